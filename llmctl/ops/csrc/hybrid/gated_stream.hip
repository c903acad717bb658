// The fp32 residual stream of sequential layers with norms on both sides of a sublayer and a gated
// residual, and the small passes around them:
//   gated_norm_add_norm_f32_  g = y sigmoid(r); x += g / rms(g) * w_post; h = x / rms(x) * w_next, one pass per row
//   embed_rmsnorm_f32         x = table[id] + pos_table[position] as the fp32 stream, and its first RMS norm
//   act_any                   relu(x)^2 or the exact (erf) GELU on a column range of a wider row
//   qk_fullnorm_prep          queries and keys normed as whole rows, turned by their position, keys and values to the cache
//   glu_act                   act(gate) * up of rows [gate | up] (silu or the tanh GELU), times an optional factor per row
// All arithmetic fp32; y, r, h in the activation dtype or fp32.
#include "hybrid_common.h"

namespace llmctl_hybrid {

namespace {
constexpr int NT = 256;
constexpr int NW = NT / 64;
constexpr int KEEP = 8;  // a thread's first KEEP values stay in registers (rows up to KEEP * NT wide are read once)

__device__ __forceinline__ float sigmoidf_(float v) { return 1.0f / (1.0f + expf(-v)); }

template <typename TY, typename TR, typename TH>
__global__ __launch_bounds__(NT) void gated_norm_add_norm_kernel(float* __restrict__ x, const TY* __restrict__ y, int64_t y_st,
                                                                 const TR* __restrict__ r, int64_t r_st, const float* __restrict__ wp,
                                                                 const float* __restrict__ wn, TH* __restrict__ h, int W, float eps) {
  __shared__ float red[NW];
  const int64_t row = blockIdx.x;
  float* xr = x + row * W;
  const TY* yr = y + row * y_st;
  const TR* rr = r + row * r_st;
  float g[KEEP];
  float q = 0.f;
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int c = threadIdx.x + i * NT;
    g[i] = c < W ? ldf(yr + c) * sigmoidf_(ldf(rr + c)) : 0.f;
    q += g[i] * g[i];
  }
  for (int c = threadIdx.x + KEEP * NT; c < W; c += NT) {
    const float v = ldf(yr + c) * sigmoidf_(ldf(rr + c));
    q += v * v;
  }
  const float rstd = 1.0f / sqrtf(block_sum<NW>(q, red) / (float)W + eps);
  float q2 = 0.f;
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int c = threadIdx.x + i * NT;
    if (c < W) {
      g[i] = xr[c] + g[i] * rstd * wp[c];
      xr[c] = g[i];
      q2 += g[i] * g[i];
    }
  }
  for (int c = threadIdx.x + KEEP * NT; c < W; c += NT) {
    const float v = xr[c] + ldf(yr + c) * sigmoidf_(ldf(rr + c)) * rstd * wp[c];
    xr[c] = v;
    q2 += v * v;
  }
  if (h == nullptr) return;
  const float rstd2 = 1.0f / sqrtf(block_sum<NW>(q2, red) / (float)W + eps);
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int c = threadIdx.x + i * NT;
    if (c < W) stf(h + row * W + c, g[i] * rstd2 * wn[c]);
  }
  for (int c = threadIdx.x + KEEP * NT; c < W; c += NT) stf(h + row * W + c, xr[c] * rstd2 * wn[c]);
}

template <typename T>
__global__ __launch_bounds__(NT) void embed_rmsnorm_kernel(const int64_t* __restrict__ ids, const int* __restrict__ pos,
                                                           const T* __restrict__ table, const T* __restrict__ ptable, const float* __restrict__ w,
                                                           float* __restrict__ x, T* __restrict__ h, int W, float eps) {
  __shared__ float red[NW];
  const int64_t row = blockIdx.x;
  const T* e = table + ids[row] * (int64_t)W;
  const T* p = ptable + (int64_t)pos[row] * W;
  float q = 0.f;
  for (int c = threadIdx.x; c < W; c += NT) {
    const float v = ldf(e + c) + ldf(p + c);
    x[row * W + c] = v;
    q += v * v;
  }
  const float rstd = 1.0f / sqrtf(block_sum<NW>(q, red) / (float)W + eps);
  for (int c = threadIdx.x; c < W; c += NT) stf(h + row * W + c, x[row * W + c] * rstd * w[c]);  // the thread's own stores
}

template <int KIND>
__device__ __forceinline__ float act_one(float v) {
  if constexpr (KIND == 0) {
    const float r = fmaxf(v, 0.f);
    return r * r;
  } else {
    return 0.5f * v * (1.0f + erff(v * 0.70710678118654752f));
  }
}

template <typename T, int KIND>
__global__ void act_kernel(const T* __restrict__ x, int64_t x_st, const float* __restrict__ scale, T* __restrict__ y, int64_t rows, int F) {
  const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= rows * F) return;
  const int64_t r = i / F;
  const int c = (int)(i - r * F);
  stf(y + i, act_one<KIND>(ldf(x + r * x_st + c)) * (scale != nullptr ? scale[r] : 1.0f));
}

template <typename T, int KIND>
__global__ void act_vec_kernel(const T* __restrict__ x, int64_t x_st, const float* __restrict__ scale, T* __restrict__ y, int64_t rows, int F) {
  constexpr int N = Vec16<T>::N;
  const int per = F / N;
  const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= rows * per) return;
  const int64_t r = i / per;
  const int c = (int)(i - r * per) * N;
  float v[N];
  Vec16<T>::load(x + r * x_st + c, v);
  const float f = scale != nullptr ? scale[r] : 1.0f;
#pragma unroll
  for (int k = 0; k < N; ++k) v[k] = act_one<KIND>(v[k]) * f;
  Vec16<T>::store(y + r * F + c, v);
}

// The tanh GELU 0.5 z (1 + tanh(y)) is z sigmoid(2 y), y = sqrt(2 / pi) (z + 0.044715 z^3).
template <int KIND>
__device__ __forceinline__ float gate_act(float z) {
  const float e = KIND == 0 ? z : 1.5957691216057308f * (z + 0.044715f * z * z * z);
  return z / (1.0f + expf(-e));
}

// gu [rows, 2F] = [gate | up] -> y [rows, F] = act(gate) up (times scale[row]); N elements a thread
template <typename T, int KIND, int N>
__global__ __launch_bounds__(256) void glu_act_kernel(const T* __restrict__ gu, int64_t gu_st, const float* __restrict__ scale, T* __restrict__ y,
                                                      int64_t rows, int F) {
  const int per = F / N;
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= rows * per) return;
  const int64_t r = i / per;
  const int c = (int)(i - r * per) * N;
  float g[N], u[N];
  if constexpr (N == 1) {
    g[0] = ldf(gu + r * gu_st + c);
    u[0] = ldf(gu + r * gu_st + F + c);
  } else {
    Vec16<T>::load(gu + r * gu_st + c, g);
    Vec16<T>::load(gu + r * gu_st + F + c, u);
  }
  const float f = scale != nullptr ? scale[r] : 1.0f;
#pragma unroll
  for (int k = 0; k < N; ++k) g[k] = gate_act<KIND>(g[k]) * u[k] * f;
  if constexpr (N == 1) stf(y + r * F + c, g[0]);
  else Vec16<T>::store(y + r * F + c, g);
}

template <typename T, int N>
__device__ __forceinline__ void ld_piece(const T* p, float* v) {  // N neighbouring elements (N == 4: one access)
  if constexpr (N == 1) {
    v[0] = ldf(p);
  } else if constexpr (sizeof(T) == 4) {
    Vec16<float>::load(reinterpret_cast<const float*>(p), v);
  } else {
    const uint2 x = *reinterpret_cast<const uint2*>(p);
    v[0] = __uint_as_float(x.x << 16), v[1] = __uint_as_float(x.x & 0xffff0000u);
    v[2] = __uint_as_float(x.y << 16), v[3] = __uint_as_float(x.y & 0xffff0000u);
  }
}
template <typename T, int N>
__device__ __forceinline__ void st_piece(T* p, const float* v) {
  if constexpr (N == 1) {
    stf(p, v[0]);
  } else if constexpr (sizeof(T) == 4) {
    Vec16<float>::store(reinterpret_cast<float*>(p), v);
  } else {
    unsigned w[2];
#pragma unroll
    for (int c = 0; c < 2; ++c)
      w[c] = (unsigned)__bfloat16_as_ushort(__float2bfloat16(v[2 * c])) | ((unsigned)__bfloat16_as_ushort(__float2bfloat16(v[2 * c + 1])) << 16);
    *reinterpret_cast<uint2*>(p) = make_uint2(w[0], w[1]);
  }
}

// z [T, >= H*dk + G*dk + G*dv] = [q | k | v | ...]: unit RMS over all of q and over all of k, times the weights;
// q times the position's temperature; rotary of q and k on the first rot entries of every head (halves, or neighbours
// when inter); [v | k] per kv group to the token's cache row.  One block per token; pieces of N neighbouring elements.
template <typename T, int N>
__global__ __launch_bounds__(NT) void qk_fullnorm_prep_kernel(const T* __restrict__ z, int64_t z_st, const float* __restrict__ wq,
                                                              const float* __restrict__ wk, const int* __restrict__ pos, T* __restrict__ q,
                                                              T* __restrict__ cache, const int64_t* __restrict__ slots, int H, int G, int dk,
                                                              int dv, float eps, float coef, int every, const float* __restrict__ freq, int rot,
                                                              int inter, float amp) {
  extern __shared__ float cs[];  // [rot / 2] cos, then [rot / 2] sin
  __shared__ float red[2 * NW];
  const int64_t t = blockIdx.x;
  const T* zr = z + t * z_st;
  const int nq = H * dk, nk = G * dk, nv = G * dv, half = rot / 2;
  const float p = (float)pos[t];
  for (int i = threadIdx.x; i < half; i += NT) {
    float s, c;
    sincosf(p * freq[i], &s, &c);
    cs[i] = c * amp;
    cs[half + i] = s * amp;
  }
  float sq = 0.f, sk = 0.f;
  for (int c = threadIdx.x * N; c < nq + nk; c += NT * N) {  // (N divides nq)
    float v[N], a = 0.f;
    ld_piece<T, N>(zr + c, v);
#pragma unroll
    for (int i = 0; i < N; ++i) a += v[i] * v[i];
    if (c < nq) sq += a;
    else sk += a;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((threadIdx.x & 63) == 0) {
    red[threadIdx.x >> 6] = sq;
    red[NW + (threadIdx.x >> 6)] = sk;
  }
  __syncthreads();
  sq = sk = 0.f;
#pragma unroll
  for (int i = 0; i < NW; ++i) sq += red[i], sk += red[NW + i];
  float temp = 1.0f;
  if (coef != 0.f) temp = 1.0f + coef * logf((float)((pos[t] + 1) / every) + 1.0f);
  const float rq = temp / sqrtf(sq / (float)nq + eps), rk = 1.0f / sqrtf(sk / (float)nk + eps);
  const int64_t slot = slots[t];
  T* row = cache + slot * (int64_t)(nk + nv);
  auto normed = [&](int c, float* v) {  // N entries of the row [q | k] from column c on, normed
    float w[N];
    ld_piece<T, N>(zr + c, v);
    ld_piece<float, N>(c < nq ? wq + c : wk + (c - nq), w);
    const float f = c < nq ? rq : rk;
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] *= f * w[i];
  };
  for (int c = threadIdx.x * N; c < nq + nk; c += NT * N) {
    const int hd = c / dk, d = c - hd * dk;
    float v[N], m[N];
    normed(c, v);
    if (d < rot) {
      if (inter) {
        if constexpr (N == 1) normed(c - d + (d ^ 1), m);
        else m[0] = v[1], m[1] = v[0], m[2] = v[3], m[3] = v[2];
#pragma unroll
        for (int i = 0; i < N; ++i) {
          const int di = d + i;
          if (di < rot) v[i] = v[i] * cs[di >> 1] + ((di & 1) ? m[i] : -m[i]) * cs[half + (di >> 1)];
        }
      } else {  // N == 4: half is a multiple of 4, so a piece lies on one side
        const bool first = d < half;
        normed(c + (first ? half : -half), m);
        const int i0 = first ? d : d - half;
#pragma unroll
        for (int i = 0; i < N; ++i) v[i] = v[i] * cs[i0 + i] + (first ? -m[i] : m[i]) * cs[half + i0 + i];
      }
    }
    if (c < nq) st_piece<T, N>(q + t * nq + c, v);
    else if (slot >= 0) st_piece<T, N>(row + (hd - H) * (dv + dk) + dv + d, v);
  }
  if (slot < 0) return;
  for (int c = threadIdx.x * N; c < nv; c += NT * N) {
    const int g = c / dv, d = c - g * dv;
    float v[N];
    ld_piece<T, N>(zr + nq + nk + c, v);
    st_piece<T, N>(row + g * (dv + dk) + d, v);
  }
}

bool f32w(const at::Tensor& w, int64_t n) { return w.is_cuda() && w.scalar_type() == at::kFloat && w.is_contiguous() && w.numel() == n; }
}  // namespace

at::Tensor gated_norm_add_norm_f32_(at::Tensor x, const at::Tensor& y, const at::Tensor& r, const at::Tensor& w_post,
                                    const c10::optional<at::Tensor>& w_next, double eps, bool out_bf16) {
  HYB_CHECK(x.is_cuda() && x.dim() == 2 && x.is_contiguous() && x.scalar_type() == at::kFloat, "x: contiguous fp32 [T, W]");
  check_rows(y, "y");
  check_rows(r, "r");
  const int64_t T = x.size(0), W = x.size(1);
  HYB_CHECK(y.sizes() == x.sizes() && r.sizes() == x.sizes(), "y and r must have x's shape");
  HYB_CHECK(f32w(w_post, W) && (!w_next.has_value() || f32w(*w_next, W)), "norm weights: fp32 [W]");
  c10::DeviceGuard guard(x.device());
  at::Tensor h = w_next.has_value() ? at::empty({T, W}, x.options().dtype(out_bf16 ? at::kBFloat16 : at::kFloat)) : at::empty({0}, x.options());
  if (T == 0) return h;
  const float* wn = w_next.has_value() ? w_next->data_ptr<float>() : nullptr;
  hipStream_t st = cur_stream();
  auto go = [&](auto* ty, auto* tr, auto* th) {
    using TY = std::remove_pointer_t<decltype(ty)>;
    using TR = std::remove_pointer_t<decltype(tr)>;
    using TH = std::remove_pointer_t<decltype(th)>;
    gated_norm_add_norm_kernel<TY, TR, TH><<<dim3((unsigned)T), NT, 0, st>>>(x.data_ptr<float>(), (const TY*)y.data_ptr(), y.stride(0),
                                                                           (const TR*)r.data_ptr(), r.stride(0), w_post.data_ptr<float>(), wn,
                                                                           wn != nullptr ? (TH*)h.data_ptr() : (TH*)nullptr, (int)W, (float)eps);
  };
  dispatch_act(y, [&](auto* ty) {
    dispatch_act(r, [&](auto* tr) {
      if (out_bf16) go(ty, tr, (bf16_t*)nullptr);
      else go(ty, tr, (float*)nullptr);
    });
  });
  return h;
}

std::tuple<at::Tensor, at::Tensor> embed_rmsnorm_f32(const at::Tensor& ids, const at::Tensor& pos, const at::Tensor& table,
                                                     const at::Tensor& pos_table, const at::Tensor& w, double eps, bool out_bf16) {
  HYB_CHECK(table.is_cuda() && table.dim() == 2 && table.is_contiguous() && pos_table.is_cuda() && pos_table.dim() == 2 && pos_table.is_contiguous() &&
                pos_table.size(1) == table.size(1) && pos_table.scalar_type() == table.scalar_type(),
            "embedding and position tables: contiguous [rows, W] of one dtype");
  const int64_t T = ids.numel(), W = table.size(1);
  HYB_CHECK(ids.is_cuda() && ids.is_contiguous() && ids.scalar_type() == at::kLong && pos.is_cuda() && pos.is_contiguous() && pos.scalar_type() == at::kInt && pos.numel() == T,
            "ids int64 [T], pos int32 [T]");
  HYB_CHECK(f32w(w, W), "norm weight: fp32 [W]");
  HYB_CHECK((table.scalar_type() == at::kBFloat16) == out_bf16, "the output has the tables' dtype");
  c10::DeviceGuard guard(table.device());
  at::Tensor x = at::empty({T, W}, table.options().dtype(at::kFloat));
  at::Tensor h = at::empty({T, W}, table.options());
  if (T == 0) return {x, h};
  dispatch_act(table, [&](auto* tag) {
    using Tt = std::remove_pointer_t<decltype(tag)>;
    embed_rmsnorm_kernel<Tt><<<dim3((unsigned)T), NT, 0, cur_stream()>>>(ids.data_ptr<int64_t>(), pos.data_ptr<int>(), (const Tt*)table.data_ptr(),
                                                                        (const Tt*)pos_table.data_ptr(), w.data_ptr<float>(), x.data_ptr<float>(),
                                                                        (Tt*)h.data_ptr(), (int)W, (float)eps);
  });
  return {x, h};
}

at::Tensor act_any(const at::Tensor& x, int64_t kind, const c10::optional<at::Tensor>& scale) {
  check_rows(x, "x");
  if (scale.has_value()) HYB_CHECK(f32w(*scale, x.size(0)), "row factors: fp32 [rows]");
  const float* sp = scale.has_value() ? scale->data_ptr<float>() : nullptr;
  HYB_CHECK(kind == 0 || kind == 1, "activation kind: 0 = squared relu, 1 = erf gelu");
  c10::DeviceGuard guard(x.device());
  const int64_t rows = x.size(0);
  const int F = (int)x.size(1);
  at::Tensor y = at::empty({rows, F}, x.options());
  const int64_t n = y.numel();
  if (n == 0) return y;
  hipStream_t st = cur_stream();
  dispatch_act(x, [&](auto* tag) {
    using T = std::remove_pointer_t<decltype(tag)>;
    const bool vec = F % Vec16<T>::N == 0 && aligned16<T>(x);
    const int64_t nv = vec ? n / Vec16<T>::N : n;
    const dim3 grid((unsigned)((nv + 255) / 256));
    if (vec) {
      if (kind == 0) act_vec_kernel<T, 0><<<grid, 256, 0, st>>>((const T*)x.data_ptr(), x.stride(0), sp, (T*)y.data_ptr(), rows, F);
      else act_vec_kernel<T, 1><<<grid, 256, 0, st>>>((const T*)x.data_ptr(), x.stride(0), sp, (T*)y.data_ptr(), rows, F);
    } else {
      if (kind == 0) act_kernel<T, 0><<<grid, 256, 0, st>>>((const T*)x.data_ptr(), x.stride(0), sp, (T*)y.data_ptr(), rows, F);
      else act_kernel<T, 1><<<grid, 256, 0, st>>>((const T*)x.data_ptr(), x.stride(0), sp, (T*)y.data_ptr(), rows, F);
    }
  });
  return y;
}

// kind: 0 = silu, 1 = tanh GELU
at::Tensor glu_act(const at::Tensor& gu, int64_t kind, const c10::optional<at::Tensor>& scale) {
  check_rows(gu, "gu");
  HYB_CHECK(gu.size(1) % 2 == 0 && (kind == 0 || kind == 1), "gu: [rows, 2F]; kind: 0 = silu, 1 = tanh gelu");
  const int64_t rows = gu.size(0);
  const int F = (int)(gu.size(1) / 2);
  if (scale.has_value()) HYB_CHECK(f32w(*scale, rows), "row factors: fp32 [rows]");
  c10::DeviceGuard guard(gu.device());
  at::Tensor y = at::empty({rows, F}, gu.options());
  if (y.numel() == 0) return y;
  const float* sp = scale.has_value() ? scale->data_ptr<float>() : nullptr;
  dispatch_act(gu, [&](auto* tag) {
    using T = std::remove_pointer_t<decltype(tag)>;
    constexpr int N = Vec16<T>::N;
    const bool vec = F % N == 0 && aligned16<T>(gu);
    const dim3 grid((unsigned)((y.numel() / (vec ? N : 1) + 255) / 256));
    auto go = [&](auto kern) { kern<<<grid, 256, 0, cur_stream()>>>((const T*)gu.data_ptr(), gu.stride(0), sp, (T*)y.data_ptr(), rows, F); };
    if (vec) {
      if (kind == 0) go(glu_act_kernel<T, 0, N>);
      else go(glu_act_kernel<T, 1, N>);
    } else {
      if (kind == 0) go(glu_act_kernel<T, 0, 1>);
      else go(glu_act_kernel<T, 1, 1>);
    }
  });
  return y;
}

at::Tensor qk_fullnorm_prep(const at::Tensor& z, int64_t H, int64_t G, int64_t dk, int64_t dv, const at::Tensor& q_norm, const at::Tensor& k_norm,
                            double eps, const at::Tensor& pos, double temp_coef, int64_t temp_every, at::Tensor cache, const at::Tensor& slots,
                            const c10::optional<at::Tensor>& freq, int64_t rot, bool interleaved, double amp) {
  check_rows(z, "z");
  const int64_t T = z.size(0);
  HYB_CHECK(H >= 1 && G >= 1 && H % G == 0 && dk >= 1 && dv >= 1 && z.size(1) >= (H + G) * dk + G * dv, "z: [T, >= H*dk + G*dk + G*dv]");
  HYB_CHECK(f32w(q_norm, H * dk) && f32w(k_norm, G * dk), "norm weights: fp32 [H*dk], [G*dk]");
  HYB_CHECK(cache.is_cuda() && cache.is_contiguous() && cache.dim() == 3 && cache.size(2) == G * (dv + dk) && cache.scalar_type() == z.scalar_type(),
            "cache: contiguous [blocks, block_size, G * (dv + dk)] of z's dtype");
  HYB_CHECK(pos.is_cuda() && pos.is_contiguous() && pos.scalar_type() == at::kInt && pos.numel() == T && slots.is_cuda() && slots.is_contiguous() &&
                slots.scalar_type() == at::kLong && slots.numel() == T,
            "pos int32 [T], slots int64 [T]");
  HYB_CHECK(temp_every >= 1, "temperature period >= 1");
  HYB_CHECK(rot >= 0 && rot % 2 == 0 && rot <= dk && rot <= 8192 && (rot == 0 || (freq.has_value() && f32w(*freq, rot / 2))),
            "rotary: even dims <= dk, fp32 frequencies [dims / 2]");
  c10::DeviceGuard guard(z.device());
  at::Tensor q = at::empty({T, H, dk}, z.options());
  if (T == 0) return q;
  dispatch_act(z, [&](auto* tag) {
    using Tt = std::remove_pointer_t<decltype(tag)>;
    auto a16 = [](const at::Tensor& t) { return reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0; };
    const bool v4 = dk % 4 == 0 && dv % 4 == 0 && (interleaved || (rot / 2) % 4 == 0) && z.stride(0) % 4 == 0 &&
                    reinterpret_cast<uintptr_t>(z.data_ptr()) % (4 * sizeof(Tt)) == 0 && a16(q_norm) && a16(k_norm) && a16(cache);
    auto go = [&](auto kern) {
      kern<<<dim3((unsigned)T), NT, (size_t)rot * sizeof(float), cur_stream()>>>(
          (const Tt*)z.data_ptr(), z.stride(0), q_norm.data_ptr<float>(), k_norm.data_ptr<float>(), pos.data_ptr<int>(), (Tt*)q.data_ptr(),
          (Tt*)cache.data_ptr(), slots.data_ptr<int64_t>(), (int)H, (int)G, (int)dk, (int)dv, (float)eps, (float)temp_coef, (int)temp_every,
          rot > 0 ? freq->data_ptr<float>() : nullptr, (int)rot, interleaved ? 1 : 0, (float)amp);
    };
    if (v4) go(qk_fullnorm_prep_kernel<Tt, 4>);
    else go(qk_fullnorm_prep_kernel<Tt, 1>);
  });
  return q;
}

}  // namespace llmctl_hybrid
