// The fp32 residual stream of layers whose sublayers read it as it is and are normed on their way out, and the small
// passes around their recurrences:
//   embed_f32        the embedding rows as the fp32 stream and in their own dtype
//   norm_add_f32_    y = s1 y1 (+ s2 y2); x += mult y / rms(y) (w + plus); h = x, one pass per row
//   gate_groupnorm   y = o silu(z), then an RMS norm of y in equal consecutive parts, times a weight
//   rotary_f32       rotary of query and key heads into fp32, keys times a factor
// All arithmetic fp32; y, z and h in the activation dtype.
#include "hybrid_common.h"

namespace llmctl_hybrid {

namespace {
constexpr int NT = 256;
constexpr int NW = NT / 64;
constexpr int KEEP = 4;  // a thread's first KEEP pieces stay in registers

template <typename T, int N>
__device__ __forceinline__ void ldn(const T* p, float* v) {  // N neighbouring elements (N == 4: one access)
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
__device__ __forceinline__ void stn(T* p, const float* v) {
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

template <typename T>
bool rows4(const at::Tensor& t) {  // rows that 4-element accesses may walk
  return t.stride(0) % 4 == 0 && reinterpret_cast<uintptr_t>(t.data_ptr()) % (4 * sizeof(T)) == 0;
}

template <typename T, int N>
__global__ __launch_bounds__(NT) void embed_f32_kernel(const int64_t* __restrict__ ids, const T* __restrict__ table, float* __restrict__ x,
                                                       T* __restrict__ h, int W) {
  const int64_t row = blockIdx.x;
  const T* e = table + ids[row] * (int64_t)W;
  for (int c = threadIdx.x * N; c < W; c += NT * N) {
    float v[N];
    ldn<T, N>(e + c, v);
    stn<T, N>(h + row * W + c, v);
    stn<float, N>(x + row * W + c, v);
  }
}

template <typename T, int N>
__global__ __launch_bounds__(NT) void norm_add_kernel(float* __restrict__ x, const T* __restrict__ y1, int64_t st1, float s1, const T* __restrict__ y2,
                                                      int64_t st2, float s2, const float* __restrict__ w, float mult, float plus, T* __restrict__ h,
                                                      int W, float eps) {
  __shared__ float red[NW];
  const int64_t row = blockIdx.x;
  float* xr = x + row * W;
  T* hr = h + row * W;
  auto sum = [&](int c, float* v) {
    ldn<T, N>(y1 + row * st1 + c, v);
    float b[N];
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] *= s1, b[i] = 0.f;
    if (y2 != nullptr) {
      ldn<T, N>(y2 + row * st2 + c, b);
#pragma unroll
      for (int i = 0; i < N; ++i) v[i] += b[i] * s2;
    }
  };
  float keep[KEEP][N], q = 0.f;
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int c = (threadIdx.x + k * NT) * N;
    if (c < W) {
      sum(c, keep[k]);
#pragma unroll
      for (int i = 0; i < N; ++i) q += keep[k][i] * keep[k][i];
    }
  }
  for (int c = (threadIdx.x + KEEP * NT) * N; c < W; c += NT * N) {
    float v[N];
    sum(c, v);
#pragma unroll
    for (int i = 0; i < N; ++i) q += v[i] * v[i];
  }
  const float f = mult / sqrtf(block_sum<NW>(q, red) / (float)W + eps);
  auto finish = [&](int c, const float* v) {
    float xv[N], wv[N];
    ldn<float, N>(xr + c, xv);
    ldn<float, N>(w + c, wv);
#pragma unroll
    for (int i = 0; i < N; ++i) xv[i] += v[i] * f * (wv[i] + plus);
    stn<float, N>(xr + c, xv);
    stn<T, N>(hr + c, xv);
  };
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int c = (threadIdx.x + k * NT) * N;
    if (c < W) finish(c, keep[k]);
  }
  for (int c = (threadIdx.x + KEEP * NT) * N; c < W; c += NT * N) {
    float v[N];
    sum(c, v);
    finish(c, v);
  }
}

// one workgroup per (row, part)
template <typename T, int N>
__global__ __launch_bounds__(NT) void gate_groupnorm_kernel(const float* __restrict__ o, const T* __restrict__ z, int64_t z_st, const float* __restrict__ w,
                                                            T* __restrict__ y, int groups, int part, float eps) {
  __shared__ float red[NW];
  const int64_t row = blockIdx.x / groups;
  const int g = (int)(blockIdx.x % groups);
  const int64_t C = (int64_t)groups * part;
  const float* orow = o + row * C + (int64_t)g * part;
  const T* zr = z + row * z_st + (int64_t)g * part;
  const float* wr = w + (int64_t)g * part;
  T* yr = y + row * C + (int64_t)g * part;
  auto gated = [&](int c, float* v) {
    float b[N];
    ldn<float, N>(orow + c, v);
    ldn<T, N>(zr + c, b);
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] *= b[i] / (1.0f + expf(-b[i]));
  };
  float keep[KEEP][N], q = 0.f;
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int c = (threadIdx.x + k * NT) * N;
    if (c < part) {
      gated(c, keep[k]);
#pragma unroll
      for (int i = 0; i < N; ++i) q += keep[k][i] * keep[k][i];
    }
  }
  for (int c = (threadIdx.x + KEEP * NT) * N; c < part; c += NT * N) {
    float v[N];
    gated(c, v);
#pragma unroll
    for (int i = 0; i < N; ++i) q += v[i] * v[i];
  }
  const float f = 1.0f / sqrtf(block_sum<NW>(q, red) / (float)part + eps);
  auto finish = [&](int c, float* v) {
    float wv[N];
    ldn<float, N>(wr + c, wv);
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] *= f * wv[i];
    stn<T, N>(yr + c, v);
  };
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int c = (threadIdx.x + k * NT) * N;
    if (c < part) finish(c, keep[k]);
  }
  for (int c = (threadIdx.x + KEEP * NT) * N; c < part; c += NT * N) {
    float v[N];
    gated(c, v);
    finish(c, v);
  }
}

// one workgroup per token; cos / sin of the token's angles once in LDS
template <typename T, int N>
__global__ __launch_bounds__(NT) void rotary_f32_kernel(const T* __restrict__ z, int64_t z_st, const int* __restrict__ pos, const float* __restrict__ freq,
                                                        float* __restrict__ out, int nq, int heads, int dk, int rot, int inter, float amp, float kscale) {
  extern __shared__ float cs[];  // [rot / 2] cos, then [rot / 2] sin
  const int64_t t = blockIdx.x;
  const int half = rot / 2;
  const float p = (float)pos[t];
  for (int i = threadIdx.x; i < half; i += NT) {
    float s, c;
    sincosf(p * freq[i], &s, &c);
    cs[i] = c * amp;
    cs[half + i] = s * amp;
  }
  __syncthreads();
  const T* zr = z + t * z_st;
  const int n = heads * dk;
  for (int e = threadIdx.x * N; e < n; e += NT * N) {
    const int hd = e / dk, d = e - hd * dk;
    float v[N], m[N];
    ldn<T, N>(zr + e, v);
    if (inter) {
#pragma unroll
      for (int i = 0; i < N; ++i) m[i] = 0.f;
      if (d < rot) {
        if constexpr (N == 1) {
          m[0] = ldf(zr + hd * dk + (d ^ 1));
        } else {
          m[0] = v[1], m[1] = v[0], m[2] = v[3], m[3] = v[2];
        }
      }
#pragma unroll
      for (int i = 0; i < N; ++i) {
        const int di = d + i;
        if (di < rot) v[i] = v[i] * cs[di >> 1] + ((di & 1) ? m[i] : -m[i]) * cs[half + (di >> 1)];
      }
    } else if (d < rot) {  // N == 4: half is a multiple of 4, so a piece lies on one side
      const bool first = d < half;
      ldn<T, N>(zr + e + (first ? half : -half), m);
      const int i0 = first ? d : d - half;
#pragma unroll
      for (int i = 0; i < N; ++i) v[i] = v[i] * cs[i0 + i] + (first ? -m[i] : m[i]) * cs[half + i0 + i];
    }
    if (hd >= nq) {
#pragma unroll
      for (int i = 0; i < N; ++i) v[i] *= kscale;
    }
    stn<float, N>(out + t * n + e, v);
  }
}

bool f32w(const at::Tensor& w, int64_t n) { return w.is_cuda() && w.scalar_type() == at::kFloat && w.is_contiguous() && w.numel() == n; }
}  // namespace

std::tuple<at::Tensor, at::Tensor> embed_f32(const at::Tensor& ids, const at::Tensor& table) {
  HYB_CHECK(table.is_cuda() && table.dim() == 2 && table.is_contiguous(), "table: contiguous [vocab, W]");
  HYB_CHECK(ids.is_cuda() && ids.is_contiguous() && ids.scalar_type() == at::kLong && ids.dim() == 1, "ids: int64 [T]");
  const int64_t T = ids.numel(), W = table.size(1);
  c10::DeviceGuard guard(table.device());
  at::Tensor x = at::empty({T, W}, table.options().dtype(at::kFloat)), h = at::empty({T, W}, table.options());
  if (T == 0) return {x, h};
  dispatch_act(table, [&](auto* tag) {
    using Tt = std::remove_pointer_t<decltype(tag)>;
    auto go = [&](auto kern) {
      kern<<<dim3((unsigned)T), NT, 0, cur_stream()>>>(ids.data_ptr<int64_t>(), (const Tt*)table.data_ptr(), x.data_ptr<float>(), (Tt*)h.data_ptr(), (int)W);
    };
    if (W % 4 == 0 && rows4<Tt>(table)) go(embed_f32_kernel<Tt, 4>);
    else go(embed_f32_kernel<Tt, 1>);
  });
  return {x, h};
}

at::Tensor norm_add_f32_(at::Tensor x, const at::Tensor& y1, double s1, const c10::optional<at::Tensor>& y2, double s2, const at::Tensor& w, double mult,
                         double eps, bool one_plus, bool out_bf16) {
  HYB_CHECK(x.is_cuda() && x.dim() == 2 && x.is_contiguous() && x.scalar_type() == at::kFloat, "x: contiguous fp32 [T, W]");
  check_rows(y1, "y1");
  const int64_t T = x.size(0), W = x.size(1);
  HYB_CHECK(y1.sizes() == x.sizes() && f32w(w, W), "y1: x's shape; w: fp32 [W]");
  HYB_CHECK((y1.scalar_type() == at::kBFloat16) == out_bf16, "the output has y1's dtype");
  if (y2.has_value()) {
    check_rows(*y2, "y2");
    HYB_CHECK(y2->sizes() == x.sizes() && y2->scalar_type() == y1.scalar_type(), "y2: y1's shape and dtype");
  }
  c10::DeviceGuard guard(x.device());
  at::Tensor h = at::empty({T, W}, y1.options());
  if (T == 0 || W == 0) return h;
  dispatch_act(y1, [&](auto* tag) {
    using Tt = std::remove_pointer_t<decltype(tag)>;
    const bool v4 = W % 4 == 0 && rows4<Tt>(y1) && (!y2.has_value() || rows4<Tt>(*y2)) && rows4<float>(x) && reinterpret_cast<uintptr_t>(w.data_ptr()) % 16 == 0;
    auto go = [&](auto kern) {
      kern<<<dim3((unsigned)T), NT, 0, cur_stream()>>>(x.data_ptr<float>(), (const Tt*)y1.data_ptr(), y1.stride(0), (float)s1,
                                                       y2.has_value() ? (const Tt*)y2->data_ptr() : nullptr, y2.has_value() ? y2->stride(0) : 0,
                                                       (float)s2, w.data_ptr<float>(), (float)mult, one_plus ? 1.0f : 0.0f, (Tt*)h.data_ptr(), (int)W, (float)eps);
    };
    if (v4) go(norm_add_kernel<Tt, 4>);
    else go(norm_add_kernel<Tt, 1>);
  });
  return h;
}

at::Tensor gate_groupnorm(const at::Tensor& o, const at::Tensor& z, const at::Tensor& w, int64_t groups, double eps, bool out_bf16) {
  HYB_CHECK(o.is_cuda() && o.dim() == 2 && o.is_contiguous() && o.scalar_type() == at::kFloat, "o: contiguous fp32 [T, C]");
  check_rows(z, "z");
  const int64_t T = o.size(0), C = o.size(1);
  HYB_CHECK(z.sizes() == o.sizes() && f32w(w, C) && groups >= 1 && C % groups == 0, "z: o's shape; w: fp32 [C]; groups must divide C");
  HYB_CHECK((z.scalar_type() == at::kBFloat16) == out_bf16, "the output has z's dtype");
  HYB_CHECK(T * groups <= 0x7fffffff, "grid too large");
  c10::DeviceGuard guard(o.device());
  at::Tensor y = at::empty({T, C}, z.options());
  if (T == 0 || C == 0) return y;
  const int part = (int)(C / groups);
  dispatch_act(z, [&](auto* tag) {
    using Tt = std::remove_pointer_t<decltype(tag)>;
    const bool v4 = part % 4 == 0 && rows4<Tt>(z) && rows4<float>(o) && reinterpret_cast<uintptr_t>(w.data_ptr()) % 16 == 0;
    auto go = [&](auto kern) {
      kern<<<dim3((unsigned)(T * groups)), NT, 0, cur_stream()>>>(o.data_ptr<float>(), (const Tt*)z.data_ptr(), z.stride(0), w.data_ptr<float>(),
                                                                  (Tt*)y.data_ptr(), (int)groups, part, (float)eps);
    };
    if (v4) go(gate_groupnorm_kernel<Tt, 4>);
    else go(gate_groupnorm_kernel<Tt, 1>);
  });
  return y;
}

at::Tensor rotary_f32(const at::Tensor& z, int64_t nq, int64_t nk, int64_t dk, const at::Tensor& pos, const at::Tensor& freq, int64_t rot, bool interleaved,
                      double amp, double kscale) {
  check_rows(z, "z");
  const int64_t T = z.size(0), heads = nq + nk;
  HYB_CHECK(nq >= 0 && nk >= 0 && heads >= 1 && dk >= 1 && z.size(1) >= heads * dk, "z: [T, >= (nq + nk) dk]");
  HYB_CHECK(rot >= 0 && rot % 2 == 0 && rot <= dk && rot <= 8192 && f32w(freq, rot / 2), "rotary: even dims <= dk, fp32 frequencies [dims / 2]");
  HYB_CHECK(pos.is_cuda() && pos.is_contiguous() && pos.scalar_type() == at::kInt && pos.numel() == T, "pos: int32 [T]");
  c10::DeviceGuard guard(z.device());
  at::Tensor out = at::empty({T, heads, dk}, z.options().dtype(at::kFloat));
  if (T == 0) return out;
  dispatch_act(z, [&](auto* tag) {
    using Tt = std::remove_pointer_t<decltype(tag)>;
    const bool v4 = dk % 4 == 0 && (interleaved || (rot / 2) % 4 == 0) && rows4<Tt>(z);
    auto go = [&](auto kern) {
      kern<<<dim3((unsigned)T), NT, (size_t)rot * sizeof(float), cur_stream()>>>((const Tt*)z.data_ptr(), z.stride(0), pos.data_ptr<int>(), freq.data_ptr<float>(),
                                                                                 out.data_ptr<float>(), (int)nq, (int)heads, (int)dk, (int)rot,
                                                                                 interleaved ? 1 : 0, (float)amp, (float)kscale);
    };
    if (v4) go(rotary_f32_kernel<Tt, 4>);
    else go(rotary_f32_kernel<Tt, 1>);
  });
  return out;
}

}  // namespace llmctl_hybrid
