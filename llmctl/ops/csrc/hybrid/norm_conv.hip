// The fp32 residual stream of layers whose sublayers read a causally convolved, group-normed input:
//   x <- x + y (or x = table[id] * scale + pos_table[position]);  h = x / rms(x per group) * w;
//   out_t = h_t + sum_j c[j] h_(t - taps + 1 + j)  per channel, zeros before position 0
// with the last taps - 1 values of h of every live sequence carried in a slot pool (fp32) between steps.
//
//   norm_conv_kernel   all of it in one pass.  A workgroup owns L consecutive packed rows and walks them in order with
//                      the last taps - 1 normed rows in registers; the rows before its first one are normed again (they
//                      belong to the neighbour, which writes them), so no row waits for another workgroup.  The stream
//                      is written to a second buffer, because a neighbour may still read the old row.
//   conv_tail_kernel   after it, for portions that continue a sequence and span workgroups: the carried rows of
//                      such a portion may still be read by its first workgroup while its last one has the new ones, so
//                      those go to a scratch row first and are copied here
//   group_norm_kernel  the norm alone (any width); the final norm, and the first half of the unfused form
// A row's group sums are formed from power-of-two lane units by shuffles and finished out of LDS in a fixed order.
#include "hybrid_common.h"

namespace llmctl_hybrid {

namespace {

struct NormConvArgs {
  const float* x;
  float* xo;
  const void* y;
  int64_t y_st;
  const int64_t* ids;  // EMB form: x = table[ids] * scale + pos_table[pos]
  const int* pos;
  const void* table;
  const void* pos_table;
  float scale;
  const float* w;   // [W]
  const float* cw;  // [taps, W]
  float* state;     // [slots, taps - 1, W]
  float* tail;      // nullptr, or [sequences, taps - 1, W]
  const int* seq_of;
  const int* cu;
  const int* start;
  const int* sslot;
  void* out;
  int T, W, L, gs, unit;  // gs: columns per group; unit: lanes per shuffle-reduced unit (4 columns a lane)
  float eps;
};

template <typename T>
__device__ __forceinline__ void ld4(const T* p, float* v);
template <>
__device__ __forceinline__ void ld4<float>(const float* p, float* v) {
  const float4 r = *reinterpret_cast<const float4*>(p);
  v[0] = r.x, v[1] = r.y, v[2] = r.z, v[3] = r.w;
}
template <>
__device__ __forceinline__ void ld4<bf16_t>(const bf16_t* p, float* v) {
  const uint2 r = *reinterpret_cast<const uint2*>(p);
  v[0] = __uint_as_float(r.x << 16), v[1] = __uint_as_float(r.x & 0xffff0000u);
  v[2] = __uint_as_float(r.y << 16), v[3] = __uint_as_float(r.y & 0xffff0000u);
}
__device__ __forceinline__ void st4(float* p, const float* v) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }
__device__ __forceinline__ void st4(bf16_t* p, const float* v) {
  const unsigned a = (unsigned)__bfloat16_as_ushort(__float2bfloat16(v[0])) | ((unsigned)__bfloat16_as_ushort(__float2bfloat16(v[1])) << 16);
  const unsigned b = (unsigned)__bfloat16_as_ushort(__float2bfloat16(v[2])) | ((unsigned)__bfloat16_as_ushort(__float2bfloat16(v[3])) << 16);
  *reinterpret_cast<uint2*>(p) = make_uint2(a, b);
}

// Thread i owns the column quads (i + k NT), k < VPT.  TY: y's (EMB: the tables') element, TH: the output's.
template <typename TY, typename TH, bool EMB, int TAPS, int VPT, int NT>
__global__ __launch_bounds__(NT) void norm_conv_kernel(NormConvArgs a) {
  extern __shared__ float units[];  // two rows of W / (4 unit) unit sums
  const int W = a.W, quads = W / 4, nunits = quads / a.unit;
  const int t0 = blockIdx.x * a.L, t1 = min(t0 + a.L, a.T);
  const float inv_gs = 1.0f / (float)a.gs;
  const int upg = a.gs / (4 * a.unit);  // units per group
  float nw[VPT][4], cw[TAPS][VPT][4], win[TAPS - 1][VPT][4];
#pragma unroll
  for (int k = 0; k < VPT; ++k) {
    const int q = threadIdx.x + k * NT;
    const bool ok = q < quads;
#pragma unroll
    for (int e = 0; e < 4; ++e) nw[k][e] = 0.f;
    if (ok) ld4(a.w + 4 * q, nw[k]);
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
#pragma unroll
      for (int e = 0; e < 4; ++e) cw[j][k][e] = 0.f;
      if (ok) ld4(a.cw + (int64_t)j * W + 4 * q, cw[j][k]);
    }
  }
  // the current sequence: its index, its rows [first, end) of the step, its first position, its state slot (scalars)
  int s, first, end, p0, slot;
  auto enter = [&](int t) {
    s = __builtin_amdgcn_readfirstlane(a.seq_of[t]);
    first = __builtin_amdgcn_readfirstlane(a.cu[s]);
    end = __builtin_amdgcn_readfirstlane(a.cu[s + 1]);
    p0 = __builtin_amdgcn_readfirstlane(a.start[s]);
    slot = __builtin_amdgcn_readfirstlane(a.sslot[s]);
  };
  enter(t0);
  // the carried rows of sequence s as its window: entry j is position start - (TAPS - 1) + j
  auto history = [&]() {
    const float* st = a.state + (int64_t)slot * (TAPS - 1) * W;
#pragma unroll
    for (int j = 0; j < TAPS - 1; ++j)
#pragma unroll
      for (int k = 0; k < VPT; ++k) {
        const int q = threadIdx.x + k * NT;
#pragma unroll
        for (int e = 0; e < 4; ++e) win[j][k][e] = 0.f;
        if (q < quads && p0 - (TAPS - 1) + j >= 0) ld4(st + (int64_t)j * W + 4 * q, win[j][k]);
      }
  };
  const int r0 = max(first, t0 - (TAPS - 1));
  if (r0 == first) {
    history();
  } else {
#pragma unroll
    for (int j = 0; j < TAPS - 1; ++j)
#pragma unroll
      for (int k = 0; k < VPT; ++k)
#pragma unroll
        for (int e = 0; e < 4; ++e) win[j][k][e] = 0.f;
  }
  float v[VPT][4], nx[VPT][4];
  auto fetch = [&](int t, float (*d)[4]) {
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
      const int q = threadIdx.x + k * NT;
#pragma unroll
      for (int e = 0; e < 4; ++e) d[k][e] = 0.f;
      if (q < quads) {
        float b[4];
        if constexpr (EMB) {
          ld4(reinterpret_cast<const TY*>(a.table) + a.ids[t] * (int64_t)W + 4 * q, d[k]);
          ld4(reinterpret_cast<const TY*>(a.pos_table) + (int64_t)a.pos[t] * W + 4 * q, b);
#pragma unroll
          for (int e = 0; e < 4; ++e) d[k][e] = d[k][e] * a.scale + b[e];
        } else {
          ld4(a.x + (int64_t)t * W + 4 * q, d[k]);
          ld4(reinterpret_cast<const TY*>(a.y) + t * a.y_st + 4 * q, b);
#pragma unroll
          for (int e = 0; e < 4; ++e) d[k][e] += b[e];
        }
      }
    }
  };
  fetch(r0, v);
  for (int t = r0; t < t1; ++t) {
    if (t == end) {  // the next sequence with rows begins
      enter(t);
      history();
    }
    if (t + 1 < t1) fetch(t + 1, nx);
    float* u = units + ((t - r0) & 1) * nunits;
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
      const int q = threadIdx.x + k * NT;
      float ss = 0.f;
#pragma unroll
      for (int e = 0; e < 4; ++e) ss += v[k][e] * v[k][e];
      for (int o = a.unit >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
      if (q < quads && (q & (a.unit - 1)) == 0) u[q / a.unit] = ss;
      if (t >= t0 && q < quads) st4(a.xo + (int64_t)t * W + 4 * q, v[k]);
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < VPT; ++k) {
      const int q = threadIdx.x + k * NT;
      if (q >= quads) continue;
      const int g = (4 * q) / a.gs;
      float ss = 0.f;
      for (int i = 0; i < upg; ++i) ss += u[g * upg + i];
      const float rstd = 1.0f / sqrtf(ss * inv_gs + a.eps);
      float h[4], o[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        h[e] = v[k][e] * rstd * nw[k][e];
        float c = cw[TAPS - 1][k][e] * h[e];
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j) c += cw[j][k][e] * win[j][k][e];
        o[e] = h[e] + c;
      }
      if (t >= t0) st4(reinterpret_cast<TH*>(a.out) + (int64_t)t * W + 4 * q, o);
#pragma unroll
      for (int j = 0; j + 1 < TAPS - 1; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) win[j][k][e] = win[j + 1][k][e];
#pragma unroll
      for (int e = 0; e < 4; ++e) win[TAPS - 2][k][e] = h[e];
    }
    if (t == end - 1) {  // the sequence's last row of the step: the window is its new state
      auto save = [&](float* st) {
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j)
#pragma unroll
          for (int k = 0; k < VPT; ++k) {
            const int q = threadIdx.x + k * NT;
            if (q < quads) st4(st + (int64_t)j * W + 4 * q, win[j][k]);
          }
      };
      if (a.tail == nullptr || p0 == 0 || (end - 1) / a.L == first / a.L) save(a.state + (int64_t)slot * (TAPS - 1) * W);
      else save(a.tail + (int64_t)s * (TAPS - 1) * W);
    }
#pragma unroll
    for (int k = 0; k < VPT; ++k)
#pragma unroll
      for (int e = 0; e < 4; ++e) v[k][e] = nx[k][e];
  }
}

__global__ __launch_bounds__(256) void conv_tail_kernel(const float* __restrict__ tail, float* __restrict__ state, const int* __restrict__ cu,
                                                        const int* __restrict__ start, const int* __restrict__ sslot, int n, int L) {
  const int s = blockIdx.y;
  const int a = cu[s], b = cu[s + 1];
  if (a == b || start[s] == 0 || (b - 1) / L == a / L) return;
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i < n) state[(int64_t)sslot[s] * n + i] = tail[(int64_t)s * n + i];
}

// One workgroup per row, its waves take the groups in turn.
template <typename TY, typename TH>
__global__ __launch_bounds__(256) void group_norm_kernel(const float* __restrict__ x, const TY* __restrict__ y, int64_t y_st, float* __restrict__ xo,
                                                         const float* __restrict__ w, TH* __restrict__ h, int W, int groups, float eps) {
  const int64_t t = blockIdx.x;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int gs = W / groups;
  for (int g = wave; g < groups; g += 4) {
    float q = 0.f;
    for (int c = g * gs + lane; c < (g + 1) * gs; c += 64) {
      const float v = x[t * W + c] + (y != nullptr ? ldf(y + t * y_st + c) : 0.f);
      if (xo != nullptr) xo[t * W + c] = v;
      q += v * v;
    }
    const float rstd = 1.0f / sqrtf(wave_sum(q) / (float)gs + eps);
    for (int c = g * gs + lane; c < (g + 1) * gs; c += 64) {
      const float v = x[t * W + c] + (y != nullptr ? ldf(y + t * y_st + c) : 0.f);
      stf(h + t * W + c, v * rstd * w[c]);
    }
  }
}

bool f32n(const at::Tensor& t, int64_t n) { return t.is_cuda() && t.scalar_type() == at::kFloat && t.is_contiguous() && t.numel() == n; }
bool i32n(const at::Tensor& t, int64_t n) { return t.is_cuda() && t.scalar_type() == at::kInt && t.is_contiguous() && t.numel() == n; }
bool al16(const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; }

constexpr int MAX_QUADS = 2 * 1024;  // widest row of the one-pass form: 8192 columns

void launch_norm_conv(NormConvArgs a, int taps, const at::Tensor& table_or_y, bool emb, bool out_bf16, int64_t ns, bool carried,
                      const at::Tensor& like) {
  const int quads = a.W / 4;
  // rows per workgroup: enough workgroups to fill the chip first, then fewer rows normed twice at the borders
  a.L = std::max(1, std::min(8, a.T / 512));
  const int g4 = a.gs / 4;
  a.unit = 1;
  while (a.unit < 64 && g4 % (a.unit * 2) == 0) a.unit *= 2;
  at::Tensor tail;
  if (carried && a.L < a.T) {
    tail = at::empty({ns, taps - 1, a.W}, like.options().dtype(at::kFloat));
    a.tail = tail.data_ptr<float>();
  }
  const size_t lds = (size_t)2 * (quads / a.unit) * sizeof(float);
  const dim3 grid((unsigned)((a.T + a.L - 1) / a.L));
  hipStream_t st = cur_stream();
  auto by_shape = [&](auto* ty, auto* th, auto e) {
    using TY = std::remove_pointer_t<decltype(ty)>;
    using TH = std::remove_pointer_t<decltype(th)>;
    constexpr bool EMB = decltype(e)::value;
    auto by_taps = [&](auto tp) {
      constexpr int TAPS = decltype(tp)::value;
      if (quads <= 256) norm_conv_kernel<TY, TH, EMB, TAPS, 1, 256><<<grid, 256, lds, st>>>(a);
      else if (quads <= 512) norm_conv_kernel<TY, TH, EMB, TAPS, 1, 512><<<grid, 512, lds, st>>>(a);
      else if (quads <= 1024) norm_conv_kernel<TY, TH, EMB, TAPS, 1, 1024><<<grid, 1024, lds, st>>>(a);
      else norm_conv_kernel<TY, TH, EMB, TAPS, 2, 1024><<<grid, 1024, lds, st>>>(a);
    };
    if (taps == 2) by_taps(std::integral_constant<int, 2>{});
    else if (taps == 3) by_taps(std::integral_constant<int, 3>{});
    else by_taps(std::integral_constant<int, 4>{});
  };
  dispatch_act(table_or_y, [&](auto* ty) {
    using TY = std::remove_pointer_t<decltype(ty)>;
    if (emb) {  // the output has the tables' dtype
      by_shape(ty, (TY*)nullptr, std::true_type{});
    } else if (out_bf16) {
      by_shape(ty, (bf16_t*)nullptr, std::false_type{});
    } else {
      if constexpr (std::is_same_v<TY, float>) by_shape(ty, (float*)nullptr, std::false_type{});
      else HYB_CHECK(false, "an fp32 output takes an fp32 y");
    }
  });
  if (a.tail != nullptr) {
    const int n = (taps - 1) * a.W;
    conv_tail_kernel<<<dim3((unsigned)((n + 255) / 256), (unsigned)ns), 256, 0, st>>>(a.tail, a.state, a.cu, a.start, a.sslot, n, a.L);
  }
}

NormConvArgs common_args(const at::Tensor& w, int64_t groups, double eps, const at::Tensor& cw, at::Tensor& state, const at::Tensor& seq_of,
                         const at::Tensor& cu, const at::Tensor& start, const at::Tensor& sslot, int64_t T, int64_t W) {
  const int64_t taps = cw.size(0), ns = start.numel();
  HYB_CHECK(f32n(w, W) && groups >= 1 && W % groups == 0, "norm weight: fp32 [W]; the groups must divide W");
  HYB_CHECK(cw.dim() == 2 && f32n(cw, taps * W) && taps >= 2 && taps <= 4, "conv weight: contiguous fp32 [taps, W], 2 to 4 taps");
  HYB_CHECK(W % 4 == 0 && (W / groups) % 4 == 0 && W / 4 <= MAX_QUADS, "the one-pass form takes groups of whole column quads");
  HYB_CHECK(state.is_cuda() && state.is_contiguous() && state.scalar_type() == at::kFloat && state.dim() == 3 && state.size(1) == taps - 1 && state.size(2) == W,
            "state: contiguous fp32 [slots, taps - 1, W]");
  HYB_CHECK(i32n(seq_of, T) && i32n(cu, ns + 1) && i32n(start, ns) && i32n(sslot, ns), "seq_of [T], cu [n + 1], start [n], slots [n]: int32");
  HYB_CHECK(ns <= 65535, "too many sequences for one launch");
  HYB_CHECK(al16(w.data_ptr()) && al16(cw.data_ptr()) && al16(state.data_ptr()), "weights and state must be 16-byte aligned");
  NormConvArgs a{};
  a.w = w.data_ptr<float>();
  a.cw = cw.data_ptr<float>();
  a.state = state.data_ptr<float>();
  a.seq_of = seq_of.data_ptr<int>();
  a.cu = cu.data_ptr<int>();
  a.start = start.data_ptr<int>();
  a.sslot = sslot.data_ptr<int>();
  a.T = (int)T;
  a.W = (int)W;
  a.gs = (int)(W / groups);
  a.eps = (float)eps;
  return a;
}
}  // namespace

// carried: some portion of more than one row continues a sequence (start > 0)
std::tuple<at::Tensor, at::Tensor> add_norm_conv(const at::Tensor& x, const at::Tensor& y, const at::Tensor& w, int64_t groups, double eps,
                                                 const at::Tensor& cw, at::Tensor state, const at::Tensor& seq_of, const at::Tensor& cu,
                                                 const at::Tensor& start, const at::Tensor& sslot, bool carried, bool out_bf16) {
  HYB_CHECK(x.is_cuda() && x.dim() == 2 && x.is_contiguous() && x.scalar_type() == at::kFloat, "x: contiguous fp32 [T, W]");
  check_rows(y, "y");
  HYB_CHECK(y.sizes() == x.sizes() && y.stride(0) % 4 == 0 && reinterpret_cast<uintptr_t>(y.data_ptr()) % 16 == 0, "y: x's shape, aligned rows");
  const int64_t T = x.size(0), W = x.size(1);
  NormConvArgs a = common_args(w, groups, eps, cw, state, seq_of, cu, start, sslot, T, W);
  c10::DeviceGuard guard(x.device());
  at::Tensor xo = at::empty_like(x);
  at::Tensor h = at::empty({T, W}, x.options().dtype(out_bf16 ? at::kBFloat16 : at::kFloat));
  if (T == 0) return {xo, h};
  a.x = x.data_ptr<float>();
  a.xo = xo.data_ptr<float>();
  a.y = y.data_ptr();
  a.y_st = y.stride(0);
  a.out = h.data_ptr();
  launch_norm_conv(a, (int)cw.size(0), y, false, out_bf16, start.numel(), carried, x);
  return {xo, h};
}

std::tuple<at::Tensor, at::Tensor> embed_norm_conv(const at::Tensor& ids, const at::Tensor& pos, const at::Tensor& table,
                                                   const at::Tensor& pos_table, double scale, const at::Tensor& w, int64_t groups, double eps,
                                                   const at::Tensor& cw, at::Tensor state, const at::Tensor& seq_of, const at::Tensor& cu,
                                                   const at::Tensor& start, const at::Tensor& sslot, bool carried) {
  HYB_CHECK(table.is_cuda() && table.dim() == 2 && table.is_contiguous() && pos_table.is_cuda() && pos_table.dim() == 2 && pos_table.is_contiguous() &&
                pos_table.size(1) == table.size(1) && pos_table.scalar_type() == table.scalar_type() && al16(table.data_ptr()) && al16(pos_table.data_ptr()),
            "embedding and position tables: contiguous [rows, W] of one dtype");
  const int64_t T = ids.numel(), W = table.size(1);
  HYB_CHECK(ids.is_cuda() && ids.is_contiguous() && ids.scalar_type() == at::kLong && i32n(pos, T), "ids int64 [T], pos int32 [T]");
  NormConvArgs a = common_args(w, groups, eps, cw, state, seq_of, cu, start, sslot, T, W);
  c10::DeviceGuard guard(table.device());
  at::Tensor xo = at::empty({T, W}, table.options().dtype(at::kFloat));
  at::Tensor h = at::empty({T, W}, table.options());
  if (T == 0) return {xo, h};
  a.xo = xo.data_ptr<float>();
  a.ids = ids.data_ptr<int64_t>();
  a.pos = pos.data_ptr<int>();
  a.table = table.data_ptr();
  a.pos_table = pos_table.data_ptr();
  a.scale = (float)scale;
  a.out = h.data_ptr();
  launch_norm_conv(a, (int)cw.size(0), table, true, false, start.numel(), carried, table);
  return {xo, h};
}

// (x + y, group norm of it); without y the first result is empty (the stream stays as it is)
std::tuple<at::Tensor, at::Tensor> group_norm_f32(const at::Tensor& x, const c10::optional<at::Tensor>& y, const at::Tensor& w, int64_t groups,
                                                  double eps, bool out_bf16) {
  HYB_CHECK(x.is_cuda() && x.dim() == 2 && x.is_contiguous() && x.scalar_type() == at::kFloat, "x: contiguous fp32 [T, W]");
  const int64_t T = x.size(0), W = x.size(1);
  HYB_CHECK(f32n(w, W) && groups >= 1 && W % groups == 0, "norm weight: fp32 [W]; the groups must divide W");
  if (y.has_value()) {
    check_rows(*y, "y");
    HYB_CHECK(y->sizes() == x.sizes(), "y: x's shape");
  }
  c10::DeviceGuard guard(x.device());
  at::Tensor xo = y.has_value() ? at::empty_like(x) : at::empty({0}, x.options());
  at::Tensor h = at::empty({T, W}, x.options().dtype(out_bf16 ? at::kBFloat16 : at::kFloat));
  if (T == 0) return {xo, h};
  auto go = [&](auto* ty, auto* th) {
    using TY = std::remove_pointer_t<decltype(ty)>;
    using TH = std::remove_pointer_t<decltype(th)>;
    group_norm_kernel<TY, TH><<<dim3((unsigned)T), 256, 0, cur_stream()>>>(x.data_ptr<float>(), y.has_value() ? (const TY*)y->data_ptr() : nullptr,
                                                                          y.has_value() ? y->stride(0) : 0, y.has_value() ? xo.data_ptr<float>() : nullptr,
                                                                          w.data_ptr<float>(), (TH*)h.data_ptr(), (int)W, (int)groups, (float)eps);
  };
  dispatch_act(y.has_value() ? *y : x, [&](auto* ty) {
    if (out_bf16) go(ty, (bf16_t*)nullptr);
    else go(ty, (float*)nullptr);
  });
  return {xo, h};
}

}  // namespace llmctl_hybrid
