// Short causal convolution over time on every channel of a step's packed tokens, with the last
// taps - 1 inputs of each live sequence carried in a slot pool between steps:
//   y_t = (add_input ? u_t : 0) + sum_j w[j][c] * u_(t - taps + 1 + j),   zeros before position 0
// (the weights arrive tap-major, [taps, C], so that neighbouring channels are neighbouring loads).
// A token whose tap reaches before the step's first row of its sequence reads the carried inputs; a
// sequence that starts at position 0 ignores what its slot holds.
//
//   causal_conv_kernel        one thread per (token, channel); fp32 arithmetic
//   causal_conv_vec_kernel    the same with 16-byte accesses (8 bf16 / 4 fp32 channels per thread), for
//                             channel counts and row pitches that allow them
//   causal_conv_state_kernel  after it (stream order): the slot's new content from the step's rows and,
//                             for portions shorter than taps - 1, the slot's old content
//   causal_conv_short_kernel  steps whose portions are all short (decode rows): one thread per (sequence,
//                             channel) walks the portion's tokens and then writes the slot, in one launch
//   conv_silu_unit_kernel     silu(convolution + bias) for the inputs of a recurrence, the first groups of channels as unit
//                             vectors in fp32: a group's lanes walk a few tokens with the last inputs in registers;
//                             steps of short portions write the slots in the same launch
#include "hybrid_common.h"

namespace llmctl_hybrid {

constexpr int CONV_MAX_TAPS = 16;

template <typename T>
__global__ __launch_bounds__(256) void causal_conv_kernel(const T* __restrict__ u, int64_t u_stride, const float* __restrict__ w,
                                                          const float* __restrict__ state, const int* __restrict__ seq_of,
                                                          const int* __restrict__ cu, const int* __restrict__ start,
                                                          const int* __restrict__ sslot, T* __restrict__ y, int64_t y_stride, int C,
                                                          int taps, int add_input) {
  const int64_t t = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  const int s = seq_of[t];
  const int li = (int)t - cu[s];  // index inside the step's portion
  const int p0 = start[s];        // position of the portion's first token
  const float* st = state + (int64_t)sslot[s] * (taps - 1) * C;
  const float* wc = w + c;  // tap j of this channel: wc[j * C]
  const float cur = ldf(u + t * u_stride + c);
  float acc = wc[(int64_t)(taps - 1) * C] * cur;
  for (int k = 1; k < taps; ++k) {
    const int i = li - k;
    float v = 0.f;
    if (i >= 0) v = ldf(u + (t - k) * u_stride + c);
    else if (p0 + i >= 0) v = st[(int64_t)(taps - 1 + i) * C + c];
    acc += wc[(int64_t)(taps - 1 - k) * C] * v;
  }
  if (add_input) acc += cur;
  stf(y + t * y_stride + c, acc);
}

template <typename T>
__global__ __launch_bounds__(256) void causal_conv_vec_kernel(const T* __restrict__ u, int64_t u_stride, const float* __restrict__ w,
                                                              const float* __restrict__ state, const int* __restrict__ seq_of,
                                                              const int* __restrict__ cu, const int* __restrict__ start,
                                                              const int* __restrict__ sslot, T* __restrict__ y, int C, int taps,
                                                              int add_input) {
  constexpr int N = Vec16<T>::N;
  const int64_t t = blockIdx.x;
  const int c = (blockIdx.y * 256 + threadIdx.x) * N;
  if (c >= C) return;
  const int s = seq_of[t];
  const int li = (int)t - cu[s];
  const int p0 = start[s];
  const float* st = state + (int64_t)sslot[s] * (taps - 1) * C;
  float cur[N], acc[N], v[N], wk[N];
  Vec16<T>::load(u + t * u_stride + c, cur);
#pragma unroll
  for (int i = 0; i < N; i += 4) Vec16<float>::load(w + (int64_t)(taps - 1) * C + c + i, wk + i);
#pragma unroll
  for (int i = 0; i < N; ++i) acc[i] = wk[i] * cur[i];
  for (int k = 1; k < taps; ++k) {
    const int i0 = li - k;
    if (i0 >= 0) {
      Vec16<T>::load(u + (t - k) * u_stride + c, v);
    } else if (p0 + i0 >= 0) {
#pragma unroll
      for (int i = 0; i < N; i += 4) Vec16<float>::load(st + (int64_t)(taps - 1 + i0) * C + c + i, v + i);
    } else {
      continue;
    }
#pragma unroll
    for (int i = 0; i < N; i += 4) Vec16<float>::load(w + (int64_t)(taps - 1 - k) * C + c + i, wk + i);
#pragma unroll
    for (int i = 0; i < N; ++i) acc[i] += wk[i] * v[i];
  }
  if (add_input) {
#pragma unroll
    for (int i = 0; i < N; ++i) acc[i] += cur[i];
  }
  Vec16<T>::store(y + t * (int64_t)C + c, acc);
}

// Portions of at most CONV_SHORT tokens: thread (sequence, channel) keeps the last taps - 1 inputs in
// registers, walks the portion and writes the slot back; the convolution and the state update are one launch.
constexpr int CONV_SHORT = 4;
template <typename T>
__global__ __launch_bounds__(256) void causal_conv_short_kernel(const T* __restrict__ u, int64_t u_stride, const float* __restrict__ w,
                                                                float* __restrict__ state, const int* __restrict__ cu,
                                                                const int* __restrict__ start, const int* __restrict__ sslot,
                                                                T* __restrict__ y, int C, int taps, int add_input) {
  const int s = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  const int a = cu[s], n = cu[s + 1] - a;
  if (n <= 0) return;
  const int p0 = start[s];
  float* st = state + (int64_t)sslot[s] * (taps - 1) * C;
  float h[CONV_MAX_TAPS];  // h[j]: the input taps - 1 - j positions before the current token (h[taps-1] = current)
  for (int j = 0; j < taps - 1; ++j) h[j] = (p0 - (taps - 1) + j >= 0) ? st[(int64_t)j * C + c] : 0.f;
  const float* wc = w + c;
  for (int i = 0; i < n; ++i) {
    const float cur = ldf(u + (int64_t)(a + i) * u_stride + c);
    h[taps - 1] = cur;
    float acc = add_input ? cur : 0.f;
    for (int j = 0; j < taps; ++j) acc += wc[(int64_t)j * C] * h[j];
    stf(y + (int64_t)(a + i) * C + c, acc);
    for (int j = 0; j < taps - 1; ++j) h[j] = h[j + 1];
  }
  for (int j = 0; j < taps - 1; ++j) st[(int64_t)j * C + c] = h[j];
}

template <typename T>
__global__ __launch_bounds__(256) void causal_conv_state_kernel(const T* __restrict__ u, int64_t u_stride, float* __restrict__ state,
                                                                const int* __restrict__ cu, const int* __restrict__ start,
                                                                const int* __restrict__ sslot, int C, int taps) {
  const int s = blockIdx.x;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= C) return;
  const int a = cu[s], n = cu[s + 1] - a;
  if (n <= 0) return;
  const int p0 = start[s];
  float* st = state + (int64_t)sslot[s] * (taps - 1) * C;
  // entry j holds the input of position (p0 + n) - (taps - 1) + j; ascending j reads old entries
  // j + n > j only, so the update is safe in place
  for (int j = 0; j < taps - 1; ++j) {
    const int li = n - (taps - 1) + j;
    float v = 0.f;
    if (li >= 0) v = ldf(u + (int64_t)(a + li) * u_stride + c);
    else if (p0 + li >= 0) v = st[(int64_t)(j + n) * C + c];
    st[(int64_t)j * C + c] = v;
  }
}

// max_len: the longest portion of the step if the host knows it (0 = unknown)
at::Tensor causal_conv(const at::Tensor& u, const at::Tensor& w, at::Tensor state, const at::Tensor& seq_of, const at::Tensor& cu,
                       const at::Tensor& start, const at::Tensor& sslot, bool add_input, int64_t max_len) {
  check_rows(u, "u");
  const int64_t T = u.size(0), C = u.size(1);
  HYB_CHECK(w.is_cuda() && w.dim() == 2 && w.is_contiguous() && w.scalar_type() == at::kFloat && w.size(1) == C, "w: contiguous fp32 [taps, C]");
  const int64_t taps = w.size(0);
  HYB_CHECK(taps >= 1 && taps <= CONV_MAX_TAPS, "taps in [1, 16]");
  HYB_CHECK(state.is_cuda() && state.is_contiguous() && state.scalar_type() == at::kFloat && state.dim() == 3 && state.size(1) == taps - 1 && state.size(2) == C,
            "state: contiguous fp32 [slots, taps - 1, C]");
  auto i32 = [](const at::Tensor& t) { return t.is_cuda() && t.is_contiguous() && t.scalar_type() == at::kInt; };
  HYB_CHECK(i32(seq_of) && i32(cu) && i32(start) && i32(sslot), "seq_of, cu, start, slots: contiguous int32 GPU tensors");
  const int64_t ns = start.numel();
  HYB_CHECK(seq_of.numel() == T && cu.numel() == ns + 1 && sslot.numel() == ns, "seq_of [T], cu [n + 1], start [n], slots [n]");
  c10::DeviceGuard guard(u.device());
  at::Tensor y = at::empty({T, C}, u.options());
  if (T == 0) return y;
  const unsigned cb = (unsigned)((C + 255) / 256);
  HYB_CHECK(cb <= 65535, "too many channels for one launch");
  dispatch_act(u, [&](auto* tag) {
    using Tt = std::remove_pointer_t<decltype(tag)>;
    if (max_len >= 1 && max_len <= CONV_SHORT) {
      causal_conv_short_kernel<Tt><<<dim3((unsigned)ns, cb), 256, 0, cur_stream()>>>(
          (const Tt*)u.data_ptr(), u.stride(0), w.data_ptr<float>(), state.data_ptr<float>(), cu.data_ptr<int>(), start.data_ptr<int>(),
          sslot.data_ptr<int>(), (Tt*)y.data_ptr(), (int)C, (int)taps, add_input ? 1 : 0);
      return;
    }
    constexpr int N = Vec16<Tt>::N;
    if (C % 8 == 0 && aligned16<Tt>(u) && reinterpret_cast<uintptr_t>(state.data_ptr()) % 16 == 0 && reinterpret_cast<uintptr_t>(w.data_ptr()) % 16 == 0)
      causal_conv_vec_kernel<Tt><<<dim3((unsigned)T, (unsigned)((C / N + 255) / 256)), 256, 0, cur_stream()>>>(
          (const Tt*)u.data_ptr(), u.stride(0), w.data_ptr<float>(), state.data_ptr<float>(), seq_of.data_ptr<int>(), cu.data_ptr<int>(),
          start.data_ptr<int>(), sslot.data_ptr<int>(), (Tt*)y.data_ptr(), (int)C, (int)taps, add_input ? 1 : 0);
    else
      causal_conv_kernel<Tt><<<dim3((unsigned)T, cb), 256, 0, cur_stream()>>>(
          (const Tt*)u.data_ptr(), u.stride(0), w.data_ptr<float>(), state.data_ptr<float>(), seq_of.data_ptr<int>(), cu.data_ptr<int>(),
          start.data_ptr<int>(), sslot.data_ptr<int>(), (Tt*)y.data_ptr(), C, (int)C, (int)taps, add_input ? 1 : 0);
    if (taps > 1)
      causal_conv_state_kernel<Tt><<<dim3((unsigned)ns, cb), 256, 0, cur_stream()>>>(
          (const Tt*)u.data_ptr(), u.stride(0), state.data_ptr<float>(), cu.data_ptr<int>(), start.data_ptr<int>(), sslot.data_ptr<int>(),
          (int)C, (int)taps);
  });
  return y;
}

namespace {
struct ConvUnitArgs {
  const void* u;
  int64_t u_st;
  const float* w;     // [taps, C]
  const float* bias;  // nullptr or [C]
  float* state;       // [slots, taps - 1, C]
  const int* seq_of;
  const int* cu;
  const int* start;
  const int* sslot;
  float* qk;  // [T, ng, dk]
  void* y;    // [T, C - ng * dk]
  int T, C, taps, ng, nq, dk, lg, whole;  // lg lanes per unit; whole: a sequence per walk
  float qscale, eps;
};

// the sum over a unit's ``lg`` lanes (a power of two), in each of them: inside a row of 16 by lane permutations, then across rows
__device__ __forceinline__ float unit_sum(float v, int lg) {
  auto add = [&](auto ctrl) { v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), decltype(ctrl)::value, 0xf, 0xf, true)); };
  if (lg > 1) add(std::integral_constant<int, 0xB1>());   // neighbours of a pair
  if (lg > 2) add(std::integral_constant<int, 0x4E>());   // pairs of a quad
  if (lg > 4) add(std::integral_constant<int, 0x141>());  // quads of a half row
  if (lg > 8) add(std::integral_constant<int, 0x140>());  // halves of a row
  if (lg > 16) v += __shfl_xor(v, 16, 64);
  if (lg > 32) v += __shfl_xor(v, 32, 64);
  return v;
}

// A unit is a group of dk channels, or a span of lg * VEC * NI of the other channels.  TAPS == 0: any number of taps.  A walk of
// WALK tokens that lies inside one sequence, its taps inside the step's rows, runs without branches on rows requested at
// once; any other walk goes token by token.
template <typename T, int VEC, int NI, int TAPS, int WALK>
__global__ __launch_bounds__(256) void conv_silu_unit_kernel(ConvUnitArgs a) {
  constexpr int NH = TAPS > 1 ? TAPS - 1 : 1;
  const int lane = threadIdx.x % a.lg;
  const int unit = ((int)blockIdx.y * 256 + (int)threadIdx.x) / a.lg;
  const int taps = TAPS > 0 ? TAPS : a.taps;
  const int span = a.lg * VEC * NI, gw = a.ng * a.dk;
  const bool grp = unit < a.ng;
  const int base = grp ? unit * a.dk : gw + (unit - a.ng) * span;
  const int lim = grp ? base + a.dk : min(base + span, a.C);
  if (base >= a.C) return;  // (the unit's lanes leave together)
  int t_lo, t_hi;
  if (a.whole) {
    t_lo = a.cu[blockIdx.x], t_hi = a.cu[blockIdx.x + 1];
    if (t_lo >= t_hi) return;
  } else {
    t_lo = (int)blockIdx.x * WALK, t_hi = min(t_lo + WALK, a.T);
  }
  const T* u = reinterpret_cast<const T*>(a.u);
  int ch[NI];
  bool ok[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    ch[i] = base + (i * a.lg + lane) * VEC;
    ok[i] = ch[i] < lim;  // VEC divides the group and the row
    if (!ok[i]) ch[i] = base;
  }
  auto load_row = [&](const T* p, float* v) {
    if constexpr (VEC == 4 && sizeof(T) == 4) {
      Vec16<float>::load(reinterpret_cast<const float*>(p), v);
    } else if constexpr (VEC == 4) {
      const uint2 x = *reinterpret_cast<const uint2*>(p);
      v[0] = __uint_as_float(x.x << 16), v[1] = __uint_as_float(x.x & 0xffff0000u);
      v[2] = __uint_as_float(x.y << 16), v[3] = __uint_as_float(x.y & 0xffff0000u);
    } else {
      v[0] = ldf(p);
    }
  };
  auto load_f = [&](const float* p, float* v) {
    if constexpr (VEC == 4) Vec16<float>::load(p, v);
    else v[0] = p[0];
  };
  // silu in place, then the unit's result for token t
  auto activate = [&](float (&x)[NI][VEC]) {
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
      for (int c = 0; c < VEC; ++c) {
        x[i][c] *= __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * x[i][c]));
        if (ok[i]) ss += x[i][c] * x[i][c];
      }
    return ss;
  };
  auto emit = [&](int t, float (&x)[NI][VEC], float ss) {
    if (grp) {
      const float f = (unit < a.nq ? a.qscale : 1.0f) / sqrtf(ss + a.eps);
      float* o = a.qk + ((int64_t)t * a.ng + unit) * a.dk - base;
#pragma unroll
      for (int i = 0; i < NI; ++i) {
#pragma unroll
        for (int c = 0; c < VEC; ++c) x[i][c] *= f;
        if (ok[i]) {
          if constexpr (VEC == 4) Vec16<float>::store(o + ch[i], x[i]);
          else o[ch[i]] = x[i][0];
        }
      }
    } else {
      T* o = reinterpret_cast<T*>(a.y) + (int64_t)t * (a.C - gw) - gw;
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        if (!ok[i]) continue;
        if constexpr (VEC == 4 && sizeof(T) == 4) {
          Vec16<float>::store(reinterpret_cast<float*>(o) + ch[i], x[i]);
        } else if constexpr (VEC == 4) {
          unsigned w[2];
#pragma unroll
          for (int c = 0; c < 2; ++c)
            w[c] = (unsigned)__bfloat16_as_ushort(__float2bfloat16(x[i][2 * c])) | ((unsigned)__bfloat16_as_ushort(__float2bfloat16(x[i][2 * c + 1])) << 16);
          *reinterpret_cast<uint2*>(o + ch[i]) = make_uint2(w[0], w[1]);
        } else {
          stf(o + ch[i], x[i][0]);
        }
      }
    }
  };
  float wk[TAPS > 0 ? TAPS : 1][NI][VEC], bs[NI][VEC];
#pragma unroll
  for (int i = 0; i < NI; ++i) {
#pragma unroll
    for (int c = 0; c < VEC; ++c) bs[i][c] = 0.f;
    if (a.bias != nullptr) load_f(a.bias + ch[i], bs[i]);
    if constexpr (TAPS > 0) {
#pragma unroll
      for (int k = 0; k < TAPS; ++k) load_f(a.w + (int64_t)k * a.C + ch[i], wk[k][i]);
    }
  }
  int s = a.whole ? (int)blockIdx.x : a.seq_of[t_lo];
  int s0 = a.cu[s], s1 = a.cu[s + 1], p0 = a.start[s];
  if constexpr (TAPS > 0 && NI == 1 && WALK > 1) {
    if (!a.whole && t_hi - t_lo == WALK && t_hi <= s1 && t_lo - s0 >= TAPS - 1) {
      const T* up = u + (int64_t)(t_lo - (TAPS - 1)) * a.u_st + ch[0];
      float r[WALK + TAPS - 1][VEC];
#pragma unroll
      for (int j = 0; j < WALK + TAPS - 1; ++j) {
        load_row(up, r[j]);
        up += a.u_st;
      }
      float x[WALK][1][VEC], ss[WALK];
#pragma unroll
      for (int j = 0; j < WALK; ++j) {
#pragma unroll
        for (int c = 0; c < VEC; ++c) {
          float acc = bs[0][c];
#pragma unroll
          for (int k = 0; k < TAPS; ++k) acc += wk[k][0][c] * r[j + k][c];
          x[j][0][c] = acc;
        }
        ss[j] = activate(x[j]);
      }
      if (grp) {
#pragma unroll
        for (int j = 0; j < WALK; ++j) ss[j] = unit_sum(ss[j], a.lg);
      }
#pragma unroll
      for (int j = 0; j < WALK; ++j) emit(t_lo + j, x[j], ss[j]);
      return;
    }
  }
  // the input ``k`` positions before token t of the sequence that begins at row s0, position p0
  auto past = [&](int t, int k, const float* st, int i, float* v) {
    const int j = t - s0 - k;
    if (j >= 0) {
      load_row(u + (int64_t)(t - k) * a.u_st + ch[i], v);
    } else if (p0 + j >= 0) {
      load_f(st + (int64_t)(taps - 1 + j) * a.C + ch[i], v);
    } else {
#pragma unroll
      for (int c = 0; c < VEC; ++c) v[c] = 0.f;
    }
  };
  float hist[NH][NI][VEC];  // hist[k]: the input k + 1 positions before the current token
  float* st = a.state + (int64_t)a.sslot[s] * (taps - 1) * a.C;
#pragma unroll 1
  for (int t = t_lo; t < t_hi; ++t) {
    bool reload = t == t_lo;
    if (t >= s1) {
      s = a.seq_of[t];
      s0 = a.cu[s], s1 = a.cu[s + 1], p0 = a.start[s];
      st = a.state + (int64_t)a.sslot[s] * (taps - 1) * a.C;
      reload = true;
    }
    if constexpr (TAPS > 1) {
      if (reload) {
#pragma unroll
        for (int k = 0; k < TAPS - 1; ++k)
#pragma unroll
          for (int i = 0; i < NI; ++i) past(t, k + 1, st, i, hist[k][i]);
      }
    }
    float x[NI][VEC];
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      float cur[VEC];
      load_row(u + (int64_t)t * a.u_st + ch[i], cur);
      if constexpr (TAPS > 0) {  // (the oldest tap first, as on the other path)
#pragma unroll
        for (int c = 0; c < VEC; ++c) {
          float acc = bs[i][c];
#pragma unroll
          for (int k = TAPS - 2; k >= 0; --k) acc += wk[TAPS - 2 - k][i][c] * hist[k][i][c];
          x[i][c] = acc + wk[TAPS - 1][i][c] * cur[c];
        }
#pragma unroll
        for (int k = TAPS - 2; k > 0; --k)
#pragma unroll
          for (int c = 0; c < VEC; ++c) hist[k][i][c] = hist[k - 1][i][c];
        if constexpr (TAPS > 1) {
#pragma unroll
          for (int c = 0; c < VEC; ++c) hist[0][i][c] = cur[c];
        }
      } else {
        float w1[VEC], v[VEC];
        load_f(a.w + (int64_t)(taps - 1) * a.C + ch[i], w1);
#pragma unroll
        for (int c = 0; c < VEC; ++c) x[i][c] = bs[i][c] + w1[c] * cur[c];
        for (int k = 1; k < taps; ++k) {
          past(t, k, st, i, v);
          load_f(a.w + (int64_t)(taps - 1 - k) * a.C + ch[i], w1);
#pragma unroll
          for (int c = 0; c < VEC; ++c) x[i][c] += w1[c] * v[c];
        }
      }
    }
    const float ss = activate(x);
    emit(t, x, grp ? unit_sum(ss, a.lg) : 0.f);
  }
  if (a.whole) {  // the slot's new content; entry j is the input taps - 1 - j positions before the portion's end
    for (int j = 0; j < taps - 1; ++j) {
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        float v[VEC];
        past(t_hi, taps - 1 - j, st, i, v);  // (ascending j reads entries that are not yet rewritten)
        if (ok[i]) {
#pragma unroll
          for (int c = 0; c < VEC; ++c) st[(int64_t)j * a.C + ch[i] + c] = v[c];
        }
      }
    }
  }
}
}  // namespace

// max_len: the longest portion of the step
std::tuple<at::Tensor, at::Tensor> conv_silu_unit(const at::Tensor& u, const at::Tensor& w, const c10::optional<at::Tensor>& bias, at::Tensor state,
                                                  const at::Tensor& seq_of, const at::Tensor& cu, const at::Tensor& start, const at::Tensor& sslot,
                                                  int64_t nq, int64_t nk, int64_t dk, double qscale, double eps, int64_t max_len) {
  check_rows(u, "u");
  const int64_t T = u.size(0), C = u.size(1), ng = nq + nk;
  auto f32c = [](const at::Tensor& t) { return t.is_cuda() && t.is_contiguous() && t.scalar_type() == at::kFloat; };
  HYB_CHECK(f32c(w) && w.dim() == 2 && w.size(1) == C && w.size(0) >= 1 && w.size(0) <= CONV_MAX_TAPS, "w: contiguous fp32 [taps, C], 1 .. 16 taps");
  const int64_t taps = w.size(0);
  HYB_CHECK(!bias.has_value() || (f32c(*bias) && bias->numel() == C), "bias: fp32 [C]");
  HYB_CHECK(f32c(state) && state.dim() == 3 && state.size(1) == taps - 1 && state.size(2) == C, "state: contiguous fp32 [slots, taps - 1, C]");
  auto i32 = [](const at::Tensor& t) { return t.is_cuda() && t.is_contiguous() && t.scalar_type() == at::kInt; };
  HYB_CHECK(i32(seq_of) && i32(cu) && i32(start) && i32(sslot), "seq_of, cu, start, slots: contiguous int32 GPU tensors");
  const int64_t ns = start.numel();
  HYB_CHECK(seq_of.numel() == T && cu.numel() == ns + 1 && sslot.numel() == ns, "seq_of [T], cu [n + 1], start [n], slots [n]");
  HYB_CHECK(nq >= 0 && nk >= 0 && (ng == 0 || (dk >= 1 && dk <= 256)) && ng * dk <= C, "groups of 1 .. 256 channels inside the row");
  if (ng == 0) dk = 0;
  c10::DeviceGuard guard(u.device());
  at::Tensor qk = at::empty({T, ng, dk}, u.options().dtype(at::kFloat));
  at::Tensor y = at::empty({T, C - ng * dk}, u.options());
  if (T == 0 || C == 0) return {qk, y};
  const bool v4 = dk % 4 == 0 && C % 4 == 0 && u.stride(0) % 4 == 0 && reinterpret_cast<uintptr_t>(u.data_ptr()) % (4 * u.element_size()) == 0;
  const int64_t vec = v4 ? 4 : 1;
  int lg = 64;
  if (ng > 0)
    for (lg = 1; lg < 64 && lg * vec < dk;) lg *= 2;
  const int ni = ng > 0 ? (int)((dk + lg * vec - 1) / (lg * vec)) : 1;  // 1, or up to 4 in the scalar form
  ConvUnitArgs a;
  a.u = u.data_ptr(), a.u_st = u.stride(0), a.w = w.data_ptr<float>(), a.bias = bias.has_value() ? bias->data_ptr<float>() : nullptr;
  a.state = state.data_ptr<float>(), a.seq_of = seq_of.data_ptr<int>(), a.cu = cu.data_ptr<int>(), a.start = start.data_ptr<int>(), a.sslot = sslot.data_ptr<int>();
  a.qk = qk.data_ptr<float>(), a.y = y.data_ptr();
  a.T = (int)T, a.C = (int)C, a.taps = (int)taps, a.ng = (int)ng, a.nq = (int)nq, a.dk = (int)dk, a.lg = lg;
  a.whole = max_len >= 1 && max_len <= CONV_SHORT ? 1 : 0;
  a.qscale = (float)qscale, a.eps = (float)eps;
  const int NIv = ni > 1 ? 4 : 1;
  const int64_t span = (int64_t)lg * vec * NIv, units = ng + (C - ng * dk + span - 1) / span;
  const int64_t by = (units * lg + 255) / 256;
  HYB_CHECK(by <= 65535, "too many channels for one launch");
  // tokens per walk: 8 where that leaves the chip a thousand workgroups
  const int walk = (T + 7) / 8 * by >= 1024 ? 8 : 4;
  const dim3 grid((unsigned)(a.whole ? ns : (T + walk - 1) / walk), (unsigned)by);
  dispatch_act(u, [&](auto* tag) {
    using Tt = std::remove_pointer_t<decltype(tag)>;
    auto go = [&](auto kern) { kern<<<grid, 256, 0, cur_stream()>>>(a); };
    auto taps_of = [&](auto vc, auto nc, auto wc) {
      constexpr int V = decltype(vc)::value, N = decltype(nc)::value, WK = decltype(wc)::value;
      switch (taps) {
        case 2: go(conv_silu_unit_kernel<Tt, V, N, 2, WK>); break;
        case 3: go(conv_silu_unit_kernel<Tt, V, N, 3, WK>); break;
        case 4: go(conv_silu_unit_kernel<Tt, V, N, 4, WK>); break;
        default: go(conv_silu_unit_kernel<Tt, V, N, 0, WK>); break;
      }
    };
    auto sized = [&](auto vc, auto nc) {
      if (walk == 8) taps_of(vc, nc, std::integral_constant<int, 8>());
      else taps_of(vc, nc, std::integral_constant<int, 4>());
    };
    if (v4) sized(std::integral_constant<int, 4>(), std::integral_constant<int, 1>());
    else if (NIv == 1) sized(std::integral_constant<int, 1>(), std::integral_constant<int, 1>());
    else sized(std::integral_constant<int, 1>(), std::integral_constant<int, 4>());
    if (!a.whole && taps > 1)
      causal_conv_state_kernel<Tt><<<dim3((unsigned)ns, (unsigned)((C + 255) / 256)), 256, 0, cur_stream()>>>(
          (const Tt*)u.data_ptr(), u.stride(0), state.data_ptr<float>(), cu.data_ptr<int>(), start.data_ptr<int>(), sslot.data_ptr<int>(), (int)C, (int)taps);
  });
  return {qk, y};
}

}  // namespace llmctl_hybrid
