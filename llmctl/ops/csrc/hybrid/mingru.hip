// An elementwise gated recurrence whose gates read only the current token, fused with its output gate:
//   zeta = sigmoid(z + z_bias), u = x + x_bias, cand = u + 1/2 (u >= 0) or sigmoid(u) (u < 0),
//   S_t = (1 - zeta) S_(t-1) + zeta cand,   out_t = S_t silu(g_t)
// over packed rows [z | x | g] (W columns each); the state pool S [slots, W] is fp32, a sequence that starts at
// position 0 begins from zeros.
//
//   mingru_seq_kernel    one thread per (sequence, channel), token by token (decode rows and short portions)
//   mingru_local_kernel  long portions in chunks, all chunks at once: the chunk's total decay A (the product of its
//                        1 - zeta) and its end state B from zeros (the first chunk: from the carried state, which
//                        it also copies aside); no outputs
//   mingru_out_kernel    every chunk again: its first state folded from the (A, B) of the chunks before it
//                        (S <- A S + B), outputs token by token, and the last chunk writes the new carried state
// Two neighbouring channels a thread where the rows allow 4-byte (bf16) / 8-byte (fp32) accesses.
#include "hybrid_common.h"

namespace llmctl_hybrid {

namespace {
constexpr int UNR = 8;  // tokens fetched ahead as one batch

struct MinGruArgs {
  const void* z;  // [T, >= 3 W]
  int64_t z_st;
  const float* zb;
  const float* xb;
  float* S;
  const int* slots;
  const int* cu;
  const int* start;
  void* out;  // [T, W]
  float* A;   // [sequences, chunks, W]
  float* B;   // [sequences, chunks, W]
  float* S0;  // [sequences, W]
  int W, chunk, nchunks, seq0;  // the launch's first sequence
};

__device__ __forceinline__ float rcp_(float v) { return __builtin_amdgcn_rcpf(v); }

// sigmoid(v) and sigmoid(-v), each to full relative precision
__device__ __forceinline__ void sig_pair(float v, float& p, float& n) {
  const float e = __expf(-fabsf(v));
  const float r = rcp_(1.0f + e);
  p = v >= 0.f ? r : e * r;
  n = v >= 0.f ? e * r : r;
}

__device__ __forceinline__ void coeffs(float zv, float u, float& keep, float& add) {
  float zeta, s, d;
  sig_pair(zv, zeta, keep);
  sig_pair(u, s, d);
  add = zeta * (u >= 0.f ? u + 0.5f : s);
}

template <typename T, int V>
__device__ __forceinline__ void ldv(const T* p, float* v) {
  if constexpr (V == 1) {
    v[0] = ldf(p);
  } else if constexpr (std::is_same_v<T, float>) {
    const float2 r = *reinterpret_cast<const float2*>(p);
    v[0] = r.x, v[1] = r.y;
  } else {
    const unsigned r = *reinterpret_cast<const unsigned*>(p);
    v[0] = __uint_as_float(r << 16), v[1] = __uint_as_float(r & 0xffff0000u);
  }
}
template <typename T, int V>
__device__ __forceinline__ void stv(T* p, const float* v) {
  if constexpr (V == 1) {
    stf(p, v[0]);
  } else if constexpr (std::is_same_v<T, float>) {
    *reinterpret_cast<float2*>(p) = make_float2(v[0], v[1]);
  } else {
    *reinterpret_cast<unsigned*>(p) = (unsigned)__bfloat16_as_ushort(__float2bfloat16(v[0])) | ((unsigned)__bfloat16_as_ushort(__float2bfloat16(v[1])) << 16);
  }
}

// Rows [t0, t1) of one channel group from the state S (in place): outputs when OUT, the running decay product when PROD.
template <typename T, int V, bool OUT, bool PROD>
__device__ __forceinline__ void walk(const MinGruArgs& a, int c, int t0, int t1, float* S, float* A) {
  const T* zp = reinterpret_cast<const T*>(a.z) + c;
  T* op = reinterpret_cast<T*>(a.out) + c;
  float zb[V], xb[V];
#pragma unroll
  for (int i = 0; i < V; ++i) zb[i] = a.zb[c + i], xb[i] = a.xb[c + i];
  for (int t = t0; t < t1; t += UNR) {
    float zv[UNR][V], xv[UNR][V], gv[UNR][V];
#pragma unroll
    for (int k = 0; k < UNR; ++k) {
      const T* r = zp + (int64_t)min(t + k, t1 - 1) * a.z_st;
      ldv<T, V>(r, zv[k]);
      ldv<T, V>(r + a.W, xv[k]);
      if constexpr (OUT) ldv<T, V>(r + 2 * a.W, gv[k]);
    }
#pragma unroll
    for (int k = 0; k < UNR; ++k) {
      if (t + k < t1) {
        float o[V];
#pragma unroll
        for (int i = 0; i < V; ++i) {
          float keep, add;
          coeffs(zv[k][i] + zb[i], xv[k][i] + xb[i], keep, add);
          S[i] = keep * S[i] + add;
          if constexpr (PROD) A[i] *= keep;
          if constexpr (OUT) {
            float sp, sn;
            sig_pair(gv[k][i], sp, sn);
            o[i] = S[i] * gv[k][i] * sp;
          }
        }
        if constexpr (OUT) stv<T, V>(op + (int64_t)(t + k) * a.W, o);
      }
    }
  }
}

template <typename T, int V>
__global__ __launch_bounds__(64) void mingru_seq_kernel(MinGruArgs a) {
  const int s = a.seq0 + blockIdx.y;
  const int c = (blockIdx.x * 64 + threadIdx.x) * V;
  const int t0 = a.cu[s], t1 = a.cu[s + 1];
  if (c >= a.W || t0 >= t1) return;
  float* Sp = a.S + (int64_t)a.slots[s] * a.W + c;
  float S[V];
#pragma unroll
  for (int i = 0; i < V; ++i) S[i] = a.start[s] == 0 ? 0.f : Sp[i];
  walk<T, V, true, false>(a, c, t0, t1, S, nullptr);
#pragma unroll
  for (int i = 0; i < V; ++i) Sp[i] = S[i];
}

template <typename T, int V>
__global__ __launch_bounds__(64) void mingru_local_kernel(MinGruArgs a) {
  const int k = blockIdx.y, sl = blockIdx.z, s = a.seq0 + sl;
  const int c = (blockIdx.x * 64 + threadIdx.x) * V;
  const int t0 = a.cu[s] + k * a.chunk, t1 = min(t0 + a.chunk, a.cu[s + 1]);
  if (c >= a.W || t0 >= t1) return;
  float S[V], A[V];
#pragma unroll
  for (int i = 0; i < V; ++i) S[i] = 0.f, A[i] = 1.f;
  if (k == 0) {
    const float* Sp = a.S + (int64_t)a.slots[s] * a.W + c;
#pragma unroll
    for (int i = 0; i < V; ++i) {
      if (a.start[s] != 0) S[i] = Sp[i];
      a.S0[(int64_t)sl * a.W + c + i] = S[i];
    }
  }
  walk<T, V, false, true>(a, c, t0, t1, S, A);
  const int64_t o = ((int64_t)sl * a.nchunks + k) * a.W + c;
#pragma unroll
  for (int i = 0; i < V; ++i) a.A[o + i] = A[i], a.B[o + i] = S[i];
}

template <typename T, int V>
__global__ __launch_bounds__(64) void mingru_out_kernel(MinGruArgs a) {
  const int k = blockIdx.y, sl = blockIdx.z, s = a.seq0 + sl;
  const int c = (blockIdx.x * 64 + threadIdx.x) * V;
  const int t0 = a.cu[s] + k * a.chunk, end = a.cu[s + 1], t1 = min(t0 + a.chunk, end);
  if (c >= a.W || t0 >= t1) return;
  float S[V];
  if (k == 0) {
#pragma unroll
    for (int i = 0; i < V; ++i) S[i] = a.S0[(int64_t)sl * a.W + c + i];
  } else {
    const float* Ap = a.A + (int64_t)sl * a.nchunks * a.W + c;
    const float* Bp = a.B + (int64_t)sl * a.nchunks * a.W + c;
#pragma unroll
    for (int i = 0; i < V; ++i) S[i] = Bp[i];  // chunk 0's end state holds the carried one
    for (int j = 1; j < k; j += UNR) {
      float av[UNR][V], bv[UNR][V];
#pragma unroll
      for (int q = 0; q < UNR; ++q) {
        const int64_t o = (int64_t)min(j + q, k - 1) * a.W;
        ldv<float, V>(Ap + o, av[q]);
        ldv<float, V>(Bp + o, bv[q]);
      }
#pragma unroll
      for (int q = 0; q < UNR; ++q)
        if (j + q < k) {
#pragma unroll
          for (int i = 0; i < V; ++i) S[i] = av[q][i] * S[i] + bv[q][i];
        }
    }
  }
  walk<T, V, true, false>(a, c, t0, t1, S, nullptr);
  if (t1 == end) {
    float* Sp = a.S + (int64_t)a.slots[s] * a.W + c;
#pragma unroll
    for (int i = 0; i < V; ++i) Sp[i] = S[i];
  }
}
}  // namespace

// z [T, >= 3 W] = [z | x | g | ...].  The first ``portions`` sequences may be long (their longest has ``max_q`` rows), the
// others bring one row each.
at::Tensor mingru_scan(const at::Tensor& z, const at::Tensor& z_bias, const at::Tensor& x_bias, at::Tensor S, const at::Tensor& slots,
                       const at::Tensor& cu, const at::Tensor& start, int64_t portions, int64_t max_q, int64_t chunk) {
  check_rows(z, "z");
  HYB_CHECK(S.is_cuda() && S.is_contiguous() && S.dim() == 2 && S.scalar_type() == at::kFloat, "S: contiguous fp32 [slots, W]");
  const int64_t T = z.size(0), W = S.size(1), ns = start.numel();
  HYB_CHECK(z.size(1) >= 3 * W, "z: [T, >= 3 W]");
  auto f32 = [&](const at::Tensor& t) { return t.is_cuda() && t.is_contiguous() && t.scalar_type() == at::kFloat && t.numel() == W; };
  auto i32 = [](const at::Tensor& t, int64_t n) { return t.is_cuda() && t.is_contiguous() && t.scalar_type() == at::kInt && t.numel() == n; };
  HYB_CHECK(f32(z_bias) && f32(x_bias), "biases: fp32 [W]");
  HYB_CHECK(i32(slots, ns) && i32(cu, ns + 1) && i32(start, ns), "slots [n], cu [n + 1], start [n]: int32");
  HYB_CHECK(portions >= 0 && portions <= ns && max_q >= 0 && chunk >= 1 && ns <= 65535, "portions lie in 0 .. n; chunk >= 1");
  c10::DeviceGuard guard(z.device());
  at::Tensor out = at::empty({T, W}, z.options());
  if (T == 0) return out;
  MinGruArgs a{};
  a.z = z.data_ptr();
  a.z_st = z.stride(0);
  a.zb = z_bias.data_ptr<float>();
  a.xb = x_bias.data_ptr<float>();
  a.S = S.data_ptr<float>();
  a.slots = slots.data_ptr<int>();
  a.cu = cu.data_ptr<int>();
  a.start = start.data_ptr<int>();
  a.out = out.data_ptr();
  a.W = (int)W;
  const bool chunked = portions > 0 && max_q >= 2 * chunk;
  at::Tensor ws;
  if (chunked) {
    a.chunk = (int)chunk;
    a.nchunks = (int)((max_q + chunk - 1) / chunk);
    HYB_CHECK(a.nchunks <= 65535, "too many chunks");
    ws = at::empty({portions * (2 * (int64_t)a.nchunks + 1) * W}, S.options());
    a.A = ws.data_ptr<float>();
    a.B = a.A + portions * a.nchunks * W;
    a.S0 = a.B + portions * a.nchunks * W;
  }
  hipStream_t st = cur_stream();
  dispatch_act(z, [&](auto* tag) {
    using Tt = std::remove_pointer_t<decltype(tag)>;
    const bool pair = W % 2 == 0 && z.stride(0) % 2 == 0 && reinterpret_cast<uintptr_t>(z.data_ptr()) % (2 * sizeof(Tt)) == 0;
    auto go = [&](auto vv) {
      constexpr int V = decltype(vv)::value;
      const unsigned cb = (unsigned)((W + 64 * V - 1) / (64 * V));
      if (chunked) {
        a.seq0 = 0;
        const dim3 grid(cb, (unsigned)a.nchunks, (unsigned)portions);
        mingru_local_kernel<Tt, V><<<grid, 64, 0, st>>>(a);
        mingru_out_kernel<Tt, V><<<grid, 64, 0, st>>>(a);
      }
      const int64_t rest = chunked ? ns - portions : ns;
      if (rest > 0) {
        a.seq0 = chunked ? (int)portions : 0;
        mingru_seq_kernel<Tt, V><<<dim3(cb, (unsigned)rest), 64, 0, st>>>(a);
      }
    };
    if (pair) go(std::integral_constant<int, 2>{});
    else go(std::integral_constant<int, 1>{});
  });
  return out;
}

}  // namespace llmctl_hybrid
