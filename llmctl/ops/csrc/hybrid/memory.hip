// Matrix memories with one decay per head and token: per (sequence, head) a memory S [dk, dv] (fp32) with
//   S_t = g_t S_(t-1) + k_t u_t^T,   u_t = beta_t v_t or beta_t (v_t - g_t S_(t-1)^T k_t),   o_t = S_t^T q_t (+ skip v_t),
// the decay g and the write strength beta formed here in fp32 (kinds: 0 fixed decay and beta = 1; 1 state-space: beta = dt =
// softplus(ga + dt_bias), g = exp(-exp(a_log) dt); 2 delta: g likewise, beta = sigmoid(gb), and the subtracting form of u).
//
//   memory_decode        one token per sequence: S is read once into registers, S^T k and S^T q are summed together, S is
//                        written back (o = g S^T q + (k . q) u needs no second sweep)
//   memory_chunks        chunks of 64 tokens from the memory at their first token.  With L_t the running sum of log g inside
//                        the chunk, o_t = e^(L_t) S_0^T q_t + sum_(s <= t) e^(L_t - L_s) (q_t . k_s) u_s; for the delta kind the
//                        u solve (I + A) U = beta (V - e^L K S_0) with A_ts = beta_t e^(L_t - L_s) (k_t . k_s), s < t, block by
//                        block (16 x 16 diagonal blocks are inverted by substitution).  Called on whole portions it also
//                        writes the new memory, e^(L_n) S_0 + sum_t e^(L_n - L_t) k_t u_t^T.
//                        Both of these can end in the mixer's head norm: o over its root mean square, a weight, a silu gate.
//   memory_chunk_local   every chunk from a zero memory: its own contribution, its total decay and, for the delta kind, the
//                        matrix that carries a memory over the chunk (the same solve on the columns of K)
//   memory_combine       the memory at every chunk's first token in order, and the sequence's new carried memory
//
// All products run on the fp32 matrix cores (MFMA 16x16x4) in fp32.  A step j of such a product takes logical index 4 g + j of a
// 16-wide block from lane group g = lane / 16 on both sides, so that a lane's A operands are 16 neighbouring bytes and a
// result (rows 4 g + r, column lane % 16) is a B operand as it stands: values, solved rows and memories stay in registers
// from product to product, and only K, Q and the score blocks go through LDS.  A wave owns 16 value columns.
#include "hybrid_common.h"

namespace llmctl_hybrid {

namespace {
using f32x4 = float __attribute__((ext_vector_type(4)));

constexpr int CH = 64;            // tokens per chunk
constexpr int AS = CH + 4;        // row stride of the score blocks in LDS
constexpr int TBS = 20;           // row stride of an inverted diagonal block
enum { KIND_FIXED = 0, KIND_SSM = 1, KIND_DELTA = 2 };

struct MemArgs {
  const void* q;
  const void* k;
  const void* v;
  int64_t q_st, q_sh, k_st, k_sh, v_st, v_sh;  // token and head strides (elements)
  const void* ga;  // [T, H] gate columns in v's dtype (kinds 1, 2)
  const void* gb;  // kind 2
  int64_t ga_st, gb_st;
  const float* a_log;
  const float* dt_bias;
  const float* log_decay;
  const float* skip;  // nullptr or [H]
  float* S;           // [slots, H, dk, dv]
  const int* slots;
  const int* cu;
  const int* start;
  const float* init;  // memory_chunks on the chunks of longer portions: [chunks, H, dk, dv] (nullptr: whole portions, read from S)
  float* loc;         // memory_chunk_local: [chunks, H, dk, dv]
  float* dec;         // [chunks, H]
  float* trans;       // [chunks, H, dkp, dkp]
  float* out;         // [T, H, dv]
  // fused head norm (y given, out not): y = o / rms(o over dv) * hn_w (if given) * hn_g sigmoid(hn_g), [T, H * dv] in v's dtype
  void* y;
  const float* hn_w;  // nullptr or [H * dv]
  const void* hn_g;   // [T, H * dv] in v's dtype
  int64_t hn_st;
  float hn_eps;
  int kind, H, rep, dk, dv, vec, row0;
};

// z sigmoid(z); the hardware's exponential and reciprocal are good to an ulp
__device__ __forceinline__ float silu(float z) { return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z)); }

// (log g, beta) of head h from the raw gate columns
__device__ __forceinline__ void gate_values(const MemArgs& a, int h, float ga, float gb, float& la, float& beta) {
  if (a.kind == KIND_FIXED) {
    la = a.log_decay[h];
    beta = 1.0f;
    return;
  }
  const float x = ga + a.dt_bias[h];
  const float dt = fmaxf(x, 0.f) + log1pf(expf(-fabsf(x)));
  la = -expf(a.a_log[h]) * dt;
  beta = a.kind == KIND_SSM ? dt : 1.0f / (1.0f + expf(-gb));
}

// ------------------------------------------------------------------------------------------ decode
// 16 thread groups share the dk rows of S; a thread owns VEC neighbouring value columns of its rows, CL threads a row.
template <typename TQ, typename TV, int VEC, int NR, int CL>
__global__ __launch_bounds__(16 * CL) void memory_decode_kernel(MemArgs a) {
  constexpr int NWV = 16 * CL / 64, NS = 2 * VEC + 1;
  __shared__ float red[NWV][CL][NS];
  const int n = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int wave = tid >> 6, cl = tid % CL, rg = tid / CL;
  const int64_t t = a.row0 + n;
  const int dk = a.dk, dv = a.dv;
  const int col = blockIdx.z * CL * VEC + cl * VEC;
  const bool cok = col < dv;  // VEC divides dv
  const int colc = cok ? col : 0;
  const TQ* qp = reinterpret_cast<const TQ*>(a.q) + t * a.q_st + (h / a.rep) * a.q_sh;
  const TQ* kp = reinterpret_cast<const TQ*>(a.k) + t * a.k_st + (h / a.rep) * a.k_sh;
  const TV* vp = reinterpret_cast<const TV*>(a.v) + t * a.v_st + h * a.v_sh + colc;
  float* Sb = a.S + ((int64_t)a.slots[n] * a.H + h) * dk * dv + colc;
  const bool fresh = a.start[n] == 0;
  float S[NR][VEC], kr[NR], qr[NR], v[VEC], gt[VEC];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int d = rg + 16 * i;
    const bool ok = d < dk;
#pragma unroll
    for (int c = 0; c < VEC; ++c) S[i][c] = 0.f;
    if (ok && !fresh) {
      if constexpr (VEC == 4) Vec16<float>::load(Sb + (int64_t)d * dv, S[i]);
      else S[i][0] = Sb[(int64_t)d * dv];
    }
    kr[i] = ok ? ldf(kp + d) : 0.f;
    qr[i] = ok ? ldf(qp + d) : 0.f;
  }
#pragma unroll
  for (int c = 0; c < VEC; ++c) {
    v[c] = ldf(vp + c);
    gt[c] = a.y != nullptr ? ldf(reinterpret_cast<const TV*>(a.hn_g) + t * a.hn_st + h * dv + colc + c) : 0.f;
  }
  float la, beta;
  gate_values(a, h, a.kind != KIND_FIXED ? ldf(reinterpret_cast<const TV*>(a.ga) + t * a.ga_st + h) : 0.f,
              a.kind == KIND_DELTA ? ldf(reinterpret_cast<const TV*>(a.gb) + t * a.gb_st + h) : 0.f, la, beta);
  const float g = expf(la);
  float sum[NS];
#pragma unroll
  for (int c = 0; c < NS; ++c) sum[c] = 0.f;
#pragma unroll
  for (int i = 0; i < NR; ++i) {
#pragma unroll
    for (int c = 0; c < VEC; ++c) {
      sum[c] += S[i][c] * kr[i];
      sum[VEC + c] += S[i][c] * qr[i];
    }
    sum[2 * VEC] += kr[i] * qr[i];
  }
#pragma unroll
  for (int c = 0; c < NS; ++c) {
#pragma unroll
    for (int o = CL; o < 64; o <<= 1) sum[c] += __shfl_xor(sum[c], o, 64);
  }
  if ((tid & 63) < CL) {
#pragma unroll
    for (int c = 0; c < NS; ++c) red[wave][cl][c] = sum[c];
  }
  __syncthreads();
#pragma unroll
  for (int c = 0; c < NS; ++c) {
    sum[c] = 0.f;
#pragma unroll
    for (int w = 0; w < NWV; ++w) sum[c] += red[w][cl][c];
  }
  float u[VEC];
#pragma unroll
  for (int c = 0; c < VEC; ++c) u[c] = beta * (a.kind == KIND_DELTA ? v[c] - g * sum[c] : v[c]);
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int d = rg + 16 * i;
    if (cok && d < dk) {
#pragma unroll
      for (int c = 0; c < VEC; ++c) S[i][c] = g * S[i][c] + kr[i] * u[c];
      if constexpr (VEC == 4) Vec16<float>::store(Sb + (int64_t)d * dv, S[i]);
      else Sb[(int64_t)d * dv] = S[i][0];
    }
  }
  if (rg == 0) {  // (CL lanes of the first wave)
    const float sk = a.skip != nullptr ? a.skip[h] : 0.f;
    float o[VEC];
#pragma unroll
    for (int c = 0; c < VEC; ++c) o[c] = g * sum[VEC + c] + sum[2 * VEC] * u[c] + sk * v[c];
    if (a.y != nullptr) {  // (one column tile: the lanes hold the whole head)
      float q = 0.f;
#pragma unroll
      for (int c = 0; c < VEC; ++c) q += cok ? o[c] * o[c] : 0.f;
#pragma unroll
      for (int x = CL / 2; x > 0; x >>= 1) q += __shfl_xor(q, x, 64);
      if (!cok) return;
      const float f = 1.0f / sqrtf(q / (float)dv + a.hn_eps);
      TV* yp = reinterpret_cast<TV*>(a.y) + (t * a.H + h) * dv + col;
#pragma unroll
      for (int c = 0; c < VEC; ++c) stf(yp + c, o[c] * f * (a.hn_w != nullptr ? a.hn_w[h * dv + col + c] : 1.f) * silu(gt[c]));
      return;
    }
    if (!cok) return;
    float* op = a.out + (t * a.H + h) * dv + col;
    if constexpr (VEC == 4) Vec16<float>::store(op, o);
    else op[0] = o[0];
  }
}

// ------------------------------------------------------------------------------------------ chunks
__device__ __forceinline__ f32x4 mfma4(float x, float y, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(x, y, c, 0, 0, 0); }
__device__ __forceinline__ f32x4 lds4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }

// the sum over the 16 lanes of a row, in each of them (rotations inside the row: no LDS)
__device__ __forceinline__ float sum16(float v) {
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x128, 0xf, 0xf, true));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x124, 0xf, 0xf, true));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x122, 0xf, 0xf, true));
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x121, 0xf, 0xf, true));
  return v;
}

// acc += X Y over one 16-wide block: x4 the lane's four A operands, y its four B operands
__device__ __forceinline__ f32x4 block_product(f32x4 x4, f32x4 y, f32x4 acc) {
#pragma unroll
  for (int j = 0; j < 4; ++j) acc = mfma4(x4[j], y[j], acc);
  return acc;
}

// n rows of one head to LDS as fp32 [CH][dkp + 4]; rows past n and columns past dk become zeros
template <typename T>
__device__ __forceinline__ void stage_rows(float* dst, int stride, const T* src, int64_t st, int n, int dk, int dkp, bool vec) {
  const int nt = blockDim.x;
  if (vec) {
    const int per = dkp / 4;
    for (int e = threadIdx.x; e < CH * per; e += nt) {
      const int r = e / per, c = (e - r * per) * 4;
      float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
      if (r < n && c < dk) {
        const T* p = src + (int64_t)r * st + c;
        if constexpr (sizeof(T) == 4) {
          x = *reinterpret_cast<const float4*>(p);
        } else {
          const uint2 w = *reinterpret_cast<const uint2*>(p);
          x = make_float4(__uint_as_float(w.x << 16), __uint_as_float(w.x & 0xffff0000u), __uint_as_float(w.y << 16),
                          __uint_as_float(w.y & 0xffff0000u));
        }
      }
      *reinterpret_cast<float4*>(dst + r * stride + c) = x;
    }
  } else {
    for (int e = threadIdx.x; e < CH * dkp; e += nt) {
      const int r = e / dkp, c = e - r * dkp;
      dst[r * stride + c] = (r < n && c < dk) ? ldf(src + (int64_t)r * st + c) : 0.f;
    }
  }
}

struct ChunkGates {  // LDS arrays of CH floats each
  float* hi;    // L_t, the running sum of log g, as a pair of floats (differences of large sums stay exact)
  float* lo;
  float* beta;
  float* grow;  // e^(L_t)
  float* rest;  // e^(L_n - L_t)
};

// The first wave fills the arrays (tokens past n: no decay, no write).  Raw gate values are requested ahead of the rows'
// staging and used after it.
struct RawGates {
  float x, y;
};
template <typename TV>
__device__ __forceinline__ RawGates load_gates(const MemArgs& a, int h, int t0, int n) {
  RawGates r = {0.f, 0.f};
  if ((int)threadIdx.x < n && a.kind != KIND_FIXED) {
    const int64_t t = t0 + (int)threadIdx.x;
    r.x = ldf(reinterpret_cast<const TV*>(a.ga) + t * a.ga_st + h);
    if (a.kind == KIND_DELTA) r.y = ldf(reinterpret_cast<const TV*>(a.gb) + t * a.gb_st + h);
  }
  return r;
}

__device__ __forceinline__ void chunk_gates(const MemArgs& a, const ChunkGates& cg, RawGates raw, int h, int n) {
  if (threadIdx.x < CH) {
    const int t = threadIdx.x;
    float la = 0.f, beta = 0.f;
    if (t < n) gate_values(a, h, raw.x, raw.y, la, beta);
    double L = (double)la;
#pragma unroll
    for (int o = 1; o < CH; o <<= 1) {
      const double up = __shfl_up(L, o, 64);
      if (t >= o) L += up;
    }
    const double end = __shfl(L, CH - 1, 64);
    cg.hi[t] = (float)L;
    cg.lo[t] = (float)(L - (double)(float)L);
    cg.beta[t] = beta;
    cg.grow[t] = expf((float)L);
    cg.rest[t] = expf((float)(end - L));
  }
}

// inverses of the four 16 x 16 diagonal blocks of I + A (A strictly lower): one wave, lane = (block, column)
__device__ __forceinline__ void invert_diagonals(const float* A, float* Tb) {
  if (threadIdx.x >= 64) return;
  const int b = threadIdx.x >> 4, j = threadIdx.x & 15;
  const float* Ab = A + (16 * b) * AS + 16 * b;
  float x[16];
#pragma unroll
  for (int i = 0; i < 16; ++i) {
    float s = i == j ? 1.f : 0.f;
#pragma unroll
    for (int c4 = 0; c4 < i; c4 += 4) {
      const f32x4 a4 = lds4(Ab + i * AS + c4);
#pragma unroll
      for (int c = 0; c < 4; ++c)
        if (c4 + c < i) s -= a4[c] * x[c4 + c];
    }
    x[i] = s;
    Tb[(b * 16 + i) * TBS + j] = s;
  }
}

// y <- (I + A)^-1 y, the 64 rows of y as four blocks in registers
__device__ __forceinline__ void solve(const float* A, const float* Tb, f32x4 (&y)[4], int lane) {
  const int r = lane & 15, g4 = (lane >> 4) * 4;
#pragma unroll
  for (int b = 0; b < 4; ++b) {
    f32x4 acc = y[b];
#pragma unroll
    for (int c = 0; c < b; ++c) acc = block_product(-lds4(A + (16 * b + r) * AS + 16 * c + g4), y[c], acc);
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
    y[b] = block_product(lds4(Tb + (b * 16 + r) * TBS + g4), acc, zero);
  }
}

__device__ __forceinline__ void lower_tile(int i, int& ti, int& tj) {  // the ten 16 x 16 tiles on and below the diagonal
  ti = i < 1 ? 0 : (i < 3 ? 1 : (i < 6 ? 2 : 3));
  tj = i - ti * (ti + 1) / 2;
}

// one score tile: rows 16 ti .. of X against rows 16 tj .. of Y (both [CH][ks] in LDS)
template <int NKK>
__device__ __forceinline__ f32x4 score_tile(const float* X, const float* Y, int ks, int nkk, int ti, int tj, int lane) {
  const float* xr = X + (16 * ti + (lane & 15)) * ks + (lane >> 4) * 4;
  const float* yr = Y + (16 * tj + (lane & 15)) * ks + (lane >> 4) * 4;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  if constexpr (NKK > 0) {
#pragma unroll
    for (int kk = 0; kk < NKK; ++kk) acc = block_product(lds4(xr + 16 * kk), lds4(yr + 16 * kk), acc);
  } else {
    for (int kk = 0; kk < nkk; ++kk) acc = block_product(lds4(xr + 16 * kk), lds4(yr + 16 * kk), acc);
  }
  return acc;
}

// a score tile times e^(L_t - L_s) (rows t, columns s; zero above the diagonal, or from it on when ``strict``) times a factor
// per row or per column, to LDS
__device__ __forceinline__ void put_tile(float* A, f32x4 acc, const ChunkGates& cg, int ti, int tj, int lane, bool strict,
                                         const float* row_f, const float* col_f) {
  const int s = 16 * tj + (lane & 15);
  const float shi = cg.hi[s], slo = cg.lo[s], cf = col_f != nullptr ? col_f[s] : 1.f;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int t = 16 * ti + (lane >> 4) * 4 + r;
    const bool on = strict ? s < t : s <= t;
    const float f = on ? expf((cg.hi[t] - shi) + (cg.lo[t] - slo)) * cf * (row_f != nullptr ? row_f[t] : 1.f) : 0.f;
    A[t * AS + s] = on ? acc[r] * f : 0.f;
  }
}

constexpr int MAX_TILES = 3;  // score tiles per wave (ten tiles over at least four waves)

// NKK > 0: the keys fill up to 16 * NKK channels, known at compile time (0: any width).
// LDS: K [CH][ks] | (delta) A [CH][AS] | inverted blocks | gate arrays.  A wave takes up to two column tiles, one after the other:
// the value columns first, then (delta) the columns of the transition matrix.
template <typename TQ, typename TV, bool DELTA, int NKK>
__global__ __launch_bounds__(512, 4) void memory_chunk_local_kernel(MemArgs a) {
  extern __shared__ __attribute__((aligned(16))) float smem[];
  const int p = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int lane = tid & 63, wave = tid >> 6, nw = blockDim.x >> 6;
  const int t0 = a.cu[p], n = a.cu[p + 1] - t0;
  const int dk = a.dk, dv = a.dv, dkt = (dk + 15) & ~15, nkk = NKK > 0 ? NKK : dkt / 16, dkp = 16 * nkk, ks = dkp + 4;
  float* Ks = smem;
  float* A = Ks + CH * ks;
  float* Tb = A + (DELTA ? CH * AS : 0);
  float* gl = Tb + (DELTA ? 4 * 16 * TBS : 0);
  const ChunkGates cg{gl, gl + CH, gl + 2 * CH, gl + 3 * CH, gl + 4 * CH};
  const int vtiles = (dv + 15) / 16, tiles = vtiles + (DELTA ? dkt / 16 : 0);
  const int g4 = (lane >> 4) * 4;
  const TQ* kp = reinterpret_cast<const TQ*>(a.k) + t0 * a.k_st + (h / a.rep) * a.k_sh;
  const TV* vp = reinterpret_cast<const TV*>(a.v) + t0 * a.v_st + h * a.v_sh;
  const RawGates raw = load_gates<TV>(a, h, t0, n);
  f32x4 y[4];
  auto load_values = [&](int ct) {
    const int col = ct * 16 + (lane & 15);
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * m + g4 + r;
        y[m][r] = (ct < vtiles && col < dv && t < n) ? ldf(vp + t * a.v_st + col) : 0.f;
      }
  };
  int ct = (int)blockIdx.z * 2 * nw + wave;
  load_values(ct);
  stage_rows(Ks, ks, kp, a.k_st, n, dk, dkp, a.vec != 0);
  chunk_gates(a, cg, raw, h, n);
  __syncthreads();
  if constexpr (DELTA) {
    for (int i = wave; i < 10; i += nw) {
      int ti, tj;
      lower_tile(i, ti, tj);
      put_tile(A, score_tile<NKK>(Ks, Ks, ks, nkk, ti, tj, lane), cg, ti, tj, lane, true, cg.beta, nullptr);
    }
    __syncthreads();
    invert_diagonals(A, Tb);
    __syncthreads();
  }
  if (blockIdx.z == 0 && tid == 0) a.dec[(int64_t)p * a.H + h] = cg.grow[CH - 1];
#pragma unroll 1
  for (int half = 0; half < 2; ++half, ct += nw) {
    if (ct >= tiles) return;
    asm volatile("" ::: "memory");  // the second tile reads LDS again: kept in registers over the loop, it would spill
    if (half > 0) load_values(ct);
    const bool carry = DELTA && ct >= vtiles;  // columns of the transition matrix
    const int col = (carry ? ct - vtiles : ct) * 16 + (lane & 15);
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * m + g4 + r;
        if (carry) y[m][r] = -cg.grow[t] * Ks[t * ks + col];
        y[m][r] *= cg.beta[t];
      }
    if constexpr (DELTA) solve(A, Tb, y, lane);
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) y[m][r] *= cg.rest[16 * m + g4 + r];
    const float all = cg.grow[CH - 1];
    for (int dt = 0; dt < dkt / 16; ++dt) {
      f32x4 acc;
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[r] = (carry && 16 * dt + g4 + r == col) ? all : 0.f;
#pragma unroll
      for (int m = 0; m < 4; ++m)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc = mfma4(Ks[(16 * m + g4 + j) * ks + 16 * dt + (lane & 15)], y[m][j], acc);
      if (carry) {
        float* o = a.trans + (((int64_t)p * a.H + h) * dkt + 16 * dt + g4) * dkt + col;
#pragma unroll
        for (int r = 0; r < 4; ++r) o[r * dkt] = acc[r];
      } else if (col < dv) {
        float* o = a.loc + (((int64_t)p * a.H + h) * dk + 16 * dt + g4) * dv + col;
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (16 * dt + g4 + r < dk) o[(int64_t)r * dv] = acc[r];
      }
    }
  }
}

// LDS: K [CH][ks] | Q [CH][ks], later the read-out scores [CH][AS] | (delta) A [CH][AS] | inverted blocks | gate arrays
template <typename TQ, typename TV, bool DELTA, int NKK>
__global__ __launch_bounds__(512, NKK == 8 && DELTA ? 2 : 4) void memory_chunks_kernel(MemArgs a) {
  extern __shared__ __attribute__((aligned(16))) float smem[];
  const int p = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int lane = tid & 63, wave = tid >> 6, nw = blockDim.x >> 6;
  const int t0 = a.cu[p], n = a.cu[p + 1] - t0;
  if (n <= 0) return;
  const int dk = a.dk, dv = a.dv, nkk = NKK > 0 ? NKK : (dk + 15) / 16, dkp = 16 * nkk, ks = dkp + 4;
  float* Ks = smem;
  float* Qs = Ks + CH * ks;
  float* A = Qs + CH * (ks > AS ? ks : AS);
  float* Tb = A + (DELTA ? CH * AS : 0);
  float* gl = Tb + (DELTA ? 4 * 16 * TBS : 0);
  const ChunkGates cg{gl, gl + CH, gl + 2 * CH, gl + 3 * CH, gl + 4 * CH};
  const bool whole = a.init == nullptr;
  const int ct = blockIdx.z * nw + wave;
  const int col = ct * 16 + (lane & 15), g4 = (lane >> 4) * 4;
  const bool live = ct * 16 < dv, cok = col < dv;
  const int colc = cok ? col : dv - 1;
  const TQ* qp = reinterpret_cast<const TQ*>(a.q) + t0 * a.q_st + (h / a.rep) * a.q_sh;
  const TQ* kp = reinterpret_cast<const TQ*>(a.k) + t0 * a.k_st + (h / a.rep) * a.k_sh;
  const TV* vp = reinterpret_cast<const TV*>(a.v) + t0 * a.v_st + h * a.v_sh;
  const bool fresh = whole && a.start[p] == 0;
  const float* S0 = (whole ? a.S + ((int64_t)a.slots[p] * a.H + h) * dk * dv : a.init + ((int64_t)p * a.H + h) * dk * dv) + colc;
  const RawGates raw = load_gates<TV>(a, h, t0, n);
  f32x4 y[4];
#pragma unroll
  for (int m = 0; m < 4; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 16 * m + g4 + r;
      y[m][r] = (cok && t < n) ? ldf(vp + t * a.v_st + col) : 0.f;
    }
  // this wave's columns of the memory, requested ahead of everything that does not need them
  f32x4 s0[NKK > 0 ? NKK : 1];
  auto load_memory = [&](int kk) {
    f32x4 s;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int d = 16 * kk + g4 + j;
      s[j] = (live && !fresh && d < dk) ? S0[(int64_t)d * dv] : 0.f;
    }
    return s;
  };
  if constexpr (NKK > 0) {
#pragma unroll
    for (int kk = 0; kk < NKK; ++kk) s0[kk] = load_memory(kk);
  }
  stage_rows(Ks, ks, kp, a.k_st, n, dk, dkp, a.vec != 0);
  stage_rows(Qs, ks, qp, a.q_st, n, dk, dkp, a.vec != 0);
  const bool fused = a.y != nullptr;  // (one column tile per wave covers the head)
  f32x4 gt[4];
  auto load_gate = [&]() {
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * m + g4 + r;
        gt[m][r] = (fused && cok && t < n) ? ldf(reinterpret_cast<const TV*>(a.hn_g) + (t0 + t) * a.hn_st + h * dv + col) : 0.f;
      }
  };
  if constexpr (NKK != 8) load_gate();  // (the widest form has no registers to spare for it)
  chunk_gates(a, cg, raw, h, n);
  __syncthreads();
  // scores of this wave's tiles (kept in registers: they overwrite Q), and this wave's columns of Q S_0 and K S_0
  f32x4 sq[MAX_TILES];
#pragma unroll
  for (int i = 0; i < MAX_TILES; ++i) {
    const int tile = wave + i * nw;
    if (tile < 10) {
      int ti, tj;
      lower_tile(tile, ti, tj);
      sq[i] = score_tile<NKK>(Qs, Ks, ks, nkk, ti, tj, lane);
      if constexpr (DELTA) put_tile(A, score_tile<NKK>(Ks, Ks, ks, nkk, ti, tj, lane), cg, ti, tj, lane, true, cg.beta, nullptr);
    }
  }
  f32x4 oq[4], ok[4];
#pragma unroll
  for (int m = 0; m < 4; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) oq[m][r] = 0.f, ok[m][r] = 0.f;
  if (live && !fresh) {
    const int row = (lane & 15) * ks + g4;
    auto read_out = [&](int kk, f32x4 s) {
#pragma unroll
      for (int m = 0; m < 4; ++m) {
        oq[m] = block_product(lds4(Qs + 16 * m * ks + row + 16 * kk), s, oq[m]);
        if constexpr (DELTA) ok[m] = block_product(lds4(Ks + 16 * m * ks + row + 16 * kk), s, ok[m]);
      }
    };
    if constexpr (NKK > 0) {
#pragma unroll
      for (int kk = 0; kk < NKK; ++kk) read_out(kk, s0[kk]);
    } else {
      for (int kk = 0; kk < nkk; ++kk) read_out(kk, load_memory(kk));
    }
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < MAX_TILES; ++i) {
    const int tile = wave + i * nw;
    if (tile < 10) {
      int ti, tj;
      lower_tile(tile, ti, tj);
      put_tile(Qs, sq[i], cg, ti, tj, lane, false, nullptr, DELTA ? nullptr : cg.beta);
    }
  }
  if constexpr (DELTA) invert_diagonals(A, Tb);
  __syncthreads();
  if (!live && !fused) return;
  const float sk = a.skip != nullptr ? a.skip[h] : 0.f;
  if constexpr (DELTA) {
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * m + g4 + r;
        y[m][r] = cg.beta[t] * (y[m][r] - cg.grow[t] * ok[m][r]);
      }
    solve(A, Tb, y, lane);
  }
#pragma unroll
  for (int m = 0; m < 4; ++m) {
    f32x4 o;
#pragma unroll
    for (int r = 0; r < 4; ++r) o[r] = cg.grow[16 * m + g4 + r] * oq[m][r] + (DELTA ? 0.f : sk * y[m][r]);
#pragma unroll
    for (int c = 0; c <= m; ++c) o = block_product(lds4(Qs + (16 * m + (lane & 15)) * AS + 16 * c + g4), y[c], o);
    oq[m] = o;
  }
  if (fused) {
    float* rstd = gl + 5 * CH;
    float* part = rstd + CH;  // [waves][CH] sums of squares of a wave's columns
    if constexpr (NKK == 8) load_gate();
#pragma unroll
    for (int m = 0; m < 4; ++m) {
      f32x4 q;
#pragma unroll
      for (int r = 0; r < 4; ++r) q[r] = sum16(cok ? oq[m][r] * oq[m][r] : 0.f);
      if ((lane & 15) == 0) *reinterpret_cast<f32x4*>(part + wave * CH + 16 * m + g4) = q;
    }
    __syncthreads();
    if (tid < CH) {
      float q = 0.f;
      for (int x = 0; x < nw; ++x) q += part[x * CH + tid];
      rstd[tid] = 1.0f / sqrtf(q / (float)dv + a.hn_eps);
    }
    __syncthreads();
    const float w = (a.hn_w != nullptr && cok) ? a.hn_w[h * dv + col] : 1.f;
    TV* yp = reinterpret_cast<TV*>(a.y) + ((int64_t)t0 * a.H + h) * dv + col;
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * m + g4 + r;
        if (cok && t < n) stf(yp + (int64_t)t * a.H * dv, oq[m][r] * rstd[t] * w * silu(gt[m][r]));
      }
    if (!live) return;
  } else {
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * m + g4 + r;
        if (cok && t < n) a.out[((int64_t)(t0 + t) * a.H + h) * dv + col] = oq[m][r];
      }
  }
  if (!whole) return;
#pragma unroll
  for (int m = 0; m < 4; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 16 * m + g4 + r;
      y[m][r] *= cg.rest[t] * (DELTA ? 1.f : cg.beta[t]);
    }
  float* Sw = a.S + ((int64_t)a.slots[p] * a.H + h) * dk * dv + colc;  // a lane rewrites the entries that it alone has read
  const float all = cg.grow[CH - 1];
  for (int dt = 0; dt < nkk; ++dt) {
    f32x4 acc;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * dt + g4 + r;
      acc[r] = (!fresh && d < dk) ? all * Sw[(int64_t)d * dv] : 0.f;
    }
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
      for (int j = 0; j < 4; ++j) acc = mfma4(Ks[(16 * m + g4 + j) * ks + 16 * dt + (lane & 15)], y[m][j], acc);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * dt + g4 + r;
      if (cok && d < dk) Sw[(int64_t)d * dv] = acc[r];
    }
  }
}

// ------------------------------------------------------------------------------------------ combine
// Sequence s has chunks [base[s], base[s+1]).  One thread per memory entry; contributions are fetched a batch ahead.
constexpr int CB = 8;
__global__ __launch_bounds__(256) void memory_combine_kernel(float* __restrict__ S, const int* __restrict__ slots, const int* __restrict__ start,
                                                             const int* __restrict__ base, const float* __restrict__ loc,
                                                             const float* __restrict__ dec, float* __restrict__ init, int H, int64_t per) {
  const int s = blockIdx.x, h = blockIdx.y;
  const int64_t e = (int64_t)blockIdx.z * 256 + threadIdx.x;
  const int lo = base[s], hi = base[s + 1];
  if (e >= per || lo == hi) return;
  float* real = S + ((int64_t)slots[s] * H + h) * per + e;
  float val = start[s] == 0 ? 0.f : *real;
  float l[CB], d[CB], nl[CB], nd[CB];
  auto fetch = [&](int p0) {
#pragma unroll
    for (int i = 0; i < CB; ++i) {
      const int64_t p = min(p0 + i, hi - 1);
      nl[i] = loc[(p * H + h) * per + e];
      nd[i] = dec[p * H + h];
    }
  };
  fetch(lo);
  for (int p0 = lo; p0 < hi; p0 += CB) {
#pragma unroll
    for (int i = 0; i < CB; ++i) l[i] = nl[i], d[i] = nd[i];
    if (p0 + CB < hi) fetch(p0 + CB);
#pragma unroll
    for (int i = 0; i < CB; ++i) {
      if (p0 + i < hi) {
        init[((int64_t)(p0 + i) * H + h) * per + e] = val;
        val = d[i] * val + l[i];
      }
    }
  }
  *real = val;
}

// The delta kind: S' = P S + loc.  A workgroup owns 16 value columns of one head, wave w the rows 16 w .. of the memory.  Every
// step's P rows and contribution are requested PD chunks ahead; the memory goes from wave to wave through LDS, column by
// column.
template <int KK, int PD>
__global__ __launch_bounds__(64 * KK) void memory_combine_delta_kernel(float* __restrict__ S, const int* __restrict__ slots,
                                                                       const int* __restrict__ start, const int* __restrict__ base,
                                                                       const float* __restrict__ loc, const float* __restrict__ trans,
                                                                       float* __restrict__ init, int H, int dk, int dv) {
  constexpr int DKP = 16 * KK, SS = DKP + 4;
  __shared__ __attribute__((aligned(16))) float mem[2][16][SS];
  const int s = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int lo = base[s], hi = base[s + 1];
  if (lo == hi) return;
  const int c16 = lane & 15, g4 = (lane >> 4) * 4, d0 = 16 * wave + g4;
  const int col = blockIdx.z * 16 + c16;
  const bool cok = col < dv;
  const int colc = cok ? col : dv - 1;
  float* real = S + ((int64_t)slots[s] * H + h) * dk * dv + colc;
  const bool fresh = start[s] == 0;
  f32x4 val;
#pragma unroll
  for (int r = 0; r < 4; ++r) val[r] = (!fresh && d0 + r < dk) ? real[(int64_t)(d0 + r) * dv] : 0.f;
  f32x4 pf[PD][KK], lf[PD];
  auto fetch = [&](int b, int p) {
    const int64_t ph = (int64_t)min(p, hi - 1) * H + h;
    const float* tp = trans + (ph * DKP + 16 * wave + c16) * DKP + g4;
#pragma unroll
    for (int kk = 0; kk < KK; ++kk) pf[b][kk] = *reinterpret_cast<const f32x4*>(tp + 16 * kk);
    const float* lp = loc + ph * dk * dv + colc;
#pragma unroll
    for (int r = 0; r < 4; ++r) lf[b][r] = d0 + r < dk ? lp[(int64_t)(d0 + r) * dv] : 0.f;
  };
#pragma unroll
  for (int b = 0; b < PD; ++b) fetch(b, lo + b);
  int buf = 0;
  for (int p0 = lo; p0 < hi; p0 += PD) {
#pragma unroll
    for (int b = 0; b < PD; ++b) {
      const int p = p0 + b;
      if (p < hi) {
        *reinterpret_cast<f32x4*>(&mem[buf][c16][d0]) = val;
        float* ip = init + ((int64_t)p * H + h) * dk * dv + colc;
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (cok && d0 + r < dk) ip[(int64_t)(d0 + r) * dv] = val[r];
        __syncthreads();  // (two buffers: the reads of the one before last are behind this barrier)
        f32x4 acc = lf[b];
#pragma unroll
        for (int kk = 0; kk < KK; ++kk) acc = block_product(pf[b][kk], lds4(&mem[buf][c16][16 * kk + g4]), acc);
        val = acc;
        if (p + PD < hi) fetch(b, p + PD);
        buf ^= 1;
      }
    }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r)
    if (cok && d0 + r < dk) real[(int64_t)(d0 + r) * dv] = val[r];
}

// ------------------------------------------------------------------------------------------ host
bool f32vec(const at::Tensor& t, int64_t n) { return t.is_cuda() && t.is_contiguous() && t.scalar_type() == at::kFloat && t.numel() == n; }
bool i32(const at::Tensor& t) { return t.is_cuda() && t.is_contiguous() && t.scalar_type() == at::kInt && t.dim() == 1; }

using OptT = c10::optional<at::Tensor>;

MemArgs mem_args(const at::Tensor& q, const at::Tensor& k, const at::Tensor& v, int64_t kind, const OptT& ga, const OptT& gb, const OptT& a_log,
                 const OptT& dt_bias, const OptT& log_decay, const OptT& skip) {
  for (const at::Tensor* t : {&q, &k, &v})
    HYB_CHECK(t->is_cuda() && t->dim() == 3 && (t->size(2) == 1 || t->stride(2) == 1), "q, k, v: [T, heads, d] with unit last stride");
  const int64_t T = v.size(0), H = v.size(1), KH = q.size(1), dk = q.size(2);
  HYB_CHECK(q.size(0) == T && k.size(0) == T && k.size(1) == KH && k.size(2) == dk && q.scalar_type() == k.scalar_type(), "q and k: one shape and dtype");
  HYB_CHECK(KH >= 1 && H % KH == 0 && dk >= 1 && dk <= 256 && v.size(2) >= 1 && H <= 65535, "key heads must divide the heads; key size 1 .. 256");
  HYB_CHECK(q.scalar_type() == at::kFloat || q.scalar_type() == v.scalar_type(), "q, k: fp32 or v's dtype");
  HYB_CHECK(kind >= 0 && kind <= 2, "kind: 0 fixed, 1 state-space, 2 delta");
  MemArgs a = {};
  a.q = q.data_ptr(), a.k = k.data_ptr(), a.v = v.data_ptr();
  a.q_st = q.stride(0), a.q_sh = q.stride(1), a.k_st = k.stride(0), a.k_sh = k.stride(1), a.v_st = v.stride(0), a.v_sh = v.stride(1);
  auto column = [&](const OptT& t, const char* name) {
    HYB_CHECK(t.has_value() && t->is_cuda() && t->dim() == 2 && t->size(0) == T && t->size(1) == H && (H == 1 || t->stride(1) == 1) && t->scalar_type() == v.scalar_type(),
              name, ": [T, H] of v's dtype");
    return t->data_ptr();
  };
  auto perhead = [&](const OptT& t, const char* name) {
    HYB_CHECK(t.has_value() && f32vec(*t, H), name, ": fp32 [H]");
    return t->data_ptr<float>();
  };
  if (kind == KIND_FIXED) {
    a.log_decay = perhead(log_decay, "log_decay");
  } else {
    a.ga = column(ga, "ga"), a.ga_st = ga->stride(0);
    a.a_log = perhead(a_log, "a_log"), a.dt_bias = perhead(dt_bias, "dt_bias");
    if (kind == KIND_DELTA) a.gb = column(gb, "gb"), a.gb_st = gb->stride(0);
  }
  if (skip.has_value()) {
    HYB_CHECK(kind != KIND_DELTA, "the delta kind takes no skip");
    a.skip = perhead(skip, "skip");
  }
  a.kind = (int)kind, a.H = (int)H, a.rep = (int)(H / KH), a.dk = (int)dk, a.dv = (int)v.size(2);
  const size_t quad = 4 * q.element_size();
  auto rows4 = [&](const at::Tensor& t) {
    return reinterpret_cast<uintptr_t>(t.data_ptr()) % quad == 0 && t.stride(0) % 4 == 0 && t.stride(1) % 4 == 0;
  };
  a.vec = dk % 4 == 0 && rows4(q) && rows4(k);
  return a;
}

void set_pool(MemArgs& a, const at::Tensor& S) {
  HYB_CHECK(S.is_cuda() && S.is_contiguous() && S.scalar_type() == at::kFloat && S.dim() == 4 && S.size(1) == a.H && S.size(2) == a.dk && S.size(3) == a.dv,
            "state: contiguous fp32 [slots, H, dk, dv]");
  a.S = S.data_ptr<float>();
}

// the outputs: fp32 [T, H, dv], or (a gate given) the head norm's result [T, H * dv] in v's dtype
void set_out(MemArgs& a, const at::Tensor& out, const at::Tensor& v, const OptT& hn_w, const OptT& hn_g, double eps) {
  const int64_t T = v.size(0), n = a.H * (int64_t)a.dv;
  if (!hn_g.has_value()) {
    HYB_CHECK(f32vec(out, T * n) && !hn_w.has_value(), "out: fp32 [T, H, dv]");
    a.out = out.data_ptr<float>();
    return;
  }
  HYB_CHECK(a.dv % 4 == 0 && a.dv <= 128, "the fused head norm takes value sizes up to 128 in quads");
  HYB_CHECK(out.is_cuda() && out.is_contiguous() && out.scalar_type() == v.scalar_type() && out.numel() == T * n, "out: [T, H * dv] of v's dtype");
  check_rows(*hn_g, "gate");
  HYB_CHECK(hn_g->size(0) == T && hn_g->size(1) == n && hn_g->scalar_type() == v.scalar_type(), "gate: [T, H * dv] of v's dtype");
  HYB_CHECK(!hn_w.has_value() || f32vec(*hn_w, n), "norm weight: fp32 [H * dv]");
  a.y = out.data_ptr(), a.hn_g = hn_g->data_ptr(), a.hn_st = hn_g->stride(0), a.hn_eps = (float)eps;
  a.hn_w = hn_w.has_value() ? hn_w->data_ptr<float>() : nullptr;
}

// q / k dtype x v dtype: (v, v) or (fp32, v)
template <typename F>
void dispatch_qv(const at::Tensor& q, const at::Tensor& v, F&& f) {
  dispatch_act(v, [&](auto* tv) {
    if (q.scalar_type() == at::kFloat) f((float*)nullptr, tv);
    else f(tv, tv);
  });
}

int waves_for(int dv) { return dv > 64 ? 8 : 4; }

// channels that a chunk's keys take in LDS: the compile-time widths 32, 64 and 128, else filled up to 16
int staged_width(int dk) { return dk <= 32 ? 32 : (dk <= 64 ? 64 : (dk <= 128 && dk > 96 ? 128 : (dk + 15) / 16 * 16)); }
template <typename F>
void by_width(int dk, F&& f) {
  if (dk <= 32) f(std::integral_constant<int, 2>());
  else if (dk <= 64) f(std::integral_constant<int, 4>());
  else if (dk <= 128 && dk > 96) f(std::integral_constant<int, 8>());
  else f(std::integral_constant<int, 0>());
}

template <typename K>
void launch_lds(K kern, dim3 grid, int threads, size_t lds, const MemArgs& a) {
  HYB_CHECK(lds <= 160 * 1024, "keys too wide for LDS");
  if (lds > 64 * 1024)
    HYB_CHECK(hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) == hipSuccess, "LDS size");
  kern<<<grid, threads, lds, cur_stream()>>>(a);
}
}  // namespace

void memory_decode(const at::Tensor& q, const at::Tensor& k, const at::Tensor& v, int64_t kind, const OptT& ga, const OptT& gb, const OptT& a_log,
                   const OptT& dt_bias, const OptT& log_decay, const OptT& skip, at::Tensor S, const at::Tensor& slots, const at::Tensor& start,
                   at::Tensor out, const OptT& hn_w, const OptT& hn_g, double hn_eps, int64_t row0) {
  MemArgs a = mem_args(q, k, v, kind, ga, gb, a_log, dt_bias, log_decay, skip);
  set_pool(a, S);
  set_out(a, out, v, hn_w, hn_g, hn_eps);
  HYB_CHECK(i32(slots) && i32(start) && slots.numel() == start.numel() && row0 >= 0 && row0 + slots.numel() == v.size(0), "slots [n], start [n]: the last n rows");
  const int64_t n = slots.numel();
  if (n == 0) return;
  a.slots = slots.data_ptr<int>(), a.start = start.data_ptr<int>(), a.row0 = (int)row0;
  c10::DeviceGuard guard(v.device());
  const bool v4 = a.dv % 4 == 0, wide = v4 && a.dv > 64 && a.dv <= 128;  // (a head of up to 128 values is one tile)
  const int tile = wide ? 128 : (v4 ? 64 : 16);
  const dim3 grid((unsigned)n, (unsigned)a.H, (unsigned)((a.dv + tile - 1) / tile));
  dispatch_qv(q, v, [&](auto* tq, auto* tv) {
    using TQ = std::remove_pointer_t<decltype(tq)>;
    using TV = std::remove_pointer_t<decltype(tv)>;
    auto go = [&](auto kern, int cl) { kern<<<grid, 16 * cl, 0, cur_stream()>>>(a); };
    auto rows = [&](auto vec, auto lanes) {
      constexpr int V = decltype(vec)::value, CL = decltype(lanes)::value;
      if (a.dk <= 16) go(memory_decode_kernel<TQ, TV, V, 1, CL>, CL);
      else if (a.dk <= 32) go(memory_decode_kernel<TQ, TV, V, 2, CL>, CL);
      else if (a.dk <= 64) go(memory_decode_kernel<TQ, TV, V, 4, CL>, CL);
      else if (a.dk <= 128) go(memory_decode_kernel<TQ, TV, V, 8, CL>, CL);
      else go(memory_decode_kernel<TQ, TV, V, 16, CL>, CL);
    };
    if (wide) rows(std::integral_constant<int, 4>(), std::integral_constant<int, 32>());
    else if (v4) rows(std::integral_constant<int, 4>(), std::integral_constant<int, 16>());
    else rows(std::integral_constant<int, 1>(), std::integral_constant<int, 16>());
  });
}

// init == None: the rows [cu[s], cu[s+1]) are whole portions of at most 64 tokens, from and to the pool S; otherwise they are the chunks
// of longer ones and start from init
void memory_chunks(const at::Tensor& q, const at::Tensor& k, const at::Tensor& v, int64_t kind, const OptT& ga, const OptT& gb, const OptT& a_log,
                   const OptT& dt_bias, const OptT& log_decay, const OptT& skip, at::Tensor S, const OptT& slots, const at::Tensor& cu,
                   const OptT& start, const OptT& init, at::Tensor out, const OptT& hn_w, const OptT& hn_g, double hn_eps, int64_t rows) {
  MemArgs a = mem_args(q, k, v, kind, ga, gb, a_log, dt_bias, log_decay, skip);
  set_pool(a, S);
  set_out(a, out, v, hn_w, hn_g, hn_eps);
  HYB_CHECK(i32(cu) && cu.numel() >= 1 && rows >= 0 && rows <= v.size(0), "cu: int32 [n + 1]");
  const int64_t n = cu.numel() - 1;
  if (n == 0 || rows == 0) return;
  a.cu = cu.data_ptr<int>();
  if (init.has_value()) {
    HYB_CHECK(f32vec(*init, n * a.H * a.dk * a.dv), "chunk-start memories: fp32 [chunks, H, dk, dv]");
    a.init = init->data_ptr<float>();
  } else {
    HYB_CHECK(slots.has_value() && start.has_value() && i32(*slots) && i32(*start) && slots->numel() == n && start->numel() == n, "slots [n], start [n]: int32");
    a.slots = slots->data_ptr<int>(), a.start = start->data_ptr<int>();
  }
  c10::DeviceGuard guard(v.device());
  const int nw = waves_for(a.dv), ks = staged_width(a.dk) + 4;
  const bool delta = kind == KIND_DELTA;
  const size_t lds = sizeof(float) * (size_t)(CH * ks + CH * std::max(ks, AS) + (delta ? CH * AS + 4 * 16 * TBS : 0) + 5 * CH + (a.y != nullptr ? (nw + 1) * CH : 0));
  const dim3 grid((unsigned)n, (unsigned)a.H, (unsigned)(((a.dv + 15) / 16 + nw - 1) / nw));
  dispatch_qv(q, v, [&](auto* tq, auto* tv) {
    using TQ = std::remove_pointer_t<decltype(tq)>;
    using TV = std::remove_pointer_t<decltype(tv)>;
    auto go = [&](auto nkk) {
      constexpr int N = decltype(nkk)::value;
      if (delta) launch_lds(memory_chunks_kernel<TQ, TV, true, N>, grid, 64 * nw, lds, a);
      else launch_lds(memory_chunks_kernel<TQ, TV, false, N>, grid, 64 * nw, lds, a);
    };
    by_width(a.dk, go);
  });
}

void memory_chunk_local(const at::Tensor& q, const at::Tensor& k, const at::Tensor& v, int64_t kind, const OptT& ga, const OptT& gb, const OptT& a_log,
                        const OptT& dt_bias, const OptT& log_decay, const OptT& skip, const at::Tensor& cu, at::Tensor loc, at::Tensor dec,
                        const OptT& trans) {
  MemArgs a = mem_args(q, k, v, kind, ga, gb, a_log, dt_bias, log_decay, skip);
  HYB_CHECK(i32(cu) && cu.numel() >= 1, "cu: int32 [chunks + 1]");
  const int64_t n = cu.numel() - 1;
  if (n == 0) return;
  const int nw = waves_for(a.dv), dkp = (a.dk + 15) / 16 * 16, ks = staged_width(a.dk) + 4;
  const bool delta = kind == KIND_DELTA;
  HYB_CHECK(f32vec(loc, n * a.H * a.dk * a.dv) && f32vec(dec, n * a.H), "loc: fp32 [chunks, H, dk, dv], dec: fp32 [chunks, H]");
  HYB_CHECK(trans.has_value() == delta && (!delta || f32vec(*trans, n * a.H * dkp * dkp)), "trans: fp32 [chunks, H, dkp, dkp] (delta kind), dkp = dk filled up to 16");
  a.cu = cu.data_ptr<int>(), a.loc = loc.data_ptr<float>(), a.dec = dec.data_ptr<float>();
  a.trans = delta ? trans->data_ptr<float>() : nullptr;
  c10::DeviceGuard guard(v.device());
  const size_t lds = sizeof(float) * (size_t)(CH * ks + (delta ? CH * AS + 4 * 16 * TBS : 0) + 5 * CH);
  const int tiles = (a.dv + 15) / 16 + (delta ? dkp / 16 : 0);
  const dim3 grid((unsigned)n, (unsigned)a.H, (unsigned)((tiles + 2 * nw - 1) / (2 * nw)));
  dispatch_qv(q, v, [&](auto* tq, auto* tv) {
    using TQ = std::remove_pointer_t<decltype(tq)>;
    using TV = std::remove_pointer_t<decltype(tv)>;
    auto go = [&](auto nkk) {
      constexpr int N = decltype(nkk)::value;
      if (delta) launch_lds(memory_chunk_local_kernel<TQ, TV, true, N>, grid, 64 * nw, lds, a);
      else launch_lds(memory_chunk_local_kernel<TQ, TV, false, N>, grid, 64 * nw, lds, a);
    };
    by_width(a.dk, go);
  });
}

void memory_combine(at::Tensor S, const at::Tensor& slots, const at::Tensor& start, const at::Tensor& base, const at::Tensor& loc, const at::Tensor& dec,
                    const OptT& trans, at::Tensor init) {
  HYB_CHECK(S.is_cuda() && S.is_contiguous() && S.scalar_type() == at::kFloat && S.dim() == 4, "state: contiguous fp32 [slots, H, dk, dv]");
  const int64_t H = S.size(1), dk = S.size(2), dv = S.size(3), per = dk * dv;
  HYB_CHECK(loc.dim() == 4 && f32vec(loc, loc.size(0) * H * per) && f32vec(init, loc.numel()) && f32vec(dec, loc.size(0) * H), "loc, init: fp32 [chunks, H, dk, dv]; dec: fp32 [chunks, H]");
  HYB_CHECK(i32(slots) && i32(start) && i32(base) && start.numel() == slots.numel() && base.numel() == slots.numel() + 1, "slots [n], start [n], base [n + 1]: int32");
  const int64_t ns = slots.numel(), P = loc.size(0);
  if (ns == 0 || P == 0) return;
  c10::DeviceGuard guard(S.device());
  if (!trans.has_value()) {
    HYB_CHECK((per + 255) / 256 <= 65535, "grid too large");
    memory_combine_kernel<<<dim3((unsigned)ns, (unsigned)H, (unsigned)((per + 255) / 256)), 256, 0, cur_stream()>>>(
        S.data_ptr<float>(), slots.data_ptr<int>(), start.data_ptr<int>(), base.data_ptr<int>(), loc.data_ptr<float>(), dec.data_ptr<float>(),
        init.data_ptr<float>(), (int)H, per);
    return;
  }
  const int64_t kk = (dk + 15) / 16, dkp = 16 * kk;
  HYB_CHECK(f32vec(*trans, P * H * dkp * dkp) && dk <= 256, "trans: fp32 [chunks, H, dkp, dkp]");
  const dim3 grid((unsigned)ns, (unsigned)H, (unsigned)((dv + 15) / 16));
  auto go = [&](auto kern, int KK) {
    kern<<<grid, 64 * KK, 0, cur_stream()>>>(S.data_ptr<float>(), slots.data_ptr<int>(), start.data_ptr<int>(), base.data_ptr<int>(),
                                             loc.data_ptr<float>(), trans->data_ptr<float>(), init.data_ptr<float>(), (int)H, (int)dk, (int)dv);
  };
  switch (kk) {
#define CASE(N, PD) case N: go(memory_combine_delta_kernel<N, PD>, N); break
    CASE(1, 8); CASE(2, 8); CASE(3, 8); CASE(4, 6); CASE(5, 4); CASE(6, 4); CASE(7, 4); CASE(8, 4);
    CASE(9, 2); CASE(10, 2); CASE(11, 2); CASE(12, 2); CASE(13, 1); CASE(14, 1); CASE(15, 1); CASE(16, 1);
#undef CASE
    default: HYB_CHECK(false, "key size 1 .. 256");
  }
}

}  // namespace llmctl_hybrid
