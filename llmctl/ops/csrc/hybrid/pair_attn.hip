// Differential attention over a paged row cache: every head has two attention maps (queries and keys of their own,
// width ``dk`` each) over the same values, and its output is
//   o = a_1 - lambda a_2,   o <- post * o / sqrt(mean(o^2) + eps)   (the mean over the head's dv values),
// where a_m is the ordinary causal softmax attention of map m inside a sliding window (i - j < window).
//
// A token's cache row holds G sub-rows [v (dv) | k_1 (dk) | k_2 (dk)], one per kv head; query head h reads sub-row
// h / (H / G).  Queries are rows [H][2][dk] at a row pitch of their own (columns of the fused projection's output).
//
//   pair_attn_mfma_kernel     bf16, MFMA 32x32x16; prompt portions and decode rows.  A workgroup (4 waves) owns 128
//                             query rows = TB tokens x HB heads; 64-key tiles are gathered through the block table into
//                             LDS once (a row image of both maps' keys, a transposed-read image of the values), the two
//                             maps' scores and softmaxes follow one another and their P V products share every value
//                             fragment; the combination and the norm happen in the epilogue (query on the lane, so
//                             the sum over the values is lane-local but for one exchange of the two lane halves)
//   pair_merge_kernel         decode rows whose keys were split over workgroups, and values wider than 128, whose column
//                             tiles are: both maps' parts merged, then combination and norm
//   pair_attn_generic_kernel  any shape, fp32 or bf16: one workgroup per (query row, head)
#include "attn_common.h"
#include "hybrid_common.h"

namespace llmctl_hybrid {
using namespace llmctl::attn;

namespace {
constexpr int PKB = 64;         // keys per tile
constexpr int PROWB = 256;      // bytes of a row of a 128-column block image
constexpr int PIMG = PKB * PROWB;
constexpr float kRescale = 8.f;

struct PairArgs {
  const void* q;
  int64_t q_st;  // row pitch of the queries (elements)
  const void* cache;
  void* out;  // [rows, H * dv]
  const int* bt;
  const int* cu;  // nullptr: one query row per sequence (decode)
  const int* ctx;
  const float* lam;  // one number
  int H, G, dk, dv, rs, bs, maxb, window, HB, hpg;
  float scale_log2, scale, post, eps;
  int nsplit, nvt;  // key splits (decode), value tiles of a head
  // with several splits or value tiles a workgroup leaves its unnormalised parts here and pair_merge_kernel finishes
  float* ws_o;   // [rows * H, nsplit, 2, dv]
  float* ws_ml;  // [rows * H, nsplit, 2, 2]
};

// KB: 128-column blocks of the key image; a map takes 64 KB of its columns (dk <= 64 KB).  NDB: 32-column blocks of values.
template <int KB, int NDB>
__global__ __launch_bounds__(256, 1) void pair_attn_mfma_kernel(PairArgs a) {
  constexpr int NKM = 4 * KB;  // 16-wide steps per map
  constexpr int NTB = (NDB + 3) / 4;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  constexpr int BUFB = (KB + NTB) * PIMG;  // one of the two tile buffers
  const unsigned short* cache = reinterpret_cast<const unsigned short*>(a.cache);

  const int tid = threadIdx.x;
  const int lane = tid & 63, wave = tid >> 6;
  const int r = lane & 31, hh = lane >> 5;
  const int n = blockIdx.y;
  const int P = a.H / a.G;
  const int zi = blockIdx.z / a.nvt, v0 = (blockIdx.z % a.nvt) * (NDB * 32);  // this workgroup's first value column
  const int grp = zi / a.hpg, hsub = (zi % a.hpg) * a.HB;
  const int q_begin = a.cu ? a.cu[n] : n;
  const int qlen = a.cu ? a.cu[n + 1] - q_begin : 1;
  const int HB = a.HB, TB = 128 / HB;
  const int split = a.nsplit > 1 ? blockIdx.x : 0;
  const int tok0 = a.nsplit > 1 ? 0 : (int)(gridDim.x - 1 - blockIdx.x) * TB;
  if (tok0 >= qlen) return;
  const int ctx = a.ctx[n];
  const int pos0 = ctx - qlen;
  const int row = wave * 32 + r;
  const int my_tok = tok0 + row / HB, my_head = grp * P + hsub + row % HB;
  const bool valid = my_tok < qlen && hsub + row % HB < P;
  const int tokc = min(my_tok, qlen - 1), headc = grp * P + min(hsub + row % HB, P - 1);
  const int my_pos = pos0 + tokc;
  const int* btn = a.bt + (long)n * a.maxb;

  bf16x8_t qf[2 * NKM];
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    const unsigned short* Qp = reinterpret_cast<const unsigned short*>(a.q) + (q_begin + tokc) * a.q_st + (long)(headc * 2 + m) * a.dk;
#pragma unroll
    for (int ks = 0; ks < NKM; ++ks) {
      const int col = ks * 16 + 8 * hh;
      uint4 v = make_uint4(0, 0, 0, 0);
      if (col < a.dk) v = gload16(Qp + col);
      qf[m * NKM + ks] = __builtin_bit_cast(bf16x8_t, v);
    }
  }
  f32x16 o[2][NDB];
  float m_i[2], l_i[2];
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    m_i[m] = -INFINITY;
    l_i[m] = 0.f;
#pragma unroll
    for (int d = 0; d < NDB; ++d)
#pragma unroll
      for (int i = 0; i < 16; ++i) o[m][d][i] = 0.f;
  }

  const int first_pos = pos0 + tok0, last_pos = pos0 + min(tok0 + TB, qlen) - 1;
  auto first_key = [&](int p) { return max(p - a.window + 1, 0); };
  int t_lo = first_key(first_pos) / PKB, t_hi = last_pos / PKB + 1;
  if (a.nsplit > 1) {
    const int per = (t_hi - t_lo + a.nsplit - 1) / a.nsplit;
    t_lo += split * per;
    t_hi = min(t_hi, t_lo + per);
  }
  const int w_first = pos0 + min(tok0 + (wave * 32) / HB, qlen - 1);
  const int w_last = pos0 + min(tok0 + (wave * 32 + 31) / HB, qlen - 1);
  const bool wave_live = tok0 + (wave * 32) / HB < qlen && hsub + (HB >= 32 ? (wave * 32) % HB : 0) < P;
  const int w_lo = first_key(w_first), w_lo_last = first_key(w_last), my_lo = first_key(my_pos);
  int tr_lo[4], tr_hi[4];
#pragma unroll
  for (int c = 0; c < 4; ++c) tr_frag_offs<128>(c * 32, lane, tr_lo[c], tr_hi[c]);
  const int k_row = r * PROWB, k_x = (hh ^ (r & 15)) << 4;

  const int wave_u = __builtin_amdgcn_readfirstlane(wave);
  const unsigned lds_base = lds_addr(smem);
  int* slot_lds = reinterpret_cast<int*>(smem + 2 * BUFB);  // cache slots of a tile's keys, two tiles
  auto slot_of = [&](int t) {
    const int key = min(t * PKB + tid, ctx - 1);
    return btn[key / a.bs] * a.bs + key % a.bs;
  };
  // image columns past a map's width or past the row's end read a valid neighbour (finite data): such columns meet
  // zero query entries, or are value columns that are never stored
  auto fill = [&](int buf) {
#pragma unroll 4
    for (int g = wave_u; g < 16 * (KB + NTB); g += 4) {
      const int img = g >> 4, rg = g & 15;
      const int krow = rg * 4 + (lane >> 4), chp = lane & 15;
      const long slot = slot_lds[buf * PKB + krow];
      int col;
      if (img < KB) {
        const int c = (img * 16 + (chp ^ swz_row<128>(krow))) * 8;
        const int m = c >= 64 * KB ? 1 : 0;
        col = a.dv + m * a.dk + min(c - m * 64 * KB, a.dk - 8);
      } else {
        col = min(v0 + ((img - KB) * 16 + (chp ^ swz_tr<128>(krow))) * 8, a.rs - 8);
      }
      dma16(cache + (slot * a.G + grp) * a.rs + col, lds_base + (unsigned)(buf * BUFB + img * PIMG + rg * 1024));
    }
  };
  // slots of tile t + 2 are requested before the fill of tile t + 1 is issued, so that no wave waits on its own fill in
  // between (a wave's memory operations complete in order)
  int pend = 0;
  if (t_lo < t_hi) {
    if (tid < PKB) slot_lds[tid] = slot_of(t_lo);
    __syncthreads();
    if (t_lo + 1 < t_hi && tid < PKB) pend = slot_of(t_lo + 1);
    fill(0);
  }
  for (int t = t_lo; t < t_hi; ++t) {
    const int buf = (t - t_lo) & 1;
    const unsigned char* Ks = smem + buf * BUFB;
    const unsigned char* Vs = Ks + KB * PIMG;
    // after the barrier every wave's pieces of tile t have landed, every wave is done with tile t - 1 (its images
    // may be overwritten) and the slots of t + 1 are visible
    if (t + 1 < t_hi && tid < PKB) slot_lds[(buf ^ 1) * PKB + tid] = pend;
    vm_wait<0>();
    __syncthreads();
    if (t + 2 < t_hi && tid < PKB) pend = slot_of(t + 2);
    if (t + 1 < t_hi) fill(buf ^ 1);
    const int kv0 = t * PKB;
    if (!wave_live || kv0 > w_last || kv0 + PKB - 1 < w_lo) continue;
    const bool whole = kv0 + PKB - 1 <= w_first && kv0 >= w_lo_last && kv0 + PKB - 1 < ctx;  // no row masks a key of the tile

    bf16x8_t pb[2][2][2];
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      f32x16 s[2];
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
#pragma unroll
        for (int i = 0; i < 16; ++i) s[kb][i] = 0.f;
#pragma unroll
        for (int ks = 0; ks < NKM; ++ks) {
          const int gs = m * NKM + ks;
          const bf16x8_t kf = lds_read_b128(Ks + (gs >> 3) * PIMG + kb * 32 * PROWB, k_row + (k_x ^ (((2 * gs) & 15) << 4)));
          s[kb] = mfma32(kf, qf[gs], s[kb]);
        }
      }
      float mx = -INFINITY;
      if (whole) {
#pragma unroll
        for (int kb = 0; kb < 2; ++kb)
#pragma unroll
          for (int i = 0; i < 16; ++i) {
            s[kb][i] *= a.scale_log2;
            mx = fmaxf(mx, s[kb][i]);
          }
        if (!valid) mx = -INFINITY;  // such a row must not trigger the wave's rescale
      } else {
#pragma unroll
        for (int kb = 0; kb < 2; ++kb)
#pragma unroll
          for (int i = 0; i < 16; ++i) {
            float x = s[kb][i] * a.scale_log2;
            const int key = kv0 + kb * 32 + acc_row(i, hh);
            if (!valid || key > my_pos || key < my_lo) x = -INFINITY;
            s[kb][i] = x;
            mx = fmaxf(mx, x);
          }
      }
      mx = xor32_max(mx);
      const bool grow = __builtin_amdgcn_ballot_w64(mx > m_i[m] + kRescale) != 0;
      const float m_raw = grow ? fmaxf(m_i[m], mx) : m_i[m];
      const float m_new = m_raw == -INFINITY ? 0.f : m_raw;  // nothing seen yet
      float rs = 0.f;
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
        float p[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          p[i] = fast_exp2(s[kb][i] - m_new);
          rs += p[i];
        }
        pb[m][kb][0] = to_bf16x8(p);
        pb[m][kb][1] = to_bf16x8(p + 8);
      }
      rs = xor32_add(rs);
      if (grow) {
        const float alpha = fast_exp2(m_i[m] - m_new);
        l_i[m] *= alpha;
#pragma unroll
        for (int d = 0; d < NDB; ++d)
#pragma unroll
          for (int i = 0; i < 16; ++i) o[m][d][i] *= alpha;
      }
      l_i[m] += rs;
      m_i[m] = m_raw;
    }
#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
#pragma unroll
      for (int st = 0; st < 2; ++st)
#pragma unroll
        for (int d = 0; d < NDB; ++d) {
          const bf16x8_t vf = tr_frag_at<128>(Vs + (d >> 2) * PIMG, kb * 32 + 16 * st, tr_lo[d & 3], tr_hi[d & 3]);
          o[0][d] = mfma32(vf, pb[0][kb][st], o[0][d]);
          o[1][d] = mfma32(vf, pb[1][kb][st], o[1][d]);
        }
  }

  if (a.ws_o != nullptr) {
    if (!valid) return;
    const long rowi = (long)(q_begin + my_tok) * a.H + my_head;
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      float* Wp = a.ws_o + ((rowi * a.nsplit + split) * 2 + m) * a.dv;
#pragma unroll
      for (int d = 0; d < NDB; ++d)
#pragma unroll
        for (int g = 0; g < 4; ++g) {
          const int col = v0 + d * 32 + 8 * g + 4 * hh;
          if (col < a.dv) *reinterpret_cast<float4*>(Wp + col) = make_float4(o[m][d][4 * g], o[m][d][4 * g + 1], o[m][d][4 * g + 2], o[m][d][4 * g + 3]);
        }
      if (hh == 0 && v0 == 0) {
        a.ws_ml[((rowi * a.nsplit + split) * 2 + m) * 2] = m_i[m];
        a.ws_ml[((rowi * a.nsplit + split) * 2 + m) * 2 + 1] = l_i[m];
      }
    }
    return;
  }
  const float f0 = 1.f / l_i[0], f1 = a.lam[0] / l_i[1];
  float ss = 0.f;
#pragma unroll
  for (int d = 0; d < NDB; ++d)
#pragma unroll
    for (int g = 0; g < 4; ++g) {
      const int col = d * 32 + 8 * g + 4 * hh;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float v = o[0][d][4 * g + j] * f0 - o[1][d][4 * g + j] * f1;
        o[0][d][4 * g + j] = v;
        if (col < a.dv) ss += v * v;
      }
    }
  ss = xor32_add(ss);
  const float rstd = a.post / sqrtf(ss / (float)a.dv + a.eps);
  if (!valid) return;
  unsigned short* Op = reinterpret_cast<unsigned short*>(a.out) + ((long)(q_begin + my_tok) * a.H + my_head) * a.dv;
#pragma unroll
  for (int d = 0; d < NDB; ++d)
#pragma unroll
    for (int g = 0; g < 4; ++g) {
      const int col = d * 32 + 8 * g + 4 * hh;
      if (col < a.dv) {
        unsigned short w4[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) w4[j] = __bfloat16_as_ushort(__float2bfloat16(o[0][d][4 * g + j] * rstd));
        *reinterpret_cast<uint2*>(Op + col) = make_uint2((unsigned)w4[0] | ((unsigned)w4[1] << 16), (unsigned)w4[2] | ((unsigned)w4[3] << 16));
      }
    }
}

// One workgroup per (row, head); splits that saw nothing: m = -inf, l = 0.  dv <= 128 MERGE_COLS.
constexpr int MERGE_COLS = 8;
__global__ __launch_bounds__(128) void pair_merge_kernel(const float* __restrict__ ws_o, const float* __restrict__ ws_ml,
                                                         unsigned short* __restrict__ out, const float* __restrict__ lam, int nsplit, int dv,
                                                         float post, float eps) {
  __shared__ float red[2];
  const long row = blockIdx.x;
  const float* ml = ws_ml + row * nsplit * 4;
  float inv[2], M[2];
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    M[m] = -INFINITY;
    for (int s = 0; s < nsplit; ++s) M[m] = fmaxf(M[m], ml[s * 4 + m * 2]);
    float L = 0.f;
    for (int s = 0; s < nsplit; ++s) L += ml[s * 4 + m * 2] == -INFINITY ? 0.f : ml[s * 4 + m * 2 + 1] * fast_exp2(ml[s * 4 + m * 2] - M[m]);
    inv[m] = (m == 0 ? 1.f : lam[0]) / L;
  }
  float v[MERGE_COLS], ss = 0.f;
#pragma unroll
  for (int i = 0; i < MERGE_COLS; ++i) {
    const int c = threadIdx.x + 128 * i;
    v[i] = 0.f;
    if (c < dv) {
      float p[2] = {0.f, 0.f};
      for (int s = 0; s < nsplit; ++s)
#pragma unroll
        for (int m = 0; m < 2; ++m) {
          const float mv = ml[s * 4 + m * 2];
          if (mv != -INFINITY) p[m] += ws_o[((row * nsplit + s) * 2 + m) * dv + c] * fast_exp2(mv - M[m]);
        }
      v[i] = p[0] * inv[0] - p[1] * inv[1];
      ss += v[i] * v[i];
    }
  }
  const float rstd = post / sqrtf(block_sum<2>(ss, red) / (float)dv + eps);
#pragma unroll
  for (int i = 0; i < MERGE_COLS; ++i) {
    const int c = threadIdx.x + 128 * i;
    if (c < dv) out[row * dv + c] = __bfloat16_as_ushort(__float2bfloat16(v[i] * rstd));
  }
}

// grid (query rows of the longest portion, sequences, heads); each of 4 waves takes 64 keys at a time (one per lane for the
// scores of both maps, lanes over the value columns for the weighted sums)
template <typename T, int NA>
__global__ __launch_bounds__(256) void pair_attn_generic_kernel(PairArgs a) {
  extern __shared__ float sm[];
  const int n = blockIdx.y, h = blockIdx.z;
  const int q_begin = a.cu ? a.cu[n] : n;
  const int qlen = a.cu ? a.cu[n + 1] - q_begin : 1;
  if ((int)blockIdx.x >= qlen) return;
  const int dk = a.dk, dv = a.dv;
  int64_t* ro = reinterpret_cast<int64_t*>(sm);  // [4][64] rows of a wave's keys
  float* pw = reinterpret_cast<float*>(ro + 256);  // [4][2][64] weights
  float* ml = pw + 512;                            // [4][2][2]
  float* qs = ml + 16;                             // [2][dk]
  float* ac = qs + 2 * dk;                         // [4][2][dv]
  float* red = ac + 8 * dv;                        // [4]
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int pos = a.ctx[n] - qlen + (int)blockIdx.x;
  const int lo = max(pos - a.window + 1, 0), nk = pos + 1 - lo;
  const int64_t qrow = q_begin + (int)blockIdx.x;
  const T* qp = reinterpret_cast<const T*>(a.q) + qrow * a.q_st + (int64_t)h * 2 * dk;
  for (int d = threadIdx.x; d < 2 * dk; d += 256) qs[d] = ldf(qp + d);
  __syncthreads();
  const T* cache = reinterpret_cast<const T*>(a.cache);
  const int* btn = a.bt + (int64_t)n * a.maxb;
  const int grp = h / (a.H / a.G);
  float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};
  float acc[2][NA];
#pragma unroll
  for (int i = 0; i < NA; ++i) acc[0][i] = acc[1][i] = 0.f;
  for (int c = wave * 64; c < nk; c += 256) {
    const bool ok = c + lane < nk;
    const int j = lo + min(c + lane, nk - 1);
    const int64_t off = (((int64_t)btn[j / a.bs] * a.bs + j % a.bs) * a.G + grp) * a.rs;
    const T* key = cache + off + dv;
    ro[wave * 64 + lane] = off;
#pragma unroll
    for (int mm = 0; mm < 2; ++mm) {
      float s = 0.f;
      for (int d = 0; d < dk; ++d) s += qs[mm * dk + d] * ldf(key + mm * dk + d);
      s = ok ? s * a.scale : -INFINITY;
      const float mn = fmaxf(m[mm], wave_max(s));  // at least one key of the 64 is visible: finite
      const float p = ok ? expf(s - mn) : 0.f, corr = expf(m[mm] - mn);
      l[mm] = l[mm] * corr + wave_sum(p);
      m[mm] = mn;
      pw[(wave * 2 + mm) * 64 + lane] = p;
#pragma unroll
      for (int i = 0; i < NA; ++i) acc[mm][i] *= corr;
    }
    __builtin_amdgcn_wave_barrier();
    const int cnt = min(64, nk - c);
    for (int jj = 0; jj < cnt; ++jj) {
      const float p0 = pw[wave * 128 + jj], p1 = pw[wave * 128 + 64 + jj];
      const T* vr = cache + ro[wave * 64 + jj];
#pragma unroll
      for (int i = 0; i < NA; ++i) {
        const int d = lane + 64 * i;
        if (d < dv) {
          const float x = ldf(vr + d);
          acc[0][i] += p0 * x;
          acc[1][i] += p1 * x;
        }
      }
    }
    __builtin_amdgcn_wave_barrier();
  }
#pragma unroll
  for (int mm = 0; mm < 2; ++mm) {
    if (lane == 0) {
      ml[(wave * 2 + mm) * 2] = m[mm];
      ml[(wave * 2 + mm) * 2 + 1] = l[mm];
    }
#pragma unroll
    for (int i = 0; i < NA; ++i) {
      const int d = lane + 64 * i;
      if (d < dv) ac[(wave * 2 + mm) * dv + d] = acc[mm][i];
    }
  }
  __syncthreads();
  float f[2][4];
#pragma unroll
  for (int mm = 0; mm < 2; ++mm) {
    float M = -INFINITY, L = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) M = fmaxf(M, ml[(w * 2 + mm) * 2]);
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      f[mm][w] = ml[(w * 2 + mm) * 2 + 1] > 0.f ? expf(ml[(w * 2 + mm) * 2] - M) : 0.f;
      L += ml[(w * 2 + mm) * 2 + 1] * f[mm][w];
    }
    const float g = (mm == 0 ? 1.f : a.lam[0]) / L;
#pragma unroll
    for (int w = 0; w < 4; ++w) f[mm][w] *= g;
  }
  float ss = 0.f;
  for (int d = threadIdx.x; d < dv; d += 256) {  // every thread reads and rewrites its own columns
    float v = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) v += ac[w * 2 * dv + d] * f[0][w] - ac[(w * 2 + 1) * dv + d] * f[1][w];
    ac[d] = v;
    ss += v * v;
  }
  const float rstd = a.post / sqrtf(block_sum<4>(ss, red) / (float)dv + a.eps);
  T* op = reinterpret_cast<T*>(a.out) + (qrow * a.H + h) * dv;
  for (int d = threadIdx.x; d < dv; d += 256) stf(op + d, ac[d] * rstd);
}

// [v | k_1 | k_2] of every kv head from the columns of z to the token's cache row; 16-byte pieces (N elements) or single ones
template <typename T, int N>
__global__ __launch_bounds__(256) void kv_rows_write_kernel(const T* __restrict__ k, int64_t k_st, const T* __restrict__ v, int64_t v_st,
                                                            T* __restrict__ cache, const int64_t* __restrict__ slots, int G, int kw, int dv,
                                                            int64_t total) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const int rs = kw + dv, per = G * rs / N;
  const int64_t t = i / per;
  const int c = (int)(i - t * per) * N;
  const int64_t slot = slots[t];
  if (slot < 0) return;
  const int g = c / rs, d = c - g * rs;
  const T* src = d < dv ? v + t * v_st + (int64_t)g * dv + d : k + t * k_st + (int64_t)g * kw + (d - dv);
  T* dst = cache + slot * (int64_t)G * rs + c;
  if constexpr (N == 1) *dst = *src;
  else *reinterpret_cast<uint4*>(dst) = *reinterpret_cast<const uint4*>(src);
}

bool i32c(const at::Tensor& t, int64_t n) { return t.is_cuda() && t.is_contiguous() && t.scalar_type() == at::kInt && t.numel() == n; }
}  // namespace

void kv_rows_write(const at::Tensor& k, const at::Tensor& v, at::Tensor cache, const at::Tensor& slots, int64_t groups) {
  check_rows(k, "k");
  check_rows(v, "v");
  const int64_t T = k.size(0), G = groups;
  HYB_CHECK(G >= 1 && v.size(0) == T && k.size(1) % G == 0 && v.size(1) % G == 0 && k.scalar_type() == v.scalar_type(), "k and v: [T, groups * width] of one dtype");
  HYB_CHECK(cache.is_cuda() && cache.is_contiguous() && cache.dim() == 3 && cache.size(2) == k.size(1) + v.size(1) && cache.scalar_type() == k.scalar_type(),
            "cache: contiguous [blocks, block_size, groups * row width] of k's dtype");
  HYB_CHECK(slots.is_cuda() && slots.is_contiguous() && slots.scalar_type() == at::kLong && slots.numel() == T, "slots: int64 [T]");
  if (T == 0) return;
  c10::DeviceGuard guard(k.device());
  const int kw = (int)(k.size(1) / G), dv = (int)(v.size(1) / G);
  dispatch_act(k, [&](auto* tag) {
    using Tt = std::remove_pointer_t<decltype(tag)>;
    constexpr int N = Vec16<Tt>::N;
    const bool vec = kw % N == 0 && dv % N == 0 && aligned16<Tt>(k) && aligned16<Tt>(v) && reinterpret_cast<uintptr_t>(cache.data_ptr()) % 16 == 0;
    const int64_t total = T * G * (kw + dv) / (vec ? N : 1);
    const dim3 grid((unsigned)((total + 255) / 256));
    auto go = [&](auto kern) {
      kern<<<grid, 256, 0, cur_stream()>>>((const Tt*)k.data_ptr(), k.stride(0), (const Tt*)v.data_ptr(), v.stride(0), (Tt*)cache.data_ptr(),
                                           slots.data_ptr<int64_t>(), (int)G, kw, dv, total);
    };
    if (vec) go(kv_rows_write_kernel<Tt, N>);
    else go(kv_rows_write_kernel<Tt, 1>);
  });
}

// q [rows, >= H * 2 * dk] (row-strided view); cu empty: decode, one row per sequence.  Writes out [rows, H * dv].
void diff_attn(const at::Tensor& q, const at::Tensor& cache, const at::Tensor& bt, const c10::optional<at::Tensor>& cu, const at::Tensor& ctx,
               int64_t heads, int64_t groups, int64_t dk, int64_t dv, int64_t window, double scale, const at::Tensor& lam, double post, double eps,
               int64_t max_q, int64_t max_ctx, bool mfma, at::Tensor out) {
  check_rows(q, "q");
  const int64_t rows = q.size(0), H = heads, G = groups, ns = ctx.numel();
  HYB_CHECK(H >= 1 && G >= 1 && H % G == 0 && dk >= 1 && dv >= 1 && q.size(1) >= H * 2 * dk, "q: [rows, >= heads * 2 * dk]; kv heads divide the heads");
  HYB_CHECK(cache.is_cuda() && cache.is_contiguous() && cache.dim() == 3 && cache.size(2) == G * (dv + 2 * dk) && cache.scalar_type() == q.scalar_type(),
            "cache: contiguous [blocks, block_size, kv heads * (dv + 2 dk)] of q's dtype");
  HYB_CHECK(bt.is_cuda() && bt.is_contiguous() && bt.scalar_type() == at::kInt && bt.dim() == 2 && bt.size(0) == ns && i32c(ctx, ns), "block tables [n, max_blocks], ctx [n]: int32");
  HYB_CHECK(cu.has_value() ? (i32c(*cu, ns + 1) && max_q >= 1) : rows == ns, "portions: cu int32 [n + 1], max_q >= 1; decode: one row per sequence");
  HYB_CHECK(lam.is_cuda() && lam.scalar_type() == at::kFloat && lam.numel() == 1, "lambda: one fp32 number");
  HYB_CHECK(out.is_cuda() && out.is_contiguous() && out.scalar_type() == q.scalar_type() && out.numel() == rows * H * dv, "out: contiguous [rows, heads * dv] of q's dtype");
  HYB_CHECK(window >= 1 && ns <= 65535 && H <= 65535, "window >= 1; grid too large");
  if (rows == 0 || ns == 0) return;
  c10::DeviceGuard guard(q.device());
  PairArgs a{};
  a.q = q.data_ptr();
  a.q_st = q.stride(0);
  a.cache = cache.data_ptr();
  a.out = out.data_ptr();
  a.bt = bt.data_ptr<int>();
  a.cu = cu.has_value() ? cu->data_ptr<int>() : nullptr;
  a.ctx = ctx.data_ptr<int>();
  a.lam = lam.data_ptr<float>();
  a.H = (int)H, a.G = (int)G, a.dk = (int)dk, a.dv = (int)dv;
  a.rs = (int)(dv + 2 * dk);
  a.bs = (int)cache.size(1), a.maxb = (int)bt.size(1);
  a.window = (int)std::min<int64_t>(window, (int64_t)1 << 30);
  a.scale = (float)scale;
  a.scale_log2 = (float)(scale * 1.4426950408889634);
  a.post = (float)post, a.eps = (float)eps;
  a.nsplit = 1;
  hipStream_t st = cur_stream();
  const bool fits = q.scalar_type() == at::kBFloat16 && dk % 8 == 0 && dv % 8 == 0 && dk <= 128 && dv <= 128 * MERGE_COLS && aligned16<bf16_t>(q) &&
                    reinterpret_cast<uintptr_t>(cache.data_ptr()) % 16 == 0;
  if (mfma && fits) {
    const int64_t P = H / G;
    int HB = 1;
    const int64_t longest = cu.has_value() ? max_q : 1;
    if (longest < 64)
      while (HB < P && HB < 128) HB *= 2;
    const int TB = 128 / HB;
    a.HB = HB;
    a.hpg = (int)((P + HB - 1) / HB);
    const int NDBv = dv <= 64 ? 2 : 4;
    a.nvt = (int)((dv + NDBv * 32 - 1) / (NDBv * 32));
    HYB_CHECK(G * a.hpg * a.nvt <= 65535, "grid too large");
    at::Tensor ws_o, ws_ml;
    if (!cu.has_value()) {  // decode: split the visible key tiles over workgroups, one for every CU at most (a CU holds one)
      const int64_t span = std::min<int64_t>(a.window, max_ctx > 0 ? max_ctx : (int64_t)1 << 30);
      const int tiles = (int)std::min<int64_t>((span + PKB - 1) / PKB + 1, 1 << 20);
      const long blocks = (long)ns * G * a.hpg * a.nvt;
      while (a.nsplit < tiles && a.nsplit < 32 && blocks * a.nsplit * 2 <= 256) a.nsplit *= 2;
    }
    if (a.nsplit > 1 || a.nvt > 1) {
      ws_o = at::empty({rows * H * a.nsplit * 2 * dv}, q.options().dtype(at::kFloat));
      ws_ml = at::empty({rows * H * a.nsplit * 4}, q.options().dtype(at::kFloat));
      a.ws_o = ws_o.data_ptr<float>();
      a.ws_ml = ws_ml.data_ptr<float>();
    }
    const dim3 grid(a.nsplit > 1 ? (unsigned)a.nsplit : (unsigned)((longest + TB - 1) / TB), (unsigned)ns, (unsigned)(G * a.hpg * a.nvt));
    auto go = [&](auto kern, int KB, int NDB) {
      const size_t lds = (size_t)2 * (KB + (NDB + 3) / 4) * PIMG + 2 * PKB * sizeof(int);
      HYB_CHECK(hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) == hipSuccess, "LDS size");
      kern<<<grid, 256, lds, st>>>(a);
    };
    if (dk <= 64) {
      if (NDBv == 2) go(pair_attn_mfma_kernel<1, 2>, 1, 2);
      else go(pair_attn_mfma_kernel<1, 4>, 1, 4);
    } else {
      if (NDBv == 2) go(pair_attn_mfma_kernel<2, 2>, 2, 2);
      else go(pair_attn_mfma_kernel<2, 4>, 2, 4);
    }
    if (a.ws_o != nullptr)
      pair_merge_kernel<<<dim3((unsigned)(rows * H)), 128, 0, st>>>(a.ws_o, a.ws_ml, (unsigned short*)a.out, a.lam, a.nsplit, (int)dv, a.post, a.eps);
    return;
  }
  const size_t lds = 256 * 8 + (size_t)(512 + 16 + 2 * dk + 8 * dv + 4) * 4;
  HYB_CHECK(dv <= 1024 && lds <= 64 * 1024, "key or value too wide");
  const dim3 grid((unsigned)(cu.has_value() ? max_q : 1), (unsigned)ns, (unsigned)H);
  dispatch_act(q, [&](auto* tag) {
    using Tt = std::remove_pointer_t<decltype(tag)>;
    if (dv <= 128) pair_attn_generic_kernel<Tt, 2><<<grid, 256, lds, st>>>(a);
    else pair_attn_generic_kernel<Tt, 16><<<grid, 256, lds, st>>>(a);
  });
}

}  // namespace llmctl_hybrid
