// A gated delta rule with a decay per key channel over a step's rows, with the request's state in its slot; everything is 32-bit.
//
// Per head a state S [d, dv] (key channel i, value channel j), a token's unit key k and query q, value v, decays g [d], beta:
//     S <- diag(g) S;   w = beta (v - S^T k);   S <- S + k w^T;   o = S^T q
// low_rank: log g = -rate softplus(W_a a + bias) and the output gate sigmoid(W_g b) of every (token, head, channel): two products
//     over a small inner size on v_mfma_f32_16x16x4_f32 (true 32-bit), the inner activations straight from the projection's sums.
// scan: a workgroup a (row, head), tokens in order.  A lane is a column of S, a wave owns R rows of it in registers.  With
//     S' = diag(g) S the sums S'^T k and S'^T q are taken in one pass over the rows (o = S'^T q + (k . q) w), the waves' shares
//     meet in the LDS: one barrier a token.  Unit vectors come as factors on the sums.  A head's output is divided by its root
//     mean square, times the weight and the gate, and rounded once.
//
// Rows of many tokens run in chunks of 64 on the matrix cores, in 32-bit.  G_t is the sum of log g over a chunk's tokens up to t
// (a vector over the channels), S_0 the state the chunk starts from.  Unrolled,
//     S_t = diag(e^G_t) S_0 + sum_(s <= t) diag(e^(G_t - G_s)) k_s w_s^T
// so that with  A_ts = sum_i k_ti k_si e^(G_ti - G_si)  (s < t)  and  Q_ts  the same with q_t for k_t (s <= t)
//     (I + diag(beta) A) w = diag(beta) (v - (e^G k) S_0)      =>      w = U - W S_0,   [U | W] = (I + diag(beta) A)^-1 diag(beta) [v | e^G k]
//     S_end = diag(e^G_end) S_0 + (e^(G_end - G) k)^T w,        o = (e^G q) S_0 + Q w.
// (1) chunk_solve, a workgroup a (chunk, head): A, Q, the inverse, U and W;  (2) chunk_fold, per (row, head, 16 columns), chunk after
// chunk: w and S_end, leaving every chunk's S_0 and w;  (3) chunk_outputs: o, its norm, weight and gate.
// No exponent is ever positive: within 16 tokens A and Q are taken pair by pair; for tokens s of an earlier 16 both factors are
// taken against the sum R at the start of t's 16, e^(G_t - R) and e^(R - G_s), so that the product runs on the matrix cores.
// The inverse is built from 16 x 16 blocks: the diagonal ones by substitution, X_ab = -X_aa sum_c M_ac X_cb below them.
#include "common.hpp"

typedef float f32x4 __attribute__((ext_vector_type(4)));
constexpr float LOG2E = 1.4426950408889634f;

// max(z, 0) + log(1 + e), e = 2^(-|z| log2 e): with u = 1 + e as rounded, log(1 + e) = log(u) e / (u - 1) (Kahan's correction: what u
// lost of e is made up by the factor), so the hardware's logarithm and reciprocal are enough
__device__ __forceinline__ float softplus(float z) {
  const float e = __builtin_amdgcn_exp2f(-fabsf(z) * LOG2E), u = 1.0f + e, d = u - 1.0f;
  const float l = d == 0.f ? e : __builtin_amdgcn_logf(u) * 0.6931471805599453f * (e * __builtin_amdgcn_rcpf(d));
  return fmaxf(z, 0.f) + l;
}
__device__ __forceinline__ float gate_sigmoid(float z) { return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-z * LOG2E)); }
__device__ __forceinline__ float pow2(float x) { return __builtin_amdgcn_exp2f(x); }      // below 2^-126: 0
// The waves meet over the LDS only: loads and stores of global memory stay on their way (__syncthreads would wait for them)
__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}
__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// ---- decays and gates: a wave 16 channels of 16 TT tokens.  Operand A lane (n, g): token n, B: channel n; both take inner numbers
// 16 kb + 4 g + j at step j (the order of the inner numbers is the same for both, so it may be any).  R: inner sizes, multiples of 16.
template <int TT>
__global__ void __launch_bounds__(256)
low_rank_kernel(const float* __restrict__ sums, long ld, int a_col, int g_col, const float* __restrict__ w_decay, int ra,
                const float* __restrict__ w_gate, int rg, const float* __restrict__ rate, const float* __restrict__ decay_bias,
                float* __restrict__ la, float* __restrict__ gate, int tokens, int H, int d, int dv, int decay_blocks) {
  const bool is_gate = (int)blockIdx.y >= decay_blocks;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, n = lane & 15, g = lane >> 4;
  const int channels = is_gate ? H * dv : H * d, R = is_gate ? rg : ra;
  const int c0 = ((int)blockIdx.y - (is_gate ? decay_blocks : 0)) * 64 + 16 * wave;
  if (c0 >= channels) return;
  const int c = c0 + n, t0 = blockIdx.x * 16 * TT;
  const float* __restrict__ wp = (is_gate ? w_gate : w_decay) + (size_t)(c < channels ? c : channels - 1) * R + 4 * g;
  const float* __restrict__ ip = sums + (is_gate ? g_col : a_col) + 4 * g;
  f32x4 acc[TT];
  size_t at[TT];
#pragma unroll
  for (int i = 0; i < TT; ++i) {
    acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int t = t0 + 16 * i + n;
    at[i] = (size_t)(t < tokens ? t : tokens - 1) * ld;
  }
#pragma unroll 4
  for (int kb = 0; kb < R; kb += 16) {
    const f32x4 w = *reinterpret_cast<const f32x4*>(wp + kb);
#pragma unroll
    for (int i = 0; i < TT; ++i) {
      const f32x4 a = *reinterpret_cast<const f32x4*>(ip + at[i] + kb);
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[i] = mfma4(a[j], w[j], acc[i]);
    }
  }
  if (c >= channels) return;
  const float r = is_gate ? 0.f : -rate[c / d], b = is_gate ? 0.f : decay_bias[c];
#pragma unroll
  for (int i = 0; i < TT; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = t0 + 16 * i + 4 * g + e;
      if (t >= tokens) continue;
      if (is_gate) gate[(size_t)t * channels + c] = gate_sigmoid(acc[i][e]);
      else la[(size_t)t * channels + c] = r * softplus(acc[i][e] + b);
    }
}

struct DeltaArgs {
  const float* q; const float* k; const float* v; long ld_u;      // first columns of queries, keys, values; rows ld_u floats apart
  int per_group;                 // heads that share a query/key head
  const float* beta; long ld;    // one a head, before its sigmoid
  const float* la;               // [T, H d] logarithms of the decays
  const float* gate;             // [T, H dv]
  const float* norm_weight; float eps, q_scale;
  float* state;                  // [slots, H, d, dv]
  const int* row_start; const int* slots;
  void* out;                     // [T, H dv]
  int H, d, dv;
  int first_row;                 // the launch's rows begin here
};

// ---- rows token by token.  threads: CB blocks of 64 columns x RG groups of R rows
constexpr int TB = 8;            // tokens staged in the LDS at a time
template <int R, typename TO>
__global__ void __launch_bounds__(1024)
scan_kernel(DeltaArgs a, int CB) {
  extern __shared__ __align__(16) float lds[];
  const int d = a.d, dv = a.dv, H = a.H, tid = threadIdx.x, nthreads = blockDim.x;
  const int lane = tid & 63, wave = tid >> 6, waves = nthreads >> 6, RG = waves / CB, cb = wave % CB, rg = wave / CB;
  const int DP = RG * R, CW = CB * 64;
  float* sq = lds;                       // [TB][DP] raw
  float* sk = sq + TB * DP;
  float* sg = sk + TB * DP;              // decays
  float* part = sg + TB * DP;            // [2][RG][2][CW]
  float* so = part + 4 * RG * CW;        // [TB][CW]
  float* sv = so + TB * CW;              // [TB][CW]
  float* sf = sv + TB * CW;              // [TB][4]: factors of q and k, k . q, beta
  const int row = a.first_row + blockIdx.x, h = blockIdx.y, hk = h / a.per_group, col = cb * 64 + lane;
  const int begin = a.row_start[row], end = a.row_start[row + 1];
  const bool active = col < dv;
  float* __restrict__ st = a.state + ((size_t)a.slots[row] * H + h) * d * dv + (active ? col : 0);
  const int r0 = rg * R;
  float S[R];
#pragma unroll
  for (int i = 0; i < R; ++i) S[i] = active && r0 + i < d ? st[(size_t)(r0 + i) * dv] : 0.f;
  int buf = 0;
  for (int t0 = begin; t0 < end; t0 += TB) {
    const int nt = end - t0 < TB ? end - t0 : TB;
    __syncthreads();
    for (int e = tid; e < nt * DP; e += nthreads) {
      const int tt = e / DP, i = e - tt * DP;
      const bool in = i < d;
      const size_t at = (size_t)(t0 + tt) * a.ld_u + (size_t)hk * d + (in ? i : 0);
      sq[e] = in ? a.q[at] : 0.f;
      sk[e] = in ? a.k[at] : 0.f;
      sg[e] = in ? expf(a.la[((size_t)(t0 + tt) * H + h) * d + i]) : 0.f;
    }
    for (int tt = rg; tt < nt; tt += RG) sv[tt * CW + col] = active ? a.v[(size_t)(t0 + tt) * a.ld_u + (size_t)h * dv + col] : 0.f;
    __syncthreads();
    for (int tt = wave; tt < nt; tt += waves) {
      float qq = 0.f, kk = 0.f, qk = 0.f;
      for (int i = lane; i < d; i += 64) {
        const float x = sq[tt * DP + i], y = sk[tt * DP + i];
        qq = fmaf(x, x, qq);
        kk = fmaf(y, y, kk);
        qk = fmaf(x, y, qk);
      }
      qq = wave_sum(qq);
      kk = wave_sum(kk);
      qk = wave_sum(qk);
      if (lane == 0) {
        const float fq = a.q_scale / sqrtf(qq + 1e-6f), fk = 1.0f / sqrtf(kk + 1e-6f);
        sf[4 * tt] = fq;
        sf[4 * tt + 1] = fk;
        sf[4 * tt + 2] = qk * fq * fk;
        sf[4 * tt + 3] = mie_sigmoid(a.beta[(size_t)(t0 + tt) * a.ld + h]);
      }
    }
    __syncthreads();
#pragma unroll 1
    for (int tt = 0; tt < nt; ++tt) {
      const float4* q4 = reinterpret_cast<const float4*>(sq + tt * DP + r0);
      const float4* k4 = reinterpret_cast<const float4*>(sk + tt * DP + r0);
      const float4* g4 = reinterpret_cast<const float4*>(sg + tt * DP + r0);
      float p = 0.f, o = 0.f;
#pragma unroll
      for (int i = 0; i < R / 4; ++i) {
        const float4 gg = g4[i], kk = k4[i], qq = q4[i];
        S[4 * i + 0] *= gg.x; p = fmaf(S[4 * i + 0], kk.x, p); o = fmaf(S[4 * i + 0], qq.x, o);
        S[4 * i + 1] *= gg.y; p = fmaf(S[4 * i + 1], kk.y, p); o = fmaf(S[4 * i + 1], qq.y, o);
        S[4 * i + 2] *= gg.z; p = fmaf(S[4 * i + 2], kk.z, p); o = fmaf(S[4 * i + 2], qq.z, o);
        S[4 * i + 3] *= gg.w; p = fmaf(S[4 * i + 3], kk.w, p); o = fmaf(S[4 * i + 3], qq.w, o);
      }
      float* mine = part + buf * 2 * RG * CW;
      mine[(rg * 2) * CW + col] = p;
      mine[(rg * 2 + 1) * CW + col] = o;
      __syncthreads();                   // two buffers: the one written next was read before this barrier
      p = o = 0.f;
      for (int w = 0; w < RG; ++w) {
        p += mine[(w * 2) * CW + col];
        o += mine[(w * 2 + 1) * CW + col];
      }
      buf ^= 1;
      const float fk = sf[4 * tt + 1], w = sf[4 * tt + 3] * (sv[tt * CW + col] - p * fk), wk = w * fk;
#pragma unroll
      for (int i = 0; i < R / 4; ++i) {
        const float4 kk = k4[i];
        S[4 * i + 0] = fmaf(kk.x, wk, S[4 * i + 0]);
        S[4 * i + 1] = fmaf(kk.y, wk, S[4 * i + 1]);
        S[4 * i + 2] = fmaf(kk.z, wk, S[4 * i + 2]);
        S[4 * i + 3] = fmaf(kk.w, wk, S[4 * i + 3]);
      }
      if (rg == 0) so[tt * CW + col] = fmaf(sf[4 * tt + 2], w, o * sf[4 * tt]);
    }
    __syncthreads();
    for (int tt = wave; tt < nt; tt += waves) {        // a wave a token: sums in lane order, the same whatever the step holds
      float ss = 0.f;
      for (int e = lane; e < dv; e += 64) ss = fmaf(so[tt * CW + e], so[tt * CW + e], ss);
      const float rstd = 1.0f / sqrtf(wave_sum(ss) / (float)dv + a.eps);
      const size_t at = ((size_t)(t0 + tt) * H + h) * dv;
      for (int e = lane; e < dv; e += 64)
        ((TO*)a.out)[at + e] = from_float<TO>(so[tt * CW + e] * rstd * a.norm_weight[e] * a.gate[at + e]);
    }
  }
  if (active) {
#pragma unroll
    for (int i = 0; i < R; ++i)
      if (r0 + i < d) st[(size_t)(r0 + i) * dv] = S[i];
  }
}

// ---- long rows: chunks of 64 tokens.  Scratch of a (chunk, head), padded with zeros to DP channels and VP columns:
constexpr int CH = 64, MS = CH + 4;
struct ChunkArgs {
  DeltaArgs s;
  int max_chunks, units, VP;      // units: rows * max_chunks
  float* W;        // [unit][64][DP]
  float* KT;       // [unit][DP][64]   e^(G_end - G_s) k_s, a channel's tokens side by side
  float* QT;       // [unit][64][DP]   e^G_t q_t
  float* U;        // [unit][64][VP]   U, then w
  float* AQ;       // [unit][64][64]   Q (blocks above the diagonal are not written)
  float* EG;       // [unit][DP]       e^G_end
  float* ST;       // [unit][DP][VP]   S_0
};

// Grids run over the heads first: workgroups go to the eight XCDs in turn, so where H is a multiple of 8 all passes of a head run
// on one XCD and find in its L2 what the pass before left.
#define CHUNK_OF_ROW                                                                                                    \
  const int place = blockIdx.y + gridDim.y * blockIdx.z;                                                                \
  if (place >= p.units) return;                                                                                         \
  const int rr = place / p.max_chunks, ci = place - rr * p.max_chunks, row = a.first_row + rr, h = blockIdx.x;          \
  const int t0 = a.row_start[row] + ci * CH, t_end = a.row_start[row + 1];                                              \
  if (t0 >= t_end) return;                                                                                              \
  const int nt = t_end - t0 < CH ? t_end - t0 : CH;                                                                     \
  const size_t unit = (size_t)place * a.H + h

constexpr int SOLVE_THREADS = 512;

template <int DP>
__global__ void __launch_bounds__(SOLVE_THREADS)
chunk_solve_kernel(ChunkArgs p) {
  constexpr int DS = DP + 4;
  extern __shared__ __align__(16) float lds[];
  float* sk = lds;                   // [64][DS] unit keys
  float* sq = sk + CH * DS;          // unit queries, scaled
  float* sG = sq + CH * DS;          // G in units of log 2
  float* M = sG + CH * DS;           // [64][MS] diag(beta) A, strictly below the diagonal
  float* X = M + CH * MS;            // [64][MS] (I + M)^-1
  float* sb = X + CH * MS;           // [64] beta
  float* so = sb + CH;               // [4][DP] sums of 16 tokens
  const DeltaArgs& a = p.s;
  CHUNK_OF_ROW;
  const int tid = threadIdx.x, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int d = a.d, dv = a.dv, H = a.H, hk = h / a.per_group;
  // ---- unit vectors and decays into the LDS, a wave eight tokens, four at a time
  constexpr int E = (DP + 63) / 64;
#pragma unroll 1
  for (int g4 = 0; g4 < 8; g4 += 4) {
    float q[4][E], k[4][E], l[4][E], qq[4], kk[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int tt = 8 * wave + g4 + u, t = t0 + (tt < nt ? tt : nt - 1);
#pragma unroll
      for (int e = 0; e < E; ++e) {
        const int i = lane + 64 * e, ic = i < d ? i : d - 1;
        q[u][e] = a.q[(size_t)t * a.ld_u + (size_t)hk * d + ic];
        k[u][e] = a.k[(size_t)t * a.ld_u + (size_t)hk * d + ic];
        l[u][e] = a.la[((size_t)t * H + h) * d + ic];
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      qq[u] = kk[u] = 0.f;
#pragma unroll
      for (int e = 0; e < E; ++e)
        if (lane + 64 * e < d) {
          qq[u] = fmaf(q[u][e], q[u][e], qq[u]);
          kk[u] = fmaf(k[u][e], k[u][e], kk[u]);
        }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1)
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        qq[u] += __shfl_xor(qq[u], o, 64);
        kk[u] += __shfl_xor(kk[u], o, 64);
      }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int tt = 8 * wave + g4 + u;
      const float fq = a.q_scale / sqrtf(qq[u] + 1e-6f), fk = 1.0f / sqrtf(kk[u] + 1e-6f);
#pragma unroll
      for (int e = 0; e < E; ++e) {
        const int i = lane + 64 * e;
        const bool in = i < d && tt < nt;
        if (i < DP) {
          sq[tt * DS + i] = in ? q[u][e] * fq : 0.f;
          sk[tt * DS + i] = in ? k[u][e] * fk : 0.f;
          sG[tt * DS + i] = in ? l[u][e] * LOG2E : 0.f;
        }
      }
    }
  }
  if (tid < CH) sb[tid] = tid < nt ? mie_sigmoid(a.beta[(size_t)(t0 + tid) * a.ld + h]) : 0.f;
  for (int e = tid; e < CH * MS; e += SOLVE_THREADS) M[e] = X[e] = 0.f;
  lds_barrier();
  // ---- sums over the tokens: within 16 tokens, then the 16s before them
  {
    const int i = tid % DP, part = tid / DP;
    float run = 0.f, at[16];
    if (part < 4) {
#pragma unroll
      for (int t = 0; t < 16; ++t) at[t] = run += sG[(16 * part + t) * DS + i];
      so[part * DP + i] = run;
    }
    lds_barrier();
    if (part < 4) {
      float before = 0.f;
      for (int w = 0; w < part; ++w) before += so[w * DP + i];
#pragma unroll
      for (int t = 0; t < 16; ++t) sG[(16 * part + t) * DS + i] = before + at[t];
    }
  }
  lds_barrier();
  float* __restrict__ AQ = p.AQ + unit * CH * CH;
  // ---- pairs within 16 tokens: two waves a block, a lane one token t and two tokens s, four channels at a time
  {
    const int t = 16 * (wave >> 1) + 2 * (lane >> 3) + (wave & 1), si = 16 * (wave >> 1) + 2 * (lane & 7);
    float ak[2] = {0.f, 0.f}, aq[2] = {0.f, 0.f};
    if (t >= si) {
#pragma unroll 4
      for (int i = 0; i < DP; i += 4) {
        const f32x4 kt = *reinterpret_cast<const f32x4*>(sk + t * DS + i), qt = *reinterpret_cast<const f32x4*>(sq + t * DS + i);
        const f32x4 gt = *reinterpret_cast<const f32x4*>(sG + t * DS + i);
#pragma unroll
        for (int w = 0; w < 2; ++w) {
          const f32x4 ks = *reinterpret_cast<const f32x4*>(sk + (si + w) * DS + i), gs = *reinterpret_cast<const f32x4*>(sG + (si + w) * DS + i);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const float x = ks[e] * pow2(fminf(gt[e] - gs[e], 0.f));       // a pair above the diagonal is not used
            ak[w] = fmaf(kt[e], x, ak[w]);
            aq[w] = fmaf(qt[e], x, aq[w]);
          }
        }
      }
    }
#pragma unroll
    for (int w = 0; w < 2; ++w) {
      const int s = si + w;
      if (t > s) M[t * MS + s] = sb[t] * ak[w];
      AQ[t * CH + s] = t >= s ? aq[w] : 0.f;
    }
  }
  // ---- tokens of an earlier 16, on the matrix cores: the blocks (x, y) below the diagonal, one a wave
  if (wave < 6) {
    const int blk = wave, x = blk < 3 ? 3 : blk < 5 ? 2 : 1, y = blk < 3 ? blk : blk < 5 ? blk - 3 : 0;
    const float* __restrict__ ref = sG + (16 * x - 1) * DS;
    f32x4 acc_k = f32x4{0.f, 0.f, 0.f, 0.f}, acc_q = acc_k;
#pragma unroll 2
    for (int i = 4 * g; i < DP; i += 16) {
      const f32x4 r = *reinterpret_cast<const f32x4*>(ref + i);
      const f32x4 gt = *reinterpret_cast<const f32x4*>(sG + (16 * x + n) * DS + i), gs = *reinterpret_cast<const f32x4*>(sG + (16 * y + n) * DS + i);
      const f32x4 kt = *reinterpret_cast<const f32x4*>(sk + (16 * x + n) * DS + i), qt = *reinterpret_cast<const f32x4*>(sq + (16 * x + n) * DS + i);
      const f32x4 ks = *reinterpret_cast<const f32x4*>(sk + (16 * y + n) * DS + i);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float et = pow2(gt[e] - r[e]), right = ks[e] * pow2(r[e] - gs[e]);
        acc_k = mfma4(kt[e] * et, right, acc_k);
        acc_q = mfma4(qt[e] * et, right, acc_q);
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = 16 * x + 4 * g + e, s = 16 * y + n;
      M[t * MS + s] = sb[t] * acc_k[e];
      AQ[t * CH + s] = acc_q[e];
    }
  }
  lds_barrier();
  // ---- the inverse: diagonal blocks by substitution, a lane a column
  if (wave < 4) {
    const float* __restrict__ m = M + 16 * wave * MS + 16 * wave;
    float x[16];
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      float v = t == n ? 1.f : 0.f;
#pragma unroll
      for (int s = 0; s < t; ++s) v = fmaf(-m[t * MS + s], x[s], v);
      x[t] = v;
    }
    if (g == 0) {
#pragma unroll
      for (int t = 0; t < 16; ++t) X[(16 * wave + t) * MS + 16 * wave + n] = x[t];
    }
  }
  lds_barrier();
#pragma unroll 1
  for (int dist = 1; dist < 4; ++dist) {
    if (wave + dist < 4) {
      const int x = wave + dist, y = wave;
      f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
      for (int c = y; c < x; ++c) {
        const f32x4 m = *reinterpret_cast<const f32x4*>(M + (16 * x + n) * MS + 16 * c + 4 * g);
#pragma unroll
        for (int j = 0; j < 4; ++j) s = mfma4(m[j], X[(16 * c + 4 * g + j) * MS + 16 * y + n], s);
      }
      // a result's rows 4 g + e are what the next product's operand wants as its rows 4 g + j
      const f32x4 xx = *reinterpret_cast<const f32x4*>(X + (16 * x + n) * MS + 16 * x + 4 * g);
      f32x4 r = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < 4; ++j) r = mfma4(xx[j], s[j], r);
#pragma unroll
      for (int e = 0; e < 4; ++e) X[(16 * x + 4 * g + e) * MS + 16 * y + n] = -r[e];
    }
    lds_barrier();
  }
  // ---- W and U: a wave every eighth 16 columns
  float* __restrict__ W = p.W + unit * CH * DP;
  float* __restrict__ U = p.U + unit * CH * p.VP;
  const int col_tiles = DP / 16 + p.VP / 16;
  for (int ct = wave; ct < col_tiles; ct += SOLVE_THREADS / 64) {
    const bool of_w = ct < DP / 16;
    const int c = (of_w ? ct : ct - DP / 16) * 16 + n;
    f32x4 acc[4];
#pragma unroll
    for (int x = 0; x < 4; ++x) acc[x] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int y = 0; y < 4; ++y) {
      float b[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int s = 16 * y + 4 * g + j;
        if (of_w) b[j] = sk[s * DS + c] * pow2(sG[s * DS + c]) * sb[s];
        else b[j] = c < dv ? a.v[(size_t)(t0 + (s < nt ? s : nt - 1)) * a.ld_u + (size_t)h * dv + c] * sb[s] : 0.f;
      }
#pragma unroll
      for (int x = y; x < 4; ++x) {
        const f32x4 m = *reinterpret_cast<const f32x4*>(X + (16 * x + n) * MS + 16 * y + 4 * g);
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[x] = mfma4(m[j], b[j], acc[x]);
      }
    }
#pragma unroll
    for (int x = 0; x < 4; ++x)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = 16 * x + 4 * g + e;
        if (of_w) W[(size_t)t * DP + c] = acc[x][e];
        else U[(size_t)t * p.VP + c] = acc[x][e];
      }
  }
  // ---- what the other passes want of keys and queries
  float* __restrict__ KT = p.KT + unit * DP * CH;
  float* __restrict__ QT = p.QT + unit * CH * DP;
  for (int e = tid; e < CH * DP; e += SOLVE_THREADS) {
    const int s = e & (CH - 1), i = e / CH;
    KT[e] = sk[s * DS + i] * pow2(sG[(CH - 1) * DS + i] - sG[s * DS + i]);
    const int t = e / DP, j = e % DP;
    QT[e] = sq[t * DS + j] * pow2(sG[t * DS + j]);
  }
  for (int i = tid; i < DP; i += SOLVE_THREADS) p.EG[unit * DP + i] = pow2(sG[(CH - 1) * DS + i]);
}

// (2) grid (H, rows, VP / 16): the workgroups of a head are H apart, on one XCD where H is a multiple of 8
template <int DP>
__global__ void __launch_bounds__(256)
chunk_fold_kernel(ChunkArgs p) {
  constexpr int CS = 20, KB = DP / 16, RT = (KB + 3) / 4;       // RT: 16-row tiles of the state a wave owns
  __shared__ __align__(16) float sS[DP * CS], sU[CH * CS];
  const DeltaArgs& a = p.s;
  const int h = blockIdx.x, rr = blockIdx.y, row = a.first_row + rr, c0 = blockIdx.z * 16;
  const int tid = threadIdx.x, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int d = a.d, dv = a.dv, H = a.H, VP = p.VP, col = c0 + n;
  const int chunks = (a.row_start[row + 1] - a.row_start[row] + CH - 1) / CH;
  float* __restrict__ st = a.state + ((size_t)a.slots[row] * H + h) * d * dv;
  f32x4 S[RT];
#pragma unroll
  for (int i = 0; i < RT; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int r = 16 * (wave + 4 * i) + 4 * g + e;
      S[i][e] = r < d && col < dv ? st[(size_t)r * dv + col] : 0.f;
    }
  struct Ahead {                          // what a chunk needs, asked for two chunks ahead
    f32x4 w[KB], kt[RT][4], eg[RT];
    float u[4];
  };
  auto unit_of = [&](int c) { return ((size_t)rr * p.max_chunks + c) * H + h; };
  auto fetch_first = [&](Ahead& A, int c) {         // of the first product: W and U
    c = c < chunks ? c : chunks - 1;
    const float* __restrict__ W = p.W + unit_of(c) * CH * DP + (size_t)(16 * wave + n) * DP + 4 * g;
#pragma unroll
    for (int kb = 0; kb < KB; ++kb) A.w[kb] = *reinterpret_cast<const f32x4*>(W + 16 * kb);
    const float* __restrict__ U = p.U + unit_of(c) * CH * VP + col;
#pragma unroll
    for (int e = 0; e < 4; ++e) A.u[e] = U[(size_t)(16 * wave + 4 * g + e) * VP];
  };
  auto fetch_second = [&](Ahead& A, int c) {        // of the second: keys and the chunk's decay
    c = c < chunks ? c : chunks - 1;
#pragma unroll
    for (int i = 0; i < RT; ++i) {
      const int tile = wave + 4 * i < KB ? wave + 4 * i : KB - 1;
      const float* __restrict__ K = p.KT + unit_of(c) * DP * CH + (size_t)(16 * tile + n) * CH + 4 * g;
#pragma unroll
      for (int sb = 0; sb < 4; ++sb) A.kt[i][sb] = *reinterpret_cast<const f32x4*>(K + 16 * sb);
      A.eg[i] = *reinterpret_cast<const f32x4*>(p.EG + unit_of(c) * DP + 16 * tile + 4 * g);
    }
  };
  // What a later chunk needs is asked for without a condition (the last chunk's once more at the end): the waits below then count
  // exactly what was issued since, and never wait for more than they need.
  auto step = [&](Ahead& A, int c) {
    float* __restrict__ ST = p.ST + unit_of(c) * DP * VP + col;
#pragma unroll
    for (int i = 0; i < RT; ++i)
      if (KB % 4 == 0 || wave + 4 * i < KB) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int r = 16 * (wave + 4 * i) + 4 * g + e;
          sS[r * CS + n] = S[i][e];
          ST[(size_t)r * VP] = S[i][e];
        }
      }
    lds_barrier();
    f32x4 acc[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
    float right[KB][4];                   // all of it asked for before the first product
#pragma unroll
    for (int kb = 0; kb < KB; ++kb)
#pragma unroll
      for (int j = 0; j < 4; ++j) right[kb][j] = sS[(16 * kb + 4 * g + j) * CS + n];
    asm volatile("" ::: "memory");
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int kb = 0; kb < KB; ++kb) acc[kb & 1] = mfma4(A.w[kb][j], right[kb][j], acc[kb & 1]);
    float* __restrict__ U = p.U + unit_of(c) * CH * VP + col;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = 16 * wave + 4 * g + e;
      const float x = A.u[e] - (acc[0][e] + acc[1][e]);
      sU[t * CS + n] = x;
      U[(size_t)t * VP] = x;
    }
    fetch_first(A, c + 2);
    lds_barrier();
    float down[4][4];
#pragma unroll
    for (int sb = 0; sb < 4; ++sb)
#pragma unroll
      for (int j = 0; j < 4; ++j) down[sb][j] = sU[(16 * sb + 4 * g + j) * CS + n];
    asm volatile("" ::: "memory");
#pragma unroll
    for (int i = 0; i < RT; ++i) S[i] = S[i] * A.eg[i];
#pragma unroll
    for (int sb = 0; sb < 4; ++sb)
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int i = 0; i < RT; ++i) S[i] = mfma4(A.kt[i][sb][j], down[sb][j], S[i]);
    fetch_second(A, c + 2);
  };
  Ahead even, odd;
  fetch_first(even, 0);                   // in the order in which the steps will ask, so that the waits agree
  asm volatile("" ::: "memory");
  fetch_second(even, 0);
  asm volatile("" ::: "memory");
  fetch_first(odd, 1);
  asm volatile("" ::: "memory");
  fetch_second(odd, 1);
  asm volatile("" ::: "memory");
  for (int c = 0; c < chunks; c += 2) {
    step(even, c);
    if (c + 1 < chunks) step(odd, c + 1);
  }
#pragma unroll
  for (int i = 0; i < RT; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int r = 16 * (wave + 4 * i) + 4 * g + e;
      if (r < d && col < dv) st[(size_t)r * dv + col] = S[i][e];
    }
}

// (3) a wave 16 tokens of all columns: o = (e^G q) S_0, then Q w, 32 rows of the right operand in the LDS at a time
template <int DP, int NV, typename TO>
__global__ void __launch_bounds__(256)
chunk_outputs_kernel(ChunkArgs p) {
  constexpr int VP = 16 * NV, VS = VP + 4, PIECES = DP / 32 + 2;
  __shared__ __align__(16) float piece[32 * VS];
  const DeltaArgs& a = p.s;
  CHUNK_OF_ROW;
  const int tid = threadIdx.x, lane = tid & 63, n = lane & 15, g = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const float* __restrict__ ST = p.ST + unit * DP * VP;
  const float* __restrict__ U = p.U + unit * CH * VP;
  const float* __restrict__ QT = p.QT + unit * CH * DP + (size_t)(16 * wave + n) * DP + 4 * g;
  const float* __restrict__ AQ = p.AQ + unit * CH * CH + (size_t)(16 * wave + n) * CH + 4 * g;
  f32x4 O[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) O[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  constexpr int PER = 32 * VP / 4 / 256;             // 16-byte parts a thread brings of a piece
  f32x4 next[PER > 0 ? PER : 1], ops[2], ops_next[2];
  auto fetch = [&](int pc) {
    const float* __restrict__ src = pc < DP / 32 ? ST + (size_t)pc * 32 * VP : U + (size_t)(pc - DP / 32) * 32 * VP;
#pragma unroll
    for (int i = 0; i < PER; ++i) next[i] = *reinterpret_cast<const f32x4*>(src + 4 * (tid + 256 * i));
#pragma unroll
    for (int k = 0; k < 2; ++k)
      ops_next[k] = *reinterpret_cast<const f32x4*>(pc < DP / 32 ? QT + 32 * pc + 16 * k : AQ + 32 * (pc - DP / 32) + 16 * k);
  };
  fetch(0);
#pragma unroll 1
  for (int pc = 0; pc < PIECES; ++pc) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int e = tid + 256 * i, r = e / (VP / 4), c = e % (VP / 4);
      *reinterpret_cast<f32x4*>(piece + r * VS + 4 * c) = next[i];
    }
    ops[0] = ops_next[0];
    ops[1] = ops_next[1];
    __syncthreads();
    if (pc + 1 < PIECES) fetch(pc + 1);
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      if (pc >= DP / 32 && 2 * (pc - DP / 32) + k > wave) continue;      // blocks above the diagonal
#pragma unroll
      for (int i = 0; i < NV; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) O[i] = mfma4(ops[k][j], piece[(16 * k + 4 * g + j) * VS + 16 * i + n], O[i]);
    }
  }
  // the norm over a head's numbers: a token's are spread over 16 lanes
  const int dv = a.dv, H = a.H;
  float ss[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    ss[e] = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) ss[e] = fmaf(O[i][e], O[i][e], ss[e]);
  }
#pragma unroll
  for (int o = 8; o > 0; o >>= 1)
#pragma unroll
    for (int e = 0; e < 4; ++e) ss[e] += __shfl_xor(ss[e], o, 64);
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int tt = 16 * wave + 4 * g + e;
    if (tt >= nt) continue;
    const float rstd = 1.0f / sqrtf(ss[e] / (float)dv + a.eps);
    const size_t at = ((size_t)(t0 + tt) * H + h) * dv;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = 16 * i + n;
      if (c < dv) ((TO*)a.out)[at + c] = from_float<TO>(O[i][e] * rstd * a.norm_weight[c] * a.gate[at + c]);
    }
  }
}

MIE_EXPORT const char* gated_delta_last_error() { return g_mie_error; }

template <typename TO>
static int scan_launch(const DeltaArgs& a, int rows, hipStream_t s) {
  const int CB = (a.dv + 63) / 64;
  int R = 8;
  while (R < 64 && CB * ((a.d + R - 1) / R) > 16) R *= 2;
  const int RG = (a.d + R - 1) / R, waves = CB * RG;
  if (waves > 16) MIE_FAIL("gated_delta: states of %d x %d do not fit a workgroup", a.d, a.dv);
  const size_t lds = ((size_t)3 * TB * RG * R + (size_t)4 * RG * CB * 64 + (size_t)2 * TB * CB * 64 + 4 * TB) * sizeof(float);
  if (lds > 64 * 1024) MIE_FAIL("gated_delta: %zu bytes of LDS", lds);
#define SCAN(R_) hipLaunchKernelGGL((scan_kernel<R_, TO>), dim3(rows, a.H), dim3(waves * 64), lds, s, a, CB)
  if (R == 8) SCAN(8);
  else if (R == 16) SCAN(16);
  else if (R == 32) SCAN(32);
  else SCAN(64);
#undef SCAN
  MIE_CHECK_LAUNCH("gated_delta (scan)");
  return 0;
}

template <int DP, typename TO>
static int chunks_launch(const ChunkArgs& p, int rows, hipStream_t s) {
  const size_t lds = ((size_t)3 * CH * (DP + 4) + (size_t)2 * CH * MS + CH + 4 * DP) * sizeof(float);
  static bool allowed[64] = {};
  int dev = 0;
  if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 64) MIE_FAIL("gated_delta: no current device");
  if (lds > 64 * 1024 && !allowed[dev]) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(chunk_solve_kernel<DP>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) MIE_FAIL("gated_delta: %zu bytes of LDS refused: %s", lds, hipGetErrorString(e));
    allowed[dev] = true;
  }
  const dim3 units(p.s.H, p.units < 32768 ? p.units : 32768, (p.units + 32767) / 32768);
  hipLaunchKernelGGL(chunk_solve_kernel<DP>, units, dim3(SOLVE_THREADS), lds, s, p);
  MIE_CHECK_LAUNCH("gated_delta (chunks: solve)");
  hipLaunchKernelGGL(chunk_fold_kernel<DP>, dim3(p.s.H, rows, p.VP / 16), dim3(256), 0, s, p);
  MIE_CHECK_LAUNCH("gated_delta (chunks: fold)");
  switch (p.VP) {
#define OUTPUTS(NV_) case 16 * NV_: hipLaunchKernelGGL((chunk_outputs_kernel<DP, NV_, TO>), units, dim3(256), 0, s, p); break
    OUTPUTS(2);
    OUTPUTS(4);
    OUTPUTS(8);
    OUTPUTS(16);
#undef OUTPUTS
    default: MIE_FAIL("gated_delta: columns padded to %d", p.VP);
  }
  MIE_CHECK_LAUNCH("gated_delta (chunks: outputs)");
  return 0;
}

// floats of scratch a (chunk, head) takes; DP and VP: sizes padded to 32, 64, 128 (columns also 256)
MIE_EXPORT int mie_gated_delta_unit_floats(int DP, int VP) { return 3 * CH * DP + CH * VP + CH * CH + DP + DP * VP; }

// la, gate: scratch of tokens * H * d and tokens * H * dv floats.  w_decay [H d, ra], w_gate [H dv, rg], ra and rg multiples of 16 (zero
// columns beyond the inner sizes), and so are the columns decay_col and gate_col of the sums and the rows' distance ld; the columns up
// to the padded inner sizes exist.  Rows [0, whole_rows) run token by token, the others in chunks of 64 tokens, at most max_chunks
// a row, with scratch of (rows - whole_rows) * max_chunks * H * mie_gated_delta_unit_floats(DP, VP) floats.
MIE_EXPORT int mie_gated_delta(const float* u, long ld_u, int q_col, int k_col, int v_col, const float* sums, long ld, int beta_col,
                               int decay_col, int gate_col, const float* w_decay, int ra, const float* rate, const float* decay_bias,
                               const float* w_gate, int rg, float q_scale, const float* norm_weight, float eps, float* state,
                               const int* row_start, const int* slots, float* la, float* gate, void* out, int out_dtype, int tokens,
                               int rows, int whole_rows, int H, int G, int d, int dv, int max_chunks, int DP, int VP, float* scratch,
                               hipStream_t s) {
  if (tokens <= 0 || rows <= 0) return 0;
  if (H <= 0 || G <= 0 || H % G || d <= 0 || dv <= 0 || d > 256 || dv > 256)
    MIE_FAIL("gated_delta: %d heads on %d query/key heads of %d x %d (up to 256 x 256)", H, G, d, dv);
  if (H > 65535 || rows > 65535) MIE_FAIL("gated_delta: %d heads, %d rows are beyond the grid", H, rows);
  if (ra < 16 || ra % 16 || rg < 16 || rg % 16 || decay_col % 16 || gate_col % 16 || ld % 16 || (uintptr_t)sums % 16 ||
      (uintptr_t)w_decay % 16 || (uintptr_t)w_gate % 16)
    MIE_FAIL("gated_delta: inner sizes %d and %d, columns %d and %d, rows of %ld (multiples of 16)", ra, rg, decay_col, gate_col, ld);
  if (ld < (long)decay_col + ra || ld < (long)gate_col + rg || ld < (long)beta_col + H) MIE_FAIL("gated_delta: columns beyond the rows of %ld", ld);
  if (out_dtype != MIE_F32 && out_dtype != MIE_BF16) MIE_FAIL("gated_delta: dtype code %d", out_dtype);
  if (!u || !rate || !decay_bias || !norm_weight || !state || !row_start || !slots || !la || !gate || !out) MIE_FAIL("gated_delta: a null operand");
  if (whole_rows < 0 || whole_rows > rows) MIE_FAIL("gated_delta: %d of %d rows whole", whole_rows, rows);
  const int decay_blocks = (H * d + 63) / 64, blocks = decay_blocks + (H * dv + 63) / 64;
  if (blocks > 65535) MIE_FAIL("gated_delta: %d channels are beyond the grid", H * (d + dv));
#define LOW_RANK(TT_)                                                                                                                     \
  hipLaunchKernelGGL(low_rank_kernel<TT_>, dim3((tokens + 16 * TT_ - 1) / (16 * TT_), blocks), dim3(256), 0, s, sums, ld, decay_col, gate_col, \
                     w_decay, ra, w_gate, rg, rate, decay_bias, la, gate, tokens, H, d, dv, decay_blocks)
  if (tokens <= 256) LOW_RANK(1);
  else LOW_RANK(4);
#undef LOW_RANK
  MIE_CHECK_LAUNCH("gated_delta (decays and gates)");
  DeltaArgs a{u + q_col, u + k_col, u + v_col, ld_u, H / G, sums + beta_col, ld, la, gate, norm_weight, eps, q_scale, state,
              row_start, slots, out, H, d, dv, 0};
  if (whole_rows > 0) {
    const int rc = out_dtype == MIE_F32 ? scan_launch<float>(a, whole_rows, s) : scan_launch<bf16>(a, whole_rows, s);
    if (rc) return rc;
  }
  if (whole_rows == rows) return 0;
  const int n = rows - whole_rows;
  if (max_chunks < 1 || !scratch || DP < d || VP < dv || (uintptr_t)scratch % 16) MIE_FAIL("gated_delta: chunks, %d a row, padded to %d x %d", max_chunks, DP, VP);
  if ((long)n * max_chunks > 2147483647L) MIE_FAIL("gated_delta: %d rows of %d chunks are beyond the grid", n, max_chunks);
  a.first_row = whole_rows;
  const size_t units = (size_t)n * max_chunks * H;      // of scratch
  ChunkArgs p{a, max_chunks, n * max_chunks, VP, nullptr, nullptr, nullptr, nullptr, nullptr, nullptr, nullptr};
  float* at = scratch;
  auto take = [&](size_t per) { float* q = at; at += units * per; return q; };
  p.W = take((size_t)CH * DP);
  p.KT = take((size_t)CH * DP);
  p.QT = take((size_t)CH * DP);
  p.U = take((size_t)CH * VP);
  p.AQ = take((size_t)CH * CH);
  p.ST = take((size_t)DP * VP);
  p.EG = take((size_t)DP);
#define CHUNKS(DP_) return out_dtype == MIE_F32 ? chunks_launch<DP_, float>(p, n, s) : chunks_launch<DP_, bf16>(p, n, s)
  if (DP == 32) CHUNKS(32);
  if (DP == 64) CHUNKS(64);
  if (DP == 128) CHUNKS(128);
#undef CHUNKS
  MIE_FAIL("gated_delta: channels padded to %d", DP);
}
