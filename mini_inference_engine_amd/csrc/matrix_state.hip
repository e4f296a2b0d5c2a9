// Recurrences whose state a head is a matrix with one decay a token: S [d, dv] <- e^la S + c k v^T, o = S^T q, over a step's
// rows, the request's state in its slot.  Everything is 32-bit.  Two mixers use it:
//   state space (Mamba-2): k = B, q = C (shared by the heads of a group), v = x, la = -rate dt, c = dt, dt = softplus(.);
//     y = o + skip x, then y silu(z), RMS-normed in equal parts of all heads' numbers, times a weight.
//   matrix memory (mLSTM): la = f + m - m', c = exp(i - m') with capped log gates i, f and the running maximum
//     m' = max(f + m, i); a normaliser n [d] runs along (n <- e^la n + c k); o / (max(|n . q|, exp(-m')) + 1e-6), each head
//     over its root mean square, times a weight and sigmoid(g).
//
// ssm_prepare / mlstm_prepare: la and c of every (token, head).  The maximum is a scan: a token maps m to max(f + m, i), two
//     tokens after one another map it to max(f1 + f2 + m, max(f2 + i1, i2)), so a wave takes 64 tokens of a (row, head) at a
//     time with six exchanges.
// matrix_scan: a workgroup a (row, head, 64 columns of the state), tokens in order.  A lane is a column, a wave owns R rows of
//     it in registers; q, k and decays of a few tokens come in through the LDS at a time, the waves' shares of an output are
//     added in the order of the rows.
// ssm_finish / mlstm_finish: what follows the recurrence, rounded once.
//
// Long rows run in chunks of 64 tokens side by side, on the matrix cores in 32-bit (v_mfma_f32_16x16x4_f32).  With A_t the sum
// of la over a chunk's tokens up to t, and S_0 the state the chunk starts from,
//     S_end = e^A_end S_0 + B,   B = sum_s e^(A_end - A_s) c_s k_s v_s^T
//     o_t = e^A_t S_0^T q_t + sum_(s <= t) e^(A_t - A_s) c_s (q_t . k_s) v_s
// so that (1) chunk_sums computes every chunk's B, (2) chunk_fold walks a row's chunks, a thread an entry: it leaves S_0 of
// every chunk where B was and the end of the row in its slot, (3) chunk_outputs computes the outputs, three products a
// (chunk, head, columns).  All exponents are <= 0.  The normaliser takes the same way with ones for v.
#include "common.hpp"

__device__ __forceinline__ float softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }
__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }

// dt columns of the sums -> la, c [T, H]
__global__ void __launch_bounds__(256)
ssm_prepare_kernel(const float* __restrict__ dt_in, long ld, const float* __restrict__ dt_bias, const float* __restrict__ rate,
                   float* __restrict__ la, float* __restrict__ c, int tokens, int H) {
  const int e = blockIdx.x * 256 + threadIdx.x;
  if (e >= tokens * H) return;
  const int t = e / H, h = e - t * H;
  const float dt = softplus(dt_in[(size_t)t * ld + h] + dt_bias[h]);
  la[e] = -rate[h] * dt;
  c[e] = dt;
}

// gate columns -> la, c and exp(-m) [T, H]; the slot's maximum moves on.  A workgroup a (row, head), a wave 64 tokens of it at
// a time: every wave sums up its own tokens, then joins what the waves before it found.
__global__ void __launch_bounds__(1024)
mlstm_prepare_kernel(const float* __restrict__ gi, const float* __restrict__ gf, long ld, const float* __restrict__ i_bias,
                     const float* __restrict__ f_bias, float cap, float* __restrict__ maximum, const int* __restrict__ row_start,
                     const int* __restrict__ slots, float* __restrict__ la, float* __restrict__ c, float* __restrict__ low, int H) {
  __shared__ float tot_f[16], tot_i[16];
  const int row = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, waves = blockDim.x >> 6;
  const int begin = row_start[row], end = row_start[row + 1];
  float m0 = maximum[(size_t)slots[row] * H + h];
  const float ib = i_bias[h], fb = f_bias[h], inv_cap = 1.0f / cap;
  for (int t0 = begin; t0 < end; t0 += 64 * waves) {
    const int t = t0 + 64 * wave + lane;
    const bool ok = t < end;
    const size_t at = (size_t)(ok ? t : end - 1) * ld + h;
    const float i = ok ? cap * tanhf((gi[at] + ib) * inv_cap) : -INFINITY;
    const float f = ok ? log_sigmoid(cap * tanhf((gf[at] + fb) * inv_cap)) : 0.f;
    float F = f, I = i;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float F1 = __shfl_up(F, o, 64), I1 = __shfl_up(I, o, 64);
      if (lane >= o) {
        I = fmaxf(F + I1, I);
        F += F1;
      }
    }
    if (waves > 1) {
      __syncthreads();                       // the totals of the round before have been read
      if (lane == 63) {
        tot_f[wave] = F;
        tot_i[wave] = I;
      }
      __syncthreads();
    }
    float start = m0;                        // the maximum before this wave's tokens, and behind the last wave's
    for (int w = 0; w < wave; ++w) start = fmaxf(tot_f[w] + start, tot_i[w]);
    const float m = fmaxf(F + start, I);
    float before = __shfl_up(m, 1, 64);
    if (lane == 0) before = start;
    if (waves > 1) {
      for (int w = wave; w < waves; ++w) start = fmaxf(tot_f[w] + start, tot_i[w]);
      m0 = start;
    } else {
      m0 = __shfl(m, 63, 64);                // tokens beyond the row's end pass the maximum on
    }
    if (ok) {
      const size_t e = (size_t)t * H + h;
      la[e] = fminf(f + before - m, 0.f);
      c[e] = expf(i - m);
      low[e] = expf(-m);
    }
  }
  if (threadIdx.x == 0) maximum[(size_t)slots[row] * H + h] = m0;
}

struct ScanArgs {
  const float* q; const float* k; const float* v; long ld_qk, ld_v;
  int per_group;                 // heads that share a head of q and k
  float q_scale;
  const float* la; const float* c;           // [T, H]
  float* state;                  // [slots, H, d, dv]
  float* normaliser;             // [slots, H, d] or null
  const int* row_start; const int* slots;
  float* o;                      // [T, H, dv]
  float* nq;                     // [T, H] (with a normaliser)
  int H, d, dv;
};

template <int R, int TB>
__global__ void __launch_bounds__(1024)
matrix_scan_kernel(ScanArgs a) {
  extern __shared__ __align__(16) float lds[];
  const int d = a.d, dv = a.dv, H = a.H;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, waves = blockDim.x >> 6, DP = waves * R;
  float* sq = lds;                       // [TB][DP]
  float* sk = sq + TB * DP;              // [TB][DP], times c
  float* part = sk + TB * DP;            // [waves][TB][64]
  float* pn = part + waves * TB * 64;    // [waves][TB]
  float* sa = pn + waves * TB;           // [TB] decays
  const int row = blockIdx.x, h = blockIdx.y, col = blockIdx.z * 64 + lane, g = h / a.per_group;
  const int begin = a.row_start[row], end = a.row_start[row + 1], slot = a.slots[row];
  const bool active = col < dv, with_n = a.normaliser && blockIdx.z == 0;
  float* __restrict__ st = a.state + ((size_t)slot * H + h) * d * dv + (active ? col : 0);
  const int r0 = wave * R;
  float S[R];
#pragma unroll
  for (int i = 0; i < R; ++i) S[i] = active && r0 + i < d ? st[(size_t)(r0 + i) * dv] : 0.f;
  float* nrm = with_n ? a.normaliser + ((size_t)slot * H + h) * d : nullptr;
  float n = with_n && lane < R && r0 + lane < d ? nrm[r0 + lane] : 0.f;
  for (int t0 = begin; t0 < end; t0 += TB) {
    const int nt = end - t0 < TB ? end - t0 : TB;
    __syncthreads();
    for (int e = tid; e < nt * DP; e += blockDim.x) {
      const int tt = e / DP, i = e - tt * DP;
      const size_t at = (size_t)(t0 + tt) * a.ld_qk + (size_t)g * d + i;
      sq[e] = i < d ? a.q[at] * a.q_scale : 0.f;
      sk[e] = i < d ? a.k[at] * a.c[(size_t)(t0 + tt) * H + h] : 0.f;
    }
    if (tid < nt) sa[tid] = expf(a.la[(size_t)(t0 + tid) * H + h]);
    float v[TB];
#pragma unroll
    for (int tt = 0; tt < TB; ++tt) v[tt] = active && tt < nt ? a.v[(size_t)(t0 + tt) * a.ld_v + (size_t)h * dv + col] : 0.f;
    __syncthreads();
#pragma unroll
    for (int tt = 0; tt < TB; ++tt) {
      if (tt >= nt) break;
      const float decay = sa[tt];
      const float4* q4 = reinterpret_cast<const float4*>(sq + tt * DP + r0);
      const float4* k4 = reinterpret_cast<const float4*>(sk + tt * DP + r0);
      float o = 0.f;
#pragma unroll
      for (int i = 0; i < R / 4; ++i) {
        const float4 qq = q4[i], kk = k4[i];
        S[4 * i + 0] = fmaf(kk.x, v[tt], decay * S[4 * i + 0]); o = fmaf(S[4 * i + 0], qq.x, o);
        S[4 * i + 1] = fmaf(kk.y, v[tt], decay * S[4 * i + 1]); o = fmaf(S[4 * i + 1], qq.y, o);
        S[4 * i + 2] = fmaf(kk.z, v[tt], decay * S[4 * i + 2]); o = fmaf(S[4 * i + 2], qq.z, o);
        S[4 * i + 3] = fmaf(kk.w, v[tt], decay * S[4 * i + 3]); o = fmaf(S[4 * i + 3], qq.w, o);
      }
      part[(wave * TB + tt) * 64 + lane] = o;
      if (with_n) {
        float p = 0.f;
        if (lane < R) {
          n = fmaf(decay, n, sk[tt * DP + r0 + lane]);
          p = n * sq[tt * DP + r0 + lane];
        }
        p = wave_sum(p);
        if (lane == 0) pn[wave * TB + tt] = p;
      }
    }
    __syncthreads();
    for (int e = tid; e < nt * 64; e += blockDim.x) {
      const int tt = e >> 6, l = e & 63, cc = blockIdx.z * 64 + l;
      float o = 0.f;
      for (int w = 0; w < waves; ++w) o += part[(w * TB + tt) * 64 + l];
      if (cc < dv) a.o[((size_t)(t0 + tt) * H + h) * dv + cc] = o;
    }
    if (with_n && tid < nt) {
      float s = 0.f;
      for (int w = 0; w < waves; ++w) s += pn[w * TB + tid];
      a.nq[(size_t)(t0 + tid) * H + h] = s;
    }
  }
  if (active) {
#pragma unroll
    for (int i = 0; i < R; ++i)
      if (r0 + i < d) st[(size_t)(r0 + i) * dv] = S[i];
  }
  if (with_n && lane < R && r0 + lane < d) nrm[r0 + lane] = n;
}

// ---- long rows: chunks of 64 tokens side by side
typedef float f32x4 __attribute__((ext_vector_type(4)));
constexpr int CH = 64;            // tokens a chunk
constexpr int DB = 32;            // state rows chunk_outputs takes at a time
constexpr int QS = DB + 4;        // a row of q or k in the LDS (reads of four numbers by 16 rows meet no bank twice)

struct ChunkArgs {
  ScanArgs s;
  int max_chunks, vec;            // vec: rows and pieces of q, k, v, states start on 16 bytes
  float* starts;                  // [rows * max_chunks, H, d, dv]: B, then S_0
  float* n_starts;                // [rows * max_chunks, H, d] (with a normaliser)
  float* ends;                    // [rows * max_chunks, H]: A_end
};

// four numbers of a row from p + i on, zeros where i is at n or beyond
__device__ __forceinline__ f32x4 load4(const float* __restrict__ p, int i, int n, bool vec) {
  f32x4 r = {0.f, 0.f, 0.f, 0.f};
  if (vec) {
    if (i < n) r = *reinterpret_cast<const f32x4*>(p + i);       // n is a multiple of 4
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (i + e < n) r[e] = p[i + e];
  }
  return r;
}

// the chunk's sums A and inputs' factors c into the LDS, by the first wave: A_t inclusive, tokens beyond the end add nothing
__device__ __forceinline__ void chunk_decays(const ScanArgs& a, int t0, int nt, int h, float* A, float* c) {
  if (threadIdx.x < 64) {
    const int l = threadIdx.x;
    const size_t e = (size_t)(t0 + (l < nt ? l : nt - 1)) * a.H + h;
    float x = l < nt ? a.la[e] : 0.f;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float y = __shfl_up(x, o, 64);
      if (l >= o) x += y;
    }
    A[l] = x;
    c[l] = l < nt ? a.c[e] : 0.f;
  }
}

#define CHUNK_OF_ROW                                                          \
  const int row = blockIdx.x / p.max_chunks, ci = blockIdx.x - row * p.max_chunks; \
  const int t0 = a.row_start[row] + ci * CH, t_end = a.row_start[row + 1];    \
  if (t0 >= t_end) return;                                                    \
  const int nt = t_end - t0 < CH ? t_end - t0 : CH

// (1) B of 64 state rows and 16 NT columns: A operand k (times its factor) by state row, B operand v; a wave 16 state rows
template <int NT>
__global__ void __launch_bounds__(256)
chunk_sums_kernel(ChunkArgs p, int row_tiles) {
  constexpr int VS = 16 * NT + 4, KST = 64 + 4;
  __shared__ __align__(16) float sk[CH * KST], sv[CH * VS], A[CH], cc[CH];
  const ScanArgs& a = p.s;
  CHUNK_OF_ROW;
  const int h = blockIdx.y, dt = blockIdx.z % row_tiles, vt = blockIdx.z / row_tiles;
  const int d0 = dt * 64, v0 = vt * 16 * NT, tid = threadIdx.x;
  const float* __restrict__ kp = a.k + (size_t)t0 * a.ld_qk + (size_t)(h / a.per_group) * a.d;
  const float* __restrict__ vp = a.v + (size_t)t0 * a.ld_v + (size_t)h * a.dv;
  chunk_decays(a, t0, nt, h, A, cc);
  f32x4 kr[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int e = tid + 256 * i, t = e >> 4;
    kr[i] = load4(kp + (size_t)(t < nt ? t : nt - 1) * a.ld_qk, d0 + 4 * (e & 15), a.d, p.vec);
  }
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int e = tid + 256 * i, t = e / (4 * NT), c = 4 * (e % (4 * NT));
    f32x4 v = load4(vp + (size_t)(t < nt ? t : nt - 1) * a.ld_v, v0 + c, a.dv, p.vec);
    *reinterpret_cast<f32x4*>(sv + t * VS + c) = v;
  }
  __syncthreads();                              // A and cc are there
  const float end = A[CH - 1];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int e = tid + 256 * i, t = e >> 4;
    *reinterpret_cast<f32x4*>(sk + t * KST + 4 * (e & 15)) = kr[i] * (expf(end - A[t]) * cc[t]);      // cc 0 beyond the end
  }
  __syncthreads();
  const int lane = tid & 63, wave = tid >> 6, n = lane & 15, g = lane >> 4;
  f32x4 acc[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int t = g; t < CH; t += 4) {
    const float kk = sk[t * KST + 16 * wave + n];
#pragma unroll
    for (int i = 0; i < NT; ++i) acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(kk, sv[t * VS + 16 * i + n], acc[i], 0, 0, 0);
  }
  const size_t unit = (size_t)blockIdx.x * a.H + h;
  float* __restrict__ B = p.starts + unit * a.d * a.dv;
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int r = d0 + 16 * wave + 4 * g + e, c = v0 + 16 * i + n;
      if (r < a.d && c < a.dv) B[(size_t)r * a.dv + c] = acc[i][e];
    }
  if (vt == 0 && a.normaliser && tid < 64 && d0 + tid < a.d) {
    float s = 0.f;
    for (int t = 0; t < CH; ++t) s += sk[t * KST + tid];
    p.n_starts[unit * a.d + d0 + tid] = s;
  }
  if (dt == 0 && vt == 0 && tid == 0) p.ends[unit] = end;
}

// (2) a thread an entry (of the states, then of the normalisers): S_0 in B's place chunk by chunk, the end into the slot
__global__ void __launch_bounds__(256)
chunk_fold_kernel(ChunkArgs p) {
  extern __shared__ float decay[];              // [chunks of this row]
  const ScanArgs& a = p.s;
  const int row = blockIdx.x, h = blockIdx.y, d = a.d, dv = a.dv, H = a.H;
  const int chunks = (a.row_start[row + 1] - a.row_start[row] + CH - 1) / CH;
  const size_t unit0 = (size_t)row * p.max_chunks * H + h;
  for (int c = threadIdx.x; c < chunks; c += blockDim.x) decay[c] = expf(p.ends[unit0 + (size_t)c * H]);
  __syncthreads();
  const int slot = a.slots[row], total = d * dv + (a.normaliser ? d : 0);
  for (int e = blockIdx.z * blockDim.x + threadIdx.x; e < total; e += gridDim.z * blockDim.x) {
    const bool of_state = e < d * dv;
    const int i = of_state ? e : e - d * dv, per = of_state ? d * dv : d;
    float* __restrict__ st = (of_state ? a.state : a.normaliser) + ((size_t)slot * H + h) * per + i;
    float* __restrict__ at = (of_state ? p.starts : p.n_starts) + unit0 * per + i;
    const size_t stride = (size_t)H * per;
    float s = *st;
    for (int c = 0; c < chunks; c += 8) {       // the loads of eight chunks on their way together
      float b[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) b[u] = at[(size_t)(c + u < chunks ? c + u : chunks - 1) * stride];
#pragma unroll
      for (int u = 0; u < 8; ++u)
        if (c + u < chunks) {
          at[(size_t)(c + u) * stride] = s;
          s = fmaf(decay[c + u], s, b[u]);
        }
    }
    *st = s;
  }
}

// (3) outputs of a chunk, 16 NT columns of a head: a wave 16 tokens.  P = Q K^T and O = Q S_0 together, DB state rows at a
// time through the LDS (q read once for both), then O <- e^A_t O + (P masked and weighted) V.
template <int NT>
__global__ void __launch_bounds__(256)
chunk_outputs_kernel(ChunkArgs p) {
  constexpr int VS = 16 * NT + 4, PS = CH + 4;
  constexpr int QKS = 2 * CH * QS + DB * VS, VP = CH * VS + CH * PS, FLOATS = QKS > VP ? QKS : VP;
  __shared__ __align__(16) float buf[FLOATS];           // q, k, S_0; after the products over the state rows v and the weights
  __shared__ float A[CH], cc[CH], sn[DB], rows_sum[CH];
  float* sq = buf;
  float* sk = buf + CH * QS;
  float* ss = buf + 2 * CH * QS;
  float* sv = buf;
  float* sp = buf + CH * VS;
  const ScanArgs& a = p.s;
  CHUNK_OF_ROW;
  const int h = blockIdx.y, v0 = blockIdx.z * 16 * NT, tid = threadIdx.x;
  const int lane = tid & 63, n = lane & 15, g = lane >> 4;
  // whose 16 tokens: later tokens see more, so the SIMDs take turns (a scalar: the branches on it are uniform)
  const int wave = __builtin_amdgcn_readfirstlane(((tid >> 6) + blockIdx.x) & 3);
  const bool with_n = a.normaliser && blockIdx.z == 0;
  const size_t unit = (size_t)blockIdx.x * a.H + h;
  const float* __restrict__ qp = a.q + (size_t)t0 * a.ld_qk + (size_t)(h / a.per_group) * a.d;
  const float* __restrict__ kp = a.k + (size_t)t0 * a.ld_qk + (size_t)(h / a.per_group) * a.d;
  const float* __restrict__ vp = a.v + (size_t)t0 * a.ld_v + (size_t)h * a.dv;
  const float* __restrict__ S0 = p.starts + unit * a.d * a.dv;
  const float* __restrict__ n0 = with_n ? p.n_starts + unit * a.d : nullptr;
  chunk_decays(a, t0, nt, h, A, cc);
  f32x4 O[NT], P[4];
#pragma unroll
  for (int i = 0; i < NT; ++i) O[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < 4; ++i) P[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  float qn = 0.f;
  constexpr int SR = DB * 4 * NT / 256;         // pieces of S_0 a thread carries
  f32x4 rq[2], rk[2], rs[SR];
  float rn = 0.f;
  auto fetch = [&](int d0) {
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int e = tid + 256 * i, t = e >> 3, c = d0 + 4 * (e & 7);
      const size_t at = (size_t)(t < nt ? t : nt - 1) * a.ld_qk;
      rq[i] = load4(qp + at, c, a.d, p.vec);
      rk[i] = load4(kp + at, c, a.d, p.vec);
    }
#pragma unroll
    for (int i = 0; i < SR; ++i) {
      const int e = tid + 256 * i, r = d0 + e / (4 * NT);
      rs[i] = load4(S0 + (size_t)(r < a.d ? r : a.d - 1) * a.dv, v0 + 4 * (e % (4 * NT)), a.dv, p.vec);
    }
    if (with_n && tid < DB) rn = d0 + tid < a.d ? n0[d0 + tid] : 0.f;
  };
  fetch(0);
  for (int d0 = 0; d0 < a.d; d0 += DB) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int e = tid + 256 * i, at = (e >> 3) * QS + 4 * (e & 7);
      *reinterpret_cast<f32x4*>(sq + at) = rq[i] * a.q_scale;
      *reinterpret_cast<f32x4*>(sk + at) = rk[i];
    }
#pragma unroll
    for (int i = 0; i < SR; ++i) {
      const int e = tid + 256 * i;
      *reinterpret_cast<f32x4*>(ss + (e / (4 * NT)) * VS + 4 * (e % (4 * NT))) = rs[i];     // rows beyond d meet zeros of q
    }
    if (with_n && tid < DB) sn[tid] = rn;
    __syncthreads();
    if (d0 + DB < a.d) fetch(d0 + DB);          // on its way during the products
#pragma unroll
    for (int kb = 0; kb < DB / 16; ++kb) {
      // state row 16 kb + 4 g + j is step j's of lane group g, for both operands
      const f32x4 q = *reinterpret_cast<const f32x4*>(sq + (16 * wave + n) * QS + 16 * kb + 4 * g);
#pragma unroll
      for (int st = 0; st < 4; ++st)
        if (st <= wave) {
          const f32x4 k = *reinterpret_cast<const f32x4*>(sk + (16 * st + n) * QS + 16 * kb + 4 * g);
#pragma unroll
          for (int j = 0; j < 4; ++j) P[st] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[j], k[j], P[st], 0, 0, 0);
        }
#pragma unroll
      for (int i = 0; i < NT; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          O[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[j], ss[(16 * kb + 4 * g + j) * VS + 16 * i + n], O[i], 0, 0, 0);
      if (with_n) {
#pragma unroll
        for (int j = 0; j < 4; ++j) qn = fmaf(q[j], sn[16 * kb + 4 * g + j], qn);
      }
    }
  }
  f32x4 rv[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int e = tid + 256 * i, t = e / (4 * NT);
    rv[i] = load4(vp + (size_t)(t < nt ? t : nt - 1) * a.ld_v, v0 + 4 * (e % (4 * NT)), a.dv, p.vec);     // beyond the end: meets zeros
  }
  __syncthreads();                              // everybody is done with q, k and S_0
  // a lane holds rows (tokens) 4 g + e of the wave's 16 and column n of every tile
  float At[4], eA[4], sum[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    At[e] = A[16 * wave + 4 * g + e];
    eA[e] = expf(At[e]);
  }
#pragma unroll
  for (int st = 0; st < 4; ++st) {
    const int s = 16 * st + n;
    const float As = A[s], cs = cc[s];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = 16 * wave + 4 * g + e;
      const float w = st <= wave && s <= t ? P[st][e] * (expf(At[e] - As) * cs) : 0.f;
      sp[t * PS + s] = w;
      sum[e] += w;
    }
  }
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) O[i][e] *= eA[e];
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int e = tid + 256 * i;
    *reinterpret_cast<f32x4*>(sv + (e / (4 * NT)) * VS + 4 * (e % (4 * NT))) = rv[i];
  }
  if (with_n) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      sum[e] += __shfl_xor(sum[e], 1, 64);
      sum[e] += __shfl_xor(sum[e], 2, 64);
      sum[e] += __shfl_xor(sum[e], 4, 64);
      sum[e] += __shfl_xor(sum[e], 8, 64);
      if (n == 0) rows_sum[16 * wave + 4 * g + e] = sum[e];
    }
    qn += __shfl_xor(qn, 16, 64);
    qn += __shfl_xor(qn, 32, 64);
  }
  __syncthreads();
  if (with_n && g == 0 && 16 * wave + n < nt) {
    const int t = 16 * wave + n;
    a.nq[(size_t)(t0 + t) * a.H + h] = fmaf(expf(A[t]), qn, rows_sum[t]);
  }
#pragma unroll
  for (int kb = 0; kb < 4; ++kb)
    if (kb <= wave) {
      const f32x4 w = *reinterpret_cast<const f32x4*>(sp + (16 * wave + n) * PS + 16 * kb + 4 * g);
#pragma unroll
      for (int i = 0; i < NT; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          O[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(w[j], sv[(16 * kb + 4 * g + j) * VS + 16 * i + n], O[i], 0, 0, 0);
    }
#pragma unroll
  for (int i = 0; i < NT; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = 16 * wave + 4 * g + e, c = v0 + 16 * i + n;
      if (t < nt && c < a.dv) a.o[((size_t)(t0 + t) * a.H + h) * a.dv + c] = O[i][e];
    }
}

// y = (o + skip x) silu(z) over one part of a token's numbers, over its root mean square, times weight and scale
template <typename TO>
__global__ void __launch_bounds__(256)
ssm_finish_kernel(const float* __restrict__ o, const float* __restrict__ x, long ldx, const float* __restrict__ z, long ldz,
                  const float* __restrict__ skip, const float* __restrict__ weight, float eps, float scale, TO* __restrict__ out,
                  long ldo, int inner, int dv, int size) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, c0 = blockIdx.y * size;
  auto value = [&](int c) {
    const float zz = z[(size_t)t * ldz + c];
    return fmaf(skip[c / dv], x[(size_t)t * ldx + c], o[(size_t)t * inner + c]) * (zz / (1.0f + expf(-zz)));
  };
  float ss = 0.f;
  for (int c = c0 + threadIdx.x; c < c0 + size; c += blockDim.x) {
    const float y = value(c);
    ss = fmaf(y, y, ss);
  }
  const float r = 1.0f / sqrtf(block_sum(ss, scratch) / (float)size + eps);
  for (int c = c0 + threadIdx.x; c < c0 + size; c += blockDim.x)
    out[(size_t)t * ldo + c] = from_float<TO>(value(c) * r * weight[c] * scale);
}

// a wave a (token, head)
template <typename TO>
__global__ void __launch_bounds__(256)
mlstm_finish_kernel(const float* __restrict__ o, const float* __restrict__ nq, const float* __restrict__ low,
                    const float* __restrict__ g, long ldg, const float* __restrict__ weight, float eps, float scale,
                    TO* __restrict__ out, long ldo, int tokens, int H, int dv) {
  const int job = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (job >= tokens * H) return;
  const int t = job / H, h = job - t * H;
  const float inv = 1.0f / (fmaxf(fabsf(nq[job]), low[job]) + 1e-6f);
  const float* __restrict__ oh = o + (size_t)job * dv;
  float ss = 0.f;
  for (int e = lane; e < dv; e += 64) {
    const float y = oh[e] * inv;
    ss = fmaf(y, y, ss);
  }
  const float r = inv / sqrtf(wave_sum(ss) / (float)dv + eps);
  for (int e = lane; e < dv; e += 64) {
    const int c = h * dv + e;
    out[(size_t)t * ldo + c] = from_float<TO>(oh[e] * r * weight[c] * mie_sigmoid(g[(size_t)t * ldg + c]) * scale);
  }
}

MIE_EXPORT const char* matrix_state_last_error() { return g_mie_error; }

constexpr long WIDE_FROM = 256;       // workgroups

template <int NT>
static int chunk_launch_nt(const ChunkArgs& p, int rows, hipStream_t s) {
  const ScanArgs& a = p.s;
  const int vt = (a.dv + 16 * NT - 1) / (16 * NT), dt = (a.d + 63) / 64;
  if ((long)vt * dt > 65535) MIE_FAIL("matrix state in chunks: states of %d x %d are beyond the grid", a.d, a.dv);
  const dim3 units(rows * p.max_chunks, a.H);
  hipLaunchKernelGGL(chunk_sums_kernel<NT>, dim3(units.x, units.y, vt * dt), dim3(256), 0, s, p, dt);
  MIE_CHECK_LAUNCH("chunk_sums");
  const long entries = (long)a.d * a.dv + (a.normaliser ? a.d : 0);
  const int per = (int)((entries + 255) / 256 < 1024 ? (entries + 255) / 256 : 1024);
  hipLaunchKernelGGL(chunk_fold_kernel, dim3(rows, a.H, per), dim3(256), (size_t)p.max_chunks * sizeof(float), s, p);
  MIE_CHECK_LAUNCH("chunk_fold");
  hipLaunchKernelGGL(chunk_outputs_kernel<NT>, dim3(units.x, units.y, vt), dim3(256), 0, s, p);
  MIE_CHECK_LAUNCH("chunk_outputs");
  return 0;
}

static int scan_launch(const ScanArgs& a, int rows, int max_chunks, float* starts, float* n_starts, float* ends, hipStream_t s) {
  if (max_chunks > 0) {
    if (!starts || !ends || (a.normaliser && !n_starts)) MIE_FAIL("matrix state in chunks: no scratch");
    if ((long)rows * max_chunks > 2000000000L || a.H > 65535 || max_chunks > 16000)
      MIE_FAIL("matrix state in chunks: %d rows of %d chunks, %d heads", rows, max_chunks, a.H);
    const uintptr_t all = (uintptr_t)a.q | (uintptr_t)a.k | (uintptr_t)a.v | (uintptr_t)starts;
    const int vec = (all & 15) == 0 && a.ld_qk % 4 == 0 && a.ld_v % 4 == 0 && a.d % 4 == 0 && a.dv % 4 == 0;
    ChunkArgs p{a, max_chunks, vec, starts, n_starts, ends};
    // 128 columns a workgroup where that still gives every compute unit one (the scores are then made half as often)
    const bool wide = a.dv > 64 && (long)rows * max_chunks * a.H * ((a.dv + 127) / 128) >= WIDE_FROM;
    return wide ? chunk_launch_nt<8>(p, rows, s) : chunk_launch_nt<4>(p, rows, s);
  }
  if (a.d > 1024) MIE_FAIL("matrix_scan: states of %d rows (at most 1024)", a.d);
  const int tiles = (a.dv + 63) / 64;
  if (a.H > 65535 || tiles > 65535) MIE_FAIL("matrix_scan: %d heads of %d columns are beyond the grid", a.H, a.dv);
  auto lds = [&](int R, int TB, int waves) { return (size_t)(2 * TB * waves * R + waves * TB * 65 + TB) * sizeof(float); };
  if (a.d <= 256) {
    const int waves = (a.d + 15) / 16;
    hipLaunchKernelGGL((matrix_scan_kernel<16, 8>), dim3(rows, a.H, tiles), dim3(waves * 64), lds(16, 8, waves), s, a);
  } else {
    const int waves = (a.d + 63) / 64;
    hipLaunchKernelGGL((matrix_scan_kernel<64, 4>), dim3(rows, a.H, tiles), dim3(waves * 64), lds(64, 4, waves), s, a);
  }
  MIE_CHECK_LAUNCH("matrix_scan");
  return 0;
}

// u points at x (rows ld_u floats apart), B and C at columns b_col, c_col of it; dt and z point at their first columns of the
// sums (rows ld floats apart).  la, c: scratch [tokens, H]; o: scratch [tokens, H dv].  out rows are ldo numbers apart.
MIE_EXPORT int mie_state_space(const float* u, long ld_u, int b_col, int c_col, const float* z, const float* dt, long ld,
                               const float* dt_bias, const float* rate, const float* skip, const float* norm_weight, float eps,
                               float scale, float* state, const int* row_start, const int* slots, float* la, float* c, float* o,
                               void* out, int out_dtype, long ldo, int tokens, int rows, int H, int groups, int d, int dv,
                               int norm_groups, int max_chunks, float* starts, float* ends, hipStream_t s) {
  if (tokens <= 0 || rows <= 0) return 0;
  if (H <= 0 || groups <= 0 || H % groups || d <= 0 || dv <= 0 || norm_groups <= 0 || (H * dv) % norm_groups || ldo < (long)H * dv)
    MIE_FAIL("state_space: %d heads of %d x %d in %d groups, %d norm groups, output rows %ld apart", H, d, dv, groups, norm_groups, ldo);
  if (out_dtype != MIE_F32 && out_dtype != MIE_BF16) MIE_FAIL("state_space: dtype code %d", out_dtype);
  if (!u || !z || !dt || !dt_bias || !rate || !skip || !norm_weight || !state || !row_start || !slots || !la || !c || !o || !out)
    MIE_FAIL("state_space: a null operand");
  hipLaunchKernelGGL(ssm_prepare_kernel, dim3((tokens * H + 255) / 256), dim3(256), 0, s, dt, ld, dt_bias, rate, la, c, tokens, H);
  MIE_CHECK_LAUNCH("ssm_prepare");
  ScanArgs a{u + c_col, u + b_col, u, ld_u, ld_u, H / groups, 1.0f, la, c, state, nullptr, row_start, slots, o, nullptr, H, d, dv};
  if (scan_launch(a, rows, max_chunks, starts, nullptr, ends, s)) return -1;
  const int size = H * dv / norm_groups;
  if (norm_groups > 65535) MIE_FAIL("state_space: %d norm groups are beyond the grid", norm_groups);
  const int threads = size <= 256 ? 64 : 256;
  if (out_dtype == MIE_F32)
    hipLaunchKernelGGL(ssm_finish_kernel<float>, dim3(tokens, norm_groups), dim3(threads), 0, s, o, u, ld_u, z, ld, skip, norm_weight,
                       eps, scale, (float*)out, ldo, H * dv, dv, size);
  else
    hipLaunchKernelGGL(ssm_finish_kernel<bf16>, dim3(tokens, norm_groups), dim3(threads), 0, s, o, u, ld_u, z, ld, skip, norm_weight,
                       eps, scale, (bf16*)out, ldo, H * dv, dv, size);
  MIE_CHECK_LAUNCH("ssm_finish");
  return 0;
}

// max_chunks > 0: rows run in chunks of 64 tokens, at most that many a row, with scratch starts [rows * max_chunks, H, d, dv],
// ends [rows * max_chunks, H] (and n_starts [rows * max_chunks, H, d]); 0: rows run whole.
// sums: rows ld floats apart with q, k (H d each), v, g (H dv each), gates i, f (H each) from their columns on.  la, c, low,
// nq: scratch [tokens, H]; o: scratch [tokens, H dv].
MIE_EXPORT int mie_mlstm(const float* sums, long ld, int q_col, int k_col, int v_col, int g_col, int i_col, int f_col,
                         const float* i_bias, const float* f_bias, float cap, float q_scale, const float* norm_weight, float eps,
                         float scale, float* state, float* normaliser, float* maximum, const int* row_start, const int* slots,
                         float* la, float* c, float* low, float* nq, float* o, void* out, int out_dtype, long ldo, int tokens,
                         int rows, int H, int d, int dv, int longest, int max_chunks, float* starts, float* n_starts, float* ends,
                         hipStream_t s) {
  if (tokens <= 0 || rows <= 0) return 0;
  if (H <= 0 || d <= 0 || dv <= 0 || !(cap > 0.f) || ldo < (long)H * dv)
    MIE_FAIL("mlstm: %d heads of %d x %d, cap %g, output rows %ld apart", H, d, dv, (double)cap, ldo);
  if (H > 65535) MIE_FAIL("mlstm: %d heads are beyond the grid", H);
  if (out_dtype != MIE_F32 && out_dtype != MIE_BF16) MIE_FAIL("mlstm: dtype code %d", out_dtype);
  if (!sums || !i_bias || !f_bias || !norm_weight || !state || !normaliser || !maximum || !row_start || !slots || !la || !c || !low ||
      !nq || !o || !out)
    MIE_FAIL("mlstm: a null operand");
  const int waves = (longest + 63) / 64 < 1 ? 1 : (longest + 63) / 64 > 16 ? 16 : (longest + 63) / 64;
  hipLaunchKernelGGL(mlstm_prepare_kernel, dim3(rows, H), dim3(64 * waves), 0, s, sums + i_col, sums + f_col, ld, i_bias, f_bias, cap, maximum,
                     row_start, slots, la, c, low, H);
  MIE_CHECK_LAUNCH("mlstm_prepare");
  ScanArgs a{sums + q_col, sums + k_col, sums + v_col, ld, ld, 1, q_scale, la, c, state, normaliser, row_start, slots, o, nq, H, d, dv};
  if (scan_launch(a, rows, max_chunks, starts, n_starts, ends, s)) return -1;
  const dim3 grid((tokens * H + 3) / 4);
  if (out_dtype == MIE_F32)
    hipLaunchKernelGGL(mlstm_finish_kernel<float>, grid, dim3(256), 0, s, o, nq, low, sums + g_col, ld, norm_weight, eps, scale,
                       (float*)out, ldo, tokens, H, dv);
  else
    hipLaunchKernelGGL(mlstm_finish_kernel<bf16>, grid, dim3(256), 0, s, o, nq, low, sums + g_col, ld, norm_weight, eps, scale,
                       (bf16*)out, ldo, tokens, H, dv);
  MIE_CHECK_LAUNCH("mlstm_finish");
  return 0;
}
