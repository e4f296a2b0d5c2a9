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

// gate columns -> la, c and exp(-m) [T, H]; the slot's maximum moves on.  A wave a (row, head).
__global__ void __launch_bounds__(64)
mlstm_prepare_kernel(const float* __restrict__ gi, const float* __restrict__ gf, long ld, const float* __restrict__ i_bias,
                     const float* __restrict__ f_bias, float cap, float* __restrict__ maximum, const int* __restrict__ row_start,
                     const int* __restrict__ slots, float* __restrict__ la, float* __restrict__ c, float* __restrict__ low, int H) {
  const int row = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const int begin = row_start[row], end = row_start[row + 1];
  float m0 = maximum[(size_t)slots[row] * H + h];
  const float ib = i_bias[h], fb = f_bias[h], inv_cap = 1.0f / cap;
  for (int t0 = begin; t0 < end; t0 += 64) {
    const int t = t0 + lane;
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
    const float m = fmaxf(F + m0, I);
    float before = __shfl_up(m, 1, 64);
    if (lane == 0) before = m0;
    if (ok) {
      const size_t e = (size_t)t * H + h;
      la[e] = fminf(f + before - m, 0.f);
      c[e] = expf(i - m);
      low[e] = expf(-m);
    }
    m0 = __shfl(m, 63, 64);                  // lanes beyond the row's end pass the maximum on
  }
  if (lane == 0) maximum[(size_t)slots[row] * H + h] = m0;
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

static int scan_launch(const ScanArgs& a, int rows, hipStream_t s) {
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
                               int norm_groups, hipStream_t s) {
  if (tokens <= 0 || rows <= 0) return 0;
  if (H <= 0 || groups <= 0 || H % groups || d <= 0 || dv <= 0 || norm_groups <= 0 || (H * dv) % norm_groups || ldo < (long)H * dv)
    MIE_FAIL("state_space: %d heads of %d x %d in %d groups, %d norm groups, output rows %ld apart", H, d, dv, groups, norm_groups, ldo);
  if (out_dtype != MIE_F32 && out_dtype != MIE_BF16) MIE_FAIL("state_space: dtype code %d", out_dtype);
  if (!u || !z || !dt || !dt_bias || !rate || !skip || !norm_weight || !state || !row_start || !slots || !la || !c || !o || !out)
    MIE_FAIL("state_space: a null operand");
  hipLaunchKernelGGL(ssm_prepare_kernel, dim3((tokens * H + 255) / 256), dim3(256), 0, s, dt, ld, dt_bias, rate, la, c, tokens, H);
  MIE_CHECK_LAUNCH("ssm_prepare");
  ScanArgs a{u + c_col, u + b_col, u, ld_u, ld_u, H / groups, 1.0f, la, c, state, nullptr, row_start, slots, o, nullptr, H, d, dv};
  if (scan_launch(a, rows, s)) return -1;
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

// sums: rows ld floats apart with q, k (H d each), v, g (H dv each), gates i, f (H each) from their columns on.  la, c, low,
// nq: scratch [tokens, H]; o: scratch [tokens, H dv].
MIE_EXPORT int mie_mlstm(const float* sums, long ld, int q_col, int k_col, int v_col, int g_col, int i_col, int f_col,
                         const float* i_bias, const float* f_bias, float cap, float q_scale, const float* norm_weight, float eps,
                         float scale, float* state, float* normaliser, float* maximum, const int* row_start, const int* slots,
                         float* la, float* c, float* low, float* nq, float* o, void* out, int out_dtype, long ldo, int tokens,
                         int rows, int H, int d, int dv, hipStream_t s) {
  if (tokens <= 0 || rows <= 0) return 0;
  if (H <= 0 || d <= 0 || dv <= 0 || !(cap > 0.f) || ldo < (long)H * dv)
    MIE_FAIL("mlstm: %d heads of %d x %d, cap %g, output rows %ld apart", H, d, dv, (double)cap, ldo);
  if (H > 65535) MIE_FAIL("mlstm: %d heads are beyond the grid", H);
  if (out_dtype != MIE_F32 && out_dtype != MIE_BF16) MIE_FAIL("mlstm: dtype code %d", out_dtype);
  if (!sums || !i_bias || !f_bias || !norm_weight || !state || !normaliser || !maximum || !row_start || !slots || !la || !c || !low ||
      !nq || !o || !out)
    MIE_FAIL("mlstm: a null operand");
  hipLaunchKernelGGL(mlstm_prepare_kernel, dim3(rows, H), dim3(64), 0, s, sums + i_col, sums + f_col, ld, i_bias, f_bias, cap, maximum,
                     row_start, slots, la, c, low, H);
  MIE_CHECK_LAUNCH("mlstm_prepare");
  ScanArgs a{sums + q_col, sums + k_col, sums + v_col, ld, ld, 1, q_scale, la, c, state, normaliser, row_start, slots, o, nq, H, d, dv};
  if (scan_launch(a, rows, s)) return -1;
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
