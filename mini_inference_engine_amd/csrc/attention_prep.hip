// Between a q/k/v projection's float32 sums and attention, for mixers that want more than a rotation there:
// an RMS norm over a token's whole query (key) projection (or head by head, with one weight of a head's size for all
// heads), the rotation of the first numbers of every head by
// angles computed here in 32-bit (adjacent pairs or the two halves of the turned part), a temperature a query
// head, the projection's biases, a query temperature that grows with the logarithm of the position, values that are the keys as projected, and heads kept in the cache at a padded size.
//
// qkv_finish: one workgroup a token.  Queries go out as [T, Hq, P], keys to k_cache [pages, Hkv, page, P], values
// to v_cache [pages, Hkv, P, page] (transposed within a page), zeros beyond dim / vdim.  Everything is computed in
// 32-bit from the sums and rounded once on the way out.
// qkv_conv_finish: the same for projections that first pass a short causal convolution over time (with biases before it, norms
// head by head before the rotation or, without weights, after it, either pairing turned, a factor on cosines and sines, values
// left for or mixed with another layer's).
// head_gate:  o[t, h, :] *= sigmoid(gate[t, h]).
// gate_heads: out[t, h vdim + d] = scale * o[t, h P + d] * sigmoid(gate[t, h vdim + d]), d < vdim.
#include "common.hpp"

enum { LAYOUT_INTERLEAVED = 0, LAYOUT_HALF = 1 };

struct FinishArgs {
  const float* sums; long ld; int q_col, k_col, v_col;      // v_col < 0: the values are the keys as projected
  const float* q_norm; const float* k_norm; float eps;
  int norm_per_head;            // the norms are taken head by head; q_norm and k_norm hold dim numbers each
  const float* inv_freq; int nf, layout;
  const float* q_head_scale;
  const float* col_bias;        // one number a column of the sums, added to queries, keys and values first (or null)
  float temp_coef; int temp_every;   // queries times 1 + temp_coef * ln(floor((p + 1) / temp_every) + 1) at position p (temp_every 0: not)
  const int* positions; const int* slots;
  void* q_out; void* k_cache; void* v_cache;
  int Hq, Hkv, dim, vdim, P, page;
};

template <typename TO>
__global__ void __launch_bounds__(256)
qkv_finish_kernel(FinishArgs a) {
  __shared__ float scratch[16];
  // blockIdx.y: which share of the token's heads this workgroup makes (every one takes the norms' sums itself)
  const int t = blockIdx.x;
  const float* __restrict__ row = a.sums + (size_t)t * a.ld;
  const float* __restrict__ q = row + a.q_col;
  const float* __restrict__ k = row + a.k_col;
  const float* __restrict__ qb = a.col_bias ? a.col_bias + a.q_col : nullptr;
  const float* __restrict__ kb = a.col_bias ? a.col_bias + a.k_col : nullptr;
  const float* __restrict__ vb = a.col_bias ? a.col_bias + (a.v_col < 0 ? a.k_col : a.v_col) : nullptr;
  const int nq = a.Hq * a.dim, nk = a.Hkv * a.dim;
  float rq = 1.f, rk = 1.f;
  if (a.q_norm && !a.norm_per_head) {
    float ss = 0.f;
    for (int i = threadIdx.x; i < nq; i += blockDim.x) {
      const float v = qb ? q[i] + qb[i] : q[i];
      ss = fmaf(v, v, ss);
    }
    rq = 1.0f / sqrtf(block_sum(ss, scratch) / (float)nq + a.eps);
  }
  if (a.k_norm && !a.norm_per_head) {
    float ss = 0.f;
    for (int i = threadIdx.x; i < nk; i += blockDim.x) {
      const float v = kb ? k[i] + kb[i] : k[i];
      ss = fmaf(v, v, ss);
    }
    rk = 1.0f / sqrtf(block_sum(ss, scratch) / (float)nk + a.eps);
  }
  // the angles' cosines and sines once a token: every head turns by the same ones
  extern __shared__ float cs[];                 // cos [nf], sin [nf]
  const float pos = (float)a.positions[t];
  const float temperature = a.temp_every > 0 ? 1.0f + a.temp_coef * logf((float)((a.positions[t] + 1) / a.temp_every) + 1.0f) : 1.0f;
  for (int i = threadIdx.x; i < a.nf; i += blockDim.x) sincosf(pos * a.inv_freq[i], &cs[a.nf + i], &cs[i]);
  __syncthreads();
  // A wave a head (query heads first, then key heads with their values), lanes over the head's pairs and then over what
  // does not turn: both members of a pair come from one lane, which reads each of its numbers once.
  const int turned = 2 * a.nf, lane = threadIdx.x & 63;
  const int wave = blockIdx.y * (blockDim.x >> 6) + (threadIdx.x >> 6), waves = gridDim.y * (blockDim.x >> 6);
  const int slot = a.slots[t];
  const size_t pg = slot / a.page, off = slot % a.page;
  TO* __restrict__ qo = (TO*)a.q_out + (size_t)t * a.Hq * a.P;
  TO* __restrict__ kc = (TO*)a.k_cache;
  TO* __restrict__ vc = (TO*)a.v_cache;
  const float* __restrict__ vals = a.v_col < 0 ? k : row + a.v_col;
  for (int job = wave; job < a.Hq + a.Hkv; job += waves) {
    const bool is_q = job < a.Hq;
    const int h = is_q ? job : job - a.Hq;
    const float* __restrict__ x = (is_q ? q : k) + (size_t)h * a.dim;
    const float* __restrict__ xb = (is_q ? qb : kb) ? (is_q ? qb : kb) + (size_t)h * a.dim : nullptr;
    const float* __restrict__ w = is_q ? a.q_norm : a.k_norm;
    if (w && !a.norm_per_head) w += (size_t)h * a.dim;
    float r = is_q ? rq : rk;
    if (w && a.norm_per_head) {       // the wave owns the head: its root mean square by a sum over the lanes
      float ss = 0.f;
      for (int d = lane; d < a.dim; d += 64) {
        const float v = xb ? x[d] + xb[d] : x[d];
        ss = fmaf(v, v, ss);
      }
      r = 1.0f / sqrtf(wave_sum(ss) / (float)a.dim + a.eps);
    }
    const float mult = is_q ? (a.q_head_scale ? a.q_head_scale[h] * temperature : temperature) : 1.f;
    TO* __restrict__ dst = is_q ? qo + (size_t)h * a.P : kc + ((pg * a.Hkv + h) * a.page + off) * a.P;
    for (int i = lane; i < a.nf; i += 64) {
      const int d1 = a.layout == LAYOUT_INTERLEAVED ? 2 * i : i, d2 = a.layout == LAYOUT_INTERLEAVED ? 2 * i + 1 : i + a.nf;
      const float y1 = xb ? x[d1] + xb[d1] : x[d1], y2 = xb ? x[d2] + xb[d2] : x[d2];
      const float x1 = w ? y1 * r * w[d1] : y1, x2 = w ? y2 * r * w[d2] : y2;
      float o1, o2;
      rotate_pair(x1, x2, cs[i], cs[a.nf + i], o1, o2);
      dst[d1] = from_float<TO>(o1 * mult);
      dst[d2] = from_float<TO>(o2 * mult);
    }
    for (int d = turned + lane; d < a.P; d += 64) {
      const float y = d < a.dim ? (xb ? x[d] + xb[d] : x[d]) : 0.f;
      const float v = d < a.dim ? (w ? y * r * w[d] : y) * mult : 0.f;
      dst[d] = from_float<TO>(v);
    }
    if (!is_q) {
      const float* __restrict__ vh = vals + (size_t)h * a.vdim;
      const float* __restrict__ vhb = vb ? vb + (size_t)h * a.vdim : nullptr;
      TO* __restrict__ vd = vc + (pg * a.Hkv + h) * a.P * a.page + off;
      for (int d = lane; d < a.P; d += 64) vd[(size_t)d * a.page] = from_float<TO>(d < a.vdim ? (vhb ? vh[d] + vhb[d] : vh[d]) : 0.f);
    }
  }
}

// ---- projections through a short convolution
struct ConvFinishArgs {
  const float* sums; long ld; int col;                      // queries, keys, values side by side from column ``col`` on
  const float* col_bias;        // [C], added to the inputs of the convolution (the tail holds biased inputs), or null
  const float* taps;            // [C, K], C = (Hq + Hkv) dim + Hkv vdim in that order
  float* tail;                  // [slots, K - 1, C]: the row's last inputs, oldest first
  const int* token_row; const int* row_start; const int* state_slots;
  int K, move_tail;             // move_tail: every row is one token, and the waves move the tail on themselves
  const float* q_norm; const float* k_norm; float eps;      // dim numbers each, or null
  int norm_turned;              // no weights: heads over their root mean square after the rotation
  const float* inv_freq; int nf, layout; float rot_scale;
  const int* positions; const int* slots;
  float* values_out; const float* mix_other; float mix;     // values as projected / (1 - mix) v + mix * other
  void* q_out; void* k_cache; void* v_cache;
  int Hq, Hkv, dim, vdim, P, page, C, row_floats;
};

// A workgroup a (token, share of its heads), a wave a head of queries, keys or values: its convolved numbers go into the
// wave's own stretch of the LDS with the sum of their squares on the way, then out normed and turned.  KT: the taps (0: any
// number).
template <typename TO, int KT>
__global__ void __launch_bounds__(256)
qkv_conv_finish_kernel(ConvFinishArgs a) {
  extern __shared__ float lds[];
  const int t = blockIdx.x, lane = threadIdx.x & 63, wv = threadIdx.x >> 6;
  float* mine = lds + (size_t)wv * a.row_floats;
  const int K = KT ? KT : a.K, keep = K - 1;
  const int r = a.token_row[t], j = t - a.row_start[r];
  float* __restrict__ tl = a.tail + (size_t)a.state_slots[r] * (keep > 0 ? keep : 1) * a.C;
  const float pos = (float)a.positions[t];
  const int slot = a.slots[t];
  const size_t pg = slot / a.page, off = slot % a.page;
  const int jobs = a.Hq + 2 * a.Hkv;
  for (int job = blockIdx.y * 4 + wv; job < jobs; job += gridDim.y * 4) {
    const bool is_q = job < a.Hq, is_v = job >= a.Hq + a.Hkv;
    const int h = is_q ? job : is_v ? job - a.Hq - a.Hkv : job - a.Hq;
    const int n = is_v ? a.vdim : a.dim;
    const int c0 = is_q ? h * a.dim : is_v ? (a.Hq + a.Hkv) * a.dim + h * a.vdim : (a.Hq + h) * a.dim;
    float ss = 0.f;
    const float grown = a.norm_turned ? a.rot_scale * a.rot_scale : 1.f;      // what the rotation does to a pair's sum of squares
    for (int d = lane; d < n; d += 64) {
      const int c = c0 + d;
      const float* __restrict__ x = a.sums + (size_t)t * a.ld + a.col + c;
      const float b = a.col_bias ? a.col_bias[c] : 0.f;
      float acc = 0.f;
      if constexpr (KT > 0) {
        float in[KT];
#pragma unroll
        for (int i = 0; i < KT; ++i) {          // tokens t - K + 1 .. t
          const int back = KT - 1 - i;
          const float* src = back <= j ? x - (long)back * a.ld : tl + (size_t)(keep + j - back) * a.C + c;
          in[i] = *src + (back <= j ? b : 0.f);
        }
#pragma unroll
        for (int i = 0; i < KT; ++i) acc = fmaf(a.taps[(size_t)c * KT + i], in[i], acc);
        if (a.move_tail) {
#pragma unroll
          for (int i = 0; i < KT - 1; ++i) tl[(size_t)i * a.C + c] = in[i + 1];      // a row of one token: its inputs are the tail's and its own
        }
      } else {
        for (int i = 0; i < K; ++i) {
          const int back = K - 1 - i;
          acc = fmaf(a.taps[(size_t)c * K + i], back <= j ? x[-(long)back * a.ld] + b : tl[(size_t)(keep + j - back) * a.C + c], acc);
        }
        if (a.move_tail)
          for (int i = 0; i < keep; ++i) tl[(size_t)i * a.C + c] = i + 1 < keep ? tl[(size_t)(i + 1) * a.C + c] : x[0] + b;
      }
      mine[d] = acc;
      ss = fmaf(d < 2 * a.nf ? grown * acc : acc, acc, ss);
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");      // the wave's lanes read one another's numbers below
    __builtin_amdgcn_wave_barrier();
    if (is_v) {
      TO* __restrict__ vd = (TO*)a.v_cache + (pg * a.Hkv + h) * a.P * a.page + off;
      const size_t at = ((size_t)t * a.Hkv + h) * a.vdim;
      for (int d = lane; d < a.P; d += 64) {
        float v = 0.f;
        if (d < n) {
          v = mine[d];
          if (a.values_out) a.values_out[at + d] = v;
          if (a.mix_other) v = (1.0f - a.mix) * v + a.mix * a.mix_other[at + d];
        }
        vd[(size_t)d * a.page] = from_float<TO>(v);
      }
    } else {
      const float* __restrict__ w = is_q ? a.q_norm : a.k_norm;
      const float rms = w || a.norm_turned ? 1.0f / sqrtf(wave_sum(ss) / (float)n + a.eps) : 1.f;
      TO* __restrict__ dst = is_q ? (TO*)a.q_out + ((size_t)t * a.Hq + h) * a.P
                                  : (TO*)a.k_cache + ((pg * a.Hkv + h) * a.page + off) * a.P;
      for (int i = lane; i < a.nf; i += 64) {
        float c, s, o1, o2;
        sincosf(pos * a.inv_freq[i], &s, &c);
        const int d1 = a.layout == LAYOUT_INTERLEAVED ? 2 * i : i, d2 = a.layout == LAYOUT_INTERLEAVED ? 2 * i + 1 : i + a.nf;
        const float x1 = w ? mine[d1] * rms * w[d1] : mine[d1] * rms, x2 = w ? mine[d2] * rms * w[d2] : mine[d2] * rms;
        rotate_pair(x1, x2, c * a.rot_scale, s * a.rot_scale, o1, o2);
        dst[d1] = from_float<TO>(o1);
        dst[d2] = from_float<TO>(o2);
      }
      for (int d = 2 * a.nf + lane; d < a.P; d += 64)
        dst[d] = from_float<TO>(d < n ? (w ? mine[d] * rms * w[d] : mine[d] * rms) : 0.f);
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");      // before the next head's numbers replace these
    __builtin_amdgcn_wave_barrier();
  }
}

// The same for steps with rows of many tokens: a workgroup a (16 tokens, share of the heads), a wave a head for all of the 16,
// four at a time.  A lane owns E channels of the head and carries their last inputs along, so that every number is read
// once; the angles' cosines and sines of the 16 tokens are made once a workgroup; where the 16 tokens fill a stretch of
// 16 slots of a page, the values of four go out as one run a dim.
template <typename TO, int KT, int E>
__global__ void __launch_bounds__(256)
qkv_conv_finish_tile_kernel(ConvFinishArgs a, int tokens) {
  constexpr int TT = 16, U = 4, keep = KT - 1;
  extern __shared__ __align__(16) float lds[];
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, P = a.P;
  float* cs = lds;                                            // [TT][nf] cosines, then sines
  float* sn = cs + TT * a.nf;
  float* mine = lds + 2 * TT * a.nf + (size_t)wv * U * P;     // the wave's normed heads of four tokens
  const int t_first = blockIdx.x * TT, t_end = t_first + TT < tokens ? t_first + TT : tokens;
  for (int i = threadIdx.x; i < TT * a.nf; i += 256) {
    const int tt = i / a.nf, f = i - tt * a.nf;
    float s, c;
    sincosf((float)a.positions[t_first + tt < t_end ? t_first + tt : t_end - 1] * a.inv_freq[f], &s, &c);
    cs[i] = c * a.rot_scale;
    sn[i] = s * a.rot_scale;
  }
  __syncthreads();
  // whether the 16 tokens fill one stretch of 16 slots of a page, in order (a row's tokens mostly do)
  const int slot0 = a.slots[t_first];
  const bool run = t_end - t_first == TT && a.page % TT == 0 && slot0 % TT == 0 &&
                   __builtin_amdgcn_ballot_w64(a.slots[t_first + (lane & (TT - 1) & (t_end - t_first - 1))] !=
                                               slot0 + (lane & (TT - 1) & (t_end - t_first - 1))) == 0;
  const int jobs = a.Hq + 2 * a.Hkv;
  for (int job = blockIdx.y * 4 + wv; job < jobs; job += gridDim.y * 4) {
    const bool is_q = job < a.Hq, is_v = job >= a.Hq + a.Hkv;
    const int h = is_q ? job : is_v ? job - a.Hq - a.Hkv : job - a.Hq;
    const int n = is_v ? a.vdim : a.dim;
    const int c0 = is_q ? h * a.dim : is_v ? (a.Hq + a.Hkv) * a.dim + h * a.vdim : (a.Hq + h) * a.dim;
    const float* __restrict__ w = is_q ? a.q_norm : a.k_norm;
    const bool normed = w || a.norm_turned;
    const float grown = a.norm_turned ? a.rot_scale * a.rot_scale : 1.f;      // what the rotation does to a pair's sum of squares
    float tp[E][KT], win[E][keep], wn[E], bi[E];
    int ch[E];                                                // the lane's channels, clamped into the head
#pragma unroll
    for (int e = 0; e < E; ++e) {
      const int d = lane + 64 * e;
      ch[e] = c0 + (d < n ? d : n - 1);
      wn[e] = !is_v && w && d < n ? w[d] : 1.f;
      bi[e] = a.col_bias ? a.col_bias[ch[e]] : 0.f;
#pragma unroll
      for (int k = 0; k < KT; ++k) tp[e][k] = a.taps[(size_t)ch[e] * KT + k];
    }
#pragma unroll 1
    for (int g = 0; g < TT; g += U) {
      float x[U][E], y[U][E], ss[U];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int t = t_first + g + u < t_end ? t_first + g + u : t_end - 1;
#pragma unroll
        for (int e = 0; e < E; ++e) x[u][e] = a.sums[(size_t)t * a.ld + a.col + ch[e]] + bi[e];
      }
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int t = t_first + g + u < t_end ? t_first + g + u : t_end - 1;
        const int r = a.token_row[t], j = t - a.row_start[r];
        if (g + u == 0 || j == 0) {                           // the inputs before this token: of its row, or from the tail
          const float* __restrict__ tl = a.tail + (size_t)a.state_slots[r] * keep * a.C;
#pragma unroll
          for (int e = 0; e < E; ++e)
#pragma unroll
            for (int i = 0; i < keep; ++i) {
              const int back = keep - i;
              win[e][i] = back <= j ? a.sums[(size_t)(t - back) * a.ld + a.col + ch[e]] + bi[e] : tl[(size_t)(keep + j - back) * a.C + ch[e]];
            }
        }
        ss[u] = 0.f;
#pragma unroll
        for (int e = 0; e < E; ++e) {
          float acc = 0.f;
#pragma unroll
          for (int i = 0; i < keep; ++i) acc = fmaf(tp[e][i], win[e][i], acc);
          acc = fmaf(tp[e][keep], x[u][e], acc);
#pragma unroll
          for (int i = 0; i + 1 < keep; ++i) win[e][i] = win[e][i + 1];
          win[e][keep - 1] = x[u][e];
          y[u][e] = lane + 64 * e < n ? acc : 0.f;
          ss[u] = fmaf(lane + 64 * e < 2 * a.nf ? grown * y[u][e] : y[u][e], y[u][e], ss[u]);
        }
      }
      if (is_v) {
        struct alignas(U * sizeof(TO)) Four { TO v[U]; } vals[E];
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const int t = t_first + g + u;
          if (t < t_end) {
            const size_t at = ((size_t)t * a.Hkv + h) * a.vdim;
#pragma unroll
            for (int e = 0; e < E; ++e) {
              const int d = lane + 64 * e;
              float v = y[u][e];
              if (d < n) {
                if (a.values_out) a.values_out[at + d] = v;
                if (a.mix_other) v = (1.0f - a.mix) * v + a.mix * a.mix_other[at + d];
              }
              vals[e].v[u] = from_float<TO>(v);
              if (!run && d < P) {
                const int slot = a.slots[t];
                ((TO*)a.v_cache)[(((size_t)(slot / a.page) * a.Hkv + h) * P + d) * a.page + slot % a.page] = vals[e].v[u];
              }
            }
          }
        }
        if (run) {
#pragma unroll
          for (int e = 0; e < E; ++e)
            if (lane + 64 * e < P)
              *reinterpret_cast<Four*>((TO*)a.v_cache + (((size_t)(slot0 / a.page) * a.Hkv + h) * P + lane + 64 * e) * a.page +
                                       slot0 % a.page + g) = vals[e];
        }
        continue;
      }
      if (normed) {
#pragma unroll
        for (int o = 32; o > 0; o >>= 1)
#pragma unroll
          for (int u = 0; u < U; ++u) ss[u] += __shfl_xor(ss[u], o, 64);
      }
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const float rms = normed ? 1.0f / sqrtf(ss[u] / (float)n + a.eps) : 1.f;
#pragma unroll
        for (int e = 0; e < E; ++e) {
          y[u][e] *= rms * wn[e];
          if (lane + 64 * e < P) mine[u * P + lane + 64 * e] = y[u][e];
        }
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      __builtin_amdgcn_wave_barrier();
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int t = t_first + g + u;
        if (t < t_end) {
          const int slot = a.slots[t];
          TO* __restrict__ dst = is_q ? (TO*)a.q_out + ((size_t)t * a.Hq + h) * P
                                      : (TO*)a.k_cache + (((size_t)(slot / a.page) * a.Hkv + h) * a.page + slot % a.page) * P;
#pragma unroll
          for (int e = 0; e < E; ++e) {
            const int d = lane + 64 * e;
            if (d < P) {
              float o = y[u][e];
              if (d < 2 * a.nf) {
                const bool half = a.layout == LAYOUT_HALF, low = half ? d < a.nf : (d & 1) == 0;
                const int f = half ? (low ? d : d - a.nf) : d >> 1, partner = half ? (low ? d + a.nf : f) : d ^ 1;
                const float c = cs[(g + u) * a.nf + f], s = sn[(g + u) * a.nf + f], other = mine[u * P + partner];
                o = low ? fmaf(o, c, -(other * s)) : fmaf(o, c, other * s);
              }
              dst[d] = from_float<TO>(o);
            }
          }
        }
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      __builtin_amdgcn_wave_barrier();
    }
  }
}

template <typename TO, int KT>
static void qkv_conv_tile_launch(const ConvFinishArgs& a, int tokens, hipStream_t s) {
  const int e = (a.P + 63) / 64;
  const size_t lds = ((size_t)2 * 16 * a.nf + (size_t)4 * 4 * a.P) * sizeof(float);
  const int tiles = (tokens + 15) / 16;
  int parts = (a.Hq + 2 * a.Hkv + 3) / 4;
  while (parts > 1 && (long)tiles * parts > 1536) parts = (parts + 1) / 2;       // a few workgroups a compute unit
#define QCT(E_) hipLaunchKernelGGL((qkv_conv_finish_tile_kernel<TO, KT, E_>), dim3(tiles, parts), dim3(256), lds, s, a, tokens)
  if (e <= 1) QCT(1);
  else if (e == 2) QCT(2);
  else QCT(4);
#undef QCT
}

MIE_EXPORT const char* attention_prep_last_error() { return g_mie_error; }

MIE_EXPORT int mie_qkv_finish(const float* sums, long ld, int q_col, int k_col, int v_col, const float* q_norm,
                              const float* k_norm, float eps, int norm_per_head, const float* inv_freq, int nf, int layout,
                              const float* q_head_scale, const int* positions, const int* slots, void* q_out, void* k_cache,
                              void* v_cache, int dtype, int tokens, int Hq, int Hkv, int dim, int vdim, int P, int page,
                              const float* col_bias, float temp_coef, int temp_every, hipStream_t s) {
  if (tokens <= 0) return 0;
  if (Hq <= 0 || Hkv <= 0 || dim <= 0 || vdim <= 0 || P < dim || P < vdim || page <= 0)
    MIE_FAIL("qkv_finish: %d / %d heads of %d (values %d) in %d, page %d", Hq, Hkv, dim, vdim, P, page);
  if (2 * nf > dim || nf < 0 || (nf > 0 && !inv_freq)) MIE_FAIL("qkv_finish: %d turned pairs in heads of %d", nf, dim);
  if (layout != LAYOUT_INTERLEAVED && layout != LAYOUT_HALF) MIE_FAIL("qkv_finish: layout code %d", layout);
  if (v_col < 0 && vdim != dim) MIE_FAIL("qkv_finish: values that are the keys have their size");
  if (temp_every < 0) MIE_FAIL("qkv_finish: a query temperature every %d positions", temp_every);
  FinishArgs a{sums, ld, q_col, k_col, v_col, q_norm, k_norm, eps, norm_per_head, inv_freq, nf, layout, q_head_scale, col_bias, temp_coef, temp_every,
               positions, slots, q_out, k_cache, v_cache, Hq, Hkv, dim, vdim, P, page};
  const size_t lds = (size_t)2 * (nf > 0 ? nf : 1) * sizeof(float);
  // few tokens: several workgroups a token, so that a decode step's few rows are spread over the GPU
  int parts = tokens >= 256 ? 1 : (Hq + Hkv + 3) / 4;
  parts = parts < 1 ? 1 : parts > 8 ? 8 : parts;
  if (dtype == MIE_F32) hipLaunchKernelGGL(qkv_finish_kernel<float>, dim3(tokens, parts), dim3(256), lds, s, a);
  else if (dtype == MIE_BF16) hipLaunchKernelGGL(qkv_finish_kernel<bf16>, dim3(tokens, parts), dim3(256), lds, s, a);
  else MIE_FAIL("qkv_finish: dtype code %d", dtype);
  MIE_CHECK_LAUNCH("qkv_finish");
  return 0;
}

template <typename T>
__global__ void __launch_bounds__(256)
head_gate_kernel(T* __restrict__ o, const float* __restrict__ gate, long ldg, int H, int D) {
  const int t = blockIdx.x;
  T* row = o + (size_t)t * H * D;
  for (int e = threadIdx.x; e < H * D; e += blockDim.x)
    row[e] = from_float<T>(to_float(row[e]) * mie_sigmoid(gate[(size_t)t * ldg + e / D]));
}

// gate points at the first gate column; rows are ldg floats apart
MIE_EXPORT int mie_head_gate(void* o, int dtype, const float* gate, long ldg, int tokens, int H, int D, hipStream_t s) {
  if (tokens <= 0) return 0;
  if (H <= 0 || D <= 0 || ldg < H) MIE_FAIL("head_gate: %d heads of %d, gate rows %ld apart", H, D, ldg);
  if (dtype == MIE_F32) hipLaunchKernelGGL(head_gate_kernel<float>, dim3(tokens), dim3(256), 0, s, (float*)o, gate, ldg, H, D);
  else if (dtype == MIE_BF16) hipLaunchKernelGGL(head_gate_kernel<bf16>, dim3(tokens), dim3(256), 0, s, (bf16*)o, gate, ldg, H, D);
  else MIE_FAIL("head_gate: dtype code %d", dtype);
  MIE_CHECK_LAUNCH("head_gate");
  return 0;
}

// taps [C, K] and tail [slots, max(1, K - 1), C] float32, C = (Hq + Hkv) dim + Hkv vdim channels that lie side by side in the
// sums from column col on.  move_tail: every row of the step is one token, and the tail moves on here; else the caller moves
// it afterwards.  col_bias float32 [C] or null.  norm_turned: q_norm and k_norm are null, and heads are divided by their root
// mean square after the rotation.  values_out, mix_other float32 [tokens, Hkv vdim] or null.
MIE_EXPORT int mie_qkv_conv_finish(const float* sums, long ld, int col, const float* col_bias, const float* taps, float* tail,
                                   const int* token_row, const int* row_start, const int* state_slots, int K, int move_tail,
                                   const float* q_norm, const float* k_norm, float eps, int norm_turned, const float* inv_freq, int nf,
                                   int layout, float rot_scale, const int* positions, const int* slots, float* values_out, const float* mix_other, float mix,
                                   void* q_out, void* k_cache, void* v_cache, int dtype, int tokens, int Hq, int Hkv, int dim,
                                   int vdim, int P, int page, hipStream_t s) {
  if (tokens <= 0) return 0;
  if (Hq <= 0 || Hkv <= 0 || dim <= 0 || vdim <= 0 || P < dim || P < vdim || page <= 0 || P > 1024)
    MIE_FAIL("qkv_conv_finish: %d / %d heads of %d (values %d) in %d (at most 1024), page %d", Hq, Hkv, dim, vdim, P, page);
  if (2 * nf > dim || nf < 0 || (nf > 0 && !inv_freq)) MIE_FAIL("qkv_conv_finish: %d turned pairs in heads of %d", nf, dim);
  if (K < 1 || !taps || !tail || !token_row || !row_start || !state_slots) MIE_FAIL("qkv_conv_finish: %d taps and their operands", K);
  if (layout != LAYOUT_INTERLEAVED && layout != LAYOUT_HALF) MIE_FAIL("qkv_conv_finish: layout code %d", layout);
  if (norm_turned && (q_norm || k_norm)) MIE_FAIL("qkv_conv_finish: norms after the rotation have no weights");
  const int C = (Hq + Hkv) * dim + Hkv * vdim;
  if (ld < (long)col + C) MIE_FAIL("qkv_conv_finish: %d channels from column %d in rows of %ld", C, col, ld);
  const int row_floats = (dim > vdim ? dim : vdim);
  ConvFinishArgs a{sums, ld, col, col_bias, taps, tail, token_row, row_start, state_slots, K, move_tail, q_norm, k_norm, eps, norm_turned,
                   inv_freq, nf, layout, rot_scale, positions, slots, values_out, mix_other, mix, q_out, k_cache, v_cache, Hq, Hkv, dim, vdim, P, page, C,
                   row_floats};
  // rows of many tokens: 16 tokens a workgroup (the angles' table of a workgroup has to fit beside the heads)
  if (tokens >= 64 && !move_tail && K >= 2 && K <= 4 && P <= 256 && nf <= 128) {
#define QCT_K(T_)                                        \
  switch (K) {                                           \
    case 2: qkv_conv_tile_launch<T_, 2>(a, tokens, s); break; \
    case 3: qkv_conv_tile_launch<T_, 3>(a, tokens, s); break; \
    default: qkv_conv_tile_launch<T_, 4>(a, tokens, s); \
  }
    if (dtype == MIE_F32) { QCT_K(float) }
    else if (dtype == MIE_BF16) { QCT_K(bf16) }
    else MIE_FAIL("qkv_conv_finish: dtype code %d", dtype);
#undef QCT_K
    MIE_CHECK_LAUNCH("qkv_conv_finish (tiles)");
    return 0;
  }
  const size_t lds = (size_t)4 * row_floats * sizeof(float);
  int parts = (Hq + 2 * Hkv + 3) / 4;
  const int most = tokens >= 1024 ? 4 : 16;
  parts = parts < most ? parts : most;
#define QCF(T_, K_) hipLaunchKernelGGL((qkv_conv_finish_kernel<T_, K_>), dim3(tokens, parts), dim3(256), lds, s, a)
#define QCF_K(T_)              \
  switch (K) {                 \
    case 2: QCF(T_, 2); break; \
    case 3: QCF(T_, 3); break; \
    case 4: QCF(T_, 4); break; \
    default: QCF(T_, 0);       \
  }
  if (dtype == MIE_F32) { QCF_K(float) }
  else if (dtype == MIE_BF16) { QCF_K(bf16) }
  else MIE_FAIL("qkv_conv_finish: dtype code %d", dtype);
#undef QCF_K
#undef QCF
  MIE_CHECK_LAUNCH("qkv_conv_finish");
  return 0;
}

template <typename T>
__global__ void __launch_bounds__(256)
gate_heads_kernel(const T* __restrict__ o, const float* __restrict__ gate, long ldg, T* __restrict__ out, long ldo, int H, int dv,
                  int P, float scale) {
  const int t = blockIdx.x;
  const T* __restrict__ row = o + (size_t)t * H * P;
  for (int e = blockIdx.y * blockDim.x + threadIdx.x; e < H * dv; e += gridDim.y * blockDim.x) {
    const int h = e / dv;
    out[(size_t)t * ldo + e] = from_float<T>(scale * to_float(row[h * P + e - h * dv]) * mie_sigmoid(gate[(size_t)t * ldg + e]));
  }
}

// gate points at the first gate column; rows of gate are ldg floats apart, rows of out ldo numbers
MIE_EXPORT int mie_gate_heads(const void* o, int dtype, const float* gate, long ldg, void* out, long ldo, int tokens, int H, int dv,
                              int P, float scale, hipStream_t s) {
  if (tokens <= 0) return 0;
  if (H <= 0 || dv <= 0 || P < dv || ldg < (long)H * dv || ldo < (long)H * dv)
    MIE_FAIL("gate_heads: %d heads of %d in %d, gate rows %ld apart, output rows %ld", H, dv, P, ldg, ldo);
  int by = (H * dv + 1023) / 1024;
  by = by > 16 ? 16 : by;
  if (dtype == MIE_F32)
    hipLaunchKernelGGL(gate_heads_kernel<float>, dim3(tokens, by), dim3(256), 0, s, (const float*)o, gate, ldg, (float*)out, ldo, H, dv, P, scale);
  else if (dtype == MIE_BF16)
    hipLaunchKernelGGL(gate_heads_kernel<bf16>, dim3(tokens, by), dim3(256), 0, s, (const bf16*)o, gate, ldg, (bf16*)out, ldo, H, dv, P, scale);
  else MIE_FAIL("gate_heads: dtype code %d", dtype);
  MIE_CHECK_LAUNCH("gate_heads");
  return 0;
}
