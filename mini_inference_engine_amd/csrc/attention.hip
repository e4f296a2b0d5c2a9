// Paged causal attention, one kernel for every kind of row (single decoded tokens and prompt
// portions starting anywhere), in true 32-bit arithmetic for float and bfloat16 storage.
//
// One wavefront per (token, query head).  The token sits in row r at absolute position p and
// sees keys lo..p of its own request, lo = max(0, p - window + 1) or 0 (with a chunk size c
// also lo >= floor(p / c) * c: a query sees its own chunk of positions only), found through the
// row's block table in caches laid out [pages, Hkv, page, D] (keys) and [pages, Hkv, D, page]
// (values, transposed within a page).  Keys are taken 64 at a time
// (one per lane: q . k in increasing d), the softmax is kept online in 32-bit, and the 64
// probabilities then weight the value rows with the lanes spread over D.  The order of every
// sum depends only on (lo, p): the result for a token is bit-identical whatever else the
// step holds and however the request was cut into steps.  With a sink, one more term exp(sink)
// joins the softmax's denominator at the end and has no value.  With a cap c the scaled scores
// pass through c * tanh(score / c).  In the sigmoid mode there is no softmax: a visible key counts
// with sigmoid(score + the head's bias), and the weights are not normalised.  With a distance bias a key n
// positions back adds a number of its head's table to the score.  With a window and kept first keys a query also
// sees keys 0 .. keep - 1, taken before the window's.  The sink may be a number a query head.
//
// This is the reference kernel of the engine: the float32 path runs on it, and the
// bfloat16 path uses it wherever a faster kernel does not take the shape.
#include "common.hpp"

template <typename T> struct Pack;
template <> struct Pack<float> {
  typedef float4 V;
  static constexpr int N = 4;
  __device__ static __forceinline__ void unpack(const V& v, float* f) { f[0] = v.x; f[1] = v.y; f[2] = v.z; f[3] = v.w; }
};
template <> struct Pack<bf16> {
  typedef uint4 V;
  static constexpr int N = 8;
  __device__ static __forceinline__ void unpack(const V& v, float* f) {
    const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f[2 * i] = __uint_as_float(w[i] << 16);
      f[2 * i + 1] = __uint_as_float(w[i] & 0xFFFF0000u);
    }
  }
};

#define ATT_MAX_D 1024     // head sizes up to 256 run with four accumulators a lane, larger ones with sixteen

template <typename T, int NR>
__global__ void __launch_bounds__(64)
paged_attention_kernel(const T* __restrict__ q, long q_stride, const T* __restrict__ k_cache,
                       const T* __restrict__ v_cache, T* __restrict__ out, const int* __restrict__ block_tables,
                       int max_blocks, const int* __restrict__ token_row, const int* __restrict__ positions, int Hq,
                       int Hkv, int D, int page, float scale, int window, int has_sink, float sink, int chunk,
                       float softcap, int sigmoid, const float* __restrict__ head_bias,
                       const float* __restrict__ dist_bias, int dist_n, int keep, const float* __restrict__ head_sinks) {
  __shared__ float qs[NR * 64];
  __shared__ float ps[64];
  __shared__ long long base[64];     // per key of the chunk: offset of its value column
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const int row = token_row[t], pos = positions[t];
  const int kvh = h / (Hq / Hkv);
  int lo = window > 0 ? (pos - window + 1 > 0 ? pos - window + 1 : 0) : 0;
  if (chunk > 0 && pos / chunk * chunk > lo) lo = pos / chunk * chunk;
  const float hb = sigmoid && head_bias ? head_bias[h] : 0.f;
  const float* db = dist_bias ? dist_bias + (size_t)h * dist_n : nullptr;
  const int* bt = block_tables + (size_t)row * max_blocks;
  const T* qp = q + (size_t)t * q_stride + (size_t)h * D;
  for (int d = lane; d < D; d += 64) qs[d] = to_float(qp[d]);
  __syncthreads();

  typedef Pack<T> P;
  float m = -INFINITY, l = 0.f;
  float acc[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) acc[i] = 0.f;

  const int kept = keep < lo ? keep : lo;             // keys [0, kept) first, then [lo, pos]
  for (int c0 = kept > 0 ? 0 : lo, next; c0 <= pos; c0 = next) {
    const int limit = c0 < kept ? kept : pos + 1;     // end of this stretch of keys
    next = c0 + 64;
    if (c0 < kept && next >= kept) next = lo;
    const int key = c0 + lane;
    const bool valid = key < limit;
    float s = -INFINITY;
    if (valid) {
      const int pg = bt[key / page];
      const long long off = (((long long)pg * Hkv + kvh) * page + key % page) * D;
      base[lane] = ((long long)pg * Hkv + kvh) * page * D + key % page;
      const typename P::V* kp = reinterpret_cast<const typename P::V*>(k_cache + off);
      float dot = 0.f;
      for (int d0 = 0; d0 < D; d0 += P::N) {
        float f[P::N];
        P::unpack(kp[d0 / P::N], f);
#pragma unroll
        for (int e = 0; e < P::N; ++e) dot = fmaf(qs[d0 + e], f[e], dot);
      }
      s = dot * scale;
      if (softcap > 0.f) s = softcap * tanhf(s / softcap);
      if (db) s += db[pos - key < dist_n ? pos - key : dist_n - 1];
    }
    float alpha = 1.f, p;
    if (sigmoid) {
      p = valid ? mie_sigmoid(s + hb) : 0.f;
    } else {
      const float m_new = fmaxf(m, wave_max(s));    // finite: key c0 < limit is valid
      alpha = expf(m - m_new);                      // 0 on the first chunk (m = -inf)
      p = valid ? expf(s - m_new) : 0.f;
      l = l * alpha + wave_sum(p);
      m = m_new;
    }
    ps[lane] = p;
    __syncthreads();
    const int nk = limit - c0 < 64 ? limit - c0 : 64;
#pragma unroll
    for (int i = 0; i < NR; ++i) acc[i] *= alpha;
    for (int j = 0; j < nk; ++j) {
      const float pj = ps[j];
      const T* vp = v_cache + base[j];
#pragma unroll
      for (int i = 0; i < NR; ++i) {
        const int d = lane + 64 * i;
        if (d < D) acc[i] = fmaf(pj, to_float(vp[(size_t)d * page]), acc[i]);
      }
    }
    __syncthreads();
  }
  if (head_sinks) sink = head_sinks[h];
  if (has_sink && !sigmoid) {                     // one more term exp(sink) in the denominator, with no value
    const float m_new = fmaxf(m, sink);
    const float alpha = expf(m - m_new);
    l = l * alpha + expf(sink - m_new);
#pragma unroll
    for (int i = 0; i < NR; ++i) acc[i] *= alpha;
  }
  const float inv = sigmoid ? 1.0f : 1.0f / l;
  T* op = out + ((size_t)t * Hq + h) * D;
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int d = lane + 64 * i;
    if (d < D) op[d] = from_float<T>(acc[i] * inv);
  }
}

MIE_EXPORT const char* attention_last_error() { return g_mie_error; }

static int paged_attention_launch(const void* q, long q_stride, const void* k_cache, const void* v_cache, void* out,
                                   int dtype, const int* block_tables, int max_blocks, const int* token_row,
                                   const int* positions, int tokens, int Hq, int Hkv, int D, int page, float scale,
                                   int window, int has_sink, float sink, int chunk, float softcap, int sigmoid,
                                   const float* head_bias, const float* dist_bias, int dist_n, int keep,
                                   const float* head_sinks, hipStream_t stream) {
  if (tokens <= 0) return 0;
  if (keep < 0 || (keep > 0 && window <= 0)) MIE_FAIL("paged_attention: %d kept first keys belong beside a window", keep);
  if (dist_bias && dist_n < 1) MIE_FAIL("paged_attention: a distance bias of %d entries a head", dist_n);
  if (chunk < 0 || softcap < 0.f) MIE_FAIL("paged_attention: chunk %d, score cap %g", chunk, (double)softcap);
  if (sigmoid && has_sink) MIE_FAIL("paged_attention: a sink belongs to a softmax; the weights asked for are sigmoids");
  if (D % 16 || D < 16 || D > ATT_MAX_D) MIE_FAIL("paged_attention: head_dim %d (multiples of 16 up to %d)", D, ATT_MAX_D);
  if (Hkv <= 0 || Hq % Hkv) MIE_FAIL("paged_attention: %d query heads on %d kv heads", Hq, Hkv);
  if (Hq > 65535) MIE_FAIL("paged_attention: %d query heads is beyond the grid", Hq);
  if (page <= 0 || max_blocks <= 0) MIE_FAIL("paged_attention: page %d, max_blocks %d", page, max_blocks);
  if (q_stride < (long)Hq * D) MIE_FAIL("paged_attention: q row stride %ld < %d", q_stride, Hq * D);
  dim3 grid(tokens, Hq), block(64);
#define PA_LAUNCH(T_, NR_)                                                                                               \
  hipLaunchKernelGGL((paged_attention_kernel<T_, NR_>), grid, block, 0, stream, (const T_*)q, q_stride, (const T_*)k_cache, \
                     (const T_*)v_cache, (T_*)out, block_tables, max_blocks, token_row, positions, Hq, Hkv, D, page, scale,  \
                     window, has_sink, sink, chunk, softcap, sigmoid, head_bias, dist_bias, dist_n, keep, head_sinks)
  if (dtype == MIE_F32 && D <= 256) PA_LAUNCH(float, 4);
  else if (dtype == MIE_F32) PA_LAUNCH(float, 16);
  else if (dtype == MIE_BF16 && D <= 256) PA_LAUNCH(bf16, 4);
  else if (dtype == MIE_BF16) PA_LAUNCH(bf16, 16);
  else MIE_FAIL("paged_attention: dtype code %d", dtype);
#undef PA_LAUNCH
  MIE_CHECK_LAUNCH("paged_attention");
  return 0;
}

MIE_EXPORT int mie_paged_attention(const void* q, long q_stride, const void* k_cache, const void* v_cache, void* out,
                                   int dtype, const int* block_tables, int max_blocks, const int* token_row,
                                   const int* positions, int tokens, int Hq, int Hkv, int D, int page, float scale,
                                   int window, int has_sink, float sink, hipStream_t stream) {
  return paged_attention_launch(q, q_stride, k_cache, v_cache, out, dtype, block_tables, max_blocks, token_row, positions,
                                tokens, Hq, Hkv, D, page, scale, window, has_sink, sink, 0, 0.f, 0, nullptr, nullptr, 0, 0, nullptr, stream);
}

// The same with what a design may put between scores and weights: a chunk size (0: none), a cap on the scores
// (0: none), sigmoid weights with a bias per query head (head_bias float32 [Hq] or null) instead of the softmax, a bias
// on the score by the key's distance (dist_bias float32 [Hq, dist_n] or null: a key n positions back adds entry
// min(n, dist_n - 1) of the head's row, after scale and cap), keep first keys beside the window (0: none), a sink per
// query head (head_sinks float32 [Hq] or null; has_sink is then set).
MIE_EXPORT int mie_paged_attention_scored(const void* q, long q_stride, const void* k_cache, const void* v_cache, void* out,
                                          int dtype, const int* block_tables, int max_blocks, const int* token_row,
                                          const int* positions, int tokens, int Hq, int Hkv, int D, int page, float scale,
                                          int window, int has_sink, float sink, int chunk, float softcap, int sigmoid,
                                          const float* head_bias, const float* dist_bias, int dist_n, int keep,
                                          const float* head_sinks, hipStream_t stream) {
  return paged_attention_launch(q, q_stride, k_cache, v_cache, out, dtype, block_tables, max_blocks, token_row, positions,
                                tokens, Hq, Hkv, D, page, scale, window, has_sink, sink, chunk, softcap, sigmoid, head_bias,
                                dist_bias, dist_n, keep, head_sinks, stream);
}
