// Attention over the paged cache, general kernel: any value size up to 512, any key size up to 4096, any number
// of heads and groups, any page size, optional window or chunks, float32 or bfloat16.
//
// One wave per (query token, head).  Keys are taken 64 at a time: each lane scores one
// key (a full dot product with the query, which sits in LDS), the tile's maximum and
// sum update the running softmax in float32, then lanes switch to owning output
// elements and add p_j * V[j] for the tile's keys.  The order of keys is ascending and
// does not depend on what else is in the batch or on which pages hold the keys.
//
// Query token t belongs to request r = token_req[t]; its position is
// context_lens[r] - q_len_r + (t - cu_seqlens[r]) and it sees keys lo..pos with
// lo = max(0, pos - window + 1) when window > 0, pos - pos mod chunk when chunk > 0, else 0.
//
// Capped scores: with softcap > 0 a scaled score s becomes softcap * tanh(s / softcap) before the softmax.
//
// Kept first keys: with keep_first > 0 a windowed query also sees keys 0..keep_first-1 (those of them that lie
// before lo; they are visited first, so the order of keys stays ascending).
// Sink: with sink [heads] float32 the softmax's denominator holds one more term, exp(sink[h]), that has no key and
// no value; it is added once, after the last key, whatever the scale.
//
// Optional bias by distance: dist_bias [heads, bias_len] float32 is added to the scaled score of query position
// pos and key j as dist_bias[h, min(pos - j, bias_len - 1)] (the scale does not multiply it).
#include <math.h>

#include "common.h"

#define ATT_MAX_ACC 8      // value size <= 64 * ATT_MAX_ACC
#define ATT_MAX_KEY 4096   // key size (the query row lies in LDS)

template <typename T>
__global__ __launch_bounds__(64) void paged_attention_kernel(
    const T* __restrict__ q, const T* __restrict__ k_cache, const T* __restrict__ v_cache,
    const int* __restrict__ block_tables, int table_width, const int* __restrict__ cu_seqlens,
    const int* __restrict__ context_lens, const int* __restrict__ token_req, T* __restrict__ out, int n_heads,
    int n_kv, int head_dim, int page_size, float scale, int window, const float* __restrict__ dist_bias, int bias_len,
    int value_dim, int keep_first, const float* __restrict__ sink, int chunk, float softcap) {
  extern __shared__ float qs[];  // the query row, float32
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const int r = token_req[t];
  const int q_start = cu_seqlens[r];
  const int q_len = cu_seqlens[r + 1] - q_start;
  const int pos = context_lens[r] - q_len + (t - q_start);
  const int lo = chunk > 0 ? pos / chunk * chunk : (window > 0 && pos - window + 1 > 0) ? pos - window + 1 : 0;
  const int kvh = h / (n_heads / n_kv);
  const T* qrow = q + ((size_t)t * n_heads + h) * head_dim;
  for (int d = lane; d < head_dim; d += TP_WAVE) qs[d] = to_float(qrow[d]);
  __syncthreads();
  const int* table = block_tables + (size_t)r * table_width;

  float m = -INFINITY, l = 0.f;
  float acc[ATT_MAX_ACC];
#pragma unroll
  for (int i = 0; i < ATT_MAX_ACC; ++i) acc[i] = 0.f;

  // two runs of keys: the kept first ones that the window has left behind, then the window (or everything)
  const int kept_end = (keep_first > 0 && lo > 0) ? min(keep_first, lo) : 0;
  for (int seg = kept_end > 0 ? 0 : 1; seg < 2; ++seg) {
  const int seg_lo = seg == 0 ? 0 : lo, seg_hi = seg == 0 ? kept_end - 1 : pos;
  for (int j0 = seg_lo; j0 <= seg_hi; j0 += TP_WAVE) {
    const int j = j0 + lane;
    const bool valid = j <= seg_hi;
    int row = 0;   // cache row of this lane's key: (page * n_kv + kvh) * page_size + offset
    int vbase = 0; // its value column: values are stored [page, kv_head, head_dim, page_size]
    float s = -INFINITY;
    if (valid) {
      const int page = table[j / page_size];
      row = (page * n_kv + kvh) * page_size + j % page_size;
      vbase = (page * n_kv + kvh);
      const T* kr = k_cache + (size_t)row * head_dim;
      float dot = 0.f;
      for (int d = 0; d < head_dim; ++d) dot = fmaf(qs[d], to_float(kr[d]), dot);
      s = dot * scale;
      if (softcap > 0.f) s = softcap * tanhf(s / softcap);
      if (dist_bias != nullptr) s += dist_bias[(size_t)h * bias_len + min(pos - j, bias_len - 1)];
    }
    const float m_new = fmaxf(m, wave_max(s));
    const float alpha = expf(m - m_new);  // first tile: exp(-inf) = 0
    const float p = valid ? expf(s - m_new) : 0.f;
    l = l * alpha + wave_sum(p);
    m = m_new;
#pragma unroll
    for (int i = 0; i < ATT_MAX_ACC; ++i) acc[i] *= alpha;
    const int n_valid = min(TP_WAVE, seg_hi - j0 + 1);
    for (int jj = 0; jj < n_valid; ++jj) {
      const float pj = __shfl(p, jj, TP_WAVE);
      const int vb = __shfl(vbase, jj, TP_WAVE);
      const T* vr = v_cache + (size_t)vb * value_dim * page_size + (j0 + jj) % page_size;
#pragma unroll
      for (int i = 0; i < ATT_MAX_ACC; ++i) {
        const int d = lane + i * TP_WAVE;
        if (d < value_dim) acc[i] = fmaf(pj, to_float(vr[(size_t)d * page_size]), acc[i]);
      }
    }
  }
  }
  if (sink != nullptr) {
    const float sk = sink[h];
    const float m_new = fmaxf(m, sk);
    const float alpha = expf(m - m_new);
    l = l * alpha + expf(sk - m_new);
#pragma unroll
    for (int i = 0; i < ATT_MAX_ACC; ++i) acc[i] *= alpha;
  }
  const float inv = 1.0f / l;
  T* o = out + ((size_t)t * n_heads + h) * value_dim;
#pragma unroll
  for (int i = 0; i < ATT_MAX_ACC; ++i) {
    const int d = lane + i * TP_WAVE;
    if (d < value_dim) from_float(o + d, acc[i] * inv);
  }
}

// Defined in attention_mfma.hip: takes bfloat16 shapes it is built for, returns -1 otherwise.
int tp_paged_attention_fast(const void* q, const void* k_cache, const void* v_cache, const int* block_tables,
                            int table_width, const int* cu_seqlens, const int* context_lens, void* out, int n_tokens,
                            int n_req, int n_heads, int n_kv, int head_dim, int page_size, float scale, int window,
                            int max_q_len, int num_single, int num_splits, float* scratch, const int* token_req,
                            int portion_splits, int portion_min_steps, float* portion_scratch, const float* dist_bias,
                            int bias_len, int keep_first, const float* sink, int value_dim, int chunk, float softcap,
                            hipStream_t s);

extern "C" int tp_paged_attention(const void* q, int dt, const void* k_cache, const void* v_cache,
                                  const int* block_tables, int table_width, const int* cu_seqlens,
                                  const int* context_lens, const int* token_req, void* out, int n_tokens,
                                  int n_req, int n_heads, int n_kv, int head_dim, int page_size, float scale,
                                  int window, int max_q_len, int max_ctx, int allow_fast, int num_single,
                                  int num_splits, float* scratch, int portion_splits, int portion_min_steps,
                                  float* portion_scratch, const float* dist_bias, int bias_len, int value_dim,
                                  int keep_first, const float* sink, int chunk, float softcap, hipStream_t s) {
  // value_dim: the size of a value head (0: head_dim): v_cache is [page, kv_head, value_dim, page_size] and out
  // [n, heads * value_dim]; the matrix-core kernels take equal sizes and a few pairs with wider keys.
  if (value_dim <= 0) value_dim = head_dim;
  // num_single: how many requests bring exactly one token (they go to the split decode kernel,
  // which, with more than one split, needs `scratch` of n_req * n_heads * num_splits * (head_dim + 2)
  // floats).  portion_splits > 1: the keys of every longer request are split over that many blocks,
  // which needs `portion_scratch` of n_tokens * n_heads * portion_splits * (head_dim + 4) floats.
  TP_REQUIRE(n_tokens >= 0 && n_req >= 0 && n_heads > 0 && n_kv > 0 && head_dim > 0 && page_size > 0,
             "paged_attention: bad sizes");
  TP_REQUIRE(n_heads % n_kv == 0, "paged_attention: %d heads is not a multiple of %d kv heads", n_heads, n_kv);
  TP_REQUIRE(head_dim <= ATT_MAX_KEY && value_dim <= TP_WAVE * ATT_MAX_ACC, "paged_attention: head sizes %d / %d exceed %d / %d",
             head_dim, value_dim, ATT_MAX_KEY, TP_WAVE * ATT_MAX_ACC);
  TP_REQUIRE(window >= 0, "paged_attention: window must be >= 0");
  TP_REQUIRE(keep_first >= 0, "paged_attention: keep_first must be >= 0");
  TP_REQUIRE(chunk >= 0 && (chunk == 0 || window == 0), "paged_attention: chunks and a window exclude each other");
  TP_REQUIRE(softcap >= 0.f && (softcap == 0.f || dist_bias == nullptr), "paged_attention: a cap and a distance bias exclude each other");
  if (chunk == 1) {   // (a chunk of one position: the query itself)
    chunk = 0;
    window = 1;
  }
  if (window == 0) keep_first = 0;   // (without a window every key is seen anyway)
  TP_REQUIRE(n_heads <= 65535, "paged_attention: too many heads");
  if (n_tokens == 0) return 0;
  TP_REQUIRE(dist_bias == nullptr || bias_len > 0, "paged_attention: empty distance bias table");
  if (dt == TP_BF16 && allow_fast) {
    const int rc = tp_paged_attention_fast(q, k_cache, v_cache, block_tables, table_width, cu_seqlens,
                                           context_lens, out, n_tokens, n_req, n_heads, n_kv, head_dim,
                                           page_size, scale, window, max_q_len, num_single, num_splits, scratch, token_req,
                                           portion_splits, portion_min_steps, portion_scratch, dist_bias, bias_len, keep_first, sink, value_dim, chunk,
                                           softcap, s);
    if (rc >= 0) return rc;
  }
  const dim3 grid(n_tokens, n_heads);
  const size_t shmem = (size_t)head_dim * sizeof(float);
  if (dt == TP_F32)
    hipLaunchKernelGGL(paged_attention_kernel<float>, grid, dim3(64), shmem, s, (const float*)q,
                       (const float*)k_cache, (const float*)v_cache, block_tables, table_width, cu_seqlens,
                       context_lens, token_req, (float*)out, n_heads, n_kv, head_dim, page_size, scale, window, dist_bias, bias_len, value_dim, keep_first, sink, chunk, softcap);
  else if (dt == TP_BF16)
    hipLaunchKernelGGL(paged_attention_kernel<bf16_t>, grid, dim3(64), shmem, s, (const bf16_t*)q,
                       (const bf16_t*)k_cache, (const bf16_t*)v_cache, block_tables, table_width, cu_seqlens,
                       context_lens, token_req, (bf16_t*)out, n_heads, n_kv, head_dim, page_size, scale, window, dist_bias, bias_len, value_dim, keep_first, sink, chunk, softcap);
  else
    TP_REQUIRE(false, "paged_attention: unknown dtype %d", dt);
  TP_CHECK_LAUNCH("paged_attention");
  return 0;
}
