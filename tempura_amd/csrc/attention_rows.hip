// What lies between an attention's float32 projection rows and its cache, and between its heads' outputs and the
// output product, for attentions that need more than a rotation there:
//  * qkv_rows: biases on q, k and v, an RMS norm over the whole q and the whole k projection or over each of their heads,
//    rotation of q and k, rotation of the values by their own positions, cache write;
//  * latent_rows_write: queries into a latent's space beside one normed latent and one rotated key part a token;
//  * turn_gate: outputs turned back by the query's position and multiplied by a sigmoid gate.
// All pairs that turn together are neighbouring elements (2 i, 2 i + 1) of a head.  Float32 arithmetic throughout; a row's
// result depends on no other row and not on how the launch is cut.
#include <math.h>

#include "common.h"

template <int V>
struct Elems {
  float x[V];
};
template <int V>
__device__ inline Elems<V> load_elems(const float* p) {
  Elems<V> r;
  if constexpr (V == 4) {
    const float4 f = *(const float4*)p;
    r.x[0] = f.x; r.x[1] = f.y; r.x[2] = f.z; r.x[3] = f.w;
  } else {
    r.x[0] = p[0];
    r.x[1] = p[1];
  }
  return r;
}
template <int V, typename T>
__device__ inline void store_elems(T* p, const Elems<V>& r) {
  if constexpr (V == 4) {
    from_float4(p, r.x[0], r.x[1], r.x[2], r.x[3]);
  } else {
    from_float(p, r.x[0]);
    from_float(p + 1, r.x[1]);
  }
}

// Turns the pairs of elements i, i + 1, .. (i even) of one head that lie below 2 * half by position * inv_freq[pair]
// (table: this step's cosines and sines [n, half], or nullptr); sign -1 turns back.
template <int V>
__device__ inline void turn_pairs(Elems<V>& r, int i, int half, int t, int pos, const double* inv_freq, const float2* table,
                                  float factor, float sign) {
#pragma unroll
  for (int e = 0; e < V / 2; ++e) {
    const int pr = i / 2 + e;
    if (pr >= half) continue;
    float c, sn;
    if (table != nullptr) {
      const float2 cs = table[(size_t)t * half + pr];
      c = cs.x;
      sn = cs.y;
    } else {
      rope_cos_sin(pos, inv_freq[pr], factor, c, sn);
    }
    sn *= sign;
    const float a = r.x[2 * e], b = r.x[2 * e + 1];
    r.x[2 * e] = a * c - b * sn;
    r.x[2 * e + 1] = a * sn + b * c;
  }
}

struct QkvRows {
  const float* rows;        // [n, stride]: q heads | k heads | v heads (more columns may follow)
  size_t stride;
  const float *q_bias, *k_bias, *v_bias;   // per column, or nullptr
  const float *q_norm, *k_norm;            // weights of the norm over the whole projection, or nullptr
  float eps;
  const int *positions, *slots;            // slots: page * page_size + offset
  const double* inv_freq;
  const float2* table;
  int rotary_dim;
  float factor;
  const double* v_inv_freq;                // [vdim / 2], or nullptr: values are not turned
  const float2* v_table;
  int heads, kv, dim, vdim, out_dim, page_size;
  int q_slices, k_slices, v_slices;        // blocks a token, per section
  int per_slice;                           // groups of V elements a block stores
};

// grid: (tokens, q_slices + k_slices + v_slices).  Every block of a section forms the section's sum of squares itself
// (from the same elements in the same order) and stores its slice.
template <typename T, int V>
__global__ __launch_bounds__(256) void qkv_rows_kernel(QkvRows a, T* __restrict__ q_out, T* __restrict__ k_cache, T* __restrict__ v_cache) {
  __shared__ float scratch[32];
  const int t = blockIdx.x;
  int slice = blockIdx.y, sec = 0;
  if (slice >= a.q_slices) {
    slice -= a.q_slices;
    sec = 1;
    if (slice >= a.k_slices) {
      slice -= a.k_slices;
      sec = 2;
    }
  }
  const int qd = a.heads * a.dim, kd = a.kv * a.dim;
  const int width = sec == 0 ? qd : sec == 1 ? kd : a.kv * a.vdim;
  const int hdim = sec == 2 ? a.vdim : a.dim;
  const float* row = a.rows + (size_t)t * a.stride + (sec == 0 ? 0 : sec == 1 ? qd : qd + kd);
  const float* bias = sec == 0 ? a.q_bias : sec == 1 ? a.k_bias : a.v_bias;
  const float* w = sec == 0 ? a.q_norm : sec == 1 ? a.k_norm : nullptr;
  float rstd = 1.f;
  if (w != nullptr) {   // (uniform over the block)
    float ss = 0.f;
    for (int g = threadIdx.x; g < width / V; g += blockDim.x) {
      Elems<V> x = load_elems<V>(row + g * V);
      if (bias != nullptr) {
        const Elems<V> b = load_elems<V>(bias + g * V);
#pragma unroll
        for (int e = 0; e < V; ++e) x.x[e] += b.x[e];
      }
#pragma unroll
      for (int e = 0; e < V; ++e) ss = fmaf(x.x[e], x.x[e], ss);
    }
    ss = block_sum(ss, scratch);
    rstd = 1.0f / sqrtf(ss / (float)width + a.eps);
  }
  const int slot = a.slots[t], pos = a.positions[t];
  const size_t page = (size_t)(slot / a.page_size), off = (size_t)(slot % a.page_size);
  const int end = min(width / V, (slice + 1) * a.per_slice);
  for (int g = slice * a.per_slice + threadIdx.x; g < end; g += blockDim.x) {
    const int h = g * V / hdim, i = g * V % hdim;
    Elems<V> x = load_elems<V>(row + g * V);
    if (bias != nullptr) {
      const Elems<V> b = load_elems<V>(bias + g * V);
#pragma unroll
      for (int e = 0; e < V; ++e) x.x[e] += b.x[e];
    }
    if (w != nullptr) {
      const Elems<V> wv = load_elems<V>(w + g * V);
#pragma unroll
      for (int e = 0; e < V; ++e) x.x[e] = x.x[e] * rstd * wv.x[e];
    }
    if (sec == 2) {
      if (a.v_inv_freq != nullptr) turn_pairs<V>(x, i, a.vdim / 2, t, pos, a.v_inv_freq, a.v_table, 1.0f, 1.0f);
      T* o = v_cache + ((page * a.kv + h) * a.vdim + i) * a.page_size + off;
#pragma unroll
      for (int e = 0; e < V; ++e) from_float(o + (size_t)e * a.page_size, x.x[e]);
      continue;
    }
    turn_pairs<V>(x, i, a.rotary_dim / 2, t, pos, a.inv_freq, a.table, a.factor, 1.0f);
    T* o = sec == 0 ? q_out + ((size_t)t * a.heads + h) * a.out_dim : k_cache + ((page * a.kv + h) * a.page_size + off) * a.out_dim;
    store_elems<V>(o + i, x);
    Elems<V> zero;
#pragma unroll
    for (int e = 0; e < V; ++e) zero.x[e] = 0.f;
    for (int z = a.dim + i; z < a.out_dim; z += a.dim) store_elems<V>(o + z, zero);   // (zeros behind the head's own elements)
  }
}

// The same with a norm over every head by itself (weights q_norm and k_norm [dim], shared by the heads; nullptr: no norm):
// `group` neighbouring lanes (a power of two) take one head of one token.  units: tokens times per_token, the heads of a
// token that this launch takes (q, k and, in short steps, v).
template <typename T, int V>
__global__ __launch_bounds__(256) void qkv_heads_kernel(QkvRows a, long units, int per_token, int group, T* __restrict__ q_out, T* __restrict__ k_cache,
                                                        T* __restrict__ v_cache) {
  const long mine = ((long)blockIdx.x * 256 + threadIdx.x) / group, unit = min(mine, units - 1);   // (every lane takes part in the sums)
  const int lane = threadIdx.x % group;
  const int t = (int)(unit / per_token), hh = (int)(unit % per_token);
  const int sec = hh < a.heads ? 0 : hh < a.heads + a.kv ? 1 : 2;
  const int h = sec == 0 ? hh : sec == 1 ? hh - a.heads : hh - a.heads - a.kv;
  const int hdim = sec == 2 ? a.vdim : a.dim;
  const int qd = a.heads * a.dim, kd = a.kv * a.dim;
  const float* row = a.rows + (size_t)t * a.stride + (sec == 0 ? 0 : sec == 1 ? qd : qd + kd) + (size_t)h * hdim;
  const float* bias = sec == 0 ? a.q_bias : sec == 1 ? a.k_bias : a.v_bias;
  if (bias != nullptr) bias += (size_t)h * hdim;
  const float* w = sec == 0 ? a.q_norm : sec == 1 ? a.k_norm : nullptr;
  auto load = [&](int i) {
    Elems<V> x = load_elems<V>(row + i);
    if (bias != nullptr) {
      const Elems<V> b = load_elems<V>(bias + i);
#pragma unroll
      for (int e = 0; e < V; ++e) x.x[e] += b.x[e];
    }
    return x;
  };
  float rstd = 1.f;
  if (a.q_norm != nullptr) {   // (uniform over the wave; a value head's sum is not used)
    float ss = 0.f;
    for (int i = lane * V; i < hdim; i += group * V) {
      const Elems<V> x = load(i);
#pragma unroll
      for (int e = 0; e < V; ++e) ss = fmaf(x.x[e], x.x[e], ss);
    }
    ss = lanes_sum_of(ss, group);
    rstd = 1.0f / sqrtf(ss / (float)hdim + a.eps);
  }
  if (mine >= units) return;
  const int pos = a.positions[t], slot = a.slots[t];
  const size_t page = (size_t)(slot / a.page_size), off = (size_t)(slot % a.page_size);
  if (sec == 2) {
    T* o = v_cache + ((page * a.kv + h) * a.vdim) * a.page_size + off;
    for (int i = lane * V; i < hdim; i += group * V) {
      Elems<V> x = load(i);
      if (a.v_inv_freq != nullptr) turn_pairs<V>(x, i, a.vdim / 2, t, pos, a.v_inv_freq, a.v_table, 1.0f, 1.0f);
#pragma unroll
      for (int e = 0; e < V; ++e) from_float(o + (size_t)(i + e) * a.page_size, x.x[e]);
    }
    return;
  }
  T* o = sec == 0 ? q_out + ((size_t)t * a.heads + h) * a.out_dim : k_cache + ((page * a.kv + h) * a.page_size + off) * a.out_dim;
  for (int i = lane * V; i < a.out_dim; i += group * V) {
    Elems<V> x;
    if (i < hdim) {
      x = load(i);
      if (w != nullptr) {
        const Elems<V> wv = load_elems<V>(w + i);
#pragma unroll
        for (int e = 0; e < V; ++e) x.x[e] = x.x[e] * rstd * wv.x[e];
      }
      turn_pairs<V>(x, i, a.rotary_dim / 2, t, pos, a.inv_freq, a.table, a.factor, 1.0f);
    } else {   // (zeros behind the head's own elements)
#pragma unroll
      for (int e = 0; e < V; ++e) x.x[e] = 0.f;
    }
    store_elems<V>(o + i, x);
  }
}

// The values of long steps: a thread takes one element of one head for sixteen consecutive tokens and stores each run
// of eight places that starts at a multiple of eight as one piece of the transposed layout.
// grid: (ceil(n / 16), kv heads); block: vdim threads rounded up to whole waves (a pair's two elements are neighbours
// of one wave; vdim is even wherever values are turned).
template <typename T>
__global__ void qkv_values_kernel(QkvRows a, int n, T* __restrict__ v_cache) {
  const int t0 = blockIdx.x * 16, kh = blockIdx.y, d = min((int)threadIdx.x, a.vdim - 1);
  const bool mine = (int)threadIdx.x < a.vdim;
  const int col0 = (a.heads + a.kv) * a.dim + kh * a.vdim + d;
  const float b = a.v_bias != nullptr ? a.v_bias[kh * a.vdim + d] : 0.f;
  float y[16];
#pragma unroll
  for (int i = 0; i < 16; ++i) y[i] = t0 + i < n ? a.rows[(size_t)(t0 + i) * a.stride + col0] + b : 0.f;
  if (a.v_inv_freq != nullptr) {
    const int half = a.vdim / 2;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const float other = __shfl_xor(y[i], 1, TP_WAVE);   // (every lane takes part)
      const int t = min(t0 + i, n - 1);
      float c, sn;
      if (a.v_table != nullptr) {
        const float2 cs = a.v_table[(size_t)t * half + d / 2];
        c = cs.x;
        sn = cs.y;
      } else {
        rope_cos_sin(a.positions[t], a.v_inv_freq[d / 2], 1.0f, c, sn);
      }
      y[i] = (d & 1) ? other * sn + y[i] * c : y[i] * c - other * sn;
    }
  }
  if (!mine) return;
#pragma unroll
  for (int g = 0; g < 2; ++g) {
    const int tg = t0 + 8 * g;
    if (tg >= n) break;
    const int s0 = a.slots[tg];
    bool run = tg + 8 <= n && (s0 & 7) == 0 && a.page_size % 8 == 0;
    if (run) {
#pragma unroll
      for (int i = 1; i < 8; ++i) run = run && a.slots[tg + i] == s0 + i;
    }
    if (run) {
      T* o = v_cache + (((size_t)(s0 / a.page_size) * a.kv + kh) * a.vdim + d) * a.page_size + s0 % a.page_size;
      from_float4(o, y[8 * g], y[8 * g + 1], y[8 * g + 2], y[8 * g + 3]);
      from_float4(o + 4, y[8 * g + 4], y[8 * g + 5], y[8 * g + 6], y[8 * g + 7]);
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        if (tg + i >= n) break;
        const int sl = a.slots[tg + i];
        from_float(v_cache + (((size_t)(sl / a.page_size) * a.kv + kh) * a.vdim + d) * a.page_size + sl % a.page_size, y[8 * g + i]);
      }
    }
  }
}

static inline bool all_aligned16(const void* a, const void* b, const void* c, const void* d, const void* e, const void* f) {
  return (((uintptr_t)a | (uintptr_t)b | (uintptr_t)c | (uintptr_t)d | (uintptr_t)e | (uintptr_t)f) & 15) == 0;
}

// rows float32 [n, stride] with q | k | v from column 0 on (`width`: how many columns of a row lie behind that one).  q_norm
// and k_norm come together; per_head: they have dim elements and norm every head by itself.  out_dim >= dim: q_out
// [n, heads, out_dim], keys [page, kv, page_size, out_dim] with zeros behind a head's own elements; values transposed
// [page, kv, vdim, page_size].  dt: the type of q_out and of both caches.
extern "C" int tp_qkv_rows(const float* rows, size_t stride, size_t width, const float* q_bias, const float* k_bias, const float* v_bias,
                           const float* q_norm, const float* k_norm, float eps, const int* positions, const int* slots,
                           const double* inv_freq, const float* table, int rotary_dim, float factor, const double* v_inv_freq,
                           const float* v_table, int n, int heads, int kv, int dim, int vdim, int out_dim, void* q_out,
                           void* k_cache, void* v_cache, int dt, int page_size, int per_head, hipStream_t s) {
  TP_REQUIRE(n >= 0 && heads > 0 && kv > 0 && dim > 0 && vdim > 0 && page_size > 0, "qkv_rows: bad sizes");
  TP_REQUIRE(dim % 2 == 0 && vdim % 2 == 0 && out_dim >= dim && out_dim % 2 == 0 && stride % 2 == 0, "qkv_rows: head sizes and row length must be even");
  TP_REQUIRE(vdim <= 1024 && kv <= 65535, "qkv_rows: value size %d or %d key heads too large", vdim, kv);
  TP_REQUIRE(rotary_dim >= 0 && rotary_dim % 2 == 0 && rotary_dim <= dim && (rotary_dim == 0 || inv_freq != nullptr), "qkv_rows: bad rotation");
  TP_REQUIRE(width <= stride && width >= (size_t)(heads + kv) * dim + (size_t)kv * vdim, "qkv_rows: rows too short");
  TP_REQUIRE((q_norm == nullptr) == (k_norm == nullptr), "qkv_rows: the norms of q and k come together");
  TP_REQUIRE(dt == TP_F32 || dt == TP_BF16, "qkv_rows: unknown dtype %d", dt);
  if (n == 0) return 0;
  QkvRows a;
  a.rows = rows; a.stride = stride;
  a.q_bias = q_bias; a.k_bias = k_bias; a.v_bias = v_bias;
  a.q_norm = q_norm; a.k_norm = k_norm; a.eps = eps;
  a.positions = positions; a.slots = slots;
  a.inv_freq = inv_freq; a.table = (const float2*)table; a.rotary_dim = rotary_dim; a.factor = factor;
  a.v_inv_freq = v_inv_freq; a.v_table = (const float2*)v_table;
  a.heads = heads; a.kv = kv; a.dim = dim; a.vdim = vdim; a.out_dim = out_dim; a.page_size = page_size;
  const bool four = dim % 4 == 0 && vdim % 4 == 0 && out_dim % 4 == 0 && stride % 4 == 0 && all_aligned16(rows, q_bias, k_bias, v_bias, q_norm, k_norm);
  const int V = four ? 4 : 2;
  // a few rows: many blocks a token, so that a decode step fills more than a handful of CUs; long steps: one block per
  // token and section, values sixteen tokens at a time
  const bool lng = n >= 256;
  if (per_head) {
    const int per_token = heads + kv + (lng ? 0 : kv);
    const long units = (long)n * per_token;
    int group = 1;
    while (group < TP_WAVE && group * V < out_dim) group *= 2;
    TP_REQUIRE(units * group / 256 + 1 < 0x7fffffffL, "qkv_rows: too many rows");
    const dim3 grid((unsigned)((units * group + 255) / 256));
#define QKV_HEADS(T)                                                                                                                 \
  do {                                                                                                                               \
    if (four)                                                                                                                        \
      hipLaunchKernelGGL((qkv_heads_kernel<T, 4>), grid, dim3(256), 0, s, a, units, per_token, group, (T*)q_out, (T*)k_cache, (T*)v_cache); \
    else                                                                                                                             \
      hipLaunchKernelGGL((qkv_heads_kernel<T, 2>), grid, dim3(256), 0, s, a, units, per_token, group, (T*)q_out, (T*)k_cache, (T*)v_cache); \
    if (lng)                                                                                                                         \
      hipLaunchKernelGGL(qkv_values_kernel<T>, dim3((n + 15) / 16, kv), dim3((vdim + 63) / 64 * 64), 0, s, a, n, (T*)v_cache);       \
  } while (0)
    if (dt == TP_F32)
      QKV_HEADS(float);
    else
      QKV_HEADS(bf16_t);
#undef QKV_HEADS
    TP_CHECK_LAUNCH("qkv_rows");
    return 0;
  }
  const int widest = heads * dim > kv * vdim ? heads * dim : kv * vdim;
  a.per_slice = lng ? (widest > kv * dim ? widest : kv * dim) / V : 256;
  auto slices = [&](int width) { return (width / V + a.per_slice - 1) / a.per_slice; };
  a.q_slices = slices(heads * dim);
  a.k_slices = slices(kv * dim);
  a.v_slices = lng ? 0 : slices(kv * vdim);
  const dim3 grid(n, a.q_slices + a.k_slices + a.v_slices);
  TP_REQUIRE(grid.y <= 65535, "qkv_rows: too many heads");
#define QKV(T)                                                                                                        \
  do {                                                                                                                \
    if (four)                                                                                                         \
      hipLaunchKernelGGL((qkv_rows_kernel<T, 4>), grid, dim3(256), 0, s, a, (T*)q_out, (T*)k_cache, (T*)v_cache);     \
    else                                                                                                              \
      hipLaunchKernelGGL((qkv_rows_kernel<T, 2>), grid, dim3(256), 0, s, a, (T*)q_out, (T*)k_cache, (T*)v_cache);     \
    if (lng)                                                                                                          \
      hipLaunchKernelGGL(qkv_values_kernel<T>, dim3((n + 15) / 16, kv), dim3((vdim + 63) / 64 * 64), 0, s, a, n, (T*)v_cache); \
  } while (0)
  if (dt == TP_F32)
    QKV(float);
  else
    QKV(bf16_t);
#undef QKV
  TP_CHECK_LAUNCH("qkv_rows");
  return 0;
}

// ---- queries in a latent's space, one latent and one rotated key part a token --------------------
// rows float32 [n, stride]: at q_col0 the queries, q_head elements a head, whose rot rotated elements start at q_rot; the
// latent elements follow them, or (latent_follows 0) somebody else writes the latent part of q_out.  At d_col0 the
// latent before its norm [latent] and the shared rotated key part [rot].  The latent becomes c = x / sqrt(mean(x^2) +
// eps) * w.  Written: q_out [n, heads, out_dim] and keys [page, 1, page_size, out_dim] as [rotated | latent | zeros],
// values [page, 1, value_dim, page_size] as [latent | zeros], transposed.
// grid: (tokens, 1 + q_slices); block 0 of a token writes key and value, the others a slice of its queries.
template <typename T, int V>
__global__ __launch_bounds__(256) void latent_rows_write_kernel(const float* __restrict__ rows, size_t stride, int q_col0, int d_col0,
                                                                const float* __restrict__ w, float eps, const int* __restrict__ positions,
                                                                const int* __restrict__ slots, const double* __restrict__ inv_freq,
                                                                const float2* __restrict__ table, float factor, int heads, int rot, int latent,
                                                                int out_dim, int value_dim, T* __restrict__ q_out, T* __restrict__ k_cache,
                                                                T* __restrict__ v_cache, int page_size, int per_slice, int q_head, int q_rot,
                                                                int latent_follows) {
  __shared__ float scratch[32];
  const int t = blockIdx.x, pos = positions[t];
  const float* row = rows + (size_t)t * stride;
  if (blockIdx.y == 0) {
    const float* x = row + d_col0;
    float ss = 0.f;
    for (int i = threadIdx.x; i < latent; i += blockDim.x) ss = fmaf(x[i], x[i], ss);
    ss = block_sum(ss, scratch);
    const float rstd = 1.0f / sqrtf(ss / (float)latent + eps);
    const int slot = slots[t];
    const size_t page = (size_t)(slot / page_size), off = (size_t)(slot % page_size);
    T* k = k_cache + (page * page_size + off) * out_dim;
    T* v = v_cache + page * value_dim * page_size + off;
    for (int p = threadIdx.x; p < rot / 2; p += blockDim.x) {
      Elems<2> r;
      r.x[0] = x[latent + 2 * p];
      r.x[1] = x[latent + 2 * p + 1];
      turn_pairs<2>(r, 2 * p, rot / 2, t, pos, inv_freq, table, factor, 1.0f);
      store_elems<2>(k + 2 * p, r);
    }
    const int most = max(out_dim - rot, value_dim);
    for (int i = threadIdx.x; i < most; i += blockDim.x) {
      const float c = i < latent ? x[i] * rstd * w[i] : 0.f;
      if (i < out_dim - rot) from_float(k + rot + i, c);
      if (i < value_dim) from_float(v + (size_t)i * page_size, c);
    }
    return;
  }
  // a head's elements that this kernel writes: all of them, or all but the latent part
  const int key = rot + latent, skip = latent_follows ? 0 : latent, span = out_dim - skip;
  const int end = min(heads * span / V, (int)blockIdx.y * per_slice);
  for (int g = ((int)blockIdx.y - 1) * per_slice + threadIdx.x; g < end; g += blockDim.x) {
    const int h = g * V / span, j = g * V % span, i = j < rot ? j : j + skip;
    Elems<V> r;
    if (i < key) {
      r = load_elems<V>(row + q_col0 + (size_t)h * q_head + q_rot + i);
      turn_pairs<V>(r, i, rot / 2, t, pos, inv_freq, table, factor, 1.0f);
    } else {
#pragma unroll
      for (int e = 0; e < V; ++e) r.x[e] = 0.f;
    }
    store_elems<V>(q_out + ((size_t)t * heads + h) * out_dim + i, r);
  }
}

extern "C" int tp_latent_rows_write(const float* rows, size_t stride, int q_col0, int d_col0, const float* w, float eps,
                                    const int* positions, const int* slots, const double* inv_freq, const float* table, float factor,
                                    int n, int heads, int rot, int latent, int out_dim, int value_dim, void* q_out, void* k_cache,
                                    void* v_cache, int dt, int page_size, int q_head, int q_rot, int latent_follows, hipStream_t s) {
  TP_REQUIRE(n >= 0 && heads > 0 && rot >= 0 && latent > 0 && q_col0 >= 0 && d_col0 >= 0 && page_size > 0, "latent_rows_write: bad sizes");
  const int key = rot + latent;
  TP_REQUIRE(rot % 2 == 0 && key % 2 == 0 && out_dim % 2 == 0 && out_dim >= key && value_dim >= latent, "latent_rows_write: head sizes must be even");
  TP_REQUIRE(stride % 2 == 0 && q_col0 % 2 == 0 && q_head % 2 == 0 && q_rot % 2 == 0 && q_rot >= 0 &&
                 q_head >= q_rot + rot + (latent_follows ? latent : 0) && stride >= (size_t)q_col0 + (size_t)heads * q_head &&
                 stride >= (size_t)d_col0 + key,
             "latent_rows_write: rows too short or odd");
  TP_REQUIRE(rot == 0 || inv_freq != nullptr, "latent_rows_write: no frequency table");
  TP_REQUIRE(dt == TP_F32 || dt == TP_BF16, "latent_rows_write: unknown dtype %d", dt);
  if (n == 0) return 0;
  const bool four = key % 4 == 0 && rot % 4 == 0 && (latent_follows || latent % 4 == 0) && q_head % 4 == 0 && q_rot % 4 == 0 && out_dim % 4 == 0 && stride % 4 == 0 && q_col0 % 4 == 0 && ((uintptr_t)rows & 15) == 0;
  const int V = four ? 4 : 2;
  const int per_slice = n >= 256 ? 1024 : 256;
  const int span = latent_follows ? out_dim : out_dim - latent;
  const dim3 grid(n, 1 + (heads * span / V + per_slice - 1) / per_slice);
  TP_REQUIRE(grid.y <= 65535, "latent_rows_write: too many heads");
#define LAT(T, VV)                                                                                                            \
  hipLaunchKernelGGL((latent_rows_write_kernel<T, VV>), grid, dim3(256), 0, s, rows, stride, q_col0, d_col0, w, eps, positions, slots, \
                     inv_freq, (const float2*)table, factor, heads, rot, latent, out_dim, value_dim, (T*)q_out, (T*)k_cache,  \
                     (T*)v_cache, page_size, per_slice, q_head, q_rot, latent_follows)
  if (dt == TP_F32) {
    if (four) LAT(float, 4); else LAT(float, 2);
  } else {
    if (four) LAT(bf16_t, 4); else LAT(bf16_t, 2);
  }
#undef LAT
  TP_CHECK_LAUNCH("latent_rows_write");
  return 0;
}

// ---- outputs turned back, times a gate ------------------------------------------------------------
// out[t, c] = (a[t] with every head's pairs (2 m, 2 m + 1) turned by -positions[t] * inv_freq[m])[c] *
// sigmoid(gate[t, gate_col0 + c]) (gate nullptr: no gate).  a and out [n, heads * dim].
template <typename T, int V>
__global__ void turn_gate_kernel(const T* __restrict__ a, const int* __restrict__ positions, const double* __restrict__ inv_freq,
                                 const float2* __restrict__ table, const float* __restrict__ gate, size_t gate_stride, int gate_col0,
                                 T* __restrict__ out, int width, int dim, size_t groups) {
  const size_t g = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (g >= groups) return;
  const int per = width / V;
  const int t = (int)(g / per), c = (int)(g % per) * V;
  Elems<V> r;
  if constexpr (V == 4 && sizeof(T) == 2) {
    const uint2 raw = *(const uint2*)(a + (size_t)t * width + c);
    r.x[0] = bf16_to_float(bf16_t{(uint16_t)(raw.x & 0xffff)});
    r.x[1] = bf16_to_float(bf16_t{(uint16_t)(raw.x >> 16)});
    r.x[2] = bf16_to_float(bf16_t{(uint16_t)(raw.y & 0xffff)});
    r.x[3] = bf16_to_float(bf16_t{(uint16_t)(raw.y >> 16)});
  } else {
#pragma unroll
    for (int e = 0; e < V; ++e) r.x[e] = to_float(a[(size_t)t * width + c + e]);
  }
  turn_pairs<V>(r, c % dim, dim / 2, t, positions[t], inv_freq, table, 1.0f, -1.0f);
  if (gate != nullptr) {
    const Elems<V> z = load_elems<V>(gate + (size_t)t * gate_stride + gate_col0 + c);
#pragma unroll
    for (int e = 0; e < V; ++e) r.x[e] *= 1.0f / (1.0f + expf(-z.x[e]));
  }
  store_elems<V>(out + (size_t)t * width + c, r);
}

extern "C" int tp_turn_gate(const void* a, int dt, const int* positions, const double* inv_freq, const float* table, const float* gate,
                            size_t gate_stride, int gate_col0, void* out, int n, int heads, int dim, hipStream_t s) {
  TP_REQUIRE(n >= 0 && heads > 0 && dim > 0 && dim % 2 == 0 && inv_freq != nullptr, "turn_gate: bad sizes");
  TP_REQUIRE(gate == nullptr || (gate_col0 >= 0 && gate_stride >= (size_t)gate_col0 + (size_t)heads * dim), "turn_gate: gate rows too short");
  TP_REQUIRE(dt == TP_F32 || dt == TP_BF16, "turn_gate: unknown dtype %d", dt);
  if (n == 0) return 0;
  const int width = heads * dim;
  const bool four = dim % 4 == 0 && (gate == nullptr || (gate_stride % 4 == 0 && gate_col0 % 4 == 0)) && all_aligned16(a, out, gate, a, a, a);
  const size_t groups = (size_t)n * (width / (four ? 4 : 2));
  TP_REQUIRE((groups + 255) / 256 < ((size_t)1 << 31), "turn_gate: too many tokens");
  const dim3 grid((unsigned)((groups + 255) / 256));
#define TG(T, VV)                                                                                                               \
  hipLaunchKernelGGL((turn_gate_kernel<T, VV>), grid, dim3(256), 0, s, (const T*)a, positions, inv_freq, (const float2*)table, gate, \
                     gate_stride, gate_col0, (T*)out, width, dim, groups)
  if (dt == TP_F32) {
    if (four) TG(float, 4); else TG(float, 2);
  } else {
    if (four) TG(bf16_t, 4); else TG(bf16_t, 2);
  }
#undef TG
  TP_CHECK_LAUNCH("turn_gate");
  return 0;
}
