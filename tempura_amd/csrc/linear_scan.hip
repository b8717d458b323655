// A linear recurrence with a decay per key channel over a batch of requests that each bring a run of tokens, and the
// mixes of a token's row with the row before it that feed one of its mixers.  Per head, with a state S [dim, vdim]:
//   S <- diag(w) S + k v^T
// read either behind the update, o = S^T q, or in front of it with a bonus u, o = (S + diag(u) k v^T)^T q.
// All arithmetic is float32; the state [heads, vdim, dim] (a head's matrix column by column) lives in float32 rows of a
// per-request state tensor (row = request slot).
//
// A request r of the batch owns tokens cu_seqlens[r] .. cu_seqlens[r + 1] - 1 and the state row state_slots[r]; everything
// is read from device memory, so the same launches serve prompt portions, single decoded tokens and captured steps.
// How a run is cut changes rounding only.
#include <math.h>

#include "common.h"
#include "column_sum.h"

// ---- mixes of a row and the row before it ------------------------------------------------------
// out[s][t][c] = x[t][c] + (x'[c] - x[t][c]) * mu[s][c]; x' is the row before t in its request: row t - 1 of the step, or for a
// run's first token what the request's state row holds from state_off on.
template <typename TO, int V>
__global__ void token_shift_kernel(const float* __restrict__ x, const float* __restrict__ mu, float* __restrict__ state, size_t state_stride,
                                   size_t state_off, const int* __restrict__ cu_seqlens, const int* __restrict__ token_req,
                                   const int* __restrict__ state_slots, TO* __restrict__ out, size_t out_stride_mix, int width, int mixes,
                                   int channel_blocks, int single, int blocked) {
  const int t = blockIdx.x / channel_blocks;
  const int c = ((blockIdx.x % channel_blocks) * blockDim.x + threadIdx.x) * V;
  if (c >= width) return;
  const int r = token_req[t];
  float* st = state + (size_t)state_slots[r] * state_stride + state_off + c;
  const float* xr = x + (size_t)t * width + c;
  const float* before = t > cu_seqlens[r] ? xr - width : st;
  float cur[V], gap[V];
  if constexpr (V == 4) {
    const float4 a = *(const float4*)xr;
    cur[0] = a.x; cur[1] = a.y; cur[2] = a.z; cur[3] = a.w;
  } else {
    cur[0] = xr[0];
  }
#pragma unroll
  for (int e = 0; e < V; ++e) gap[e] = before[e] - cur[e];   // (a state row's place need not be aligned)
  // every run one token long: the thread that has read a channel of the state is the only one that does
  if (single) {
#pragma unroll
    for (int e = 0; e < V; ++e) st[e] = cur[e];
  }
  for (int s = 0; s < mixes; ++s) {
    const float* m = mu + (size_t)s * width + c;
    TO* o = out + (size_t)s * out_stride_mix + (blocked ? ((size_t)(c >> 3) * (gridDim.x / channel_blocks) + t) * 8 + (c & 7) : (size_t)t * width + c);
    if constexpr (V == 4) {
      const float4 mv = *(const float4*)m;
      from_float4(o, fmaf(gap[0], mv.x, cur[0]), fmaf(gap[1], mv.y, cur[1]), fmaf(gap[2], mv.z, cur[2]), fmaf(gap[3], mv.w, cur[3]));
    } else {
      from_float(o, fmaf(gap[0], m[0], cur[0]));
    }
  }
}

__global__ void last_row_kernel(const float* __restrict__ x, float* __restrict__ state, size_t state_stride, size_t state_off,
                                const int* __restrict__ cu_seqlens, const int* __restrict__ state_slots, int width) {
  const int r = blockIdx.x;
  const int c = blockIdx.y * blockDim.x + threadIdx.x;
  const int end = cu_seqlens[r + 1];
  if (c >= width || end <= cu_seqlens[r]) return;
  state[(size_t)state_slots[r] * state_stride + state_off + c] = x[(size_t)(end - 1) * width + c];
}

// single: every run of the step is one token long; blocked: every mix leaves as [width / 8, n, 8] (see decode_groups.hip)
extern "C" int tp_token_shift(const float* x, const float* mu, float* state, size_t state_stride, size_t state_off, const int* cu_seqlens,
                              const int* token_req, const int* state_slots, void* out, int out_dt, int n, int n_req, int width, int mixes,
                              int single, int blocked, hipStream_t s) {
  TP_REQUIRE(n >= 0 && n_req >= 0 && width > 0 && mixes > 0, "token_shift: bad sizes");
  TP_REQUIRE(state_stride >= state_off + (size_t)width, "token_shift: state rows too short");
  TP_REQUIRE(out_dt == TP_F32 || out_dt == TP_BF16, "token_shift: unknown dtype %d", out_dt);
  TP_REQUIRE(!blocked || width % 8 == 0, "token_shift: k-blocked rows need a width that is a multiple of eight");
  TP_REQUIRE(!single || n <= n_req, "token_shift: %d tokens are not %d runs of one", n, n_req);
  if (n == 0 || n_req == 0) return 0;
  const bool four = width % 4 == 0 && (((uintptr_t)x | (uintptr_t)mu | (uintptr_t)out) & 15) == 0;
  const int units = four ? width / 4 : width;
  const int threads = units >= 256 ? 256 : 64;
  const int cb = (units + threads - 1) / threads;
  TP_REQUIRE((long)n * cb < 0x7fffffffL && (width + 255) / 256 <= 65535, "token_shift: too many channels or tokens");
  const dim3 grid((unsigned)((long)n * cb));
#define SHIFT(T, V)                                                                                                                        \
  hipLaunchKernelGGL((token_shift_kernel<T, V>), grid, dim3(threads), 0, s, x, mu, state, state_stride, state_off, cu_seqlens, token_req, \
                     state_slots, (T*)out, (size_t)n * width, width, mixes, cb, single, blocked)
  if (out_dt == TP_F32) {
    if (four) SHIFT(float, 4);
    else SHIFT(float, 1);
  } else {
    if (four) SHIFT(bf16_t, 4);
    else SHIFT(bf16_t, 1);
  }
#undef SHIFT
  if (!single)
    hipLaunchKernelGGL(last_row_kernel, dim3(n_req, (width + 255) / 256), dim3(256), 0, s, x, state, state_stride, state_off, cu_seqlens,
                       state_slots, width);
  TP_CHECK_LAUNCH("token_shift");
  return 0;
}

// ---- the recurrence ---------------------------------------------------------------------------
// A block owns one request (or one piece of its run), one head and CB = WAVES * TP * 64 / KS value columns; a thread holds PER
// consecutive key channels of TP neighbouring columns in registers, and the KS neighbouring lanes that share those columns
// split the key channels among them (their partial read-outs meet by row permutes).  Several columns a thread share
// what a token's q, k and w cost in LDS reads.  Tokens are taken TC at a time through LDS (rows padded to KS * PER channels
// with q = k = 0 and w = 1, so the run itself needs no bounds); the next chunk's values travel from memory into registers
// while this chunk runs.
//
// With the bonus the read-out of column j is sum_i q_i S_ij + (sum_i q_i u_i k_i) v_j: the second sum is the same for all
// columns, so a lane adds its share of it times v_j to its partial read-out.
//
// Long runs (keys of at most 128) are cut into pieces of `piece` tokens that run side by side.  Three launches:
//   ends         every piece's end state from a zero state and, per key channel, the product of its decays, to scratch.  The end
//                state is sum_j (k_j times the decays of the piece's tokens behind j) v_j^T: a float32 product on the matrix
//                cores, the tokens walked backwards so that every factor is a product of decays (nothing is divided);
//   carry        per state entry, piece by piece: the state a piece starts from is decay(piece before) * (the state the piece
//                before started from) + (its end state from zero); what the last piece leaves is the request's state;
//   SCAN_PIECES  every piece from the state it starts from, writing o (a run of one piece runs as in SCAN_DIRECT and is left
//                out of the other two).
// Short runs take SCAN_DIRECT: one launch, from the request's state to its new state.
enum { SCAN_DIRECT = 0, SCAN_PIECES = 1 };

struct LinearScan {
  const float *q, *k, *v;      // first column of each, rows of their own strides
  int q_stride, k_stride, v_stride;
  const float* decay;          // [n, heads * dim]
  const float* bonus;          // [heads * dim], or nullptr: read behind the update
  float q_scale;
  float* state;
  size_t state_stride, state_off;
  const int* cu_seqlens;
  const int* state_slots;
  float* y;                    // [n, heads * vdim]
  int heads, dim, vdim;
  int mode, piece;
  float* piece_state;          // [pieces, heads, vdim, dim]; a request's pieces start at cu_seqlens[r] / piece + r
  float* piece_decay;          // [pieces, heads, dim]
};

template <int PER, int KS, int TP, int WAVES, bool BONUS>
__global__ __launch_bounds__(WAVES * 64) void linear_scan_kernel(LinearScan a) {
  constexpr int THREADS = WAVES * 64;
  constexpr int DP = PER * KS, CW = TP_WAVE / KS * TP, CB = WAVES * CW;
  constexpr int TC = DP <= 128 ? 16 : 2048 / DP;
  constexpr int NI = (TC * DP + THREADS - 1) / THREADS, NV = (TC * CB + THREADS - 1) / THREADS;
  __shared__ __attribute__((aligned(16))) float qs[TC * DP];
  __shared__ __attribute__((aligned(16))) float ks_[TC * DP];
  __shared__ __attribute__((aligned(16))) float ws[TC * DP];
  __shared__ __attribute__((aligned(16))) float vs[TC * CB];
  const int r = blockIdx.x, h = blockIdx.y;
  const int slices = (a.vdim + CB - 1) / CB;
  const int slice = blockIdx.z % slices, pc = blockIdx.z / slices;
  const int run0 = a.cu_seqlens[r], run_len = a.cu_seqlens[r + 1] - run0;
  if (run_len <= 0) return;
  int mode = a.mode;
  if (mode != SCAN_DIRECT) {
    if ((long)pc * a.piece >= run_len) return;
    if (run_len <= a.piece) mode = SCAN_DIRECT;
  }
  const int start = run0 + (mode == SCAN_DIRECT ? 0 : pc * a.piece);
  const int len = mode == SCAN_DIRECT ? run_len : min(a.piece, run_len - pc * a.piece);
  const int tid = threadIdx.x, wave = tid / TP_WAVE, lane = tid % TP_WAVE;
  const int ks = lane % KS, jl = wave * CW + lane / KS * TP;
  const int j0 = slice * CB + jl;

  float* S_mem = a.state + (size_t)a.state_slots[r] * a.state_stride + a.state_off + (size_t)h * a.vdim * a.dim;
  const size_t place = a.piece > 0 ? (size_t)(run0 / a.piece + r + pc) * a.heads + h : 0;
  if (mode != SCAN_DIRECT) S_mem = a.piece_state + place * a.vdim * a.dim;
  const bool vec = a.dim % 4 == 0 && ((uintptr_t)S_mem % 16) == 0;
  float S[TP][PER];
#pragma unroll
  for (int j = 0; j < TP; ++j) {
    const bool have = j0 + j < a.vdim;
    const float* col = S_mem + (size_t)(have ? j0 + j : 0) * a.dim;
#pragma unroll
    for (int e4 = 0; e4 < PER / 4; ++e4) {
      const int i = ks * PER + e4 * 4;
      if (vec && have && i < a.dim) {
        const float4 f = *(const float4*)(col + i);
        S[j][e4 * 4 + 0] = f.x; S[j][e4 * 4 + 1] = f.y; S[j][e4 * 4 + 2] = f.z; S[j][e4 * 4 + 3] = f.w;
      } else {
#pragma unroll
        for (int c = 0; c < 4; ++c) S[j][e4 * 4 + c] = (have && i + c < a.dim) ? col[i + c] : 0.f;
      }
    }
  }
  float u[PER];
#pragma unroll
  for (int e = 0; e < PER; ++e) {
    const int i = ks * PER + e;
    u[e] = (BONUS && i < a.dim) ? a.bonus[(size_t)h * a.dim + i] : 0.f;
  }
  const size_t hd = (size_t)a.heads * a.dim, out_width = (size_t)a.heads * a.vdim;
  const float *q0 = a.q + (size_t)h * a.dim, *k0 = a.k + (size_t)h * a.dim, *v0 = a.v + (size_t)h * a.vdim, *w0 = a.decay + (size_t)h * a.dim;

  float fq[NI], fk[NI], fw[NI], fv[NV];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int it = 0; it < NI; ++it) {
      const int idx = it * THREADS + tid;
      const int t = idx / DP, i = idx % DP;
      const bool in = idx < TC * DP && t0 + t < len && i < a.dim;
      const size_t row = (size_t)(start + t0 + t);
      fq[it] = in ? q0[row * a.q_stride + i] * a.q_scale : 0.f;
      fk[it] = in ? k0[row * a.k_stride + i] : 0.f;
      fw[it] = in ? w0[row * hd + i] : 1.f;
    }
#pragma unroll
    for (int it = 0; it < NV; ++it) {
      const int idx = it * THREADS + tid;
      const int t = idx / CB, col = slice * CB + idx % CB;
      fv[it] = (idx < TC * CB && t0 + t < len && col < a.vdim) ? v0[(size_t)(start + t0 + t) * a.v_stride + col] : 0.f;
    }
  };
  struct Tok {
    float4 q[PER / 4], k[PER / 4], w[PER / 4];
    float v[TP];
  };
  auto take = [&](Tok& x, int t) {
    const int off = t * DP + ks * PER;
#pragma unroll
    for (int e4 = 0; e4 < PER / 4; ++e4) {
      x.q[e4] = ((const float4*)(qs + off))[e4];
      x.k[e4] = ((const float4*)(ks_ + off))[e4];
      x.w[e4] = ((const float4*)(ws + off))[e4];
    }
    const float* vr = vs + t * CB + jl;
    if constexpr (TP == 4) {
      const float4 f = *(const float4*)vr;
      x.v[0] = f.x; x.v[1] = f.y; x.v[2] = f.z; x.v[3] = f.w;
    } else if constexpr (TP == 2) {
      const float2 f = *(const float2*)vr;
      x.v[0] = f.x; x.v[1] = f.y;
    } else {
      x.v[0] = vr[0];
    }
  };
  auto step = [&](const Tok& x, int t_run) {
    float part[TP], own = 0.f;
#pragma unroll
    for (int j = 0; j < TP; ++j) part[j] = 0.f;
#pragma unroll
    for (int e4 = 0; e4 < PER / 4; ++e4) {
      const float qa[4] = {x.q[e4].x, x.q[e4].y, x.q[e4].z, x.q[e4].w}, ka[4] = {x.k[e4].x, x.k[e4].y, x.k[e4].z, x.k[e4].w},
                  wa[4] = {x.w[e4].x, x.w[e4].y, x.w[e4].z, x.w[e4].w};
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        const int e = e4 * 4 + c;
        if (BONUS) own = fmaf(u[e] * ka[c], qa[c], own);
#pragma unroll
        for (int j = 0; j < TP; ++j) {
          if (BONUS) part[j] = fmaf(S[j][e], qa[c], part[j]);   // (the state as the token before left it)
          S[j][e] = fmaf(wa[c], S[j][e], ka[c] * x.v[j]);
          if (!BONUS) part[j] = fmaf(S[j][e], qa[c], part[j]);
        }
      }
    }
#pragma unroll
    for (int j = 0; j < TP; ++j) {
      if (BONUS) part[j] = fmaf(own, x.v[j], part[j]);
      part[j] = column_sum<KS>(part[j]);
    }
    // a column's sum is in all of its lanes: lane j of them stores column j (TP <= KS wherever TP > 1)
    float out = part[0];
#pragma unroll
    for (int j = 1; j < TP; ++j) out = ks == j ? part[j] : out;
    if (ks < TP && j0 + ks < a.vdim) a.y[(size_t)(start + t_run) * out_width + (size_t)h * a.vdim + j0 + ks] = out;
  };
  fetch(0);
  for (int t0 = 0; t0 < len; t0 += TC) {
    const int tc = min(TC, len - t0);
    __syncthreads();   // the chunk before has been consumed
#pragma unroll
    for (int it = 0; it < NI; ++it) {
      const int idx = it * THREADS + tid;
      if (idx < TC * DP) {
        qs[idx] = fq[it];
        ks_[idx] = fk[it];
        ws[idx] = fw[it];
      }
    }
#pragma unroll
    for (int it = 0; it < NV; ++it) {
      const int idx = it * THREADS + tid;
      if (idx < TC * CB) vs[idx] = fv[it];
    }
    __syncthreads();
    if (t0 + TC < len) fetch(t0 + TC);   // on its way while this chunk runs
    // two tokens a turn, each token's LDS reads issued before the token ahead of it is worked on
    Tok A, B;
    take(A, 0);
    for (int t = 0; t < tc; t += 2) {
      if (t + 1 < tc) take(B, t + 1);
      step(A, t0 + t);
      if (t + 1 < tc) {
        if (t + 2 < tc) take(A, t + 2);
        step(B, t0 + t + 1);
      }
    }
  }
  if (mode == SCAN_PIECES) return;   // (the carry has left the state after the run)
#pragma unroll
  for (int j = 0; j < TP; ++j) {
    const bool have = j0 + j < a.vdim;
    float* col = S_mem + (size_t)(have ? j0 + j : 0) * a.dim;
#pragma unroll
    for (int e4 = 0; e4 < PER / 4; ++e4) {
      const int i = ks * PER + e4 * 4;
      if (vec && have && i < a.dim) {
        *(float4*)(col + i) = make_float4(S[j][e4 * 4 + 0], S[j][e4 * 4 + 1], S[j][e4 * 4 + 2], S[j][e4 * 4 + 3]);
      } else {
#pragma unroll
        for (int c = 0; c < 4; ++c)
          if (have && i + c < a.dim) col[i + c] = S[j][e4 * 4 + c];
      }
    }
  }
}

// The end state of every piece from zero, and the products of its decays.  DT: 16-row tiles of key channels (16 DT >= dim).
// grid: (requests, heads, pieces times slices of 64 value columns); a wave owns 16 columns.  Chunks of sixteen tokens, the
// last first: 256 / (16 DT) groups of threads each take a run of the chunk's tokens, a thread one key channel; what decays a
// group's keys beyond its own tokens is the product of the later groups' decays and of the chunks behind.
// Operands of the 16x16x4 product: lane l holds row (column) l % 16 at k = l / 16; result rows (l / 16) * 4 + r of column l % 16.
typedef float f32x4_t __attribute__((ext_vector_type(4)));

template <int DT>
__global__ __launch_bounds__(256) void linear_ends_kernel(LinearScan a) {
  constexpr int DP = DT * 16, G = 256 / DP, TG = 16 / G;   // groups, tokens of a group
  __shared__ float ks[16][DP + 1];
  __shared__ float vs[16][64 + 1];
  __shared__ float gp[G][DP];
  const int r = blockIdx.x, h = blockIdx.y;
  const int slices = (a.vdim + 63) / 64;
  const int slice = blockIdx.z % slices, pc = blockIdx.z / slices;
  const int run0 = a.cu_seqlens[r], run_len = a.cu_seqlens[r + 1] - run0;
  if (run_len <= a.piece || (long)pc * a.piece >= run_len) return;
  const int start = run0 + pc * a.piece, len = min(a.piece, run_len - pc * a.piece);
  const size_t place = (size_t)(run0 / a.piece + r + pc) * a.heads + h;
  const int tid = threadIdx.x, wave = tid / TP_WAVE, lane = tid % TP_WAVE;
  const int d = tid % DP, g = tid / DP;
  const bool d_ok = d < a.dim;
  const size_t hd = (size_t)a.heads * a.dim;
  const float *k0 = a.k + (size_t)h * a.dim + (d_ok ? d : 0), *w0 = a.decay + (size_t)h * a.dim + (d_ok ? d : 0);
  const float* v0 = a.v + (size_t)h * a.vdim;
  const int col = slice * 64 + tid % 64;   // (of the value that this thread fetches)

  float fk[TG], fw[TG], fv[4];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int i = 0; i < TG; ++i) {
      const int t = t0 + g * TG + i;
      const bool in = d_ok && t < len;
      const size_t row = (size_t)(start + (in ? t : 0));
      fk[i] = in ? k0[row * a.k_stride] : 0.f;
      fw[i] = in ? w0[row * hd] : 1.f;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = t0 + i * 4 + tid / 64;
      const bool in = t < len && col < a.vdim;
      fv[i] = in ? v0[(size_t)(start + t) * a.v_stride + col] : 0.f;
    }
  };
  f32x4_t acc[DT];
#pragma unroll
  for (int i = 0; i < DT; ++i) acc[i] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
  float behind = 1.f;   // the decays of the chunks behind this one, of key channel d
  const int chunks = (len + 15) / 16;
  fetch((chunks - 1) * 16);
  for (int ch = chunks - 1; ch >= 0; --ch) {
    float own = 1.f;
#pragma unroll
    for (int i = 0; i < TG; ++i) own *= fw[i];
    __syncthreads();   // (the chunk before has been consumed)
    gp[g][d] = own;
#pragma unroll
    for (int i = 0; i < 4; ++i) vs[i * 4 + tid / 64][tid % 64] = fv[i];
    __syncthreads();
    float later = behind, all = 1.f;
#pragma unroll
    for (int j = 0; j < G; ++j) {
      const float p = gp[j][d];
      all *= p;
      if (j > g) later *= p;
    }
#pragma unroll
    for (int i = TG - 1; i >= 0; --i) {
      ks[g * TG + i][d] = fk[i] * later;
      later *= fw[i];
    }
    behind *= all;
    if (ch > 0) fetch((ch - 1) * 16);   // on its way while this chunk is multiplied
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < 4; ++kk) {
      const int t = kk * 4 + (lane >> 4);
      const float b = vs[t][wave * 16 + (lane & 15)];
#pragma unroll
      for (int i = 0; i < DT; ++i) acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(ks[t][i * 16 + (lane & 15)], b, acc[i], 0, 0, 0);
    }
  }
  const int j = slice * 64 + wave * 16 + (lane & 15);
  if (j < a.vdim) {
    float* out = a.piece_state + (place * a.vdim + j) * a.dim;
#pragma unroll
    for (int i = 0; i < DT; ++i) {
      const int row = i * 16 + (lane >> 4) * 4;
      if (a.dim % 4 == 0 && row < a.dim) {
        *(float4*)(out + row) = make_float4(acc[i][0], acc[i][1], acc[i][2], acc[i][3]);
      } else {
#pragma unroll
        for (int c = 0; c < 4; ++c)
          if (row + c < a.dim) out[row + c] = acc[i][c];
      }
    }
  }
  if (slice == 0 && g == 0 && d_ok) a.piece_decay[place * a.dim + d] = behind;
}

// grid: (requests, heads, blocks of 256 state entries); the state each piece starts from, in place of what it ended with from
// zero, and the state after the run
__global__ __launch_bounds__(256) void linear_carry_kernel(LinearScan a) {
  const int r = blockIdx.x, h = blockIdx.y, size = a.dim * a.vdim;
  const int i = blockIdx.z * 256 + threadIdx.x;
  const int run0 = a.cu_seqlens[r], run_len = a.cu_seqlens[r + 1] - run0;
  if (run_len <= a.piece || i >= size) return;
  const int pieces = (run_len + a.piece - 1) / a.piece;
  float* S = a.state + (size_t)a.state_slots[r] * a.state_stride + a.state_off + (size_t)h * size + i;
  const size_t place = (size_t)(run0 / a.piece + r) * a.heads + h;
  float* ps = a.piece_state + place * size + i;
  const float* pd = a.piece_decay + place * a.dim + i % a.dim;
  const size_t ps_step = (size_t)a.heads * size, pd_step = (size_t)a.heads * a.dim;
  float cur = *S, local = *ps, decay = *pd;
  for (int p = 0; p < pieces; ++p) {
    float next_local = 0.f, next_decay = 0.f;
    if (p + 1 < pieces) {   // (on its way while this piece's entry is written)
      next_local = ps[(size_t)(p + 1) * ps_step];
      next_decay = pd[(size_t)(p + 1) * pd_step];
    }
    ps[(size_t)p * ps_step] = cur;
    cur = fmaf(decay, cur, local);
    local = next_local;
    decay = next_decay;
  }
  *S = cur;
}

// q, k, v: first column of float32 rows.  bonus may be missing.  piece 0: no run is cut (max_run then does not matter); else runs
// longer than `piece` are, and scratch holds float32 [pieces * heads * dim * (vdim + 1)] with pieces >= n / piece + n_req.
extern "C" int tp_linear_scan(const float* q, int q_stride, const float* k, int k_stride, const float* v, int v_stride, const float* decay,
                              const float* bonus, float q_scale, float* state, size_t state_stride, size_t state_off,
                              const int* cu_seqlens, const int* state_slots, float* y, int n, int n_req, int heads, int dim, int vdim,
                              int max_run, int piece, int pieces, float* scratch, hipStream_t s) {
  TP_REQUIRE(n >= 0 && n_req >= 0 && heads > 0 && dim > 0 && vdim > 0 && max_run >= 0 && max_run <= n, "linear_scan: bad sizes");
  TP_REQUIRE(dim <= 1024, "linear_scan: key size %d exceeds 1024", dim);
  TP_REQUIRE(q_stride >= heads * dim && k_stride >= heads * dim && v_stride >= heads * vdim, "linear_scan: rows too short");
  TP_REQUIRE(state_stride >= state_off + (size_t)heads * dim * vdim, "linear_scan: state rows too short");
  TP_REQUIRE(heads <= 65535, "linear_scan: too many heads");
  TP_REQUIRE(piece == 0 || dim <= 128, "linear_scan: runs of keys of %d are not cut", dim);
  TP_REQUIRE(piece == 0 || (piece > 0 && scratch != nullptr && pieces >= n / piece + n_req), "linear_scan: no room for the pieces");
  if (n == 0 || n_req == 0) return 0;
  LinearScan a;
  a.q = q; a.k = k; a.v = v;
  a.q_stride = q_stride; a.k_stride = k_stride; a.v_stride = v_stride;
  a.decay = decay; a.bonus = bonus; a.q_scale = q_scale;
  a.state = state; a.state_stride = state_stride; a.state_off = state_off;
  a.cu_seqlens = cu_seqlens; a.state_slots = state_slots; a.y = y;
  a.heads = heads; a.dim = dim; a.vdim = vdim;
  a.piece = piece;
  a.piece_state = scratch;
  a.piece_decay = piece ? scratch + (size_t)pieces * heads * dim * vdim : nullptr;
  // PER key channels a lane (8 up to a key size of 128, then 16, then 32), KS lanes a column (a power of two), TP columns a
  // lane and WAVES waves a block: as many columns a lane as fill a wave without columns to spare, as many waves as the
  // columns need (at most four); single tokens take one column a lane (more blocks, nothing to share)
  const int per = dim <= 128 ? 8 : (dim <= 256 ? 16 : 32);
  int ks = 1;
  while (ks * per < dim) ks *= 2;
  if (per == 32 && ks < 16) ks = 16;
  int tp = 1;
  const int most = per == 32 ? 1 : (per == 16 ? 2 : (ks >= 8 ? 4 : (ks == 4 ? 2 : 1)));
  while (tp < most && max_run > 4 && 64 / ks * tp * 2 <= vdim) tp *= 2;
  const int cw = 64 / ks * tp;
  const int waves = tp == 4 && vdim <= 2 * cw ? 2 : 4;
  const int cb = cw * waves;
  const int slices = (vdim + cb - 1) / cb, end_slices = (vdim + 63) / 64;
  const int most_pieces = piece ? (max_run + piece - 1) / piece : 1;
  TP_REQUIRE((long)(slices > end_slices ? slices : end_slices) * most_pieces <= 65535 && ((long)dim * vdim + 255) / 256 <= 65535,
             "linear_scan: too many value columns or pieces");
#define SCAN_(P, K, T, W, B) hipLaunchKernelGGL((linear_scan_kernel<P, K, T, W, B>), grid, dim3(W * 64), 0, s, a)
#define SCAN(P, K, T, W)         \
  do {                           \
    if (bonus != nullptr)        \
      SCAN_(P, K, T, W, true);   \
    else                         \
      SCAN_(P, K, T, W, false);  \
  } while (0)
  auto launch = [&](int mode, int across) {
    a.mode = mode;
    const dim3 grid(n_req, heads, slices * across);
    if (per == 8) {
      if (ks == 1) SCAN(8, 1, 1, 4);
      else if (ks == 2) SCAN(8, 2, 1, 4);
      else if (ks == 4 && tp == 1) SCAN(8, 4, 1, 4);
      else if (ks == 4) SCAN(8, 4, 2, 4);
      else if (ks == 8 && tp == 1) SCAN(8, 8, 1, 4);
      else if (ks == 8 && tp == 2) SCAN(8, 8, 2, 4);
      else if (ks == 8 && waves == 2) SCAN(8, 8, 4, 2);
      else if (ks == 8) SCAN(8, 8, 4, 4);
      else if (tp == 1) SCAN(8, 16, 1, 4);
      else if (tp == 2) SCAN(8, 16, 2, 4);
      else if (waves == 2) SCAN(8, 16, 4, 2);
      else SCAN(8, 16, 4, 4);
    } else if (per == 16) {
      if (tp == 1) SCAN(16, 16, 1, 4);
      else SCAN(16, 16, 2, 4);
    } else {
      if (ks <= 16) SCAN(32, 16, 1, 4);
      else SCAN(32, 32, 1, 4);
    }
  };
#undef SCAN
#undef SCAN_
  if (piece == 0 || max_run <= piece) {
    launch(SCAN_DIRECT, 1);
  } else {
    const dim3 grid(n_req, heads, end_slices * most_pieces);
    if (dim <= 16) hipLaunchKernelGGL(linear_ends_kernel<1>, grid, dim3(256), 0, s, a);
    else if (dim <= 32) hipLaunchKernelGGL(linear_ends_kernel<2>, grid, dim3(256), 0, s, a);
    else if (dim <= 64) hipLaunchKernelGGL(linear_ends_kernel<4>, grid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL(linear_ends_kernel<8>, grid, dim3(256), 0, s, a);
    hipLaunchKernelGGL(linear_carry_kernel, dim3(n_req, heads, (dim * vdim + 255) / 256), dim3(256), 0, s, a);
    launch(SCAN_PIECES, most_pieces);
  }
  TP_CHECK_LAUNCH("linear_scan");
  return 0;
}
