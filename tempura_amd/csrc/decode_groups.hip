// Products of decode steps (at most 16 bfloat16 rows) that come in groups: several products whose inputs differ in one
// launch, and the two products of a layer of routed experts.  Their time is the weights' stream from memory, so a launch per
// group pays its start and its end once for all, and the weights of experts that no row of the step has chosen are not read.
//
// Rows are k-blocked, [K / 8, M, 8], weights tiled, [N / 16][K / 32][64][8] (see gemm_mfma.hip): every load of a wave is
// one run of neighbouring bytes.  A block owns 16 result columns; its eight waves split K in runs of 128 (run r of a weight
// goes to wave r % 8, whatever else is skipped), and their sums meet through LDS in the order of the waves, so a row's
// result has the same bits whatever the other rows are.
#include <math.h>

#include "common.h"
#include "activations.h"

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef unsigned int u32x4_t __attribute__((ext_vector_type(4)));

#define DG_WAVES 8
#define DG_MAX_GROUPS 8
#define DG_MAX_EXPERTS 512

__device__ inline f32x4_t dg_mfma(u32x4_t w, u32x4_t x, f32x4_t acc) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, w), __builtin_bit_cast(bf16x8_t, x), acc, 0, 0, 0);
}

// acc += the wave's runs of one 16-row tile of a weight: wp this lane's first piece of the tile, xp of the rows; steps of 32 k
__device__ inline f32x4_t dg_tile(const u32x4_t* wp, const u32x4_t* xp, int xstep, int steps, int wave, f32x4_t acc) {
  for (int s0 = wave * 4; s0 < steps; s0 += DG_WAVES * 8) {
    u32x4_t a[2][4], b[2][4];
#pragma unroll
    for (int d = 0; d < 2; ++d)
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int s = min(s0 + d * DG_WAVES * 4 + u, steps - 1);   // (steps past the end repeat the last one and are dropped below)
        a[d][u] = __builtin_nontemporal_load(wp + (size_t)s * 64);
        b[d][u] = xp[(size_t)s * xstep];
      }
#pragma unroll
    for (int d = 0; d < 2; ++d)
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (s0 + d * DG_WAVES * 4 + u < steps) acc = dg_mfma(a[d][u], b[d][u], acc);
  }
  return acc;
}

// the waves' sums of element q (lane q / 4, register q % 4) in wave order
__device__ inline float dg_sum(const float (*red)[256], int q) {
  float v = 0.f;
#pragma unroll
  for (int i = 0; i < DG_WAVES; ++i) v += red[i][q];
  return v;
}

// ---- several products in one launch -------------------------------------------------------------
// Rows n of the stacked weight belong to the first group g with n < end[g] (multiples of 16) and multiply the rows x + g * M * K.
struct GroupEnds {
  int end[DG_MAX_GROUPS];
};

__global__ __launch_bounds__(DG_WAVES * 64) void group_linear_kernel(const bf16_t* __restrict__ x, const bf16_t* __restrict__ w,
                                                                      float* __restrict__ out, GroupEnds ends, int M, int N, int K) {
  __shared__ float red[DG_WAVES][256];
  const int lane = threadIdx.x % 64, wave = threadIdx.x / 64;
  const int n0 = blockIdx.x * 16;
  int g = 0;
#pragma unroll
  for (int i = 0; i < DG_MAX_GROUPS - 1; ++i) g += n0 >= ends.end[i] ? 1 : 0;
  const u32x4_t* wp = (const u32x4_t*)(w + (size_t)n0 * K) + lane;
  const int row = min(lane & 15, M - 1);
  const u32x4_t* xp = (const u32x4_t*)(x + (size_t)g * M * K + ((size_t)(lane >> 4) * M + row) * 8);
  const f32x4_t acc = dg_tile(wp, xp, 4 * M, K / 32, wave, (f32x4_t){0.f, 0.f, 0.f, 0.f});
#pragma unroll
  for (int r = 0; r < 4; ++r) red[wave][lane * 4 + r] = acc[r];
  __syncthreads();
  const int q = threadIdx.x;
  if (q >= 256) return;
  const int l = q / 4, m = l & 15;
  const float v = dg_sum(red, q);
  if (m < M) out[(size_t)m * N + n0 + (l >> 4) * 4 + q % 4] = v;
}

// x: bfloat16, groups times [K / 8, M, 8]; w: tiled [N, K]; ends: host array, ends[groups - 1] == N; out float32 [M, N]
extern "C" int tp_group_linear(const void* x, const void* w, float* out, const int* ends, int groups, int M, int N, int K, hipStream_t s) {
  TP_REQUIRE(M > 0 && M <= 16 && N > 0 && N % 16 == 0 && K > 0 && K % 64 == 0, "group_linear: sizes M %d N %d K %d", M, N, K);
  TP_REQUIRE(groups > 0 && groups <= DG_MAX_GROUPS && ends[groups - 1] == N, "group_linear: %d groups", groups);
  TP_REQUIRE((((uintptr_t)x | (uintptr_t)w) & 15) == 0, "group_linear: operands must be aligned to 16 bytes");
  GroupEnds e;
  for (int i = 0; i < DG_MAX_GROUPS; ++i) {
    e.end[i] = i < groups ? ends[i] : N;
    TP_REQUIRE(e.end[i] % 16 == 0 && e.end[i] <= N && e.end[i] > (i > 0 && i < groups ? e.end[i - 1] : 0), "group_linear: bad group borders");
  }
  hipLaunchKernelGGL(group_linear_kernel, dim3(N / 16), dim3(DG_WAVES * 64), 0, s, (const bf16_t*)x, (const bf16_t*)w, out, e, M, N, K);
  TP_CHECK_LAUNCH("group_linear");
  return 0;
}

// ---- routed experts ---------------------------------------------------------------------------------
// Up: a[m][e * ff + c] = f(x_m . up_e[c]) * dense[m][e] as bfloat16, k-blocked over the columns of all experts; experts whose
// column of `dense` is zero for all rows are skipped (their columns stay unwritten).  GATED: the weight's rows alternate
// eight gate rows and eight up rows, and f is silu(gate) * up.
template <bool GATED>
__global__ __launch_bounds__(DG_WAVES * 64) void moe_up_kernel(const bf16_t* __restrict__ x, const bf16_t* __restrict__ w,
                                                                const float* __restrict__ dense, bf16_t* __restrict__ a, int M, int experts,
                                                                int rows, int K, int kind) {
  __shared__ float red[DG_WAVES][256];
  const int lane = threadIdx.x % 64, wave = threadIdx.x / 64;
  const int n0 = blockIdx.x * 16, e = n0 / rows;
  const float mine = lane < M ? dense[(size_t)lane * experts + e] : 0.f;
  if (__ballot(mine != 0.f) == 0ull) return;   // (the same for every wave of the block)
  const u32x4_t* wp = (const u32x4_t*)(w + (size_t)n0 * K) + lane;
  const int row = min(lane & 15, M - 1);
  const u32x4_t* xp = (const u32x4_t*)(x + ((size_t)(lane >> 4) * M + row) * 8);
  const f32x4_t acc = dg_tile(wp, xp, 4 * M, K / 32, wave, (f32x4_t){0.f, 0.f, 0.f, 0.f});
#pragma unroll
  for (int r = 0; r < 4; ++r) red[wave][lane * 4 + r] = acc[r];
  __syncthreads();
  const int q = threadIdx.x;
  if (q >= (GATED ? 128 : 256)) return;
  const int l = q / 4, m = l & 15;
  if (m >= M) return;
  const float weight = dense[(size_t)m * experts + e];
  const float v = dg_sum(red, q);
  float y;
  if (GATED) {
    const float u = dg_sum(red, q + 128);   // (a gate row's up row is eight further on)
    y = act_f(v, 1) * u;
  } else {
    y = act_f(v, kind);
  }
  const int n = (GATED ? n0 / 2 : n0) + (l >> 4) * 4 + q % 4;
  a[((size_t)(n >> 3) * M + m) * 8 + (n & 7)] = float_to_bf16(weight == 0.f ? 0.f : y * weight);
}

// Down: y[m] (+)= sum_e a[m][e] . down_e, experts ascending; the same experts are skipped.  w: every expert's tiled [N, ff], one
// behind the other.
__global__ __launch_bounds__(DG_WAVES * 64) void moe_down_kernel(const bf16_t* __restrict__ a, const bf16_t* __restrict__ w,
                                                                  const float* __restrict__ dense, float* __restrict__ y, int M, int experts,
                                                                  int ff, int N, int accumulate) {
  __shared__ float red[DG_WAVES][256];
  __shared__ int list[DG_MAX_EXPERTS];
  __shared__ int counts[DG_WAVES];
  const int lane = threadIdx.x % 64, wave = threadIdx.x / 64;
  // the experts in use, ascending
  bool used = false;
  if ((int)threadIdx.x < experts)
    for (int m = 0; m < M; ++m) used = used || dense[(size_t)m * experts + threadIdx.x] != 0.f;
  const unsigned long long mask = __ballot(used);
  if (lane == 0) counts[wave] = __popcll(mask);
  __syncthreads();
  int before = 0, total = 0;
#pragma unroll
  for (int i = 0; i < DG_WAVES; ++i) {
    if (i < wave) before += counts[i];
    total += counts[i];
  }
  if (used) list[before + __popcll(mask & ((1ull << lane) - 1ull))] = threadIdx.x;
  __syncthreads();

  const int n0 = blockIdx.x * 16, steps = ff / 32, runs = (steps + 3) / 4;
  const int row = min(lane & 15, M - 1);
  const int xstep = 4 * M;
  const u32x4_t* w_lane = (const u32x4_t*)(w + (size_t)n0 * ff) + lane;
  const u32x4_t* x_lane = (const u32x4_t*)(a + ((size_t)(lane >> 4) * M + row) * 8);
  const size_t w_expert = (size_t)N * ff / 8, x_expert = (size_t)(ff / 8) * M;   // in pieces of 16 bytes
  // run r of expert e goes to wave (e * runs + r) % 8: `per` turns an expert
  const int per = (runs + DG_WAVES - 1) / DG_WAVES;
  f32x4_t acc = (f32x4_t){0.f, 0.f, 0.f, 0.f};
  for (int it = 0; it < total * per; it += 2) {
    u32x4_t av[2][4], bv[2][4];
    int left[2];
#pragma unroll
    for (int d = 0; d < 2; ++d) {
      const int i = min(it + d, total * per - 1);
      const int e = __builtin_amdgcn_readfirstlane(list[i / per]);
      const int run = i % per * DG_WAVES + ((wave - e * runs) & (DG_WAVES - 1));
      left[d] = it + d < total * per && run < runs ? min(4, steps - run * 4) : 0;
      const u32x4_t* wp = w_lane + (size_t)e * w_expert;
      const u32x4_t* xp = x_lane + (size_t)e * x_expert;
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int s = min(run * 4 + u, steps - 1);
        av[d][u] = __builtin_nontemporal_load(wp + (size_t)s * 64);
        bv[d][u] = xp[(size_t)s * xstep];
      }
    }
#pragma unroll
    for (int d = 0; d < 2; ++d)
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (u < left[d]) acc = dg_mfma(av[d][u], bv[d][u], acc);
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) red[wave][lane * 4 + r] = acc[r];
  __syncthreads();
  const int q = threadIdx.x;
  if (q >= 256) return;
  const int l = q / 4, m = l & 15;
  if (m >= M) return;
  float* o = y + (size_t)m * N + n0 + (l >> 4) * 4 + q % 4;
  const float v = dg_sum(red, q);
  *o = accumulate ? *o + v : v;
}

// x: bfloat16 [K / 8, M, 8]; w_up: tiled [experts * rows, K], rows = ff, or 2 ff with gated (kind is then not read); w_down: experts
// tiled [N, ff]; dense float32 [M, experts]; a: bfloat16 scratch [experts * ff / 8, M, 8]; y float32 [M, N].
extern "C" int tp_moe_few(const void* x, const void* w_up, const void* w_down, const float* dense, void* a, float* y, int M, int experts,
                          int ff, int K, int N, int gated, int kind, int accumulate, hipStream_t s) {
  TP_REQUIRE(M > 0 && M <= 16 && experts > 0 && experts <= DG_MAX_EXPERTS, "moe_few: %d rows, %d experts", M, experts);
  TP_REQUIRE(ff > 0 && ff % 64 == 0 && K > 0 && K % 64 == 0 && N > 0 && N % 16 == 0, "moe_few: sizes ff %d K %d N %d", ff, K, N);
  TP_REQUIRE(gated || (kind >= 0 && kind <= 3), "moe_few: unknown activation %d", kind);
  TP_REQUIRE((((uintptr_t)x | (uintptr_t)w_up | (uintptr_t)w_down | (uintptr_t)a) & 15) == 0, "moe_few: operands must be aligned to 16 bytes");
  const int rows = gated ? 2 * ff : ff;
  TP_REQUIRE((long)experts * rows < 0x7fffffffL, "moe_few: too many rows");
  const dim3 up(experts * rows / 16), block(DG_WAVES * 64);
  if (gated)
    hipLaunchKernelGGL(moe_up_kernel<true>, up, block, 0, s, (const bf16_t*)x, (const bf16_t*)w_up, dense, (bf16_t*)a, M, experts, rows, K, 0);
  else
    hipLaunchKernelGGL(moe_up_kernel<false>, up, block, 0, s, (const bf16_t*)x, (const bf16_t*)w_up, dense, (bf16_t*)a, M, experts, rows, K, kind);
  hipLaunchKernelGGL(moe_down_kernel, dim3(N / 16), block, 0, s, (const bf16_t*)a, (const bf16_t*)w_down, dense, y, M, experts, ff, N, accumulate);
  TP_CHECK_LAUNCH("moe_few");
  return 0;
}

// bfloat16 rows [M, K] -> [K / 8, M, 8]
__global__ void block_rows_kernel(const u32x4_t* __restrict__ x, u32x4_t* __restrict__ out, int M, int pieces) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= M * pieces) return;
  const int m = i / pieces, p = i % pieces;
  out[(size_t)p * M + m] = x[i];
}

extern "C" int tp_block_rows(const void* x, void* out, int M, int K, hipStream_t s) {
  TP_REQUIRE(M > 0 && K > 0 && K % 8 == 0 && (long)M * (K / 8) < 0x7fffffffL && (((uintptr_t)x | (uintptr_t)out) & 15) == 0, "block_rows: bad rows");
  const int total = M * (K / 8);
  hipLaunchKernelGGL(block_rows_kernel, dim3((total + 255) / 256), dim3(256), 0, s, (const u32x4_t*)x, (u32x4_t*)out, M, K / 8);
  TP_CHECK_LAUNCH("block_rows");
  return 0;
}
