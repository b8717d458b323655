// A product of its own for every head: out[m, h, :] = scale * sigmoid(gate[m, h]) * W[h] x[m, h, :], bfloat16 weights
// [heads, N, K] on the gfx950 matrix cores with float32 accumulation.  The rows of x and out are strided, so that the
// operands are pieces of wider rows: x may be the float32 sums of a projection (rounded to bfloat16 here), out a part of
// the rows that an attention or an output product reads.
//
// A wave owns 16 NT weight rows and 16 MT rows of x (four times sixteen of each in steps of many rows, where what it reads
// would otherwise come from L2 once for every sixteen rows): the weight rows are the first operand, so a result lane holds four
// neighbouring columns of one row.  Everything is read straight from memory (a head's weights are a few hundred KB and
// shared by all row tiles; the heads run fastest in the grid, so that with a multiple of eight heads each XCD's L2
// holds the weights of an eighth of them).
#include <math.h>

#include "common.h"

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef float f32x2_t __attribute__((ext_vector_type(2)));
typedef __bf16 bf16x2_t __attribute__((ext_vector_type(2)));
typedef unsigned int u32x4_t __attribute__((ext_vector_type(4)));

namespace {
__device__ inline unsigned pack2(float a, float b) {
  const f32x2_t f = {a, b};
  return __builtin_bit_cast(unsigned, __builtin_convertvector(f, bf16x2_t));
}
__device__ inline bf16x8_t eight(const bf16_t* p) { return __builtin_bit_cast(bf16x8_t, *(const u32x4_t*)p); }
__device__ inline bf16x8_t eight(const float* p) {
  const f32x4_t a = *(const f32x4_t*)p, b = *(const f32x4_t*)(p + 4);
  const u32x4_t v = {pack2(a[0], a[1]), pack2(a[2], a[3]), pack2(b[0], b[1]), pack2(b[2], b[3])};
  return __builtin_bit_cast(bf16x8_t, v);
}
}  // namespace

// grid: (heads, ceil(row tiles * column groups / 4)); block: four waves, each a (tile of 16 MT rows, group of 16 NT columns).
template <typename TX, int NT, int MT>
__global__ __launch_bounds__(256) void head_linear_kernel(const TX* __restrict__ x, size_t x_row, int x_head, const bf16_t* __restrict__ w,
                                                          bf16_t* __restrict__ out, size_t out_row, int out_head,
                                                          const float* __restrict__ gate, size_t gate_row, float scale, int M, int N, int K) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int g = lane >> 4, c = lane & 15;
  const int h = blockIdx.x;
  const int groups = (N + 16 * NT - 1) / (16 * NT);
  const long item = (long)blockIdx.y * 4 + wave;
  const int m0 = (int)(item / groups) * 16 * MT, n0 = (int)(item % groups) * 16 * NT;
  if (m0 >= M) return;
  const TX* xr[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i)          // (rows past the end repeat the last one, never written)
    xr[i] = x + (size_t)min(m0 + i * 16 + c, M - 1) * x_row + (size_t)h * x_head + g * 8;
  const bf16_t* wr[NT];
#pragma unroll
  for (int j = 0; j < NT; ++j) wr[j] = w + ((size_t)h * N + min(n0 + j * 16, N - 16) + c) * K + g * 8;   // (a tile past N repeats the last one)
  f32x4_t acc[MT][NT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[i][j] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll(MT == 1 ? 4 : 2)
  for (int k = 0; k < K; k += 32) {
    bf16x8_t a[NT], b[MT];
#pragma unroll
    for (int i = 0; i < MT; ++i) b[i] = eight(xr[i] + k);
#pragma unroll
    for (int j = 0; j < NT; ++j) a[j] = eight(wr[j] + k);
#pragma unroll
    for (int i = 0; i < MT; ++i)
#pragma unroll
      for (int j = 0; j < NT; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[j], b[i], acc[i][j], 0, 0, 0);
  }
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const int m = m0 + i * 16 + c;
    if (m >= M) break;
    float f = scale;
    if (gate != nullptr) f *= 1.0f / (1.0f + expf(-gate[(size_t)m * gate_row + h]));
    bf16_t* o = out + (size_t)m * out_row + (size_t)h * out_head;
#pragma unroll
    for (int j = 0; j < NT; ++j) {
      const int n = n0 + j * 16 + 4 * g;
      if (n0 + j * 16 < N) {
        uint2 v;
        v.x = pack2(acc[i][j][0] * f, acc[i][j][1] * f);
        v.y = pack2(acc[i][j][2] * f, acc[i][j][3] * f);
        *(uint2*)(o + n) = v;
      }
    }
  }
}

// x (TP_F32 or TP_BF16): element (m, h, k) at m * x_row + h * x_head + k; out (bfloat16): (m, h, n) at m * out_row +
// h * out_head + n; gate (optional): (m, h) at m * gate_row + h.  K % 32 == 0, N % 16 == 0; x pieces start at multiples of
// 16 bytes, out pieces at multiples of eight.
extern "C" int tp_head_linear(const void* x, int x_dt, size_t x_row, int x_head, const void* w, void* out, size_t out_row, int out_head,
                              const float* gate, size_t gate_row, float scale, int M, int H, int N, int K, hipStream_t s) {
  TP_REQUIRE(M >= 0 && H > 0 && N > 0 && K > 0, "head_linear: bad sizes");
  TP_REQUIRE(K % 32 == 0 && N % 16 == 0, "head_linear: needs K %% 32 == 0 and N %% 16 == 0 (N=%d K=%d)", N, K);
  TP_REQUIRE(x_dt == TP_F32 || x_dt == TP_BF16, "head_linear: unknown dtype %d", x_dt);
  const int piece = x_dt == TP_F32 ? 4 : 8;
  TP_REQUIRE(((uintptr_t)x & 15) == 0 && ((uintptr_t)w & 15) == 0 && ((uintptr_t)out & 7) == 0 && x_row % piece == 0 && x_head % piece == 0 &&
                 out_row % 4 == 0 && out_head % 4 == 0, "head_linear: operands are not aligned");
  if (M == 0) return 0;
  // (a wave for every sixteen rows and columns up to 64 rows; wider tiles where they leave every CU some waves)
  const int nt = M <= 64 ? 1 : 4;
  const long groups = (N + 16 * nt - 1) / (16 * nt);
  int mt = nt == 1 ? 1 : 4;
  while (mt > 1 && (long)((M + 16 * mt - 1) / (16 * mt)) * groups * H < 2048) mt >>= 1;
  const long items = (long)((M + 16 * mt - 1) / (16 * mt)) * groups;
  TP_REQUIRE((items + 3) / 4 <= 65535, "head_linear: too many rows (%d)", M);
  const dim3 grid(H, (unsigned)((items + 3) / 4));
#define HL(TX, NT_, MT_)                                                                                                                   \
  hipLaunchKernelGGL((head_linear_kernel<TX, NT_, MT_>), grid, dim3(256), 0, s, (const TX*)x, x_row, x_head, (const bf16_t*)w, (bf16_t*)out, \
                     out_row, out_head, gate, gate_row, scale, M, N, K)
#define HL_ROWS(TX)                                \
  do {                                             \
    if (nt == 1) HL(TX, 1, 1);                     \
    else if (mt == 1) HL(TX, 4, 1);                \
    else if (mt == 2) HL(TX, 4, 2);                \
    else HL(TX, 4, 4);                             \
  } while (0)
  if (x_dt == TP_F32) HL_ROWS(float);
  else HL_ROWS(bf16_t);
#undef HL_ROWS
#undef HL
  TP_CHECK_LAUNCH("head_linear");
  return 0;
}
