// Products of many rows with few outputs: y (M, N) = x (M, K) W^T, N at most 64, bfloat16 operands, float32 sums, float32 or
// bfloat16 results.  What a gate of a few numbers a head, or a bottleneck, needs of a prompt portion: the tiled kernels give
// such a product one or two blocks a hundred rows and leave the chip idle.
//
// A block owns 16 rows and all outputs; its eight wavefronts share K out between them in turns of 32, each loading both
// operands straight in the matrix cores' order (v_mfma_f32_16x16x32_bf16: lane l holds row l % 16, eight consecutive k at
// 8 (l / 16)), and their sums are added through LDS in wavefront order.  A row's result depends on nothing but the row.
#include "common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 nr_bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float nr_f32x4_t;
typedef __attribute__((ext_vector_type(4))) unsigned nr_u32x4_t;

#define NR_WAVES 8

template <int NT, typename TO>
__global__ __launch_bounds__(NR_WAVES * 64) void gemm_narrow_kernel(const bf16* __restrict__ x, int ldx,
                                                                    const bf16* __restrict__ w, TO* __restrict__ y, int ldy,
                                                                    int M, int N, int K) {
  __shared__ float part[NR_WAVES][NT][16][17];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r16 = lane & 15, g = lane >> 4;
  const int m0 = blockIdx.x * 16;
  const int mrow = m0 + r16 < M ? m0 + r16 : M - 1;
  const bf16* xp = x + (size_t)mrow * ldx;
  const bf16* wp[NT];
#pragma unroll
  for (int j = 0; j < NT; ++j) {
    const int n = 16 * j + r16 < N ? 16 * j + r16 : N - 1;
    wp[j] = w + (size_t)n * K;
  }
  nr_f32x4_t acc[NT];
#pragma unroll
  for (int j = 0; j < NT; ++j) acc[j] = nr_f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k0 = 32 * wave; k0 < K; k0 += 32 * NR_WAVES) {
    const bool in = k0 + 8 * g < K;                  // K in whole pieces of 8: a piece is inside or outside
    const int k = in ? k0 + 8 * g : 0;
    nr_u32x4_t a = *reinterpret_cast<const nr_u32x4_t*>(xp + k);
    a = in ? a : nr_u32x4_t{0u, 0u, 0u, 0u};
    nr_u32x4_t b[NT];
#pragma unroll
    for (int j = 0; j < NT; ++j) {
      b[j] = *reinterpret_cast<const nr_u32x4_t*>(wp[j] + k);
      b[j] = in ? b[j] : nr_u32x4_t{0u, 0u, 0u, 0u};
    }
#pragma unroll
    for (int j = 0; j < NT; ++j)
      acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(nr_bf16x8_t, a), __builtin_bit_cast(nr_bf16x8_t, b[j]),
                                                       acc[j], 0, 0, 0);
  }
#pragma unroll
  for (int j = 0; j < NT; ++j)
#pragma unroll
    for (int e = 0; e < 4; ++e) part[wave][j][4 * g + e][r16] = acc[j][e];
  __syncthreads();
  for (int i = threadIdx.x; i < 16 * 16 * NT; i += NR_WAVES * 64) {
    const int m = i / (16 * NT), n = i - m * 16 * NT;
    if (m0 + m >= M || n >= N) continue;
    float s = 0.f;
#pragma unroll
    for (int v = 0; v < NR_WAVES; ++v) s += part[v][n >> 4][m][n & 15];
    y[(size_t)(m0 + m) * ldy + n] = from_f32<TO>(s);
  }
}

extern "C" int gs_gemm_narrow(const void* x, int ldx, const void* w, void* y, int y_dtype, int ldy, int M, int N, int K,
                              hipStream_t stream) {
  GS_REQUIRE(M >= 0 && N > 0 && N <= 64 && K > 0 && K % 8 == 0, "gemm_narrow: bad sizes M=%d N=%d K=%d", M, N, K);
  GS_REQUIRE(ldx >= K && ldx % 8 == 0 && ldy >= N, "gemm_narrow: bad row strides %d, %d", ldx, ldy);
  GS_REQUIRE((((uintptr_t)x | (uintptr_t)w) & 15) == 0, "gemm_narrow: operands must be 16-byte aligned");
  if (M == 0) return 0;
  const int blocks = gs_ceil_div(M, 16), nt = gs_ceil_div(N, 16);
#define GS_RUN(NT, TO) \
  gemm_narrow_kernel<NT, TO><<<blocks, NR_WAVES * 64, 0, stream>>>((const bf16*)x, ldx, (const bf16*)w, (TO*)y, ldy, M, N, K)
#define GS_RUN_T(TO)                 \
  switch (nt) {                      \
    case 1: GS_RUN(1, TO); break;    \
    case 2: GS_RUN(2, TO); break;    \
    case 3: GS_RUN(3, TO); break;    \
    default: GS_RUN(4, TO); break;   \
  }
  if (y_dtype == GS_F32) {
    GS_RUN_T(float)
  } else if (y_dtype == GS_BF16) {
    GS_RUN_T(bf16)
  } else {
    GS_REQUIRE(false, "gemm_narrow: unknown dtype %d", y_dtype);
  }
#undef GS_RUN_T
#undef GS_RUN
  GS_LAUNCH_CHECK("gemm_narrow");
  return 0;
}
