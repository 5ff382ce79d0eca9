// fp32 GEMM for the exact-replay path: C[M,N] = A[M,K] . B[N,K]^T (+ bias), true fp32 products
// (v_mfma_f32_16x16x4_f32). 64x64 output tile, 4 waves of 32x32, 32-deep K slices through LDS.
#include "seq_common.h"
using namespace ragk;

namespace {

constexpr int FT = 64, FK = 32, FLD = FK + 4;

__global__ __launch_bounds__(256) void gemm_f32_kernel(const float* __restrict__ A, int lda, const float* __restrict__ B,
                                                       int ldb, float* C, int ldc, const float* __restrict__ bias, int M,
                                                       int N, int K) {
  __shared__ __attribute__((aligned(16))) float sa[FT][FLD], sb[FT][FLD];
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int fr = lane & 15, fh = lane >> 4, wr = (wid >> 1) * 32, wc = (wid & 1) * 32;
  const int m0 = blockIdx.y * FT, n0 = blockIdx.x * FT;
  f32x4 acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) acc[i][j] = (f32x4){0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < K; k0 += FK) {
#pragma unroll
    for (int i = 0; i < 2; ++i) {  // 64 rows x 8 vectors of 4
      const int v = tid + i * 256, r = v >> 3, c = (v & 7) * 4;
      *reinterpret_cast<f32x4*>(&sa[r][c]) =
          *reinterpret_cast<const f32x4*>(A + (size_t)min(m0 + r, M - 1) * lda + k0 + c);
      *reinterpret_cast<f32x4*>(&sb[r][c]) =
          *reinterpret_cast<const f32x4*>(B + (size_t)min(n0 + r, N - 1) * ldb + k0 + c);
    }
    __syncthreads();
#pragma unroll
    for (int s = 0; s < FK; s += 4) {
      float a[2], b[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        a[i] = sa[wr + 16 * i + fr][s + fh];
        b[i] = sb[wc + 16 * i + fr][s + fh];
      }
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[j], acc[i][j], 0, 0, 0);
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = m0 + wr + 16 * i + 4 * fh + r, col = n0 + wc + 16 * j + fr;
        if (row < M && col < N) C[(size_t)row * ldc + col] = acc[i][j][r] + (bias ? bias[col] : 0.f);
      }
}

}  // namespace

// K % 32 == 0, row strides multiples of 4. bias (fp32 [N]) may be null.
RAGK_API int ragk_gemm_f32(const float* A, int lda, const float* B, int ldb, float* C, int ldc, const float* bias, int M,
                           int N, int K, hipStream_t st) {
  if (M <= 0 || N <= 0) return 0;
  if (K % FK || lda % 4 || ldb % 4) return (int)hipErrorInvalidValue;
  hipLaunchKernelGGL(gemm_f32_kernel, dim3((N + FT - 1) / FT, (M + FT - 1) / FT), dim3(256), 0, st, A, lda, B, ldb, C, ldc,
                     bias, M, N, K);
  return (int)hipGetLastError();
}
