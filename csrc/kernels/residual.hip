// Residual-stream kernels: the stream h is fp32 rows, padded to the GEMM tile (padding columns are zero).
//
//  * embed_residual : h[t] = table[ids[t]] in fp32 (ids may be carried over from the previous step's samples).
//  * residual_norm  : h += norm(y) * w_post; out = norm(h) * w_next, one pass over the row. y is a sublayer's
//    output: fp32 split-K slabs (summed here, so a decode GEMM needs no reduction launch), fp32 rows or bf16
//    rows. Without w_post the sublayer is added as it is; without y only the norm runs; without w_next only
//    the add. norm(x) = x / sqrt(mean(x^2) + eps) over the n real columns.
//  * glu_clip       : the clipped gated unit over packed [64 gate | 64 up] tiles (fp32 path; the bf16 GEMMs
//    have it as an epilogue).
#include "seq_common.h"
using namespace ragk;

namespace {

template <typename T>
__global__ __launch_bounds__(256) void embed_residual_kernel(int* __restrict__ ids, const T* __restrict__ table, float* h,
                                                             int W, int vocab, const int* __restrict__ carry,
                                                             const int* __restrict__ prev) {
  const int t = blockIdx.x;
  int id = ids[t];
  if (carry != nullptr) {
    const int c = carry[t];
    if (c >= 0) {
      id = prev[c];
      __syncthreads();  // every lane has read ids[t] before lane 0 overwrites it
      if (threadIdx.x == 0) ids[t] = id;
    }
  }
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  for (int v = threadIdx.x; v < (W >> 3); v += 256) {
    float f[8];
    ld8(table + (size_t)id * W + v * 8, f);
    st8(h + (size_t)t * W + v * 8, f);
  }
}

template <int MAXV, typename TY, typename TO>
__global__ __launch_bounds__(256) void residual_norm_kernel(float* h, const TY* __restrict__ y, int ldy, int S, size_t slab,
                                                            const float* __restrict__ w_post,
                                                            const float* __restrict__ w_next, TO* out, int W, float n,
                                                            float eps) {
  __shared__ float red[4];
  const int row = blockIdx.x, nvec = W >> 3;
  float* hr = h + (size_t)row * W;
  // everything the row needs is requested before the first reduction (rows up to 8192 columns)
  constexpr bool PRE = MAXV <= 4;
  constexpr int PV = PRE ? MAXV : 1;
  float v[MAXV][8], hv[PV][8], wp[PV][8], wn[PV][8];
  if constexpr (PRE) {
#pragma unroll
    for (int i = 0; i < MAXV; ++i) {
      const int vi = min((int)threadIdx.x + i * 256, nvec - 1);
      ld8(hr + vi * 8, hv[i]);
      if (w_post != nullptr) ld8(w_post + vi * 8, wp[i]);
      if (w_next != nullptr) ld8(w_next + vi * 8, wn[i]);
    }
  }
  float ss = 0.f;
  if (y != nullptr) {
#pragma unroll
    for (int i = 0; i < MAXV; ++i) {
      const int vi = threadIdx.x + i * 256;
      if (vi < nvec) {
        const TY* yp = y + (size_t)row * ldy + vi * 8;
        if constexpr (sizeof(TY) == 4) sum_slabs8(yp, S, slab, v[i]);
        else ld8(yp, v[i]);
#pragma unroll
        for (int e = 0; e < 8; ++e) ss += v[i][e] * v[i][e];
      }
    }
    float inv = 1.f;
    if (w_post != nullptr) inv = rsqrtf(block_sum(ss, red) / n + eps);
    ss = 0.f;
#pragma unroll
    for (int i = 0; i < MAXV; ++i) {
      const int vi = threadIdx.x + i * 256;
      if (vi < nvec) {
        if constexpr (!PRE) {
          ld8(hr + vi * 8, hv[0]);
          if (w_post != nullptr) ld8(w_post + vi * 8, wp[0]);
        }
        const int k = PRE ? i : 0;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          v[i][e] = hv[k][e] + (w_post != nullptr ? v[i][e] * inv * wp[k][e] : v[i][e]);
          ss += v[i][e] * v[i][e];
        }
        st8(hr + vi * 8, v[i]);
      }
    }
  } else {
#pragma unroll
    for (int i = 0; i < MAXV; ++i) {
      const int vi = threadIdx.x + i * 256;
      if (vi < nvec) {
        if constexpr (!PRE) ld8(hr + vi * 8, hv[0]);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          v[i][e] = hv[PRE ? i : 0][e];
          ss += v[i][e] * v[i][e];
        }
      }
    }
  }
  if (w_next == nullptr) return;
  const float inv = rsqrtf(block_sum(ss, red) / n + eps);
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const int vi = threadIdx.x + i * 256;
    if (vi < nvec) {
      if constexpr (!PRE) ld8(w_next + vi * 8, wn[0]);
      float o[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) o[e] = v[i][e] * inv * wn[PRE ? i : 0][e];
      st8(out + (size_t)row * W + vi * 8, o);
    }
  }
}

template <typename TY, typename TO>
int launch_residual_norm(float* h, const void* y, int ldy, int S, size_t slab, const float* wp, const float* wn, void* out,
                         int M, int W, float n, float eps, hipStream_t st) {
  const int per = (W / 8 + 255) / 256;
#define RAGK_RN(V)                                                                                                \
  hipLaunchKernelGGL((residual_norm_kernel<V, TY, TO>), dim3(M), dim3(256), 0, st, h, (const TY*)y, ldy, S, slab, \
                     wp, wn, (TO*)out, W, n, eps)
  if (per <= 1) RAGK_RN(1);
  else if (per <= 2) RAGK_RN(2);
  else if (per <= 4) RAGK_RN(4);
  else if (per <= 8) RAGK_RN(8);
  else return (int)hipErrorInvalidValue;
#undef RAGK_RN
  return (int)hipGetLastError();
}

// out[m][c] = sum_s P[s][m][c] (+ bias[c]): split-K slabs to activation rows, for consumers that take rows
template <typename T>
__global__ __launch_bounds__(256) void slab_rows_kernel(const float* __restrict__ P, int S, size_t slab,
                                                        const T* __restrict__ bias, T* out, int N) {
  const int row = blockIdx.x;
  for (int v = threadIdx.x; v < (N >> 3); v += 256) {
    float a[8];
    sum_slabs8(P + (size_t)row * N + v * 8, S, slab, a);
    if (bias != nullptr) {
      float b[8];
      ld8(bias + v * 8, b);
#pragma unroll
      for (int e = 0; e < 8; ++e) a[e] += b[e];
    }
    st8(out + (size_t)row * N + v * 8, a);
  }
}

__global__ __launch_bounds__(256) void glu_clip_kernel(const float* __restrict__ x, float* out, int F,
                                                       const float* __restrict__ par) {
  const int t = blockIdx.x;
  const float limit = par[0], alpha = par[1], shift = par[2];
  for (int j = threadIdx.x; j < F; j += 256) {
    const float* p = x + (size_t)t * 2 * F + (j >> 6) * 128 + (j & 63);
    const float g = fminf(p[0], limit), u = fminf(fmaxf(p[64], -limit), limit);
    out[(size_t)t * F + j] = g / (1.f + expf(-alpha * g)) * (u + shift);
  }
}

}  // namespace

// table: [vocab][W] bf16 (f32 = 0) or fp32; h: fp32 [T][W], W % 8 == 0. carry / prev may be null.
RAGK_API int ragk_embed_residual(int* ids, const void* table, float* h, int T, int W, int vocab, const int* carry,
                                 const int* prev, int f32, hipStream_t st) {
  if (T <= 0) return 0;
  if (W % 8) return (int)hipErrorInvalidValue;
  if (f32)
    hipLaunchKernelGGL(embed_residual_kernel<float>, dim3(T), dim3(256), 0, st, ids, (const float*)table, h, W, vocab,
                       carry, prev);
  else
    hipLaunchKernelGGL(embed_residual_kernel<bf16_t>, dim3(T), dim3(256), 0, st, ids, (const bf16_t*)table, h, W, vocab,
                       carry, prev);
  return (int)hipGetLastError();
}

// h: fp32 [M][W]. y: null, fp32 slabs [S][M][ldy] (y_bf16 = 0) or bf16 rows [M][ldy] (S = 1). out: [M][W], fp32
// when out_f32. W % 8 == 0, W <= 16384.
RAGK_API int ragk_residual_norm(float* h, const void* y, int ldy, int S, int y_bf16, const float* w_post,
                                const float* w_next, void* out, int out_f32, int M, int W, int n, float eps,
                                hipStream_t st) {
  if (M <= 0) return 0;
  if (W % 8 || ldy % 8 || (y && S < 1) || (y_bf16 && S != 1) || (w_next && !out)) return (int)hipErrorInvalidValue;
  const size_t slab = (size_t)M * ldy;
  const float fn = (float)n;
  if (y_bf16)
    return out_f32 ? launch_residual_norm<bf16_t, float>(h, y, ldy, 1, slab, w_post, w_next, out, M, W, fn, eps, st)
                   : launch_residual_norm<bf16_t, bf16_t>(h, y, ldy, 1, slab, w_post, w_next, out, M, W, fn, eps, st);
  return out_f32 ? launch_residual_norm<float, float>(h, y, ldy, S, slab, w_post, w_next, out, M, W, fn, eps, st)
                 : launch_residual_norm<float, bf16_t>(h, y, ldy, S, slab, w_post, w_next, out, M, W, fn, eps, st);
}

// x: fp32 [M][2F] in packed gate/up tiles, out: fp32 [M][F], F % 64 == 0; par = {limit, alpha, shift} on the device.
RAGK_API int ragk_glu_clip(const float* x, float* out, int M, int F, const float* par, hipStream_t st) {
  if (M <= 0) return 0;
  if (F % 64) return (int)hipErrorInvalidValue;
  hipLaunchKernelGGL(glu_clip_kernel, dim3(M), dim3(256), 0, st, x, out, F, par);
  return (int)hipGetLastError();
}

// P: fp32 slabs [S][M][N], bias [N] or null -> out [M][N] (bf16, or fp32 when f32). N % 8 == 0.
RAGK_API int ragk_slab_rows(const float* P, int S, const void* bias, void* out, int M, int N, int f32, hipStream_t st) {
  if (M <= 0) return 0;
  if (S < 1 || N % 8) return (int)hipErrorInvalidValue;
  const size_t slab = (size_t)M * N;
  if (f32)
    hipLaunchKernelGGL(slab_rows_kernel<float>, dim3(M), dim3(256), 0, st, P, S, slab, (const float*)bias, (float*)out, N);
  else
    hipLaunchKernelGGL(slab_rows_kernel<bf16_t>, dim3(M), dim3(256), 0, st, P, S, slab, (const bf16_t*)bias, (bf16_t*)out,
                       N);
  return (int)hipGetLastError();
}
