// Element helpers shared by the kernels that run in bf16 (serving) or fp32 (exact replay).
#pragma once
#include "common.h"

namespace ragk {

template <typename T>
__device__ __forceinline__ float ld1(const T* p);
template <>
__device__ __forceinline__ float ld1<bf16_t>(const bf16_t* p) { return bf2f(*p); }
template <>
__device__ __forceinline__ float ld1<float>(const float* p) { return *p; }

__device__ __forceinline__ void st1(bf16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void st1(float* p, float v) { *p = v; }

__device__ __forceinline__ void ld8(const bf16_t* p, float* f) { unpack8(*reinterpret_cast<const u32x4*>(p), f); }
__device__ __forceinline__ void ld8(const float* p, float* f) {
  const f32x4 a = reinterpret_cast<const f32x4*>(p)[0], b = reinterpret_cast<const f32x4*>(p)[1];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    f[e] = a[e];
    f[4 + e] = b[e];
  }
}
__device__ __forceinline__ void st8(bf16_t* p, const float* f) { *reinterpret_cast<u32x4*>(p) = pack8(f); }
__device__ __forceinline__ void st8(float* p, const float* f) {
  reinterpret_cast<f32x4*>(p)[0] = (f32x4){f[0], f[1], f[2], f[3]};
  reinterpret_cast<f32x4*>(p)[1] = (f32x4){f[4], f[5], f[6], f[7]};
}

// sequence that packed token t belongs to: the last s with cu[s] <= t (cu has S + 1 entries, cu[0] = 0)
__device__ __forceinline__ int seq_of(const int* cu, int S, int t) {
  int lo = 0, hi = S - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (cu[mid] <= t) lo = mid;
    else hi = mid - 1;
  }
  return lo;
}

// ln(1 + e^z), exact to fp32 rounding over the whole range
__device__ __forceinline__ float softplusf(float z) { return z > 20.f ? z + log1pf(expf(-z)) : log1pf(expf(z)); }
// z * sigmoid(z) with IEEE division (norms and gates that must hold fp32 accuracy)
__device__ __forceinline__ float silu_exact(float z) { return z / (1.f + expf(-z)); }

}  // namespace ragk
