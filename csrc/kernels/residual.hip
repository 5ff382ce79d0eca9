// Residual-stream kernels: the stream h is fp32 rows, padded to the GEMM tile (padding columns are zero).
//
//  * embed_residual : h[t] = table[ids[t]] * scale in fp32 (ids may be carried over from the previous step's samples),
//    plus the sinusoid of the token's position: angles are reduced in fp64, so they are exact to fp32 rounding at any
//    position.
//  * residual_norm  : h += norm(y) * w_post; out = norm(h) * w_next, one pass over the row. y is a sublayer's
//    output: fp32 split-K slabs (summed here, so a decode GEMM needs no reduction launch), fp32 rows or bf16
//    rows. Without w_post the sublayer is added as it is; without y only the norm runs; without w_next only
//    the add. norm(x) = x / sqrt(mean(x^2) + eps) over the n real columns.
//  * gated_residual : h += norm(y * sigmoid(z + b)) * w, the sublayer gated element by element before its norm; then
//    the rows themselves and / or the token-shifted rows, for a next sublayer that reads the stream without a norm.
//  * token_shift    : x[t] + (x[t-1] - x[t]) * mix; the row before a sequence's first new token is its state.
//  * glu_clip       : the clipped gated unit over packed [64 gate | 64 up] tiles (fp32 path; the bf16 GEMMs
//    have it as an epilogue).
#include "seq_common.h"
using namespace ragk;

namespace {

template <typename T>
__global__ __launch_bounds__(256) void embed_residual_kernel(int* __restrict__ ids, const T* __restrict__ table, float* h,
                                                             int W, int vocab, const int* __restrict__ carry,
                                                             const int* __restrict__ prev, float scale, int n,
                                                             const int* __restrict__ pos,
                                                             const double* __restrict__ turns) {
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
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] *= scale;
    if (pos != nullptr) {  // columns 2i / 2i + 1: sin / cos of pos * turns[i] whole turns
      const double p = pos[t];
#pragma unroll
      for (int e = 0; e < 8; e += 2) {
        const int c = v * 8 + e;
        if (c < n) {
          const double a = p * turns[c >> 1];
          float sn, cs;
          sincospif((float)(2.0 * (a - rint(a))), &sn, &cs);
          f[e] += sn;
          if (c + 1 < n) f[e + 1] += cs;
        }
      }
    }
    st8(h + (size_t)t * W + v * 8, f);
  }
}

// new row of one vector of the stream -> the shifted row (prev: the row before it)
template <typename TO>
__device__ __forceinline__ void put_shifted(TO* dst, const float* x, const float* prev, const float* mix) {
  float o[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) o[e] = x[e] + (prev[e] - x[e]) * mix[e];
  st8(dst, o);
}

struct GatedArgs {
  float* h; int W; float n, eps;
  const void* y; int S; const void* z; int SZ; size_t slab;  // rows, or fp32 split-K slabs
  const float* zb; const float* w;                            // [W]; zb null: y is not gated
  void* out;                                                   // the new rows, or null
  const float* mix; void* shifted; float* state;              // decode: one row per sequence; null: no shift
  const int* slots; const int* kv_lens;
};

template <int NT, int MAXV, typename TY, typename TO>
__global__ __launch_bounds__(NT) void gated_residual_kernel(GatedArgs a) {
  __shared__ float red[NT / 64];
  const int row = blockIdx.x, nvec = a.W >> 3;
  const size_t base = (size_t)row * a.W;
  constexpr bool PRE = MAXV <= 2;  // the stream's row and the weights are requested before the reduction
  constexpr int PV = PRE ? MAXV : 1;
  float v[MAXV][8], hv[PV][8], wv[PV][8];
  auto fetch = [&](int i, int k) {
    const int vi = min((int)threadIdx.x + i * NT, nvec - 1);
    ld8(a.h + base + vi * 8, hv[k]);
    ld8(a.w + vi * 8, wv[k]);
  };
  if constexpr (PRE) {
#pragma unroll
    for (int i = 0; i < MAXV; ++i) fetch(i, i);
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const int vi = threadIdx.x + i * NT;
    if (vi < nvec) {
      const TY* yp = (const TY*)a.y + base + vi * 8;
      const TY* zp = (const TY*)a.z + base + vi * 8;
      float z[8], b[8];
      if constexpr (sizeof(TY) == 4) {  // both sets of slabs in flight together
        f32x4 py[PSU][2], pz[PSU][2];
        load_slabs8(yp, a.S, a.slab, py);
        if (a.zb != nullptr) {
          load_slabs8(zp, a.SZ, a.slab, pz);
          ld8(a.zb + vi * 8, b);
        }
        add_slabs8(py, yp, a.S, a.slab, v[i]);
        if (a.zb != nullptr) add_slabs8(pz, zp, a.SZ, a.slab, z);
      } else {
        ld8(yp, v[i]);
        if (a.zb != nullptr) {
          ld8(zp, z);
          ld8(a.zb + vi * 8, b);
        }
      }
      if (a.zb != nullptr) {
#pragma unroll
        for (int e = 0; e < 8; ++e) v[i][e] /= 1.f + expf(-(z[e] + b[e]));
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += v[i][e] * v[i][e];
    }
  }
  const float inv = rsqrtf(block_sum(ss, red) / a.n + a.eps);
  float* st = nullptr;
  bool fresh = false;
  if (a.mix != nullptr) {
    st = a.state + (size_t)a.slots[row] * a.W;
    fresh = a.kv_lens[row] == 1;
  }
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const int vi = threadIdx.x + i * NT;
    if (vi < nvec) {
      const int k = PRE ? i : 0;
      if constexpr (!PRE) fetch(i, 0);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[i][e] = hv[k][e] + v[i][e] * inv * wv[k][e];
      st8(a.h + base + vi * 8, v[i]);
      if (a.out != nullptr) st8((TO*)a.out + base + vi * 8, v[i]);
      if (st != nullptr) {
        float p[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f}, m[8];
        if (!fresh) ld8(st + vi * 8, p);
        ld8(a.mix + vi * 8, m);
        put_shifted((TO*)a.shifted + base + vi * 8, v[i], p, m);
        st8(st + vi * 8, v[i]);
      }
    }
  }
}

template <int NT, typename TY, typename TO>
int launch_gated_nt(const GatedArgs& a, int M, hipStream_t st) {
  const int per = (a.W / 8 + NT - 1) / NT;
  if (per <= 1) hipLaunchKernelGGL((gated_residual_kernel<NT, 1, TY, TO>), dim3(M), dim3(NT), 0, st, a);
  else if (per <= 2) hipLaunchKernelGGL((gated_residual_kernel<NT, 2, TY, TO>), dim3(M), dim3(NT), 0, st, a);
  else if (per <= 4) hipLaunchKernelGGL((gated_residual_kernel<NT, 4, TY, TO>), dim3(M), dim3(NT), 0, st, a);
  else if (per <= 8) hipLaunchKernelGGL((gated_residual_kernel<NT, 8, TY, TO>), dim3(M), dim3(NT), 0, st, a);
  else return (int)hipErrorInvalidValue;
  return (int)hipGetLastError();
}
template <typename TY, typename TO>
int launch_gated(const GatedArgs& a, int M, hipStream_t st) {
  // few rows of slabs: one vector a thread, so that a row is one round of loads
  if (sizeof(TY) == 4 && a.W > 2048 && M <= 256) return launch_gated_nt<512, TY, TO>(a, M, st);
  return launch_gated_nt<256, TY, TO>(a, M, st);
}

// cu null: one token per sequence. The block of a sequence's first new token reads the state and then replaces it by
// the last new row, element by element in the same thread.
template <typename TO>
__global__ __launch_bounds__(256) void token_shift_kernel(const float* __restrict__ h, int W, const float* __restrict__ mix,
                                                          float* state, const int* __restrict__ slots,
                                                          const int* __restrict__ cu, const int* __restrict__ kv_lens,
                                                          int S, TO* out, TO* shifted) {
  const int t = blockIdx.x;
  const int s = cu ? seq_of(cu, S, t) : t, q0 = cu ? cu[s] : t, q1 = cu ? cu[s + 1] : t + 1;
  const bool first = t == q0, fresh = kv_lens[s] == q1 - q0;
  float* st = state + (size_t)slots[s] * W;
  for (int v = threadIdx.x; v < (W >> 3); v += 256) {
    float x[8], p[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f}, m[8];
    ld8(h + (size_t)t * W + v * 8, x);
    ld8(mix + v * 8, m);
    if (!first) ld8(h + (size_t)(t - 1) * W + v * 8, p);
    else if (!fresh) ld8(st + v * 8, p);
    if (out != nullptr) st8(out + (size_t)t * W + v * 8, x);
    put_shifted(shifted + (size_t)t * W + v * 8, x, p, m);
    if (first) {
      float l[8];
      ld8(h + (size_t)(q1 - 1) * W + v * 8, l);
      st8(st + v * 8, l);
    }
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

// table: [vocab][W] bf16 (f32 = 0) or fp32; h: fp32 [T][W], W % 8 == 0. carry / prev may be null. pos [T] and turns
// [(n + 1) / 2] (fp64, turns per position of each column pair), or null: no sinusoid.
RAGK_API int ragk_embed_residual(int* ids, const void* table, float* h, int T, int W, int vocab, const int* carry,
                                 const int* prev, float scale, int n, const int* pos, const double* turns, int f32,
                                 hipStream_t st) {
  if (T <= 0) return 0;
  if (W % 8 || n > W || (pos && !turns)) return (int)hipErrorInvalidValue;
  if (f32)
    hipLaunchKernelGGL(embed_residual_kernel<float>, dim3(T), dim3(256), 0, st, ids, (const float*)table, h, W, vocab,
                       carry, prev, scale, n, pos, turns);
  else
    hipLaunchKernelGGL(embed_residual_kernel<bf16_t>, dim3(T), dim3(256), 0, st, ids, (const bf16_t*)table, h, W, vocab,
                       carry, prev, scale, n, pos, turns);
  return (int)hipGetLastError();
}

// h: fp32 [M][W] += norm(y * sigmoid(z + zb)) * w. y, z: bf16 rows [M][W] (y_bf16, S = SZ = 1) or fp32 slabs [S][M][W].
// out / shifted: [M][W], fp32 when out_f32; either may be null. shifted takes mix [W], state [slots][W], slots, kv_lens [M]
// (one token per sequence).
RAGK_API int ragk_gated_residual(float* h, const void* y, int S, const void* z, int SZ, int y_bf16, const float* zb,
                                 const float* w, void* out, const float* mix, void* shifted, float* state,
                                 const int* slots, const int* kv_lens, int out_f32, int M, int W, int n, float eps,
                                 hipStream_t st) {
  if (M <= 0) return 0;
  if (W % 8 || W > 16384 || !y || !w || S < 1 || SZ < 1 || (y_bf16 && (S != 1 || SZ != 1)) || (zb && !z) ||
      (mix && (!shifted || !state || !slots || !kv_lens)))
    return (int)hipErrorInvalidValue;
  const GatedArgs a{h, W, (float)n, eps, y, S, z, SZ, (size_t)M * W, zb, w, out, mix, shifted, state, slots, kv_lens};
  if (y_bf16) return out_f32 ? launch_gated<bf16_t, float>(a, M, st) : launch_gated<bf16_t, bf16_t>(a, M, st);
  return out_f32 ? launch_gated<float, float>(a, M, st) : launch_gated<float, bf16_t>(a, M, st);
}

// h: fp32 [T][W]; cu [S + 1] or null (one token per sequence); out (may be null) / shifted: [T][W], fp32 when f32
RAGK_API int ragk_token_shift(const float* h, int T, int W, const float* mix, float* state, const int* slots, const int* cu,
                              const int* kv_lens, int S, void* out, void* shifted, int f32, hipStream_t st) {
  if (T <= 0) return 0;
  if (W % 8 || !mix || !state || !slots || !kv_lens || !shifted || (!cu && S != T)) return (int)hipErrorInvalidValue;
  if (f32)
    hipLaunchKernelGGL(token_shift_kernel<float>, dim3(T), dim3(256), 0, st, h, W, mix, state, slots, cu, kv_lens, S,
                       (float*)out, (float*)shifted);
  else
    hipLaunchKernelGGL(token_shift_kernel<bf16_t>, dim3(T), dim3(256), 0, st, h, W, mix, state, slots, cu, kv_lens, S,
                       (bf16_t*)out, (bf16_t*)shifted);
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
