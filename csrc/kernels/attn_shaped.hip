// Attention with shaped scores over the paged cache (K pages [blocks][G][64][DK], V pages [blocks][G][64][DV]):
//
//   s_ij = softcap * tanh(q_i . k_j * scale / softcap) + table[h][min(i - j, far)]
//   j visible to i:  j <= i  and  (window == 0 or i - j < window or j < keep)
//   out_i = gate_ih * sum_j exp(s_ij) v_j / (sink + sum_j exp(s_ij)),  sink in {0, 1}
//
// Positions are the tokens' own in the sequence, so the kept first tokens enter with their true distances.
// Scores, softmax and the bias are fp32.
//
//  * kv_store     : k, and v mixed with the first mixing layer's values of the same token, into the pages.
//  * attn_rows    : one wave per (token, query head), plain fp32 arithmetic. Any head size; the fp32 path.
#include "seq_common.h"
using namespace ragk;

namespace {

struct ShapedArgs {
  const void* q; int ldq;      // projection rows; head h at h * DK, gates at off_g
  const void* kc; const void* vc;
  const int* block_tables; int bt_stride;
  const int* cu_q;             // [S + 1]; null: one token per sequence
  const int* kv_lens;          // [S]
  const float* table;          // [H][far + 1] or null
  void* out; int ldo;
  int T, S, H, G, DK, DV;
  int off_g;                   // column of the gates, -1: no gate
  int window, keep, far, sink;
  float scale, softcap;
};

template <typename T>
__global__ __launch_bounds__(256) void kv_store_kernel(const T* __restrict__ row, int ld, int off_k, int off_v, int G, int DK,
                                                       int DV, const int* __restrict__ slots, T* kc, T* vc,
                                                       const T* __restrict__ v_first, int ldf,
                                                       const float* __restrict__ lam) {
  const int t = blockIdx.x, slot = slots[t];
  if (slot < 0) return;
  const int blk = slot >> 6, off = slot & 63;
  const T* r = row + (size_t)t * ld;
  const int nk = G * DK / 8, nv = G * DV / 8;
  for (int i = threadIdx.x; i < nk + nv; i += 256) {
    float f[8];
    if (i < nk) {
      const int g = i / (DK / 8), c = (i % (DK / 8)) * 8;
      ld8(r + off_k + i * 8, f);
      st8(kc + (((size_t)blk * G + g) * 64 + off) * DK + c, f);
    } else {
      const int j = i - nk, g = j / (DV / 8), c = (j % (DV / 8)) * 8;
      ld8(r + off_v + j * 8, f);
      if (v_first != nullptr) {
        const float lm = lam[0];
        float w[8];
        ld8(v_first + (size_t)t * ldf + j * 8, w);
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] = (1.f - lm) * f[e] + lm * w[e];
      }
      st8(vc + (((size_t)blk * G + g) * 64 + off) * DV + c, f);
    }
  }
}

template <typename T>
__global__ __launch_bounds__(64) void attn_rows_kernel(ShapedArgs a) {
  __shared__ float sq[256], sp[64];
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const int s = a.cu_q ? seq_of(a.cu_q, a.S, t) : t;
  const int q0 = a.cu_q ? a.cu_q[s] : t, q1 = a.cu_q ? a.cu_q[s + 1] : t + 1;
  const int L = a.kv_lens[s], i = L - (q1 - q0) + (t - q0);
  const int g = h / (a.H / a.G);
  const T* qr = (const T*)a.q + (size_t)t * a.ldq;
  for (int d = lane; d < a.DK; d += 64) sq[d] = ld1(qr + h * a.DK + d);
  __syncthreads();
  const int* bt = a.block_tables + (size_t)s * a.bt_stride;
  const int n_pages = i / 64 + 1;
  const int keep_pages = a.window > 0 ? min(n_pages, (a.keep + 63) / 64) : n_pages;
  const int first_win = a.window > 0 ? max(keep_pages, max(0, i - a.window + 1) / 64) : n_pages;
  const int n_it = keep_pages + max(0, n_pages - first_win);
  float m = a.sink ? 0.f : -INFINITY, l = a.sink ? 1.f : 0.f;
  float acc[4] = {0.f, 0.f, 0.f, 0.f};
  for (int it = 0; it < n_it; ++it) {
    const int pg = it < keep_pages ? it : first_win + it - keep_pages;
    const int blk = bt[pg], j = pg * 64 + lane;
    const T* kr = (const T*)a.kc + (((size_t)blk * a.G + g) * 64 + lane) * a.DK;
    const bool ok = j <= i && (a.window <= 0 || i - j < a.window || j < a.keep);
    float x = 0.f;
    if (ok) {
      for (int d = 0; d < a.DK; d += 8) {
        float f[8];
        ld8(kr + d, f);
#pragma unroll
        for (int e = 0; e < 8; ++e) x = fmaf(sq[d + e], f[e], x);
      }
      x *= a.scale;
      if (a.softcap > 0.f) x = a.softcap * tanhf(x / a.softcap);
      if (a.table) x += a.table[(size_t)h * (a.far + 1) + min(i - j, a.far)];
    } else {
      x = -INFINITY;
    }
    const float mn = fmaxf(m, wave_max(x));
    if (mn == -INFINITY) continue;  // nothing visible yet (uniform over the wave)
    const float alpha = expf(m - mn);
    const float p = expf(x - mn);
    m = mn;
    l = l * alpha + wave_sum(p);
    __syncthreads();
    sp[lane] = p;
    __syncthreads();
    const T* vb = (const T*)a.vc + ((size_t)blk * a.G + g) * 64 * a.DV;
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      const int d = lane + 64 * c;
      if (d < a.DV) {
        acc[c] *= alpha;
        const int nj = min(64, i + 1 - pg * 64);
        for (int k = 0; k < nj; ++k) acc[c] = fmaf(sp[k], ld1(vb + (size_t)k * a.DV + d), acc[c]);
      }
    }
  }
  const float inv = l > 0.f ? 1.f / l : 0.f;
  float gate = 1.f;
  if (a.off_g >= 0) gate = 1.f / (1.f + expf(-ld1(qr + a.off_g + h)));
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    const int d = lane + 64 * c;
    if (d < a.DV) st1((T*)a.out + (size_t)t * a.ldo + h * a.DV + d, acc[c] * inv * gate);
  }
}

}  // namespace

// row: projection rows [T][ld] (fp32 when f32). v_first: [T][ldf] own values of the first mixing layer, or null.
RAGK_API int ragk_shaped_kv_store(const void* row, int ld, int off_k, int off_v, int T, int G, int DK, int DV,
                                  const int* slots, void* kc, void* vc, const void* v_first, int ldf, const float* lam,
                                  int f32, hipStream_t st) {
  if (T <= 0) return 0;
  if (DK % 8 || DV % 8 || ld % 8 || off_k % 8 || off_v % 8 || ldf % 8 || (v_first && !lam))
    return (int)hipErrorInvalidValue;
  if (f32)
    hipLaunchKernelGGL(kv_store_kernel<float>, dim3(T), dim3(256), 0, st, (const float*)row, ld, off_k, off_v, G, DK, DV,
                       slots, (float*)kc, (float*)vc, (const float*)v_first, ldf, lam);
  else
    hipLaunchKernelGGL(kv_store_kernel<bf16_t>, dim3(T), dim3(256), 0, st, (const bf16_t*)row, ld, off_k, off_v, G, DK, DV,
                       slots, (bf16_t*)kc, (bf16_t*)vc, (const bf16_t*)v_first, ldf, lam);
  return (int)hipGetLastError();
}

RAGK_API int ragk_shaped_attn_rows(const void* q, int ldq, const void* kc, const void* vc, const int* block_tables,
                                   int bt_stride, const int* cu_q, const int* kv_lens, const float* table, void* out,
                                   int ldo, int T, int S, int H, int G, int DK, int DV, int off_g, int window, int keep,
                                   int far, int sink, float scale, float softcap, int f32, hipStream_t st) {
  if (T <= 0) return 0;
  if (DK % 8 || DK > 256 || DV > 256 || H % G || H > 65535) return (int)hipErrorInvalidValue;
  const ShapedArgs a{q, ldq, kc, vc, block_tables, bt_stride, cu_q, kv_lens, table, out, ldo, T, S, H, G, DK, DV,
                     off_g, window, keep, far, sink, scale, softcap};
  if (f32) hipLaunchKernelGGL(attn_rows_kernel<float>, dim3(T, H), dim3(64), 0, st, a);
  else hipLaunchKernelGGL(attn_rows_kernel<bf16_t>, dim3(T, H), dim3(64), 0, st, a);
  return (int)hipGetLastError();
}
