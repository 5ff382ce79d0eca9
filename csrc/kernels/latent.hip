// Latent attention: a token's cache entry is one normed latent row c [R]; keys and values of every head are linear in it
// (k_h = Uk_h c, v_h = Uv_h c).
//
//  * Prompts expand: the latents of the visible tokens (their own rows of this step, latent_store, or gathered from the
//    pages, latent_gather) go through one GEMM with [Uk | Uv] and the row attention of attn_shaped.hip.
//  * Decoding absorbs: q'_h = Uk_h^T q_h (latent_absorb), attention of all heads over the latent pages, each page serving
//    as keys and as values (latent_decode), then o_h = Uv_h (sum_j p_j c_j) with the output gate (latent_out). The
//    projection arrives as fp32 split-K slabs (or as rows), so slab sums, the latent's norm and the cache append need no
//    launch of their own.
//
// Cache: pages [blocks][64][Rp], Rp = R rounded up to 128 (zero columns). Scores, softmax, norms and the partial outputs
// are fp32; the softmax weights enter P.C as bf16 high + low parts.
#include "attn_tiles.h"
#include "seq_common.h"
using namespace ragk;

namespace {

constexpr float LOG2E = 1.4426950408889634f;
constexpr int NORM_T = 128;  // threads per latent row: 8 columns each, R up to 1024

// x [8 per thread] -> rms-normed * w; red: NORM_T / 64 floats
template <int NT>
__device__ __forceinline__ void norm_row(float* f, const float* __restrict__ w, int R, float eps, int c, bool in, float* red) {
  float ss = 0.f;
  if (in) {
#pragma unroll
    for (int e = 0; e < 8; ++e) ss += f[e] * f[e];
  }
  const float inv = rsqrtf(block_sum(ss, red) / (float)R + eps);
  if (in) {
    float g[8];
    ld8(w + c, g);
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] *= inv * g[e];
  }
}

// rows [T][ld] at column off_c -> normed latents in the pages and in crows [T + pad][Rp] (pad rows zero)
template <typename T>
__global__ __launch_bounds__(NORM_T) void latent_store_kernel(const T* __restrict__ row, int ld, int off_c, int R, int Rp,
                                                              const float* __restrict__ w, float eps,
                                                              const int* __restrict__ slots, T* pages, T* crows, int n) {
  __shared__ float red[NORM_T / 64];
  const int t = blockIdx.x, c = threadIdx.x * 8;
  const bool in = c < Rp;
  float f[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
  if (t < n) {
    if (in) ld8(row + (size_t)t * ld + off_c + c, f);
    norm_row<NORM_T>(f, w, R, eps, c, in, red);
    const int slot = slots[t];
    if (in && slot >= 0) st8(pages + (size_t)slot * Rp + c, f);
  }
  if (in && crows) st8(crows + (size_t)t * Rp + c, f);
}

// packed key rows of the step: row r of sequence s is position r - key_off[s]; rows past the last are zero
template <typename T>
__global__ __launch_bounds__(NORM_T) void latent_gather_kernel(const T* __restrict__ pages, int Rp, const int* __restrict__ bt,
                                                               int bt_stride, const int* __restrict__ cu_k,
                                                               const int* __restrict__ key_off, int S, int n, T* out) {
  const int r = blockIdx.x, c = threadIdx.x * 8;
  if (c >= Rp) return;
  float f[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
  if (r < n) {
    const int s = seq_of(cu_k, S, r), p = r - key_off[s];
    ld8(pages + ((size_t)bt[(size_t)s * bt_stride + (p >> 6)] * 64 + (p & 63)) * Rp + c, f);
  }
  st8(out + (size_t)r * Rp + c, f);
}

// y[t][h][n] = sum_k x[t][h][k] w[h][n][k] (* sigmoid(gate[t][h][n])), plain fp32
__global__ __launch_bounds__(256) void head_proj_f32_kernel(const float* __restrict__ x, int ldx, int K,
                                                            const float* __restrict__ w, int N, const float* __restrict__ g,
                                                            int ldg, float* y, int ldy) {
  __shared__ float sx[1024];
  const int h = blockIdx.x, t = blockIdx.y;
  for (int k = threadIdx.x; k < K; k += 256) sx[k] = x[(size_t)t * ldx + (size_t)h * K + k];
  __syncthreads();
  for (int n = threadIdx.x; n < N; n += 256) {
    const float* wr = w + ((size_t)h * N + n) * K;
    float a = 0.f;
    for (int k = 0; k < K; k += 4) {
      const f32x4 v = *reinterpret_cast<const f32x4*>(wr + k);
#pragma unroll
      for (int e = 0; e < 4; ++e) a = fmaf(sx[k + e], v[e], a);
    }
    if (g) a /= 1.f + expf(-g[(size_t)t * ldg + (size_t)h * N + n]);
    y[(size_t)t * ldy + (size_t)h * N + n] = a;
  }
}

// projection rows of a decode step: fp32 slabs [S][B][ld] or bf16 rows [B][ld]
template <typename TP>
struct Proj {
  const TP* P; int S; size_t slab; int ld;
  __device__ __forceinline__ void row8(int b, int col, float* f) const {
    const TP* p = P + (size_t)b * ld + col;
    if constexpr (sizeof(TP) == 4) sum_slabs8(p, S, slab, f);
    else ld8(p, f);
  }
};

constexpr int DB = 16;  // sequences per block (one MFMA column each)

template <typename TP>
struct AbsorbArgs {
  Proj<TP> P;
  int B, H, Rp, R, off_c;
  const bf16_t* wuk;   // [H][Rp][DK]
  bf16_t* qa;          // [B][H][Rp]
  bf16_t* pages; const int* slots; const float* norm; float eps;  // pages null: the latent belongs to another layer
};

// grid: (H * Rp / 128 blocks of 128 latent columns of one head, then DB append blocks; batch / DB)
template <typename TP, int DK>
__global__ __launch_bounds__(256) void latent_absorb_kernel(AbsorbArgs<TP> a) {
  __shared__ __attribute__((aligned(16))) bf16_t s_q[DB * (DK + 8)];
  __shared__ float red[4];
  const int nt = a.Rp / 128, bx = blockIdx.x, b0 = blockIdx.y * DB, nb = min(DB, a.B - b0);
  if (bx >= a.H * nt) {
    const int b = b0 + bx - a.H * nt;
    if (b >= a.B) return;  // block-uniform, before any barrier
    const int c = threadIdx.x * 8;
    const bool in = c < a.Rp;
    float f[8];
    if (in) a.P.row8(b, a.off_c + c, f);
    norm_row<256>(f, a.norm, a.R, a.eps, c, in, red);
    const int slot = a.slots[b];
    if (in && slot >= 0) st8(a.pages + (size_t)slot * a.Rp + c, f);
    return;
  }
  const int h = bx / nt, lane = threadIdx.x & 63, wid = threadIdx.x >> 6, fr = lane & 15, fh = lane >> 4;
  const int r0 = (bx % nt) * 128 + wid * 32;
  constexpr int KS = DK / 32;
  bf16x8 wf[2][KS];  // requested before the slab sums
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int s = 0; s < KS; ++s)
      wf[t][s] = *reinterpret_cast<const bf16x8*>(a.wuk + ((size_t)h * a.Rp + r0 + 16 * t + fr) * DK + 32 * s + 8 * fh);
  for (int i = threadIdx.x; i < DB * (DK / 8); i += 256) {
    const int b = i / (DK / 8), c = (i % (DK / 8)) * 8;
    float f[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (b < nb) a.P.row8(b0 + b, h * DK + c, f);
    st8(s_q + b * (DK + 8) + c, f);
  }
  __syncthreads();
  f32x4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
  for (int s = 0; s < KS; ++s) {
    const bf16x8 q = *reinterpret_cast<const bf16x8*>(s_q + fr * (DK + 8) + 32 * s + 8 * fh);
#pragma unroll
    for (int t = 0; t < 2; ++t) acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[t][s], q, acc[t], 0, 0, 0);
  }
  if (fr < nb) {
    bf16_t* o = a.qa + ((size_t)(b0 + fr) * a.H + h) * a.Rp + r0 + 4 * fh;
#pragma unroll
    for (int t = 0; t < 2; ++t)
      *reinterpret_cast<uint2*>(o + 16 * t) = make_uint2(pk2bf(acc[t][0], acc[t][1]), pk2bf(acc[t][2], acc[t][3]));
  }
}

// ---- attention over latent pages ----
struct LatentArgs {
  const bf16_t* qa;    // [B][H][Rp]
  const bf16_t* pages; // [blocks][64][Rp]
  const int* block_tables; int bt_stride;
  const int* kv_lens;
  float* part_o;       // [B][H][max_parts][Rp], not normalised
  float* part_ml;      // [B][H][max_parts][2]: maximum (log2 units) and sum
  int B, H, window, min_tiles, max_parts;
  float scale;
};
__device__ __forceinline__ int first_page(int pos, int window) { return window > 0 ? max(0, pos - window + 1) / KT : 0; }
__device__ __forceinline__ int part_pages(int n, int min_tiles, int max_parts) {
  return max(min_tiles, (n + max_parts - 1) / max_parts);
}
// the latent tile serves row reads (keys) and transposed reads (values): 32-B granules kept, 8 rows on distinct banks
__device__ __forceinline__ int cswz(int row) { return 2 * (row & 7); }
__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
  __builtin_amdgcn_sched_barrier(0);
}

constexpr int P_STRIDE = 72;  // bf16 per head row of the weights in LDS (64 keys, padded)

// grid: (max_parts, groups of 16 NHT heads, batch); 4 waves share each 64-token page: a wave scores 16 of its tokens for
// all the block's heads and accumulates a quarter of the latent columns.
template <int NR, int NHT>
__global__ __launch_bounds__(256, 1) void latent_decode_kernel(LatentArgs a) {
  constexpr int Rp = 128 * NR, ROWB = 2 * Rp, NC = Rp / 8, TILE = KT * ROWB, PIECES = TILE / 1024 / 4, BUFS = NR <= 4 ? 2 : 1;
  constexpr int KS = Rp / 32, DT = Rp / 64, NH = 16 * NHT;  // k-steps of a score; 16-column tiles per wave; heads
  extern __shared__ __attribute__((aligned(16))) char smem[];
  bf16_t* s_p = reinterpret_cast<bf16_t*>(smem + BUFS * TILE);   // [hi | lo][NH][P_STRIDE]
  float* s_m = reinterpret_cast<float*>(s_p + 2 * NH * P_STRIDE);  // [4][NH]
  const int lane = threadIdx.x & 63, wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int fr = lane & 15, fh = lane >> 4;
  const int part = blockIdx.x, h0 = blockIdx.y * NH, b = blockIdx.z;
  const int pos = a.kv_lens[b] - 1, p0 = first_page(pos, a.window), np = pos / KT + 1 - p0;
  const int pt = part_pages(np, a.min_tiles, a.max_parts), it0 = part * pt;
  if (it0 >= np) return;  // block-uniform, before any barrier
  const int it1 = min(it0 + pt, np);
  const int* bt = a.block_tables + (size_t)b * a.bt_stride + p0;

  int off[PIECES];
#pragma unroll
  for (int i = 0; i < PIECES; ++i) {
    const int idx = (wid + 4 * i) * 64 + lane, row = idx / NC, ph = idx % NC;
    off[i] = row * ROWB + 16 * (ph ^ cswz(row));
  }
  const unsigned lds0 = lds_addr(smem);
  auto stage = [&](int it, int buf) {
    const i32x4 srd = make_srd(a.pages + (size_t)__builtin_amdgcn_readfirstlane(bt[it]) * KT * Rp, TILE);
#pragma unroll
    for (int i = 0; i < PIECES; ++i) blds16_asm(srd, off[i], 0, lds0 + buf * TILE + (wid + 4 * i) * 1024);
  };
  stage(it0, 0);

  bf16x8 qf[NHT][KS];
#pragma unroll
  for (int t = 0; t < NHT; ++t) {
    const bf16_t* q = a.qa + ((size_t)b * a.H + min(h0 + 16 * t + fr, a.H - 1)) * Rp + 8 * fh;
#pragma unroll
    for (int s = 0; s < KS; ++s) qf[t][s] = *reinterpret_cast<const bf16x8*>(q + 32 * s);
  }
  f32x4 o[DT][NHT];
#pragma unroll
  for (int d = 0; d < DT; ++d)
#pragma unroll
    for (int t = 0; t < NHT; ++t) o[d][t] = (f32x4){0.f, 0.f, 0.f, 0.f};
  float m[NHT], l[NHT];
#pragma unroll
  for (int t = 0; t < NHT; ++t) {
    m[t] = -INFINITY;
    l[t] = 0.f;
  }
  const float c = a.scale * LOG2E;
  const int win = a.window > 0 ? a.window : 0x7fffffff;
  wait_vmcnt0();
  lds_barrier();

  for (int it = it0; it < it1; ++it) {
    const int buf = BUFS == 2 ? (it - it0) & 1 : 0, k0 = (p0 + it) * KT;
    const char* tile = smem + buf * TILE;
    if (BUFS == 2 && it + 1 < it1) stage(it + 1, buf ^ 1);
    f32x4 s4[NHT];
#pragma unroll
    for (int t = 0; t < NHT; ++t) s4[t] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const int row = 16 * wid + fr;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const bf16x8 kf = *reinterpret_cast<const bf16x8*>(tile + row * ROWB + 16 * ((4 * s + fh) ^ cswz(row)));
#pragma unroll
      for (int t = 0; t < NHT; ++t) s4[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[t][s], s4[t], 0, 0, 0);
    }
    const int d0 = pos - k0 - 16 * wid - 4 * fh;  // distance of this lane's first token
    const bool edge = pos < k0 + KT - 1 || pos - k0 >= win;
#pragma unroll
    for (int t = 0; t < NHT; ++t) {
      float mx = -INFINITY;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = d0 - r;
        s4[t][r] = !edge || (d >= 0 && d < win) ? s4[t][r] * c : -INFINITY;
        mx = fmaxf(mx, s4[t][r]);
      }
      mx = max_xor32(max_xor16(mx));
      if (fh == 0) s_m[wid * NH + 16 * t + fr] = mx;
    }
    lds_barrier();
#pragma unroll
    for (int t = 0; t < NHT; ++t) {
      float mn = m[t];
#pragma unroll
      for (int w = 0; w < 4; ++w) mn = fmaxf(mn, s_m[w * NH + 16 * t + fr]);
      const float mu = mn == -INFINITY ? 0.f : mn, alpha = __builtin_amdgcn_exp2f(m[t] - mu);
      m[t] = mn;
      float p[4], sum = 0.f;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        p[r] = __builtin_amdgcn_exp2f(s4[t][r] - mu);
        sum += p[r];
      }
      l[t] = l[t] * alpha + sum;
      const unsigned a0 = pk2bf(p[0], p[1]), a1 = pk2bf(p[2], p[3]);
      bf16_t* dst = s_p + (16 * t + fr) * P_STRIDE + 16 * wid + 4 * fh;
      *reinterpret_cast<uint2*>(dst) = make_uint2(a0, a1);
      *reinterpret_cast<uint2*>(dst + NH * P_STRIDE) =
          make_uint2(pk2bf(p[0] - __uint_as_float(a0 << 16), p[1] - __uint_as_float(a0 & 0xffff0000u)),
                     pk2bf(p[2] - __uint_as_float(a1 << 16), p[3] - __uint_as_float(a1 & 0xffff0000u)));
#pragma unroll
      for (int d = 0; d < DT; ++d) o[d][t] *= alpha;
    }
    lds_barrier();
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      bf16x8 pf[2][NHT];  // tokens 32 ks + 4 fh + 0..3 and 16 further, as load_vt orders them
#pragma unroll
      for (int t = 0; t < NHT; ++t)
#pragma unroll
        for (int x = 0; x < 2; ++x) {
          const bf16_t* src = s_p + (x * NH + 16 * t + fr) * P_STRIDE + 32 * ks + 4 * fh;
          const bf16x4 u = *reinterpret_cast<const bf16x4*>(src), v = *reinterpret_cast<const bf16x4*>(src + 16);
          pf[x][t] = (bf16x8){u[0], u[1], u[2], u[3], v[0], v[1], v[2], v[3]};
        }
      const int r0 = 32 * ks + 4 * fh + (fr >> 2), r1 = r0 + 16;
#pragma unroll
      for (int d = 0; d < DT; ++d) {
        const int chunk = 2 * (wid * DT + d) + ((fr >> 1) & 1);
        const bf16x4 u = tr_read(tile + r0 * ROWB + 16 * (chunk ^ cswz(r0)) + 8 * (fr & 1));
        const bf16x4 v = tr_read(tile + r1 * ROWB + 16 * (chunk ^ cswz(r1)) + 8 * (fr & 1));
        const bf16x8 vf = (bf16x8){u[0], u[1], u[2], u[3], v[0], v[1], v[2], v[3]};
#pragma unroll
        for (int t = 0; t < NHT; ++t) {
          o[d][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[0][t], o[d][t], 0, 0, 0);
          o[d][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[1][t], o[d][t], 0, 0, 0);
        }
      }
    }
    if (BUFS == 1 && it + 1 < it1) {
      lds_barrier();  // every wave has read the page
      stage(it + 1, 0);
    }
    wait_vmcnt0();
    lds_barrier();  // the next page has landed; the weights and maxima of this one are read
  }

#pragma unroll
  for (int t = 0; t < NHT; ++t) {
    l[t] += __shfl_xor(l[t], 16, 64);
    l[t] += __shfl_xor(l[t], 32, 64);
    if (fh == 0) s_m[wid * NH + 16 * t + fr] = l[t];
  }
  lds_barrier();
#pragma unroll
  for (int t = 0; t < NHT; ++t) {
    const int h = h0 + 16 * t + fr;
    if (h >= a.H) continue;
    const size_t pi = ((size_t)b * a.H + h) * a.max_parts + part;
    float* po = a.part_o + pi * Rp + wid * (16 * DT) + 4 * fh;
#pragma unroll
    for (int d = 0; d < DT; ++d) *reinterpret_cast<f32x4*>(po + 16 * d) = o[d][t];
    if (wid == 0 && fh == 0) {
      float L = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) L += s_m[w * NH + 16 * t + fr];
      a.part_ml[pi * 2] = m[t];
      a.part_ml[pi * 2 + 1] = L;
    }
  }
}

constexpr int MAX_PARTS = 64;

template <typename TP>
struct OutArgs {
  Proj<TP> P; int off_g;     // output gates, one per value element (off_g < 0: none)
  const float* part_o; const float* part_ml; const int* kv_lens;
  const bf16_t* wuv;         // [H][DV][Rp]
  bf16_t* out; int ldo;
  int B, H, DV, window, min_tiles, max_parts;
};

// grid: (H * ceil(DV / 64), batch / DB): joins the partitions of one head, 64 rows of its value map, gate
template <typename TP, int NR>
__global__ __launch_bounds__(256) void latent_out_kernel(OutArgs<TP> a) {
  constexpr int Rp = 128 * NR, KS = Rp / 32, ST = Rp + 8;
  __shared__ __attribute__((aligned(16))) bf16_t s_c[DB * ST];
  __shared__ float s_w[DB * MAX_PARTS];  // exp2(m_p - M) / L
  const int nd = (a.DV + 63) / 64, h = blockIdx.x / nd, d0 = (blockIdx.x % nd) * 64;
  const int b0 = blockIdx.y * DB, nb = min(DB, a.B - b0);
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, fr = lane & 15, fh = lane >> 4;
  const int dr = d0 + 16 * wid;  // this wave's 16 value rows
  const bool live = dr < a.DV;   // DV is a multiple of 16
  bf16x8 wf[KS];
  if (live) {
#pragma unroll
    for (int s = 0; s < KS; ++s)
      wf[s] = *reinterpret_cast<const bf16x8*>(a.wuv + ((size_t)h * a.DV + dr + fr) * Rp + 32 * s + 8 * fh);
  }
  // partition weights: 16 lanes per sequence
  {
    const int b = threadIdx.x >> 4, q = threadIdx.x & 15;
    int n = 0;
    if (b < nb) {
      const int pos = a.kv_lens[b0 + b] - 1, np = pos / KT + 1 - first_page(pos, a.window);
      const int pt = part_pages(np, a.min_tiles, a.max_parts);
      n = (np + pt - 1) / pt;
    }
    const float* ml = a.part_ml + ((size_t)(b0 + min(b, nb - 1)) * a.H + h) * a.max_parts * 2;
    float M = -INFINITY, L = 0.f;
    for (int p = q; p < n; p += 16) M = fmaxf(M, ml[2 * p]);
#pragma unroll
    for (int x = 1; x < 16; x <<= 1) M = fmaxf(M, __shfl_xor(M, x, 64));
    const float Mu = M == -INFINITY ? 0.f : M;
    for (int p = q; p < n; p += 16) L += ml[2 * p + 1] * __builtin_amdgcn_exp2f(ml[2 * p] - Mu);
#pragma unroll
    for (int x = 1; x < 16; x <<= 1) L += __shfl_xor(L, x, 64);
    const float inv = L > 0.f ? 1.f / L : 0.f;
    for (int p = q; p < MAX_PARTS; p += 16)
      s_w[b * MAX_PARTS + p] = p < n ? __builtin_amdgcn_exp2f(ml[2 * p] - Mu) * inv : 0.f;
  }
  __syncthreads();
  for (int i = threadIdx.x; i < DB * (Rp / 4); i += 256) {
    const int b = i / (Rp / 4), c = (i % (Rp / 4)) * 4;
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
    if (b < nb) {
      const float* po = a.part_o + ((size_t)(b0 + b) * a.H + h) * a.max_parts * Rp + c;
      const int pos = a.kv_lens[b0 + b] - 1, np = pos / KT + 1 - first_page(pos, a.window);
      const int pt = part_pages(np, a.min_tiles, a.max_parts), n = (np + pt - 1) / pt;
      for (int p = 0; p < n; p += 8) {
        f32x4 u[8];
#pragma unroll
        for (int k = 0; k < 8; ++k) u[k] = *reinterpret_cast<const f32x4*>(po + (size_t)min(p + k, n - 1) * Rp);
#pragma unroll
        for (int k = 0; k < 8; ++k)
          if (p + k < n) v += u[k] * s_w[b * MAX_PARTS + p + k];
      }
    }
    *reinterpret_cast<uint2*>(s_c + b * ST + c) = make_uint2(pk2bf(v[0], v[1]), pk2bf(v[2], v[3]));
  }
  __syncthreads();
  if (!live) return;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int s = 0; s < KS; ++s) {
    const bf16x8 cf = *reinterpret_cast<const bf16x8*>(s_c + fr * ST + 32 * s + 8 * fh);
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[s], cf, acc, 0, 0, 0);
  }
  if (fr >= nb) return;
  const int col = h * a.DV + dr + 4 * fh;
  if (a.off_g >= 0) {
    const TP* g = a.P.P + (size_t)(b0 + fr) * a.P.ld + a.off_g + col;
    f32x4 z = {0.f, 0.f, 0.f, 0.f};
    if constexpr (sizeof(TP) == 4) {
      for (int s = 0; s < a.P.S; ++s) z += *reinterpret_cast<const f32x4*>(g + (size_t)s * a.P.slab);
    } else {
      const bf16x4 zz = *reinterpret_cast<const bf16x4*>(g);
#pragma unroll
      for (int r = 0; r < 4; ++r) z[r] = bf2f_s(zz[r]);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) acc[r] *= __builtin_amdgcn_rcpf(1.f + __expf(-z[r]));
  }
  *reinterpret_cast<uint2*>(a.out + (size_t)(b0 + fr) * a.ldo + col) = make_uint2(pk2bf(acc[0], acc[1]), pk2bf(acc[2], acc[3]));
}

template <int NR, int NHT>
int launch_decode(const LatentArgs& a, hipStream_t st) {
  constexpr int NH = 16 * NHT;
  constexpr int lds = (NR <= 4 ? 2 : 1) * KT * 256 * NR + 2 * NH * P_STRIDE * 2 + 4 * NH * 4;
  (void)hipFuncSetAttribute((const void*)latent_decode_kernel<NR, NHT>, hipFuncAttributeMaxDynamicSharedMemorySize, lds);
  hipLaunchKernelGGL((latent_decode_kernel<NR, NHT>), dim3(a.max_parts, (a.H + NH - 1) / NH, a.B), dim3(256), lds, st, a);
  return (int)hipGetLastError();
}
template <int NR>
int launch_decode_nr(const LatentArgs& a, int heads, hipStream_t st) {
  if constexpr (NR <= 4)
    if (heads == 32) return launch_decode<NR, 2>(a, st);
  return heads == 16 ? launch_decode<NR, 1>(a, st) : (int)hipErrorInvalidValue;
}

template <typename TP>
int launch_absorb(const AbsorbArgs<TP>& a, int DK, hipStream_t st) {
  const dim3 grid(a.H * (a.Rp / 128) + (a.pages ? DB : 0), (a.B + DB - 1) / DB);
  if (DK == 32) hipLaunchKernelGGL((latent_absorb_kernel<TP, 32>), grid, dim3(256), 0, st, a);
  else if (DK == 64) hipLaunchKernelGGL((latent_absorb_kernel<TP, 64>), grid, dim3(256), 0, st, a);
  else if (DK == 128) hipLaunchKernelGGL((latent_absorb_kernel<TP, 128>), grid, dim3(256), 0, st, a);
  else if (DK == 256) hipLaunchKernelGGL((latent_absorb_kernel<TP, 256>), grid, dim3(256), 0, st, a);
  else return (int)hipErrorInvalidValue;
  return (int)hipGetLastError();
}
template <int NR, typename TP>
int launch_out(const OutArgs<TP>& a, hipStream_t st) {
  hipLaunchKernelGGL((latent_out_kernel<TP, NR>), dim3(a.H * ((a.DV + 63) / 64), (a.B + DB - 1) / DB), dim3(256), 0, st, a);
  return (int)hipGetLastError();
}

#define RAGK_LATENT_DISPATCH(RP, CALL)         \
  switch ((RP) / 128) {                        \
    case 1: { constexpr int NR = 1; return CALL; } \
    case 2: { constexpr int NR = 2; return CALL; } \
    case 3: { constexpr int NR = 3; return CALL; } \
    case 4: { constexpr int NR = 4; return CALL; } \
    case 5: { constexpr int NR = 5; return CALL; } \
    case 6: { constexpr int NR = 6; return CALL; } \
    case 7: { constexpr int NR = 7; return CALL; } \
    case 8: { constexpr int NR = 8; return CALL; } \
    default: return (int)hipErrorInvalidValue;  \
  }

bool rank_ok(int R, int Rp) { return Rp % 128 == 0 && Rp <= 1024 && R >= 1 && R <= Rp; }

}  // namespace

// row: [n][ld] (bf16, fp32 when f32); pages [blocks][64][Rp] and crows [n + pad][Rp] (or null) in the same type
RAGK_API int ragk_latent_store(const void* row, int ld, int off_c, int R, int Rp, const float* norm, float eps,
                               const int* slots, void* pages, void* crows, int n, int pad, int f32, hipStream_t st) {
  if (n <= 0) return 0;
  if (!rank_ok(R, Rp) || ld % 8 || off_c % 8 || off_c + Rp > ld || pad < 0) return (int)hipErrorInvalidValue;
  const dim3 grid(crows ? n + pad : n);
  if (f32)
    hipLaunchKernelGGL(latent_store_kernel<float>, grid, dim3(NORM_T), 0, st, (const float*)row, ld, off_c, R, Rp, norm, eps,
                       slots, (float*)pages, (float*)crows, n);
  else
    hipLaunchKernelGGL(latent_store_kernel<bf16_t>, grid, dim3(NORM_T), 0, st, (const bf16_t*)row, ld, off_c, R, Rp, norm,
                       eps, slots, (bf16_t*)pages, (bf16_t*)crows, n);
  return (int)hipGetLastError();
}

// out [n + pad][Rp]; cu_k [S + 1] packed row offsets, key_off[s] = cu_k[s] - first position kept of sequence s
RAGK_API int ragk_latent_gather(const void* pages, int Rp, const int* block_tables, int bt_stride, const int* cu_k,
                                const int* key_off, int S, int n, int pad, void* out, int f32, hipStream_t st) {
  if (n <= 0) return 0;
  if (!rank_ok(1, Rp) || S < 1 || pad < 0) return (int)hipErrorInvalidValue;
  if (f32)
    hipLaunchKernelGGL(latent_gather_kernel<float>, dim3(n + pad), dim3(NORM_T), 0, st, (const float*)pages, Rp, block_tables,
                       bt_stride, cu_k, key_off, S, n, (float*)out);
  else
    hipLaunchKernelGGL(latent_gather_kernel<bf16_t>, dim3(n + pad), dim3(NORM_T), 0, st, (const bf16_t*)pages, Rp,
                       block_tables, bt_stride, cu_k, key_off, S, n, (bf16_t*)out);
  return (int)hipGetLastError();
}

// x: [T][ldx], head h at h * K; w: [H][N][K]; gate [T][ldg] (head h at h * N) or null; y: [T][ldy], head h at h * N
RAGK_API int ragk_head_proj_f32(const float* x, int ldx, int K, const float* w, int N, const float* gate, int ldg, float* y,
                                int ldy, int T, int H, hipStream_t st) {
  if (T <= 0) return 0;
  if (K % 4 || K > 1024 || T > 65535) return (int)hipErrorInvalidValue;
  hipLaunchKernelGGL(head_proj_f32_kernel, dim3(H, T), dim3(256), 0, st, x, ldx, K, w, N, gate, ldg, y, ldy);
  return (int)hipGetLastError();
}

// P: fp32 slabs [S][B][ld], or bf16 rows [B][ld] (p_bf16, S = 1); queries of head h at column h * DK. qa [B][H][Rp].
// pages null: nothing is appended.
RAGK_API int ragk_latent_absorb(const void* P, int p_bf16, int S, int ld, int B, int H, int DK, int R, int Rp, int off_c,
                                const void* wuk, void* qa, void* pages, const int* slots, const float* norm, float eps,
                                hipStream_t st) {
  if (B <= 0) return 0;
  if (!rank_ok(R, Rp) || S < 1 || (p_bf16 && S != 1) || ld % 8 || H * DK > ld ||
      (pages && (!slots || !norm || off_c % 8 || off_c + Rp > ld)))
    return (int)hipErrorInvalidValue;
  if (p_bf16)
    return launch_absorb(AbsorbArgs<bf16_t>{{(const bf16_t*)P, 1, 0, ld}, B, H, Rp, R, off_c, (const bf16_t*)wuk,
                                            (bf16_t*)qa, (bf16_t*)pages, slots, norm, eps}, DK, st);
  return launch_absorb(AbsorbArgs<float>{{(const float*)P, S, (size_t)B * ld, ld}, B, H, Rp, R, off_c, (const bf16_t*)wuk,
                                         (bf16_t*)qa, (bf16_t*)pages, slots, norm, eps}, DK, st);
}

// heads: query heads per block, 16, or 32 for Rp <= 512
RAGK_API int ragk_latent_decode(const void* qa, const void* pages, const int* block_tables, int bt_stride, const int* kv_lens,
                                float* part_o, float* part_ml, int B, int H, int Rp, int window, int min_tiles,
                                int max_parts, int heads, float scale, hipStream_t st) {
  if (B <= 0) return 0;
  if (!rank_ok(1, Rp) || window < 0 || min_tiles < 1 || max_parts < 1 || max_parts > MAX_PARTS || B > 65535)
    return (int)hipErrorInvalidValue;
  const LatentArgs a{(const bf16_t*)qa, (const bf16_t*)pages, block_tables, bt_stride, kv_lens, part_o, part_ml, B, H,
                     window, min_tiles, max_parts, scale};
  RAGK_LATENT_DISPATCH(Rp, (launch_decode_nr<NR>(a, heads, st)));
}

// joins what latent_decode left, applies the value map and the output gate; out [B][ldo], head h at h * DV
RAGK_API int ragk_latent_out(const void* P, int p_bf16, int S, int ld, int off_g, const float* part_o, const float* part_ml,
                             const int* kv_lens, const void* wuv, void* out, int ldo, int B, int H, int DV, int Rp,
                             int window, int min_tiles, int max_parts, hipStream_t st) {
  if (B <= 0) return 0;
  if (!rank_ok(1, Rp) || S < 1 || (p_bf16 && S != 1) || DV % 16 || ldo % 4 || ld % 4 || off_g % 4 || max_parts < 1 ||
      max_parts > MAX_PARTS || min_tiles < 1)
    return (int)hipErrorInvalidValue;
  if (p_bf16) {
    const OutArgs<bf16_t> a{{(const bf16_t*)P, 1, 0, ld}, off_g, part_o, part_ml, kv_lens, (const bf16_t*)wuv,
                            (bf16_t*)out, ldo, B, H, DV, window, min_tiles, max_parts};
    RAGK_LATENT_DISPATCH(Rp, (launch_out<NR>(a, st)));
  }
  const OutArgs<float> a{{(const float*)P, S, (size_t)B * ld, ld}, off_g, part_o, part_ml, kv_lens, (const bf16_t*)wuv,
                         (bf16_t*)out, ldo, B, H, DV, window, min_tiles, max_parts};
  RAGK_LATENT_DISPATCH(Rp, (launch_out<NR>(a, st)));
}
