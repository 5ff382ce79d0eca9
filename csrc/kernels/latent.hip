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
  float* part_ml;      // [B][H][max_parts][2]: reference of the exponentials (log2 units) and sum
  int B, H, window, min_tiles, max_parts;
  float scale;
};
// A tile is TT tokens of a page; BUFS of them are in LDS, BUFS - 1 of them in flight while one is computed.
template <int NR>
struct LatentTile {
  static constexpr int TT = NR <= 2 ? 64 : 32;
  static constexpr int BYTES = TT * 256 * NR;
  static constexpr int BUFS = NR <= 4 ? 4 : NR == 5 ? 3 : 2;
  static constexpr int PIECES = BYTES / 1024 / 4;  // 1-KiB pieces per wave
};
// A query visits tiles first .. first + n - 1, `per` of them in each partition.
struct Split {
  int first, n, per;
  __device__ __forceinline__ Split(int pos, int window, int tt, int min_tiles, int max_parts) {
    first = window > 0 ? max(0, pos - window + 1) / tt : 0;
    n = pos / tt + 1 - first;
    per = max(min_tiles, (n + max_parts - 1) / max_parts);
  }
  __device__ __forceinline__ int parts() const { return (n + per - 1) / per; }
};
// the latent tile serves row reads (keys) and transposed reads (values): 32-B granules kept, 8 rows on distinct banks
__device__ __forceinline__ int cswz(int row) { return 2 * (row & 7); }
__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
  __builtin_amdgcn_sched_barrier(0);
}
template <int N>
__device__ __forceinline__ void wait_vmcnt() {
  static_assert(N < 64, "vmcnt has six bits");
  asm volatile("s_waitcnt vmcnt(%0)" ::"n"(N) : "memory");
}

// grid: (max_parts, groups of 16 NHT heads, batch). The 4 waves share every tile: each scores a part of its tokens and
// heads, the scores meet in LDS, and each accumulates a quarter of the latent columns for all heads, with the whole
// softmax in its own registers. Queries and latents come by LDS-DMA alone and the page list is read once, so no load
// of the loop makes the compiler drain the DMA queue.
template <int NR, int NHT>
__global__ __launch_bounds__(256, 1) void latent_decode_kernel(LatentArgs a) {
  using C = LatentTile<NR>;
  constexpr int Rp = 128 * NR, ROWB = 2 * Rp, NC = Rp / 8, TT = C::TT, BUFS = C::BUFS, PIECES = C::PIECES;
  constexpr int KS = Rp / 32, DT = Rp / 64, NH = 16 * NHT;  // k-steps of a score; 16-column tiles per wave; heads
  constexpr int QT = TT == 64 ? NHT : 1;                    // head tiles that one wave scores
  constexpr int SS = TT + 4;                                // floats per head of the scores in LDS
  static_assert(NH <= TT, "the queries pass through one tile buffer");
  extern __shared__ __attribute__((aligned(16))) char smem[];
  float* s_s = reinterpret_cast<float*>(smem + BUFS * C::BYTES);  // [NH][SS]
  int* s_bt = reinterpret_cast<int*>(s_s + NH * SS);              // this partition's page list
  const int lane = threadIdx.x & 63, wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int fr = lane & 15, fh = lane >> 4;
  const int part = blockIdx.x, h0 = blockIdx.y * NH, b = blockIdx.z;
  const int pos = a.kv_lens[b] - 1;
  const Split sp(pos, a.window, TT, a.min_tiles, a.max_parts);
  if (part * sp.per >= sp.n) return;  // block-uniform, before any barrier
  const int it0 = sp.first + part * sp.per, it1 = sp.first + min((part + 1) * sp.per, sp.n);
  const int pg0 = it0 * TT / KT, npg = ((it1 - 1) * TT) / KT + 1 - pg0;
  const int* bt = a.block_tables + (size_t)b * a.bt_stride + pg0;
  for (int i = threadIdx.x; i < npg; i += 256) s_bt[i] = bt[i];

  const unsigned lds0 = lds_addr(smem);
  int off[PIECES];
#pragma unroll
  for (int i = 0; i < PIECES; ++i) {
    const int idx = (wid + 4 * i) * 64 + lane, row = idx / NC, ph = idx % NC;
    off[i] = row * ROWB + 16 * (ph ^ cswz(row));
  }
  auto stage = [&](int it) {
    const int pg = __builtin_amdgcn_readfirstlane(s_bt[it * TT / KT - pg0]), buf = (it - it0) % BUFS;
    const i32x4 srd = make_srd(a.pages + ((size_t)pg * KT + it * TT % KT) * Rp, C::BYTES);
#pragma unroll
    for (int i = 0; i < PIECES; ++i) blds16_asm(srd, off[i], 0, lds0 + buf * C::BYTES + (wid + 4 * i) * 1024);
  };
  __syncthreads();  // page list
  {                 // queries into the buffer that the first tiles leave free (heads past the last repeat it)
    const int last = min(NH, a.H - h0) - 1;
    const i32x4 srd = make_srd(a.qa + ((size_t)b * a.H + h0) * Rp, (last + 1) * ROWB);
#pragma unroll
    for (int i = 0; i < NH * NR / 16; ++i) {
      const int idx = (wid + 4 * i) * 64 + lane, row = idx / NC, ph = idx % NC;
      blds16_asm(srd, min(row, last) * ROWB + 16 * (ph ^ cswz(row)), 0, lds0 + (BUFS - 1) * C::BYTES + (wid + 4 * i) * 1024);
    }
  }
#pragma unroll
  for (int k = 0; k < BUFS - 1; ++k)
    if (it0 + k < it1) stage(it0 + k);
  if (it1 - it0 >= BUFS - 1) wait_vmcnt<(BUFS - 1) * PIECES>();
  else wait_vmcnt0();
  lds_barrier();
  const int tg = TT == 64 ? wid : wid & 1, ht = TT == 64 ? 0 : wid >> 1;  // the tokens and heads this wave scores
  const bool scores = ht < NHT;
  bf16x8 qf[QT][KS];
  if (scores) {
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      const int row = 16 * (ht + t) + fr;
#pragma unroll
      for (int s = 0; s < KS; ++s)
        qf[t][s] = *reinterpret_cast<const bf16x8*>(smem + (BUFS - 1) * C::BYTES + row * ROWB + 16 * ((4 * s + fh) ^ cswz(row)));
    }
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

  for (int it = it0; it < it1; ++it) {
    const int k0 = it * TT;
    const char* tile = smem + ((it - it0) % BUFS) * C::BYTES;
    if (it1 - it > BUFS - 2) wait_vmcnt<(BUFS - 2) * PIECES>();
    else wait_vmcnt0();
    lds_barrier();  // the tile has landed for all waves; the buffer of the one before it and the scores are free
    if (it + BUFS - 1 < it1) stage(it + BUFS - 1);
    if (scores) {
      f32x4 s4[QT][2];
#pragma unroll
      for (int t = 0; t < QT; ++t) s4[t][0] = s4[t][1] = (f32x4){0.f, 0.f, 0.f, 0.f};
      const int row = 16 * tg + fr;
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const bf16x8 kf = *reinterpret_cast<const bf16x8*>(tile + row * ROWB + 16 * ((4 * s + fh) ^ cswz(row)));
#pragma unroll
        for (int t = 0; t < QT; ++t) s4[t][s & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[t][s], s4[t][s & 1], 0, 0, 0);
      }
      const int d0 = pos - k0 - 16 * tg - 4 * fh;  // distance of this lane's first token
      const bool edge = pos < k0 + TT - 1 || pos - k0 >= win;
#pragma unroll
      for (int t = 0; t < QT; ++t) {
        f32x4 x = (s4[t][0] + s4[t][1]) * c;
        if (edge) {
#pragma unroll
          for (int r = 0; r < 4; ++r) x[r] = d0 - r >= 0 && d0 - r < win ? x[r] : -INFINITY;
        }
        *reinterpret_cast<f32x4*>(s_s + (16 * (ht + t) + fr) * SS + 16 * tg + 4 * fh) = x;
      }
    }
    lds_barrier();
    bf16x8 hi[TT / 32][NHT], lo[TT / 32][NHT];  // tokens 32 ks + 4 fh + 0..3 and 16 further, as the value fragments order them
    float alpha[NHT];
#pragma unroll
    for (int t = 0; t < NHT; ++t) {
      f32x4 x[TT / 16];
      float mx = -INFINITY;
#pragma unroll
      for (int g = 0; g < TT / 16; ++g) {
        x[g] = *reinterpret_cast<const f32x4*>(s_s + (16 * t + fr) * SS + 16 * g + 4 * fh);
        mx = fmaxf(fmaxf(mx, fmaxf(x[g][0], x[g][1])), fmaxf(x[g][2], x[g][3]));
      }
      mx = max_xor32(max_xor16(mx));
      alpha[t] = 1.f;
      if (mx > m[t] + RESCALE_LOG2) {
        alpha[t] = m[t] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m[t] - mx);
        m[t] = mx;
      }
      const float mu = m[t] == -INFINITY ? 0.f : m[t];
      float sum = 0.f;
#pragma unroll
      for (int g = 0; g < TT / 16; ++g)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          x[g][r] = __builtin_amdgcn_exp2f(x[g][r] - mu);
          sum += x[g][r];
        }
      l[t] = l[t] * alpha[t] + sum;
#pragma unroll
      for (int ks = 0; ks < TT / 32; ++ks) split_p(x[2 * ks], x[2 * ks + 1], hi[ks][t], lo[ks][t]);
    }
    bool moved = false;
#pragma unroll
    for (int t = 0; t < NHT; ++t) moved |= alpha[t] != 1.f;
    if (__builtin_amdgcn_ballot_w64(moved)) {
#pragma unroll
      for (int d = 0; d < DT; ++d)
#pragma unroll
        for (int t = 0; t < NHT; ++t) o[d][t] *= alpha[t];
    }
#pragma unroll
    for (int ks = 0; ks < TT / 32; ++ks) {
      const int r0 = 32 * ks + 4 * fh + (fr >> 2), r1 = r0 + 16;
#pragma unroll
      for (int d = 0; d < DT; ++d) {
        const int chunk = 2 * (wid * DT + d) + ((fr >> 1) & 1);
        const bf16x4 u = tr_read(tile + r0 * ROWB + 16 * (chunk ^ cswz(r0)) + 8 * (fr & 1));
        const bf16x4 v = tr_read(tile + r1 * ROWB + 16 * (chunk ^ cswz(r1)) + 8 * (fr & 1));
        const bf16x8 vf = (bf16x8){u[0], u[1], u[2], u[3], v[0], v[1], v[2], v[3]};
#pragma unroll
        for (int t = 0; t < NHT; ++t) o[d][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, hi[ks][t], o[d][t], 0, 0, 0);
#pragma unroll
        for (int t = 0; t < NHT; ++t) o[d][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, lo[ks][t], o[d][t], 0, 0, 0);
      }
    }
  }

#pragma unroll
  for (int t = 0; t < NHT; ++t) {
    l[t] += __shfl_xor(l[t], 16, 64);
    l[t] += __shfl_xor(l[t], 32, 64);
    const int h = h0 + 16 * t + fr;
    if (h >= a.H) continue;
    const size_t pi = ((size_t)b * a.H + h) * a.max_parts + part;
    float* po = a.part_o + pi * Rp + wid * (16 * DT) + 4 * fh;
#pragma unroll
    for (int d = 0; d < DT; ++d) *reinterpret_cast<f32x4*>(po + 16 * d) = o[d][t];
    if (wid == 0 && fh == 0) {
      a.part_ml[pi * 2] = m[t];
      a.part_ml[pi * 2 + 1] = l[t];
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

// grid: (H * ceil(DV / 64), batch / NB): joins the partitions of one head for NB sequences, 64 rows of its value map, gate
template <typename TP, int NR, int NB>
__global__ __launch_bounds__(256) void latent_out_kernel(OutArgs<TP> a) {
  constexpr int Rp = 128 * NR, KS = Rp / 32, ST = Rp + 8, TT = LatentTile<NR>::TT;
  constexpr int U = NB <= 4 ? 16 : 8;  // partitions requested at a time
  __shared__ __attribute__((aligned(16))) bf16_t s_c[NB * ST];
  __shared__ float s_w[NB * MAX_PARTS];  // exp2(m_p - M) / L
  __shared__ int s_n[NB];                // partitions
  const int nd = (a.DV + 63) / 64, h = blockIdx.x / nd, d0 = (blockIdx.x % nd) * 64;
  const int b0 = blockIdx.y * NB, nb = min(NB, a.B - b0);
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, fr = lane & 15, fh = lane >> 4;
  const int dr = d0 + 16 * wid;  // this wave's 16 value rows
  const bool live = dr < a.DV;   // DV is a multiple of 16
  const int col = h * a.DV + dr + 4 * fh;
  bf16x8 wf[KS];
  f32x4 z = {0.f, 0.f, 0.f, 0.f};
  if (live) {  // requested before the join
#pragma unroll
    for (int s = 0; s < KS; ++s)
      wf[s] = *reinterpret_cast<const bf16x8*>(a.wuv + ((size_t)h * a.DV + dr + fr) * Rp + 32 * s + 8 * fh);
    if (a.off_g >= 0) {
      const TP* g = a.P.P + (size_t)(b0 + min(fr, nb - 1)) * a.P.ld + a.off_g + col;
      if constexpr (sizeof(TP) == 4) {
        for (int s0 = 0; s0 < a.P.S; s0 += PSU) {
          f32x4 u[PSU];
#pragma unroll
          for (int k = 0; k < PSU; ++k) u[k] = *reinterpret_cast<const f32x4*>(g + (size_t)min(s0 + k, a.P.S - 1) * a.P.slab);
#pragma unroll
          for (int k = 0; k < PSU; ++k)
            if (s0 + k < a.P.S) z += u[k];
        }
      } else {
        const bf16x4 zz = *reinterpret_cast<const bf16x4*>(g);
#pragma unroll
        for (int r = 0; r < 4; ++r) z[r] = bf2f_s(zz[r]);
      }
    }
  }
  // partition weights: 16 lanes per sequence
  if (threadIdx.x < 16 * NB) {
    const int b = threadIdx.x >> 4, q = threadIdx.x & 15;
    int n = 0;
    if (b < nb) n = Split(a.kv_lens[b0 + b] - 1, a.window, TT, a.min_tiles, a.max_parts).parts();
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
    if (q == 0) s_n[b] = n;
  }
  __syncthreads();
  for (int i = threadIdx.x; i < NB * (Rp / 4); i += 256) {
    const int b = i / (Rp / 4), c = (i % (Rp / 4)) * 4, n = s_n[b];
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
    const float* po = a.part_o + ((size_t)(b0 + min(b, nb - 1)) * a.H + h) * a.max_parts * Rp + c;
    for (int p = 0; p < n; p += U) {
      f32x4 u[U];
#pragma unroll
      for (int k = 0; k < U; ++k) u[k] = *reinterpret_cast<const f32x4*>(po + (size_t)min(p + k, n - 1) * Rp);
#pragma unroll
      for (int k = 0; k < U; ++k)
        if (p + k < n) v += u[k] * s_w[b * MAX_PARTS + p + k];
    }
    *reinterpret_cast<uint2*>(s_c + b * ST + c) = make_uint2(pk2bf(v[0], v[1]), pk2bf(v[2], v[3]));
  }
  __syncthreads();
  if (!live) return;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int s = 0; s < KS; ++s) {  // matrix columns past NB repeat and are dropped
    const bf16x8 cf = *reinterpret_cast<const bf16x8*>(s_c + fr % NB * ST + 32 * s + 8 * fh);
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[s], cf, acc, 0, 0, 0);
  }
  if (fr >= nb) return;
  if (a.off_g >= 0) {
#pragma unroll
    for (int r = 0; r < 4; ++r) acc[r] *= __builtin_amdgcn_rcpf(1.f + __expf(-z[r]));
  }
  *reinterpret_cast<uint2*>(a.out + (size_t)(b0 + fr) * a.ldo + col) = make_uint2(pk2bf(acc[0], acc[1]), pk2bf(acc[2], acc[3]));
}

template <int NR, int NHT>
int launch_decode(const LatentArgs& a, hipStream_t st) {
  using C = LatentTile<NR>;
  constexpr int NH = 16 * NHT, lds = C::BUFS * C::BYTES + NH * (C::TT + 4) * 4 + MAX_BT * 4;
  static_assert(lds <= 160 * 1024, "LDS of a CU");
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
  const int gx = a.H * ((a.DV + 63) / 64);  // fewer sequences a block where that is what fills the chip
  if (gx * ((a.B + 15) / 16) >= 256) hipLaunchKernelGGL((latent_out_kernel<TP, NR, 16>), dim3(gx, (a.B + 15) / 16), dim3(256), 0, st, a);
  else if (gx * ((a.B + 7) / 8) >= 256) hipLaunchKernelGGL((latent_out_kernel<TP, NR, 8>), dim3(gx, (a.B + 7) / 8), dim3(256), 0, st, a);
  else hipLaunchKernelGGL((latent_out_kernel<TP, NR, 4>), dim3(gx, (a.B + 3) / 4), dim3(256), 0, st, a);
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
  if (!rank_ok(1, Rp) || window < 0 || min_tiles < 1 || max_parts < 1 || max_parts > MAX_PARTS || B > 65535 || bt_stride > MAX_BT)
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
