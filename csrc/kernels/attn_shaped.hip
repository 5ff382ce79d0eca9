// Attention with shaped scores over the paged cache (K pages [blocks][G][64][DK], V pages [blocks][G][64][DV]),
// or over packed key / value rows of the step (row_attn_*: keys of a sequence in consecutive rows):
//
//   s_ij = softcap * tanh(q_i . k_j * scale / softcap) + table[h][min(i - j, far)]
//   j visible to i:  j <= i  and  (window == 0 or i - j < window or j < keep)
//   out_i = gate_ih * sum_j exp(s_ij) v_j / (sink + sum_j exp(s_ij)),  sink in {0, 1}
//   gate_ih: none, one sigmoid per head, or one per head and value element
//
// Positions are the tokens' own in the sequence, so the kept first tokens enter with their true distances.
// Scores, softmax and the bias are fp32.
//
//  * kv_store     : k, and v mixed with the first mixing layer's values of the same token, into the pages.
//  * attn_rows    : one wave per (token, query head), plain fp32 arithmetic. Any head size; the fp32 path.
//  * attn_prefill : MFMA flash attention over 64-key pages, 4 waves = GB query heads of one KV head x (4 / GB)
//                   groups of 32 query rows. Only pages with a visible key are visited: the pages of the kept first
//                   tokens, then those of the window. The bias table row of each head sits in LDS.
//  * attn_decode  : one query per sequence. Takes the projection as fp32 split-K slabs, so the slab sum, the bias
//                   add, the value mix and the cache append need no launch of their own; the pages of a
//                   sequence are split over partitions (attn_merge joins them) when batch x KV heads is small.
//
// The MFMA kernels keep the softmax weights at 16 significant bits for P.V (bf16 high + low part, two products).
#include "attn_tiles.h"
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
  int gate_vec;                // 1: a gate per head and value element, 0: one per head
  int window, keep, far, sink;
  float scale, softcap;
  // keys: entry e of a sequence's page list starts at kc + e * k_unit + kv head * k_head, rows k_row apart. Paged:
  // e = block table entry; packed rows: e = key_off[seq] + first position of the page.
  const int* key_off;          // [S] row of position 0 of each sequence (may be negative), null: paged
  long long k_unit, v_unit;
  int k_head, k_row, v_head, v_row;
  __device__ __forceinline__ int entry(const int* bt, int seq, int page) const {
    return key_off ? key_off[seq] + page * 64 : bt[page];
  }
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

// NC: value columns per lane, sizes up to 64 NC
template <typename T, int NC>
__global__ __launch_bounds__(64) void attn_rows_kernel(ShapedArgs a) {
  __shared__ float sq[64 * NC], sp[64];
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
  float acc[NC];
#pragma unroll
  for (int c = 0; c < NC; ++c) acc[c] = 0.f;
  for (int it = 0; it < n_it; ++it) {
    const int pg = it < keep_pages ? it : first_win + it - keep_pages;
    const int e0 = a.entry(bt, s, pg), j = pg * 64 + lane;
    const T* kr = (const T*)a.kc + e0 * a.k_unit + (size_t)g * a.k_head + (size_t)lane * a.k_row;
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
    const T* vb = (const T*)a.vc + e0 * a.v_unit + (size_t)g * a.v_head;
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const int d = lane + 64 * c;
      if (d < a.DV) {
        acc[c] *= alpha;
        const int nj = min(64, i + 1 - pg * 64);
        for (int k = 0; k < nj; ++k) acc[c] = fmaf(sp[k], ld1(vb + (size_t)k * a.v_row + d), acc[c]);
      }
    }
  }
  const float inv = l > 0.f ? 1.f / l : 0.f;
  float gate = 1.f;
  if (a.off_g >= 0 && !a.gate_vec) gate = 1.f / (1.f + expf(-ld1(qr + a.off_g + h)));
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int d = lane + 64 * c;
    if (d < a.DV && a.off_g >= 0 && a.gate_vec) gate = 1.f / (1.f + expf(-ld1(qr + a.off_g + h * a.DV + d)));
    if (d < a.DV) st1((T*)a.out + (size_t)t * a.ldo + h * a.DV + d, acc[c] * inv * gate);
  }
}

// ---- visited pages of a query range [qmin, qmax]: the kept first pages, then the window's ----
struct Pages {
  int n_keep, first, n;  // iteration it -> page it < n_keep ? it : first + it - n_keep
  __device__ __forceinline__ int page(int it) const { return it < n_keep ? it : first + it - n_keep; }
};
__device__ __forceinline__ Pages visited(int qmin, int qmax, int window, int keep) {
  const int n_pages = qmax / KT + 1;
  if (window <= 0) return Pages{n_pages, n_pages, n_pages};
  const int nk = min(n_pages, (keep + KT - 1) / KT);
  const int f = max(nk, max(0, qmin - window + 1) / KT);
  return Pages{nk, f, nk + max(0, n_pages - f)};
}

// softcapped score in log2 units: cap2 * tanh(x / cap) = cap2 - 2 cap2 / (1 + 2^(x * c1)); c1 = 2 scale log2e / cap
struct Shape {
  float c1, cap2, c;  // cap2 > 0: soft-capped; else s = x * c
  __device__ __forceinline__ float sigma(float x) const {  // 1 / (1 + 2^(x * c1))
    return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(x * c1));
  }
};
// tanh(y) / y as a polynomial in y^2, |error of tanh| < 1.4e-7 for |y| <= TANH_R (least-maximum fit): cheaper than the
// exponential and the reciprocal, which on this ALU take four issue slots each
constexpr float TANH_R = 0.5f;
constexpr float TANH_C[4] = {0.999997676f, -0.333206551f, 0.131451449f, -0.0433724665f};

constexpr float LOG2E = 1.4426950408889634f;
__device__ __forceinline__ Shape make_shape(float scale, float softcap) {
  return Shape{softcap > 0.f ? 2.f * scale * LOG2E / softcap : 0.f, softcap > 0.f ? softcap * LOG2E : 0.f, scale * LOG2E};
}

struct ShapedPrefill {
  ShapedArgs a;
  const int* tiles; int n_hg, gb;  // work list (seq, first query); head groups; heads per block
  int sb_stride;                   // floats per head of the LDS bias table, 0: none
};

// PLAIN: no soft cap, bias, kept first tokens or zero score, and a positive scale: the maxima run over the raw products.
// BOUNDED: every score is known to stay within a range whose exponentials fp32 holds (soft cap + largest bias), so
// the sums need no running maximum: the weights are 2^s, and the extra zero score adds exactly 1.
enum PrefillMode { GENERAL, BOUNDED, PLAIN };
template <int DK, int DV, PrefillMode MODE>
__global__ __launch_bounds__(256, (DK <= 128 && DV <= 128) ? 2 : 1) void attn_shaped_prefill_kernel(ShapedPrefill pa) {
  using CK = Cfg<DK>;
  using CV = Cfg<DV>;
  const ShapedArgs& a = pa.a;
  extern __shared__ __attribute__((aligned(16))) char smem[];  // [buf][K | V], page list, bias tables
  int* s_bt = reinterpret_cast<int*>(smem + 2 * (CK::TILEB + CV::TILEB));
  float* s_bias = reinterpret_cast<float*>(s_bt + MAX_BT);

  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int wid_u = __builtin_amdgcn_readfirstlane(wid);
  const int tix = (int)blockIdx.x / pa.n_hg, hg = (int)blockIdx.x - tix * pa.n_hg;
  const int seq = pa.tiles[2 * tix], q_start = pa.tiles[2 * tix + 1];
  const int G = a.H / a.G, gb = pa.gb, per_kv = G / gb;
  const int kvh = hg / per_kv, h0 = kvh * G + (hg % per_kv) * gb, hb = wid_u % gb, hq = h0 + hb;
  const int pbase = q_start + (wid_u / gb) * 32;
  const int q_off = a.cu_q[seq], q_len = a.cu_q[seq + 1] - q_off, kv_len = a.kv_lens[seq];
  const int ctx0 = kv_len - q_len;
  const int qt_rows = 32 * (4 / gb);
  const int keep = MODE == PLAIN ? 0 : a.keep, sink = MODE == PLAIN ? 0 : a.sink;
  const Pages pg = visited(ctx0 + q_start, ctx0 + min(q_start + qt_rows, q_len) - 1, a.window, keep);
  const int wave_pmin = ctx0 + pbase, wave_pmax = ctx0 + min(pbase + 31, q_len - 1);
  const int fr = lane & 15, fh = lane >> 4;

  bf16x8 qf[2][CK::KS];
#pragma unroll
  for (int qt = 0; qt < 2; ++qt) {
    const int qi = min(pbase + 16 * qt + fr, q_len - 1);
    const bf16_t* qp = (const bf16_t*)a.q + (size_t)(q_off + qi) * a.ldq + hq * DK + 8 * fh;
#pragma unroll
    for (int s = 0; s < CK::KS; ++s) qf[qt][s] = *reinterpret_cast<const bf16x8*>(qp + 32 * s);
  }
  f32x4 o[CV::DT][2];
#pragma unroll
  for (int dt = 0; dt < CV::DT; ++dt)
#pragma unroll
    for (int qt = 0; qt < 2; ++qt) o[dt][qt] = (f32x4){0.f, 0.f, 0.f, 0.f};
  // the extra zero score: running max 0, one unit in the sum (one of a query's four lanes holds it)
  float m_i[2], l_i[2];
#pragma unroll
  for (int qt = 0; qt < 2; ++qt) {
    m_i[qt] = sink ? 0.f : -INFINITY;
    l_i[qt] = sink && fh == 0 ? 1.f : 0.f;
  }
  const int* bt = a.block_tables + (size_t)seq * a.bt_stride;
  for (int i = threadIdx.x; i < pg.n; i += 256) s_bt[i] = a.entry(bt, seq, pg.page(i));
  if (MODE != PLAIN && a.table && pa.sb_stride)
    for (int h = 0; h < gb; ++h)
      for (int i = threadIdx.x; i <= a.far; i += 256)
        s_bias[h * pa.sb_stride + i] = a.table[(size_t)(h0 + h) * (a.far + 1) + i] * LOG2E;
  __syncthreads();
  const float* tb = MODE != PLAIN && a.table ? a.table + (size_t)hq * (a.far + 1) : nullptr;
  const float* s_tb = s_bias + hb * pa.sb_stride;  // the same row in LDS, in log2 units
  const float far_bias = tb ? tb[a.far] * LOG2E : 0.f;
  const Shape shape = make_shape(a.scale, a.softcap);
  const bool capped = MODE != PLAIN && shape.cap2 > 0.f;
  const int win = a.window > 0 ? a.window : 0x7fffffff;
  // the polynomial in the raw product x: s = x (q0 + x^2 (q1 + ...)), good while |x| <= x_lim
  const float yx = capped ? a.scale / a.softcap : 0.f, yx2 = yx * yx, x_lim = capped ? TANH_R / yx : 0.f;
  const float q0 = shape.cap2 * yx * TANH_C[0], q1 = shape.cap2 * yx * yx2 * TANH_C[1];
  const float q2 = shape.cap2 * yx * yx2 * yx2 * TANH_C[2], q3 = shape.cap2 * yx * yx2 * yx2 * yx2 * TANH_C[3];

  // a page's rows by LDS-DMA, each wave a quarter of the 1-KiB pieces; per-lane source offsets are fixed
  constexpr int KP = CK::PIECES / 4, VP = CV::PIECES / 4;
  int koff[KP], voff[VP];
#pragma unroll
  for (int i = 0; i < KP; ++i) {
    const int row = (wid_u + 4 * i) * CK::RPP + lane / CK::NC, ph = lane % CK::NC;
    koff[i] = row * a.k_row * 2 + 16 * (ph ^ kswz<DK>(row));
  }
#pragma unroll
  for (int i = 0; i < VP; ++i) {
    const int row = (wid_u + 4 * i) * CV::RPP + lane / CV::NC, ph = lane % CV::NC;
    voff[i] = row * a.v_row * 2 + 16 * (ph ^ vswz<DV>(row));
  }
  const unsigned lds0 = lds_addr(smem);
  auto stage = [&](int entry, int buf) {
    const int e0 = __builtin_amdgcn_readfirstlane(entry);
    const i32x4 srd_k = make_srd((const bf16_t*)a.kc + e0 * a.k_unit + kvh * a.k_head, (63 * a.k_row + DK) * 2);
    const i32x4 srd_v = make_srd((const bf16_t*)a.vc + e0 * a.v_unit + kvh * a.v_head, (63 * a.v_row + DV) * 2);
    const unsigned l = lds0 + buf * (CK::TILEB + CV::TILEB);
#pragma unroll
    for (int i = 0; i < KP; ++i) blds16_asm(srd_k, koff[i], 0, l + (wid_u + 4 * i) * 1024);
#pragma unroll
    for (int i = 0; i < VP; ++i) blds16_asm(srd_v, voff[i], 0, l + CK::TILEB + (wid_u + 4 * i) * 1024);
  };
  stage(s_bt[0], 0);  // pg.n >= 1: a query always sees its own page
  wait_vmcnt0();
  __syncthreads();

  for (int it = 0; it < pg.n; ++it) {
    const int cur = it & 1, k0 = pg.page(it) * KT;
    const char* sK = smem + cur * (CK::TILEB + CV::TILEB);
    const char* sV = sK + CK::TILEB;
    const bool active = k0 <= wave_pmax && (wave_pmin - (k0 + KT - 1) < win || k0 < keep);
    const int next = s_bt[min(it + 1, pg.n - 1)];
    f32x4 s[4][2];
    if (active) {
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        s[t][0] = (f32x4){0.f, 0.f, 0.f, 0.f};
        s[t][1] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < CK::KS; ++ks) {
          const bf16x8 kf = load_k<DK>(sK, t, ks, lane);
          s[t][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[0][ks], s[t][0], 0, 0, 0);
          s[t][1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[1][ks], s[t][1], 0, 0, 0);
        }
      }
    }
    if (it + 1 < pg.n) stage(next, cur ^ 1);  // DMA of the next page behind the QK^T products
    if (active) {
      const bool all_visible = k0 + KT - 1 <= wave_pmin && (wave_pmax - k0 < win || k0 + KT <= keep);
      const bool far_only = !tb || wave_pmin - (k0 + KT - 1) >= a.far;  // one bias for the whole page
      // scores in log2 units, with the page-wide bias; wave-uniform branches around whole pages of elements
      const float base = far_only ? far_bias : 0.f;
#pragma unroll
      for (int qt = 0; qt < 2; ++qt) {
        if (capped) {
          float ax = 0.f;
#pragma unroll
          for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) ax = fmaxf(ax, fabsf(s[t][qt][r]));
          if (!__builtin_amdgcn_ballot_w64(!(ax <= x_lim))) {
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
              for (int r = 0; r < 4; ++r) {
                const float x = s[t][qt][r], z = x * x;
                const float q = __builtin_fmaf(z, __builtin_fmaf(z, __builtin_fmaf(z, q3, q2), q1), q0);
                s[t][qt][r] = __builtin_fmaf(x, q, base);
              }
          } else {
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
              for (int r = 0; r < 4; ++r)
                s[t][qt][r] = __builtin_fmaf(-2.f * shape.cap2, shape.sigma(s[t][qt][r]), base + shape.cap2);
          }
        } else if constexpr (MODE != PLAIN) {
#pragma unroll
          for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) s[t][qt][r] = __builtin_fmaf(s[t][qt][r], shape.c, base);
        }
      }
      if (!far_only) {
        if (pa.sb_stride) {
#pragma unroll
          for (int qt = 0; qt < 2; ++qt) {
            const int d0 = ctx0 + pbase + 16 * qt + fr - k0 - 4 * fh;  // distance of this lane's key 0
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
              for (int r = 0; r < 4; ++r) s[t][qt][r] += s_tb[max(0, min(d0 - 16 * t - r, a.far))];
          }
        } else {
#pragma unroll
          for (int qt = 0; qt < 2; ++qt) {
            const int d0 = ctx0 + pbase + 16 * qt + fr - k0 - 4 * fh;
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
              for (int r = 0; r < 4; ++r)
                s[t][qt][r] = __builtin_fmaf(tb[max(0, min(d0 - 16 * t - r, a.far))], LOG2E, s[t][qt][r]);
          }
        }
      }
      if (!all_visible) {
#pragma unroll
        for (int qt = 0; qt < 2; ++qt) {
          const int qpos = ctx0 + pbase + 16 * qt + fr, d0 = qpos - k0 - 4 * fh;
#pragma unroll
          for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              const int d = d0 - 16 * t - r;
              const bool ok = (d >= 0) & ((d < win) | (qpos - d < keep));
              s[t][qt][r] = ok ? s[t][qt][r] : -INFINITY;
            }
        }
      }
      if constexpr (MODE == BOUNDED) {
#pragma unroll
        for (int qt = 0; qt < 2; ++qt)
#pragma unroll
          for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              const float p = __builtin_amdgcn_exp2f(s[t][qt][r]);
              s[t][qt][r] = p;
              l_i[qt] += p;
            }
      } else {
        float alpha[2];
#pragma unroll
        for (int qt = 0; qt < 2; ++qt) {
          float mx = -INFINITY;
#pragma unroll
          for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) mx = fmaxf(mx, s[t][qt][r]);
          mx = max_xor32(max_xor16(mx));
          if constexpr (MODE == PLAIN) mx *= shape.c;
          alpha[qt] = 1.f;
          if (mx > m_i[qt] + RESCALE_LOG2) {
            alpha[qt] = m_i[qt] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m_i[qt] - mx);
            m_i[qt] = mx;
          }
          const float mref = m_i[qt] == -INFINITY ? 0.f : m_i[qt];
          float ls = 0.f;
#pragma unroll
          for (int t = 0; t < 4; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              const float p = __builtin_amdgcn_exp2f(__builtin_fmaf(s[t][qt][r], MODE == PLAIN ? shape.c : 1.f, -mref));
              s[t][qt][r] = p;
              ls += p;
            }
          l_i[qt] = l_i[qt] * alpha[qt] + ls;
        }
        if (__builtin_amdgcn_ballot_w64(alpha[0] != 1.f || alpha[1] != 1.f)) {
#pragma unroll
          for (int dt = 0; dt < CV::DT; ++dt)
#pragma unroll
            for (int qt = 0; qt < 2; ++qt) o[dt][qt] *= alpha[qt];
        }
      }
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        bf16x8 hi[2], lo[2];
#pragma unroll
        for (int qt = 0; qt < 2; ++qt) split_p(s[2 * ks][qt], s[2 * ks + 1][qt], hi[qt], lo[qt]);
#pragma unroll
        for (int dt = 0; dt < CV::DT; ++dt) {
          const bf16x8 vf = load_vt<DV>(sV, dt, ks, lane);
#pragma unroll
          for (int qt = 0; qt < 2; ++qt) o[dt][qt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, hi[qt], o[dt][qt], 0, 0, 0);
#pragma unroll
          for (int qt = 0; qt < 2; ++qt) o[dt][qt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, lo[qt], o[dt][qt], 0, 0, 0);
        }
      }
    }
    wait_vmcnt0();
    __syncthreads();
  }

#pragma unroll
  for (int qt = 0; qt < 2; ++qt) {
    float l = l_i[qt];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    float inv = l > 0.f ? 1.f / l : 0.f;
    const int qi = pbase + 16 * qt + fr;
    if (qi < q_len) {
      const bf16_t* gp = nullptr;
      if (a.off_g >= 0 && a.gate_vec) {
        gp = (const bf16_t*)a.q + (size_t)(q_off + qi) * a.ldq + a.off_g + hq * DV + 4 * fh;
      } else if (a.off_g >= 0) {
        const float g = bf2f(((const bf16_t*)a.q)[(size_t)(q_off + qi) * a.ldq + a.off_g + hq]);
        inv *= __builtin_amdgcn_rcpf(1.f + __expf(-g));
      }
      bf16_t* op = (bf16_t*)a.out + (size_t)(q_off + qi) * a.ldo + hq * DV + 4 * fh;
#pragma unroll
      for (int dt = 0; dt < CV::DT; ++dt) {
        f32x4 v = o[dt][qt] * inv;
        if (gp) {
          const bf16x4 g = *reinterpret_cast<const bf16x4*>(gp + 16 * dt);
#pragma unroll
          for (int r = 0; r < 4; ++r) v[r] *= __builtin_amdgcn_rcpf(1.f + __expf(-bf2f_s(g[r])));
        }
        *reinterpret_cast<uint2*>(op + 16 * dt) = make_uint2(pk2bf(v[0], v[1]), pk2bf(v[2], v[3]));
      }
    }
  }
}

// ---- decode ----
struct ShapedDecode {
  const float* P; int S; int ldp; size_t slab;  // projection slabs [S][B][ldp]
  const bf16_t* bias;                            // [ldp] or null
  bf16_t* kc; bf16_t* vc;
  const int* block_tables; int bt_stride;
  const int* kv_lens; const int* slots;
  const float* table;
  const float* v_first; const float* lam;        // [B][G * DV] values to mix in, or null
  float* v_own;                                  // [B][G * DV] own values out, or null
  bf16_t* out; int ldo;
  float* part_o; float* part_ml;                 // [B][H][max_parts][DV], [B][H][max_parts][2]
  int B, H, G, off_k, off_v, off_g;
  int window, keep, far, sink, min_tiles, max_parts;
  float scale, softcap;
};

__device__ __forceinline__ void slab_row8(const ShapedDecode& a, int b, int col, float* f) {
  sum_slabs8(a.P + (size_t)b * a.ldp + col, a.S, a.slab, f);
  if (a.bias) {
    float w[8];
    ld8(a.bias + col, w);
#pragma unroll
    for (int e = 0; e < 8; ++e) f[e] += w[e];
  }
}
__device__ __forceinline__ float slab_gate(const ShapedDecode& a, int b, int h) {
  if (a.off_g < 0) return 1.f;
  float g = a.bias ? bf2f(a.bias[a.off_g + h]) : 0.f;
  for (int s = 0; s < a.S; ++s) g += a.P[s * a.slab + (size_t)b * a.ldp + a.off_g + h];
  return __builtin_amdgcn_rcpf(1.f + __expf(-g));
}
// pages per partition: the visited pages spread over all partitions, at least min_tiles each
__device__ __forceinline__ int part_pages(int n, const ShapedDecode& a) {
  return max(a.min_tiles, (n + a.max_parts - 1) / a.max_parts);
}

constexpr int DEC_HEADS = 16;  // query heads per decode block (one MFMA column each)

// grid: (max_parts, KV heads x groups of 16 query heads, batch), 4 waves; a wave takes every 4th page
template <int DK, int DV>
__global__ __launch_bounds__(256, (DK <= 128 && DV <= 128) ? 2 : 1) void attn_shaped_decode_kernel(ShapedDecode a) {
  using CK = Cfg<DK>;
  using CV = Cfg<DV>;
  __shared__ __attribute__((aligned(16))) char smem[4 * CV::TILEB + DEC_HEADS * DK * 2 + 4 * (16 + 64) * 4];
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int wid_u = __builtin_amdgcn_readfirstlane(wid);
  const int part = blockIdx.x, b = blockIdx.z;
  const int Gq = a.H / a.G, chunks = (Gq + DEC_HEADS - 1) / DEC_HEADS;
  const int kvh = blockIdx.y / chunks, hc = blockIdx.y % chunks;
  const int h0 = kvh * Gq + hc * DEC_HEADS, nh = min(DEC_HEADS, Gq - hc * DEC_HEADS);
  const int pos = a.kv_lens[b] - 1;
  const Pages pg = visited(pos, pos, a.window, a.keep);
  const int pt = part_pages(pg.n, a);
  const int it0 = part * pt;
  if (it0 >= pg.n) return;  // block-uniform, before any barrier
  const int it1 = min(it0 + pt, pg.n), nparts = (pg.n + pt - 1) / pt;
  const int fr = lane & 15, fh = lane >> 4;
  const int* bt = a.block_tables + (size_t)b * a.bt_stride;
  char* sV = smem + wid_u * CV::TILEB;
  bf16_t* s_q = reinterpret_cast<bf16_t*>(smem + 4 * CV::TILEB);

  // the wave's first page is requested before the prologue (not the page that the new token goes into)
  const bool pre = it0 + wid_u < it1 && it0 + wid_u != pg.n - 1;
  bf16x8 kf[4][CK::KS];
  auto request = [&](int it) {
    const size_t pgi = (size_t)bt[pg.page(it)] * a.G + kvh;
    const bf16_t* kb = a.kc + pgi * KT * DK;
    const bf16_t* vb = a.vc + pgi * KT * DV;
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int s = 0; s < CK::KS; ++s)
        kf[t][s] = *reinterpret_cast<const bf16x8*>(kb + (size_t)(16 * t + fr) * DK + 32 * s + 8 * fh);
    __builtin_amdgcn_sched_barrier(0);  // K before V: the scores and the softmax run while V is landing
    stage_kv<DV, true, false, 1>(sV, 0, 1, lane, [&](int r) { return vb + (size_t)r * DV; });
  };
  if (pre) request(it0 + wid_u);

  constexpr int QV = DK / 8, VV = DV / 8;
  const bool append = it1 == pg.n;
  const int n_q = nh * QV, n_all = n_q + (append ? QV + VV : 0);
  for (int i = threadIdx.x; i < n_all; i += 256) {
    float f[8];
    if (i < n_q) {
      slab_row8(a, b, h0 * DK + i * 8, f);
      st8(s_q + i * 8, f);
    } else {
      const int slot = a.slots[b];
      const size_t row = ((size_t)(slot >> 6) * a.G + kvh) * KT + (slot & 63);
      const int j = i - n_q;
      if (j < QV) {
        slab_row8(a, b, a.off_k + kvh * DK + j * 8, f);
        st8(a.kc + row * DK + j * 8, f);
      } else {
        const int c = (j - QV) * 8;
        slab_row8(a, b, a.off_v + kvh * DV + c, f);
        const size_t vo = ((size_t)b * a.G + kvh) * DV + c;
        if (a.v_own) st8(a.v_own + vo, f);
        if (a.v_first) {
          const float lm = a.lam[0];
          float w[8];
          ld8(a.v_first + vo, w);
#pragma unroll
          for (int e = 0; e < 8; ++e) f[e] = (1.f - lm) * f[e] + lm * w[e];
        }
        st8(a.vc + row * DV + c, f);
      }
    }
  }
  __syncthreads();  // q in LDS; the appended row visible to the whole block
  bf16x8 qf[CK::KS];
#pragma unroll
  for (int s = 0; s < CK::KS; ++s)
    qf[s] = fr < nh ? *reinterpret_cast<const bf16x8*>(s_q + fr * DK + 32 * s + 8 * fh) : (bf16x8){0, 0, 0, 0, 0, 0, 0, 0};

  const Shape shape = make_shape(a.scale, a.softcap);
  const float* tb = a.table ? a.table + (size_t)(h0 + min(fr, nh - 1)) * (a.far + 1) : nullptr;
  const float far_bias = tb ? tb[a.far] * LOG2E : 0.f;
  const bool capped = shape.cap2 > 0.f;
  const int win = a.window > 0 ? a.window : 0x7fffffff;
  f32x4 o[CV::DT];
#pragma unroll
  for (int dt = 0; dt < CV::DT; ++dt) o[dt] = (f32x4){0.f, 0.f, 0.f, 0.f};
  float m_i = -INFINITY, l_i = 0.f;
  for (int it = it0 + wid_u; it < it1; it += 4) {
    if (!(pre && it == it0 + wid_u)) {
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // the previous page's V reads have retired
      request(it);
    }
    const int k0 = pg.page(it) * KT;
    f32x4 s4[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      s4[t] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < CK::KS; ++s) s4[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[t][s], qf[s], s4[t], 0, 0, 0);
    }
    const int d0 = pos - k0 - 4 * fh;  // distance of this lane's key 0
    const bool far_only = !tb || pos - (k0 + KT - 1) >= a.far;
    const float base = (capped ? shape.cap2 : 0.f) + (far_only ? far_bias : 0.f);
    if (capped) {
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) s4[t][r] = __builtin_fmaf(-2.f * shape.cap2, shape.sigma(s4[t][r]), base);
    } else {
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) s4[t][r] = __builtin_fmaf(s4[t][r], shape.c, base);
    }
    if (!far_only) {
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          s4[t][r] = __builtin_fmaf(tb[max(0, min(d0 - 16 * t - r, a.far))], LOG2E, s4[t][r]);
    }
    if (!(k0 + KT - 1 <= pos && (pos - k0 < win || k0 + KT <= a.keep))) {
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int d = d0 - 16 * t - r;
          const bool ok = (d >= 0) & ((d < win) | (pos - d < a.keep));
          s4[t][r] = ok ? s4[t][r] : -INFINITY;
        }
    }
    float mx = -INFINITY;
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) mx = fmaxf(mx, s4[t][r]);
    mx = max_xor32(max_xor16(mx));
    const float m_new = fmaxf(m_i, mx), m_use = m_new == -INFINITY ? 0.f : m_new;
    const float alpha = __builtin_amdgcn_exp2f(m_i - m_use);
    float ls = 0.f;
#pragma unroll
    for (int t = 0; t < 4; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float p = __builtin_amdgcn_exp2f(s4[t][r] - m_use);
        s4[t][r] = p;
        ls += p;
      }
    l_i = l_i * alpha + ls;
    m_i = m_new;
#pragma unroll
    for (int dt = 0; dt < CV::DT; ++dt) o[dt] *= alpha;
    bf16x8 hi[2], lo[2];
    split_p(s4[0], s4[1], hi[0], lo[0]);
    split_p(s4[2], s4[3], hi[1], lo[1]);
    wait_vmcnt0();  // the V page is in this wave's LDS
#pragma unroll
    for (int dt = 0; dt < CV::DT; ++dt)
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        const bf16x8 vf = load_vt<DV>(sV, dt, ks, lane);
        o[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, hi[ks], o[dt], 0, 0, 0);
        o[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, lo[ks], o[dt], 0, 0, 0);
      }
  }

  // combine the 4 waves: O [4][16][DV] reuses the V pages, statistics sit behind the q rows
  __syncthreads();
  float* so = reinterpret_cast<float*>(smem);
  float* sm = reinterpret_cast<float*>(smem + 4 * CV::TILEB + DEC_HEADS * DK * 2);
  float* sl = sm + 64;
  if (fh == 0) sm[wid * 16 + fr] = m_i;
  sl[wid * 64 + lane] = l_i;
#pragma unroll
  for (int dt = 0; dt < CV::DT; ++dt)
#pragma unroll
    for (int r = 0; r < 4; ++r) so[(wid * 16 + fr) * DV + 16 * dt + 4 * fh + r] = o[dt][r];
  __syncthreads();
  for (int e = threadIdx.x; e < nh * DV; e += 256) {
    const int g = e / DV, d = e % DV, h = h0 + g;
    float M = nparts == 1 && a.sink ? 0.f : -INFINITY;
#pragma unroll
    for (int w = 0; w < 4; ++w) M = fmaxf(M, sm[w * 16 + g]);
    const float Mu = M == -INFINITY ? 0.f : M;
    float L = nparts == 1 && a.sink ? __builtin_amdgcn_exp2f(-Mu) : 0.f, O = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float sc = __builtin_amdgcn_exp2f(sm[w * 16 + g] - Mu);
      L += (sl[w * 64 + g] + sl[w * 64 + g + 16] + sl[w * 64 + g + 32] + sl[w * 64 + g + 48]) * sc;
      O += so[(w * 16 + g) * DV + d] * sc;
    }
    if (nparts == 1) {
      a.out[(size_t)b * a.ldo + h * DV + d] = f2bf(L > 0.f ? O / L * slab_gate(a, b, h) : 0.f);
    } else {
      const size_t pi = ((size_t)b * a.H + h) * a.max_parts + part;
      a.part_o[pi * DV + d] = O;
      if (d == 0) {
        a.part_ml[pi * 2] = M;
        a.part_ml[pi * 2 + 1] = L;
      }
    }
  }
}

// join the partitions of one (head, sequence), add the extra zero score, apply the gate; DV threads
__global__ void attn_shaped_merge_kernel(ShapedDecode a, int DV) {
  const int h = blockIdx.x, b = blockIdx.y, d = threadIdx.x;
  const int pos = a.kv_lens[b] - 1;
  const int n = visited(pos, pos, a.window, a.keep).n, pt = part_pages(n, a), nparts = (n + pt - 1) / pt;
  if (nparts == 1) return;  // written by the decode kernel
  const size_t p0 = ((size_t)b * a.H + h) * a.max_parts;
  float M = a.sink ? 0.f : -INFINITY;
  for (int p = 0; p < nparts; ++p) M = fmaxf(M, a.part_ml[(p0 + p) * 2]);
  const float Mu = M == -INFINITY ? 0.f : M;
  float L = a.sink ? __builtin_amdgcn_exp2f(-Mu) : 0.f, O = 0.f;
  int p = 0;
  for (; p + 4 <= nparts; p += 4) {
    float v[4], m[4], l[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      v[i] = a.part_o[(p0 + p + i) * DV + d];
      m[i] = a.part_ml[(p0 + p + i) * 2];
      l[i] = a.part_ml[(p0 + p + i) * 2 + 1];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float sc = __builtin_amdgcn_exp2f(m[i] - Mu);
      L += l[i] * sc;
      O += v[i] * sc;
    }
  }
  for (; p < nparts; ++p) {
    const float sc = __builtin_amdgcn_exp2f(a.part_ml[(p0 + p) * 2] - Mu);
    L += a.part_ml[(p0 + p) * 2 + 1] * sc;
    O += a.part_o[(p0 + p) * DV + d] * sc;
  }
  a.out[(size_t)b * a.ldo + h * DV + d] = f2bf(L > 0.f ? O / L * slab_gate(a, b, h) : 0.f);
}

template <int DK, int DV, PrefillMode MODE>
int launch_prefill_mode(const ShapedPrefill& pa, int n_tiles, int lds, hipStream_t st) {
  (void)hipFuncSetAttribute((const void*)attn_shaped_prefill_kernel<DK, DV, MODE>, hipFuncAttributeMaxDynamicSharedMemorySize,
                            lds);
  hipLaunchKernelGGL((attn_shaped_prefill_kernel<DK, DV, MODE>), dim3(n_tiles * pa.n_hg), dim3(256), lds, st, pa);
  return (int)hipGetLastError();
}
template <int DK, int DV>
int launch_prefill(ShapedPrefill pa, int n_tiles, int bounded, hipStream_t st) {
  constexpr int base = 2 * (Cfg<DK>::TILEB + Cfg<DV>::TILEB) + MAX_BT * 4;
  constexpr int room = ((DK <= 128 && DV <= 128) ? 80 * 1024 : 160 * 1024) - base;
  const ShapedArgs& a = pa.a;
  int extra = a.table ? pa.gb * (a.far + 1) * 4 : 0;
  if (extra > room) extra = 0;  // a very long table is read through the caches
  pa.sb_stride = extra ? a.far + 1 : 0;
  const int lds = base + (extra + 15) / 16 * 16;
  if (bounded) return launch_prefill_mode<DK, DV, BOUNDED>(pa, n_tiles, lds, st);
  if (!a.table && !a.keep && !a.sink && !(a.softcap > 0.f) && a.scale > 0.f)
    return launch_prefill_mode<DK, DV, PLAIN>(pa, n_tiles, lds, st);
  return launch_prefill_mode<DK, DV, GENERAL>(pa, n_tiles, lds, st);
}

template <int DK, int DV>
int launch_decode(const ShapedDecode& a, hipStream_t st) {
  const int chunks = (a.H / a.G + DEC_HEADS - 1) / DEC_HEADS;
  hipLaunchKernelGGL((attn_shaped_decode_kernel<DK, DV>), dim3(a.max_parts, a.G * chunks, a.B), dim3(256), 0, st, a);
  if (a.max_parts > 1)
    hipLaunchKernelGGL(attn_shaped_merge_kernel, dim3(a.H, a.B), dim3(DV), 0, st, a, DV);
  return (int)hipGetLastError();
}

#define RAGK_SHAPED_DISPATCH(FN, ...)                                  \
  do {                                                                 \
    if (DK == 32 && DV == 32) return FN<32, 32>(__VA_ARGS__);          \
    if (DK == 32 && DV == 64) return FN<32, 64>(__VA_ARGS__);          \
    if (DK == 32 && DV == 128) return FN<32, 128>(__VA_ARGS__);        \
    if (DK == 32 && DV == 256) return FN<32, 256>(__VA_ARGS__);        \
    if (DK == 64 && DV == 32) return FN<64, 32>(__VA_ARGS__);          \
    if (DK == 64 && DV == 64) return FN<64, 64>(__VA_ARGS__);          \
    if (DK == 64 && DV == 128) return FN<64, 128>(__VA_ARGS__);        \
    if (DK == 64 && DV == 256) return FN<64, 256>(__VA_ARGS__);        \
    if (DK == 128 && DV == 32) return FN<128, 32>(__VA_ARGS__);        \
    if (DK == 128 && DV == 64) return FN<128, 64>(__VA_ARGS__);        \
    if (DK == 128 && DV == 128) return FN<128, 128>(__VA_ARGS__);      \
    if (DK == 128 && DV == 256) return FN<128, 256>(__VA_ARGS__);      \
    if (DK == 256 && DV == 32) return FN<256, 32>(__VA_ARGS__);        \
    if (DK == 256 && DV == 64) return FN<256, 64>(__VA_ARGS__);        \
    if (DK == 256 && DV == 128) return FN<256, 128>(__VA_ARGS__);      \
    if (DK == 256 && DV == 256) return FN<256, 256>(__VA_ARGS__);      \
    return (int)hipErrorInvalidValue;                                  \
  } while (0)

}  // namespace

namespace {
ShapedArgs paged_args(const void* q, int ldq, const void* kc, const void* vc, const int* bt, int bt_stride, const int* cu_q,
                      const int* kv_lens, const float* table, void* out, int ldo, int T, int S, int H, int G, int DK,
                      int DV, int off_g, int window, int keep, int far, int sink, float scale, float softcap) {
  return ShapedArgs{q, ldq, kc, vc, bt, bt_stride, cu_q, kv_lens, table, out, ldo, T, S, H, G, DK, DV, off_g, 0, window,
                    keep, far, sink, scale, softcap, nullptr, (long long)G * 64 * DK, (long long)G * 64 * DV, 64 * DK, DK,
                    64 * DV, DV};
}
// packed rows [keys][ldk]: keys at column h * DK, values at off_v + h * DV; one gate per value element
ShapedArgs rows_args(const void* q, int ldq, const void* kv, int ldk, int off_v, size_t elem, const int* key_off,
                     const int* cu_q, const int* kv_lens, void* out, int ldo, int T, int S, int H, int DK, int DV, int off_g,
                     int window, float scale) {
  return ShapedArgs{q, ldq, kv, (const char*)kv + off_v * elem, nullptr, 0, cu_q, kv_lens, nullptr, out, ldo, T, S, H, H, DK,
                    DV, off_g, 1, window, 0, 0, 0, scale, 0.f, key_off, ldk, ldk, DK, ldk, DV, ldk};
}
template <typename T>
void launch_rows(const ShapedArgs& a, hipStream_t st) {
  if (a.DK <= 256 && a.DV <= 256) hipLaunchKernelGGL((attn_rows_kernel<T, 4>), dim3(a.T, a.H), dim3(64), 0, st, a);
  else hipLaunchKernelGGL((attn_rows_kernel<T, 16>), dim3(a.T, a.H), dim3(64), 0, st, a);
}
int dispatch_prefill(int DK, int DV, const ShapedPrefill& pa, int n_tiles, int bounded, hipStream_t st) {
  RAGK_SHAPED_DISPATCH(launch_prefill, pa, n_tiles, bounded, st);
}
}  // namespace

// bf16. tiles: [n_tiles][2] (sequence, first query) of 128 / gb query rows each; gb in {1, 2, 4} divides H / G.
// bounded: the caller knows that (softcap + largest |bias|) * log2e < 80 (every 2^score and the sum over any context fit).
RAGK_API int ragk_shaped_attn_prefill(const void* q, int ldq, const void* kc, const void* vc, const int* block_tables,
                                      int bt_stride, const int* cu_q, const int* kv_lens, const int* tiles, int n_tiles,
                                      int gb, const float* table, void* out, int ldo, int H, int G, int DK, int DV,
                                      int off_g, int window, int keep, int far, int sink, int bounded, float scale,
                                      float softcap, hipStream_t st) {
  if (n_tiles <= 0) return 0;
  if (H % G || (gb != 1 && gb != 2 && gb != 4) || (H / G) % gb || bt_stride > MAX_BT || ldq % 8 || ldo % 4 || !cu_q ||
      window < 0 || keep < 0 || far < 0 || (bounded && !(softcap > 0.f)))
    return (int)hipErrorInvalidValue;
  const ShapedArgs a = paged_args(q, ldq, kc, vc, block_tables, bt_stride, cu_q, kv_lens, table, out, ldo, 0, 0, H, G, DK,
                                  DV, off_g, window, keep, far, sink, scale, softcap);
  const ShapedPrefill pa{a, tiles, H / gb, gb, 0};
  return dispatch_prefill(DK, DV, pa, n_tiles, bounded, st);
}

// The same kernel over packed key / value rows kv [rows][ldk] (bf16): H heads of their own, position p of sequence s in
// row key_off[s] + p. Whole 64-row groups are read: every group that starts at a key must lie inside the rows.
RAGK_API int ragk_row_attn_prefill(const void* q, int ldq, const void* kv, int ldk, int off_v, const int* key_off,
                                   const int* cu_q, const int* kv_lens, const int* tiles, int n_tiles, void* out, int ldo,
                                   int H, int DK, int DV, int off_g, int window, int max_pages, float scale,
                                   hipStream_t st) {
  if (n_tiles <= 0) return 0;
  if (max_pages > MAX_BT || ldq % 8 || ldk % 8 || off_v % 8 || ldo % 4 || off_g % 4 || !cu_q || !key_off || window < 0 ||
      H < 1 || off_v < H * DK || off_v + H * DV > ldk)
    return (int)hipErrorInvalidValue;
  const ShapedPrefill pa{rows_args(q, ldq, kv, ldk, off_v, 2, key_off, cu_q, kv_lens, out, ldo, 0, 0, H, DK, DV, off_g,
                                   window, scale),
                         tiles, H, 1, 0};
  return dispatch_prefill(DK, DV, pa, n_tiles, 0, st);
}

// plain fp32 arithmetic over the same packed rows (fp32 when f32, else bf16); any head size up to 256
RAGK_API int ragk_row_attn_rows(const void* q, int ldq, const void* kv, int ldk, int off_v, const int* key_off,
                                const int* cu_q, const int* kv_lens, void* out, int ldo, int T, int S, int H, int DK,
                                int DV, int off_g, int window, float scale, int f32, hipStream_t st) {
  if (T <= 0) return 0;
  if (DK % 8 || DK > 256 || DV > 256 || H > 65535 || ldk % 8 || off_v % 8 || !cu_q || !key_off)
    return (int)hipErrorInvalidValue;
  const ShapedArgs a = rows_args(q, ldq, kv, ldk, off_v, f32 ? 4 : 2, key_off, cu_q, kv_lens, out, ldo, T, S, H, DK, DV,
                                 off_g, window, scale);
  if (f32) launch_rows<float>(a, st);
  else launch_rows<bf16_t>(a, st);
  return (int)hipGetLastError();
}

// bf16 caches, fp32 slabs P [S][B][ldp] (+ bias). The new token's k / v go to `slots`; out [B][ldo].
RAGK_API int ragk_shaped_attn_decode(const float* P, int S, int ldp, const void* bias, void* kc, void* vc,
                                     const int* block_tables, int bt_stride, const int* kv_lens, const int* slots,
                                     const float* table, const float* v_first, const float* lam, float* v_own, void* out,
                                     int ldo, float* part_o, float* part_ml, int B, int H, int G, int DK, int DV,
                                     int off_k, int off_v, int off_g, int window, int keep, int far, int sink,
                                     int min_tiles, int max_parts, float scale, float softcap, hipStream_t st) {
  if (B <= 0) return 0;
  if (S < 1 || H % G || ldp % 8 || off_k % 8 || off_v % 8 || min_tiles < 1 || max_parts < 1 || (v_first && !lam) ||
      (max_parts > 1 && (!part_o || !part_ml)) || B > 65535 || window < 0 || keep < 0 || far < 0)
    return (int)hipErrorInvalidValue;
  const ShapedDecode a{P, S, ldp, (size_t)B * ldp, (const bf16_t*)bias, (bf16_t*)kc, (bf16_t*)vc, block_tables, bt_stride,
                       kv_lens, slots, table, v_first, lam, v_own, (bf16_t*)out, ldo, part_o, part_ml, B, H, G, off_k,
                       off_v, off_g, window, keep, far, sink, min_tiles, max_parts, scale, softcap};
  RAGK_SHAPED_DISPATCH(launch_decode, a, st);
}

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
  if (DK % 8 || DK > 1024 || DV > 1024 || H % G || H > 65535) return (int)hipErrorInvalidValue;
  const ShapedArgs a = paged_args(q, ldq, kc, vc, block_tables, bt_stride, cu_q, kv_lens, table, out, ldo, T, S, H, G, DK,
                                  DV, off_g, window, keep, far, sink, scale, softcap);
  if (f32) launch_rows<float>(a, st);
  else launch_rows<bf16_t>(a, st);
  return (int)hipGetLastError();
}
