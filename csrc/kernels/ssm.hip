// Selective state-space layer (Mamba-2 form: one scalar decay per head, B and C shared by a group of heads).
//
// Projection row: [z: H*P | x: H*P | B: G*N | C: G*N | dt: H]. Per sequence, one state slot holds
//   conv_state [taps - 1][H*P + 2*G*N] fp32 : the last inputs of the short convolution, oldest first
//   ssm_state  [H][N][P] fp32
// A sequence whose first new token is its position 0 starts from zero state, whatever its slot held.
//
//   xbc   = silu(conv(x | B | C) + b)                              causal, per channel
//   dt    = softplus(dt + dt_bias),  decay = exp(-A dt)            A = exp(A_log), formed at load
//   S_t   = decay S_(t-1) + dt B_t x_t^T,  y_t = S_t^T C_t + D x_t
//   out   = group_norm(y * silu(z)) * w
//
// Everything that enters the recurrence besides xbc is fp32.
//
//  * conv_silu / conv_tail : the convolution over packed prompts, then the new conv_state.
//  * scan_seq              : the recurrence token by token, one block per (head, sequence). Any size; the fp32 path.
//  * scan_chunk            : the recurrence in 64-token chunks on MFMA (bf16 prompts). One block per (head, sequence,
//                            32 / 64 state columns) walks a sequence's chunks; inside a chunk, with c_t the running sum
//                            of log-decays,  y_t = sum_(s<=t) e^(c_t - c_s) dt_s (C_t.B_s) x_s + e^(c_t) S^T C_t  and
//                            S <- e^(c_end) S + sum_s B_s (e^(c_end - c_s) dt_s x_s)^T. The fp32 operands (the weighted
//                            C.B products, the weighted x, the state) enter the products as bf16 high + low parts.
//  * gate_norm             : the gate and the grouped norm, one block per (token, norm group); gate_norm_wave is its
//                            vectorised form, one wave per (token, group).
//  * dec_act / dec_state   : one new token per sequence from the projection's fp32 split-K slabs: convolution (and
//                            its state), activations, softplus; then the state update, read once and written once.
#include "attn_tiles.h"
#include "seq_common.h"
using namespace ragk;

namespace {

constexpr int CONV_TT = 16;  // tokens per conv block
constexpr int MAX_TAPS = 8;

struct SeqArgs {
  const int* cu_q;     // [S + 1]; null: one token per sequence
  const int* kv_lens;  // [S]
  const int* states;   // [S]
  int T, S;
};

__device__ __forceinline__ void seq_span(const SeqArgs& q, int s, int& t0, int& n, bool& fresh) {
  t0 = q.cu_q ? q.cu_q[s] : s;
  n = q.cu_q ? q.cu_q[s + 1] - t0 : 1;
  fresh = q.kv_lens[s] == n;
}

// out[t][c] = silu(b[c] + sum_k w[k][c] u[t - (taps - 1) + k][c]); one thread per channel, CONV_TT tokens
template <typename T>
__global__ __launch_bounds__(256) void conv_silu_kernel(SeqArgs q, const T* __restrict__ row, int ld, int off,
                                                        const float* __restrict__ w, const float* __restrict__ b,
                                                        const float* __restrict__ conv_state, T* out, int ch, int taps) {
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= ch) return;
  int t = blockIdx.x * CONV_TT;
  const int t_end = min(t + CONV_TT, q.T);
  int s = q.cu_q ? seq_of(q.cu_q, q.S, t) : t;
  float wk[MAX_TAPS];
#pragma unroll
  for (int k = 0; k < MAX_TAPS; ++k) wk[k] = k < taps ? w[(size_t)k * ch + c] : 0.f;
  const float bias = b[c];
  while (t < t_end) {
    int t0, n;
    bool fresh;
    seq_span(q, s, t0, n, fresh);
    const float* cs = conv_state + (size_t)q.states[s] * (taps - 1) * ch + c;
    float hist[MAX_TAPS];  // hist[k]: input at (t - (taps - 1) + k)
    auto input = [&](int local) -> float {
      if (local >= 0) return ld1(row + (size_t)(t0 + local) * ld + off + c);
      return fresh ? 0.f : cs[(size_t)(taps - 1 + local) * ch];
    };
#pragma unroll
    for (int k = 0; k < MAX_TAPS; ++k)
      if (k < taps - 1) hist[k] = input(t - t0 - (taps - 1) + k);
    const int stop = min(t_end, t0 + n);
    for (; t < stop; ++t) {
      const float u = ld1(row + (size_t)t * ld + off + c);
      float y = bias;
#pragma unroll
      for (int k = 0; k < MAX_TAPS; ++k)
        if (k < taps) y = fmaf(wk[k], k == taps - 1 ? u : hist[k], y);
      st1(out + (size_t)t * ch + c, silu_exact(y));
#pragma unroll
      for (int k = 0; k + 1 < MAX_TAPS; ++k)
        if (k < taps - 1) hist[k] = k == taps - 2 ? u : hist[k + 1];
    }
    ++s;
  }
}

// conv_silu on 16-B vectors: 8 channels per thread (bf16, ch % 8 == 0)
template <int TAPS>
__global__ __launch_bounds__(256) void conv_silu_vec_kernel(SeqArgs q, const bf16_t* __restrict__ row, int ld, int off,
                                                            const float* __restrict__ w, const float* __restrict__ b,
                                                            const float* __restrict__ conv_state, bf16_t* out, int ch) {
  const int c = (blockIdx.y * 256 + threadIdx.x) * 8;
  if (c >= ch) return;
  int t = blockIdx.x * CONV_TT;
  const int t_end = min(t + CONV_TT, q.T);
  int s = q.cu_q ? seq_of(q.cu_q, q.S, t) : t;
  float wk[TAPS][8], bias[8];
#pragma unroll
  for (int k = 0; k < TAPS; ++k) ld8(w + (size_t)k * ch + c, wk[k]);
  ld8(b + c, bias);
  while (t < t_end) {
    int t0, n;
    bool fresh;
    seq_span(q, s, t0, n, fresh);
    const float* cs = conv_state + (size_t)q.states[s] * (TAPS - 1) * ch + c;
    float hist[TAPS][8];  // rotating window of the last inputs, oldest first
#pragma unroll
    for (int k = 0; k < TAPS - 1; ++k) {
      const int local = t - t0 - (TAPS - 1) + k;
      if (local >= 0) ld8(row + (size_t)(t0 + local) * ld + off + c, hist[k]);
      else if (!fresh) ld8(cs + (size_t)(TAPS - 1 + local) * ch, hist[k]);
      else
#pragma unroll
        for (int e = 0; e < 8; ++e) hist[k][e] = 0.f;
    }
    const int stop = min(t_end, t0 + n);
    for (; t < stop; ++t) {
      float y[8];
      ld8(row + (size_t)t * ld + off + c, hist[TAPS - 1]);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        y[e] = bias[e];
#pragma unroll
        for (int k = 0; k < TAPS; ++k) y[e] = fmaf(wk[k][e], hist[k][e], y[e]);
        y[e] = silu(y[e]);
#pragma unroll
        for (int k = 0; k + 1 < TAPS; ++k) hist[k][e] = hist[k + 1][e];
      }
      st8(out + (size_t)t * ch + c, y);
    }
    ++s;
  }
}

// conv_state[slot] = the last taps - 1 inputs (older ones shift down when fewer tokens are new)
template <typename T>
__global__ __launch_bounds__(256) void conv_tail_kernel(SeqArgs q, const T* __restrict__ row, int ld, int off,
                                                        float* conv_state, int ch, int taps) {
  const int c = blockIdx.y * 256 + threadIdx.x, s = blockIdx.x;
  if (c >= ch) return;
  int t0, n;
  bool fresh;
  seq_span(q, s, t0, n, fresh);
  float* cs = conv_state + (size_t)q.states[s] * (taps - 1) * ch + c;
  float v[MAX_TAPS];
#pragma unroll
  for (int k = 0; k < MAX_TAPS; ++k)
    if (k < taps - 1) {
      const int local = n - (taps - 1) + k;
      v[k] = local >= 0 ? ld1(row + (size_t)(t0 + local) * ld + off + c)
                        : (fresh ? 0.f : cs[(size_t)(taps - 1 + local) * ch]);
    }
#pragma unroll
  for (int k = 0; k < MAX_TAPS; ++k)
    if (k < taps - 1) cs[(size_t)k * ch] = v[k];
}

// One block per (head, sequence, SEQ_COLS columns): thread (r, p) owns column p of state rows r, r + R, ...
constexpr int SEQ_COLS = 64;
template <typename T>
__global__ __launch_bounds__(256) void scan_seq_kernel(SeqArgs q, const T* __restrict__ xbc, int ch, const T* __restrict__ row,
                                                       int ld, int off_dt, const float* __restrict__ dt_bias,
                                                       const float* __restrict__ A, const float* __restrict__ D,
                                                       float* ssm_state, float* y, int H, int P, int N, int G, int PP) {
  extern __shared__ float sm[];
  const int h = blockIdx.x, s = blockIdx.y, tid = threadIdx.x;
  const int p0 = blockIdx.z * SEQ_COLS, W = min(SEQ_COLS, P - p0);
  float* S = sm;            // [N][W]
  float* sb = S + N * W;    // [N] dt * B
  float* sc = sb + N;       // [N] C
  float* part = sc + N;     // [256]
  const int g = h / (H / G), R = 256 / PP, r = tid / PP, p = tid % PP;
  int t0, n;
  bool fresh;
  seq_span(q, s, t0, n, fresh);
  float* st = ssm_state + ((size_t)q.states[s] * H + h) * N * P + p0;
  for (int i = tid; i < N * W; i += 256) S[i] = fresh ? 0.f : st[(size_t)(i / W) * P + i % W];
  const float a = A[h], d = D[h], db = dt_bias[h];
  __syncthreads();
  for (int t = t0; t < t0 + n; ++t) {
    const T* xr = xbc + (size_t)t * ch;
    const float dt = softplusf(ld1(row + (size_t)t * ld + off_dt + h) + db);
    const float decay = expf(-a * dt);
    for (int i = tid; i < N; i += 256) {
      sb[i] = dt * ld1(xr + H * P + g * N + i);
      sc[i] = ld1(xr + H * P + G * N + g * N + i);
    }
    __syncthreads();
    float acc = 0.f, x = 0.f;
    if (p < W) {
      x = ld1(xr + h * P + p0 + p);
      for (int i = r; i < N; i += R) {
        const float v = decay * S[i * W + p] + sb[i] * x;
        S[i * W + p] = v;
        acc = fmaf(v, sc[i], acc);
      }
    }
    part[tid] = acc;
    __syncthreads();
    if (r == 0 && p < W) {
      float o = d * x;
      for (int i = 0; i < R; ++i) o += part[i * PP + p];
      y[(size_t)t * H * P + h * P + p0 + p] = o;
    }
  }
  __syncthreads();
  for (int i = tid; i < N * W; i += 256) st[(size_t)(i / W) * P + i % W] = S[i];
}

// ---- chunked scan (bf16) ----
struct ChunkArgs {
  SeqArgs q;
  const bf16_t* xbc; int ch;
  const bf16_t* row; int ld, off_dt;
  const float* dt_bias; const float* A; const float* D;
  float* ssm_state;
  bf16_t* y;
  int H, P, N, G;
};

constexpr int CQ = 64;  // chunk length

// inclusive sum over the wave's lanes, on the VALU (row shifts, then the two row broadcasts)
template <int CTRL, int ROWS>
__device__ __forceinline__ float dpp_add(float v) {
  return v + __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, ROWS, 0xf, false));
}
__device__ __forceinline__ float wave_scan(float v) {
  v = dpp_add<0x111, 0xf>(v);  // row_shr:1
  v = dpp_add<0x112, 0xf>(v);  // row_shr:2
  v = dpp_add<0x114, 0xf>(v);  // row_shr:4
  v = dpp_add<0x118, 0xf>(v);  // row_shr:8
  v = dpp_add<0x142, 0xa>(v);  // row_bcast:15 into rows 1 and 3
  return dpp_add<0x143, 0xc>(v);  // row_bcast:31 into rows 2 and 3
}

// split 8 floats into bf16 high and low parts
__device__ __forceinline__ void split8(const float* f, u32x4& hi, u32x4& lo) {
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    hi[i] = pk2bf(f[2 * i], f[2 * i + 1]);
    lo[i] = pk2bf(f[2 * i] - __uint_as_float(hi[i] << 16), f[2 * i + 1] - __uint_as_float(hi[i] & 0xffff0000u));
  }
}

// NP: padded state rows (N <= NP), PS: state columns per block. 4 waves: wave w computes the outputs of chunk
// tokens 16w .. 16w + 15 and owns state rows 16w, 16(w + 4), ... of the running state (fp32 accumulators).
template <int NP, int PS>
__global__ __launch_bounds__(256, NP <= 128 ? 2 : 1) void scan_chunk_kernel(ChunkArgs a) {
  using CB = Cfg<NP>;
  using CX = Cfg<PS>;
  constexpr int NT16 = NP / 16, SPW = (NT16 + 3) / 4;  // state row tiles, tiles per wave
  constexpr int PT = PS / 16;
  constexpr int SROW = NP * 2 + 16;  // bytes per state column in LDS (padded against bank conflicts)
  __shared__ __attribute__((aligned(16))) char smem[CB::TILEB + 3 * CX::TILEB + 2 * PS * SROW + 2 * CQ * 4];
  char* sB = smem;                  // B rows [token][n], row-read swizzle
  char* sX = sB + CB::TILEB;        // x rows [token][p], transposed-read swizzle
  char* sXh = sX + CX::TILEB;       // e^(c_end - c_s) dt_s x_s, high part
  char* sXl = sXh + CX::TILEB;      // ... low part
  char* sSh = sXl + CX::TILEB;      // state entering the chunk [p][n], high part
  char* sSl = sSh + PS * SROW;      // ... low part
  float* s_cum = reinterpret_cast<float*>(sSl + PS * SROW);  // running log-decay (log2 units)
  float* s_dt = s_cum + CQ;

  const int lane = threadIdx.x & 63, wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), tid = threadIdx.x;
  const int fr = lane & 15, fh = lane >> 4;
  const int h = blockIdx.x, seq = blockIdx.y, p0 = blockIdx.z * PS;
  const int g = h / (a.H / a.G);
  int t0, n;
  bool fresh;
  seq_span(a.q, seq, t0, n, fresh);
  if (n <= 0) return;
  float* st = a.ssm_state + ((size_t)a.q.states[seq] * a.H + h) * a.N * a.P;
  const float decay_rate = a.A[h] * 1.4426950408889634f, dskip = a.D[h], dbias = a.dt_bias[h];
  const int inner = a.H * a.P, offB = inner + g * a.N, offC = inner + (a.G + g) * a.N;

  // running state: S[n][p], row tile i of this wave = rows 16 (wid + 4 i); lane holds rows 4fh + r, column fr
  f32x4 S[SPW][PT];
#pragma unroll
  for (int i = 0; i < SPW; ++i)
#pragma unroll
    for (int j = 0; j < PT; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int nn = 16 * (wid + 4 * i) + 4 * fh + r, pp = p0 + 16 * j + fr;
        S[i][j][r] = (!fresh && nn < a.N && pp < a.P) ? st[(size_t)nn * a.P + pp] : 0.f;
      }
  auto store_state = [&]() {  // high / low parts into LDS, [p][n]: four consecutive n per lane
#pragma unroll
    for (int i = 0; i < SPW; ++i)
      if (wid + 4 * i < NT16) {
#pragma unroll
        for (int j = 0; j < PT; ++j) {
          const f32x4 v = S[i][j];
          const unsigned h0 = pk2bf(v[0], v[1]), h1 = pk2bf(v[2], v[3]);
          const unsigned l0 = pk2bf(v[0] - __uint_as_float(h0 << 16), v[1] - __uint_as_float(h0 & 0xffff0000u));
          const unsigned l1 = pk2bf(v[2] - __uint_as_float(h1 << 16), v[3] - __uint_as_float(h1 & 0xffff0000u));
          const int off = (16 * j + fr) * SROW + (16 * (wid + 4 * i) + 4 * fh) * 2;
          *reinterpret_cast<uint2*>(sSh + off) = make_uint2(h0, h1);
          *reinterpret_cast<uint2*>(sSl + off) = make_uint2(l0, l1);
        }
      }
  };
  store_state();

  constexpr int BV = CQ * NP / 8 / 256, XV = (CQ * PS / 8 + 255) / 256;
  u32x4 rb[BV], rx[XV];
  bf16x8 cf[CB::KS];
  float rdt = 0.f;
  const u32x4 zero4 = (u32x4){0u, 0u, 0u, 0u};
  auto fetch = [&](int c0) {  // chunk rows into registers (zeros past the sequence or past N / P)
#pragma unroll
    for (int i = 0; i < BV; ++i) {
      const int v = tid + 256 * i, t = v / (NP / 8), c = (v % (NP / 8)) * 8;
      rb[i] = (c0 + t < n && c < a.N)
                  ? *reinterpret_cast<const u32x4*>(a.xbc + (size_t)(t0 + c0 + t) * a.ch + offB + c) : zero4;
    }
#pragma unroll
    for (int i = 0; i < XV; ++i) {
      const int v = tid + 256 * i, t = v / (PS / 8), c = (v % (PS / 8)) * 8;
      rx[i] = (t < CQ && c0 + t < n && p0 + c < a.P)
                  ? *reinterpret_cast<const u32x4*>(a.xbc + (size_t)(t0 + c0 + t) * a.ch + h * a.P + p0 + c) : zero4;
    }
    const int tq = c0 + 16 * wid + fr;
#pragma unroll
    for (int s = 0; s < CB::KS; ++s) {
      const int c = 32 * s + 8 * fh;
      cf[s] = (tq < n && c < a.N)
                  ? *reinterpret_cast<const bf16x8*>(a.xbc + (size_t)(t0 + tq) * a.ch + offC + c)
                  : (bf16x8){0, 0, 0, 0, 0, 0, 0, 0};
    }
    rdt = c0 + lane < n ? bf2f(a.row[(size_t)(t0 + c0 + lane) * a.ld + a.off_dt + h]) : 0.f;
  };
  fetch(0);

  for (int c0 = 0; c0 < n; c0 += CQ) {
    // every wave forms the chunk's running log-decay (lane = token) and keeps what it needs of it
    const float dt = c0 + lane < n ? softplusf(rdt + dbias) : 0.f;
    const float cum = wave_scan(-decay_rate * dt);
    const float c_end = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(cum), 63));
    const float wgt = __builtin_amdgcn_exp2f(c_end - cum) * dt;  // what this lane's token leaves in the state
    if (wid == 0) {
      s_cum[lane] = cum;
      s_dt[lane] = dt;
    }
#pragma unroll
    for (int i = 0; i < BV; ++i) {
      const int v = tid + 256 * i, t = v / (NP / 8), c = v % (NP / 8);
      *reinterpret_cast<u32x4*>(sB + t * CB::ROWB + 16 * (c ^ kswz<NP>(t))) = rb[i];
    }
    bf16x8 cq[CB::KS];
#pragma unroll
    for (int s = 0; s < CB::KS; ++s) cq[s] = cf[s];
#pragma unroll
    for (int i = 0; i < XV; ++i) {
      const int v = tid + 256 * i, t = v / (PS / 8), c = v % (PS / 8);
      const float wt = __shfl(wgt, t & 63, 64);
      if (t < CQ) {
        const int off = t * CX::ROWB + 16 * (c ^ vswz<PS>(t));
        float f[8];
        unpack8(rx[i], f);
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] *= wt;
        u32x4 hi, lo;
        split8(f, hi, lo);
        *reinterpret_cast<u32x4*>(sX + off) = rx[i];
        *reinterpret_cast<u32x4*>(sXh + off) = hi;
        *reinterpret_cast<u32x4*>(sXl + off) = lo;
      }
    }
    __syncthreads();
    if (c0 + CQ < n) fetch(c0 + CQ);  // in flight during the products

    // ---- M^T[s][t] = (B_s . C_t) e^(c_t - c_s) dt_s for s <= t; t = 16 wid + fr ----
    const int tq = 16 * wid + fr;
    const float c_t = s_cum[tq];
    f32x4 m[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      m[j] = (f32x4){0.f, 0.f, 0.f, 0.f};
      if (j <= wid) {
#pragma unroll
        for (int s = 0; s < CB::KS; ++s)
          m[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(load_k<NP>(sB, j, s, lane), cq[s], m[j], 0, 0, 0);
        const f32x4 cs = *reinterpret_cast<const f32x4*>(s_cum + 16 * j + 4 * fh);
        const f32x4 ds = *reinterpret_cast<const f32x4*>(s_dt + 16 * j + 4 * fh);
#pragma unroll
        for (int r = 0; r < 4; ++r)
          m[j][r] = 16 * j + 4 * fh + r <= tq ? m[j][r] * __builtin_amdgcn_exp2f(c_t - cs[r]) * ds[r] : 0.f;
      }
    }
    // ---- y^T[p][t] = e^(c_t) S^T C_t + x^T M^T + D x_t ----
    f32x4 y[PT];
    const float e_t = __builtin_amdgcn_exp2f(c_t);
#pragma unroll
    for (int j = 0; j < PT; ++j) {
      y[j] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < CB::KS; ++s) {
        const int off = (16 * j + fr) * SROW + (32 * s + 8 * fh) * 2;
        y[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(sSh + off), cq[s], y[j], 0, 0, 0);
        y[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(sSl + off), cq[s], y[j], 0, 0, 0);
      }
      y[j] *= e_t;
    }
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      if (2 * ks > wid) continue;  // keys 32 ks .. are all later than this wave's tokens
      float f[8];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        f[r] = m[2 * ks][r];
        f[4 + r] = m[2 * ks + 1][r];
      }
      u32x4 hi, lo;
      split8(f, hi, lo);
#pragma unroll
      for (int j = 0; j < PT; ++j) {
        const bf16x8 xf = load_vt<PS>(sX, j, ks, lane);
        y[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xf, __builtin_bit_cast(bf16x8, hi), y[j], 0, 0, 0);
        y[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xf, __builtin_bit_cast(bf16x8, lo), y[j], 0, 0, 0);
      }
    }
    if (c0 + tq < n) {
      bf16_t* yr = a.y + (size_t)(t0 + c0 + tq) * inner + h * a.P + p0;
#pragma unroll
      for (int j = 0; j < PT; ++j) {
        const int c = 16 * j + 4 * fh;
        const uint2 xv = *reinterpret_cast<const uint2*>(sX + tq * CX::ROWB + 16 * ((c >> 3) ^ vswz<PS>(tq)) + (c & 4) * 2);
        const float x0 = __uint_as_float(xv.x << 16), x1 = __uint_as_float(xv.x & 0xffff0000u);
        const float x2 = __uint_as_float(xv.y << 16), x3 = __uint_as_float(xv.y & 0xffff0000u);
        if (p0 + c < a.P)
          *reinterpret_cast<uint2*>(yr + c) =
              make_uint2(pk2bf(__builtin_fmaf(dskip, x0, y[j][0]), __builtin_fmaf(dskip, x1, y[j][1])),
                         pk2bf(__builtin_fmaf(dskip, x2, y[j][2]), __builtin_fmaf(dskip, x3, y[j][3])));
      }
    }
    // ---- S <- e^(c_end) S + B^T (w x) ----
    const float e_end = __builtin_amdgcn_exp2f(c_end);
#pragma unroll
    for (int i = 0; i < SPW; ++i) {
      if (wid + 4 * i >= NT16) continue;
#pragma unroll
      for (int j = 0; j < PT; ++j) S[i][j] *= e_end;
    }
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      bf16x8 xh[PT], xl[PT];
#pragma unroll
      for (int j = 0; j < PT; ++j) {
        xh[j] = load_vt<PS>(sXh, j, ks, lane);
        xl[j] = load_vt<PS>(sXl, j, ks, lane);
      }
#pragma unroll
      for (int i = 0; i < SPW; ++i) {
        if (wid + 4 * i >= NT16) continue;
        // B^T fragment (rows n, tokens in the transposed-read order) from the row-read swizzled tile
        const int hh = lane >> 4, ii = lane & 15, chunk = 2 * (wid + 4 * i) + ((ii >> 1) & 1);
        const int r0 = 32 * ks + 4 * hh + (ii >> 2), r1 = r0 + 16;
        const bf16x4 b0 = tr_read(sB + r0 * CB::ROWB + 16 * (chunk ^ kswz<NP>(r0)) + 8 * (ii & 1));
        const bf16x4 b1 = tr_read(sB + r1 * CB::ROWB + 16 * (chunk ^ kswz<NP>(r1)) + 8 * (ii & 1));
        const bf16x8 bf = (bf16x8){b0[0], b0[1], b0[2], b0[3], b1[0], b1[1], b1[2], b1[3]};
#pragma unroll
        for (int j = 0; j < PT; ++j) {
          S[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf, xh[j], S[i][j], 0, 0, 0);
          S[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf, xl[j], S[i][j], 0, 0, 0);
        }
      }
    }
    __syncthreads();  // every wave has read this chunk's tiles and the entering state
    store_state();    // ordered before its readers by the next chunk's barrier
  }
#pragma unroll
  for (int i = 0; i < SPW; ++i)
#pragma unroll
    for (int j = 0; j < PT; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int nn = 16 * (wid + 4 * i) + 4 * fh + r, pp = p0 + 16 * j + fr;
        if (nn < a.N && pp < a.P) st[(size_t)nn * a.P + pp] = S[i][j][r];
      }
}

// ---- decode: one token per sequence from projection slabs P [S][B][ld] ----
// act[b] = [silu(z) : inner | silu(conv) : ch | softplus(dt) : H], fp32; the conv state moves on by one token
__global__ __launch_bounds__(256) void dec_act_kernel(const float* __restrict__ P, int S, size_t slab, int ld,
                                                      const int* __restrict__ kv_lens, const int* __restrict__ states,
                                                      const float* __restrict__ cw, const float* __restrict__ cb,
                                                      const float* __restrict__ dt_bias, float* conv_state, float* act,
                                                      int inner, int ch, int H, int taps) {
  const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y;
  if (c >= inner + ch + H) return;
  float u = 0.f;
  for (int s0 = 0; s0 < S; s0 += 8) {  // 8 slab loads in flight
    float v[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = P[(size_t)min(s0 + i, S - 1) * slab + (size_t)b * ld + c];
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (s0 + i < S) u += v[i];
  }
  float* o = act + (size_t)b * ld + c;
  if (c < inner) {
    *o = silu_exact(u);
  } else if (c < inner + ch) {
    const int k = c - inner;
    const bool fresh = kv_lens[b] == 1;
    float* cs = conv_state + (size_t)states[b] * (taps - 1) * ch + k;
    float y = cb[k], hist[MAX_TAPS];
#pragma unroll
    for (int t = 0; t < MAX_TAPS; ++t) hist[t] = t < taps - 1 && !fresh ? cs[(size_t)t * ch] : 0.f;
#pragma unroll
    for (int t = 0; t < MAX_TAPS; ++t)
      if (t < taps) y = fmaf(cw[(size_t)t * ch + k], t == taps - 1 ? u : hist[t], y);
#pragma unroll
    for (int t = 0; t < MAX_TAPS; ++t)
      if (t < taps - 1) cs[(size_t)t * ch] = t == taps - 2 ? u : hist[t + 1];
    *o = silu_exact(y);
  } else {
    *o = softplusf(u + dt_bias[c - inner - ch]);
  }
}

// One block per (head, sequence): S <- decay S + dt B x^T (read and written once), y = (S^T C + D x) silu(z).
// Thread (r, v): 4 consecutive columns 4v .. of state rows r, r + R, ...; P % 4 == 0.
__global__ __launch_bounds__(256) void dec_state_kernel(const float* __restrict__ act, int ld,
                                                        const int* __restrict__ kv_lens, const int* __restrict__ states,
                                                        const float* __restrict__ A, const float* __restrict__ D,
                                                        float* ssm_state, float* yz, int H, int P, int N, int G, int PV) {
  __shared__ float part[256][4];
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const int g = h / (H / G), R = 256 / PV, r = tid / PV, v = tid % PV, inner = H * P;
  const bool col = 4 * v < P, fresh = kv_lens[b] == 1;
  const float* ar = act + (size_t)b * ld;
  const float* Bp = ar + 2 * inner + g * N;
  const float* Cp = Bp + G * N;
  float* st = ssm_state + ((size_t)states[b] * H + h) * N * P + 4 * v;
  const float dt = ar[2 * inner + 2 * G * N + h], decay = expf(-A[h] * dt);
  f32x4 acc = (f32x4){0.f, 0.f, 0.f, 0.f}, x = acc;
  if (col) {
    x = *reinterpret_cast<const f32x4*>(ar + inner + h * P + 4 * v);
    const f32x4 dx = x * dt;
    for (int n0 = r; n0 < N; n0 += 8 * R) {
      f32x4 s[8];
      float bb[8], cc[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int n = min(n0 + i * R, N - 1);
        s[i] = fresh ? (f32x4){0.f, 0.f, 0.f, 0.f} : *reinterpret_cast<const f32x4*>(st + (size_t)n * P);
        bb[i] = Bp[n];
        cc[i] = Cp[n];
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int n = n0 + i * R;
        if (n < N) {
          const f32x4 w = s[i] * decay + dx * bb[i];
          *reinterpret_cast<f32x4*>(st + (size_t)n * P) = w;
          acc += w * cc[i];
        }
      }
    }
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) part[tid][e] = acc[e];
  __syncthreads();
  if (tid < P) {
    const int vv = tid >> 2, e = tid & 3;
    float o = D[h] * ar[inner + h * P + tid];
    for (int i = 0; i < R; ++i) o += part[i * PV + vv][e];
    yz[(size_t)b * inner + h * P + tid] = o * ar[h * P + tid];
  }
}

// out[t] = group_norm(y * silu(z)) * w with 16-B vectors, one wave per (token, group); z null: y is gated already
template <int MAXV, typename TY>
__global__ __launch_bounds__(256) void gate_norm_wave_kernel(const TY* __restrict__ y, const bf16_t* __restrict__ row, int ld,
                                                             const float* __restrict__ w, bf16_t* out, int ldo, int T,
                                                             int inner, int gsz, int groups, float eps) {
  const int lane = threadIdx.x & 63, item = blockIdx.x * 4 + (threadIdx.x >> 6);
  const int t = item / groups, c0 = (item - t * groups) * gsz;
  if (t >= T) return;
  const int nv = gsz >> 3;
  float f[MAXV][8], ss = 0.f;
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const int v = lane + 64 * i;
    if (v < nv) {
      ld8(y + (size_t)t * inner + c0 + v * 8, f[i]);
      if (row) {
        float z[8];
        ld8(row + (size_t)t * ld + c0 + v * 8, z);
#pragma unroll
        for (int e = 0; e < 8; ++e) f[i][e] *= silu_exact(z[e]);
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += f[i][e] * f[i][e];
    }
  }
  const float inv = rsqrtf(wave_sum(ss) / (float)gsz + eps);
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const int v = lane + 64 * i;
    if (v < nv) {
      float g[8];
      ld8(w + c0 + v * 8, g);
#pragma unroll
      for (int e = 0; e < 8; ++e) f[i][e] *= inv * g[e];
      st8(out + (size_t)t * ldo + c0 + v * 8, f[i]);
    }
  }
}

template <typename TY>
int launch_gate_norm_wave(const TY* y, const bf16_t* row, int ld, const float* w, bf16_t* out, int ldo, int T, int inner,
                          int groups, float eps, hipStream_t st) {
  const int gsz = inner / groups, per = (gsz / 8 + 63) / 64;
  const dim3 grid((unsigned)(((long long)T * groups + 3) / 4));
#define RAGK_GN(V)                                                                                                       \
  hipLaunchKernelGGL((gate_norm_wave_kernel<V, TY>), grid, dim3(256), 0, st, y, row, ld, w, out, ldo, T, inner, gsz,      \
                     groups, eps)
  if (per <= 1) RAGK_GN(1);
  else if (per <= 2) RAGK_GN(2);
  else if (per <= 4) RAGK_GN(4);
  else if (per <= 8) RAGK_GN(8);
  else return (int)hipErrorInvalidValue;
#undef RAGK_GN
  return (int)hipGetLastError();
}

template <int NP, int PS>
int launch_scan_chunk(const ChunkArgs& a, hipStream_t st) {
  hipLaunchKernelGGL((scan_chunk_kernel<NP, PS>), dim3(a.H, a.q.S, (a.P + PS - 1) / PS), dim3(256), 0, st, a);
  return (int)hipGetLastError();
}

// y or yz with one thread per element, any group size; z as in gate_norm_wave
template <typename TY, typename T>
__global__ __launch_bounds__(256) void gate_norm_kernel(const TY* __restrict__ y, const T* __restrict__ row, int ld,
                                                        const float* __restrict__ w, T* out, int ldo, int inner, int gsz,
                                                        float eps) {
  __shared__ float red[4];
  const int t = blockIdx.x, c0 = blockIdx.y * gsz;
  const TY* yr = y + (size_t)t * inner + c0;
  const T* zr = row ? row + (size_t)t * ld + c0 : nullptr;
  float ss = 0.f;
  for (int i = threadIdx.x; i < gsz; i += 256) {
    const float v = ld1(yr + i) * (zr ? silu_exact(ld1(zr + i)) : 1.f);
    ss += v * v;
  }
  const float inv = rsqrtf(block_sum(ss, red) / (float)gsz + eps);
  for (int i = threadIdx.x; i < gsz; i += 256) {
    const float v = ld1(yr + i) * (zr ? silu_exact(ld1(zr + i)) : 1.f);
    st1(out + (size_t)t * ldo + c0 + i, v * inv * w[c0 + i]);
  }
}

template <typename T>
int launch_conv(const SeqArgs& q, const void* row, int ld, int off, const float* w, const float* b, float* conv_state,
                void* out, int ch, int taps, hipStream_t st) {
  hipLaunchKernelGGL(conv_silu_kernel<T>, dim3((q.T + CONV_TT - 1) / CONV_TT, (ch + 255) / 256), dim3(256), 0, st, q,
                     (const T*)row, ld, off, w, b, conv_state, (T*)out, ch, taps);
  if (taps > 1)
    hipLaunchKernelGGL(conv_tail_kernel<T>, dim3(q.S, (ch + 255) / 256), dim3(256), 0, st, q, (const T*)row, ld, off,
                       conv_state, ch, taps);
  return (int)hipGetLastError();
}

}  // namespace

// row: [T][ld] (fp32 when f32), the convolution's inputs at column off; out: [T][ch]. conv_state is updated.
RAGK_API int ragk_ssm_conv(const int* cu_q, const int* kv_lens, const int* states, int T, int S, const void* row, int ld,
                           int off, const float* w, const float* b, float* conv_state, void* out, int ch, int taps,
                           int f32, hipStream_t st) {
  if (T <= 0) return 0;
  if (taps < 1 || taps > MAX_TAPS || S < 1 || (!cu_q && S != T)) return (int)hipErrorInvalidValue;
  const SeqArgs q{cu_q, kv_lens, states, T, S};
  if (!f32 && ch % 8 == 0 && ld % 8 == 0 && off % 8 == 0 && taps >= 2 && taps <= 4) {
    const dim3 grid((T + CONV_TT - 1) / CONV_TT, (ch / 8 + 255) / 256);
#define RAGK_CV(TP)                                                                                                  \
  hipLaunchKernelGGL(conv_silu_vec_kernel<TP>, grid, dim3(256), 0, st, q, (const bf16_t*)row, ld, off, w, b, conv_state, \
                     (bf16_t*)out, ch)
    if (taps == 2) RAGK_CV(2);
    else if (taps == 3) RAGK_CV(3);
    else RAGK_CV(4);
#undef RAGK_CV
    hipLaunchKernelGGL(conv_tail_kernel<bf16_t>, dim3(S, (ch + 255) / 256), dim3(256), 0, st, q, (const bf16_t*)row, ld, off,
                       conv_state, ch, taps);
    return (int)hipGetLastError();
  }
  return f32 ? launch_conv<float>(q, row, ld, off, w, b, conv_state, out, ch, taps, st)
             : launch_conv<bf16_t>(q, row, ld, off, w, b, conv_state, out, ch, taps, st);
}

// Token-by-token scan. y: fp32 [T][H*P]. 66 N floats must fit the LDS.
RAGK_API int ragk_ssm_scan_seq(const int* cu_q, const int* kv_lens, const int* states, int T, int S, const void* xbc, int ch,
                               const void* row, int ld, int off_dt, const float* dt_bias, const float* A, const float* D,
                               float* ssm_state, float* y, int H, int P, int N, int G, int f32, hipStream_t st) {
  if (T <= 0) return 0;
  const int W = P < SEQ_COLS ? P : SEQ_COLS;
  const size_t lds = ((size_t)N * W + 2 * N + 256) * 4;
  if (H % G || lds > 160 * 1024 || S < 1 || S > 65535 || (!cu_q && S != T)) return (int)hipErrorInvalidValue;
  int PP = 1;
  while (PP < W) PP *= 2;
  const dim3 grid(H, S, (P + SEQ_COLS - 1) / SEQ_COLS);
  const SeqArgs q{cu_q, kv_lens, states, T, S};
  if (f32) {
    (void)hipFuncSetAttribute((const void*)scan_seq_kernel<float>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL(scan_seq_kernel<float>, grid, dim3(256), lds, st, q, (const float*)xbc, ch, (const float*)row,
                       ld, off_dt, dt_bias, A, D, ssm_state, y, H, P, N, G, PP);
  } else {
    (void)hipFuncSetAttribute((const void*)scan_seq_kernel<bf16_t>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL(scan_seq_kernel<bf16_t>, grid, dim3(256), lds, st, q, (const bf16_t*)xbc, ch,
                       (const bf16_t*)row, ld, off_dt, dt_bias, A, D, ssm_state, y, H, P, N, G, PP);
  }
  return (int)hipGetLastError();
}

static int g_scan_cols = 0;
// value columns per scan block: 32, 64, or 0 = by the grid (tests, measurements)
RAGK_API int ragk_ssm_scan_set_cols(int cols) {
  if (cols != 0 && cols != 32 && cols != 64) return (int)hipErrorInvalidValue;
  g_scan_cols = cols;
  return 0;
}

// Chunked scan (bf16). y: bf16 [T][H*P]. P % 8 == 0, N % 8 == 0, N <= 256, ch % 8 == 0.
RAGK_API int ragk_ssm_scan_chunk(const int* cu_q, const int* kv_lens, const int* states, int T, int S, const void* xbc,
                                 int ch, const void* row, int ld, int off_dt, const float* dt_bias, const float* A,
                                 const float* D, float* ssm_state, void* y, int H, int P, int N, int G, hipStream_t st) {
  if (T <= 0) return 0;
  if (P % 8 || N % 8 || N > 256 || ch % 8 || H % G || S < 1 || S > 65535 || (!cu_q && S != T))
    return (int)hipErrorInvalidValue;
  const ChunkArgs a{{cu_q, kv_lens, states, T, S}, (const bf16_t*)xbc, ch, (const bf16_t*)row, ld, off_dt, dt_bias, A, D,
                    ssm_state, (bf16_t*)y, H, P, N, G};
  // narrow column slices when one block per (head, sequence) would leave CUs idle
  const bool narrow = P <= 32 || (g_scan_cols ? g_scan_cols == 32 : (long long)H * S * ((P + 63) / 64) <= 256);
#define RAGK_SC(NPV) return narrow ? launch_scan_chunk<NPV, 32>(a, st) : launch_scan_chunk<NPV, 64>(a, st)
  if (N <= 32) RAGK_SC(32);
  if (N <= 64) RAGK_SC(64);
  if (N <= 128) RAGK_SC(128);
  RAGK_SC(256);
#undef RAGK_SC
}

// One token per sequence. P: fp32 slabs [S][B][ld]; act: fp32 [B][ld] scratch; yz: fp32 [B][inner]. P % 4 == 0, P <= 256.
RAGK_API int ragk_ssm_decode(const float* slabs, int S, int ld, const int* kv_lens, const int* states, const float* conv_w,
                             const float* conv_b, const float* dt_bias, const float* A, const float* D, float* conv_state,
                             float* ssm_state, float* act, float* yz, int B, int H, int P, int N, int G, int taps,
                             hipStream_t st) {
  if (B <= 0) return 0;
  if (S < 1 || B > 65535 || P % 4 || P > 256 || N % 4 || H % G || taps < 1 || taps > MAX_TAPS || ld % 4)
    return (int)hipErrorInvalidValue;
  const int inner = H * P, ch = inner + 2 * G * N;
  int PV = 1;
  while (4 * PV < P) PV *= 2;
  hipLaunchKernelGGL(dec_act_kernel, dim3((inner + ch + H + 255) / 256, B), dim3(256), 0, st, slabs, S, (size_t)B * ld, ld,
                     kv_lens, states, conv_w, conv_b, dt_bias, conv_state, act, inner, ch, H, taps);
  hipLaunchKernelGGL(dec_state_kernel, dim3(H, B), dim3(256), 0, st, act, ld, kv_lens, states, A, D, ssm_state, yz, H, P, N,
                     G, PV);
  return (int)hipGetLastError();
}

// out[t] = group_norm(y[t] * silu(row[t][0 : inner])) * w; y [T][inner] fp32 or bf16 (y_bf16), out [T][ldo] bf16, or
// fp32 when f32. row null: y is gated already.
RAGK_API int ragk_ssm_gate_norm(const void* y, int y_bf16, const void* row, int ld, const float* w, void* out, int ldo, int T,
                                int inner, int groups, float eps, int f32, hipStream_t st) {
  if (T <= 0) return 0;
  if (groups < 1 || inner % groups || (f32 && y_bf16)) return (int)hipErrorInvalidValue;
  const int gsz = inner / groups;
  if (!f32 && gsz % 8 == 0 && gsz <= 4096 && ld % 8 == 0 && ldo % 8 == 0)
    return y_bf16 ? launch_gate_norm_wave<bf16_t>((const bf16_t*)y, (const bf16_t*)row, ld, w, (bf16_t*)out, ldo, T, inner,
                                                  groups, eps, st)
                  : launch_gate_norm_wave<float>((const float*)y, (const bf16_t*)row, ld, w, (bf16_t*)out, ldo, T, inner,
                                                 groups, eps, st);
  const dim3 grid(T, groups);
  if (f32)
    hipLaunchKernelGGL((gate_norm_kernel<float, float>), grid, dim3(256), 0, st, (const float*)y, (const float*)row, ld, w,
                       (float*)out, ldo, inner, gsz, eps);
  else if (y_bf16)
    hipLaunchKernelGGL((gate_norm_kernel<bf16_t, bf16_t>), grid, dim3(256), 0, st, (const bf16_t*)y, (const bf16_t*)row, ld,
                       w, (bf16_t*)out, ldo, inner, gsz, eps);
  else
    hipLaunchKernelGGL((gate_norm_kernel<float, bf16_t>), grid, dim3(256), 0, st, (const float*)y, (const bf16_t*)row, ld,
                       w, (bf16_t*)out, ldo, inner, gsz, eps);
  return (int)hipGetLastError();
}
