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
//  * gate_norm             : the gate and the grouped norm, one block per (token, norm group).
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

// One block per (head, sequence): thread (r, p) owns column p of state rows r, r + R, ...
template <typename T>
__global__ __launch_bounds__(256) void scan_seq_kernel(SeqArgs q, const T* __restrict__ xbc, int ch, const T* __restrict__ row,
                                                       int ld, int off_dt, const float* __restrict__ dt_bias,
                                                       const float* __restrict__ A, const float* __restrict__ D,
                                                       float* ssm_state, float* y, int H, int P, int N, int G, int PP) {
  extern __shared__ float sm[];
  float* S = sm;            // [N][P]
  float* sb = S + N * P;    // [N] dt * B
  float* sc = sb + N;       // [N] C
  float* part = sc + N;     // [256]
  const int h = blockIdx.x, s = blockIdx.y, tid = threadIdx.x;
  const int g = h / (H / G), R = 256 / PP, r = tid / PP, p = tid % PP;
  int t0, n;
  bool fresh;
  seq_span(q, s, t0, n, fresh);
  float* st = ssm_state + ((size_t)q.states[s] * H + h) * N * P;
  for (int i = tid; i < N * P; i += 256) S[i] = fresh ? 0.f : st[i];
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
    if (p < P) {
      x = ld1(xr + h * P + p);
      for (int i = r; i < N; i += R) {
        const float v = decay * S[i * P + p] + sb[i] * x;
        S[i * P + p] = v;
        acc = fmaf(v, sc[i], acc);
      }
    }
    part[tid] = acc;
    __syncthreads();
    if (r == 0 && p < P) {
      float o = d * x;
      for (int i = 0; i < R; ++i) o += part[i * PP + p];
      y[(size_t)t * H * P + h * P + p] = o;
    }
  }
  __syncthreads();
  for (int i = tid; i < N * P; i += 256) st[i] = S[i];
}

template <typename TY, typename T>
__global__ __launch_bounds__(256) void gate_norm_kernel(const TY* __restrict__ y, const T* __restrict__ row, int ld,
                                                        const float* __restrict__ w, T* out, int ldo, int inner, int gsz,
                                                        float eps) {
  __shared__ float red[4];
  const int t = blockIdx.x, c0 = blockIdx.y * gsz;
  const TY* yr = y + (size_t)t * inner + c0;
  const T* zr = row + (size_t)t * ld + c0;
  float ss = 0.f;
  for (int i = threadIdx.x; i < gsz; i += 256) {
    const float v = ld1(yr + i) * silu_exact(ld1(zr + i));
    ss += v * v;
  }
  const float inv = rsqrtf(block_sum(ss, red) / (float)gsz + eps);
  for (int i = threadIdx.x; i < gsz; i += 256) {
    const float v = ld1(yr + i) * silu_exact(ld1(zr + i));
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
  return f32 ? launch_conv<float>(q, row, ld, off, w, b, conv_state, out, ch, taps, st)
             : launch_conv<bf16_t>(q, row, ld, off, w, b, conv_state, out, ch, taps, st);
}

// Token-by-token scan. y: fp32 [T][H*P]. N * P fp32 must fit the LDS with room for two rows of N.
RAGK_API int ragk_ssm_scan_seq(const int* cu_q, const int* kv_lens, const int* states, int T, int S, const void* xbc, int ch,
                               const void* row, int ld, int off_dt, const float* dt_bias, const float* A, const float* D,
                               float* ssm_state, float* y, int H, int P, int N, int G, int f32, hipStream_t st) {
  if (T <= 0) return 0;
  const size_t lds = ((size_t)N * P + 2 * N + 256) * 4;
  if (P > 256 || H % G || lds > 160 * 1024 || S < 1 || S > 65535 || (!cu_q && S != T)) return (int)hipErrorInvalidValue;
  int PP = 1;
  while (PP < P) PP *= 2;
  const SeqArgs q{cu_q, kv_lens, states, T, S};
  if (f32) {
    (void)hipFuncSetAttribute((const void*)scan_seq_kernel<float>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL(scan_seq_kernel<float>, dim3(H, S), dim3(256), lds, st, q, (const float*)xbc, ch, (const float*)row,
                       ld, off_dt, dt_bias, A, D, ssm_state, y, H, P, N, G, PP);
  } else {
    (void)hipFuncSetAttribute((const void*)scan_seq_kernel<bf16_t>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL(scan_seq_kernel<bf16_t>, dim3(H, S), dim3(256), lds, st, q, (const bf16_t*)xbc, ch,
                       (const bf16_t*)row, ld, off_dt, dt_bias, A, D, ssm_state, y, H, P, N, G, PP);
  }
  return (int)hipGetLastError();
}

// out[t] = group_norm(y[t] * silu(row[t][0 : inner])) * w; y fp32 [T][inner], out [T][ldo]
RAGK_API int ragk_ssm_gate_norm(const float* y, const void* row, int ld, const float* w, void* out, int ldo, int T, int inner,
                                int groups, float eps, int f32, hipStream_t st) {
  if (T <= 0) return 0;
  if (groups < 1 || inner % groups) return (int)hipErrorInvalidValue;
  const dim3 grid(T, groups);
  if (f32)
    hipLaunchKernelGGL((gate_norm_kernel<float, float>), grid, dim3(256), 0, st, y, (const float*)row, ld, w, (float*)out,
                       ldo, inner, inner / groups, eps);
  else
    hipLaunchKernelGGL((gate_norm_kernel<float, bf16_t>), grid, dim3(256), 0, st, y, (const bf16_t*)row, ld, w,
                       (bf16_t*)out, ldo, inner, inner / groups, eps);
  return (int)hipGetLastError();
}
