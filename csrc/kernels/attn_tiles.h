// Attention tile helpers for gfx950: swizzled LDS K / V tiles of 64 rows, LDS-DMA staging, MFMA fragments
// (row fragments by ds_read_b128, transposed fragments by ds_read_b64_tr_b16).
#pragma once
#include "common.h"

namespace ragk {

constexpr int KT = 64;  // keys per tile == KV-cache page size
constexpr int MAX_BT = 2048;  // prefill block-table row cached in LDS (128k tokens)
constexpr float RESCALE_LOG2 = 8.f;  // deferred-rescale threshold (log2 units)

// max with the xor-16 / xor-32 lane partner without an LDS round trip (gfx950
// v_permlane{16,32}_swap). With both operands = v the swap returns, per lane, {v, partner} in
// some order, so max(r0, r1) is the pairwise max on every lane.
__device__ __forceinline__ float max_xor32(float v) {
  const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  return fmaxf(__uint_as_float(r[0]), __uint_as_float(r[1]));
}
__device__ __forceinline__ float max_xor16(float v) {
  const auto r = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  return fmaxf(__uint_as_float(r[0]), __uint_as_float(r[1]));
}

template <int D>
struct Cfg {
  static constexpr int NC = D / 8;               // 16-B chunks per row
  static constexpr int ROWB = D * 2;             // bytes per row
  static constexpr int TILEB = KT * D * 2;       // bytes per K or V tile
  static constexpr int PIECES = TILEB / 1024;    // 1-KiB glds pieces per tile
  static constexpr int RPP = 1024 / ROWB;        // rows per piece
  static constexpr int KS = D / 32;              // k-steps of QK^T
  static constexpr int DT = D / 16;              // 16-wide d tiles of O
  static constexpr int GR = D / 16;              // 32-B granules per row
  static constexpr int RB = GR <= 8 ? 8 / GR : 1;  // rows per 256-B bank row
};

// K tile: swizzle for row reads (ds_read_b128)
template <int D>
__device__ __forceinline__ int kswz(int row) {
  constexpr int NC = Cfg<D>::NC;
  if constexpr (NC > 16) return row & 15;
  else return (row / (16 / NC)) & (NC - 1);
}
// V tile: swizzle for transposed reads (keeps 32-B granules intact)
template <int D>
__device__ __forceinline__ int vswz(int row) {
  return 2 * ((row / Cfg<D>::RB) & (Cfg<D>::GR - 1));
}

__device__ __forceinline__ bf16x4 tr_read(const char* p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) bf16x4*)(p));
}

// Stage one 64-row tile (K or V) into LDS with glds; `pieces_per_wave` pieces per wave.
// row_src(row) returns the global row pointer for tile row `row`.
template <int D, bool IS_V, bool NT = false, int NW = 0, typename RowSrc>
__device__ __forceinline__ void stage_kv(char* lds_tile, int wid, int nwaves, int lane, RowSrc row_src) {
  constexpr int NC = Cfg<D>::NC, PIECES = Cfg<D>::PIECES, RPP = Cfg<D>::RPP;
  constexpr int PPW = NW > 0 ? PIECES / NW : PIECES;  // NW > 0: compile-time wave count, unrolled
#pragma unroll
  for (int i = 0; i < PPW; ++i) {
    const int p = NW > 0 ? wid + NW * i : wid + nwaves * i;
    if (NW == 0 && p >= PIECES) break;
    const int row = p * RPP + lane / NC;
    const int ph = lane % NC;
    const int c = ph ^ (IS_V ? vswz<D>(row) : kswz<D>(row));
    if constexpr (NT)  // once-read K/V stream (decode): non-temporal LDS-DMA
      __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(row_src(row) + c * 8),
                                       (__attribute__((address_space(3))) void*)(lds_tile + p * 1024), 16, 0, 2);
    else
      glds16(row_src(row) + c * 8, lds_tile + p * 1024);
  }
}

// V^T A-fragment for d-tile dt and key k-step ks (32 keys) from a V tile in LDS.
template <int D>
__device__ __forceinline__ bf16x8 load_vt(const char* sV, int dt, int ks, int lane) {
  const int h = lane >> 4, i = lane & 15;
  const int chunk = 2 * dt + ((i >> 1) & 1);
  const int r0 = 32 * ks + 4 * h + (i >> 2);
  const int r1 = r0 + 16;
  const bf16x4 a = tr_read(sV + r0 * Cfg<D>::ROWB + 16 * (chunk ^ vswz<D>(r0)) + 8 * (i & 1));
  const bf16x4 b = tr_read(sV + r1 * Cfg<D>::ROWB + 16 * (chunk ^ vswz<D>(r1)) + 8 * (i & 1));
  return (bf16x8){a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
}

template <int D>
__device__ __forceinline__ bf16x8 load_k(const char* sK, int t, int s, int lane) {
  const int R = 16 * t + (lane & 15);
  const int c = 4 * s + (lane >> 4);
  return *reinterpret_cast<const bf16x8*>(sK + R * Cfg<D>::ROWB + 16 * (c ^ kswz<D>(R)));
}

__device__ __forceinline__ bf16x8 pack_p(const f32x4& a, const f32x4& b) {
  return (bf16x8){f2bf_s(a[0]), f2bf_s(a[1]), f2bf_s(a[2]), f2bf_s(a[3]),
                  f2bf_s(b[0]), f2bf_s(b[1]), f2bf_s(b[2]), f2bf_s(b[3])};
}

// high and low bf16 parts of 8 probabilities as MFMA operands
__device__ __forceinline__ void split_p(const f32x4& a, const f32x4& b, bf16x8& hi, bf16x8& lo) {
  u32x4 h, l;
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    h[i] = pk2bf(a[2 * i], a[2 * i + 1]);
    h[2 + i] = pk2bf(b[2 * i], b[2 * i + 1]);
    l[i] = pk2bf(a[2 * i] - __uint_as_float(h[i] << 16), a[2 * i + 1] - __uint_as_float(h[i] & 0xffff0000u));
    l[2 + i] = pk2bf(b[2 * i] - __uint_as_float(h[2 + i] << 16), b[2 * i + 1] - __uint_as_float(h[2 + i] & 0xffff0000u));
  }
  hi = __builtin_bit_cast(bf16x8, h);
  lo = __builtin_bit_cast(bf16x8, l);
}

// LDS-DMA piece as inline asm: the compiler's waitcnt pass cannot tell which LDS bytes a
// buffer_load ... lds intrinsic writes, so it drained vmcnt(0) before the next ds_read of ANY slot
// (an HBM round trip per fragment read). A kernel that uses this orders its slots itself (vmcnt + barrier per
// iteration) and issues every LDS-DMA through it, so M0 is never live for the compiler. The s_nop is the wait state between
// the write of M0 and the DMA that reads it.
__device__ __forceinline__ void blds16_asm(i32x4 srd, int voff, int soff, unsigned lds_addr) {
  asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tbuffer_load_dwordx4 %1, %2, %3 offen lds" ::"s"(lds_addr), "v"(voff), "s"(srd),
               "s"(soff));
}
__device__ __forceinline__ unsigned lds_addr(const void* p) {
  return (unsigned)(unsigned long long)(const __attribute__((address_space(3))) char*)p;
}

}  // namespace ragk
