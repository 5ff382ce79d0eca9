"""Shape-checked entry points of the residual-stream, shaped-attention, latent-attention and state-space kernels
(GPU tensors).

Operands are checked on the host before every launch, as in ops/native.py. `f32` paths (exact replay) take
fp32 tensors throughout; otherwise activations and caches are bf16 and the residual stream, split-K slabs,
norm weights and recurrent states fp32.
"""
from __future__ import annotations

from dataclasses import dataclass

import numpy as np
import torch

from . import _lib
from ._lib import check, ptr, stream_ptr
from .native import _req
from .specs import LatentSpec

BF16, F32, I32 = torch.bfloat16, torch.float32, torch.int32


def _act(t, name):
    _req(t.is_cuda and t.dtype in (BF16, F32) and t.dim() == 2 and t.stride(1) == 1, "%s must be 2-D bf16/fp32 rows" % name)
    return int(t.dtype == F32)


def _vec(t, n, dtype, name):
    _req(t.is_cuda and t.dtype == dtype and t.is_contiguous() and t.numel() == n, "%s must be %s[%d]" % (name, dtype, n))


# ------------------------------------------------------------------------------------- residual stream
def embed_residual(ids, table, carry=None, prev=None, scale=1.0, pos=None, turns=None, n=0):
    """fp32 rows table[ids] * scale, plus the sinusoid of `pos` over the first n columns (turns: fp64 turns per
    position of every column pair)."""
    _req(ids.dtype == I32 and ids.is_cuda and ids.is_contiguous() and table.is_contiguous(), "ids int32, table dense")
    V, W = table.shape
    f32 = _act(table, "table")
    if carry is not None:
        _req(carry.dtype == I32 and prev.dtype == I32 and carry.numel() >= ids.numel(), "carry int32")
    if pos is not None:
        _vec(pos, ids.numel(), I32, "pos")
        _vec(turns, (n + 1) // 2, torch.float64, "turns")
    h = torch.empty((ids.numel(), W), dtype=F32, device=table.device)
    check(_lib.lib().ragk_embed_residual(ids.data_ptr(), table.data_ptr(), h.data_ptr(), ids.numel(), W, V, ptr(carry),
                                         ptr(prev) if carry is not None else None, float(scale), n, ptr(pos),
                                         ptr(turns) if pos is not None else None, f32, stream_ptr()),
          "ragk_embed_residual")
    return h


def _slabs(y, M, W, name):
    """(rows are bf16, number of slabs) of rows [M, W] or fp32 slabs [S, M, W]."""
    _req(y.is_cuda and y.dtype in (BF16, F32) and y.is_contiguous() and y.shape[-2:] == (M, W) and y.dim() in (2, 3), name)
    bf, S = int(y.dtype == BF16), y.shape[0] if y.dim() == 3 else 1
    _req(S == 1 or not bf, "bf16 rows come as one slab")
    return bf, S


def _shift_state(mix, state, meta, M, W):
    _vec(mix, W, F32, "mix")
    _req(state.dtype == F32 and state.is_contiguous() and state.dim() == 2 and state.shape[1] == W, "shift state")
    S = meta.kv_lens.numel()
    _req(meta.states is not None and meta.states.dtype == I32 and meta.states.numel() == S, "state slots")
    _req(meta.kind != "decode" or S == M, "one token per sequence")
    return S


def gated_residual(h, y, z, zb, w, eps, n, out_dtype, keep=False, shift=None, meta=None):
    """h += norm(y * sigmoid(z + zb)) * w in place. y / z: rows, or fp32 slabs. Returns (h in out_dtype if `keep`,
    the token-shifted rows if `shift` = (mix, state), decode steps only)."""
    M, W = h.shape
    _req(h.is_cuda and h.dtype == F32 and h.is_contiguous() and W % 8 == 0 and W <= 16384, "h fp32 [M, W]")
    bf, S = _slabs(y, M, W, "y rows / slabs")
    SZ = 1
    if z is not None:
        bz, SZ = _slabs(z, M, W, "z rows / slabs")
        _req(bz == bf, "y and z of one type")
        _vec(zb, W, F32, "zb")
    _vec(w, W, F32, "w")
    out = torch.empty((M, W), dtype=out_dtype, device=h.device) if keep else None
    mix = state = xs = None
    if shift is not None:
        mix, state = shift
        _req(meta.kind == "decode", "shifted rows of a decode step")
        _shift_state(mix, state, meta, M, W)
        xs = torch.empty((M, W), dtype=out_dtype, device=h.device)
    check(_lib.lib().ragk_gated_residual(
        h.data_ptr(), y.data_ptr(), S, ptr(z), SZ, bf, ptr(zb) if z is not None else None, w.data_ptr(), ptr(out), ptr(mix),
        ptr(xs), ptr(state), meta.states.data_ptr() if shift is not None else None,
        meta.kv_lens.data_ptr() if shift is not None else None, int(out_dtype == F32), M, W, n, float(eps), stream_ptr()),
        "ragk_gated_residual")
    return out, xs


def token_shift(h, mix, state, meta, out_dtype, keep=True):
    """(h in out_dtype if `keep`, h[t] + (h[t - 1] - h[t]) * mix); the state holds each sequence's last row."""
    M, W = h.shape
    _req(h.is_cuda and h.dtype == F32 and h.is_contiguous() and W % 8 == 0, "h fp32 [M, W]")
    S = _shift_state(mix, state, meta, M, W)
    _, cu = _meta(meta, M, meta.kind == "decode")
    out = torch.empty((M, W), dtype=out_dtype, device=h.device) if keep else None
    xs = torch.empty((M, W), dtype=out_dtype, device=h.device)
    check(_lib.lib().ragk_token_shift(h.data_ptr(), M, W, mix.data_ptr(), state.data_ptr(), meta.states.data_ptr(), cu,
                                      meta.kv_lens.data_ptr(), S, ptr(out), xs.data_ptr(), int(out_dtype == F32),
                                      stream_ptr()), "ragk_token_shift")
    return out, xs


def residual_norm(h, y, w_post, w_next, eps, n, out_dtype):
    """h += norm(y) * w_post (in place), returns norm(h) * w_next in out_dtype. y: rows [M, W] (bf16 / fp32),
    fp32 slabs [S, M, W], or None."""
    M, W = h.shape
    _req(h.is_cuda and h.dtype == F32 and h.is_contiguous() and W % 8 == 0 and W <= 16384, "h fp32 [M, W]")
    S, bf, ldy = 1, 0, W
    if y is not None:
        _req(y.is_cuda and y.dtype in (BF16, F32) and y.is_contiguous() and y.shape[-2:] == (M, W), "y rows / slabs")
        bf = int(y.dtype == BF16)
        S = y.shape[0] if y.dim() == 3 else 1
        _req(S == 1 or not bf, "bf16 rows come as one slab")
    for w, name in ((w_post, "w_post"), (w_next, "w_next")):
        if w is not None:
            _vec(w, W, F32, name)
    out = torch.empty((M, W), dtype=out_dtype, device=h.device) if w_next is not None else None
    check(_lib.lib().ragk_residual_norm(h.data_ptr(), ptr(y), ldy, S, bf, ptr(w_post), ptr(w_next), ptr(out),
                                        int(out_dtype == F32), M, W, n, float(eps), stream_ptr()), "ragk_residual_norm")
    return out


def slab_rows(P, bias, dtype):
    S, M, N = P.shape
    _req(P.is_cuda and P.dtype == F32 and P.is_contiguous() and N % 8 == 0, "slabs fp32 [S, M, N]")
    if bias is not None:
        _vec(bias, N, dtype, "bias")
    out = torch.empty((M, N), dtype=dtype, device=P.device)
    check(_lib.lib().ragk_slab_rows(P.data_ptr(), S, ptr(bias), out.data_ptr(), M, N, int(dtype == F32), stream_ptr()),
          "ragk_slab_rows")
    return out


def gemm_f32(x, w, bias=None):
    _req(_act(x, "x") and _act(w, "w") and x.shape[1] == w.shape[1] and x.shape[1] % 32 == 0, "gemm_f32 operands")
    _req(x.stride(0) % 4 == 0 and w.stride(0) % 4 == 0, "gemm_f32 row strides")
    M, K = x.shape
    N = w.shape[0]
    if bias is not None:
        _vec(bias, N, F32, "bias")
    out = torch.empty((M, N), dtype=F32, device=x.device)
    check(_lib.lib().ragk_gemm_f32(x.data_ptr(), x.stride(0), w.data_ptr(), w.stride(0), out.data_ptr(), N, ptr(bias), M, N,
                                   K, stream_ptr()), "ragk_gemm_f32")
    return out


def glu_clip_f32(x, par):
    _req(_act(x, "x") and x.is_contiguous() and x.shape[1] % 128 == 0, "packed gate/up rows")
    _vec(par, 4, F32, "par")
    M, F = x.shape[0], x.shape[1] // 2
    out = torch.empty((M, F), dtype=F32, device=x.device)
    check(_lib.lib().ragk_glu_clip(x.data_ptr(), out.data_ptr(), M, F, par.data_ptr(), stream_ptr()), "ragk_glu_clip")
    return out


# ------------------------------------------------------------------------------------- work lists
def query_tiles(q_lens, qt):
    """(seq, first query) work list of qt-row query tiles, latest (heaviest) first."""
    ql = np.asarray(q_lens, dtype=np.int64)
    nt = (ql + qt - 1) // qt
    seq = np.repeat(np.arange(len(ql)), nt)
    first = np.repeat(np.cumsum(nt) - nt, nt)
    q0 = (np.arange(int(nt.sum())) - first) * qt
    order = np.argsort(-q0, kind="stable")
    return torch.from_numpy(np.stack([seq[order], q0[order]], 1).astype(np.int32)).reshape(-1, 2)


DECODE_TARGET_BLOCKS = 512  # decode attention grid: partitions x KV heads x batch
DECODE_MIN_PAGES = 4


def decode_parts(spec, max_kv_len, batch):
    """Partitions per (sequence, KV head): the pages a query can visit, spread to fill the chip."""
    pages = -(-max_kv_len // 64)
    if spec.window > 0:
        pages = min(pages, -(-spec.keep_first // 64) + -(-spec.window // 64) + 1)
    rows = batch * spec.kv_heads * -(-spec.group // 16)
    return max(1, min(-(-DECODE_TARGET_BLOCKS // rows), -(-pages // DECODE_MIN_PAGES)))


def decode_split(specs, max_kv_len, batch, device):
    """(min pages per partition, 1, partition sums, partition statistics): one workspace all layers share."""
    need = [(batch * s.heads * p, s.dvp) for s in specs for p in [decode_parts(s, max_kv_len, batch)] if p > 1]
    if not need:
        return DECODE_MIN_PAGES, 1, None, None
    f32 = dict(dtype=F32, device=device)
    return (DECODE_MIN_PAGES, 1, torch.empty(max(r * d for r, d in need), **f32),
            torch.empty(max(r for r, _ in need) * 2, **f32))


# ------------------------------------------------------------------------------------- shaped attention
def _caches(kc, vc, spec, dtype):
    _req(kc.dim() == 4 and kc.shape[1:] == (spec.kv_heads, 64, spec.dkp) and kc.is_contiguous() and kc.dtype == dtype,
         "K pages [blocks, kv_heads, 64, dk]")
    _req(vc.shape == (kc.shape[0], spec.kv_heads, 64, spec.dvp) and vc.is_contiguous() and vc.dtype == dtype,
         "V pages [blocks, kv_heads, 64, dv]")


def kv_store(row, spec, slots, kc, vc, v_first=None, lam=None):
    """k and (mixed) v of each token into the pages at `slots`; returns the tokens' own values (a view)."""
    f32 = _act(row, "row")
    T = row.shape[0]
    _req(row.shape[1] >= spec.off_g and row.stride(0) % 8 == 0, "projection rows")
    _req(slots.dtype == I32 and slots.is_contiguous() and slots.numel() == T, "slots int32[T]")
    _caches(kc, vc, spec, row.dtype)
    ldf = 0
    if v_first is not None:
        _req(v_first.dtype == row.dtype and v_first.shape == (T, spec.kv_heads * spec.dvp) and v_first.stride(1) == 1
             and v_first.data_ptr() % 16 == 0, "v_first rows")
        _vec(lam, 1, F32, "lam")
        ldf = v_first.stride(0)
    check(_lib.lib().ragk_shaped_kv_store(row.data_ptr(), row.stride(0), spec.off_k, spec.off_v, T, spec.kv_heads, spec.dkp,
                                          spec.dvp, slots.data_ptr(), kc.data_ptr(), vc.data_ptr(), ptr(v_first), ldf,
                                          ptr(lam) if v_first is not None else None, f32, stream_ptr()),
          "ragk_shaped_kv_store")
    return row[:, spec.off_v:spec.off_g]


def _table(table, spec):
    if table is not None:
        _vec(table.reshape(-1), spec.heads * (spec.far + 1), F32, "bias table")


def _meta(meta, T, decode):
    S = meta.kv_lens.numel()
    _req(meta.kv_lens.dtype == I32 and meta.block_tables.dtype == I32 and meta.block_tables.shape[0] == S
         and meta.block_tables.stride(1) == 1, "kv_lens / block tables int32")
    if decode:
        _req(S == T, "one token per sequence")
    else:
        _req(meta.cu_q is not None and meta.cu_q.dtype == I32 and meta.cu_q.numel() == S + 1, "cu_q int32[S + 1]")
    return S, None if decode else meta.cu_q.data_ptr()


def attn_rows(row, spec, table, kc, vc, meta, out):
    """Plain attention, one wave per (token, head): any head size, bf16 or fp32."""
    f32 = _act(row, "row")
    T = row.shape[0]
    S, cu = _meta(meta, T, meta.kind == "decode")
    _caches(kc, vc, spec, row.dtype)
    _table(table, spec)
    _req(out.dtype == row.dtype and out.shape == (T, spec.out_row) and out.is_contiguous(), "out rows")
    check(_lib.lib().ragk_shaped_attn_rows(
        row.data_ptr(), row.stride(0), kc.data_ptr(), vc.data_ptr(), meta.block_tables.data_ptr(),
        meta.block_tables.stride(0), cu, meta.kv_lens.data_ptr(), ptr(table), out.data_ptr(), out.stride(0), T, S,
        spec.heads, spec.kv_heads, spec.dkp, spec.dvp, spec.off_g if spec.gate else -1, spec.window, spec.keep_first,
        spec.far, int(spec.sink), float(spec.scale), float(spec.softcap), f32, stream_ptr()), "ragk_shaped_attn_rows")
    return out


def attn_prefill(row, spec, table, kc, vc, meta, out):
    """MFMA prefill attention over the pages (bf16)."""
    T = row.shape[0]
    _req(_act(row, "row") == 0, "bf16 rows")
    S, cu = _meta(meta, T, False)
    _caches(kc, vc, spec, row.dtype)
    _table(table, spec)
    tiles = meta.qtiles[spec.q_tile]
    _req(tiles.dtype == I32 and tiles.is_cuda and tiles.is_contiguous(), "query tiles")
    _req(out.dtype == row.dtype and out.shape == (T, spec.out_row) and out.is_contiguous(), "out rows")
    _req(meta.block_tables.stride(0) <= 2048, "block tables wider than 2048 blocks (128k tokens)")
    check(_lib.lib().ragk_shaped_attn_prefill(
        row.data_ptr(), row.stride(0), kc.data_ptr(), vc.data_ptr(), meta.block_tables.data_ptr(),
        meta.block_tables.stride(0), cu, meta.kv_lens.data_ptr(), tiles.data_ptr(), tiles.shape[0], spec.heads_per_block,
        ptr(table), out.data_ptr(), out.stride(0), spec.heads, spec.kv_heads, spec.dkp, spec.dvp,
        spec.off_g if spec.gate else -1, spec.window, spec.keep_first, spec.far, int(spec.sink), int(spec.bounded),
        float(spec.scale), float(spec.softcap), stream_ptr()), "ragk_shaped_attn_prefill")
    return out


def attn_decode(P, bias, spec, table, slots, kc, vc, meta, out, v_first=None, lam=None):
    """One new token per sequence from projection slabs (bf16 caches): value mix, cache append, attention, gate.
    Returns the tokens' own values [B, kv_heads * dv] (fp32)."""
    S, B, N = P.shape
    _req(P.is_cuda and P.dtype == F32 and P.is_contiguous() and N >= spec.off_g + (spec.heads if spec.gate else 0), "slabs")
    _meta(meta, B, True)
    _caches(kc, vc, spec, BF16)
    _table(table, spec)
    _req(slots.dtype == I32 and slots.is_contiguous() and slots.numel() == B, "slots int32[B]")
    _req(out.dtype == BF16 and out.shape == (B, spec.out_row) and out.is_contiguous(), "out rows")
    if bias is not None:
        _vec(bias, N, BF16, "bias")
    nv = spec.kv_heads * spec.dvp
    if v_first is not None:
        _req(v_first.dtype == F32 and v_first.shape == (B, nv) and v_first.is_contiguous(), "v_first fp32 [B, values]")
        _vec(lam, 1, F32, "lam")
    own = torch.empty((B, nv), dtype=F32, device=P.device)
    parts = decode_parts(spec, meta.max_kv, B) if meta.ws_o is not None else 1
    if parts > 1:
        _req(meta.ws_o.numel() >= B * spec.heads * parts * spec.dvp and meta.ws_ml.numel() >= B * spec.heads * parts * 2,
             "decode workspace too small")
    check(_lib.lib().ragk_shaped_attn_decode(
        P.data_ptr(), S, N, ptr(bias), kc.data_ptr(), vc.data_ptr(), meta.block_tables.data_ptr(),
        meta.block_tables.stride(0), meta.kv_lens.data_ptr(), slots.data_ptr(), ptr(table), ptr(v_first),
        ptr(lam) if v_first is not None else None, own.data_ptr(), out.data_ptr(), out.stride(0), ptr(meta.ws_o),
        ptr(meta.ws_ml), B, spec.heads, spec.kv_heads, spec.dkp, spec.dvp, spec.off_k, spec.off_v,
        spec.off_g if spec.gate else -1, spec.window, spec.keep_first, spec.far, int(spec.sink), DECODE_MIN_PAGES, parts,
        float(spec.scale), float(spec.softcap), stream_ptr()), "ragk_shaped_attn_decode")
    return own


# ------------------------------------------------------------------------------------- latent attention
KEY_PAD = 64  # zero rows behind packed key rows: attention reads whole 64-row groups
LATENT_TARGET_BLOCKS = 256  # a decode block fills a CU's LDS
LATENT_MIN_TOKENS = 128  # of a partition
LATENT_MAX_PARTS = 64


@dataclass
class KeyRows:
    """Packed key rows of a prefill step for one window: sequence s of the first `seqs` holds positions
    first .. kv_len - 1 in rows key_off[s] + position. `gather`: rows come from the pages (a sequence continues);
    otherwise they are the step's own rows in order. The `tail` sequences behind them bring one token each and
    attend like decode rows."""
    key_off: torch.Tensor  # int32 [S]
    cu_k: torch.Tensor  # int32 [seqs + 1]
    tiles: torch.Tensor  # query tiles of the first `seqs` sequences
    rows: int
    seqs: int
    tail: int
    gather: bool


def key_rows(q_lens, kv_lens, window, device):
    ql, kl = np.asarray(q_lens, dtype=np.int64), np.asarray(kv_lens, dtype=np.int64)
    one = (ql == 1) & (kl > 1)
    tail = len(ql) if one.all() else int(np.argmin(one[::-1]))
    n = len(ql) - tail
    ctx = (kl - ql)[:n]
    first = np.maximum(0, ctx - window + 1) // 64 * 64 if window > 0 else np.zeros_like(ctx)
    cu = np.concatenate([[0], np.cumsum(kl[:n] - first)])
    off = np.zeros(len(ql), dtype=np.int64)
    off[:n] = cu[:n] - first
    i32 = lambda x: torch.from_numpy(x.astype(np.int32)).to(device)  # noqa: E731
    return KeyRows(i32(off), i32(cu), query_tiles(ql[:n], LatentSpec.q_tile).to(device), int(cu[-1]), n, tail,
                   bool((ctx > 0).any()))


def latent_tile(spec):
    """Tokens of one LDS tile of the decode kernel (its LatentTile)."""
    return 64 if spec.rp <= 256 else 32


def latent_min_tiles(spec):
    return LATENT_MIN_TOKENS // latent_tile(spec)


def latent_split(spec, max_kv_len, batch):
    """(partitions per sequence, query heads per block) of a decode step."""
    tt = latent_tile(spec)
    tiles = -(-max_kv_len // tt)
    if spec.window > 0:
        tiles = min(tiles, -(-spec.window // tt) + 1)
    most = min(-(-tiles // latent_min_tiles(spec)), LATENT_MAX_PARTS)
    wide = spec.rp <= 512 and spec.heads > 16 and batch * -(-spec.heads // 32) * most >= LATENT_TARGET_BLOCKS
    heads = 32 if wide else 16
    return min(-(-LATENT_TARGET_BLOCKS // (batch * -(-spec.heads // heads))), most), heads


def latent_parts(spec, max_kv_len, batch):
    return latent_split(spec, max_kv_len, batch)[0]


def latent_workspace(specs, max_kv_len, batch, device):
    """(partial latents, partial statistics) of one decode step, shared by all layers."""
    n = max(batch * s.heads * latent_parts(s, max_kv_len, batch) * s.rp for s in specs)
    m = max(batch * s.heads * latent_parts(s, max_kv_len, batch) for s in specs)
    f32 = dict(dtype=F32, device=device)
    return torch.empty(n, **f32), torch.empty(2 * m, **f32)


def _pages(pages, spec, dtype):
    _req(pages.dim() == 3 and pages.shape[1:] == (64, spec.rp) and pages.is_contiguous() and pages.dtype == dtype,
         "latent pages [blocks, 64, rp]")


def latent_store(row, spec, norm, eps, slots, pages, keep=True):
    """Normed latents of every token into the pages at `slots`; returns them as rows [T + KEY_PAD, rp] if `keep`."""
    f32 = _act(row, "row")
    T = row.shape[0]
    _req(spec.own and row.shape[1] >= spec.off_c + spec.rp and row.stride(0) % 8 == 0, "projection rows")
    _req(slots.dtype == I32 and slots.is_contiguous() and slots.numel() == T, "slots int32[T]")
    _vec(norm, spec.rp, F32, "latent norm")
    _pages(pages, spec, row.dtype)
    out = torch.empty((T + KEY_PAD, spec.rp), dtype=row.dtype, device=row.device) if keep else None
    check(_lib.lib().ragk_latent_store(row.data_ptr(), row.stride(0), spec.off_c, spec.rank, spec.rp, norm.data_ptr(),
                                       float(eps), slots.data_ptr(), pages.data_ptr(), ptr(out), T, KEY_PAD, f32,
                                       stream_ptr()), "ragk_latent_store")
    return out


def latent_gather(pages, spec, meta, kr):
    """Packed latent rows [kr.rows + KEY_PAD, rp] of the visible tokens of a step's sequences."""
    _pages(pages, spec, pages.dtype)
    _req(meta.block_tables.dtype == I32 and meta.block_tables.shape[0] >= kr.seqs and kr.cu_k.numel() == kr.seqs + 1
         and kr.key_off.numel() >= kr.seqs, "key rows")
    out = torch.empty((kr.rows + KEY_PAD, spec.rp), dtype=pages.dtype, device=pages.device)
    check(_lib.lib().ragk_latent_gather(pages.data_ptr(), spec.rp, meta.block_tables.data_ptr(), meta.block_tables.stride(0),
                                        kr.cu_k.data_ptr(), kr.key_off.data_ptr(), kr.seqs, kr.rows, KEY_PAD, out.data_ptr(),
                                        int(pages.dtype == F32), stream_ptr()), "ragk_latent_gather")
    return out


def row_attention(row, spec, kv, kr, meta, out):
    """Attention of the first kr.seqs sequences' tokens over expanded key / value rows, output gates applied."""
    f32 = _act(row, "row")
    T = row.shape[0]
    S, cu = _meta(meta, T, False)
    _req(kv.dtype == row.dtype and kv.dim() == 2 and kv.is_contiguous() and kv.shape[1] == spec.kv_row
         and kv.shape[0] >= kr.rows + KEY_PAD and kr.key_off.numel() == S, "key / value rows")
    _req(row.shape[1] >= spec.off_c, "projection rows")
    _req(out.dtype == row.dtype and out.shape == (T, spec.out_row) and out.is_contiguous(), "out rows")
    if f32:
        n = T - kr.tail
        check(_lib.lib().ragk_row_attn_rows(
            row.data_ptr(), row.stride(0), kv.data_ptr(), kv.stride(0), spec.off_v, kr.key_off.data_ptr(), cu,
            meta.kv_lens.data_ptr(), out.data_ptr(), out.stride(0), n, S, spec.heads, spec.dkp, spec.dvp, spec.off_g,
            spec.window, float(spec.scale), 1, stream_ptr()), "ragk_row_attn_rows")
        return out
    tiles = kr.tiles
    _req(tiles.dtype == I32 and tiles.is_cuda and tiles.is_contiguous(), "query tiles")
    check(_lib.lib().ragk_row_attn_prefill(
        row.data_ptr(), row.stride(0), kv.data_ptr(), kv.stride(0), spec.off_v, kr.key_off.data_ptr(), cu,
        meta.kv_lens.data_ptr(), tiles.data_ptr(), tiles.shape[0], out.data_ptr(), out.stride(0), spec.heads, spec.dkp,
        spec.dvp, spec.off_g, spec.window, meta.block_tables.stride(0), float(spec.scale), stream_ptr()),
        "ragk_row_attn_prefill")
    return out


def _proj(P, spec, own):
    """(bf16 rows?, slabs, B, leading dimension) of projection slabs [S, B, N] (fp32) or rows [B, N] (bf16)."""
    rows = P.dim() == 2
    S, (B, N) = 1 if rows else P.shape[0], P.shape[-2:]
    _req(P.is_cuda and P.dtype == (BF16 if rows else F32) and P.stride(-1) == 1 and (rows or P.is_contiguous())
         and N >= spec.off_c + (spec.rp if own else 0), "projection slabs / rows")
    return int(rows), S, B, P.stride(0) if rows else N


def _partials(spec, meta, B, ws):
    ws_o, ws_ml = ws if ws is not None else (meta.ws_o, meta.ws_ml)
    parts, heads = latent_split(spec, meta.max_kv, B)
    _req(ws_o.dtype == F32 and ws_ml.dtype == F32 and ws_o.numel() >= B * spec.heads * parts * spec.rp
         and ws_ml.numel() >= B * spec.heads * parts * 2, "decode workspace too small")
    return ws_o, ws_ml, parts, heads


def latent_absorb(P, spec, wuk, pages=None, slots=None, norm=None, eps=0.0):
    """Queries into latent space, qa [B, H, rp]; with `slots`, the tokens' normed latents into the pages too."""
    own = slots is not None
    rows, S, B, ld = _proj(P, spec, own)
    _req(wuk.dtype == BF16 and wuk.is_contiguous() and wuk.shape == (spec.heads, spec.rp, spec.dkp), "wuk [H, rp, dkp]")
    if own:
        _pages(pages, spec, BF16)
        _req(slots.dtype == I32 and slots.is_contiguous() and slots.numel() == B, "slots int32[B]")
        _vec(norm, spec.rp, F32, "latent norm")
    qa = torch.empty((B, spec.heads, spec.rp), dtype=BF16, device=P.device)
    check(_lib.lib().ragk_latent_absorb(P.data_ptr(), rows, S, ld, B, spec.heads, spec.dkp, spec.rank, spec.rp,
                                        spec.off_c if own else 0, wuk.data_ptr(), qa.data_ptr(), ptr(pages) if own else None,
                                        ptr(slots), ptr(norm) if own else None, float(eps), stream_ptr()),
          "ragk_latent_absorb")
    return qa


def latent_attend(qa, spec, pages, meta, ws=None):
    """Attention of one query per sequence and head over the latent pages, left as partitions in the workspace."""
    B = qa.shape[0]
    _req(qa.is_cuda and qa.dtype == BF16 and qa.is_contiguous() and qa.shape == (B, spec.heads, spec.rp), "qa [B, H, rp]")
    _meta(meta, B, True)
    _pages(pages, spec, BF16)
    ws_o, ws_ml, parts, heads = _partials(spec, meta, B, ws)
    check(_lib.lib().ragk_latent_decode(
        qa.data_ptr(), pages.data_ptr(), meta.block_tables.data_ptr(), meta.block_tables.stride(0), meta.kv_lens.data_ptr(),
        ws_o.data_ptr(), ws_ml.data_ptr(), B, spec.heads, spec.rp, spec.window, latent_min_tiles(spec), parts, heads,
        float(spec.scale), stream_ptr()), "ragk_latent_decode")


def latent_out(P, spec, wuv, meta, out, ws=None):
    """Joined partitions through the value map, times the output gates of P, into `out` rows."""
    rows, S, B, ld = _proj(P, spec, False)
    _meta(meta, B, True)
    _req(wuv.dtype == BF16 and wuv.is_contiguous() and wuv.shape == (spec.heads, spec.dvp, spec.rp), "wuv [H, dvp, rp]")
    _req(out.dtype == BF16 and out.shape == (B, spec.out_row) and out.stride(1) == 1, "out rows")
    ws_o, ws_ml, parts, _ = _partials(spec, meta, B, ws)
    check(_lib.lib().ragk_latent_out(P.data_ptr(), rows, S, ld, spec.off_g, ws_o.data_ptr(), ws_ml.data_ptr(),
                                     meta.kv_lens.data_ptr(), wuv.data_ptr(), out.data_ptr(), out.stride(0), B, spec.heads,
                                     spec.dvp, spec.rp, spec.window, latent_min_tiles(spec), parts, stream_ptr()),
          "ragk_latent_out")
    return out


def latent_decode(P, spec, wuk, wuv, pages, meta, out, slots=None, norm=None, eps=0.0, ws=None):
    """One new token per sequence from projection slabs or rows: queries into latent space, cache append (with
    `slots`), attention over the latent pages, value map, output gate (bf16 caches)."""
    qa = latent_absorb(P, spec, wuk, pages, slots, norm, eps)
    latent_attend(qa, spec, pages, meta, ws)
    return latent_out(P, spec, wuv, meta, out, ws)


def latent_decode_rows(row, spec, wuk, wuv, pages, meta, out):
    """The same from fp32 rows with plain fp32 arithmetic (exact replay); the tokens' latents are in the pages."""
    B = row.shape[0]
    _req(_act(row, "row") == 1 and row.shape[1] >= spec.off_c, "projection rows")
    _meta(meta, B, True)
    _pages(pages, spec, F32)
    _req(wuk.dtype == F32 and wuk.is_contiguous() and wuk.shape == (spec.heads, spec.rp, spec.dkp), "wuk [H, rp, dkp]")
    _req(wuv.dtype == F32 and wuv.is_contiguous() and wuv.shape == (spec.heads, spec.dvp, spec.rp), "wuv [H, dvp, rp]")
    _req(out.dtype == F32 and out.shape == (B, spec.out_row) and out.stride(1) == 1, "out rows")
    H, L = spec.heads, _lib.lib()
    qa = torch.empty((B, H * spec.rp), dtype=F32, device=row.device)
    oc = torch.empty_like(qa)
    check(L.ragk_head_proj_f32(row.data_ptr(), row.stride(0), spec.dkp, wuk.data_ptr(), spec.rp, None, 0, qa.data_ptr(),
                               qa.stride(0), B, H, stream_ptr()), "ragk_head_proj_f32")
    check(L.ragk_shaped_attn_rows(qa.data_ptr(), qa.stride(0), pages.data_ptr(), pages.data_ptr(),
                                  meta.block_tables.data_ptr(), meta.block_tables.stride(0), None, meta.kv_lens.data_ptr(),
                                  None, oc.data_ptr(), oc.stride(0), B, B, H, 1, spec.rp, spec.rp, -1, spec.window, 0, 0, 0,
                                  float(spec.scale), 0.0, 1, stream_ptr()), "ragk_shaped_attn_rows")
    g = row[:, spec.off_g:]
    check(L.ragk_head_proj_f32(oc.data_ptr(), oc.stride(0), spec.rp, wuv.data_ptr(), spec.dvp, g.data_ptr(), row.stride(0),
                               out.data_ptr(), out.stride(0), B, H, stream_ptr()), "ragk_head_proj_f32")
    return out


# ------------------------------------------------------------------------------------- state space
def _states(meta, spec, conv_state, ssm_state):
    n = ssm_state.shape[0]
    _req(meta.states is not None and meta.states.dtype == I32 and meta.states.numel() == meta.kv_lens.numel(), "state slots")
    _req(ssm_state.dtype == F32 and ssm_state.is_contiguous()
         and ssm_state.shape == (n, spec.heads, spec.state, spec.vdim), "ssm_state")
    _req(conv_state.dtype == F32 and conv_state.is_contiguous() and conv_state.shape == (n, spec.taps - 1, spec.channels),
         "conv_state")


def ssm_conv(row, spec, w, meta, conv_state, ssm_state):
    f32 = _act(row, "row")
    T = row.shape[0]
    S, cu = _meta(meta, T, meta.kind == "decode")
    _states(meta, spec, conv_state, ssm_state)
    _req(row.shape[1] >= spec.off_dt + spec.heads, "projection rows")
    _vec(w["conv_w"].reshape(-1), spec.taps * spec.channels, F32, "conv_w")
    _vec(w["conv_b"], spec.channels, F32, "conv_b")
    xbc = torch.empty((T, spec.channels), dtype=row.dtype, device=row.device)
    check(_lib.lib().ragk_ssm_conv(cu, meta.kv_lens.data_ptr(), meta.states.data_ptr(), T, S, row.data_ptr(), row.stride(0),
                                   spec.off_x, w["conv_w"].data_ptr(), w["conv_b"].data_ptr(), conv_state.data_ptr(),
                                   xbc.data_ptr(), spec.channels, spec.taps, f32, stream_ptr()), "ragk_ssm_conv")
    return xbc


def ssm_scan_seq(xbc, row, spec, w, meta, ssm_state):
    f32 = _act(row, "row")
    T = row.shape[0]
    S, cu = _meta(meta, T, meta.kind == "decode")
    for k in ("dt_bias", "A", "D"):
        _vec(w[k], spec.heads, F32, k)
    y = torch.empty((T, spec.inner), dtype=F32, device=row.device)
    check(_lib.lib().ragk_ssm_scan_seq(cu, meta.kv_lens.data_ptr(), meta.states.data_ptr(), T, S, xbc.data_ptr(),
                                       xbc.stride(0), row.data_ptr(), row.stride(0), spec.off_dt, w["dt_bias"].data_ptr(),
                                       w["A"].data_ptr(), w["D"].data_ptr(), ssm_state.data_ptr(), y.data_ptr(), spec.heads,
                                       spec.vdim, spec.state, spec.groups, f32, stream_ptr()), "ragk_ssm_scan_seq")
    return y


def scan_chunk_ok(spec):
    return spec.vdim % 8 == 0 and spec.state % 8 == 0 and spec.state <= 256


def ssm_scan_chunk(xbc, row, spec, w, meta, ssm_state):
    """MFMA chunked scan of packed prompts (bf16)."""
    _req(_act(row, "row") == 0 and xbc.dtype == BF16 and xbc.is_contiguous() and scan_chunk_ok(spec), "chunk scan operands")
    T = row.shape[0]
    S, cu = _meta(meta, T, meta.kind == "decode")
    _req(xbc.shape == (T, spec.channels), "xbc rows")
    for k in ("dt_bias", "A", "D"):
        _vec(w[k], spec.heads, F32, k)
    y = torch.empty((T, spec.inner), dtype=BF16, device=row.device)
    check(_lib.lib().ragk_ssm_scan_chunk(cu, meta.kv_lens.data_ptr(), meta.states.data_ptr(), T, S, xbc.data_ptr(),
                                         xbc.stride(0), row.data_ptr(), row.stride(0), spec.off_dt, w["dt_bias"].data_ptr(),
                                         w["A"].data_ptr(), w["D"].data_ptr(), ssm_state.data_ptr(), y.data_ptr(),
                                         spec.heads, spec.vdim, spec.state, spec.groups, stream_ptr()),
          "ragk_ssm_scan_chunk")
    return y


def ssm_decode_ok(spec):
    return spec.vdim % 4 == 0 and spec.vdim <= 256 and spec.state % 4 == 0


def ssm_decode(P, spec, w, meta, conv_state, ssm_state):
    """One token per sequence from projection slabs: convolution, state update, gate. Returns y * silu(z), fp32."""
    S, B, N = P.shape
    _req(P.is_cuda and P.dtype == F32 and P.is_contiguous() and N >= spec.off_dt + spec.heads and ssm_decode_ok(spec),
         "slabs")
    _meta(meta, B, True)
    _states(meta, spec, conv_state, ssm_state)
    _vec(w["conv_w"].reshape(-1), spec.taps * spec.channels, F32, "conv_w")
    _vec(w["conv_b"], spec.channels, F32, "conv_b")
    for k in ("dt_bias", "A", "D"):
        _vec(w[k], spec.heads, F32, k)
    act = torch.empty((B, N), dtype=F32, device=P.device)
    yz = torch.empty((B, spec.inner), dtype=F32, device=P.device)
    check(_lib.lib().ragk_ssm_decode(P.data_ptr(), S, N, meta.kv_lens.data_ptr(), meta.states.data_ptr(),
                                     w["conv_w"].data_ptr(), w["conv_b"].data_ptr(), w["dt_bias"].data_ptr(),
                                     w["A"].data_ptr(), w["D"].data_ptr(), conv_state.data_ptr(), ssm_state.data_ptr(),
                                     act.data_ptr(), yz.data_ptr(), B, spec.heads, spec.vdim, spec.state, spec.groups,
                                     spec.taps, stream_ptr()), "ragk_ssm_decode")
    return yz


def ssm_gate_norm(y, row, spec, w, eps, out):
    """group_norm(y * silu(z)) * w; z = row[:, :inner], or None when y is gated already."""
    f32 = int(out.dtype == F32)
    T = y.shape[0]
    _req(y.dtype in (BF16, F32) and y.is_contiguous() and y.shape == (T, spec.inner), "y [T, inner]")
    if row is not None:
        _req(row.dtype == out.dtype and row.shape[0] == T and row.stride(1) == 1, "projection rows")
    _req(out.is_cuda and out.shape == (T, spec.out_row) and out.is_contiguous(), "out rows")
    _vec(w["norm"], spec.inner, F32, "norm")
    check(_lib.lib().ragk_ssm_gate_norm(y.data_ptr(), int(y.dtype == BF16), ptr(row), row.stride(0) if row is not None else 0,
                                        w["norm"].data_ptr(), out.data_ptr(), out.stride(0), T, spec.inner,
                                        spec.norm_groups, float(eps), f32, stream_ptr()), "ragk_ssm_gate_norm")
    return out
