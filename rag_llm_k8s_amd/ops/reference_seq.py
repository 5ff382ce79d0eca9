"""CPU forms of the residual-stream, shaped-attention, latent-attention and state-space kernels (torch, fp32 arithmetic).

Same operands and memory layouts as the GPU kernels in csrc/kernels/residual.hip, attn_shaped.hip and ssm.hip:
paged caches [blocks, kv_heads, 64, size], per-sequence state slots, fused projection rows (ops/specs.py).
"""
from __future__ import annotations

import math

import torch
import torch.nn.functional as F

from .reference import paged_kv_view

BLOCK = 64


def rms(x, w, eps, n):
    """fp32 RMS norm over the first n columns (padding columns hold zeros)."""
    x = x.float()
    return x * torch.rsqrt(x.pow(2).sum(-1, keepdim=True) / n + eps) * w


def residual_norm(h, y, w_post, w_next, eps, n, out_dtype):
    """h (fp32, in place) += norm(y) * w_post (plain y without w_post); returns norm(h) * w_next."""
    if y is not None:
        y = y.float().sum(0) if y.dim() == 3 else y.float()
        h += rms(y, w_post, eps, n) if w_post is not None else y
    return None if w_next is None else rms(h, w_next, eps, n).to(out_dtype)


def sinusoid(pos, turns, n, width):
    """[T, width]: sin / cos of pos * turns[i] whole turns at columns 2i / 2i + 1 below n, zero from there."""
    a = pos.double()[:, None] * turns.double()[None, :]
    a = 2 * math.pi * (a - torch.round(a))
    out = torch.zeros(pos.numel(), width)
    out[:, 0:n:2] = torch.sin(a).float()
    out[:, 1:n:2] = torch.cos(a).float()[:, :n // 2]
    return out


def gated_residual(h, y, z, zb, w, eps, n):
    """h (fp32, in place) += norm(y * sigmoid(z + zb)) * w."""
    y = rows_of(y, None)
    if z is not None:
        y = y * torch.sigmoid(rows_of(z, zb))
    h += rms(y, w, eps, n)


def token_shift(h, mix, state, q_lens, kv_lens, states):
    """h[t] + (h[t - 1] - h[t]) * mix per sequence; state[slot] holds the row before the first and takes the last."""
    out, t0 = torch.empty_like(h), 0
    for s, (ql, L) in enumerate(zip(q_lens, kv_lens)):
        slot, x = int(states[s]), h[t0:t0 + ql]
        before = torch.zeros_like(x[:1]) if L == ql else state[slot][None].clone()
        out[t0:t0 + ql] = x + (torch.cat([before, x[:-1]]) - x) * mix
        state[slot] = x[-1]
        t0 += ql
    return out


def latent_store(row, spec, norm, eps, slots, pages):
    c = rms(row[:, spec.off_c:spec.off_c + spec.rp], norm, eps, spec.rank).to(pages.dtype)
    s = slots.long()
    ok = s >= 0
    pages[s[ok] // BLOCK, s[ok] % BLOCK] = c[ok]


def latent_attention(row, spec, wuk, wuv, pages, block_tables, q_lens, kv_lens, out):
    """Queries are the last q_lens[s] positions of each context; wuk [H, rp, dkp], wuv [H, dvp, rp]."""
    H, t0 = spec.heads, 0
    out.zero_()
    uk, uv = wuk.float(), wuv.float().transpose(1, 2).contiguous()
    for s, (ql, L) in enumerate(zip(q_lens, kv_lens)):
        q = row[t0:t0 + ql, :spec.off_g].float().reshape(ql, H, spec.dkp).transpose(0, 1).contiguous()
        c = paged_kv_view(pages[:, None], block_tables[s], L, BLOCK).float()[:, 0]
        k, v = torch.matmul(c, uk), torch.matmul(c, uv)  # [H, L, dkp], [H, L, dvp]
        sc = (q @ k.transpose(1, 2).contiguous()) * spec.scale
        i, j = torch.arange(L - ql, L)[:, None], torch.arange(L)[None, :]
        ok = j <= i
        if spec.window > 0:
            ok = ok & (i - j < spec.window)
        o = (torch.softmax(sc.masked_fill(~ok, -math.inf), -1) @ v).transpose(0, 1).reshape(ql, -1)
        o = o * torch.sigmoid(row[t0:t0 + ql, spec.off_g:spec.off_c].float())
        out[t0:t0 + ql, :H * spec.dvp] = o.to(out.dtype)
        t0 += ql
    return out


def glu_clip(g, u, par):
    """min(g, limit) * sigmoid(alpha g) * (clamp(u, +-limit) + shift), par = [limit, alpha, shift]."""
    limit, alpha, shift = (float(x) for x in par[:3])
    g = g.clamp(max=limit)
    return g * torch.sigmoid(alpha * g) * (u.clamp(-limit, limit) + shift)


def rows_of(P, bias):
    """Projection rows in fp32: split-K slabs [S, M, N] summed (+ bias), or plain rows."""
    x = P.float().sum(0) if P.dim() == 3 else P.float()
    return x if bias is None else x + bias.float()


def kv_store(row, spec, slots, kc, vc, v_first, lam):
    """k and (mixed) v of every token into the paged caches; returns the token's own values."""
    T = row.shape[0]
    k = row[:, spec.off_k:spec.off_v].reshape(T, spec.kv_heads, spec.dkp)
    own = row[:, spec.off_v:spec.off_g]
    v = own.float()
    if v_first is not None:
        lm = float(lam)
        v = (1.0 - lm) * v + lm * v_first.float()
    v = v.reshape(T, spec.kv_heads, spec.dvp)
    s = slots.long()
    ok = s >= 0
    s = s[ok]
    kc[s // BLOCK, :, s % BLOCK] = k[ok].to(kc.dtype)
    vc[s // BLOCK, :, s % BLOCK] = v[ok].to(vc.dtype)
    return own


def attention(row, spec, table, kc, vc, block_tables, q_lens, kv_lens, out):
    """Queries are the last q_lens[s] positions of each context."""
    H, G = spec.heads, spec.kv_heads
    t0 = 0
    out.zero_()
    for s, (ql, L) in enumerate(zip(q_lens, kv_lens)):
        q = row[t0:t0 + ql, :spec.off_k].float().reshape(ql, H, spec.dkp).transpose(0, 1)
        k = paged_kv_view(kc, block_tables[s], L, BLOCK).float().repeat_interleave(H // G, 1).transpose(0, 1)
        v = paged_kv_view(vc, block_tables[s], L, BLOCK).float().repeat_interleave(H // G, 1).transpose(0, 1)
        sc = (q @ k.transpose(1, 2).contiguous()) * spec.scale
        if spec.softcap > 0:
            sc = spec.softcap * torch.tanh(sc / spec.softcap)
        i = torch.arange(L - ql, L)[:, None]
        j = torch.arange(L)[None, :]
        if table is not None:
            sc = sc + table[:, (i - j).clamp(0, spec.far)]
        ok = j <= i
        if spec.window > 0:
            ok = ok & ((i - j < spec.window) | (j < spec.keep_first))
        sc = sc.masked_fill(~ok, -math.inf)
        if spec.sink:
            sc = torch.cat([sc, torch.zeros(H, ql, 1)], -1)
        p = torch.softmax(sc, -1)[..., :L]
        o = (p @ v).transpose(0, 1)  # [ql, H, dvp]
        if spec.gate:
            o = o * torch.sigmoid(row[t0:t0 + ql, spec.off_g:spec.off_g + H].float())[..., None]
        out[t0:t0 + ql, :H * spec.dvp] = o.reshape(ql, -1).to(out.dtype)
        t0 += ql
    return out


def ssm(row, spec, w, eps, q_lens, kv_lens, states, conv_state, ssm_state, out):
    """Short convolution, selective scan, gate and grouped norm for every sequence's new tokens."""
    H, P, N, G, K = spec.heads, spec.vdim, spec.state, spec.groups, spec.taps
    out.zero_()
    t0 = 0
    grp = torch.arange(H) // (H // G)
    for s, (ql, L) in enumerate(zip(q_lens, kv_lens)):
        slot = int(states[s])
        fresh = L == ql
        r = row[t0:t0 + ql].float()
        u = r[:, spec.off_x:spec.off_dt]
        past = torch.zeros_like(conv_state[slot]) if fresh else conv_state[slot].clone()
        full = torch.cat([past, u])
        y = w["conv_b"].expand(ql, -1).clone()
        for t in range(K):
            y = y + full[t:t + ql] * w["conv_w"][t]
        xbc = F.silu(y).to(row.dtype).float()
        if K > 1:
            conv_state[slot] = full[-(K - 1):]
        x = xbc[:, :spec.inner].reshape(ql, H, P)
        B = xbc[:, spec.inner:spec.inner + G * N].reshape(ql, G, N)[:, grp]
        C = xbc[:, spec.inner + G * N:].reshape(ql, G, N)[:, grp]
        dt = F.softplus(r[:, spec.off_dt:spec.off_dt + H] + w["dt_bias"], threshold=30.0)
        da = torch.exp(-dt * w["A"])
        S = torch.zeros_like(ssm_state[slot]) if fresh else ssm_state[slot].clone()  # [H, N, P]
        ys = torch.empty(ql, H, P)
        for t in range(ql):
            S = da[t][:, None, None] * S + (dt[t][:, None] * B[t])[:, :, None] * x[t][:, None, :]
            ys[t] = (S * C[t][:, :, None]).sum(1)
        ssm_state[slot] = S
        ys = (ys + w["D"][:, None] * x).reshape(ql, spec.inner) * F.silu(r[:, :spec.inner])
        gsz = spec.inner // spec.norm_groups
        p = ys.reshape(ql, spec.norm_groups, gsz)
        p = p * torch.rsqrt(p.pow(2).mean(-1, keepdim=True) + eps)
        out[t0:t0 + ql, :spec.inner] = (p.reshape(ql, -1) * w["norm"]).to(out.dtype)
        t0 += ql
    return out
