"""Rolesun's part of the layer benchmark: models of its sizes and its single kernels beside Llama's like ones."""
from __future__ import annotations

import torch

from ..models import rolesun as R
from .layer_bench import SIZES, VOCAB, _meta_decode, _meta_prefill, _roof, rotate, timed, timed_graph, timed_turns

RANK = {"2k": 256, "4k": 512}


def config(s, layers=4, window=4096):
    rank = next(RANK[k] for k, v in SIZES.items() if v is s)
    att = dict(heads=s["heads"], dim=128, vdim=128, kv_rank=rank, scale=128 ** -0.5, mask=dict(size=window))
    L = [dict(type="latent_attention", mixer=dict(att), mlp=dict(kind="dense", ff=s["ff"])) for _ in range(layers)]
    L[-1]["mixer"]["kv_from"] = layers - 2
    return R.RolesunConfig(vocab=VOCAB, width=s["width"], eps=1e-5, layers=L, embed_scale=0.5, residual_mult=0.3,
                           logit_scale=0.5)


def build(s, dev):
    cfg = config(s)
    return R.RolesunModel(cfg, R.RolesunWeights.from_state_dict(cfg, R.rolesun_state_dict(cfg, 0, device=dev), dev), dev)


def kernel_rows(size, mod, lla, dev, prefill=(4, 4096), decode=((1, 4096), (32, 4096), (64, 4096))):
    """[(kernel, model, microseconds, share of roofline)]"""
    be, rows, s = mod.be, [], SIZES[size]
    bf = dict(dtype=torch.bfloat16, device=dev)
    f32 = dict(dtype=torch.float32, device=dev)
    n, T = prefill
    M = n * T

    def add(kind, model, t, nbytes, flops):
        rows.append(dict(kernel=kind, model=model, us=round(t * 1e6, 1), roofline=round(_roof(nbytes, flops) / t, 3)))

    mx, LR, LW = mod.mixers[0], mod.w.layers[0], lla.w.layers[0]
    sp, lw, mlp = mx.spec, mx.lw, LR["mlp"]
    H, G, D, W, rp = sp.heads, s["kv_heads"], 128, s["width"], sp.rp
    nb = n * (-(-T // 64))
    mod.allocate_kv_cache(nb)
    lla.allocate_kv_cache(nb)
    mR, mL = _meta_prefill(mod, n, T, dev), _meta_prefill(lla, n, T, dev)
    kr = mR.key_rows[sp.window]
    row = torch.randn(M, sp.row, **bf)
    out = torch.empty(M, sp.out_row, **bf)
    kv = torch.randn(M + be.q.KEY_PAD, sp.kv_row, **bf)
    fl = 4.0 * n * T * T / 2 * H * D
    kc, vc = lla.kv_cache[0]
    kc.normal_()
    vc.normal_()
    ta, tl = timed_turns([lambda: be.q.row_attention(row, sp, kv, kr, mR, out),
                          lambda: be.attn_prefill(row, kc, vc, mL, out, H, G, D)], 8)
    add("attention prefill", "rolesun", ta, 2.0 * M * 5 * H * D, fl)
    add("attention prefill", "llama", tl, 2.0 * M * (2 * H * D + 2 * G * D), fl)
    del kv
    x = torch.randn(M, W, **bf)

    def gemm(name, model, w, a, f=None):
        add(name, model, timed(f or (lambda: be.gemm(a, w)), 8), 2.0 * (a.numel() + w.numel() + a.shape[0] * w.shape[0]),
            2.0 * a.shape[0] * w.numel())

    gemm("input GEMM prefill", "rolesun", mx.win, x)
    gemm("input GEMM prefill", "llama", LW["wqkv"], x)
    gemm("key / value expansion GEMM prefill", "rolesun", lw["ukv"], torch.randn(M + be.q.KEY_PAD, rp, **bf))
    gemm("residual gate GEMM prefill", "rolesun", LR["rg1"], x)
    gemm("out GEMM prefill", "rolesun", mx.wo, out)
    gemm("out GEMM prefill", "llama", LW["wo"], x)
    gl = (2.0 * (M * W + mlp.wgu.numel() + M * s["ff"]), 2.0 * M * mlp.wgu.numel())
    add("gate/up GEMM prefill", "rolesun", timed(lambda: be.gemm_glu(x, mlp.wgu, mlp.par), 8), *gl)
    add("gate/up GEMM prefill", "llama", timed(lambda: be.gemm(x, LW["wgu"], epi="silu_mul"), 8), *gl)
    h, y, z = torch.randn(M, W, **f32), torch.randn(M, W, **bf), torch.randn(M, W, **bf)
    zb, w1 = torch.zeros(W, device=dev), torch.ones(W, device=dev)
    add("gated norm + add prefill", "rolesun",
        timed(lambda: be.gated_residual(h, y, z, zb, w1, 1e-5, W, torch.bfloat16, keep=True), 8), M * W * 14.0, 0)
    mod.allocate_state(n + 1)
    add("token shift prefill", "rolesun",
        timed(lambda: be.token_shift(h, LR["shift"], mod.shift_state[0], mR, torch.bfloat16), 8), M * W * 8.0, 0)
    wb = torch.ones(W, **bf)
    add("norm prefill", "llama", timed(lambda: be.rmsnorm(y, wb, 1e-5), 8), M * W * 4.0, 0)
    slots = torch.arange(M, dtype=torch.int32, device=dev)
    add("latent norm + store prefill", "rolesun",
        timed(lambda: be.q.latent_store(row, sp, lw["norm"], 1e-5, slots, mx.pages), 8), 2.0 * M * 3 * rp, 0)
    kg = be.q.key_rows([T] * n, [2 * T] * n, 0, dev)
    mG = _meta_decode(mod, n, T, dev)
    kg.rows, kg.cu_k, kg.key_off = M, mR.cu_q, mR.cu_q[:-1].contiguous()
    add("latent gather prefill", "rolesun", timed(lambda: be.q.latent_gather(mx.pages, sp, mG, kg), 8), 2.0 * M * 2 * rp, 0)
    del row, out, h, y, z, x
    for B, ctx in decode:
        tag = "decode b%d" % B
        nb = B * (-(-ctx // 64))
        mR, mL = _meta_decode(mod, B, ctx, dev), _meta_decode(lla, B, ctx, dev)
        slots = (mR.block_tables[:, (ctx - 1) // 64] * 64 + (ctx - 1) % 64).int().contiguous()
        pos = torch.full((B,), ctx - 1, dtype=torch.int32, device=dev)
        xb, ob = torch.randn(B, W, **bf), torch.empty(B, sp.out_row, **bf)
        P = be.proj_rows(xb, mx.win)[0]
        cb, ub = 2.0 * B * ctx * rp, 2.0 * lw["uk"].numel()
        pages = rotate(lambda: torch.randn(nb, 64, rp, **bf), cb)
        uk, uv = rotate(lambda: lw["uk"].clone(), ub), rotate(lambda: lw["uv"].clone(), ub)
        qa = be.q.latent_absorb(P, sp, lw["uk"])
        parts = be.q.latent_parts(sp, ctx, B)
        pb = 4.0 * B * H * parts * rp
        af = 4.0 * B * ctx * H * rp
        add("absorb queries + append " + tag, "rolesun",
            timed_graph(lambda: be.q.latent_absorb(P, sp, uk(), pages(), slots, lw["norm"], 1e-5), 24),
            ub + 4.0 * P.numel() + 2.0 * qa.numel(), 0)
        add("attention " + tag, "rolesun", timed_graph(lambda: be.q.latent_attend(qa, sp, pages(), mR), 24), cb + pb, af)
        add("join + value map " + tag, "rolesun", timed_graph(lambda: be.q.latent_out(P, sp, uv(), mR, ob), 24), ub + pb, 0)
        add("attention, all three " + tag, "rolesun",
            timed_graph(lambda: be.q.latent_decode(P, sp, uk(), uv(), pages(), mR, ob, slots, lw["norm"], 1e-5), 24),
            cb + 2 * ub, af)
        del pages, uk, uv
        kvb = 2.0 * B * ctx * G * D * 2
        caches = rotate(lambda: (torch.randn(nb, G, 64, D, **bf), torch.randn(nb, G, 64, D, **bf)), kvb)
        PL = be.gemm_part(xb, LW["wqkv"])
        ol = torch.empty(B, H * D, **bf)

        def latt():
            k, v = caches()
            be.attn_decode_rope(PL, pos, lla.cos, lla.sin, slots, k, v, mL, ol, H, G, D)
        add("attention " + tag, "llama", timed_graph(latt, 24), kvb, 0)
        del caches

        def gemm_row(name, model, f, w):
            ws = rotate(lambda: w.clone(), w.numel() * 2)
            add(name + " " + tag, model, timed_graph(lambda: f(ws()), 24), 2.0 * w.numel(), 2.0 * B * w.numel())
        gemm_row("input GEMM", "rolesun", lambda w: be.proj_rows(xb, w), mx.win)
        gemm_row("input GEMM", "llama", lambda w: be.gemm_part(xb, w), LW["wqkv"])
        gemm_row("residual gate GEMM", "rolesun", lambda w: be.proj_rows(xb, w), LR["rg1"])
        gemm_row("out GEMM", "rolesun", lambda w: be.proj_rows(ob, w), mx.wo)
        gemm_row("out GEMM", "llama", lambda w: be.gemm_part(ol, w), LW["wo"])
        gemm_row("gate/up GEMM", "rolesun", lambda w: be.gemm_glu(xb, w, mlp.par), mlp.wgu)
        gemm_row("gate/up GEMM", "llama", lambda w: be.gemm(xb, w, epi="silu_mul"), LW["wgu"])
        ab = torch.randn(B, s["ff"], **bf)
        gemm_row("down GEMM", "rolesun", lambda w: be.proj_rows(ab, w), mlp.wdown)
        gemm_row("down GEMM", "llama", lambda w: be.gemm_part(ab, w), LW["wdown"])
        mod.allocate_state(B + 1)
        hb, hl = torch.randn(B, W, **f32), torch.randn(B, W, **bf)
        Pd, Z = be.proj_rows(ab, mlp.wdown)[0], be.proj_rows(xb, LR["rg2"])[0]
        sh = (LR["shift"], mod.shift_state[0])
        add("gated norm + add + shift " + tag, "rolesun",
            timed_graph(lambda: be.gated_residual(hb, Pd, Z, zb, w1, 1e-5, W, torch.bfloat16, keep=True, shift=sh, meta=mR), 24),
            (Pd.numel() + Z.numel()) * 4 + B * W * 20.0, 0)
        add("norm " + tag, "llama", timed_graph(lambda: be.add_partials_rmsnorm(Pd, hl, wb, 1e-5), 24),
            Pd.numel() * 4 + B * W * 6.0, 0)
    return rows
