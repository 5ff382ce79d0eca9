"""Throughput of a model family's layers at realistic sizes, beside Llama layers of equal size (random weights).

    python bench.py --layers niduvik | rolesun

For each size: prefill tokens/s (whole steps through model.forward) and decode tokens/s (replays of the engine's
captured decode graph), then the single kernels with the share of their roofline they reach -- the larger of
bytes / 8 TB/s and bf16 flops / 2.5 PFLOP/s -- next to the like kernel of the Llama layers. One JSON line.
"""
from __future__ import annotations

import json
import time

import torch

from ..engine.llm_engine import RUNNING, LLMEngine, SamplingParams, Sequence, no_cyclic_gc
from ..models import llama as L
from ..models import niduvik as N
from ..ops.backend import AttnMeta

HBM, FLOPS = 8.0e12, 2.5e15
VOCAB = 32768

SIZES = {
    "2k": dict(width=2048, heads=16, kv_heads=4, ff=5632, ssm_heads=64, groups=1),
    "4k": dict(width=4096, heads=32, kv_heads=8, ff=14336, ssm_heads=128, groups=8),
}


def niduvik_config(s, layers=4, window=4096):
    att = dict(heads=s["heads"], kv_heads=s["kv_heads"], dim=128, vdim=128, scale=128 ** -0.5, softcap=50.0, bias_max=128,
               v_mix=True, mask=dict(size=window, keep_first=4))
    ssm = dict(heads=s["ssm_heads"], vdim=64, state=128, groups=s["groups"], conv=4, norm_groups=s["groups"])
    mlp = dict(kind="dense", ff=s["ff"], limit=7.0)
    return N.NiduvikConfig(vocab=VOCAB, width=s["width"], eps=1e-5, layers=[
        dict(type="attention", mixer=att, mlp=mlp) if i % 2 == 0 else dict(type="mamba2", mixer=ssm, mlp=mlp)
        for i in range(layers)])


def llama_config(s, layers=4):
    return L.LlamaConfig(vocab_size=VOCAB, hidden_size=s["width"], intermediate_size=s["ff"], num_hidden_layers=layers,
                         num_attention_heads=s["heads"], num_key_value_heads=s["kv_heads"], head_dim=128)


def timed(fn, iters, warmup=2):
    for _ in range(warmup):
        fn()
    torch.cuda.synchronize()
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    a.record()
    for _ in range(iters):
        fn()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) / iters * 1e-3


def timed_turns(fns, iters, rounds=5):
    """Median seconds per call of each function, measured in turn so that clocks and power are alike."""
    ts = [[timed(f, iters) for f in fns] for _ in range(rounds)]
    return [sorted(t)[rounds // 2] for t in zip(*ts)]


def timed_graph(fn, iters):
    """Seconds per call of a decode kernel without host launch gaps: `iters` calls in one captured graph."""
    st = torch.cuda.Stream()
    st.wait_stream(torch.cuda.current_stream())
    with torch.cuda.stream(st):
        fn()
    torch.cuda.current_stream().wait_stream(st)
    g = torch.cuda.CUDAGraph()
    with no_cyclic_gc(), torch.cuda.graph(g, stream=st):
        for _ in range(iters):
            fn()
    return timed(g.replay, 4) / iters


def rotate(make, nbytes, cap=8):
    """Copies of an operand set that together exceed the 256 MB Infinity Cache, used in turn."""
    n = int(max(1, min(cap, 600e6 // max(1, nbytes) + 1)))
    sets, i = [make() for _ in range(n)], [0]

    def nxt():
        i[0] = (i[0] + 1) % n
        return sets[i[0]]
    return nxt


# ------------------------------------------------------------------------------------- whole steps
def _engine(model, tokens, batch):
    return LLMEngine(model, num_blocks=batch * (-(-tokens // 64)) + 4, max_batch=batch, max_model_len=tokens,
                     max_prefill_tokens=1 << 20, graph_buckets=[batch])


def _sequences(eng, n, length):
    out = []
    for i in range(n):
        s = Sequence(torch.randint(0, VOCAB, (length,), generator=torch.Generator().manual_seed(i)).tolist(),
                     SamplingParams(do_sample=False, ignore_eos=True), 0)
        s.status, s.computed = RUNNING, length
        eng.bm.ensure(s.id, length)
        out.append(s)
    return out


def prefill_rate(model, n, length, iters=6):
    eng = _engine(model, length, n)
    seqs = _sequences(eng, n, length)
    inp, _, ntok = eng._prefill_input([(s, 0, length) for s in seqs])
    return ntok / timed(lambda: model.forward(inp), iters)


def decode_rate(model, batch, ctx, iters=60):
    eng = _engine(model, ctx + 8, batch)
    seqs = _sequences(eng, batch, ctx)
    eng._begin_staging()
    eng._feed_decode(seqs)
    g = eng._decode_graph(batch)["graph"]
    return batch / timed(g.replay, iters, warmup=5)


# ------------------------------------------------------------------------------------- single kernels
def _roof(nbytes, flops):
    return max(nbytes / HBM, flops / FLOPS)


def _meta_prefill(model, n, length, dev):
    q = [length] * n
    cu = torch.arange(0, (n + 1) * length, length, dtype=torch.int32, device=dev)
    nb = -(-length // 64)
    bt = torch.arange(n * nb, dtype=torch.int32, device=dev).view(n, nb)
    tiles, qtiles = model.prefill_work(q, dev)
    return AttnMeta("prefill", torch.full((n,), length, dtype=torch.int32, device=dev), bt, cu_q=cu, tiles=tiles,
                    qtiles=qtiles, max_kv=length, key_rows=model.key_rows(q, q, dev), host_kv_lens=q, host_q_lens=q, states=torch.arange(1, n + 1, dtype=torch.int32, device=dev))


def _meta_decode(model, batch, ctx, dev):
    nb = -(-ctx // 64)
    bt = torch.arange(batch * nb, dtype=torch.int32, device=dev).view(batch, nb)
    pt, mp, ws_o, ws_ml = model.decode_work(ctx, batch)
    return AttnMeta("decode", torch.full((batch,), ctx, dtype=torch.int32, device=dev), bt, part_tiles=pt, max_parts=mp,
                    ws_o=ws_o, ws_ml=ws_ml, states=torch.arange(1, batch + 1, dtype=torch.int32, device=dev), max_kv=ctx)


def kernel_rows(size, nid, lla, dev, prefill=(4, 4096), decode=((1, 4096), (32, 4096))):
    """[(kernel, model, microseconds, share of roofline)]"""
    be, rows, s = nid.be, [], SIZES[size]
    bf = dict(dtype=torch.bfloat16, device=dev)
    n, T = prefill
    M = n * T

    def add(kind, model, t, nbytes, flops):
        rows.append(dict(kernel=kind, model=model, us=round(t * 1e6, 1), roofline=round(_roof(nbytes, flops) / t, 3)))

    att, ssm = nid.attn[0], nid.ssm[0]
    mlp = nid.w.layers[0]["mlp"]
    sp, ss = att.spec, ssm.spec
    H, G, D, W = sp.heads, sp.kv_heads, 128, s["width"]
    # prefill attention: causal work of both (the window covers the prompt)
    nb = n * (-(-T // 64))
    nid.allocate_kv_cache(nb)
    lla.allocate_kv_cache(nb)
    mN, mL = _meta_prefill(nid, n, T, dev), _meta_prefill(lla, n, T, dev)
    row = torch.randn(M, sp.row, **bf)
    out = torch.empty(M, sp.out_row, **bf)
    fl = 4.0 * n * T * T / 2 * H * D
    by = 2.0 * M * (2 * H * D + 2 * G * D)
    add("attention prefill", "niduvik", timed(lambda: be.shaped_attn_prefill(row, sp, att.table, att.kc, att.vc, mN, out), 8),
        by, fl)
    kc, vc = lla.kv_cache[0]
    add("attention prefill", "llama", timed(lambda: be.attn_prefill(row, kc, vc, mL, out, H, G, D), 8), by, fl)
    # projections and MLP
    x = torch.randn(M, W, **bf)
    LW = lla.w.layers[0]
    for name, wn, wl in (("qkv GEMM prefill", att.wqkv, LW["wqkv"]), ("out GEMM prefill", att.wo, LW["wo"])):
        add(name, "niduvik", timed(lambda: be.gemm(x, wn, bias=att.bqkv if wn is att.wqkv else None,
                                                   epi="bias" if wn is att.wqkv else "none"), 8),
            2.0 * (M * W + wn.numel() + M * wn.shape[0]), 2.0 * M * wn.numel())
        add(name, "llama", timed(lambda: be.gemm(x, wl), 8), 2.0 * (M * W + wl.numel() + M * wl.shape[0]),
            2.0 * M * wl.numel())
    add("in-projection GEMM prefill", "niduvik", timed(lambda: be.gemm(x, ssm.win), 8),
        2.0 * (M * W + ssm.win.numel() + M * ssm.win.shape[0]), 2.0 * M * ssm.win.numel())
    gl = (2.0 * (M * W + mlp.wgu.numel() + M * s["ff"]), 2.0 * M * mlp.wgu.numel())
    add("gate/up GEMM prefill", "niduvik", timed(lambda: be.gemm_glu(x, mlp.wgu, mlp.par), 8), *gl)
    add("gate/up GEMM prefill", "llama", timed(lambda: be.gemm(x, LW["wgu"], epi="silu_mul"), 8), *gl)
    # norms: residual + both norms against Llama's norm
    h = torch.randn(M, W, dtype=torch.float32, device=dev)
    y = torch.randn(M, W, **bf)
    w1 = torch.ones(W, device=dev)
    add("norm prefill", "niduvik", timed(lambda: be.residual_norm(h, y, w1, w1, 1e-5, W, torch.bfloat16), 8),
        M * W * (4 + 4 + 2 + 2.0), 0)
    wb = torch.ones(W, **bf)
    add("norm prefill", "llama", timed(lambda: be.rmsnorm(y, wb, 1e-5), 8), M * W * 4.0, 0)
    # KV store, state-space prefill
    slots = torch.arange(M, dtype=torch.int32, device=dev)
    add("KV store prefill", "niduvik", timed(lambda: be.shaped_kv_store(row, sp, slots, att.kc, att.vc), 8),
        2.0 * M * 2 * G * D * 2, 0)
    del row, out, h, y, x
    nid.allocate_state(n + 1)
    zrow = torch.randn(M, ss.row, **bf)
    xbc = be.q.ssm_conv(zrow, ss, ssm.w, mN, ssm.conv_state, ssm.ssm_state)
    add("conv prefill", "niduvik", timed(lambda: be.q.ssm_conv(zrow, ss, ssm.w, mN, ssm.conv_state, ssm.ssm_state), 8),
        2.0 * M * 2 * ss.channels, 0)
    Q = 64
    per = 2.0 * Q * Q / 2 * ss.state + 2.0 * Q * Q / 2 * ss.vdim + 4.0 * Q * ss.state * ss.vdim
    add("state-space scan prefill", "niduvik",
        timed(lambda: be.q.ssm_scan_chunk(xbc, zrow, ss, ssm.w, mN, ssm.ssm_state), 8),
        2.0 * M * (ss.channels + ss.heads + ss.inner), per * M / Q * ss.heads)
    yy = be.q.ssm_scan_chunk(xbc, zrow, ss, ssm.w, mN, ssm.ssm_state)
    oo = torch.empty(M, ss.out_row, **bf)
    add("gate + norm prefill", "niduvik", timed(lambda: be.q.ssm_gate_norm(yy, zrow, ss, ssm.w, 1e-5, oo), 8),
        2.0 * M * 3 * ss.inner, 0)
    add("out GEMM prefill (state space)", "niduvik", timed(lambda: be.gemm(oo, ssm.wo), 8),
        2.0 * (oo.numel() + ssm.wo.numel() + M * W), 2.0 * M * ssm.wo.numel())
    del zrow, xbc, yy, oo
    # decode
    for B, ctx in decode:
        tag = "decode b%d" % B
        nb = B * (-(-ctx // 64))
        kvb = 2.0 * B * ctx * G * D * 2
        mN, mL = _meta_decode(nid, B, ctx, dev), _meta_decode(lla, B, ctx, dev)
        slots = (mN.block_tables[:, (ctx - 1) // 64] * 64 + (ctx - 1) % 64).int().contiguous()
        pos = torch.full((B,), ctx - 1, dtype=torch.int32, device=dev)
        caches = rotate(lambda: (torch.zeros(nb, G, 64, D, **bf), torch.zeros(nb, G, 64, D, **bf)), kvb)
        xb = torch.randn(B, W, **bf)
        P, bias = be.proj_rows(xb, att.wqkv, att.bqkv)
        ob = torch.empty(B, sp.out_row, **bf)

        def natt():
            k, v = caches()
            be.shaped_attn_decode(P, bias, sp, att.table, slots, k, v, mN, ob)
        add("attention " + tag, "niduvik", timed_graph(natt, 24), kvb, 0)
        PL = be.gemm_part(xb, LW["wqkv"])

        def latt():
            k, v = caches()
            be.attn_decode_rope(PL, pos, lla.cos, lla.sin, slots, k, v, mL, ob, H, G, D)
        add("attention " + tag, "llama", timed_graph(latt, 24), kvb, 0)
        del caches

        def gemm_row(name, model, f, w):
            ws = rotate(lambda: w.clone(), w.numel() * 2)
            add(name + " " + tag, model, timed_graph(lambda: f(ws()), 24), 2.0 * w.numel(), 2.0 * B * w.numel())
        gemm_row("qkv GEMM", "niduvik", lambda w: be.proj_rows(xb, w), att.wqkv)
        gemm_row("qkv GEMM", "llama", lambda w: be.gemm_part(xb, w), LW["wqkv"])
        gemm_row("in-projection GEMM", "niduvik", lambda w: be.proj_rows(xb, w), ssm.win)
        gemm_row("gate/up GEMM", "niduvik", lambda w: be.gemm_glu(xb, w, mlp.par), mlp.wgu)
        gemm_row("gate/up GEMM", "llama", lambda w: be.gemm(xb, w, epi="silu_mul"), LW["wgu"])
        ab = torch.randn(B, s["ff"], **bf)
        gemm_row("down GEMM", "niduvik", lambda w: be.proj_rows(ab, w), mlp.wdown)
        gemm_row("down GEMM", "llama", lambda w: be.gemm_part(ab, w), LW["wdown"])
        # state update: read and written once
        nid.allocate_state(B + 1)
        P2, _ = be.proj_rows(xb, ssm.win)
        sb = 2.0 * B * ss.inner * ss.state * 4
        st = rotate(lambda: torch.zeros_like(ssm.ssm_state), sb / 2)
        add("state update " + tag, "niduvik",
            timed_graph(lambda: be.q.ssm_decode(P2, ss, ssm.w, mN, ssm.conv_state, st()), 24), sb + P2.numel() * 4, 0)
        del st
        hb = torch.randn(B, W, dtype=torch.float32, device=dev)
        hl = torch.randn(B, W, **bf)
        Pd, _ = be.proj_rows(ab, mlp.wdown)
        add("norm " + tag, "niduvik", timed_graph(lambda: be.residual_norm(hb, Pd, w1, w1, 1e-5, W, torch.bfloat16), 24),
            Pd.numel() * 4 + B * W * 10.0, 0)
        add("norm " + tag, "llama", timed_graph(lambda: be.add_partials_rmsnorm(Pd, hl, wb, 1e-5), 24),
            Pd.numel() * 4 + B * W * 6.0, 0)
    return rows


def _niduvik(s, dev):
    cfg = niduvik_config(s)
    return N.NiduvikModel(cfg, N.NiduvikWeights.from_state_dict(cfg, N.niduvik_state_dict(cfg, 0, device=dev), dev), dev)


def run(family, sizes=None, kernels=True):
    from . import layer_bench_rolesun as R

    dev = "cuda"
    build, rows_of, layers = {"niduvik": (_niduvik, kernel_rows, "4 (2 attention + 2 mamba2) / 4"),
                              "rolesun": (R.build, R.kernel_rows, "4 / 4")}[family]
    res = {}
    for size in sizes or SIZES:
        s = SIZES[size]
        mod = build(s, dev)
        lcfg = llama_config(s)
        lla = L.LlamaModel(lcfg, L.LlamaWeights.random(lcfg, dev), dev, max_positions=16384)
        r = {"layers": layers, "prefill_tok_s": {}, "decode_tok_s": {}}
        pair = ((family, mod), ("llama", lla))
        for n, T in ((1, 2048), (1, 8192), (16, 2048)):
            key = "%dx%d" % (n, T)
            r["prefill_tok_s"][key] = {k: round(prefill_rate(m, n, T)) for k, m in pair}
            print("layer bench: %s prefill %s %s" % (size, key, r["prefill_tok_s"][key]), flush=True)
        for B, ctx in ((1, 4096), (8, 4096), (32, 4096), (64, 4096)):
            key = "b%d ctx%d" % (B, ctx)
            r["decode_tok_s"][key] = {k: round(decode_rate(m, B, ctx), 1) for k, m in pair}
            print("layer bench: %s decode %s %s" % (size, key, r["decode_tok_s"][key]), flush=True)
        if kernels:
            r["kernels"] = rows_of(size, mod, lla, dev)
            for k in r["kernels"]:
                print("layer bench: %s %-34s %-8s %9.1f us  %.3f of roofline" % (size, k["kernel"], k["model"], k["us"],
                                                                               k["roofline"]), flush=True)
        res[size] = r
        del mod, lla, pair
        torch.cuda.empty_cache()
    return res


def main(family="niduvik", json_out=None):
    t0 = time.time()
    line = json.dumps({"layer_bench": "%s beside llama layers of equal size" % family, "data": "random weights and tokens",
                       "dtype": "bf16", "sizes": run(family), "seconds": round(time.time() - t0, 1)})
    print(line, flush=True)
    if json_out:
        with open(json_out, "w") as f:
            f.write(line + "\n")
