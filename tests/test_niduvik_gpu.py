"""Niduvik on the GPU: every kernel against the plain implementation's functions, then the model-level checks
(tests/decoder_cases.py) in bf16 -- the serving kernels -- and in fp32."""
import pytest
import torch

import niduvik_oracle as O
import niduvik_util as U
from decoder_cases import Cases
from rag_llm_k8s_amd.ops.backend import AttnMeta, get_backend
from rag_llm_k8s_amd.ops.specs import AttnSpec, SsmSpec, ceil_to, distance_table

pytestmark = pytest.mark.gpu
C = Cases(U)
DEV = "cuda"
F32, BF16 = torch.float32, torch.bfloat16
BOTH = [BF16, F32]


@pytest.fixture(scope="module")
def be(native):
    return get_backend(DEV)


def close(got, want, tol, what=""):
    e = float((got.double().cpu() - want.double()).abs().max())
    s = float(want.double().abs().max())
    assert e <= tol * max(s, 1e-6), (what, e, s)


# ------------------------------------------------------------------------------------- attention kernels
def attn_inputs(spec, T, dtype, seed, pairs, vmix=False):
    """Projection rows whose scores stand out at the given (query, key) pairs, one head dimension per pair."""
    g = torch.Generator().manual_seed(seed)
    q = 0.3 * torch.randn(T, spec.heads, spec.dim, generator=g)
    k = 0.3 * torch.randn(T, spec.kv_heads, spec.dim, generator=g)
    amp = (25.0 / spec.scale) ** 0.5
    for m, (i, j) in enumerate(pairs):
        q[i] = 0
        q[i, :, m % spec.dim] = amp
        k[j, :, m % spec.dim] = amp
    v = torch.randn(T, spec.kv_heads, spec.vdim, generator=g)
    gate = torch.randn(T, spec.heads, generator=g)
    first = torch.randn(T, spec.kv_heads, spec.vdim, generator=g) if vmix else None
    r = lambda t: None if t is None else t.to(dtype)  # noqa: E731
    return tuple(r(t) for t in (q, k, v, gate, first))


def pack_row(spec, q, k, v, gate):
    T = q.shape[0]
    row = torch.zeros(T, spec.row, dtype=q.dtype)
    row[:, :spec.off_k].view(T, spec.heads, spec.dkp)[:, :, :spec.dim] = q
    row[:, spec.off_k:spec.off_v].unflatten(1, (spec.kv_heads, spec.dkp))[:, :, :spec.dim] = k
    row[:, spec.off_v:spec.off_g].unflatten(1, (spec.kv_heads, spec.dvp))[:, :, :spec.vdim] = v
    row[:, spec.off_g:spec.off_g + spec.heads] = gate
    return row


def pad_values(spec, v):
    out = torch.zeros(v.shape[0], spec.kv_heads, spec.dvp, dtype=v.dtype)
    out[:, :, :spec.vdim] = v
    return out.reshape(v.shape[0], -1)


class Pages:
    """Scattered pages (reverse order, full of another request's numbers) for sequences of the given lengths."""

    def __init__(self, spec, lens, dtype):
        n = [-(-L // 64) for L in lens]
        total = sum(n) + 1
        g = torch.Generator().manual_seed(9)
        mk = lambda d: torch.randn(total, spec.kv_heads, 64, d, generator=g).to(DEV, dtype)  # noqa: E731
        self.kc, self.vc = mk(spec.dkp), mk(spec.dvp)
        self.bt = torch.zeros(len(lens), max(n) + 1, dtype=torch.int32)
        nxt = total - 1
        for s, c in enumerate(n):
            for b in range(c):
                self.bt[s, b] = nxt
                nxt -= 1

    def slots(self, s, lo, hi):
        p = torch.arange(lo, hi)
        return (self.bt[s, p // 64] * 64 + p % 64).int()


def prefill_meta(spec, pages, q_lens, kv_lens):
    from rag_llm_k8s_amd.ops.seq_native import query_tiles

    cu = torch.tensor([0] + torch.tensor(q_lens).cumsum(0).tolist(), dtype=torch.int32)
    return AttnMeta("prefill", torch.tensor(kv_lens, dtype=torch.int32, device=DEV), pages.bt.to(DEV), cu_q=cu.to(DEV),
                    qtiles={spec.q_tile: query_tiles(q_lens, spec.q_tile).to(DEV)}, host_kv_lens=list(kv_lens),
                    host_q_lens=list(q_lens))


def decode_meta(spec, pages, kv_lens, max_kv=4096):
    from rag_llm_k8s_amd.ops.seq_native import decode_split

    pt, mp, ws_o, ws_ml = decode_split([spec], max_kv, len(kv_lens), DEV)
    return AttnMeta("decode", torch.tensor(kv_lens, dtype=torch.int32, device=DEV), pages.bt.to(DEV), part_tiles=pt,
                    max_parts=mp, ws_o=ws_o, ws_ml=ws_ml, host_kv_lens=list(kv_lens), max_kv=max_kv)


def slabs_of(row, bias, S):
    """fp32 split-K slabs of rows whose bias a consumer adds."""
    x = row.float() - bias.float()
    g = torch.Generator().manual_seed(S)
    parts = [0.1 * torch.randn(x.shape, generator=g) for _ in range(S - 1)]
    return torch.stack(parts + [x - sum(parts)] if parts else [x]).to(DEV)


SPECS = {
    "g3": dict(heads=6, kv_heads=2, dim=40, vdim=24, window=70, keep_first=3, far=90),
    "g4": dict(heads=8, kv_heads=2, dim=128, vdim=72, window=33, keep_first=0, far=24),
    "g20": dict(heads=40, kv_heads=2, dim=20, vdim=200, window=200, keep_first=70, far=600),
    "g1": dict(heads=2, kv_heads=2, dim=200, vdim=32, window=64, keep_first=64, far=40),
    "g2": dict(heads=4, kv_heads=2, dim=64, vdim=128, window=129, keep_first=130, far=3000),
    "full": dict(heads=4, kv_heads=1, dim=96, vdim=64, window=0, keep_first=0, far=100),
}


def attn_setup(name, T, dtype, vmix):
    spec = AttnSpec(scale=0.11, softcap=12.0, sink=True, gate=True, **SPECS[name])
    w, kp = spec.window or 10 ** 6, spec.keep_first
    last = T - 1
    pairs = [(last, last), (last, 0), (last - 1, last - 64)]
    for i, d in ((last - 2, w - 1), (last - 3, w), (last - 4, w + 1), (last - 40, w - 1), (last - 70, w)):
        if 0 <= i - d:
            pairs.append((i, i - d))
    for i, j in ((last - 5, kp - 1), (last - 6, kp), (last - 7, 63), (last - 8, 64), (130, 127), (131, 128), (64, 63)):
        if 0 <= j <= i:
            pairs.append((i, j))
    q, k, v, gate, first = attn_inputs(spec, T, dtype, 5, pairs, vmix)
    rel = torch.randn(16, spec.heads, generator=torch.Generator().manual_seed(3))
    lam = 0.375
    mixed = v.double() if first is None else O.mix_values(v.double(), first.double(), lam)
    want = O.attention_core(q.double(), k.double(), mixed.to(dtype).double(), gate.double(), rel.double(), spec.scale,
                            spec.softcap, spec.far, spec.window or 10 ** 6, spec.keep_first)
    return spec, (q, k, v, gate, first), distance_table(rel, spec.far).to(DEV), torch.tensor([lam], device=DEV), want


def heads_of(spec, out):
    return out[:, :spec.heads * spec.dvp].reshape(-1, spec.heads, spec.dvp)[:, :, :spec.vdim].float().cpu()


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("name", sorted(SPECS))
def test_attention_prefill_in_portions(be, name, dtype):
    T = 333
    spec, (q, k, v, gate, first), table, lam, want = attn_setup(name, T, dtype, vmix=True)
    row = pack_row(spec, q, k, v, gate).to(DEV)
    vf = pad_values(spec, first).to(DEV)
    for cuts in ([T], [130, 2, 1, 63, 64, 73], [64, 269]):
        pages = Pages(spec, [T], dtype)
        outs, lo = [], 0
        for n in cuts:
            r, m = row[lo:lo + n], prefill_meta(spec, pages, [n], [lo + n])
            out = torch.zeros(n, spec.out_row, dtype=dtype, device=DEV)
            own = be.shaped_kv_store(r, spec, pages.slots(0, lo, lo + n).to(DEV), pages.kc, pages.vc, vf[lo:lo + n], lam)
            assert torch.equal(own.cpu(), pad_values(spec, v[lo:lo + n]))
            be.shaped_attn_prefill(r, spec, table, pages.kc, pages.vc, m, out)
            outs.append(heads_of(spec, out))
            lo += n
        close(torch.cat(outs), want, 1e-5 if dtype == F32 else 0.01, cuts)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("name", sorted(SPECS))
@pytest.mark.parametrize("S", [1, 5])
def test_attention_decode(be, name, dtype, S):
    """The last 80 tokens of one sequence as decode rows of a batch with a second, short one."""
    T, n = 333, 80
    spec, (q, k, v, gate, first), table, lam, want = attn_setup(name, T, dtype, vmix=True)
    row = pack_row(spec, q, k, v, gate)
    vf = pad_values(spec, first)
    pages = Pages(spec, [T, n], dtype)
    c = T - n
    be.shaped_kv_store(row[:c].to(DEV), spec, pages.slots(0, 0, c).to(DEV), pages.kc, pages.vc, vf[:c].to(DEV), lam)
    short = O.attention_core(*(x[:n].double() for x in (q, k)), O.mix_values(v[:n].double(), first[:n].double(), 0.375)
                             .to(dtype).double(), gate[:n].double(),
                             torch.randn(16, spec.heads, generator=torch.Generator().manual_seed(3)).double(), spec.scale,
                             spec.softcap, spec.far, spec.window or 10 ** 6, spec.keep_first)
    bias = (0.1 * torch.randn(spec.row, generator=torch.Generator().manual_seed(1))).to(dtype)
    got, got_short = [], []
    for i in range(n):
        rows = torch.stack([row[c + i], row[i]])
        slots = torch.cat([pages.slots(0, c + i, c + i + 1), pages.slots(1, i, i + 1)]).to(DEV)
        m = decode_meta(spec, pages, [c + i + 1, i + 1])
        out = torch.zeros(2, spec.out_row, dtype=dtype, device=DEV)
        f = torch.stack([vf[c + i], vf[i]]).to(DEV, F32)
        own = be.shaped_attn_decode(slabs_of(rows, bias, S), bias.to(DEV), spec, table, slots, pages.kc, pages.vc, m, out,
                                    v_first=f, lam=lam)
        close(own.float(), pad_values(spec, torch.stack([v[c + i], v[i]])).float(), 1e-5 if dtype == F32 else 4e-3)
        o = heads_of(spec, out)
        got.append(o[0])
        got_short.append(o[1])
    tol = 2e-5 if dtype == F32 else 0.015
    close(torch.stack(got), want[c:], tol)
    close(torch.stack(got_short), short, tol)


def test_attention_decode_partitions_agree(be):
    """A long unwindowed context split over many partitions equals one partition."""
    from rag_llm_k8s_amd.ops import seq_native

    spec, (q, k, v, gate, first), table, lam, want = attn_setup("full", 1500, BF16, vmix=False)
    row = pack_row(spec, q, k, v, gate)
    pages = Pages(spec, [1500], BF16)
    be.shaped_kv_store(row[:-1].to(DEV), spec, pages.slots(0, 0, 1499).to(DEV), pages.kc, pages.vc)
    assert seq_native.decode_parts(spec, 4096, 1) > 4
    for max_kv in (64, 1500, 4096):
        m = decode_meta(spec, pages, [1500], max_kv)
        out = torch.zeros(1, spec.out_row, dtype=BF16, device=DEV)
        be.shaped_attn_decode(slabs_of(row[-1:], torch.zeros(spec.row), 2), None, spec, table,
                              pages.slots(0, 1499, 1500).to(DEV), pages.kc, pages.vc, m, out)
        close(heads_of(spec, out), want[-1:], 0.01, max_kv)


def test_attention_options_off(be):
    """No soft cap, bias, sink, gate or window: plain causal attention."""
    spec = AttnSpec(heads=4, kv_heads=2, dim=64, vdim=64, scale=0.125)
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(200, n, 64, generator=g).bfloat16() for n in (4, 2, 2))
    row = torch.cat([x.reshape(200, -1) for x in (q, k, v)], 1)
    row = torch.nn.functional.pad(row, (0, spec.row - row.shape[1])).to(DEV)
    pages = Pages(spec, [200], BF16)
    out = torch.zeros(200, spec.out_row, dtype=BF16, device=DEV)
    be.shaped_kv_store(row, spec, pages.slots(0, 0, 200).to(DEV), pages.kc, pages.vc)
    be.shaped_attn_prefill(row, spec, None, pages.kc, pages.vc, prefill_meta(spec, pages, [200], [200]), out)
    s = (q.double().transpose(0, 1) @ k.double().repeat_interleave(2, 1).permute(1, 2, 0).contiguous()) * 0.125
    s = s.masked_fill(torch.ones(200, 200).triu(1).bool(), -torch.inf)
    want = (s.softmax(-1) @ v.double().repeat_interleave(2, 1).transpose(0, 1)).transpose(0, 1)
    close(heads_of(spec, out), want, 0.01)


# ------------------------------------------------------------------------------------- state-space kernels
SSMS = {
    "p20": dict(heads=6, vdim=20, state=24, groups=3, taps=3, norm_groups=2),
    "p64": dict(heads=4, vdim=64, state=128, groups=1, taps=4, norm_groups=4),
    "p8": dict(heads=6, vdim=8, state=40, groups=6, taps=2, norm_groups=3),
    "p12": dict(heads=3, vdim=12, state=16, groups=1, taps=5, norm_groups=1),
    "p96": dict(heads=2, vdim=96, state=256, groups=2, taps=4, norm_groups=2),
    "p30": dict(heads=2, vdim=30, state=30, groups=1, taps=4, norm_groups=4),
    "p128": dict(heads=8, vdim=128, state=64, groups=2, taps=4, norm_groups=8),
    "p200": dict(heads=2, vdim=200, state=250, groups=1, taps=8, norm_groups=4),
    "t1": dict(heads=2, vdim=16, state=32, groups=1, taps=1, norm_groups=1),
}


def ssm_setup(name, T, dtype, seed=0):
    spec = SsmSpec(**SSMS[name])
    g = torch.Generator().manual_seed(seed)
    H = spec.heads
    w = dict(conv_w=torch.randn(spec.taps, spec.channels, generator=g) * 0.6, conv_b=0.3 * torch.randn(spec.channels, generator=g),
             dt_bias=-1.5 + torch.randn(H, generator=g), A=torch.exp(-1 + 1.5 * torch.randn(H, generator=g)),
             D=torch.randn(H, generator=g), norm=1 + 0.2 * torch.randn(spec.inner, generator=g))
    row = torch.randn(T, spec.row, generator=g).to(dtype)
    return spec, w, row


def ssm_oracle(spec, w, row, eps, kept=None):
    d = {k: v.double() for k, v in w.items()}
    r = row.double()
    T = r.shape[0]
    u = O.silu(O.causal_conv(r[:, spec.off_x:spec.off_dt], d["conv_w"].T, d["conv_b"]))
    u = u.to(kept or row.dtype).double()  # prompts keep the convolution's output in the activations' type
    x, B, Cm = torch.split(u, [spec.inner, spec.groups * spec.state, spec.groups * spec.state], 1)
    dt = O.softplus(r[:, spec.off_dt:spec.off_dt + spec.heads] + d["dt_bias"])
    y, S = O.ssm(x.reshape(T, spec.heads, -1), B.reshape(T, spec.groups, -1), Cm.reshape(T, spec.groups, -1), dt,
                 torch.log(d["A"]), d["D"])
    y = O.group_rms_norm(y.reshape(T, -1) * O.silu(r[:, :spec.inner]), d["norm"], eps, spec.norm_groups)
    return y, S


def ssm_states(spec, n, fill):
    f = torch.full if fill else torch.zeros
    mk = lambda *s: f(s, 7.5, device=DEV) if fill else f(s, device=DEV)  # noqa: E731
    return mk(n, spec.taps - 1, spec.channels), mk(n, spec.heads, spec.state, spec.vdim)


def ssm_meta(q_lens, kv_lens, slots):
    cu = torch.tensor([0] + torch.tensor(q_lens).cumsum(0).tolist(), dtype=torch.int32, device=DEV)
    i = lambda x: torch.tensor(x, dtype=torch.int32, device=DEV)  # noqa: E731
    return AttnMeta("prefill", i(kv_lens), torch.zeros(len(q_lens), 1, dtype=torch.int32, device=DEV), cu_q=cu,
                    host_kv_lens=kv_lens, host_q_lens=q_lens, states=i(slots))


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("name", sorted(SSMS))
def test_ssm_portions_and_decode(be, name, dtype):
    """Two sequences packed, in portions (down to 2 and 1 tokens) over slots that held other numbers, then decoded."""
    L = [211, 70]
    spec, w, row0 = ssm_setup(name, L[0], dtype)
    _, _, row1 = ssm_setup(name, L[1], dtype, seed=1)
    wd = {k: v.to(DEV).contiguous() for k, v in w.items()}
    want = [ssm_oracle(spec, w, r, 1e-5) for r in (row0, row1)]
    conv, state = ssm_states(spec, 4, True)
    slots, got, at = [2, 1], [[], []], [0, 0]
    rows = [row0, row1]
    for step in ((64, 1), (65, 2), (2, 3), (1, 40), (69, 14)):
        r = torch.cat([rows[s][at[s]:at[s] + step[s]] for s in (0, 1)]).to(DEV)
        out = torch.zeros(sum(step), spec.out_row, dtype=dtype, device=DEV)
        be.ssm_prefill(r, spec, wd, 1e-5, ssm_meta(list(step), [at[s] + step[s] for s in (0, 1)], slots), conv, state, out)
        o = out[:, :spec.inner].float().cpu()
        got[0].append(o[:step[0]])
        got[1].append(o[step[0]:])
        at = [at[s] + step[s] for s in (0, 1)]
    for _ in range(10):
        r = torch.stack([rows[s][at[s]] for s in (0, 1)])
        m = ssm_meta([1, 1], [a + 1 for a in at], slots)
        m.kind, m.cu_q = "decode", None
        out = torch.zeros(2, spec.out_row, dtype=dtype, device=DEV)
        be.ssm_decode(slabs_of(r, torch.zeros(spec.row), 3), spec, wd, 1e-5, m, conv, state, out)
        for s in (0, 1):
            got[s].append(out[s:s + 1, :spec.inner].float().cpu())
        at = [a + 1 for a in at]
    for s in (0, 1):
        g = torch.cat(got[s])
        close(g, want[s][0], 3e-5 if dtype == F32 else 0.02)
        close(state[slots[s]], want[s][1], 1e-5 if dtype == F32 else 0.01)
    assert float(state[3].min()) == 7.5 == float(state[3].max())  # a slot nobody owns stays as it was


def test_ssm_decode_from_first_token(be):
    """A one-token sequence starts from zero state inside the decode kernels too."""
    spec, w, row = ssm_setup("p64", 30, BF16)
    wd = {k: v.to(DEV).contiguous() for k, v in w.items()}
    want, S = ssm_oracle(spec, w, row, 1e-5, kept=F32)  # decoding keeps it in fp32
    conv, state = ssm_states(spec, 2, True)
    got = []
    for t in range(30):
        m = ssm_meta([1], [t + 1], [1])
        m.kind, m.cu_q = "decode", None
        out = torch.zeros(1, spec.out_row, dtype=BF16, device=DEV)
        be.ssm_decode(slabs_of(row[t:t + 1], torch.zeros(spec.row), 1), spec, wd, 1e-5, m, conv, state, out)
        got.append(out[:, :spec.inner].float().cpu())
    close(torch.cat(got), want, 0.01)
    close(state[1], S, 1e-5)  # fp32 from slabs on: only accumulation order differs


def test_ssm_column_slices_agree(be):
    """The scan's 32- and 64-column forms (chosen by grid size) give the same numbers."""
    from rag_llm_k8s_amd.ops import _lib

    for name in ("p64", "p96", "p128"):
        spec, w, row = ssm_setup(name, 150, BF16)
        wd = {k: v.to(DEV).contiguous() for k, v in w.items()}
        res = []
        for cols in (32, 64):
            assert _lib.lib().ragk_ssm_scan_set_cols(cols) == 0
            try:
                conv, state = ssm_states(spec, 2, False)
                out = torch.zeros(150, spec.out_row, dtype=BF16, device=DEV)
                be.ssm_prefill(row.to(DEV), spec, wd, 1e-5, ssm_meta([150], [150], [1]), conv, state, out)
                res.append((out, state))
            finally:
                _lib.lib().ragk_ssm_scan_set_cols(0)
        assert torch.equal(res[0][0], res[1][0]) and torch.equal(res[0][1], res[1][1])


def test_ssm_wide_grid(be):
    """Enough (head, sequence) pairs that the scan takes its 64-column form by itself."""
    spec, w, _ = ssm_setup("p64", 1, BF16)
    wd = {k: v.to(DEV).contiguous() for k, v in w.items()}
    n, lens = 70, [130 - i for i in range(70)]
    rows = [ssm_setup("p64", L, BF16, seed=L)[2] for L in lens]
    conv, state = ssm_states(spec, n + 1, True)
    out = torch.zeros(sum(lens), spec.out_row, dtype=BF16, device=DEV)
    be.ssm_prefill(torch.cat(rows).to(DEV), spec, wd, 1e-5, ssm_meta(lens, lens, list(range(1, n + 1))), conv, state, out)
    lo = 0
    for i, L in enumerate(lens):
        if i % 17 == 0:
            y, S = ssm_oracle(spec, w, rows[i], 1e-5)
            close(out[lo:lo + L, :spec.inner].float(), y, 0.02, i)
            close(state[i + 1], S, 0.01, i)
        lo += L


# ------------------------------------------------------------------------------------- residual stream, GEMMs
@pytest.mark.parametrize("W,n", [(128, 96), (256, 256), (4096, 4096), (8192, 8100)])
@pytest.mark.parametrize("kind", ["bf16", "fp32", "slabs", "none", "plain"])
def test_residual_norm(be, W, n, kind):
    g = torch.Generator().manual_seed(W)
    M = 5
    h, y = torch.randn(M, W, generator=g), 3 * torch.randn(M, W, generator=g)
    wp, wn = 1 + 0.3 * torch.randn(W, generator=g), 1 + 0.3 * torch.randn(W, generator=g)
    for t in (h, y, wp, wn):
        t[..., n:] = 0
    yd = y
    if kind == "bf16":
        y = y.bfloat16().float()
        yd = y.bfloat16()
    elif kind == "slabs":
        p = 0.5 * torch.randn(9, M, W, generator=g)
        p[..., n:] = 0
        yd = torch.cat([p, (y - p.sum(0))[None]])
    want = h.double()
    if kind == "plain":
        want = want + y.double()
    elif kind != "none":
        want = want.clone()
        want[:, :n] += O.rms_norm(y[:, :n].double(), wp[:n].double(), 1e-5)
    wx = torch.zeros(M, W, dtype=torch.float64)
    wx[:, :n] = O.rms_norm(want[:, :n], wn[:n].double(), 1e-5)
    for dt in BOTH:
        hd = h.to(DEV)
        x = be.residual_norm(hd, None if kind == "none" else yd.to(DEV), None if kind == "plain" else wp.to(DEV),
                             wn.to(DEV), 1e-5, n, dt)
        close(hd, want, 1e-6)
        close(x.float(), wx, 1e-6 if dt == F32 else 4e-3)
    hd = h.to(DEV)
    assert be.residual_norm(hd, None if kind == "none" else yd.to(DEV), None if kind == "plain" else wp.to(DEV), None,
                            1e-5, n, BF16) is None
    close(hd, want, 1e-6)


@pytest.mark.parametrize("dtype", BOTH)
def test_embed_residual_and_gather(be, dtype):
    t = torch.randn(50, 256).to(DEV, dtype)
    ids = torch.tensor([3, 49, 0, 7], dtype=torch.int32, device=DEV)
    h = be.embed_residual(ids, t)
    assert h.dtype == F32 and torch.equal(h, t[ids.long()].float())
    carry = torch.tensor([-1, 1, -1, 0], dtype=torch.int32, device=DEV)
    prev = torch.tensor([11, 22], dtype=torch.int32, device=DEV)
    h = be.embed_residual(ids, t, carry, prev)
    assert ids.tolist() == [3, 22, 0, 11] and torch.equal(h, t[ids.long()].float())
    assert torch.equal(be.gather_rows(h, torch.tensor([2, 0], dtype=torch.int32, device=DEV)), h[[2, 0]])


@pytest.mark.parametrize("M,N,K", [(1, 64, 128), (3, 77, 256), (64, 640, 384), (65, 96, 128), (200, 1000, 512)])
def test_gemm_f32(be, M, N, K):
    g = torch.Generator().manual_seed(M)
    x, w, b = torch.randn(M, K, generator=g), torch.randn(N, K, generator=g), torch.randn(N, generator=g)
    want = x.double() @ w.double().T
    close(be.gemm(x.to(DEV), w.to(DEV)), want, 3e-6)
    close(be.gemm(x.to(DEV), w.to(DEV), bias=b.to(DEV), epi="bias"), want + b.double(), 3e-6)


@pytest.mark.parametrize("M", [1, 4, 5, 33, 64, 65, 200, 1030])
@pytest.mark.parametrize("F,K", [(128, 128), (384, 256), (8320, 256), (14336, 512)])
def test_clipped_glu_epilogue(be, M, F, K):
    """Every GEMM form the packed gate/up projection can take (register streaming, LDS ring, tiles, 256x256)."""
    from rag_llm_k8s_amd.ops.reference import pack_gate_up

    g = torch.Generator().manual_seed(M)
    x = torch.randn(M, K, generator=g).bfloat16()
    gate, up = (torch.randn(F, K, generator=g).mul(3 * K ** -0.5).bfloat16() for _ in (0, 1))
    limit, alpha, shift = 2.25, 1.702, 1.0
    par = torch.tensor([limit, alpha, shift, 0.0], device=DEV)
    a = torch.clamp(x.double() @ gate.double().T, max=limit)
    u = torch.clamp(x.double() @ up.double().T, -limit, limit)
    want = a / (1 + torch.exp(-alpha * a)) * (u + shift)
    close(be.gemm_glu(x.to(DEV), pack_gate_up(gate, up).to(DEV), par).float(), want, 6e-3)
    if F == 384:
        close(be.gemm_glu(x.float().to(DEV), pack_gate_up(gate, up).float().to(DEV), par), want, 2e-6)


# ------------------------------------------------------------------------------------- model level
@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("name", U.CONFIGS)
class TestModel:
    def test_layers(self, native, name, dtype):
        C.layers(DEV, dtype, name)

    def test_whole_prompt(self, native, name, dtype):
        C.whole_prompt(DEV, dtype, name)

    def test_token_by_token(self, native, name, dtype):
        C.token_by_token(DEV, dtype, name)

    def test_unequal_batch(self, native, name, dtype):
        C.unequal_batch(DEV, dtype, name)

    def test_greedy(self, native, name, dtype):
        C.greedy(DEV, dtype, name)

    def test_long_decode(self, native, name, dtype):
        C.long_decode(DEV, dtype, name)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("size", [2, 3, 17, 64])
def test_portions(native, dtype, size):
    for name in ("odd", "wide", "narrow"):
        C.portions(DEV, dtype, name, size)
    if size == 64:
        C.portions(DEV, dtype, "many", 64, budget=30)


@pytest.mark.parametrize("dtype", BOTH)
def test_reuse(native, dtype):
    C.reuse(DEV, dtype, "odd")
    C.reuse(DEV, dtype, "wide")


def test_decode_graph_replays_equal_eager(native):
    """Every replay of the captured decode step, with eager work and synchronizations in between, gives the
    eager step's logits: two engines over one model's weights, one with graphs and one without."""
    cfg, sd, m = U.make_model("wide", DEV, BF16)
    _, _, m2 = U.make_model("wide", DEV, BF16)
    t = {"a": U.prompt(cfg, 90, 1), "b": U.prompt(cfg, 60, 2)}
    plan = [{"a": 50, "b": 20}] + [{"a": 1, "b": 1}] * 40
    e1, e2 = U.make_engine(m), U.make_engine(m2, use_graphs=False)
    g, e = U.run(e1, t, plan), U.run(e2, t, plan)
    assert any(x["graph"] is not None for x in e1.graphs.values()) and all(x["graph"] is None for x in e2.graphs.values())
    for k in t:
        assert torch.equal(g[k], e[k])


def test_sampled_generation_async(native):
    """The asynchronous decode pipeline with requests that join and leave: every request's tokens equal the same
    request alone (same seed)."""
    from rag_llm_k8s_amd.engine.llm_engine import SamplingParams

    cfg, sd, m = U.make_model("wide", DEV, BF16)
    ps = [U.prompt(cfg, n, n) for n in (5, 70, 33, 1, 120)]
    par = [SamplingParams(max_new_tokens=k, temperature=0.0, do_sample=False, ignore_eos=True) for k in (20, 3, 11, 30, 8)]
    eng = U.make_engine(m, batch=2)
    seqs = [eng.add_request(p, q, seed=i) for i, (p, q) in enumerate(zip(ps, par))]
    eng.run_until_done()
    assert eng.bm.slots.available() == 2
    for p, q, s in zip(ps, par, seqs):
        assert len(s.out) == q.max_new_tokens
        lg = O.forward(cfg, sd, p + s.out)[len(p) - 1:-1]
        scale = float(lg.pow(2).mean().sqrt())
        for i, tok in enumerate(s.out):
            assert float(lg[i].max() - lg[i][tok]) <= 6 * U.limit(BF16) * scale
