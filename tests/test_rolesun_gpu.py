"""Rolesun on the GPU: every kernel against the plain implementation's functions, then the model-level checks
(tests/decoder_cases.py) in bf16 -- the serving kernels -- and in fp32."""
from types import SimpleNamespace

import pytest
import torch

import rolesun_oracle as O
import rolesun_util as U
from decoder_cases import Cases
from rag_llm_k8s_amd.ops.backend import AttnMeta, get_backend
from rag_llm_k8s_amd.ops.specs import LatentSpec

pytestmark = pytest.mark.gpu
C = Cases(U)
DEV = "cuda"
F32, BF16 = torch.float32, torch.bfloat16
BOTH = [BF16, F32]
EPS = 1e-4


@pytest.fixture(scope="module")
def be(native):
    return get_backend(DEV)


def close(got, want, tol, what=""):
    e = float((got.double().cpu() - want.double()).abs().max())
    s = float(want.double().abs().max())
    assert e <= tol * max(s, 1e-6), (what, e, s)


# ------------------------------------------------------------------------------------- latent attention
# ranks of every kernel width (128 .. 1024 columns), 16 and 32 heads per decode block and groups of both
SPECS = {
    "r56": dict(heads=5, dim=24, vdim=40, rank=56, window=70),
    "r130": dict(heads=3, dim=40, vdim=20, rank=130, window=33),
    "r200": dict(heads=33, dim=64, vdim=96, rank=200, window=0),
    "r384": dict(heads=17, dim=32, vdim=32, rank=384, window=128),
    "r512": dict(heads=20, dim=128, vdim=128, rank=512, window=200),
    "r500": dict(heads=40, dim=16, vdim=256, rank=500, window=65),
    "r640": dict(heads=7, dim=32, vdim=32, rank=640, window=129),
    "r768": dict(heads=2, dim=200, vdim=250, rank=768, window=64),
    "r896": dict(heads=18, dim=64, vdim=64, rank=800, window=1),
    "r1000": dict(heads=4, dim=16, vdim=16, rank=1000, window=66),
}
T = 333


class Case:
    """One sequence of T tokens: latents before their norm, maps, and queries whose scores stand out at given pairs."""

    def __init__(self, name, dtype, seed=5, own=True, scale=0.11):
        self.spec = s = LatentSpec(scale=scale, own=own, **SPECS[name])
        self.dtype = dtype
        g = torch.Generator().manual_seed(seed)
        r = lambda *n: torch.randn(*n, generator=g)  # noqa: E731
        raw = (2 * r(T, s.rank)).to(dtype)
        self.norm = 1 + 0.3 * r(s.rank)
        self.uk = (r(s.heads, s.dim, s.rank) * s.rank ** -0.5).to(dtype)
        self.uv = (r(s.heads, s.vdim, s.rank) * s.rank ** -0.5).to(dtype)
        c = O.rms(raw.double(), EPS) * self.norm.double()
        self.latents = c.to(dtype).double()
        k = torch.einsum("tr,hdr->thd", c, self.uk.double())
        q = 0.3 * r(T, s.heads, s.dim).double()
        w, last = s.window or 10 ** 6, T - 1
        pairs = [(last, last), (last, 0), (last - 1, last - 64)]
        for i, d in ((last - 2, w - 1), (last - 3, w), (last - 4, w + 1), (last - 40, w - 1), (last - 70, w), (130, w - 1),
                     (131, w)):
            if 0 <= i - d:
                pairs.append((i, i - d))
        pairs += [(last - 7, 63), (last - 8, 64), (140, 127), (141, 128), (64, 63), (65, 64), (63, 0), (1, 0)]
        for i, j in pairs:
            q[i] = k[j] * (20.0 / s.scale / (k[j] ** 2).sum(-1, keepdim=True))
        q, gate = q.to(dtype), r(T, s.heads, s.vdim).to(dtype)
        self.row = torch.zeros(T, s.row, dtype=dtype)
        self.row[:, :s.off_g].view(T, s.heads, s.dkp)[:, :, :s.dim] = q
        self.row[:, s.off_g:s.off_c].unflatten(1, (s.heads, s.dvp))[:, :, :s.vdim] = gate
        if own:
            self.row[:, s.off_c:s.off_c + s.rank] = raw
        self.want = O.latent_attention_core(q.double(), self.latents, self.uk.double(), self.uv.double(), s.scale,
                                            s.window or 10 ** 6) * O.sigmoid(gate.double())

    def weights(self):
        """Device weights in the mixer's layouts."""
        s = self.spec
        uk = torch.zeros(s.heads, s.dkp, s.rp, dtype=self.dtype)
        uv = torch.zeros(s.heads, s.dvp, s.rp, dtype=self.dtype)
        uk[:, :s.dim, :s.rank], uv[:, :s.vdim, :s.rank] = self.uk, self.uv
        norm = torch.zeros(s.rp)
        norm[:s.rank] = self.norm
        ukv = torch.cat([uk.reshape(-1, s.rp), uv.reshape(-1, s.rp)]).to(DEV)
        return dict(ukv=ukv, uv=ukv[s.off_v:].view(s.heads, s.dvp, s.rp), uk=uk.transpose(1, 2).contiguous().to(DEV),
                    norm=norm.to(DEV) if s.own else None, source=0)

    def heads_of(self, out):
        s = self.spec
        return out[:, :s.heads * s.dvp].reshape(-1, s.heads, s.dvp)[:, :, :s.vdim].float().cpu()


class Pages:
    """Scattered pages (reverse order, full of another request's numbers) for sequences of the given lengths."""

    def __init__(self, spec, lens, dtype):
        n = [-(-L // 64) for L in lens]
        total = sum(n) + 1
        self.pages = (50 * torch.randn(total, 64, spec.rp, generator=torch.Generator().manual_seed(9))).to(DEV, dtype)
        self.bt = torch.zeros(len(lens), max(n) + 1, dtype=torch.int32)
        nxt = total - 1
        for s, c in enumerate(n):
            for b in range(c):
                self.bt[s, b] = nxt
                nxt -= 1

    def slots(self, s, lo, hi):
        p = torch.arange(lo, hi)
        return (self.bt[s, p // 64] * 64 + p % 64).int()

    def put(self, s, lo, latents):
        """Latent rows [n, rank] into the pages from position lo on."""
        sl = self.slots(s, lo, lo + latents.shape[0]).long().to(DEV)
        v = torch.zeros(latents.shape[0], self.pages.shape[2])
        v[:, :latents.shape[1]] = latents.float()
        self.pages.view(-1, self.pages.shape[2])[sl] = v.to(DEV, self.pages.dtype)


def step_input(pages, seqs, q_lens, kv_lens, kind="prefill", windows=(), max_kv=4096, specs=()):
    from rag_llm_k8s_amd.ops.seq_native import key_rows, latent_workspace

    i = lambda x: torch.tensor(x, dtype=torch.int32, device=DEV)  # noqa: E731
    cu = [0] + torch.tensor(q_lens).cumsum(0).tolist()
    slots = torch.cat([pages.slots(s, k - n, k) for s, n, k in zip(seqs, q_lens, kv_lens)]).to(DEV)
    meta = AttnMeta(kind, i(kv_lens), pages.bt[seqs].contiguous().to(DEV), cu_q=i(cu) if kind == "prefill" else None,
                    host_kv_lens=list(kv_lens), host_q_lens=list(q_lens), max_kv=max_kv)
    if kind == "prefill":
        meta.key_rows = {w: key_rows(q_lens, kv_lens, w, DEV) for w in windows}
    else:
        meta.ws_o, meta.ws_ml = latent_workspace(specs, max_kv, len(q_lens), DEV)
    return SimpleNamespace(meta=meta, slots=slots)


def slabs_of(row, S):
    """fp32 split-K slabs of rows."""
    x = row.float()
    g = torch.Generator().manual_seed(S)
    parts = [0.1 * torch.randn(x.shape, generator=g) for _ in range(S - 1)]
    return torch.stack(parts + [x - sum(parts)] if parts else [x]).to(DEV)


def tol(dtype):
    return 2e-5 if dtype == F32 else 0.02


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("name", sorted(SPECS))
def test_latent_prompt_in_portions(be, name, dtype):
    c = Case(name, dtype)
    s, lw = c.spec, c.weights()
    for cuts in ([T], [130, 2, 1, 63, 64, 73], [64, 269], [70, 58, 2, 1, 1, 201]):
        pg, outs, lo = Pages(s, [T], dtype), [], 0
        for n in cuts:
            out = torch.zeros(n, s.out_row, dtype=dtype, device=DEV)
            be.latent_prefill(c.row[lo:lo + n].to(DEV), s, lw, EPS, step_input(pg, [0], [n], [lo + n], windows=[s.window]),
                              pg.pages, {}, out)
            outs.append(c.heads_of(out))
            lo += n
        close(torch.cat(outs), c.want, tol(dtype), cuts)


@pytest.mark.parametrize("dtype", BOTH)
def test_latent_prompts_packed_with_decode_rows(be, dtype):
    """One step with a new prompt, a continued one and two one-token sequences behind them."""
    cs = [Case("r130", dtype, seed=i) for i in range(4)]
    s, lw = cs[0].spec, cs[0].weights()
    for c in cs[1:]:
        c.uk, c.uv, c.norm = cs[0].uk, cs[0].uv, cs[0].norm
    have, new = [0, 150, 300, 65], [90, 33, 1, 1]
    pg = Pages(s, [T] * 4, dtype)
    rows, want = [], []
    for i, c in enumerate(cs):
        raw = c.row[:, s.off_c:s.off_c + s.rank].double()
        lat = (O.rms(raw, EPS) * cs[0].norm.double()).to(dtype)
        pg.put(i, 0, lat[:have[i]])
        q = c.row[:, :s.off_g].reshape(T, s.heads, s.dkp)[:, :, :s.dim].double()
        gate = c.row[:, s.off_g:s.off_c].reshape(T, s.heads, s.dvp)[:, :, :s.vdim].double()
        w = O.latent_attention_core(q, lat.double(), cs[0].uk.double(), cs[0].uv.double(), s.scale, s.window) * O.sigmoid(gate)
        rows.append(c.row[have[i]:have[i] + new[i]])
        want.append(w[have[i]:have[i] + new[i]])
    n = sum(new)
    out = torch.zeros(n, s.out_row, dtype=dtype, device=DEV)
    inp = step_input(pg, [0, 1, 2, 3], new, [h + k for h, k in zip(have, new)], windows=[s.window])
    assert inp.meta.key_rows[s.window].tail == 2 and inp.meta.key_rows[s.window].gather
    be.latent_prefill(torch.cat(rows).to(DEV), s, lw, EPS, inp, pg.pages, {}, out)
    close(cs[0].heads_of(out), torch.cat(want), tol(dtype))


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("name", sorted(SPECS))
@pytest.mark.parametrize("S", [1, 5])
def test_latent_decode(be, name, dtype, S):
    """The last 70 tokens of one sequence as decode rows of a batch with a second, short one."""
    n = 70
    c = Case(name, dtype)
    s, lw = c.spec, c.weights()
    pg = Pages(s, [T, n], dtype)
    pg.put(0, 0, c.latents[:T - n])
    got, short = [], []
    for i in range(n):
        t = T - n + i
        out = torch.zeros(2, s.out_row, dtype=dtype, device=DEV)
        inp = step_input(pg, [0, 1], [1, 1], [t + 1, i + 1], kind="decode", specs=[s])
        be.latent_decode(slabs_of(torch.stack([c.row[t], c.row[i]]), S), s, lw, EPS, inp, pg.pages, out)
        o = c.heads_of(out)
        got.append(o[0])
        short.append(o[1])
    close(torch.stack(got), c.want[T - n:], tol(dtype))
    close(torch.stack(short), c.want[:n], tol(dtype))


@pytest.mark.parametrize("dtype", BOTH)
def test_latents_of_another_layer(be, dtype):
    """A layer without latents of its own reads the given pages through its own maps, queries and window."""
    src, c = Case("r200", dtype), Case("r200", dtype, seed=8, own=False)
    s, lw = c.spec, c.weights()
    s.window = 90
    q = c.row[:, :s.off_g].reshape(T, s.heads, s.dkp)[:, :, :s.dim].double()
    gate = c.row[:, s.off_g:s.off_c].reshape(T, s.heads, s.dvp)[:, :, :s.vdim].double()
    want = O.latent_attention_core(q, src.latents, c.uk.double(), c.uv.double(), s.scale, 90) * O.sigmoid(gate)
    pg = Pages(s, [T], dtype)
    pg.put(0, 0, src.latents)
    before = pg.pages.clone()
    out = torch.zeros(T - 100, s.out_row, dtype=dtype, device=DEV)
    inp = step_input(pg, [0], [T - 100], [T], windows=[90])
    rows = {}
    be.latent_prefill(c.row[100:].to(DEV), s, lw, EPS, inp, pg.pages, rows, out)
    assert list(rows) == [(0, 90)]  # gathered once for every layer that reads this source through this window
    close(c.heads_of(out), want[100:], tol(dtype))
    out = torch.zeros(1, s.out_row, dtype=dtype, device=DEV)
    inp = step_input(pg, [0], [1], [T], kind="decode", specs=[s])
    be.latent_decode(slabs_of(c.row[-1:], 3), s, lw, EPS, inp, pg.pages, out)
    close(c.heads_of(out), want[-1:], tol(dtype))
    assert torch.equal(pg.pages, before)


@pytest.mark.parametrize("heads,rank", [(5, 100), (20, 256), (20, 384), (3, 512), (33, 512), (4, 600), (4, 700), (4, 800),
                                        (20, 1000)])
def test_latent_decode_partitions_agree(be, heads, rank):
    """A long unwindowed context in one partition and in many; head 0's scores rise all the way, the others' peak anywhere."""
    from rag_llm_k8s_amd.ops import seq_native

    s = LatentSpec(heads=heads, dim=64, vdim=64, rank=rank, scale=0.1)
    L = 2500
    g = torch.Generator().manual_seed(2)
    r = lambda *n: torch.randn(*n, generator=g)  # noqa: E731
    lat = r(L, rank)
    uk, uv = ((r(heads, 64, rank) * rank ** -0.5).bfloat16() for _ in (0, 1))
    q, gate = (12 * r(heads, 64)).bfloat16(), r(heads, 64).bfloat16()
    lat = lat[torch.argsort(lat @ (uk[0].float().T @ q[0].float()))].bfloat16()
    pad = lambda w: torch.nn.functional.pad(w, (0, s.rp - rank))  # noqa: E731
    lw = dict(uk=pad(uk).transpose(1, 2).contiguous().to(DEV), uv=pad(uv).to(DEV), norm=torch.ones(s.rp, device=DEV), source=0)
    k = torch.einsum("tr,hdr->htd", lat.double(), uk.double())
    v = torch.einsum("tr,hdr->htd", lat.double(), uv.double())
    p = torch.softmax((k * q.double()[:, None]).sum(-1) * s.scale, -1)
    want = ((p[..., None] * v).sum(1) * O.sigmoid(gate.double()))[None]
    pg = Pages(s, [L], BF16)
    pg.put(0, 0, lat)
    row = torch.zeros(1, s.row)
    row[:, :s.off_g], row[:, s.off_g:s.off_c] = q.reshape(1, -1).float(), gate.reshape(1, -1).float()
    s.own = False
    assert seq_native.latent_parts(s, 8192, 1) >= 16 > seq_native.latent_parts(s, 256, 1)
    for max_kv in (64, 256, 2500, 8192):
        out = torch.zeros(1, s.out_row, dtype=BF16, device=DEV)
        inp = step_input(pg, [0], [1], [L], kind="decode", specs=[s], max_kv=max_kv)
        be.latent_decode(slabs_of(row, 2), s, lw, EPS, inp, pg.pages, out)
        close(out[:, :heads * 64].reshape(1, heads, 64).float(), want, 0.02, max_kv)


@pytest.mark.parametrize("dtype", BOTH)
def test_latent_negative_scale(be, dtype):
    c = Case("r130", dtype, scale=-0.2)
    s, lw = c.spec, c.weights()
    pg = Pages(s, [T], dtype)
    out = torch.zeros(T, s.out_row, dtype=dtype, device=DEV)
    be.latent_prefill(c.row.to(DEV), s, lw, EPS, step_input(pg, [0], [T], [T], windows=[s.window]), pg.pages, {}, out)
    close(c.heads_of(out), c.want, tol(dtype))
    out = torch.zeros(1, s.out_row, dtype=dtype, device=DEV)
    be.latent_decode(slabs_of(c.row[-1:], 2), s, lw, EPS, step_input(pg, [0], [1], [T], kind="decode", specs=[s]), pg.pages, out)
    close(c.heads_of(out), c.want[-1:], tol(dtype))


@pytest.mark.parametrize("B", [16, 17, 70])
def test_latent_decode_wide_batch(be, B):
    """More sequences than one block's matrix columns, all of different lengths."""
    c = Case("r500", BF16)
    s, lw = c.spec, c.weights()
    lens = [1 + (i * 37) % T for i in range(B)]
    pg = Pages(s, lens, BF16)
    for i, L in enumerate(lens):
        if L > 1:
            pg.put(i, 0, c.latents[:L - 1])
    out = torch.zeros(B, s.out_row, dtype=BF16, device=DEV)
    rows = torch.stack([c.row[L - 1] for L in lens])
    be.latent_decode(slabs_of(rows, 4), s, lw, EPS, step_input(pg, list(range(B)), [1] * B, lens, kind="decode", specs=[s]),
                     pg.pages, out)
    close(c.heads_of(out), torch.stack([c.want[L - 1] for L in lens]), 0.02)


def test_latent_checks_refuse_what_does_not_fit(be):
    c = Case("r56", BF16)
    s, lw = c.spec, c.weights()
    pg = Pages(s, [T], BF16)
    inp = step_input(pg, [0], [1], [T], kind="decode", specs=[s])
    out = torch.zeros(1, s.out_row, dtype=BF16, device=DEV)
    P = slabs_of(c.row[-1:], 1)
    with pytest.raises(ValueError):  # pages of another width
        be.latent_decode(P, s, lw, EPS, inp, torch.zeros(4, 64, 256, dtype=BF16, device=DEV), out)
    with pytest.raises(ValueError):  # a workspace of fewer partitions
        inp.meta.ws_o = inp.meta.ws_o[:8]
        be.latent_decode(P, s, lw, EPS, inp, pg.pages, out)
    inp = step_input(pg, [0], [T], [T], windows=[s.window])
    kv = torch.zeros(T, s.kv_row, dtype=BF16, device=DEV)
    with pytest.raises(ValueError):  # no padding rows behind the keys
        be.q.row_attention(c.row.to(DEV), s, kv, inp.meta.key_rows[s.window], inp.meta,
                           torch.zeros(T, s.out_row, dtype=BF16, device=DEV))


# ------------------------------------------------------------------------------------- residual stream
@pytest.mark.parametrize("W,n", [(128, 96), (256, 256), (4096, 4096), (8192, 8100)])
@pytest.mark.parametrize("kind", ["bf16", "fp32", "slabs", "ungated"])
@pytest.mark.parametrize("shift", [False, True])
def test_gated_residual(be, W, n, kind, shift):
    g = torch.Generator().manual_seed(W)
    M = 5
    h, y, z = (torch.randn(M, W, generator=g) for _ in range(3))
    zb, mix = torch.randn(W, generator=g), torch.rand(W, generator=g)
    state = torch.randn(8, W, generator=g)
    w = torch.full((W,), 1.3 * 0.4)
    for t in (h, y, z, zb, mix, w, state):
        t[..., n:] = 0
    if kind == "bf16":
        y, z = y.bfloat16().float(), z.bfloat16().float()
    yd, zd = (y.bfloat16(), z.bfloat16()) if kind == "bf16" else (y, z)
    if kind == "slabs":
        parts = 0.5 * torch.randn(9, M, W, generator=g)
        parts[..., n:] = 0
        yd = torch.cat([parts, (y - parts.sum(0))[None]])
        zd = torch.cat([parts[:2], (z - parts[:2].sum(0))[None]])
    gated = y if kind == "ungated" else O.output_gate(y.double()[:, :n], z.double()[:, :n], torch.eye(n, dtype=torch.float64),
                                                      zb.double()[:n])
    want = torch.zeros(M, W, dtype=torch.float64)
    want[:, :n] = O.residual_add(h.double()[:, :n], gated.double()[:, :n], 1.3, EPS, 0.4)
    slots, lens = [3, 1, 7, 2, 5], [4, 1, 100, 2, 1]  # two sequences at their first token
    before = torch.stack([torch.zeros(W) if L == 1 else state[s] for s, L in zip(slots, lens)]).double()
    ws = want + (before - want) * mix.double()
    meta = AttnMeta("decode", torch.tensor(lens, dtype=torch.int32, device=DEV), None,
                    states=torch.tensor(slots, dtype=torch.int32, device=DEV))
    for dt in BOTH:
        hd, st = h.to(DEV), state.to(DEV)
        x, xs = be.gated_residual(hd, yd.to(DEV), None if kind == "ungated" else zd.to(DEV), zb.to(DEV), w.to(DEV), EPS, n, dt,
                                  keep=True, shift=(mix.to(DEV), st) if shift else None, meta=meta)
        close(hd, want, 2e-6)
        close(x.float(), want, 2e-6 if dt == F32 else 4e-3)
        if shift:
            close(xs.float(), ws, 2e-6 if dt == F32 else 4e-3)
            assert torch.equal(st[slots], hd)
            assert torch.equal(st[[0, 4, 6]].cpu(), state[[0, 4, 6]])
        else:
            assert xs is None
    assert be.gated_residual(h.to(DEV), yd.to(DEV), None, None, w.to(DEV), EPS, n, BF16) == (None, None)


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("W", [128, 2176])
def test_token_shift(be, dtype, W):
    """Two sequences packed, in portions down to one token, over state that held other numbers."""
    g = torch.Generator().manual_seed(W)
    L = [90, 40]
    xs = [torch.randn(n, W, generator=g) for n in L]
    mix = torch.rand(W, generator=g)
    want = [O.token_shift(x, mix) for x in xs]
    state = torch.full((4, W), 7.5, device=DEV)
    at, got = [0, 0], [[], []]
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)  # noqa: E731
    for step in ((64, 1), (1, 2), (2, 30), (1, 1), (1, 1), (21, 5)):
        h = torch.cat([xs[s][at[s]:at[s] + step[s]] for s in (0, 1)]).to(DEV)
        at = [at[s] + step[s] for s in (0, 1)]
        decode = step == (1, 1)
        meta = AttnMeta("decode" if decode else "prefill", i32(at), torch.zeros(2, 1, dtype=torch.int32, device=DEV),
                        cu_q=None if decode else i32([0, step[0], sum(step)]), states=i32([2, 1]))
        x, s = be.token_shift(h, mix.to(DEV), state, meta, dtype)
        assert torch.equal(x.float(), h.to(dtype).float())
        got[0].append(s[:step[0]].float().cpu())
        got[1].append(s[step[0]:].float().cpu())
    for s in (0, 1):
        close(torch.cat(got[s]), want[s], 1e-6 if dtype == F32 else 4e-3)
        assert torch.equal(state[2 - s].cpu(), xs[s][-1])
    assert float(state[[0, 3]].min()) == 7.5 == float(state[[0, 3]].max())


@pytest.mark.parametrize("dtype", BOTH)
@pytest.mark.parametrize("n,W", [(131, 256), (256, 256), (7, 128)])
def test_embedding_with_sinusoid(be, dtype, n, W):
    t = torch.randn(50, W)
    t[:, n:] = 0
    t = t.to(DEV, dtype)
    ids = torch.tensor([3, 49, 0, 7, 11], dtype=torch.int32, device=DEV)
    pos = [0, 1, 777, 131071, 50000]
    i = torch.arange((n + 1) // 2, dtype=torch.float64)
    turns = (10000.0 ** (-2 * i / n) / (2 * torch.pi)).to(DEV)
    h = be.embed_residual(ids, t, scale=0.7, pos=torch.tensor(pos, dtype=torch.int32, device=DEV), turns=turns, n=n)
    want = t[ids.long()].double().cpu() * 0.7
    want[:, :n] += O.sinusoid(pos, n)
    assert h.dtype == F32
    close(h, want, 3e-7)


@pytest.mark.parametrize("M", [1, 5, 64, 200, 1030])
def test_silu_unit(be, M):
    from rag_llm_k8s_amd.models.mixers import GluMlp

    g = torch.Generator().manual_seed(M)
    x = torch.randn(M, 250, generator=g)
    sd = {"gate": torch.randn(300, 250, generator=g) / 8, "up": torch.randn(300, 250, generator=g) / 8,
          "down": torch.randn(250, 300, generator=g) / 16}
    for dt in BOTH:
        r = {k: v.to(dt) for k, v in sd.items()}
        mlp = GluMlp.load(250, 300, lambda n: r[n], lambda t, d=dt: t.to(DEV, d).contiguous())
        xd = torch.zeros(M, 256, dtype=dt, device=DEV)
        xd[:, :250] = x.to(DEV, dt)
        want = O.gated_mlp(x.to(dt).double(), *(r[k].double() for k in ("gate", "up", "down")))
        for kind in ("prefill", "decode"):
            y = mlp.forward(be, xd, SimpleNamespace(meta=SimpleNamespace(kind=kind)))
            y = y.sum(0) if y.dim() == 3 else y
            close(y[:, :250].float(), want, 1e-5 if dt == F32 else 0.01, kind)


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
    for dtype in BOTH:
        cfg, sd, m = U.make_model("wide", DEV, dtype)
        _, _, m2 = U.make_model("wide", DEV, dtype)
        t = {"a": U.prompt(cfg, 90, 1), "b": U.prompt(cfg, 60, 2)}
        plan = [{"a": 50, "b": 20}] + [{"a": 1, "b": 1}] * 40
        e1, e2 = U.make_engine(m), U.make_engine(m2, use_graphs=False)
        g, e = U.run(e1, t, plan), U.run(e2, t, plan)
        assert any(x["graph"] is not None for x in e1.graphs.values()) and all(x["graph"] is None for x in e2.graphs.values())
        for k in t:
            assert torch.equal(g[k], e[k])


def test_generation_async(native):
    """The asynchronous decode pipeline with requests that join and leave: every request's tokens are the oracle's
    wherever its choice is clear."""
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
