"""Sublayers of residual-stream decoders: shaped attention, latent attention, Mamba-2 state space, gated MLPs.

Each mixer owns its device weights and its cache (paged K/V, or per-slot state) and maps normed rows to
either the sublayer's output rows (prefill) or fp32 split-K slabs of them (decode), which the following
residual_norm kernel sums. A model composes them; nothing here knows a model's name.

Activations are in the weights' type (bf16 when serving, fp32 for exact replay); the residual stream,
norms, scores, decays and states are fp32 in both.
"""
from __future__ import annotations

import math

import torch

from ..ops.reference import pack_gate_up
from ..ops.specs import AttnSpec, LatentSpec, SsmSpec, ceil_to, distance_table


def pad2(t, rows, cols):
    """Zero-pad a matrix to [rows, cols]."""
    if tuple(t.shape) == (rows, cols):
        return t
    out = torch.zeros(rows, cols, dtype=t.dtype, device=t.device)
    out[:t.shape[0], :t.shape[1]] = t
    return out


def pad1(t, n):
    out = torch.zeros(n, dtype=t.dtype, device=t.device)
    out[:t.shape[0]] = t
    return out


def pad_head_rows(w, heads, d, dp):
    """[heads * d, K] -> [heads * dp, K], zero rows after each head's own."""
    if d == dp:
        return w
    out = torch.zeros(heads, dp, w.shape[1], dtype=w.dtype, device=w.device)
    out[:, :d] = w.reshape(heads, d, -1)
    return out.reshape(heads * dp, -1)


class AttentionMixer:
    """Grouped-query attention with the options of ops/specs.AttnSpec."""

    recurrent = False

    def __init__(self, spec: AttnSpec, width, wqkv, bqkv, wo, table=None, vmix=None, v_source=False):
        self.spec, self.width = spec, width
        self.wqkv, self.bqkv, self.wo, self.table = wqkv, bqkv, wo, table
        self.vmix = vmix  # device scalar; None: values as projected
        self.v_source = v_source  # this layer's own values are what later layers mix in
        self.kc = self.vc = None

    @classmethod
    def load(cls, spec: AttnSpec, width, get, dev, rel=None, vmix=False, v_source=False):
        """get(name): raw tensor of 'q', 'k', 'v', 'o' and, as the spec asks, 'g', '*.b'; dev(t): to the device."""
        H, G = spec.heads, spec.kv_heads
        wp = ceil_to(width, 128)
        parts = [(get("q"), get("q.b"), H, spec.dim, spec.dkp), (get("k"), get("k.b"), G, spec.dim, spec.dkp),
                 (get("v"), get("v.b"), G, spec.vdim, spec.dvp)]
        ws = [pad_head_rows(w, n, d, dp) for w, _, n, d, dp in parts]
        bs = [pad_head_rows((torch.zeros(n * d, dtype=w.dtype, device=w.device) if b is None else b)[:, None], n, d, dp)[:, 0]
              for w, b, n, d, dp in parts]
        if spec.gate:
            ws.append(get("g"))
            bs.append(torch.zeros(H, dtype=ws[0].dtype, device=ws[0].device))
        wqkv = dev(pad2(torch.cat(ws, 0), spec.row, wp))
        bqkv = dev(pad1(torch.cat(bs, 0), spec.row))
        wo = dev(pad2(pad_head_rows(get("o").t().contiguous(), H, spec.vdim, spec.dvp).t(), wp, spec.out_row))
        table = dev(distance_table(rel, spec.far), torch.float32) if rel is not None else None
        spec.bias_bound = float(table.abs().max()) if table is not None else 0.0
        lam = dev(get("vmix").reshape(1), torch.float32) if vmix else None
        return cls(spec, width, wqkv, bqkv, wo, table, lam, v_source)

    def cache_bytes(self, itemsize):
        return self.spec.kv_heads * 64 * (self.spec.dkp + self.spec.dvp) * itemsize

    def allocate_cache(self, num_blocks, dtype, device):
        s = self.spec
        self.kc = torch.zeros(num_blocks, s.kv_heads, 64, s.dkp, dtype=dtype, device=device)
        self.vc = torch.zeros(num_blocks, s.kv_heads, 64, s.dvp, dtype=dtype, device=device)

    def _out(self, be, T, like):
        s = self.spec
        exact = s.out_row == s.heads * s.dvp
        return (torch.empty if exact else torch.zeros)((T, s.out_row), dtype=like.dtype, device=like.device)

    def forward(self, be, xn, inp, shared):
        """`shared`: values that layers of one forward hand on ({"v_first": rows})."""
        s, meta = self.spec, inp.meta
        out = self._out(be, xn.shape[0], xn)
        v_first = shared.get("v_first") if self.vmix is not None else None
        lam = self.vmix if v_first is not None else None
        if meta.kind == "decode":
            P, bias = be.proj_rows(xn, self.wqkv, self.bqkv)
            own = be.shaped_attn_decode(P, bias, s, self.table, inp.slots, self.kc, self.vc, meta, out,
                                        v_first=v_first, lam=lam)
            y = be.proj_rows(out, self.wo)[0]
        else:
            row = be.gemm(xn, self.wqkv, bias=self.bqkv, epi="bias")
            own = be.shaped_kv_store(row, s, inp.slots, self.kc, self.vc, v_first, lam)
            be.shaped_attn_prefill(row, s, self.table, self.kc, self.vc, meta, out)
            y = be.gemm(out, self.wo)
        if self.v_source:
            shared["v_first"] = own
        return y


class LatentAttentionMixer:
    """Latent attention (ops/specs.LatentSpec). A mixer with a source reads that mixer's cached latents through its own
    key and value maps."""

    recurrent = False

    def __init__(self, spec: LatentSpec, width, eps, index, win, lw, wo, source=None):
        self.spec, self.width, self.eps, self.index = spec, width, eps, index
        self.win, self.lw, self.wo, self.source = win, lw, wo, source
        self.pages = None

    @classmethod
    def load(cls, spec: LatentSpec, width, eps, index, get, dev, source=None):
        """get(name): raw tensor of 'q', 'g', 'uk', 'uv', 'o' and, in a layer of its own latents, 'dkv', 'dkv.norm'."""
        H, wp, rp = spec.heads, ceil_to(width, 128), spec.rp
        ws = [pad_head_rows(get("q"), H, spec.dim, spec.dkp), pad_head_rows(get("g"), H, spec.vdim, spec.dvp)]
        if spec.own:
            ws.append(get("dkv"))
        win = dev(pad2(torch.cat(ws, 0), spec.row, wp))
        maps = [pad2(pad_head_rows(get(n), H, d, dp), H * dp, rp)
                for n, d, dp in (("uk", spec.dim, spec.dkp), ("uv", spec.vdim, spec.dvp))]
        ukv = dev(torch.cat(maps, 0))  # expands a latent row to [k of every head | v of every head]
        lw = dict(ukv=ukv, uv=ukv[spec.off_v:].view(H, spec.dvp, rp),
                  uk=dev(maps[0].reshape(H, spec.dkp, rp).transpose(1, 2)), norm=None,
                  source=index if source is None else source.index)
        if spec.own:
            lw["norm"] = dev(pad1(get("dkv.norm").float(), rp), torch.float32)
        wo = dev(pad2(pad_head_rows(get("o").t().contiguous(), H, spec.vdim, spec.dvp).t(), wp, spec.out_row))
        return cls(spec, width, eps, index, win, lw, wo, source)

    def cache_bytes(self, itemsize):
        return 64 * self.spec.rp * itemsize if self.spec.own else 0

    def allocate_cache(self, num_blocks, dtype, device):
        if self.spec.own:
            self.pages = torch.zeros(num_blocks, 64, self.spec.rp, dtype=dtype, device=device)

    def forward(self, be, x, inp, shared):
        """`shared`: latent rows that layers of one forward hand on, by source layer."""
        s = self.spec
        pages = self.pages if self.source is None else self.source.pages
        exact = s.out_row == s.heads * s.dvp
        out = (torch.empty if exact else torch.zeros)((x.shape[0], s.out_row), dtype=x.dtype, device=x.device)
        if inp.meta.kind == "decode":
            be.latent_decode(be.proj_rows(x, self.win)[0], s, self.lw, self.eps, inp, pages, out)
            return be.proj_rows(out, self.wo)[0]
        be.latent_prefill(be.gemm(x, self.win), s, self.lw, self.eps, inp, pages, shared, out)
        return be.gemm(out, self.wo)


class Mamba2Mixer:
    """Mamba-2 layer: in-projection, short causal convolution, selective scan, gated grouped RMS norm."""

    recurrent = True

    def __init__(self, spec: SsmSpec, width, eps, win, w, wo):
        self.spec, self.width, self.eps = spec, width, eps
        self.win, self.w, self.wo = win, w, wo
        self.conv_state = self.ssm_state = None

    @classmethod
    def load(cls, spec: SsmSpec, width, eps, get, dev):
        wp = ceil_to(width, 128)
        f = torch.float32
        w = dict(conv_w=dev(get("conv").float().t(), f), conv_b=dev(get("conv.b"), f),
                 dt_bias=dev(get("dt_bias"), f), A=dev(torch.exp(get("A_log").float()), f), D=dev(get("D"), f),
                 norm=dev(get("norm"), f))
        return cls(spec, width, eps, dev(pad2(get("in"), spec.row, wp)), w, dev(pad2(get("o"), wp, spec.out_row)))

    def state_bytes(self):
        s = self.spec
        return 4 * ((s.taps - 1) * s.channels + s.inner * s.state)

    def allocate_state(self, num_slots, device):
        s = self.spec
        f32 = dict(dtype=torch.float32, device=device)
        self.conv_state = torch.zeros(num_slots, s.taps - 1, s.channels, **f32)
        self.ssm_state = torch.zeros(num_slots, s.heads, s.state, s.vdim, **f32)

    def forward(self, be, xn, inp, shared):
        s, meta = self.spec, inp.meta
        exact = s.out_row == s.inner
        out = (torch.empty if exact else torch.zeros)((xn.shape[0], s.out_row), dtype=xn.dtype, device=xn.device)
        if meta.kind == "decode":
            P, _ = be.proj_rows(xn, self.win)
            be.ssm_decode(P, s, self.w, self.eps, meta, self.conv_state, self.ssm_state, out)
            return be.proj_rows(out, self.wo)[0]
        row = be.gemm(xn, self.win)
        be.ssm_prefill(row, s, self.w, self.eps, meta, self.conv_state, self.ssm_state, out)
        return be.gemm(out, self.wo)


class GluMlp:
    """W_down (silu(g) * u), g | u = packed gate/up rows."""

    def __init__(self, wgu, wdown, par=None):
        self.wgu, self.wdown, self.par = wgu, wdown, par

    @classmethod
    def load(cls, width, ff, get, dev, par=None):
        wp, fp = ceil_to(width, 128), ceil_to(ff, 128)
        wgu = dev(pack_gate_up(pad2(get("gate"), fp, wp), pad2(get("up"), fp, wp)))
        if par is None and wgu.dtype == torch.float32:  # the fp32 unit has the clipped form only: nothing is clipped
            par = dev(torch.tensor([math.inf, 1.0, 0.0, 0.0]), torch.float32)
        return cls(wgu, dev(pad2(get("down"), wp, fp)), par)

    def forward(self, be, xn, inp):
        a = be.gemm_glu(xn, self.wgu, self.par)
        return be.proj_rows(a, self.wdown)[0] if inp.meta.kind == "decode" else be.gemm(a, self.wdown)


class ClippedGluMlp(GluMlp):
    """W_down (min(g, limit) sigmoid(alpha g) (clamp(u, +-limit) + shift))."""

    @classmethod
    def load(cls, width, ff, limit, alpha, shift, get, dev):
        return super().load(width, ff, get, dev, dev(torch.tensor([limit, alpha, shift, 0.0]), torch.float32))
