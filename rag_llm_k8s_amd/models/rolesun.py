"""Rolesun: a decoder of windowed latent attention without rotations, norms on the sublayers' outputs only.

    x  <- embed * scale + sinusoid(position)
    x  <- x + mult * norm1(mixer(shift(x)) * sigmoid(Rg1 x + b1))
    x  <- x + mult * norm2(mlp(x) * sigmoid(Rg2 x + b2))            (layers without an mlp skip this)

The sublayers read the stream itself; shift() mixes each row with the one before it, so every layer keeps one row per
sequence as state. Attention caches one latent row per token and layer; a layer with 'kv_from' reads an earlier layer's.
The residual stream is fp32. Every size and constant comes from config.json ("layers" lists them per layer).
"""
from __future__ import annotations

import json
import math
import os
from dataclasses import dataclass, field
from typing import List, Optional

import torch

from ..ops.backend import get_backend
from ..ops.specs import LatentSpec, ceil_to
from .base import DecoderModel
from .mixers import GluMlp, LatentAttentionMixer, pad1, pad2

POSITION_BASE = 10000.0


@dataclass
class RolesunConfig:
    vocab: int
    width: int
    eps: float
    layers: List[dict]  # {"type", "mixer": {...}, "mlp": {...} or None}
    embed_scale: float = 1.0
    residual_mult: float = 1.0
    logit_scale: float = 1.0
    bos_token_id: Optional[int] = None
    eos_token_id: List[int] = field(default_factory=list)
    max_position_embeddings: int = 131072
    model_type: str = "rolesun"

    @classmethod
    def from_dict(cls, d):
        eos = d.get("eos_token_id")
        c = cls(vocab=int(d["vocab"]), width=int(d["width"]), eps=float(d["norm"]["eps"]),
                layers=[dict(type=L["type"], mixer=dict(L["mixer"]), mlp=L.get("mlp")) for L in d["layers"]],
                embed_scale=float(d["embedding"]["scale"]), residual_mult=float(d["residual_mult"]),
                logit_scale=float(d["logit_scale"]), bos_token_id=d.get("bos_token_id"),
                eos_token_id=[] if eos is None else (eos if isinstance(eos, list) else [eos]),
                max_position_embeddings=int(d.get("max_position_embeddings") or 131072))
        for i, L in enumerate(c.layers):
            if L["type"] != "latent_attention":
                raise ValueError("layer %d: unknown mixer type %r" % (i, L["type"]))
            if L["mlp"] is not None and L["mlp"].get("kind", "dense") != "dense":
                raise ValueError("layer %d: unknown mlp kind %r" % (i, L["mlp"]["kind"]))
            j = L["mixer"].get("kv_from")
            if j is not None:
                if not 0 <= j < i or c.layers[j]["mixer"].get("kv_from") is not None:
                    raise ValueError("layer %d: kv_from %r is not an earlier layer with latents of its own" % (i, j))
                if c.layers[j]["mixer"]["kv_rank"] != L["mixer"]["kv_rank"]:
                    raise ValueError("layer %d: kv_rank differs from that of layer %d" % (i, j))
        return c

    @classmethod
    def from_json(cls, path):
        with open(path) as f:
            return cls.from_dict(json.load(f))

    def to_dict(self):
        d = {"architecture": "Rolesun", "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
             "embedding": {"scale": self.embed_scale}, "residual_mult": self.residual_mult,
             "logit_scale": self.logit_scale, "layers": self.layers,
             "max_position_embeddings": self.max_position_embeddings}
        if self.bos_token_id is not None:
            d["bos_token_id"] = self.bos_token_id
        if self.eos_token_id:
            d["eos_token_id"] = self.eos_token_id
        return d

    @property
    def vocab_size(self):
        return self.vocab


def latent_spec(m):
    return LatentSpec(heads=m["heads"], dim=m["dim"], vdim=m["vdim"], rank=m["kv_rank"], scale=float(m["scale"]),
                      window=int((m.get("mask") or {}).get("size") or 0), own=m.get("kv_from") is None)


class RolesunWeights:
    """Device weights in kernel layouts (matrices zero-padded to the GEMM tiles; norm weights, gate biases and shift
    coefficients fp32). A norm's single number fills a row, with the residual multiplier or logit scale in it."""

    tp_rank, vocab_offset = 0, 0

    @classmethod
    def from_get(cls, cfg: RolesunConfig, get, device, dtype=torch.bfloat16):
        """`get(name)` returns a raw tensor."""
        w = cls()
        w.cfg, w.dtype = cfg, dtype
        n, wp = cfg.width, ceil_to(cfg.width, 128)
        device = torch.device(device)

        def dev(t, dt=dtype):
            return t.to(device=device, dtype=dt).contiguous()

        def vec(name):
            return dev(pad1(get(name).float(), wp), torch.float32)

        def norm(name, mult):
            return dev(pad1(torch.full((n,), float(get(name).float()) * mult), wp), torch.float32)

        w.width_pad = wp
        w.embed = dev(pad2(get("embed"), ceil_to(cfg.vocab, 8), wp))
        w.lm_head = dev(pad2(get("head"), ceil_to(cfg.vocab, 8), wp))
        w.vocab_valid = cfg.vocab
        # turns per position of column pair i: POSITION_BASE^(-2i / width) / (2 pi)
        i = torch.arange((n + 1) // 2, dtype=torch.float64)
        w.turns = dev(torch.exp(-2.0 * i / n * math.log(POSITION_BASE)) / (2 * math.pi), torch.float64)
        w.layers, mixers = [], []
        for li, L in enumerate(cfg.layers):
            p, src = "l%d." % li, L["mixer"].get("kv_from")
            mixers.append(LatentAttentionMixer.load(latent_spec(L["mixer"]), n, cfg.eps, li,
                                                    lambda name, p=p: get(p + "mix." + name), dev,
                                                    source=None if src is None else mixers[src]))
            layer = dict(mixer=mixers[-1], shift=vec(p + "shift"), norm1=norm(p + "norm1", cfg.residual_mult),
                         rg1=dev(pad2(get(p + "rg1"), wp, wp)), rg1b=vec(p + "rg1.b"), mlp=None)
            if L["mlp"] is not None:
                layer.update(mlp=GluMlp.load(n, L["mlp"]["ff"], lambda name, p=p: get(p + "mlp." + name), dev),
                             norm2=norm(p + "norm2", cfg.residual_mult), rg2=dev(pad2(get(p + "rg2"), wp, wp)),
                             rg2b=vec(p + "rg2.b"))
            w.layers.append(layer)
        w.norm = norm("final.norm", cfg.logit_scale)
        return w

    @classmethod
    def from_checkpoint(cls, path, cfg, device, dtype=torch.bfloat16):
        from ..runtime.safetensors_io import CheckpointReader

        rd = CheckpointReader(path)
        try:
            return cls.from_get(cfg, rd.get, device, dtype)
        finally:
            rd.close()

    @classmethod
    def from_state_dict(cls, cfg, sd, device, dtype=torch.bfloat16):
        return cls.from_get(cfg, lambda n: sd[n], device, dtype)

    def nbytes(self):
        n = 0
        for L in self.layers:
            mx, ml = L["mixer"], L["mlp"]
            ts = [mx.win, mx.wo, mx.lw["ukv"], mx.lw["uk"], L["rg1"]]
            ts += [ml.wgu, ml.wdown, L["rg2"]] if ml is not None else []
            n += sum(t.numel() * t.element_size() for t in ts)
        return n + (self.embed.numel() + self.lm_head.numel()) * self.embed.element_size()


class RolesunModel(DecoderModel):
    recurrent = True  # the row before the next token, in every layer

    def __init__(self, cfg: RolesunConfig, weights: RolesunWeights, device, comm=None, max_positions=None):
        if comm is not None and comm.size > 1:
            raise ValueError("Rolesun runs on one GPU per engine (use data-parallel replicas)")
        self.cfg, self.w, self.device = cfg, weights, torch.device(device)
        self.be = get_backend(self.device)
        self.dtype = weights.dtype
        self.comm, self.tp_rank = None, 0
        self.mixers = [L["mixer"] for L in weights.layers]
        self.windows = sorted({m.spec.window for m in self.mixers})
        self.shift_state = None

    # ---- caches and work lists the engine asks for
    def kv_bytes_per_block(self):
        size = torch.tensor([], dtype=self.dtype).element_size()
        return sum(m.cache_bytes(size) for m in self.mixers)

    def allocate_kv_cache(self, num_blocks, dtype=None):
        for m in self.mixers:
            m.allocate_cache(num_blocks, dtype or self.dtype, self.device)
        return [m.pages for m in self.mixers if m.pages is not None]

    def state_bytes_per_slot(self):
        return 4 * len(self.mixers) * self.w.width_pad

    def allocate_state(self, num_slots):
        self.shift_state = torch.zeros(len(self.mixers), num_slots, self.w.width_pad, dtype=torch.float32,
                                       device=self.device)

    def prefill_work(self, q_lens, device):
        return None, {}

    def key_rows(self, q_lens, kv_lens, device):
        if self.be.name != "native":  # the CPU forms read the pages directly
            return {}
        from ..ops.seq_native import key_rows

        return {w: key_rows(q_lens, kv_lens, w, device) for w in self.windows}

    def decode_work(self, max_kv_len, batch):
        from ..ops.seq_native import latent_workspace

        return (1, 1) + latent_workspace([m.spec for m in self.mixers], max_kv_len, batch, self.device)

    # ---- one step
    def _gate(self, x, w, inp):
        return self.be.proj_rows(x, w)[0] if inp.meta.kind == "decode" else self.be.gemm(x, w)

    def _advance(self, h, y, z, zb, norm, nxt, inp):
        """Close a layer; (rows, shifted rows) for layer `nxt`, or None behind the last one."""
        be, c, meta = self.be, self.cfg, inp.meta
        if nxt is not None and meta.kind == "decode":
            return be.gated_residual(h, y, z, zb, norm, c.eps, c.width, self.dtype, keep=True,
                                     shift=(self.w.layers[nxt]["shift"], self.shift_state[nxt]), meta=meta)
        be.gated_residual(h, y, z, zb, norm, c.eps, c.width, self.dtype)
        return self._shift(h, nxt, inp) if nxt is not None else None

    def _shift(self, h, li, inp):
        return self.be.token_shift(h, self.w.layers[li]["shift"], self.shift_state[li], inp.meta, self.dtype)

    def hidden_states(self, inp, trace=None):
        """Final-normed rows selected by logits_idx, times the logit scale. `trace` (a list) receives the residual
        after every layer."""
        be, w, c = self.be, self.w, self.cfg
        n, eps, dt = c.width, c.eps, self.dtype
        h = be.embed_residual(inp.ids, w.embed, carry=inp.carry, prev=inp.carry_src, scale=c.embed_scale,
                              pos=inp.positions, turns=w.turns, n=n)
        x, xs = self._shift(h, 0, inp)
        shared = {}
        for li, L in enumerate(w.layers):
            z = self._gate(x, L["rg1"], inp)
            y = L["mixer"].forward(be, xs, inp, shared)
            zb, norm = L["rg1b"], L["norm1"]
            if L["mlp"] is not None:
                x, _ = be.gated_residual(h, y, z, zb, norm, eps, n, dt, keep=True)
                z = self._gate(x, L["rg2"], inp)
                y = L["mlp"].forward(be, x, inp)
                zb, norm = L["rg2b"], L["norm2"]
            nxt = li + 1 if li + 1 < len(w.layers) else None
            x, xs = self._advance(h, y, z, zb, norm, nxt, inp) or (None, None)
            if trace is not None:
                trace.append(h[:, :n].clone())
        if inp.logits_idx is not None:  # the final norm runs on the selected rows only
            h = be.gather_rows(h, inp.logits_idx)
        return be.residual_norm(h, None, None, w.norm, eps, n, dt)

    def logits(self, hs):
        return self.be.gemm(hs, self.w.lm_head, out_f32=True)

    def forward(self, inp):
        return self.logits(self.hidden_states(inp))


# ------------------------------------------------------------------------------------- synthetic checkpoints
def rolesun_tiny(vocab=512, **kw):
    """Four small layers with every branch: unequal heads, sizes and windows, a layer that reads another's latents
    through a window of its own, a layer without an mlp."""
    def att(**o):
        m = dict(heads=5, dim=24, vdim=40, kv_rank=56, scale=0.21, mask=dict(size=70))
        m.update(o)
        return dict(type="latent_attention", mixer=m)

    mlp = dict(kind="dense", ff=200)
    layers = [dict(att(), mlp=mlp), dict(att(heads=3, dim=40, vdim=20, kv_rank=130, mask=dict(size=33)), mlp=None),
              dict(att(heads=4, vdim=64, kv_from=0, mask=dict(size=129)), mlp=mlp), dict(att(), mlp=mlp)]
    d = dict(vocab=vocab, width=144, eps=1e-5, layers=layers, embed_scale=0.7, residual_mult=0.4, logit_scale=1.5,
             bos_token_id=vocab - 2, eos_token_id=[vocab - 1], max_position_embeddings=4096)
    d.update(kw)
    return RolesunConfig(**d)


def tensor_shapes(cfg: RolesunConfig):
    """{checkpoint tensor name: shape}."""
    W = cfg.width
    out = {"embed": (cfg.vocab, W)}
    for i, L in enumerate(cfg.layers):
        p, m = "l%d." % i, L["mixer"]
        H, R, x = m["heads"], m["kv_rank"], p + "mix."
        out[p + "norm1"] = ()
        out[x + "q"] = (H * m["dim"], W)
        if m.get("kv_from") is None:
            out.update({x + "dkv": (R, W), x + "dkv.norm": (R,)})
        out.update({x + "uk": (H * m["dim"], R), x + "uv": (H * m["vdim"], R), x + "g": (H * m["vdim"], W),
                    x + "o": (W, H * m["vdim"]), p + "shift": (W,), p + "rg1": (W, W), p + "rg1.b": (W,)})
        if L["mlp"] is not None:
            ff = L["mlp"]["ff"]
            out.update({p + "norm2": (), p + "mlp.gate": (ff, W), p + "mlp.up": (ff, W), p + "mlp.down": (W, ff),
                        p + "rg2": (W, W), p + "rg2.b": (W,)})
    out.update({"final.norm": (), "head": (cfg.vocab, W)})
    return out


def rolesun_state_dict(cfg: RolesunConfig, seed=0, device="cpu", dtype=torch.bfloat16):
    """Random weights of the architecture, generated on `device`."""
    g = torch.Generator(device=device).manual_seed(seed)
    sd = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".")[-1]
        r = torch.randn(shape, generator=g, device=device)
        if "norm" in leaf:
            t = 1 + 0.2 * r
        elif name == "embed":
            t = r
        elif leaf == "shift":
            t = torch.sigmoid(r)
        elif leaf == "b":
            t = 0.5 * r
        elif leaf in ("rg1", "rg2"):
            t = 0.5 * r * shape[-1] ** -0.5
        else:
            t = r * shape[-1] ** -0.5
        sd[name] = t.to(dtype)
    return sd


def write_rolesun_checkpoint(out_dir, cfg: RolesunConfig, seed=0, tokenizer=True):
    from ..runtime.safetensors_io import save_file

    os.makedirs(out_dir, exist_ok=True)
    with open(os.path.join(out_dir, "config.json"), "w") as f:
        json.dump(cfg.to_dict(), f, indent=2)
    save_file(rolesun_state_dict(cfg, seed), os.path.join(out_dir, "model.safetensors"), metadata={"format": "pt"})
    if tokenizer and not os.path.exists(os.path.join(out_dir, "tokenizer.json")):
        from ..utils.synthetic import train_small_bpe

        train_small_bpe(out_dir, cfg.vocab)
        with open(os.path.join(out_dir, "generation_config.json"), "w") as f:
            json.dump({"bos_token_id": cfg.bos_token_id, "eos_token_id": cfg.eos_token_id, "do_sample": True}, f)
