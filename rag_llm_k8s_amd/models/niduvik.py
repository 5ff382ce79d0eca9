"""Niduvik: a decoder whose layers mix shaped attention and Mamba-2, with norms before and after each sublayer.

    x <- x + norm1b(mixer(norm1(x)));  x <- x + norm2b(mlp(norm2(x)))      (layers without an mlp skip the second)

Attention layers: grouped queries, no rotation -- positions enter through a learned logarithmic distance
bias and a sliding window that keeps the first tokens; soft-capped scores; a softmax with one extra zero
score in its denominator; a per-head sigmoid gate; values mixed with those of the first mixing layer.
The residual stream is fp32. Every size and constant comes from config.json ("layers" lists them per layer).
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass, field
from typing import List, Optional

import torch

from ..ops.backend import get_backend
from ..ops.specs import AttnSpec, SsmSpec, ceil_to
from .base import DecoderModel
from .mixers import AttentionMixer, ClippedGluMlp, Mamba2Mixer, pad1, pad2

GLU_ALPHA, GLU_SHIFT = 1.702, 1.0


@dataclass
class NiduvikConfig:
    vocab: int
    width: int
    eps: float
    layers: List[dict]  # {"type", "mixer": {...}, "mlp": {...} or None}
    bos_token_id: Optional[int] = None
    eos_token_id: List[int] = field(default_factory=list)
    max_position_embeddings: int = 131072
    model_type: str = "niduvik"

    @classmethod
    def from_dict(cls, d):
        eos = d.get("eos_token_id")
        c = cls(vocab=int(d["vocab"]), width=int(d["width"]), eps=float(d["norm"]["eps"]),
                layers=[dict(type=L["type"], mixer=dict(L["mixer"]), mlp=L.get("mlp")) for L in d["layers"]],
                bos_token_id=d.get("bos_token_id"),
                eos_token_id=[] if eos is None else (eos if isinstance(eos, list) else [eos]),
                max_position_embeddings=int(d.get("max_position_embeddings") or 131072))
        for i, L in enumerate(c.layers):
            if L["type"] not in ("attention", "mamba2"):
                raise ValueError("layer %d: unknown mixer type %r" % (i, L["type"]))
            if L["mlp"] is not None and L["mlp"].get("kind", "dense") != "dense":
                raise ValueError("layer %d: unknown mlp kind %r" % (i, L["mlp"]["kind"]))
        shapes = {(L["mixer"]["kv_heads"], L["mixer"]["vdim"]) for L in c.layers
                  if L["type"] == "attention" and L["mixer"].get("v_mix")}
        if len(shapes) > 1:
            raise ValueError("layers that mix values need one value shape, got %s" % sorted(shapes))
        return c

    @classmethod
    def from_json(cls, path):
        with open(path) as f:
            return cls.from_dict(json.load(f))

    def to_dict(self):
        d = {"architecture": "Niduvik", "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
             "layers": self.layers, "max_position_embeddings": self.max_position_embeddings}
        if self.bos_token_id is not None:
            d["bos_token_id"] = self.bos_token_id
        if self.eos_token_id:
            d["eos_token_id"] = self.eos_token_id
        return d

    @property
    def vocab_size(self):
        return self.vocab


def attention_spec(m):
    mask = m.get("mask") or {}
    return AttnSpec(heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], scale=float(m["scale"]),
                    softcap=float(m.get("softcap") or 0.0), window=int(mask.get("size") or 0),
                    keep_first=int(mask.get("keep_first") or 0), sink=True, gate=True, far=int(m["bias_max"]))


def ssm_spec(m):
    return SsmSpec(heads=m["heads"], vdim=m["vdim"], state=m["state"], groups=m["groups"], taps=m["conv"],
                   norm_groups=m["norm_groups"])


class NiduvikWeights:
    """Device weights in kernel layouts (matrices zero-padded to the GEMM tiles, norm weights fp32)."""

    tp_rank, vocab_offset = 0, 0

    @classmethod
    def from_get(cls, cfg: NiduvikConfig, get, device, dtype=torch.bfloat16):
        """`get(name)` returns a raw tensor."""
        w = cls()
        w.cfg, w.dtype = cfg, dtype
        wp = ceil_to(cfg.width, 128)
        device = torch.device(device)

        def dev(t, dt=dtype):
            return t.to(device=device, dtype=dt).contiguous()

        def norm(name):
            return dev(pad1(get(name).float(), wp), torch.float32)

        w.width_pad = wp
        w.embed = w.lm_head = dev(pad2(get("embed"), ceil_to(cfg.vocab, 8), wp))
        w.vocab_valid = cfg.vocab
        w.layers = []
        seen_mix = False
        for i, L in enumerate(cfg.layers):
            p, m = "l%d." % i, L["mixer"]

            def mix(name, p=p):
                return get(p + "mix." + name)

            if L["type"] == "attention":
                vm = bool(m.get("v_mix"))
                mixer = AttentionMixer.load(attention_spec(m), cfg.width, mix, dev, rel=mix("rel"),
                                            vmix=vm and seen_mix, v_source=vm and not seen_mix)
                seen_mix = seen_mix or vm
            else:
                mixer = Mamba2Mixer.load(ssm_spec(m), cfg.width, cfg.eps, mix, dev)
            layer = dict(mixer=mixer, norm1=norm(p + "norm1"), norm1b=norm(p + "norm1b"), mlp=None)
            if L["mlp"] is not None:
                layer.update(mlp=ClippedGluMlp.load(cfg.width, L["mlp"]["ff"], float(L["mlp"]["limit"]), GLU_ALPHA,
                                                    GLU_SHIFT, lambda n, p=p: get(p + "mlp." + n), dev),
                             norm2=norm(p + "norm2"), norm2b=norm(p + "norm2b"))
            w.layers.append(layer)
        w.norm = norm("final.norm")
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
            ts = [mx.wqkv, mx.wo] if isinstance(mx, AttentionMixer) else [mx.win, mx.wo]
            ts += [ml.wgu, ml.wdown] if ml is not None else []
            n += sum(t.numel() * t.element_size() for t in ts)
        return n + self.embed.numel() * self.embed.element_size()


class NiduvikModel(DecoderModel):
    def __init__(self, cfg: NiduvikConfig, weights: NiduvikWeights, device, comm=None, max_positions=None):
        if comm is not None and comm.size > 1:
            raise ValueError("Niduvik runs on one GPU per engine (use data-parallel replicas)")
        self.cfg, self.w, self.device = cfg, weights, torch.device(device)
        self.be = get_backend(self.device)
        self.dtype = weights.dtype
        self.comm, self.tp_rank = None, 0
        self.attn = [L["mixer"] for L in weights.layers if isinstance(L["mixer"], AttentionMixer)]
        self.ssm = [L["mixer"] for L in weights.layers if isinstance(L["mixer"], Mamba2Mixer)]
        self.recurrent = bool(self.ssm)

    # ---- caches and work lists the engine asks for
    def kv_bytes_per_block(self):
        size = torch.tensor([], dtype=self.dtype).element_size()
        return max(1, sum(a.cache_bytes(size) for a in self.attn))

    def allocate_kv_cache(self, num_blocks, dtype=None):
        for a in self.attn:
            a.allocate_cache(num_blocks, dtype or self.dtype, self.device)
        return [(a.kc, a.vc) for a in self.attn]

    def state_bytes_per_slot(self):
        return sum(s.state_bytes() for s in self.ssm)

    def allocate_state(self, num_slots):
        for s in self.ssm:
            s.allocate_state(num_slots, self.device)

    def prefill_work(self, q_lens, device):
        from ..ops.seq_native import query_tiles

        return None, {qt: query_tiles(q_lens, qt).to(device) for qt in sorted({a.spec.q_tile for a in self.attn})}

    def decode_work(self, max_kv_len, batch):
        from ..ops.seq_native import decode_split

        return decode_split([a.spec for a in self.attn], max_kv_len, batch, self.device)

    # ---- one step
    def hidden_states(self, inp, trace=None):
        """Final-normed rows selected by logits_idx. `trace` (a list) receives the residual after every layer."""
        be, w, c = self.be, self.w, self.cfg
        n, eps, dt = c.width, c.eps, self.dtype
        h = be.embed_residual(inp.ids, w.embed, carry=inp.carry, prev=inp.carry_src)
        xn = be.residual_norm(h, None, None, w.layers[0]["norm1"], eps, n, dt)
        shared = {}
        last = w.norm if inp.logits_idx is None else None  # a prompt's final norm runs on the selected rows only
        for li, L in enumerate(w.layers):
            nxt = w.layers[li + 1]["norm1"] if li + 1 < len(w.layers) else last
            y = L["mixer"].forward(be, xn, inp, shared)
            if L["mlp"] is None:
                xn = be.residual_norm(h, y, L["norm1b"], nxt, eps, n, dt)
            else:
                xn = be.residual_norm(h, y, L["norm1b"], L["norm2"], eps, n, dt)
                xn = be.residual_norm(h, L["mlp"].forward(be, xn, inp), L["norm2b"], nxt, eps, n, dt)
            if trace is not None:
                trace.append(h[:, :n].clone())
        if last is not None:
            return xn
        h = be.gather_rows(h, inp.logits_idx)
        return be.residual_norm(h, None, None, w.norm, eps, n, dt)

    def logits(self, hs):
        return self.be.gemm(hs, self.w.lm_head, out_f32=True)

    def forward(self, inp):
        return self.logits(self.hidden_states(inp))


# ------------------------------------------------------------------------------------- synthetic checkpoints
def niduvik_tiny(vocab=512, **kw):
    """Four small layers with every branch: both mixers, an attention layer without value mixing, a layer
    without an mlp."""
    def att(**o):
        m = dict(heads=6, kv_heads=2, dim=40, vdim=24, scale=0.17, softcap=15.0, bias_max=90, v_mix=True,
                 mask=dict(size=70, keep_first=3))
        m.update(o)
        return m

    ssm = dict(heads=6, vdim=20, state=24, groups=3, conv=3, norm_groups=2)
    mlp = dict(kind="dense", ff=200, limit=2.5)
    layers = [dict(type="attention", mixer=att(), mlp=mlp), dict(type="mamba2", mixer=ssm, mlp=mlp),
              dict(type="attention", mixer=att(v_mix=False, heads=4, kv_heads=4, dim=64, vdim=32), mlp=None),
              dict(type="attention", mixer=att(), mlp=mlp)]
    d = dict(vocab=vocab, width=144, eps=1e-5, layers=layers, bos_token_id=vocab - 2, eos_token_id=[vocab - 1],
             max_position_embeddings=4096)
    d.update(kw)
    return NiduvikConfig(**d)


def tensor_shapes(cfg: NiduvikConfig, rel_rows=16):
    """{checkpoint tensor name: shape}."""
    W = cfg.width
    out = {"embed": (cfg.vocab, W), "final.norm": (W,)}
    for i, L in enumerate(cfg.layers):
        p, m = "l%d." % i, L["mixer"]
        out.update({p + "norm1": (W,), p + "norm1b": (W,)})
        x = p + "mix."
        if L["type"] == "attention":
            H, G = m["heads"], m["kv_heads"]
            for n, r in (("q", H * m["dim"]), ("k", G * m["dim"]), ("v", G * m["vdim"])):
                out.update({x + n: (r, W), x + n + ".b": (r,)})
            out.update({x + "rel": (rel_rows, H), x + "vmix": (), x + "g": (H, W), x + "o": (W, H * m["vdim"])})
        else:
            s = ssm_spec(m)
            out.update({x + "in": (s.off_dt + s.heads, W), x + "conv": (s.channels, s.taps),
                        x + "conv.b": (s.channels,), x + "dt_bias": (s.heads,), x + "A_log": (s.heads,),
                        x + "D": (s.heads,), x + "norm": (s.inner,), x + "o": (W, s.inner)})
        if L["mlp"] is not None:
            ff = L["mlp"]["ff"]
            out.update({p + "norm2": (W,), p + "norm2b": (W,), p + "mlp.gate": (ff, W), p + "mlp.up": (ff, W),
                        p + "mlp.down": (W, ff)})
    return out


def niduvik_state_dict(cfg: NiduvikConfig, seed=0, rel_rows=16, device="cpu", dtype=torch.bfloat16):
    """Random weights of the architecture, generated on `device`."""
    g = torch.Generator(device=device).manual_seed(seed)
    sd = {}
    for name, shape in tensor_shapes(cfg, rel_rows).items():
        leaf = name.split(".")[-1]
        r = torch.randn(shape, generator=g, device=device)
        if "norm" in leaf:
            t = 1 + 0.1 * r
        elif name == "embed":
            t = r
        elif leaf == "vmix":
            t = torch.sigmoid(r)
        elif leaf == "dt_bias":
            t = -2.5 + r
        elif leaf == "A_log":
            t = -1.0 + 1.5 * r
        elif leaf == "D":
            t = 1 + 0.3 * r
        elif leaf in ("b", "rel"):
            t = 0.5 * r
        elif leaf == "conv":
            t = r * shape[1] ** -0.5
        else:
            t = r * shape[-1] ** -0.5
        sd[name] = t.to(dtype)
    return sd


def write_niduvik_checkpoint(out_dir, cfg: NiduvikConfig, seed=0, tokenizer=True):
    from ..runtime.safetensors_io import save_file

    os.makedirs(out_dir, exist_ok=True)
    with open(os.path.join(out_dir, "config.json"), "w") as f:
        json.dump(cfg.to_dict(), f, indent=2)
    save_file(niduvik_state_dict(cfg, seed), os.path.join(out_dir, "model.safetensors"), metadata={"format": "pt"})
    if tokenizer and not os.path.exists(os.path.join(out_dir, "tokenizer.json")):
        from ..utils.synthetic import train_small_bpe

        train_small_bpe(out_dir, cfg.vocab)
        with open(os.path.join(out_dir, "generation_config.json"), "w") as f:
            json.dump({"bos_token_id": cfg.bos_token_id, "eos_token_id": cfg.eos_token_id, "do_sample": True}, f)
