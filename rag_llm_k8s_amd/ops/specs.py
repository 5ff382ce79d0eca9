"""Parameters of the sequence mixers beyond plain causal attention (shared by both backends).

A spec holds what a kernel needs to know about one layer: sizes, constants, and where each part sits in
the layer's fused projection row. Head sizes are padded to what the MFMA kernels tile (zero weight rows, so
padding changes no result); the padded sizes are the ones in memory.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field

import torch


def ceil_to(n: int, m: int) -> int:
    return -(-n // m) * m


HEAD_PADS = (32, 64, 128, 256)  # per-head sizes the attention kernels are built for


def pad_head(d: int) -> int:
    for p in HEAD_PADS:
        if d <= p:
            return p
    raise ValueError("head size %d exceeds %d" % (d, HEAD_PADS[-1]))


@dataclass
class AttnSpec:
    """Grouped-query attention with separate key / value sizes and optional score shaping:
    s = softcap(q.k * scale) + bias[h][min(i - j, far)], a sliding window that always keeps the first
    tokens, a softmax whose denominator holds one extra zero score, and one sigmoid gate per head.
    Projection row: [q: heads x dkp | k: kv_heads x dkp | v: kv_heads x dvp | gate: heads]."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float = 0.0  # 0: off
    window: int = 0  # 0: unlimited
    keep_first: int = 0
    sink: bool = False
    gate: bool = False
    far: int = 0  # last distance of the bias table (larger distances use it); bias off when no table is given
    bias_bound: float = math.inf  # largest |bias| of the table, when known
    dkp: int = field(init=False)
    dvp: int = field(init=False)

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ValueError("heads (%d) must be a multiple of kv_heads (%d)" % (self.heads, self.kv_heads))
        self.dkp, self.dvp = pad_head(self.dim), pad_head(self.vdim)

    @property
    def group(self):
        return self.heads // self.kv_heads

    @property
    def off_k(self):
        return self.heads * self.dkp

    @property
    def off_v(self):
        return self.off_k + self.kv_heads * self.dkp

    @property
    def off_g(self):
        return self.off_v + self.kv_heads * self.dvp

    @property
    def row(self):
        return ceil_to(self.off_g + (self.heads if self.gate else 0), 64)

    @property
    def out_row(self):
        return ceil_to(self.heads * self.dvp, 128)

    @property
    def bounded(self):
        """Every score's exponential, and a sum of a million of them, fits fp32: no running maximum needed."""
        return self.softcap > 0 and (self.softcap + self.bias_bound) * 1.4427 < 80.0

    @property
    def heads_per_block(self):
        """Query heads of one KV head that a prefill block takes (its 4 waves split heads x 32-row groups)."""
        return 4 if self.group % 4 == 0 else (2 if self.group % 2 == 0 else 1)

    @property
    def q_tile(self):
        return 128 // self.heads_per_block


@dataclass
class SsmSpec:
    """Selective state space layer (scalar decay per head). Projection row:
    [z: inner | x: inner | B: groups x state | C: groups x state | dt: heads]."""
    heads: int
    vdim: int
    state: int
    groups: int
    taps: int
    norm_groups: int

    def __post_init__(self):
        if self.heads % self.groups:
            raise ValueError("heads (%d) must be a multiple of groups (%d)" % (self.heads, self.groups))
        if self.inner % self.norm_groups:
            raise ValueError("inner size %d does not split into %d norm groups" % (self.inner, self.norm_groups))

    @property
    def inner(self):
        return self.heads * self.vdim

    @property
    def channels(self):
        return self.inner + 2 * self.groups * self.state

    @property
    def off_x(self):
        return self.inner

    @property
    def off_dt(self):
        return self.inner + self.channels

    @property
    def row(self):
        return ceil_to(self.off_dt + self.heads, 64)

    @property
    def out_row(self):
        return ceil_to(self.inner, 128)


MAX_RANK = 1024  # widest latent row the latent-attention kernels take


@dataclass
class LatentSpec:
    """Latent attention: one cached latent row of `rank` columns per token, keys and values of every head linear in
    it, a sliding window, one sigmoid output gate per value element. `own` layers project and cache the latent;
    others read an earlier layer's. Projection row: [q: heads x dkp | gate: heads x dvp | latent: rp if own]."""
    heads: int
    dim: int
    vdim: int
    rank: int
    scale: float
    window: int = 0  # 0: unlimited
    own: bool = True
    dkp: int = field(init=False)
    dvp: int = field(init=False)
    rp: int = field(init=False)

    q_tile = 128  # query rows of a prefill block: one head, 4 waves of 32

    def __post_init__(self):
        self.dkp, self.dvp, self.rp = pad_head(self.dim), pad_head(self.vdim), ceil_to(self.rank, 128)
        if self.rp > MAX_RANK:
            raise ValueError("latent size %d exceeds %d" % (self.rank, MAX_RANK))

    @property
    def off_g(self):
        return self.heads * self.dkp

    @property
    def off_c(self):
        return self.off_g + self.heads * self.dvp

    @property
    def row(self):
        return ceil_to(self.off_c + (self.rp if self.own else 0), 64)

    @property
    def off_v(self):
        """First value column of the expanded key / value rows [k: heads x dkp | v: heads x dvp]."""
        return self.heads * self.dkp

    @property
    def kv_row(self):
        return self.heads * (self.dkp + self.dvp)

    @property
    def out_row(self):
        return ceil_to(self.heads * self.dvp, 128)


def log_bucket(n: int, rows: int, far: int) -> int:
    """Distance bucket: n itself below half = rows // 2, then half + floor(ln(n / half) / ln(far / half) *
    (rows - half)), at most rows - 1. Evaluated in exact integers, so a boundary distance lands in the
    bucket that the formula names."""
    half = rows // 2
    if n < half:
        return n
    if n >= far or half == 0 or far <= half:
        return rows - 1
    m, k = rows - half, 0
    a, b = n ** m, half ** m
    while half + k + 1 < rows and a * half ** (k + 1) >= b * far ** (k + 1):
        k += 1
    return half + k


def distance_table(rel: torch.Tensor, far: int) -> torch.Tensor:
    """[heads, far + 1] fp32: the learned bias of every distance 0 .. far (beyond far it stays constant)."""
    rows = rel.shape[0]
    idx = torch.tensor([log_bucket(n, rows, far) for n in range(far + 1)], dtype=torch.long)
    return rel.float()[idx].t().contiguous()
