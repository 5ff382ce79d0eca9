"""Model families the framework serves: config.json -> family -> weights, model, limits.

The server's builder, the trace replayer and the benchmarks all construct models here.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Callable, Optional, Tuple

import torch

DTYPES = {"bf16": torch.bfloat16, "bfloat16": torch.bfloat16, "fp8": torch.bfloat16, "fp32": torch.float32,
          "float32": torch.float32}


@dataclass(frozen=True)
class Family:
    name: str
    matches: Callable[[dict], bool]
    build: Callable  # (path, raw config, device, dtype name, tp_rank, tp_size, comm, max_len) -> model
    dtypes: Tuple[str, ...]
    # kernel sources (csrc/kernels) a forward step needs; None: the whole library
    kernels: Optional[Tuple[str, ...]] = None


def _llama(path, raw, device, dtype, tp_rank, tp_size, comm, max_len):
    from .llama import LlamaConfig, LlamaModel, LlamaWeights

    c = LlamaConfig.from_dict(raw)
    w = LlamaWeights.from_checkpoint(path, c, device, tp_rank, tp_size)
    if dtype == "fp8":  # e4m3fn linear weights, per-row scales
        w.quantize_fp8()
    return LlamaModel(c, w, device, comm=comm, max_positions=min(max_len, c.max_position_embeddings))


def _gpt2(path, raw, device, dtype, tp_rank, tp_size, comm, max_len):
    from .gpt2 import GPT2Config, GPT2Model, GPT2Weights

    c = GPT2Config.from_dict(raw)
    return GPT2Model(c, GPT2Weights.from_checkpoint(path, c, device), device)


def _niduvik(path, raw, device, dtype, tp_rank, tp_size, comm, max_len):
    from .niduvik import NiduvikConfig, NiduvikModel, NiduvikWeights

    c = NiduvikConfig.from_dict(raw)
    return NiduvikModel(c, NiduvikWeights.from_checkpoint(path, c, device, DTYPES[dtype]), device, comm=comm)


def _rolesun(path, raw, device, dtype, tp_rank, tp_size, comm, max_len):
    from .rolesun import RolesunConfig, RolesunModel, RolesunWeights

    c = RolesunConfig.from_dict(raw)
    return RolesunModel(c, RolesunWeights.from_checkpoint(path, c, device, DTYPES[dtype]), device, comm=comm)


def _names(raw):
    return {str(x).lower() for x in [raw.get("model_type"), raw.get("architecture")] + list(raw.get("architectures") or [])
            if x}


FAMILIES = (
    Family("niduvik", lambda raw: "niduvik" in _names(raw), _niduvik, ("bf16", "float32"),
           ("gemm.hip", "gemm_w4.hip", "gemm_pp.hip", "gemm_stream.hip", "gemm_dec.hip", "gemm_part.hip", "gemm_f32.hip",
            "norm.hip", "residual.hip", "attn_shaped.hip", "ssm.hip", "sampling.hip")),
    Family("rolesun", lambda raw: "rolesun" in _names(raw), _rolesun, ("bf16", "float32"),
           ("gemm.hip", "gemm_w4.hip", "gemm_pp.hip", "gemm_stream.hip", "gemm_dec.hip", "gemm_part.hip", "gemm_f32.hip",
            "norm.hip", "residual.hip", "attn_shaped.hip", "latent.hip", "sampling.hip")),
    Family("gpt2", lambda raw: "gpt2" in _names(raw), _gpt2, ("bf16",)),
    Family("llama", lambda raw: True, _llama, ("bf16", "fp8")),
)


def read_config(path):
    p = os.path.join(path, "config.json")
    if not os.path.exists(p):
        raise FileNotFoundError("no config.json under %s" % path)
    with open(p) as f:
        return json.load(f)


def family_of(raw: dict) -> Family:
    return next(f for f in FAMILIES if f.matches(raw))


def norm_dtype(dtype):
    return {"bfloat16": "bf16", "fp32": "float32"}.get(dtype, dtype)


def build_model(path, device, dtype="bf16", raw=None, tp_rank=0, tp_size=1, comm=None, max_len=1 << 30):
    """The model of a checkpoint directory on `device`."""
    raw = read_config(path) if raw is None else raw
    fam = family_of(raw)
    if norm_dtype(dtype) not in fam.dtypes:
        raise ValueError("%s does not run in %s (supported: %s)" % (fam.name, dtype, ", ".join(fam.dtypes)))
    return fam.build(path, raw, device, norm_dtype(dtype), tp_rank, tp_size, comm, max_len)


def model_limits(model):
    """(longest sequence, end-of-sequence ids) of a model's configuration."""
    c = model.cfg
    n = getattr(c, "max_position_embeddings", None) or getattr(c, "n_positions", None) or 1 << 30
    eos = c.eos_token_id
    return n, list(eos) if isinstance(eos, (list, tuple)) else [eos]
