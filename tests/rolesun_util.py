"""Configurations and weights shared by the Rolesun tests (CPU and GPU)."""
import rolesun_oracle as O
from decoder_util import limit, make_engine, pieces, prompt, run, worst  # noqa: F401
from rag_llm_k8s_amd.models.rolesun import (RolesunConfig, RolesunModel, RolesunWeights, rolesun_state_dict,
                                            rolesun_tiny)


def _att(**o):
    m = dict(heads=5, dim=24, vdim=40, kv_rank=56, scale=0.21, mask=dict(size=70))
    m.update(o)
    return dict(type="latent_attention", mixer=m)


def _ff(n):
    return dict(kind="dense", ff=n)


def make_config(name):
    """Between them: head sizes that need padding and that do not, key sizes below and above value sizes, 1 to 33
    heads, latents of 40 to 700 columns, windows of 1 to 200, layers that read another's latents with other heads and
    windows (also two of one source), layers without an mlp first and last, an odd width."""
    if name == "odd":
        return rolesun_tiny(vocab=301)
    if name == "wide":
        big = dict(heads=20, dim=64, vdim=64, kv_rank=256, scale=0.125, mask=dict(size=33))
        L = [dict(_att(**big), mlp=None), dict(_att(**dict(big, heads=6, dim=128, vdim=96, kv_from=0, mask=dict(size=100))),
                                               mlp=_ff(128)), dict(_att(**dict(big, kv_rank=512)), mlp=_ff(384))]
        return RolesunConfig(vocab=128, width=256, eps=1e-6, layers=L, embed_scale=2.0, residual_mult=1.0, logit_scale=0.25)
    if name == "many":
        a = dict(heads=33, dim=16, vdim=8, kv_rank=40, scale=0.3, mask=dict(size=200))
        L = [dict(_att(**a), mlp=_ff(330)), dict(_att(**dict(a, heads=2, dim=200, vdim=130, kv_from=0, scale=0.05)), mlp=_ff(64)),
             dict(_att(**dict(a, kv_from=0, heads=17, mask=dict(size=64))), mlp=None)]
        return RolesunConfig(vocab=77, width=96, eps=1e-5, layers=L, embed_scale=1.0, residual_mult=0.7, logit_scale=1.0)
    if name == "narrow":
        L = [dict(_att(heads=1, dim=32, vdim=200, kv_rank=700, mask=dict(size=1)), mlp=_ff(64)),
             dict(_att(heads=2, dim=40, vdim=32, kv_rank=130, mask=dict(size=65)), mlp=_ff(72)),
             dict(_att(heads=3, dim=20, vdim=16, kv_rank=700, kv_from=0, mask=dict(size=64)), mlp=_ff(64))]
        return RolesunConfig(vocab=64, width=131, eps=1e-3, layers=L, embed_scale=0.3, residual_mult=0.25, logit_scale=3.0)
    raise KeyError(name)


CONFIGS = ("odd", "wide", "many", "narrow")


def weights(cfg, seed=1, sharp=3.0):
    """Random weights whose attention is decided by few keys (queries scaled up)."""
    sd = rolesun_state_dict(cfg, seed)
    return {k: v * sharp if k.endswith(".mix.q") else v for k, v in sd.items()}


def make_model(name, device, dtype, seed=1):
    """(config dict, raw weights, model)."""
    cfg = make_config(name)
    sd = weights(cfg, seed)
    return cfg.to_dict(), sd, RolesunModel(cfg, RolesunWeights.from_state_dict(cfg, sd, device, dtype), device)


def oracle(cfg, sd, toks):
    return O.forward(cfg, sd, toks)
