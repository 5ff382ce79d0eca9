"""Configurations and weights shared by the Niduvik tests (CPU and GPU)."""
import niduvik_oracle as O
from decoder_util import limit, make_engine, pieces, prompt, run, worst  # noqa: F401
from rag_llm_k8s_amd.models.niduvik import (NiduvikConfig, NiduvikModel, NiduvikWeights, niduvik_state_dict,
                                            niduvik_tiny)


def _att(**o):
    m = dict(heads=6, kv_heads=2, dim=40, vdim=24, scale=0.17, softcap=15.0, bias_max=90, v_mix=True,
             mask=dict(size=70, keep_first=3))
    m.update(o)
    return dict(type="attention", mixer=m)


def _ssm(**o):
    m = dict(heads=6, vdim=20, state=24, groups=3, conv=3, norm_groups=2)
    m.update(o)
    return dict(type="mamba2", mixer=m)


def _with(layer, mlp):
    return dict(layer, mlp=mlp)


def make_config(name):
    """(config, rows of the distance table). Between them: head sizes that need padding and that do not, 1 / 3 /
    4 / 20 query heads per value head, no kept tokens and more of them than a page, short and long windows,
    2 to 5 taps, value sizes that are multiples of 8, of 4 and of neither, one norm group and many."""
    if name == "odd":
        return niduvik_tiny(vocab=301), 16
    if name == "wide":
        mlp = dict(kind="dense", ff=128, limit=1.0)
        a = _att(heads=8, dim=128, vdim=72, scale=0.09, softcap=30.0, bias_max=24, mask=dict(size=33, keep_first=0))
        s = _ssm(heads=4, vdim=64, state=128, groups=1, conv=4, norm_groups=4)
        L = [_with(s, mlp), _with(a, mlp), _with(s, None), _with(a, mlp)]
        return NiduvikConfig(vocab=128, width=256, eps=1e-6, layers=L), 8
    if name == "many":
        mlp = dict(kind="dense", ff=330, limit=7.0)
        a = _att(heads=40, dim=20, vdim=200, scale=0.22, softcap=50.0, bias_max=600, mask=dict(size=200, keep_first=70))
        b = _att(heads=2, kv_heads=2, dim=200, vdim=32, scale=0.07, softcap=8.0, bias_max=40, v_mix=False,
                 mask=dict(size=64, keep_first=64))
        s = _ssm(heads=6, vdim=8, state=40, groups=6, conv=2, norm_groups=3)
        L = [_with(b, mlp), _with(a, mlp), _with(s, mlp), _with(a, None)]
        return NiduvikConfig(vocab=77, width=96, eps=1e-5, layers=L), 32
    if name == "narrow":
        mlp = dict(kind="dense", ff=64, limit=3.0)
        a = _att(heads=4, kv_heads=1, dim=32, vdim=64, scale=1.0, softcap=20.0, bias_max=50, mask=dict(size=1, keep_first=1))
        s = _ssm(heads=3, vdim=12, state=16, groups=1, conv=5, norm_groups=1)
        t = _ssm(heads=2, vdim=96, state=256, groups=2, conv=4, norm_groups=2)
        L = [_with(a, mlp), _with(s, mlp), _with(t, mlp), _with(_att(heads=4, kv_heads=1, dim=32, vdim=64), mlp)]
        return NiduvikConfig(vocab=64, width=128, eps=1e-5, layers=L), 10
    raise KeyError(name)


CONFIGS = ("odd", "wide", "many", "narrow")


def make_model(name, device, dtype, seed=1):
    """(config dict, raw weights, model)."""
    cfg, rows = make_config(name)
    sd = niduvik_state_dict(cfg, seed, rel_rows=rows)
    m = NiduvikModel(cfg, NiduvikWeights.from_state_dict(cfg, sd, device, dtype), device)
    return cfg.to_dict(), sd, m


def oracle(cfg, sd, toks):
    return O.forward(cfg, sd, toks)
