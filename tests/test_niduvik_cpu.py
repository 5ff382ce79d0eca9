"""Niduvik on the CPU backend: mechanisms, caches, scheduler and trace replay against the plain implementation."""
import json
import math
import os
import subprocess
import sys

import pytest
import torch

import niduvik_oracle as O
import niduvik_util as U
from decoder_cases import Cases
from rag_llm_k8s_amd.engine.kv_manager import SequenceCache, StateSlots, make_block_manager
from rag_llm_k8s_amd.models import registry
from rag_llm_k8s_amd.models.niduvik import NiduvikConfig, niduvik_tiny, write_niduvik_checkpoint
from rag_llm_k8s_amd.ops.specs import AttnSpec, SsmSpec, distance_table, log_bucket

C = Cases(U)
F32 = torch.float32
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.mark.parametrize("rows,far", [(16, 90), (32, 128), (8, 40), (10, 77), (2, 9), (64, 4096), (7, 30)])
def test_distance_buckets(rows, far):
    got = [log_bucket(n, rows, far) for n in range(far + 60)]
    assert got == [O.distance_bucket(n, rows, far) for n in range(far + 60)]
    assert got == sorted(got) and got[-1] == rows - 1
    half = rows / 2
    if rows % 2 == 0:
        for n in range(rows // 2, far):
            x = math.log(n / half) / math.log(far / half) * (rows - half)
            if abs(x - round(x)) > 1e-9:
                assert got[n] == min(rows - 1, int(half + math.floor(x)))
    # exact powers: 8, 16, 32, 64 are whole steps of a table whose far end is 128
    assert [log_bucket(n, 16, 128) for n in (8, 15, 16, 31, 32, 64, 127, 128)] == [8, 9, 10, 11, 12, 14, 15, 15]


def test_distance_table_is_constant_past_far():
    rel = torch.randn(12, 3)
    t = distance_table(rel, 50)
    assert t.shape == (3, 51)
    for n in (0, 5, 6, 20, 49, 50):
        assert torch.equal(t[:, n], rel[O.distance_bucket(n, 12, 50)])
    assert O.distance_bucket(51, 12, 50) == O.distance_bucket(5000, 12, 50) == 11


def test_specs_reject_uneven_shapes():
    with pytest.raises(ValueError):
        AttnSpec(heads=6, kv_heads=4, dim=8, vdim=8, scale=1.0)
    with pytest.raises(ValueError):
        AttnSpec(heads=2, kv_heads=2, dim=300, vdim=8, scale=1.0)
    with pytest.raises(ValueError):
        SsmSpec(heads=5, vdim=8, state=8, groups=2, taps=4, norm_groups=1)
    with pytest.raises(ValueError):
        SsmSpec(heads=4, vdim=9, state=8, groups=2, taps=4, norm_groups=5)
    d = niduvik_tiny().to_dict()
    d["layers"][3]["mixer"] = dict(d["layers"][3]["mixer"], vdim=16)
    with pytest.raises(ValueError, match="mix values"):
        NiduvikConfig.from_dict(d)


def test_oracle_is_sensitive():
    """The comparisons below can see each mechanism: a planted mistake in the oracle moves the logits."""
    cfg, sd, _ = U.make_model("odd", "cpu", F32)
    t = U.prompt(cfg, 120, 2)
    want = O.forward(cfg, sd, t)

    def moved(change_cfg=None, change_sd=None):
        c, s = json.loads(json.dumps(cfg)), dict(sd)
        if change_cfg:
            change_cfg(c)
        if change_sd:
            change_sd(s)
        return U.worst(O.forward(c, s, t), want)

    def mixers(c, kind, key, f):
        for L in c["layers"]:
            if L["type"] == kind:
                L["mixer"][key] = f(L["mixer"][key])

    big = 10 * U.limit(F32)
    assert moved(lambda c: mixers(c, "attention", "mask", lambda m: dict(m, size=m["size"] - 1))) > big
    assert moved(lambda c: mixers(c, "attention", "mask", lambda m: dict(m, keep_first=m["keep_first"] - 1))) > big
    assert moved(lambda c: mixers(c, "attention", "bias_max", lambda n: n + 8)) > big
    assert moved(lambda c: mixers(c, "attention", "softcap", lambda n: n * 1.5)) > big
    assert moved(lambda c: mixers(c, "attention", "v_mix", lambda n: False)) > big
    assert moved(lambda c: mixers(c, "mamba2", "norm_groups", lambda n: 1)) > big
    assert moved(lambda c: c["layers"][0]["mlp"].update(limit=2.0)) > big
    for name in ("l1.mix.conv.b", "l1.mix.D", "l1.mix.dt_bias", "l1.mix.A_log", "l0.mix.g", "l0.mix.k.b", "l0.mix.rel",
                 "l3.mix.vmix", "l0.norm1b", "l0.norm2b"):
        assert moved(change_sd=lambda s: s.update({name: s[name] * 0.5})) > big, name
    assert moved(change_sd=lambda s: s.update({"l0.mix.vmix": s["l0.mix.vmix"] * 0.5})) == 0.0  # the source's own is unused


@pytest.mark.parametrize("dtype", [F32, torch.bfloat16])
@pytest.mark.parametrize("name", U.CONFIGS)
def test_whole_prompt(name, dtype):
    C.whole_prompt("cpu", dtype, name)


@pytest.mark.parametrize("name", U.CONFIGS)
def test_layers(name):
    C.layers("cpu", F32, name)


@pytest.mark.parametrize("name", U.CONFIGS)
def test_token_by_token(name):
    C.token_by_token("cpu", F32, name)


@pytest.mark.parametrize("size", [2, 3, 17, 64])
def test_portions(size):
    C.portions("cpu", F32, "odd", size)
    C.portions("cpu", F32, "narrow", size)


def test_portions_by_budget():
    C.portions("cpu", F32, "many", 64, budget=30)


@pytest.mark.parametrize("name", U.CONFIGS)
def test_unequal_batch(name):
    C.unequal_batch("cpu", F32, name)


def test_reuse():
    C.reuse("cpu", F32, "odd")


def test_long_decode():
    C.long_decode("cpu", F32, "odd")


@pytest.mark.parametrize("name", U.CONFIGS)
def test_greedy(name):
    C.greedy("cpu", F32, name)


def test_state_slots():
    c = SequenceCache(make_block_manager(10), StateSlots(3))
    assert c.can_allocate(1, 64)
    c.ensure(1, 64)
    c.ensure(2, 64)
    assert {c.state(1), c.state(2)} == {1, 2}  # slot 0 is scratch
    assert not c.can_allocate(3, 1) and c.can_allocate(2, 128)
    with pytest.raises(MemoryError):
        c.ensure(3, 1)
    s = c.state(1)
    c.free(1)
    c.ensure(3, 1)
    assert c.state(3) == s
    c.free(3), c.free(3)  # twice is harmless
    assert c.slots.available() == 1
    with pytest.raises(ValueError):
        StateSlots(1)


def test_feed_refuses_what_does_not_fit():
    cfg, _, m = U.make_model("odd", "cpu", F32)
    eng = U.make_engine(m, tokens=128, batch=2)
    s = eng.open_sequence()
    with pytest.raises(ValueError):
        eng.feed([(s, [0] * 129, [])])
    a, b, c = (eng.open_sequence() for _ in range(3))
    eng.feed([(a, [1], []), (b, [1], [])])
    with pytest.raises(MemoryError):
        eng.feed([(c, [1], [])])


def test_registry(tmp_path):
    cfg = niduvik_tiny(vocab=100)
    raw = cfg.to_dict()
    assert registry.family_of(raw).name == "niduvik"
    assert registry.family_of({"model_type": "gpt2"}).name == "gpt2"
    assert registry.family_of({"model_type": "llama"}).name == registry.family_of({}).name == "llama"
    write_niduvik_checkpoint(str(tmp_path), cfg, tokenizer=False)
    m = registry.build_model(str(tmp_path), "cpu", "float32")
    assert m.dtype == F32 and registry.model_limits(m) == (4096, [99])
    with pytest.raises(ValueError, match="does not run in"):
        registry.build_model(str(tmp_path), "cpu", "fp8")
    from rag_llm_k8s_amd import _build

    srcs, _ = _build.hip_sources(registry.family_of(raw).kernels)
    assert len(srcs) == len(registry.family_of(raw).kernels)


def test_served_by_the_builder(tmp_path):
    """The server's own construction path: config.json -> engine + tokenizer, text in, tokens out."""
    from rag_llm_k8s_amd.config import RagConfig
    from rag_llm_k8s_amd.engine.llm_engine import SamplingParams
    from rag_llm_k8s_amd.server.builder import build_generator

    write_niduvik_checkpoint(str(tmp_path), niduvik_tiny(vocab=512))
    cfg = RagConfig.from_env(model_path=str(tmp_path), device="cpu", max_batch=2, max_model_len=256, kv_cache_blocks=16)
    eng, tok, _ = build_generator(cfg, "cpu")
    ids = tok.encode("what is in the document?")
    out = eng.generate([ids, ids[:3]], SamplingParams(max_new_tokens=5, temperature=0.8, top_k=20, ignore_eos=True),
                       seeds=[1, 2])
    assert [len(o) for o in out] == [5, 5] and all(0 <= t < 512 for o in out for t in o)


def test_trace_run(tmp_path):
    cfg = niduvik_tiny(vocab=90)
    write_niduvik_checkpoint(str(tmp_path / "m"), cfg, seed=4, tokenizer=False)
    from rag_llm_k8s_amd.models.niduvik import niduvik_state_dict

    sd = niduvik_state_dict(cfg, 4)
    a, b = U.prompt(cfg.to_dict(), 80, 1), U.prompt(cfg.to_dict(), 5, 2)
    out = tmp_path / "out"
    out.mkdir()
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:77], "want": [0, 63, 76]},
                                     {"id": "b", "tokens": b[:3], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[77:78], "want": []},
                                     {"id": "b", "tokens": b[3:4], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[78:79], "want": [0]},
                                     {"id": "b", "tokens": b[4:5], "want": [0]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": a[79:], "want": [0]}], "end": ["a"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "128", "--device", "cpu"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True,
                       env=dict(os.environ, PATH=os.path.dirname(sys.executable) + ":" + os.environ["PATH"]))
    assert r.returncode == 0, r.stderr
    assert r.stdout.split("\n")[:4] == ["done %d" % i for i in range(4)]
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]

    def rows(i):
        return torch.frombuffer(bytearray((out / ("%d.f32" % i)).read_bytes()), dtype=F32).reshape(-1, 90)

    wa, wb = O.forward(cfg.to_dict(), sd, a), O.forward(cfg.to_dict(), sd, b)
    assert U.worst(rows(0), wa[[0, 63, 76]]) < U.limit(F32)
    assert U.worst(rows(2), torch.stack([wa[78], wb[4]])) < U.limit(F32)
    assert U.worst(rows(3), wa[79:]) < U.limit(F32)


def test_trace_run_refuses_a_dtype_with_status_3(tmp_path):
    from rag_llm_k8s_amd.replay import EXIT_DTYPE, main

    (tmp_path / "config.json").write_text('{"model_type": "llama"}')
    assert main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path)]) == EXIT_DTYPE == 3
