"""Rolesun on the CPU backend: mechanisms, caches, scheduler and trace replay against the plain implementation."""
import json
import os
import subprocess
import sys
from types import SimpleNamespace

import pytest
import torch

import rolesun_oracle as O
import rolesun_util as U
from decoder_cases import Cases
from rag_llm_k8s_amd.models import registry
from rag_llm_k8s_amd.models.rolesun import (RolesunConfig, rolesun_state_dict, rolesun_tiny, tensor_shapes,
                                            write_rolesun_checkpoint)
from rag_llm_k8s_amd.ops import reference_seq as RS
from rag_llm_k8s_amd.ops.seq_native import key_rows
from rag_llm_k8s_amd.ops.specs import LatentSpec

C = Cases(U)
F32 = torch.float32
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def test_spec_sizes_and_limits():
    s = LatentSpec(heads=3, dim=24, vdim=40, rank=130, scale=0.5)
    assert (s.dkp, s.dvp, s.rp, s.off_g, s.off_c) == (32, 64, 256, 96, 288)
    assert s.row == 576 and s.kv_row == 288 and s.out_row == 256
    assert LatentSpec(heads=3, dim=24, vdim=40, rank=130, scale=0.5, own=False).row == 320
    for bad in (dict(dim=300), dict(vdim=257), dict(rank=1025)):
        with pytest.raises(ValueError):
            LatentSpec(**dict(dict(heads=1, dim=8, vdim=8, rank=8, scale=1.0), **bad))


def test_config_refuses_unusable_sources():
    def build(change):
        d = json.loads(json.dumps(rolesun_tiny().to_dict()))
        change(d["layers"])
        return RolesunConfig.from_dict(d)

    build(lambda L: None)
    with pytest.raises(ValueError, match="kv_from"):
        build(lambda L: L[2]["mixer"].update(kv_from=2))
    with pytest.raises(ValueError, match="kv_from"):
        build(lambda L: L[3]["mixer"].update(kv_from=2))  # a layer that has no latents of its own
    with pytest.raises(ValueError, match="kv_rank"):
        build(lambda L: L[2]["mixer"].update(kv_from=1))
    with pytest.raises(ValueError, match="mixer type"):
        build(lambda L: L[0].update(type="attention"))
    with pytest.raises(ValueError, match="mlp kind"):
        build(lambda L: L[0]["mlp"].update(kind="moe"))


@pytest.mark.parametrize("width", [6, 7, 128])
def test_sinusoid(width):
    pos = [0, 1, 2, 63, 1000, 40000]
    i = torch.arange((width + 1) // 2, dtype=torch.float64)
    turns = 10000.0 ** (-2 * i / width) / (2 * torch.pi)
    got = RS.sinusoid(torch.tensor(pos), turns, width, width + 3)
    assert torch.allclose(got[:, :width].double(), O.sinusoid(pos, width), atol=2e-7, rtol=0)
    assert float(got[:, width:].abs().max()) == 0


def test_token_shift_in_portions():
    g = torch.Generator().manual_seed(0)
    x, mix = torch.randn(40, 16, generator=g), torch.rand(16, generator=g)
    want = O.token_shift(x, mix)
    for size in (1, 2, 7, 40):
        state, got = torch.full((3, 16), 9.0), []
        for lo in range(0, 40, size):
            p = x[lo:lo + size]
            got.append(RS.token_shift(p, mix, state, [len(p)], [lo + len(p)], [2]))
        assert torch.equal(torch.cat(got), want)
        assert torch.equal(state[2], x[-1]) and float(state[:2].min()) == 9.0


def test_key_rows():
    """Which positions a prefill step expands: the new ones and the window's before them, from a page border."""
    k = key_rows([100, 5], [100, 5], 70, "cpu")
    assert not k.gather and k.tail == 0 and k.rows == 105
    assert k.cu_k.tolist() == [0, 100, 105] and k.key_off.tolist() == [0, 100]
    k = key_rows([10, 3, 1, 1], [300, 3, 500, 2], 70, "cpu")  # 290 tokens before: 221 .. 289 are visible, from page 3
    assert k.gather and (k.seqs, k.tail) == (2, 2)
    assert k.cu_k.tolist() == [0, 300 - 192, 300 - 192 + 3]
    assert k.key_off.tolist() == [-192, 108, 0, 0]
    assert k.tiles.tolist() == [[0, 0], [1, 0]]
    assert key_rows([2], [130], 0, "cpu").cu_k.tolist() == [0, 130]  # no window: everything
    assert key_rows([2], [130], 64, "cpu").cu_k.tolist() == [0, 66]  # 128 - 63 = 65: page 1
    assert key_rows([2], [129], 64, "cpu").cu_k.tolist() == [0, 65]  # 127 - 63 = 64: the border itself
    assert key_rows([2], [128], 64, "cpu").cu_k.tolist() == [0, 128]  # 126 - 63 = 63: one before it
    k = key_rows([1, 1], [1, 9], 64, "cpu")  # a first token is a prompt, whatever its length
    assert (k.seqs, k.tail, k.rows) == (1, 1, 1)
    k = key_rows([1, 1], [7, 9], 64, "cpu")
    assert (k.seqs, k.tail, k.rows) == (0, 2, 0)


def latent_case(T, spec, seed, pairs):
    """Latents, maps and queries whose scores stand out at the given (query, key) pairs."""
    g = torch.Generator().manual_seed(seed)
    c = torch.randn(T, spec.rank, generator=g)
    uk = torch.randn(spec.heads, spec.dim, spec.rank, generator=g) * spec.rank ** -0.5
    uv = torch.randn(spec.heads, spec.vdim, spec.rank, generator=g) * spec.rank ** -0.5
    q = 0.3 * torch.randn(T, spec.heads, spec.dim, generator=g)
    k = torch.einsum("tr,hdr->thd", c, uk)
    for i, j in pairs:
        q[i] = k[j] * (25.0 / spec.scale / (k[j] ** 2).sum(-1, keepdim=True))
    return c, uk, uv, q


def test_latent_attention_window_and_pages():
    """Keys just inside and outside the window, at page borders and far away, through scattered pages."""
    spec = LatentSpec(heads=2, dim=24, vdim=20, rank=72, scale=0.2, window=65)
    T = 200
    pairs = [(199, 199), (198, 198 - 64), (197, 197 - 65), (196, 0), (150, 128), (151, 127), (130, 66), (131, 66), (64, 0), (65, 0)]
    c, uk, uv, q = latent_case(T, spec, 3, pairs)
    gate = torch.randn(T, spec.heads, spec.vdim, generator=torch.Generator().manual_seed(4))
    want = O.latent_attention_core(q.double(), c.double(), uk.double(), uv.double(), spec.scale, 65) * O.sigmoid(gate.double())
    row = torch.zeros(T, spec.row)
    row[:, :spec.off_g].view(T, 2, 32)[:, :, :24] = q
    row[:, spec.off_g:spec.off_c].unflatten(1, (2, 32))[:, :, :20] = gate
    pages = torch.randn(6, 64, spec.rp)
    bt = torch.tensor([[5, 1, 3, 2]], dtype=torch.int32)
    p = torch.arange(T)
    lat = torch.zeros(T, spec.rp)
    lat[:, :72] = c
    pages[bt[0, p // 64].long(), p % 64] = lat
    wuk, wuv = torch.zeros(2, spec.rp, 32), torch.zeros(2, 32, spec.rp)
    wuk[:, :72, :24], wuv[:, :20, :72] = uk.transpose(1, 2), uv
    got = RS.latent_attention(row, spec, wuk, wuv, pages, bt, [T], [T], torch.zeros(T, spec.out_row))
    got = got[:, :64].reshape(T, 2, 32)[:, :, :20]
    assert U.worst(got.reshape(T, -1), want.reshape(T, -1)) < 1e-5
    moved = O.latent_attention_core(q.double(), c.double(), uk.double(), uv.double(), spec.scale, 64) * O.sigmoid(gate.double())
    assert (moved - want).abs().amax((1, 2))[[198, 130]].min() > 0.1  # one token fewer shows where a key is at the edge


def test_gated_residual():
    g = torch.Generator().manual_seed(1)
    h, y, z, b = (torch.randn(*s, generator=g) for s in ((4, 24), (4, 24), (4, 24), (24,)))
    gate = y.double() * O.sigmoid(z.double() + b.double())
    want = O.residual_add(h.double(), gate, 1.3, 1e-4, 0.45)
    got = h.clone()
    RS.gated_residual(got, torch.stack([0.25 * y, 0.75 * y]), z, b, torch.full((24,), 1.3 * 0.45), 1e-4, 24)
    assert torch.allclose(got.double(), want, atol=1e-6)


def test_oracle_is_sensitive():
    """The comparisons below can see each mechanism: a planted mistake in the oracle moves the logits."""
    cfg, sd, _ = U.make_model("odd", "cpu", F32)
    t = U.prompt(cfg, 150, 2)
    want = O.forward(cfg, sd, t)

    def moved(change_cfg=None, change_sd=None):
        c, s = json.loads(json.dumps(cfg)), dict(sd)
        if change_cfg:
            change_cfg(c)
        if change_sd:
            change_sd(s)
        return U.worst(O.forward(c, s, t), want)

    big = 10 * U.limit(F32)
    for li in range(4):
        assert moved(lambda c: c["layers"][li]["mixer"]["mask"].update(size=c["layers"][li]["mixer"]["mask"]["size"] - 1)) > big
    assert moved(lambda c: c["layers"][0]["mixer"].update(scale=0.2)) > big
    assert moved(lambda c: c.update(residual_mult=0.41)) > big
    assert moved(lambda c: c["embedding"].update(scale=0.71)) > big
    assert moved(lambda c: c["norm"].update(eps=1e-2)) > big
    assert moved(lambda c: c.update(logit_scale=1.6)) > big
    assert moved(lambda c: c["layers"][2]["mixer"].pop("kv_from"), lambda s: s.update(
        {"l2.mix.dkv": sd["l0.mix.dkv"], "l2.mix.dkv.norm": sd["l0.mix.dkv.norm"]})) > big
    for name in tensor_shapes(U.make_config("odd")):
        # matrices change their rows' order: a mere scale goes out in the norm behind many of them
        wrong = sd[name].flip(0) if sd[name].dim() == 2 else sd[name] * 0.5
        assert moved(change_sd=lambda s: s.update({name: wrong})) > big, name


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


def test_registry(tmp_path):
    cfg = rolesun_tiny(vocab=100)
    raw = cfg.to_dict()
    assert registry.family_of(raw).name == "rolesun"
    write_rolesun_checkpoint(str(tmp_path), cfg, tokenizer=False)
    m = registry.build_model(str(tmp_path), "cpu", "float32")
    assert m.dtype == F32 and registry.model_limits(m) == (4096, [99])
    # latents of three layers (the fourth reads the first's) and one row of state per layer
    assert m.kv_bytes_per_block() == 64 * 4 * (128 + 256 + 128) and m.state_bytes_per_slot() == 4 * 4 * 256
    with pytest.raises(ValueError, match="does not run in"):
        registry.build_model(str(tmp_path), "cpu", "fp8")
    with pytest.raises(ValueError, match="one GPU per engine"):
        registry.build_model(str(tmp_path), "cpu", "bf16", comm=SimpleNamespace(size=2))
    from rag_llm_k8s_amd import _build

    srcs, _ = _build.hip_sources(registry.family_of(raw).kernels)
    assert len(srcs) == len(registry.family_of(raw).kernels)


def test_served_by_the_builder(tmp_path):
    """The server's own construction path: config.json -> engine + tokenizer, text in, tokens out."""
    from rag_llm_k8s_amd.config import RagConfig
    from rag_llm_k8s_amd.engine.llm_engine import SamplingParams
    from rag_llm_k8s_amd.server.builder import build_generator

    write_rolesun_checkpoint(str(tmp_path), rolesun_tiny(vocab=512))
    cfg = RagConfig.from_env(model_path=str(tmp_path), device="cpu", max_batch=2, max_model_len=256, kv_cache_blocks=16)
    eng, tok, _ = build_generator(cfg, "cpu")
    ids = tok.encode("what is in the document?")
    out = eng.generate([ids, ids[:3]], SamplingParams(max_new_tokens=5, temperature=0.8, top_k=20, ignore_eos=True),
                       seeds=[1, 2])
    assert [len(o) for o in out] == [5, 5] and all(0 <= t < 512 for o in out for t in o)


def test_trace_run(tmp_path):
    cfg = rolesun_tiny(vocab=90)
    write_rolesun_checkpoint(str(tmp_path / "m"), cfg, seed=4, tokenizer=False)
    sd = rolesun_state_dict(cfg, 4)
    a, b = U.prompt(cfg.to_dict(), 80, 1), U.prompt(cfg.to_dict(), 4, 2)
    out = tmp_path / "out"
    out.mkdir()
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:78], "want": [0, 63, 77]},
                                     {"id": "b", "tokens": b[:3], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[78:79], "want": [0]},
                                     {"id": "b", "tokens": b[3:], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[79:], "want": [0]}], "end": ["a"]}]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "128", "--device", "cpu"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True,
                       env=dict(os.environ, PATH=os.path.dirname(sys.executable) + ":" + os.environ["PATH"]))
    assert r.returncode == 0, r.stderr
    assert r.stdout.split("\n")[:3] == ["done %d" % i for i in range(3)]

    def rows(i):
        return torch.frombuffer(bytearray((out / ("%d.f32" % i)).read_bytes()), dtype=F32).reshape(-1, 90)

    wa, wb = O.forward(cfg.to_dict(), sd, a), O.forward(cfg.to_dict(), sd, b)
    assert U.worst(rows(0), wa[[0, 63, 77]]) < U.limit(F32)
    assert U.worst(rows(1), torch.stack([wa[78], wb[3]])) < U.limit(F32)
    assert U.worst(rows(2), wa[79:]) < U.limit(F32)
