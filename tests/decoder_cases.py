"""Model-level checks of a decoder family, run on the CPU backend and on the GPU kernels alike.

Every check compares logits at all positions with the plain implementation's. `U` is the family's util module:
make_model(name, device, dtype) and oracle(config, weights, tokens), beside what decoder_util brings.
"""
import torch


class Cases:
    def __init__(self, util):
        self.U = util

    def whole_prompt(self, dev, dtype, name):
        U = self.U
        cfg, sd, m = U.make_model(name, dev, dtype)
        t = U.prompt(cfg, 231, 3)
        got = U.run(U.make_engine(m), {"a": t}, [{"a": len(t)}])["a"]
        assert U.worst(got, U.oracle(cfg, sd, t)) < U.limit(dtype)

    def layers(self, dev, dtype, name):
        """The residual stream after every layer."""
        U = self.U
        from rag_llm_k8s_amd.engine.llm_engine import RUNNING, SamplingParams, Sequence

        cfg, sd, m = U.make_model(name, dev, dtype)
        eng = U.make_engine(m)
        t = U.prompt(cfg, 90, 4)
        s = Sequence(t, SamplingParams(), 0)
        s.status = RUNNING
        eng.bm.ensure(s.id, len(t))
        inp, _, _ = eng._prefill_input([(s, 0, len(t))])
        got, want = [], []
        m.hidden_states(inp, trace=got)
        U.O.forward(cfg, sd, t, layers=want)
        assert len(got) == len(want)
        for g, w in zip(got, want):
            assert g.dtype == torch.float32
            assert U.worst(g.cpu(), w) < U.limit(dtype)

    def token_by_token(self, dev, dtype, name):
        U = self.U
        cfg, sd, m = U.make_model(name, dev, dtype)
        t = U.prompt(cfg, 150, 5)
        got = U.run(U.make_engine(m), {"a": t}, [{"a": 1}] * len(t))["a"]
        assert U.worst(got, U.oracle(cfg, sd, t)) < U.limit(dtype)

    def portions(self, dev, dtype, name, size, budget=None):
        """A prompt in portions, then decoding; `budget`: the engine's own prefill budget does the cutting."""
        U = self.U
        cfg, sd, m = U.make_model(name, dev, dtype)
        t = U.prompt(cfg, 140 if size < 5 else 210, 6)
        eng = U.make_engine(m, **({} if budget is None else dict(max_prefill_tokens=budget)))
        n = len(t) - 9
        plan = [{"a": n}] if budget else [{"a": k} for k in U.pieces(n, size)]
        got = U.run(eng, {"a": t}, plan + [{"a": 1}] * 9)["a"]
        assert U.worst(got, U.oracle(cfg, sd, t)) < U.limit(dtype)

    def unequal_batch(self, dev, dtype, name):
        """Requests of unequal length in one batch against the same requests alone and against the oracle."""
        U = self.U
        cfg, sd, m = U.make_model(name, dev, dtype)
        lens = {"a": 1, "b": 2, "c": 67, "d": 130, "e": 201}
        dec = {"a": 5, "b": 3, "c": 12, "d": 9, "e": 12}
        seqs = {k: U.prompt(cfg, n + dec[k], 10 + n) for k, n in lens.items()}
        plan = [dict(lens)] + [{k: 1 for k in lens if i < dec[k]} for i in range(12)]
        got = U.run(U.make_engine(m), seqs, plan)
        for k in seqs:
            alone = U.run(U.make_engine(m), {k: seqs[k]}, [{k: lens[k]}] + [{k: 1}] * dec[k])[k]
            assert U.worst(got[k], alone) < U.limit(dtype)
            assert U.worst(got[k], U.oracle(cfg, sd, seqs[k])) < U.limit(dtype)

    def reuse(self, dev, dtype, name):
        """Pages and slots that come back: more requests, one after the other, than either holds at once."""
        U = self.U
        cfg, sd, m = U.make_model(name, dev, dtype)
        eng = U.make_engine(m, tokens=256, batch=2)
        free = eng.bm.free_blocks()
        for i in range(5):
            a, b = U.prompt(cfg, 100 + 20 * i, 30 + i), U.prompt(cfg, 3 + i, 40 + i)
            got = U.run(eng, {"a": a, "b": b}, [{"a": len(a) - 4, "b": len(b) - 2}] + [{"a": 1, "b": 1}] * 2 + [{"a": 1}] * 2)
            assert U.worst(got["a"], U.oracle(cfg, sd, a)) < U.limit(dtype)
            assert U.worst(got["b"], U.oracle(cfg, sd, b)) < U.limit(dtype)
            assert eng.bm.free_blocks() == free
            if eng.bm.slots is not None:
                assert eng.bm.slots.available() == 2

    def long_decode(self, dev, dtype, name):
        """Decoding that passes the window, the page borders and the far end of the distance table."""
        U = self.U
        cfg, sd, m = U.make_model(name, dev, dtype)
        t = U.prompt(cfg, 420, 8)
        got = U.run(U.make_engine(m), {"a": t}, [{"a": 20}] + [{"a": 1}] * 400)["a"]
        assert U.worst(got, U.oracle(cfg, sd, t)) < U.limit(dtype)

    def greedy(self, dev, dtype, name):
        """Generation through the engine's own entry point and scheduler: mixed prefill + decode steps, small
        budgets, more requests than slots. Greedy tokens must be the oracle's wherever its choice is clear."""
        U = self.U
        from rag_llm_k8s_amd.engine.llm_engine import SamplingParams

        cfg, sd, m = U.make_model(name, dev, dtype)
        eng = U.make_engine(m, tokens=256, batch=3, max_prefill_tokens=48)
        prompts = [U.prompt(cfg, n, 50 + n) for n in (1, 2, 45, 100, 131)]
        outs = eng.generate(prompts, SamplingParams(max_new_tokens=12, do_sample=False, temperature=0.0, ignore_eos=True),
                            seeds=[0] * len(prompts))
        assert not eng.running and (eng.bm.slots is None or eng.bm.slots.available() == 3)
        tol = 6 * U.limit(dtype)
        for p, o in zip(prompts, outs):
            assert len(o) == 12
            lg = U.oracle(cfg, sd, p + o)[len(p) - 1:-1]
            scale = float(lg.pow(2).mean().sqrt())
            for i, tok in enumerate(o):
                assert float(lg[i].max() - lg[i][tok]) <= tol * scale, (i, tok)
