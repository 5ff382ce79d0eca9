"""Drivers shared by the decoder families' tests (CPU and GPU)."""
import torch

from rag_llm_k8s_amd.engine.llm_engine import LLMEngine


def make_engine(m, tokens=1024, batch=8, **kw):
    return LLMEngine(m, num_blocks=tokens // 64 + batch + 2, max_batch=batch, max_model_len=tokens, **kw)


def prompt(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def limit(dtype):
    """Largest allowed rms error of a position's logits, relative to the logits' rms."""
    return 3e-5 if dtype == torch.float32 else 0.04


def worst(got, want):
    d = got.double() - want.double()
    return float((d.pow(2).mean(-1).sqrt() / want.double().pow(2).mean().sqrt()).max())


def run(engine, seqs, plan):
    """Feed sequences by a plan (list of steps, each {name: count}); every position's logits, {name: [T, vocab]}."""
    live, at, out = {}, {k: 0 for k in seqs}, {k: [] for k in seqs}
    for step in plan:
        entries = []
        for k, n in step.items():
            if k not in live:
                live[k] = engine.open_sequence()
            entries.append((live[k], seqs[k][at[k]:at[k] + n], list(range(n))))
        lg, row = engine.feed(entries), 0
        for k, n in step.items():
            out[k].append(lg[row:row + n])
            row, at[k] = row + n, at[k] + n
            if at[k] == len(seqs[k]):
                engine.close_sequence(live.pop(k))
    for s in live.values():
        engine.close_sequence(s)
    return {k: torch.cat(v) for k, v in out.items()}


def pieces(total, size):
    return [min(size, total - i) for i in range(0, total, size)]
