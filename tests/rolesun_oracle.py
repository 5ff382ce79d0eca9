"""Plain, slow Rolesun: every mechanism as one function over a whole sequence, no cache, no batching.

Independent of the framework (torch CPU tensors and loops only); float64 by default so that what a
comparison shows is the product path's rounding. Weights come as {name: tensor}, the configuration
as the dict of config.json.
"""
import math

import torch


def sinusoid(positions, width, dtype=torch.float64):
    """[T, width]: sin at even columns, cos at odd ones, of p / 10000^(2i / width) for column pair i."""
    out = torch.zeros(len(positions), width, dtype=dtype)
    for c in range(width):
        i = c // 2
        for t, p in enumerate(positions):
            a = p * 10000.0 ** (-2.0 * i / width)
            out[t, c] = math.cos(a) if c % 2 else math.sin(a)
    return out


def embed(tokens, table, scale):
    x = table[torch.as_tensor(tokens, dtype=torch.long)] * scale
    return x + sinusoid(range(len(tokens)), table.shape[1], x.dtype)


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def token_shift(h, mix):
    """h_t + (h_{t-1} - h_t) * mix, h_{-1} = 0."""
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        prev = h[t - 1] if t > 0 else torch.zeros_like(h[0])
        out[t] = h[t] + (prev - h[t]) * mix
    return out


def output_gate(y, h, w, b):
    """y * sigmoid(W h + b)."""
    return y * sigmoid(h @ w.T + b)


def residual_add(x, y, g, eps, mult):
    """x + mult * rms(y) * g, g one number."""
    return x + mult * rms(y, eps) * g


def latent(h, w, norm, eps):
    return rms(h @ w.T, eps) * norm


def visible(T, size):
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    return (j <= i) & (i - j < size)


def latent_attention_core(q, c, uk, uv, scale, size):
    """q [T, H, d], c [T, R], uk [H, d, R], uv [H, e, R] -> [T, H, e]."""
    T, H, _ = q.shape
    mask = visible(T, size)
    out = torch.zeros(T, H, uv.shape[1], dtype=q.dtype)
    for h in range(H):
        k, v = c @ uk[h].T, c @ uv[h].T
        s = (q[:, h] @ k.T) * scale
        s = torch.where(mask, s, torch.full_like(s, -math.inf))
        e = torch.exp(s - s.max(-1, keepdim=True).values)
        out[:, h] = (e / e.sum(-1, keepdim=True)) @ v
    return out


def latent_attention(h, c, W, p, m):
    T = h.shape[0]
    H, d, e, R = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
    q = (h @ W[p + "q"].T).reshape(T, H, d)
    o = latent_attention_core(q, c, W[p + "uk"].reshape(H, d, R), W[p + "uv"].reshape(H, e, R), m["scale"],
                              m["mask"]["size"])
    return (o.reshape(T, H * e) * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def gated_mlp(h, gate, up, down):
    g = h @ gate.T
    return (g * sigmoid(g) * (h @ up.T)) @ down.T


def forward(cfg, weights, tokens, dtype=torch.float64, layers=None):
    """Logits [T, vocab]; `layers` (a list) receives the residual stream after every layer."""
    W = {k: v.to(dtype) for k, v in weights.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = embed(tokens, W["embed"], cfg["embedding"]["scale"])
    latents = {}
    for i, L in enumerate(cfg["layers"]):
        p, m = "l%d." % i, L["mixer"]
        h = token_shift(x, W[p + "shift"])
        src = m.get("kv_from")
        if src is None:
            latents[i] = latent(h, W[p + "mix.dkv"], W[p + "mix.dkv.norm"], eps)
        y = latent_attention(h, latents[i if src is None else src], W, p + "mix.", m)
        x = residual_add(x, output_gate(y, x, W[p + "rg1"], W[p + "rg1.b"]), W[p + "norm1"], eps, mult)
        if L["mlp"] is not None:
            y = gated_mlp(x, W[p + "mlp.gate"], W[p + "mlp.up"], W[p + "mlp.down"])
            x = residual_add(x, output_gate(y, x, W[p + "rg2"], W[p + "rg2.b"]), W[p + "norm2"], eps, mult)
        if layers is not None:
            layers.append(x.clone())
    return rms(x, eps) * W["final.norm"] @ W["head"].T * cfg["logit_scale"]
