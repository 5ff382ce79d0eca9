"""Plain, slow Niduvik: every mechanism as one function over a whole sequence, no cache, no batching.

Independent of the framework (torch CPU tensors and loops only); float64 by default so that what a
comparison shows is the product path's rounding. Weights come as {name: tensor}, the configuration
as the dict of config.json.
"""
import math

import torch


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def group_rms_norm(x, w, eps, groups):
    T, n = x.shape
    p = x.reshape(T, groups, n // groups)
    p = p / torch.sqrt((p * p).mean(-1, keepdim=True) + eps)
    return p.reshape(T, n) * w


def silu(z):
    return z / (1 + torch.exp(-z))


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30))))


def distance_bucket(n, rows, far):
    """Bucket of distance n >= 0: exact up to half the table, then logarithmic up to `far`."""
    half = rows // 2
    if n < half:
        return n
    # floor(ln(n/half) / ln(far/half) * (rows - half)), the largest k with (far/half)^k <= (n/half)^(rows-half)
    m, k = rows - half, 0
    while half + k < rows - 1 and far ** (k + 1) * half ** m <= n ** m * half ** (k + 1):
        k += 1
    return half + k


def distance_bias(rel, far, T):
    """[T, T, heads]: rel[bucket(i - j)] for j <= i, 0 elsewhere."""
    rows, H = rel.shape
    by_n = torch.stack([rel[distance_bucket(n, rows, far)] for n in range(T)]) if T else rel[:0]
    out = torch.zeros(T, T, H, dtype=rel.dtype)
    for i in range(T):
        out[i, :i + 1] = by_n[:i + 1].flip(0)
    return out


def visible(T, size, keep):
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep))


def sink_softmax(s, mask):
    """exp(s_j) / (1 + sum_j exp(s_j)) over the visible j (last dim)."""
    s = torch.where(mask, s, torch.full_like(s, -math.inf))
    m = torch.clamp(s.max(-1, keepdim=True).values, min=0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def attention_core(q, k, v, gate_logits, rel, scale, softcap, far, size, keep):
    """q [T,H,dk], k [T,G,dk], v [T,G,dv], gate logits [T,H] -> [T,H,dv]."""
    T, H = q.shape[:2]
    G = k.shape[1]
    bias = distance_bias(rel, far, T)
    mask = visible(T, size, keep)
    gate = 1 / (1 + torch.exp(-gate_logits))
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        s = softcap * torch.tanh(s / softcap) + bias[:, :, h]
        out[:, h] = sink_softmax(s, mask) @ v[:, g] * gate[:, h:h + 1]
    return out


def mix_values(v, v_first, lam):
    return (1 - lam) * v + lam * v_first


def attention(h, W, p, c, v_first):
    """Returns (output [T, width], this layer's own values [T, kv_heads * vdim])."""
    T = h.shape[0]
    H, G, dk, dv = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q = h @ W[p + "q"].T + W[p + "q.b"]
    k = h @ W[p + "k"].T + W[p + "k.b"]
    own = h @ W[p + "v"].T + W[p + "v.b"]
    v = own if v_first is None else mix_values(own, v_first, W[p + "vmix"])
    out = attention_core(q.reshape(T, H, dk), k.reshape(T, G, dk), v.reshape(T, G, dv), h @ W[p + "g"].T, W[p + "rel"],
                         c["scale"], c["softcap"], c["bias_max"], c["mask"]["size"], c["mask"]["keep_first"])
    return out.reshape(T, H * dv) @ W[p + "o"].T, own


def causal_conv(u, w, b):
    """Per-channel causal convolution; w[:, -1] multiplies the current token."""
    T, taps = u.shape[0], w.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    y = b.expand(T, -1).clone()
    for t in range(taps):
        y = y + pad[t:t + T] * w[:, t]
    return y


def ssm(x, B, C, dt, A_log, D, state=None):
    """x [T,H,P], B/C [T,G,N], dt [T,H] (after softplus). Returns y [T,H,P], final state [H,N,P]."""
    T, H, P = x.shape
    G, N = B.shape[1:]
    S = torch.zeros(H, N, P, dtype=x.dtype) if state is None else state.clone()
    grp = torch.arange(H) // (H // G)
    y = torch.zeros_like(x)
    for t in range(T):
        decay = torch.exp(-torch.exp(A_log) * dt[t])
        S = decay[:, None, None] * S + dt[t][:, None, None] * B[t][grp][:, :, None] * x[t][:, None, :]
        y[t] = (S * C[t][grp][:, :, None]).sum(1) + D[:, None] * x[t]
    return y, S


def mamba2(h, W, p, c, eps):
    T = h.shape[0]
    H, P, N, G = c["heads"], c["vdim"], c["state"], c["groups"]
    inner = H * P
    z, x, B, C, dt = torch.split(h @ W[p + "in"].T, [inner, inner, G * N, G * N, H], 1)
    u = silu(causal_conv(torch.cat([x, B, C], 1), W[p + "conv"], W[p + "conv.b"]))
    x, B, C = torch.split(u, [inner, G * N, G * N], 1)
    dt = softplus(dt + W[p + "dt_bias"])
    y, _ = ssm(x.reshape(T, H, P), B.reshape(T, G, N), C.reshape(T, G, N), dt, W[p + "A_log"], W[p + "D"])
    y = group_rms_norm(y.reshape(T, inner) * silu(z), W[p + "norm"], eps, c["norm_groups"])
    return y @ W[p + "o"].T


def clipped_glu(h, gate, up, down, limit):
    g = torch.clamp(h @ gate.T, max=limit)
    u = torch.clamp(h @ up.T, -limit, limit)
    return (g / (1 + torch.exp(-1.702 * g)) * (u + 1)) @ down.T


def forward(cfg, weights, tokens, dtype=torch.float64, layers=None):
    """Logits [T, vocab]; `layers` (a list) receives the residual stream after every layer."""
    W = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    v_first = None
    for i, L in enumerate(cfg["layers"]):
        p, m = "l%d." % i, L["mixer"]
        h = rms_norm(x, W[p + "norm1"], eps)
        if L["type"] == "attention":
            y, own = attention(h, W, p + "mix.", m, v_first if m["v_mix"] else None)
            if m["v_mix"] and v_first is None:
                v_first = own
        else:
            y = mamba2(h, W, p + "mix.", m, eps)
        x = x + rms_norm(y, W[p + "norm1b"], eps)
        if L["mlp"] is not None:
            h = rms_norm(x, W[p + "norm2"], eps)
            y = clipped_glu(h, W[p + "mlp.gate"], W[p + "mlp.up"], W[p + "mlp.down"], L["mlp"]["limit"])
            x = x + rms_norm(y, W[p + "norm2b"], eps)
        if layers is not None:
            layers.append(x.clone())
    return rms_norm(x, W["final.norm"], eps) @ W["embed"].T
