"""Plain, slow implementation of the hybrid decoder designs (attention / gated-delta layers,
a looped middle section), in torch on the CPU, one function per mechanism.

It shares no code with the product path: it reads a configuration dictionary and a
dictionary of tensors, always runs a whole sequence from its first token, and walks
recurrences token by token.  ``dtype`` (default float64) is the precision of everything.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last dimension."""
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def norm_around_one(x, w, eps):
    """RMS norm whose stored weight is the offset from one."""
    return rms(x, eps) * (1 + w)


def rotate_pairs(x, dims, base, pos0=0):
    """x [T, heads, d]: neighbours (2i, 2i+1) of the first `dims` dimensions turn by
    p * base^(-2i/dims); the other dimensions pass."""
    out = x.clone()
    p = torch.arange(pos0, pos0 + x.shape[0], dtype=torch.float64)
    for i in range(dims // 2):
        a = p * base ** (-2.0 * i / dims)
        c, s = a.cos().to(x.dtype)[:, None], a.sin().to(x.dtype)[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i] = u * c - v * s
        out[:, :, 2 * i + 1] = v * c + u * s
    return out


def attend_with_sink(q, k, v, scale, heads, kv_heads):
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e]: causal; the denominator of the
    softmax carries one extra exp(0)."""
    T = q.shape[0]
    out = torch.zeros(T, heads, v.shape[-1], dtype=q.dtype)
    mask = torch.ones(T, T, dtype=torch.bool).tril()
    for h in range(heads):
        g = h // (heads // kv_heads)
        s = (q[:, h] @ k[:, g].t()) * scale
        s = torch.where(mask, s, torch.full_like(s, -math.inf))
        top = torch.clamp(s.max(-1, keepdim=True).values, min=0.0)
        e = torch.exp(s - top)
        out[:, h] = (e @ v[:, g]) / (torch.exp(-top) + e.sum(-1, keepdim=True))
    return out


def attention_mixer(h, w, p, m, eps):
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[p + ".q"].t()).view(T, H, d)
    k = (h @ w[p + ".k"].t()).view(T, G, d)
    v = (h @ w[p + ".v"].t()).view(T, G, e)
    q = rms(rotate_pairs(q, m["rot"]["dims"], m["rot"]["base"]), eps)
    k = rms(rotate_pairs(k, m["rot"]["dims"], m["rot"]["base"]), eps)
    o = attend_with_sink(q, k, v, m["scale"], H, G).reshape(T, H * e)
    o = o * torch.sigmoid(h @ w[p + ".g"].t())
    return o @ w[p + ".o"].t()


def short_conv_silu(x, w):
    """x [T, C], w [C, taps], the last column on the current token; zeros before the start."""
    T, taps = x.shape[0], w.shape[1]
    y = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            src = t - (taps - 1 - j)
            if src >= 0:
                y[t] += w[:, j] * x[src]
    return y * torch.sigmoid(y)


def unit(x):
    return x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)


def softplus(x):
    return torch.where(x > 30, x, torch.log1p(torch.exp(torch.clamp(x, max=30.0))))


def delta_rule(q, k, v, beta, decay, heads, kv_heads):
    """q, k [T, G, d], v [T, H, e], beta / decay [T, H] -> [T, H, e]."""
    T, d, e = q.shape[0], q.shape[-1], v.shape[-1]
    out = torch.zeros(T, heads, e, dtype=q.dtype)
    for h in range(heads):
        g = h // (heads // kv_heads)
        S = torch.zeros(d, e, dtype=q.dtype)
        for t in range(T):
            S = decay[t, h] * S
            u = beta[t, h] * (v[t, h] - S.t() @ k[t, g])
            S = S + torch.outer(k[t, g], u)
            out[t, h] = S.t() @ q[t, g]
    return out


def delta_mixer(h, w, p, m, eps):
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = short_conv_silu(h @ w[p + ".q"].t(), w[p + ".q.conv"]).view(T, G, d)
    k = short_conv_silu(h @ w[p + ".k"].t(), w[p + ".k.conv"]).view(T, G, d)
    v = short_conv_silu(h @ w[p + ".v"].t(), w[p + ".v.conv"]).view(T, H, e)
    q, k = unit(q) * d ** -0.5, unit(k)
    beta = torch.sigmoid(h @ w[p + ".b"].t())
    decay = torch.exp(-torch.exp(w[p + ".A_log"]) *
                      softplus(h @ w[p + ".a"].t() + w[p + ".dt_bias"]))
    o = delta_rule(q, k, v, beta, decay, H, G)
    o = rms(o, eps) * w[p + ".norm"]
    z = (h @ w[p + ".g"].t()).view(T, H, e)
    return (o * z * torch.sigmoid(z)).reshape(T, H * e) @ w[p + ".o"].t()


def gelu_exact(x):
    return 0.5 * x * (1 + torch.erf(x / math.sqrt(2.0)))


def dense_mlp(h, w, p):
    return gelu_exact(h @ w[p + ".up"].t()) @ w[p + ".down"].t()


MIXERS = {"attention": attention_mixer, "delta": delta_mixer}


def layer(x, w, cfg, i):
    L = cfg["layers"][i]
    eps = cfg["norm"]["eps"]
    h = norm_around_one(x, w[f"l{i}.norm1"], eps)
    y = MIXERS[L["type"]](h, w, f"l{i}.mix", L["mixer"], eps)
    if L.get("mlp") is not None:
        y = y + dense_mlp(h, w, f"l{i}.mlp")
    return x + cfg["residual_mult"] * y


def enter_pass(x, x0, w, t):
    return torch.cat([x, x0], -1) @ w["loop.in"].t() + w["loop.step"][t]


def run_order(cfg):
    """[(layer, pass or None)] as executed."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, None) for i in range(n)]
    mid = [(i, t) for t in range(lp["times"]) for i in range(lp["start"], lp["stop"])]
    return ([(i, None) for i in range(lp["start"])] + mid +
            [(i, None) for i in range(lp["stop"], n)])


def forward(cfg, weights, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one sequence; layers_out collects x after every layer run."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    x0 = w["embed"][torch.as_tensor(tokens)]
    x = x0
    for i, t in run_order(cfg):
        if t is not None and i == cfg["loop"]["start"]:
            x = enter_pass(x, x0, w, t)
        x = layer(x, w, cfg, i)
        if layers_out is not None:
            layers_out.append(x)
    return norm_around_one(x, w["final.norm"], cfg["norm"]["eps"]) @ w["head"].t()
