"""Plain, slow implementation of the Revesun decoder: one function per mechanism, one sequence at
a time, no cache, no batching, no code of the product.  The tests compare the framework with it.

Weights are a dict of tensors under the checkpoint's names; ``dt`` is the arithmetic type
(float64 by default, float32 to see what rounding alone does).
"""
from __future__ import annotations

import math

import torch


def group_norm(x, w, groups, eps):
    """x [T, W] in ``groups`` consecutive parts, each over its own root mean square, times w."""
    T, W = x.shape
    parts = x.view(T, groups, W // groups)
    r = torch.sqrt((parts * parts).mean(-1, keepdim=True) + eps)
    return (parts / r).reshape(T, W) * w


def causal_conv(u, taps_w):
    """y_t[c] = sum_j w[c, j] u_(t - taps + 1 + j)[c], zeros ahead of the first token."""
    T, C = u.shape
    n = taps_w.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(n):
            s = t - n + 1 + j
            if s >= 0:
                y[t] += taps_w[:, j] * u[s]
    return y


def rotate_pairs(x, positions, base, dims):
    """x [T, heads, D]: pairs (2i, 2i + 1) of the first ``dims`` dimensions turned by
    position * base^(-2i / dims)."""
    y = x.clone()
    for i in range(dims // 2):
        a = positions.to(x.dtype) * (float(base) ** (-2.0 * i / dims))
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i] = u * c - v * s
        y[..., 2 * i + 1] = v * c + u * s
    return y


def chunk_attention(q, k, v, scale, chunk):
    """q [T, H, D], k [T, G, D], v [T, G, E]: token i sees j <= i of its own chunk; the softmax's
    denominator has one added (a key of score 0 without a value)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        lo = (i // chunk) * chunk
        for h in range(H):
            g = h // (H // G)
            s = (k[lo:i + 1, g] @ q[i, h]) * scale
            m = max(float(s.max()), 0.0)
            e = torch.exp(s - m)
            out[i, h] = (e / (e.sum() + math.exp(-m))) @ v[lo:i + 1, g]
    return out


def min_gru(z_pre, u_pre, state=None):
    """z_pre, u_pre [T, C] (biases added): S_t = (1 - z) S_(t-1) + z c(u); returns (S [T, C])."""
    z = torch.sigmoid(z_pre)
    c = torch.where(u_pre >= 0, u_pre + 0.5, torch.sigmoid(u_pre))
    s = torch.zeros(z.shape[1], dtype=z.dtype) if state is None else state.clone()
    out = torch.empty_like(z)
    for t in range(z.shape[0]):
        s = (1 - z[t]) * s + z[t] * c[t]
        out[t] = s
    return out


def poly_norm(z, coef, eps):
    """a N(z) + b N(z^2) + c N(z^3) + e; N divides each token's vector by its root mean square."""
    def n(x):
        return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)

    a, b, c, e = coef[0], coef[1], coef[2], coef[3]
    return a * n(z) + b * n(z ** 2) + c * n(z ** 3) + e


def mingru_mixer(h, w, p):
    z = h @ w[p + "z"].T + w[p + "z.b"]
    u = h @ w[p + "x"].T + w[p + "x.b"]
    g = h @ w[p + "g"].T
    return (min_gru(z, u) * (g * torch.sigmoid(g))) @ w[p + "o"].T


def attention_mixer(h, w, p, mx):
    T = h.shape[0]
    H, G, D, E = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q, k, v = (causal_conv(h @ w[p + n].T, w[p + n + ".conv"]) for n in "qkv")
    pos = torch.arange(T)
    q = rotate_pairs(q.view(T, H, D), pos, mx["rot"]["base"], mx["rot"]["dims"])
    k = rotate_pairs(k.view(T, G, D), pos, mx["rot"]["base"], mx["rot"]["dims"])
    o = chunk_attention(q, k, v.view(T, G, E), mx["scale"], mx["mask"]["size"]).reshape(T, H * E)
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def forward(cfg, weights, tokens, dt=torch.float64, collect=None):
    """Logits [T, vocab]; ``collect`` (a list) receives the residual stream after every layer."""
    w = {k: t.to(dt) for k, t in weights.items()}
    groups, eps = cfg["norm"]["groups"], cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = group_norm(x, w[p + "norm1"], groups, eps)
        if layer["type"] == "mingru":
            x = x + mingru_mixer(h, w, p + "mix.")
        else:
            x = x + attention_mixer(h, w, p + "mix.", layer["mixer"])
        if layer.get("mlp"):
            h = group_norm(x, w[p + "norm2"], groups, eps)
            x = x + poly_norm(h @ w[p + "mlp.up"].T, w[p + "mlp.act"], eps) @ w[p + "mlp.down"].T
        if collect is not None:
            collect.append(x.clone())
    return group_norm(x, w["final.norm"], groups, eps) @ w["embed"].T
