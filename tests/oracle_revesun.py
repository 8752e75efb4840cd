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


# ------------------------------------------------------------------ configurations and weights
def attention(heads, kv, dim, vdim, conv, chunk, base, rdims, scale, ff=0):
    return {"type": "attention", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv, "scale": scale,
                      "mask": {"size": chunk}, "rot": {"base": base, "dims": rdims}}}


def mingru(width, ff=0):
    return {"type": "mingru", "mlp": {"kind": "dense", "ff": ff} if ff else None, "mixer": {"width": width}}


def config(width, vocab, groups, layers, eps=1e-5):
    return {"architecture": "Revesun", "width": width, "vocab": vocab, "norm": {"groups": groups, "eps": eps},
            "layers": layers}


def tensor_shapes(cfg):
    h = cfg["width"]
    out = {"embed": (cfg["vocab"], h), "final.norm": (h,)}
    for i, layer in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", layer["mixer"]
        out[p + "norm1"] = (h,)
        if layer["type"] == "mingru":
            w = mx["width"]
            out.update({p + "mix.z": (w, h), p + "mix.z.b": (w,), p + "mix.x": (w, h), p + "mix.x.b": (w,),
                        p + "mix.g": (w, h), p + "mix.o": (h, w)})
        else:
            rows = {"q": mx["heads"] * mx["dim"], "k": mx["kv_heads"] * mx["dim"], "v": mx["kv_heads"] * mx["vdim"]}
            for n, r in rows.items():
                out[p + f"mix.{n}"] = (r, h)
                out[p + f"mix.{n}.conv"] = (r, mx["conv"])
            out[p + "mix.g"] = (mx["heads"] * mx["vdim"], h)
            out[p + "mix.o"] = (h, mx["heads"] * mx["vdim"])
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            out.update({p + "norm2": (h,), p + "mlp.up": (ff, h), p + "mlp.down": (h, ff), p + "mlp.act": (4,)})
    return out


def random_weights(cfg, seed=0):
    """bf16 tensors under the checkpoint's names, scaled so that every term of a layer counts."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        if "norm" in name:
            t = 1 + 0.2 * t
        elif name.endswith(".conv"):
            t = 0.3 * t
            t[:, -1] += 1.0
        elif name.endswith(".act"):
            t = torch.tensor([0.6, 0.35, 0.25, 0.1]) + 0.05 * t
        elif name.endswith(".b"):
            t = 0.5 * t
        elif len(shape) == 2:
            t = t * (1.0 if name == "embed" else 1.3 / math.sqrt(shape[1]))
        out[name] = t.to(torch.bfloat16)
    return out


def save(cfg, weights, path):
    """Write a model directory."""
    import json
    import os

    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(weights, os.path.join(path, "model.safetensors"))
    return str(path)


def greedy(cfg, weights, prompt, n, dt=torch.float64):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(forward(cfg, weights, seq, dt)[-1].argmax()))
    return seq[len(prompt):]
