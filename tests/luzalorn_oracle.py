"""Plain, slow reference of the Luzalorn decoder, one function per mechanism.

Everything runs on whole sequences in float64 on the CPU: no cache, no
chunks, no batching, and no code shared with the package.  Notation: h is
the [T, width] input of a mixer, W a dict of this layer's weights by the
suffix of their tensor names.
"""

from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms(x, eps, weight=None):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def layer_norm(x, weight, bias, eps):
    mu = x.mean(-1, keepdim=True)
    dev = x - mu
    return dev / torch.sqrt((dev * dev).mean(-1, keepdim=True) + eps) \
        * weight + bias


def silu(z):
    return z / (1.0 + torch.exp(-z))


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def rotate(x, positions, dims, base):
    """x [T, H, D]: turn the pair (i, i + dims/2) by p * base^(-2i/dims)."""
    out = x.clone()
    for i in range(dims // 2):
        a = positions * base ** (-2.0 * i / dims)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[:, :, i], x[:, :, i + dims // 2]
        out[:, :, i] = u * c - v * s
        out[:, :, i + dims // 2] = v * c + u * s
    return out


def retention_recurrence(q, k, v, decay, state=None):
    """q, k [T, H, D] (k already scaled), v [T, H, E] -> (o [T, H, E],
    final state [H, D, E]); S <- decay S + k v^T, o = S^T q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F64) if state is None \
        else state.clone()
    g = torch.tensor(decay, dtype=F64)[:, None, None]
    out = []
    for t in range(T):
        S = g * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def retention(h, W, m, eps):
    T = h.shape[0]
    H, D, E = m["heads"], m["dim"], m["vdim"]
    pos = torch.arange(T, dtype=F64)
    q = (h @ W["q"].T).view(T, H, D)
    k = (h @ W["k"].T).view(T, H, D)
    v = (h @ W["v"].T).view(T, H, E)
    q = rotate(q, pos, m["rot"]["dims"], m["rot"]["base"])
    k = rotate(k, pos, m["rot"]["dims"], m["rot"]["base"]) * D ** -0.5
    o, _ = retention_recurrence(q, k, v, m["decay"])
    o = rms(o, eps).reshape(T, H * E)
    return (o * silu(h @ W["g"].T)) @ W["o"].T


def window_softmax_attention(q, k, v, scale, size, sink):
    """q, k [T, H, D], v [T, H, E]; row i sees 0 <= i - j < size, and
    exp(sink_h) stands in the denominator."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        s = (q[:, h] @ k[:, h].T) * scale
        for i in range(T):
            lo = 0 if size is None else max(0, i - size + 1)
            row = s[i, lo:i + 1]
            top = max(float(row.max()), float(sink[h]))
            e = torch.exp(row - top)
            den = e.sum() + math.exp(float(sink[h]) - top)
            out[i, h] = (e[:, None] * v[lo:i + 1, h]).sum(0) / den
    return out


def latent_attention(h, W, m, eps):
    T = h.shape[0]
    H, D, E = m["heads"], m["dim"], m["vdim"]
    cq = rms(h @ W["dq"].T, eps, W["dq.norm"])
    q = (cq @ W["uq"].T).view(T, H, D)
    c = rms(h @ W["dkv"].T, eps, W["dkv.norm"])
    k = (c @ W["uk"].T).view(T, H, D)
    v = (c @ W["uv"].T).view(T, H, E)
    size = (m.get("mask") or {}).get("size")
    o = window_softmax_attention(q, k, v, m["scale"], size, W["sink"])
    return (o.reshape(T, H * E) * sigmoid(h @ W["g"].T)) @ W["o"].T


def swiglu_ff(h, W):
    return (silu(h @ W["gate"].T) * (h @ W["up"].T)) @ W["down"].T


def layer_runs(cfg):
    """Order of (layer, pass) runs; pass is None outside the loop."""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return ([(i, None) for i in range(a)] +
            [(i, t) for t in range(loop["times"]) for i in range(a, b)] +
            [(i, None) for i in range(b, n)])


MIXERS = {"retention": retention, "latent_attention": latent_attention}


def sub(weights, prefix):
    return {k[len(prefix):]: w.to(F64) for k, w in weights.items()
            if k.startswith(prefix)}


def forward(cfg, weights, tokens):
    """tokens: list of ids -> (logits [T, vocab], residual after every
    layer run [runs, T, width])."""
    eps = cfg["norm"]["eps"]
    W = {k: w.to(F64) for k, w in weights.items()}
    emb = W["embed"][torch.tensor(tokens)]
    x, trail = emb, []
    loop = cfg.get("loop")
    for i, t in layer_runs(cfg):
        if t is not None and i == loop["start"]:
            if t > 0:
                x = x + emb
            x = x + W["loop.step"][t]
        L, p = cfg["layers"][i], f"l{i}."
        h = layer_norm(x, W[p + "norm1"], W[p + "norm1.b"], eps)
        x = x + MIXERS[L["type"]](h, sub(weights, p + "mix."), L["mixer"],
                                  eps)
        if L.get("mlp"):
            h = layer_norm(x, W[p + "norm2"], W[p + "norm2.b"], eps)
            x = x + swiglu_ff(h, sub(weights, p + "mlp."))
        trail.append(x)
    y = layer_norm(x, W["final.norm"], W["final.norm.b"], eps)
    return y @ W["embed"].T, torch.stack(trail)
