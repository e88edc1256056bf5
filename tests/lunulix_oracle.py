"""Plain, slow reference of the Lunulix decoder, one function per mechanism.

Whole sequences in float64 on the CPU: no cache, no chunks, no batching, and
no code shared with the package.  h is the [T, width] input of a mixer, W a
dict of one layer's weights by the suffix of their tensor names.
"""

from __future__ import annotations

import math

import torch

F64 = torch.float64


def rms(x, eps, weight=None):
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi)
                                     * (z + 0.044715 * z ** 3)))


def short_conv(u, w, bias=None):
    """u [T, C], w [C, taps]: the last tap meets the current token, zeros
    stand before the first one."""
    T, taps = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                y[t] += w[:, j] * u[s]
    return y if bias is None else y + bias


def frequencies(dims, base, scaling=None):
    """Angle per position of every rotated pair; long wavelengths are
    slowed down by `factor`, short ones kept, those between blended."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling:
            n = scaling["original"]
            wave = 2 * math.pi / f
            if wave > n / scaling["low"]:
                f = f / scaling["factor"]
            elif wave >= n / scaling["high"]:
                s = (n / wave - scaling["low"]) / (scaling["high"]
                                                   - scaling["low"])
                f = (1 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return out


def rotate(x, positions, dims, base, scaling=None):
    """x [T, H, D]: turn the pairs (i, i + dims/2) of the first dims."""
    out = x.clone()
    for i, f in enumerate(frequencies(dims, base, scaling)):
        c = torch.cos(positions * f)[:, None]
        s = torch.sin(positions * f)[:, None]
        u, v = x[:, :, i], x[:, :, i + dims // 2]
        out[:, :, i] = u * c - v * s
        out[:, :, i + dims // 2] = v * c + u * s
    return out


def sink_attention(q, k, v, scale, sink):
    """Causal attention of q [T, H, D] over k [T, G, D], v [T, G, E] (H / G
    query heads share a key head); exp(sink_h) stands in the denominator."""
    T, H, _ = q.shape
    G = k.shape[1]
    mask = torch.ones(T, T, dtype=torch.bool).triu(1)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(mask, -math.inf)
        top = torch.clamp(s.max(-1, keepdim=True).values, min=float(sink[h]))
        e = torch.exp(s - top)
        out[:, h] = (e @ v[:, g]) / (e.sum(-1, keepdim=True)
                                     + torch.exp(sink[h] - top))
    return out


def attention_branch(h, W, m):
    T = h.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = short_conv(h @ W["q"].T, W["q.conv"]).view(T, H, D)
    k = short_conv(h @ W["k"].T, W["k.conv"]).view(T, G, D)
    v = short_conv(h @ W["v"].T, W["v.conv"]).view(T, G, E)
    r = m["rot"]
    pos = torch.arange(T, dtype=F64)
    q = rotate(q, pos, r["dims"], r["base"], r.get("scaling"))
    k = rotate(k, pos, r["dims"], r["base"], r.get("scaling"))
    o = sink_attention(q, k, v, m["scale"], W["sink"]).reshape(T, H * E)
    return (o * sigmoid(h @ W["g"].T)) @ W["o"].T


def ssd_recurrence(x, B, C, dt, A, D, state=None):
    """x [T, H, P], B, C [T, G, N], dt [T, H] (positive), A [H] (positive):
    S <- exp(-A dt) S + dt B x^T, y = S^T C + D x.  Returns (y, S)."""
    T, H, P = x.shape
    G, N = B.shape[1:]
    S = torch.zeros(H, N, P, dtype=F64) if state is None else state.clone()
    group = torch.arange(H) // (H // G)
    out = torch.zeros(T, H, P, dtype=F64)
    for t in range(T):
        a = torch.exp(-A * dt[t])[:, None, None]
        S = a * S + dt[t][:, None, None] * B[t][group][:, :, None] \
            * x[t][:, None, :]
        out[t] = (S * C[t][group][:, :, None]).sum(1) + D[:, None] * x[t]
    return out, S


def gated_group_norm(y, z, weight, parts, eps):
    T, n = y.shape
    y = (y * silu(z)).view(T, parts, n // parts)
    return rms(y, eps).reshape(T, n) * weight


def ssd_branch(h, W, m, eps):
    T = h.shape[0]
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    u = h @ W["in"].T
    z, xbc, dt = u[:, :inner], u[:, inner:2 * inner + 2 * G * N], \
        u[:, 2 * inner + 2 * G * N:]
    assert dt.shape[1] == H
    xbc = silu(short_conv(xbc, W["conv"], W["conv.b"]))
    x = xbc[:, :inner].reshape(T, H, P)
    B = xbc[:, inner:inner + G * N].reshape(T, G, N)
    C = xbc[:, inner + G * N:].reshape(T, G, N)
    y, _ = ssd_recurrence(x, B, C, softplus(dt + W["dt_bias"]),
                          torch.exp(W["A_log"]), W["D"])
    y = gated_group_norm(y.reshape(T, inner), z, W["norm"], m["norm_groups"],
                         eps)
    return y @ W["o"].T


def parallel_mixer(h, W, m, eps):
    left = attention_branch(h, sub(W, "left."), m["left"])
    right = ssd_branch(h, sub(W, "right."), m["right"], eps)
    return m["left_scale"] * left + m["right_scale"] * right


def geglu_ff(h, W):
    return (gelu_tanh(h @ W["gate"].T) * (h @ W["up"].T)) @ W["down"].T


def token_side(x, e, W, eps):
    g = gelu_tanh(x @ W["gate"].T) * e
    return rms(g @ W["proj"].T, eps, W["norm"])


def sub(weights, prefix):
    return {k[len(prefix):]: w.to(F64) for k, w in weights.items()
            if k.startswith(prefix)}


def forward(cfg, weights, tokens):
    """tokens: list of ids -> (logits [T, vocab], residual after every layer
    [layers, T, width])."""
    eps = cfg["norm"]["eps"]
    W = {k: w.to(F64) for k, w in weights.items()}
    ids = torch.tensor(tokens)
    x, trail = W["embed"][ids] * cfg["embedding"]["scale"], []
    dim = cfg["token_side"]["dim"]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = parallel_mixer(rms(x, eps, W[p + "norm1"]), sub(W, p + "mix."),
                           L["mixer"], eps)
        x = x + rms(y, eps, W[p + "norm1b"])
        if L.get("mlp"):
            y = geglu_ff(rms(x, eps, W[p + "norm2"]), sub(W, p + "mlp."))
            x = x + rms(y, eps, W[p + "norm2b"])
        e = W["side.embed"][ids][:, i * dim:(i + 1) * dim]
        x = x + token_side(x, e, sub(W, p + "side."), eps)
        trail.append(x)
    return rms(x, eps, W["final.norm"]) @ W["head"].T, torch.stack(trail)
