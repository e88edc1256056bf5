"""Plain PyTorch fp32 references for every HIP kernel (numerics contracts).

GPU tests (tests/test_gpu_kernels.py) compare each qsa_hip kernel against
these on the same random inputs; tolerances account for bf16 I/O.
"""

from __future__ import annotations

import torch


def rmsnorm_ref(x: torch.Tensor, w: torch.Tensor, eps: float = 1e-5,
                residual: torch.Tensor | None = None):
    xf = x.float()
    res_out = None
    if residual is not None:
        xf = xf + residual.float()
        res_out = xf
    var = xf.pow(2).mean(dim=-1, keepdim=True)
    y = xf * torch.rsqrt(var + eps) * w.float()
    return (y, res_out) if residual is not None else y


def swiglu_ref(gate: torch.Tensor, up: torch.Tensor):
    g = gate.float()
    return torch.nn.functional.silu(g) * up.float()


def rope_tables(max_pos: int, d_head: int, theta: float = 500000.0):
    half = d_head // 2
    inv = 1.0 / (theta ** (torch.arange(half, dtype=torch.float64) / half))
    pos = torch.arange(max_pos, dtype=torch.float64)
    ang = torch.outer(pos, inv)
    return ang.cos().float(), ang.sin().float()


def rope_ref(x: torch.Tensor, pos: torch.Tensor, cos_t: torch.Tensor,
             sin_t: torch.Tensor):
    """x [B, H, D]; llama half-rotation (x0, x1=x[d+half])."""
    B, H, D = x.shape
    half = D // 2
    xf = x.float()
    c = cos_t[pos.long()].unsqueeze(1)  # [B, 1, half]
    s = sin_t[pos.long()].unsqueeze(1)
    x0, x1 = xf[..., :half], xf[..., half:]
    return torch.cat([x0 * c - x1 * s, x0 * s + x1 * c], dim=-1)


def paged_attn_ref(q: torch.Tensor, kc: torch.Tensor, vc: torch.Tensor,
                   block_table: torch.Tensor, seq_lens: torch.Tensor,
                   scale: float) -> torch.Tensor:
    """q [B, QH, D]; kc [P, KVH, D/8, 64, 8]; vc [P, KVH, D, 64]."""
    B, QH, D = q.shape
    KVH = kc.shape[1]
    R = QH // KVH
    out = torch.zeros_like(q, dtype=torch.float32)
    # un-page K into [P, KVH, 64, D]
    kn = kc.permute(0, 1, 3, 2, 4).reshape(kc.shape[0], KVH, 64, D).float()
    vn = vc.permute(0, 1, 3, 2).float()   # -> [P, KVH, 64, D]
    for b in range(B):
        n = int(seq_lens[b])
        if n == 0:
            continue
        npages = (n + 63) // 64
        pages = block_table[b, :npages].long()
        k_seq = kn[pages].permute(1, 0, 2, 3).reshape(KVH, npages * 64, D)[:, :n]
        v_seq = vn[pages].permute(1, 0, 2, 3).reshape(KVH, npages * 64, D)[:, :n]
        for h in range(QH):
            kvh = h // R
            sc = (k_seq[kvh] @ q[b, h].float()) * scale
            p = torch.softmax(sc, dim=-1)
            out[b, h] = p @ v_seq[kvh]
    return out


def topk_cosine_ref(queries: torch.Tensor, docs: torch.Tensor, k: int):
    scores = queries.float() @ docs.float().T
    s, i = torch.topk(scores, k, dim=-1)
    return s, i.int()


def softmax_rows_ref(scores: torch.Tensor, col_offset: int = 0,
                     causal: bool = False):
    s = scores.float().clone()
    rows, cols = s.shape
    if causal:
        col = torch.arange(cols, device=s.device).unsqueeze(0)
        row = torch.arange(rows, device=s.device).unsqueeze(1)
        s.masked_fill_(col > row + col_offset, float("-inf"))
    out = torch.softmax(s, dim=-1)
    return torch.nan_to_num(out, nan=0.0)


def window_agg_ref(ts: torch.Tensor, key: torch.Tensor, value, t0: int,
                   win_ms: int, nwin: int, nkeys: int):
    counts = torch.zeros(nkeys, nwin, dtype=torch.int32)
    sums = torch.zeros(nkeys, nwin, dtype=torch.float32)
    w = ((ts - t0) // win_ms)
    ok = (w >= 0) & (w < nwin)
    for i in torch.nonzero(ok).flatten().tolist():
        counts[key[i], w[i]] += 1
        if value is not None:
            sums[key[i], w[i]] += float(value[i])
    return counts, sums


# ---- mixer decoders --------------------------------------------------------

def residual_norm_ref(res, y, table, ids, vec, w, b, eps, init, layer, post,
                      tscale):
    """In-place f32 residual update and its norm (dispatch.residual_norm)."""
    like = y if w is None else w
    if init:
        res.zero_()
    if y is not None:
        y = y.float()
        if post is not None:
            y = y / torch.sqrt(y.pow(2).mean(-1, keepdim=True) + eps) \
                * post.float()
        res.add_(y)
    if table is not None:
        res.add_(table[ids].float() * tscale)
    if vec is not None:
        res.add_(vec.float())
    x = res
    if w is None:
        return x.to(like.dtype, copy=True)
    if layer:
        x = x - x.mean(-1, keepdim=True)
    x = x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps) * w.float()
    if b is not None:
        x = x + b.float()
    return x.to(w.dtype)


def gated_act_ref(gate, factor, gelu):
    g = gate.float()
    g = torch.nn.functional.gelu(g, approximate="tanh") if gelu \
        else torch.nn.functional.silu(g)
    return (g * factor.float()).to(gate.dtype)


def conv_portions(item, off, start, len_, slots):
    """(slot, first row, first position, length) of a step's portions; without
    `item`, one token per row at position start - 1 (0: row not in use)."""
    if item is None:
        return [(s, b, p - 1, 1) for b, (s, p) in
                enumerate(zip(slots.tolist(), start.tolist()))
                if s >= 0 and p > 0]
    return list(zip(slots.tolist(), off.tolist(), start.tolist(),
                    len_.tolist()))


def short_conv_ref(x, w, tails, portions):
    """Causal filters w [taps, C] over rows of x [T, C]; tails [slots,
    taps - 1, C] carry the last inputs of every sequence.  f32 result."""
    taps = w.shape[0]
    y = torch.zeros(x.shape, dtype=torch.float32)
    for slot, r0, p0, n in portions:
        past = tails[slot].clone()
        past[:max(0, taps - 1 - p0)] = 0        # before the sequence
        u = torch.cat([past, x[r0:r0 + n]])
        for j in range(taps):
            y[r0:r0 + n] += w[j] * u[j:j + n].float()
        tails[slot] = u[n:]
    return y


def conv_qkv_ref(x, w, tails, cos_t, sin_t, rot, cache_slots, kc, vc, heads,
                 portions):
    T, (_, G, _, D), E = x.shape[0], kc.shape, vc.shape[3]
    y = short_conv_ref(x, w, tails, portions)
    pos = torch.zeros(T, dtype=torch.int64)
    live = torch.zeros(T, dtype=torch.bool)
    for _, r0, p0, n in portions:
        pos[r0:r0 + n] = torch.arange(p0, p0 + n)
        live[r0:r0 + n] = True
    qk = y[:, :(heads + G) * D].reshape(T, heads + G, D).clone()
    if rot:
        h = rot // 2
        c, s = cos_t[pos][:, None], sin_t[pos][:, None]
        a, b = qk[..., :h].clone(), qk[..., h:rot].clone()
        qk[..., :h] = a * c - b * s
        qk[..., h:rot] = b * c + a * s
    v = y[:, (heads + G) * D:].reshape(T, G, E)
    for t in range(T):
        slot = int(cache_slots[t])
        if live[t] and slot >= 0:
            kc[slot // 64, :, slot % 64] = qk[t, heads:].to(kc.dtype)
            vc[slot // 64, :, slot % 64] = v[t].to(vc.dtype)
    return qk[:, :heads].reshape(T, heads * D).to(x.dtype)


def gqa_rows_ref(q, kc, vc, block_table, row_item, row_len, sink, gate, out,
                 heads, scale, out_scale):
    R, (_, G, _, D), E = q.shape[0], kc.shape, vc.shape[3]
    for r in range(R):
        n = int(row_len[r])
        if n <= 0:
            out[r] = 0
            continue
        pos = torch.arange(n)
        page = block_table[int(row_item[r]) if row_item is not None
                           else r].long()[pos // 64]
        k = kc[page, :, pos % 64].float().transpose(0, 1)      # [G, n, D]
        v = vc[page, :, pos % 64].float().transpose(0, 1)
        s = torch.matmul(q[r].float().view(G, heads // G, D),
                         k.transpose(1, 2)) * scale
        if sink is not None:
            s = torch.cat([s, sink.view(G, -1, 1)], -1)
        o = torch.matmul(torch.softmax(s, -1)[..., :n], v).reshape(-1)
        if gate is not None:
            o = o * torch.sigmoid(gate[r].float())
        out[r] = (o * out_scale).to(out.dtype)


def ssd_ref(u, zoff, dtoff, xbc, A, dt_bias, D, state, groups, portions, out):
    """portions: (slot, first row, first position, length); state and the
    portions' rows of out are written."""
    _, H, N, P = state.shape
    inner = H * P
    for slot, r0, p0, n in portions:
        rows = xbc[r0:r0 + n].float()
        x = rows[:, :inner].reshape(n, H, P)
        B, C = (t.reshape(n, groups, N).repeat_interleave(H // groups, 1)
                for t in rows[:, inner:].chunk(2, 1))
        z = u[r0:r0 + n, zoff:zoff + inner].float()
        dt = torch.nn.functional.softplus(
            u[r0:r0 + n, dtoff:dtoff + H].float() + dt_bias)
        S = state[slot]
        if p0 == 0:
            S.zero_()
        y = torch.empty(n, H, P)
        for t in range(n):
            S.mul_(torch.exp(-A * dt[t])[:, None, None]).add_(
                (B[t] * dt[t][:, None])[:, :, None] * x[t][:, None, :])
            y[t] = torch.matmul(C[t][:, None, :], S).squeeze(1) \
                + D[:, None] * x[t]
        out[r0:r0 + n] = (y.reshape(n, inner)
                          * torch.nn.functional.silu(z)).to(out.dtype)


def latent_rows_ref(qa, cache, block_table, row_item, row_len, sink, window,
                    scale):
    R, H, KR = qa.shape[0], sink.numel(), cache.shape[2]
    out = torch.zeros(R, H, KR)
    flat = cache.reshape(-1, KR).float()
    for r in range(R):
        n = int(row_len[r])
        if n <= 0:
            continue
        lo = max(0, n - window) if window > 0 else 0
        pos = torch.arange(lo, n)
        bt = block_table[int(row_item[r]) if row_item is not None else r]
        c = flat[bt.long()[pos // 64] * 64 + pos % 64]
        s = (qa[r].float().view(H, KR) @ c.T) * scale
        p = torch.softmax(torch.cat([s, sink.float()[:, None]], 1), -1)
        out[r] = p[:, :-1] @ c
    return out.view(R, H * KR).to(qa.dtype)


def retention_ref(x, cos_t, sin_t, decay, state, portions, out, rot, kscale,
                  eps):
    """portions: (slot, first row, first position, length); state and the
    portions' rows of out are written."""
    _, H, D, E = state.shape
    half = rot // 2
    for slot, r0, p0, n in portions:
        rows = x[r0:r0 + n].float()
        q = rows[:, :H * D].reshape(n, H, D).clone()
        k = rows[:, H * D:2 * H * D].reshape(n, H, D).clone()
        v = rows[:, 2 * H * D:2 * H * D + H * E].reshape(n, H, E)
        g = rows[:, 2 * H * D + H * E:2 * H * D + 2 * H * E]
        if half:
            c = cos_t[p0:p0 + n, None, :]
            s = sin_t[p0:p0 + n, None, :]
            for t in (q, k):
                a, b = t[..., :half].clone(), t[..., half:rot].clone()
                t[..., :half] = a * c - b * s
                t[..., half:rot] = b * c + a * s
        k = k * kscale
        S = state[slot]
        if p0 == 0:
            S.zero_()
        o = torch.empty(n, H, E)
        for t in range(n):
            S.mul_(decay.view(H, 1, 1)).add_(k[t, :, :, None]
                                             * v[t, :, None, :])
            o[t] = torch.matmul(q[t, :, None, :], S).squeeze(1)
        o = o / torch.sqrt(o.pow(2).mean(-1, keepdim=True) + eps)
        out[r0:r0 + n] = (o.reshape(n, H * E)
                          * torch.nn.functional.silu(g)).to(out.dtype)
