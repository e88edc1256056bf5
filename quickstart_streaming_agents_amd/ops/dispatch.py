"""Device dispatch for the op layer.

Same call surface as the native modules (ops/hip/ops.cpp: qsa_hip,
ops/hip/lm_ops.cpp: qsa_lm_hip). CUDA tensors go to the hand-written HIP/CDNA4 kernels — fail-loud if the extension is
missing (ops/__init__.py).  CPU tensors run reference implementations with
IDENTICAL semantics (including in-place mutation contracts), which lets the
engine / model / parallel layers run under multi-process gloo tests in
CPU-only CI.  A CUDA tensor NEVER falls back to the CPU path.
"""

from __future__ import annotations

import torch

from . import ext, lm_ext


def _cuda(t: torch.Tensor) -> bool:
    return t.is_cuda


# ---- elementwise ----------------------------------------------------------

def rmsnorm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    if _cuda(x):
        return ext().rmsnorm(x, w, eps)
    xf = x.float()
    y = xf * torch.rsqrt(xf.pow(2).mean(-1, keepdim=True) + eps) * w.float()
    return y.to(x.dtype)


def rmsnorm_residual(x: torch.Tensor, res: torch.Tensor, w: torch.Tensor,
                     eps: float) -> torch.Tensor:
    """res <- res + x (in place); returns rmsnorm(res) * w."""
    if _cuda(x):
        return ext().rmsnorm_residual(x, res, w, eps)
    res.add_(x)
    rf = res.float()
    y = rf * torch.rsqrt(rf.pow(2).mean(-1, keepdim=True) + eps) * w.float()
    return y.to(x.dtype)


def swiglu(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    if _cuda(gate):
        return ext().swiglu(gate, up)
    return (torch.nn.functional.silu(gate.float()) * up.float()).to(gate.dtype)


def rope_inplace(q: torch.Tensor, k: torch.Tensor, cos_t: torch.Tensor,
                 sin_t: torch.Tensor, pos: torch.Tensor) -> None:
    if _cuda(q):
        ext().rope_inplace(q, k, cos_t, sin_t, pos)
        return
    for t in (q, k):
        D = t.shape[-1]
        half = D // 2
        c = cos_t[pos.long()].unsqueeze(1)
        s = sin_t[pos.long()].unsqueeze(1)
        tf = t.float()
        x0, x1 = tf[..., :half], tf[..., half:]
        t.copy_(torch.cat([x0 * c - x1 * s, x0 * s + x1 * c],
                          dim=-1).to(t.dtype))


def softmax_rows_(scores: torch.Tensor, col_offset: int = 0,
                  causal: bool = False, row_mod: int = 0,
                  row_limits: torch.Tensor | None = None) -> None:
    if _cuda(scores):
        ext().softmax_rows_(scores, col_offset, causal, row_mod, row_limits)
        return
    rows, cols = scores.shape
    limit = torch.full((rows,), cols, dtype=torch.int64)
    if causal:
        r = torch.arange(rows)
        pos = r % row_mod if row_mod > 0 else r
        limit = torch.minimum(limit, pos + col_offset + 1)
    if row_limits is not None:
        limit = torch.minimum(limit, row_limits.long())
    col = torch.arange(cols).unsqueeze(0)
    masked = scores.masked_fill(col >= limit.unsqueeze(1), float("-inf"))
    out = torch.softmax(masked, dim=-1)
    scores.copy_(torch.nan_to_num(out, nan=0.0))


def softmax_rows_bf16_(scores: torch.Tensor, scale: float,
                       row_limits: torch.Tensor) -> None:
    """In-place bf16 masked softmax with folded scale; beyond-limit
    columns zeroed (prefill padded-batch attention)."""
    if _cuda(scores):
        ext().softmax_rows_bf16_(scores, scale, row_limits)
        return
    rows, cols = scores.shape
    s = scores.float() * scale
    col = torch.arange(cols).unsqueeze(0)
    masked = s.masked_fill(col >= row_limits.long().unsqueeze(1),
                           float("-inf"))
    out = torch.nan_to_num(torch.softmax(masked, dim=-1), nan=0.0)
    scores.copy_(out.to(scores.dtype))


# ---- paged KV -------------------------------------------------------------

def kv_append(knew: torch.Tensor, vnew: torch.Tensor, kc: torch.Tensor,
              vc: torch.Tensor, block_table: torch.Tensor,
              seq_lens: torch.Tensor) -> None:
    """Write row b's k/v at position seq_lens[b]-1 of its paged sequence."""
    if _cuda(knew):
        ext().kv_append(knew, vnew, kc, vc, block_table, seq_lens)
        return
    B, KVH, D = knew.shape
    for b in range(B):
        n = int(seq_lens[b])
        if n <= 0:
            continue
        page = int(block_table[b, (n - 1) // 64])
        off = (n - 1) % 64
        # K layout [P, KVH, D/8, 64, 8]; V layout [P, KVH, D, 64]
        kc[page, :, :, off, :] = knew[b].reshape(KVH, D // 8, 8)
        vc[page, :, :, off] = vnew[b]


def rope_kv_append(q, k, v, kc, vc, cos_t, sin_t, block_table,
                   seq_lens) -> None:
    """Fused decode-step rope(q,k in place semantics) + cache append.
    The fused kernel rotates q in place and writes rotated k (+v) straight
    to the paged cache; CPU reference composes the two reference ops."""
    if _cuda(q):
        ext().rope_kv_append(q, k, v, kc, vc, cos_t, sin_t, block_table,
                             seq_lens)
        return
    # positions = seq_lens - 1 (clamped)
    pos = (seq_lens.long() - 1).clamp(min=0).int()
    rope_inplace(q, k, cos_t, sin_t, pos)
    kv_append(k, v, kc, vc, block_table, seq_lens)


def kv_scatter(knew: torch.Tensor, vnew: torch.Tensor, kc: torch.Tensor,
               vc: torch.Tensor, slots: torch.Tensor) -> None:
    """Write row t at global slot ids (page*64 + offset)."""
    if _cuda(knew):
        ext().kv_scatter(knew, vnew, kc, vc, slots)
        return
    T, KVH, D = knew.shape
    for t in range(T):
        s = int(slots[t])
        page, off = s // 64, s % 64
        kc[page, :, :, off, :] = knew[t].reshape(KVH, D // 8, 8)
        vc[page, :, :, off] = vnew[t]


def paged_attn_decode(q: torch.Tensor, kc: torch.Tensor, vc: torch.Tensor,
                      block_table: torch.Tensor, seq_lens: torch.Tensor,
                      scale: float) -> torch.Tensor:
    if _cuda(q):
        return ext().paged_attn_decode(q, kc, vc, block_table, seq_lens,
                                       scale)
    from .cpu_ref import paged_attn_ref
    return paged_attn_ref(q, kc, vc, block_table, seq_lens,
                          scale).to(q.dtype)


# ---- skinny decode GEMM ---------------------------------------------------

def can_pack_weight(n: int, k: int) -> bool:
    return n % 16 == 0 and k % 256 == 0


def pack_weight_frag(w: torch.Tensor) -> torch.Tensor:
    """[N,K] bf16 -> fragment-major stream layout for skinny_linear (GPU)."""
    n, k = w.shape
    return w.reshape(n // 16, 16, k // 32, 32).permute(0, 2, 1, 3).contiguous()


def skinny_linear(x: torch.Tensor, wf: torch.Tensor, n: int,
                  k: int) -> torch.Tensor:
    """x[M,K] @ W^T via the weight-streaming decode kernel (M <= 32)."""
    if x.is_cuda:
        return lm_ext().skinny_gemm(x, wf, n, k)
    w = wf.reshape(n // 16, k // 32, 16, 32).permute(0, 2, 1, 3) \
        .reshape(n, k)
    return (x.float() @ w.float().T).to(x.dtype)


# ---- fp8 weight-only decode GEMM (W8A16, per-channel scales) -------------

def pack_weight_fp8(w: torch.Tensor) -> tuple[torch.Tensor, torch.Tensor]:
    """[N,K] bf16 -> (fp8-e4m3 fragment-pair-major stream as uint8,
    per-channel f32 scales).  Layout doc: ops/hip/skinny_gemm_fp8.hip."""
    n, k = w.shape
    assert n % 16 == 0 and k % 256 == 0
    wf = w.float()
    s = wf.abs().amax(dim=1).clamp(min=1e-12) / 448.0
    q = (wf / s[:, None]).clamp(-448.0, 448.0).to(torch.float8_e4m3fn)
    qf = q.view(torch.uint8) \
        .reshape(n // 16, 16, k // 64, 2, 4, 8) \
        .permute(0, 2, 1, 4, 3, 5).contiguous()
    return qf, s.float().contiguous()


def unpack_weight_fp8(qf: torch.Tensor, scale: torch.Tensor, n: int,
                      k: int) -> torch.Tensor:
    """Inverse of pack_weight_fp8 -> dequantized f32 [N,K] (reference)."""
    q = qf.reshape(n // 16, k // 64, 16, 4, 2, 8) \
        .permute(0, 2, 1, 4, 3, 5).reshape(n, k)
    return q.view(torch.float8_e4m3fn).float() * scale[:, None].float()


def gemm_fp8_batch(x: torch.Tensor, qf: torch.Tensor,
                   scale: torch.Tensor, n: int, k: int,
                   splitk: int = 1) -> torch.Tensor:
    """Batched-M (<=256) fp8 weight-stream GEMM (decode batches)."""
    if x.is_cuda:
        return ext().gemm_fp8_batch(x, qf, scale, n, k, splitk)
    w = unpack_weight_fp8(qf, scale, n, k)
    return (x.float() @ w.T).to(x.dtype)


def skinny_linear_fp8(x: torch.Tensor, qf: torch.Tensor,
                      scale: torch.Tensor, n: int, k: int) -> torch.Tensor:
    """x[M,K] bf16 @ dequant(Q)^T via the fp8 weight-streaming kernel."""
    if x.is_cuda:
        return ext().skinny_gemm_fp8(x, qf, scale, n, k)
    w = unpack_weight_fp8(qf, scale, n, k)
    return (x.float() @ w.T).to(x.dtype)


# ---- mixer decoders (qsa_lm_hip) ------------------------------------------
# bf16 or f32 storage, f32 arithmetic, any sizes; the CPU semantics are in
# ops/cpu_ref.py.

def residual_norm(res: torch.Tensor, y: torch.Tensor | None,
                  w: torch.Tensor | None, b: torch.Tensor | None,
                  eps: float, *, table: torch.Tensor | None = None,
                  ids: torch.Tensor | None = None,
                  vec: torch.Tensor | None = None, init: bool = False,
                  layer: bool = True, post: torch.Tensor | None = None,
                  tscale: float = 1.0) -> torch.Tensor:
    """res (f32) <- (0 if init else res) + y + tscale * table[ids] + vec, in
    place; returns the layer norm (layer=True) or rms norm of it, times w,
    plus b, or without w the residual itself.  With `post`, y enters as its
    own rms norm times post."""
    if _cuda(res):
        return lm_ext().residual_norm(res, y, table, ids, vec, w, b, eps,
                                      init, layer, post, tscale)
    from .cpu_ref import residual_norm_ref
    return residual_norm_ref(res, y, table, ids, vec, w, b, eps, init, layer,
                             post, tscale)


def glu(gate: torch.Tensor, up: torch.Tensor,
        act: str = "silu") -> torch.Tensor:
    """act(gate) * up for any width and storage type; act: silu or gelu (its
    tanh form)."""
    if _cuda(gate):
        return lm_ext().glu(gate, up, act == "gelu")
    from .cpu_ref import gated_act_ref
    return gated_act_ref(gate, up, act == "gelu")


def glu_table(gate: torch.Tensor, table: torch.Tensor, ids: torch.Tensor,
              col0: int, act: str = "gelu") -> torch.Tensor:
    """act(gate [T, n]) * table[ids, col0 : col0 + n]."""
    if _cuda(gate):
        return lm_ext().glu_table(gate, table, ids, col0, act == "gelu")
    from .cpu_ref import gated_act_ref
    return gated_act_ref(gate, table[ids, col0:col0 + gate.shape[1]],
                         act == "gelu")


def argmax_rows(x: torch.Tensor) -> torch.Tensor:
    """Greedy pick per row (lowest index on ties), safe inside graphs."""
    if _cuda(x):
        return lm_ext().argmax_rows(x.contiguous())
    return torch.argmax(x, dim=-1)


def decode_slots(block_table: torch.Tensor,
                 seq_lens: torch.Tensor) -> torch.Tensor:
    """Cache slot (page*64 + offset) of each row's newest position, or -1."""
    if _cuda(block_table):
        return lm_ext().decode_slots(block_table, seq_lens)
    p = seq_lens.long() - 1
    pc = p.clamp(min=0)
    page = block_table.long().gather(1, (pc // 64)[:, None]).squeeze(1)
    return torch.where(p < 0, torch.full_like(p, -1),
                       page * 64 + pc % 64).int()


def latent_norm_store(x: torch.Tensor, wq: torch.Tensor, wk: torch.Tensor,
                      cache: torch.Tensor, slots: torch.Tensor,
                      eps: float) -> torch.Tensor:
    """x rows [q latent | kv latent | ...]: returns rms(q latent) * wq and
    writes rms(kv latent) * wk to cache [pages, 64, rank] at `slots`."""
    if _cuda(x):
        return lm_ext().latent_norm_store(x, wq, wk, cache, slots, eps)
    from .cpu_ref import rmsnorm_ref
    qr, kr = wq.numel(), wk.numel()
    c = rmsnorm_ref(x[:, qr:qr + kr], wk, eps).to(cache.dtype)
    keep = slots >= 0
    cache.view(-1, kr)[slots[keep].long()] = c[keep]
    return rmsnorm_ref(x[:, :qr], wq, eps).to(x.dtype)


def head_matmul(x: torch.Tensor, w: torch.Tensor,
                gate: torch.Tensor | None = None) -> torch.Tensor:
    """x [M, H*K], w [H, N, K] -> [M, H*N], one product per head; with
    `gate` [M, H*N] the result is multiplied by sigmoid(gate)."""
    if _cuda(x):
        return lm_ext().head_matmul(x, w, gate)
    H, N, K = w.shape
    y = torch.bmm(x.float().reshape(-1, H, K).transpose(0, 1).contiguous(),
                  w.float().transpose(1, 2).contiguous())
    y = y.transpose(0, 1).reshape(-1, H * N)
    if gate is not None:
        y = y * torch.sigmoid(gate.float())
    return y.to(x.dtype)


def latent_rows(qa: torch.Tensor, cache: torch.Tensor,
                block_table: torch.Tensor, row_item: torch.Tensor | None,
                row_len: torch.Tensor, sink: torch.Tensor, window: int,
                scale: float) -> torch.Tensor:
    """Absorbed latent attention: row r of qa [R, H*rank] at position
    row_len[r]-1 reads the latents of sequence row_item[r] (its own index
    without it) inside the window (0: all); softmax with sink."""
    if _cuda(qa):
        return lm_ext().latent_rows(qa, cache, block_table, row_item,
                                    row_len, sink, window, scale)
    from .cpu_ref import latent_rows_ref
    return latent_rows_ref(qa, cache, block_table, row_item, row_len, sink,
                           window, scale)


def window_attn_ok(h: int, d: int, e: int) -> bool:
    return lm_ext().window_attn_ok(h, d, e)


def window_attn_prefill(q, kv, gate, sink, qb_item, qb_t0, off, start, len_,
                        ctx_off, ctx_pos, out, d: int, e: int, window: int,
                        scale: float) -> None:
    """Windowed flash attention of prompt portions over expanded keys and
    values, sink and sigmoid gate included (GPU, bf16)."""
    lm_ext().window_attn_prefill(q, kv, gate, sink, qb_item, qb_t0, off,
                                 start, len_, ctx_off, ctx_pos, out, d, e,
                                 window, scale)


def retention_decode(x, cos_t, sin_t, decay, state, slots, seq_lens,
                     rot: int, kscale: float, eps: float) -> torch.Tensor:
    """One token per row; x rows [q | k | v | gate], state [slots, H, D, E]
    f32 updated in place.  Rows with seq_len 0 or slot -1 are not in use."""
    if _cuda(x):
        return lm_ext().retention_decode(x, cos_t, sin_t, decay, state,
                                         slots, seq_lens, rot, kscale, eps)
    from .cpu_ref import retention_ref
    B, (_, H, D, E) = x.shape[0], state.shape
    out = torch.zeros(B, H * E, dtype=x.dtype)
    live = [b for b in range(B) if int(seq_lens[b]) > 0 and int(slots[b]) >= 0]
    retention_ref(x, cos_t, sin_t, decay, state,
                  [(int(slots[b]), b, int(seq_lens[b]) - 1, 1) for b in live],
                  out, rot, kscale, eps)
    return out


def retention_seq(x, cos_t, sin_t, decay, state, slots, off, start, len_,
                  out, rot: int, kscale: float, eps: float) -> None:
    """Portions of several tokens, token by token (any size and type)."""
    if _cuda(x):
        lm_ext().retention_seq(x, cos_t, sin_t, decay, state, slots, off,
                               start, len_, out, rot, kscale, eps)
        return
    from .cpu_ref import retention_ref
    retention_ref(x, cos_t, sin_t, decay, state,
                  list(zip(slots.tolist(), off.tolist(), start.tolist(),
                           len_.tolist())), out, rot, kscale, eps)


def retention_chunked_ok(h: int, d: int, e: int) -> bool:
    return lm_ext().retention_chunked_ok(h, d, e)


def retention_chunked(x, cos_t, sin_t, log2_decay, state, slots, off, start,
                      len_, positions, chunk0, chunk_item, chunk_t0, out,
                      rot: int, kscale: float, eps: float) -> None:
    """Portions in chunks of 64 tokens on the matrix cores (GPU, bf16)."""
    lm_ext().retention_chunked(x, cos_t, sin_t, log2_decay, state, slots,
                               off, start, len_, positions, chunk0,
                               chunk_item, chunk_t0, out, rot, kscale, eps)


# A step's rows for the short convolutions are (item, t0, off, start, len,
# slots): portions in chunks of 16 rows, or, with item None, one token per row
# at position start - 1 (layers.StepPlan.conv).

def conv_qkv(x, filters, tails, cos_t, sin_t, rot: int, cache_slots, kc, vc,
             heads: int, item, t0, off, start, len_, slots) -> torch.Tensor:
    """x columns [q | k | v] through their causal filters [taps, C], q and k
    rotated; returns q, writes k and v to their pages [P, G, 64, .] at
    cache_slots.  tails [slots, taps - 1, C] hold the last inputs."""
    if _cuda(x):
        return lm_ext().conv_qkv(x, filters, tails, cos_t, sin_t, rot,
                                 cache_slots, kc, vc, heads, item, t0, off,
                                 start, len_, slots)
    from .cpu_ref import conv_portions, conv_qkv_ref
    return conv_qkv_ref(x, filters, tails, cos_t, sin_t, rot, cache_slots,
                        kc, vc, heads,
                        conv_portions(item, off, start, len_, slots))


def conv_silu(x, filters, bias, tails, item, t0, off, start, len_,
              slots) -> torch.Tensor:
    """silu(causal filters over x + bias), dense [T, C]."""
    if _cuda(x):
        return lm_ext().conv_silu(x, filters, bias, tails, item, t0, off,
                                  start, len_, slots)
    from .cpu_ref import conv_portions, short_conv_ref
    y = short_conv_ref(x, filters, tails,
                       conv_portions(item, off, start, len_, slots))
    return torch.nn.functional.silu(y + bias).to(x.dtype)


def gqa_rows(q, kc, vc, block_table, row_item, row_len, sink, gate, out,
             heads: int, scale: float, out_scale: float = 1.0) -> None:
    """Rows of q [R, heads*D] at positions row_len - 1 over the paged keys
    and values of sequence row_item (their own index without it): softmax with
    sink, times sigmoid(gate) and out_scale, to rows of out."""
    if _cuda(q):
        lm_ext().gqa_rows(q, kc, vc, block_table, row_item, row_len, sink,
                          gate, out, heads, scale, out_scale)
        return
    from .cpu_ref import gqa_rows_ref
    gqa_rows_ref(q, kc, vc, block_table, row_item, row_len, sink, gate, out,
                 heads, scale, out_scale)


def gqa_mfma_ok(d: int, e: int) -> bool:
    return lm_ext().gqa_mfma_ok(d, e)


def gqa_portion_rows(d: int, e: int) -> int:
    return lm_ext().gqa_portion_rows(d, e)


def gqa_portions(q, kc, vc, block_table, sink, gate, qb_item, qb_t0, off,
                 start, len_, out, heads: int, scale: float,
                 out_scale: float = 1.0) -> None:
    """The same for whole portions, flash attention (GPU, bf16)."""
    lm_ext().gqa_portions(q, kc, vc, block_table, sink, gate, qb_item, qb_t0,
                          off, start, len_, out, heads, scale, out_scale)


def ssd_decode(u, zoff: int, dtoff: int, xbc, A, dt_bias, D, state,
               groups: int, slots, seq_lens) -> torch.Tensor:
    """One token per row of a state-space layer: z and raw dt are columns of
    u, x | B | C are xbc, state [slots, H, N, P] f32 updated in place.
    Returns (S^T C + D x) * silu(z).  Rows with seq_len 0 or slot -1 are not
    in use."""
    if _cuda(u):
        return lm_ext().ssd_decode(u, zoff, dtoff, xbc, A, dt_bias, D, state,
                                   groups, slots, seq_lens)
    from .cpu_ref import conv_portions, ssd_ref
    out = torch.zeros(u.shape[0], state.shape[1] * state.shape[3],
                      dtype=u.dtype)
    ssd_ref(u, zoff, dtoff, xbc, A, dt_bias, D, state, groups,
            conv_portions(None, None, seq_lens, None, slots), out)
    return out


def ssd_seq(u, zoff: int, dtoff: int, xbc, A, dt_bias, D, state, groups: int,
            slots, off, start, len_, out) -> None:
    """Portions of several tokens, token by token (any size and type)."""
    if _cuda(u):
        lm_ext().ssd_seq(u, zoff, dtoff, xbc, A, dt_bias, D, state, groups,
                         slots, off, start, len_, out)
        return
    from .cpu_ref import ssd_ref
    ssd_ref(u, zoff, dtoff, xbc, A, dt_bias, D, state, groups,
            list(zip(slots.tolist(), off.tolist(), start.tolist(),
                     len_.tolist())), out)


def ssd_chunked_ok(h: int, n: int, p: int, groups: int) -> bool:
    return lm_ext().ssd_chunked_ok(h, n, p, groups)


def ssd_chunked(u, zoff: int, dtoff: int, xbc, A, dt_bias, D, state,
                groups: int, slots, off, start, len_, chunk0, chunk_item,
                chunk_t0, out) -> None:
    """Portions in chunks of 64 tokens on the matrix cores (GPU, bf16)."""
    lm_ext().ssd_chunked(u, zoff, dtoff, xbc, A, dt_bias, D, state, groups,
                         slots, off, start, len_, chunk0, chunk_item,
                         chunk_t0, out)


def part_norm(x: torch.Tensor, w: torch.Tensor, out: torch.Tensor,
              parts: int, eps: float) -> None:
    """out <- rms norm of `parts` equal parts of every row of x, times w."""
    if _cuda(x):
        lm_ext().part_norm(x, w, out, parts, eps)
        return
    y = x.float().view(x.shape[0], parts, -1)
    y = y / torch.sqrt(y.pow(2).mean(-1, keepdim=True) + eps)
    out.copy_((y.reshape(x.shape) * w).to(out.dtype))


# ---- retrieval / streaming ------------------------------------------------

def topk_cosine(queries: torch.Tensor, docs: torch.Tensor, k: int):
    if _cuda(queries):
        return ext().topk_cosine(queries, docs, k)
    from .cpu_ref import topk_cosine_ref
    return topk_cosine_ref(queries, docs, k)


def window_agg(ts: torch.Tensor, key: torch.Tensor,
               value: torch.Tensor | None, t0: int, win_ms: int, nwin: int,
               nkeys: int):
    if _cuda(ts):
        return ext().window_agg(ts, key, value, t0, win_ms, nwin, nkeys)
    from .cpu_ref import window_agg_ref
    return window_agg_ref(ts, key, value, t0, win_ms, nwin, nkeys)


# ---- GPU hash join (K8) ---------------------------------------------------

def hash_build(keys: torch.Tensor, ts: torch.Tensor):
    """(i64 keys, i64 event ts) -> opaque latest-per-key table.
    GPU: (tkeys, tpay) HBM tensors; CPU: a dict of key -> (ts, row).
    Event times clamp to [0, 2^40): the GPU payload packs (ts << 24 |
    row), so negative or far-future timestamps would corrupt ordering —
    clamping keeps CPU/GPU semantics identical."""
    ts = ts.clamp(min=0, max=(1 << 40) - 1)
    if _cuda(keys):
        return tuple(ext().hash_build(keys, ts.contiguous()))
    table: dict = {}
    for i, (k, t) in enumerate(zip(keys.tolist(), ts.tolist())):
        prev = table.get(k)
        if prev is None or (t, i) >= prev:
            table[k] = (t, i)
    return table


def hash_probe(table, keys: torch.Tensor, min_ts: int) -> torch.Tensor:
    """Probe -> i32 row indices (-1 = absent or event ts < min_ts)."""
    if isinstance(table, tuple):
        return ext().hash_probe(table[0], table[1], keys, int(min_ts))
    out = torch.full((keys.numel(),), -1, dtype=torch.int32)
    for i, k in enumerate(keys.tolist()):
        hit = table.get(k)
        if hit is not None and hit[0] >= min_ts:
            out[i] = hit[1]
    return out
