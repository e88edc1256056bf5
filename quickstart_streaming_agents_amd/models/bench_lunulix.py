"""Kernels of the Lunulix design against the roofline, each beside the like
kernel of the framework's other decoders (see models/bench.py)."""

from __future__ import annotations

import torch

from ..ops import dispatch as D
from ..ops import ext
from .bench import _graph_time, _i32, _report
from .layers import RopeTable, StepPlan

DEV, BF = "cuda:0", torch.bfloat16
# width 4096: 32/8 heads of 128; 64 state heads of 64, state 128, 8 groups
W, F, SIDE = 4096, 14_336, 256
H, KVH, DH = 32, 8, 128
SH, P, N, G = 64, 64, 128, 8
QKV = (H + 2 * KVH) * DH
INNER = SH * P
XBC = INNER + 2 * G * N
TAPS = 4


def rnd(*s):
    return torch.randn(*s, device=DEV, dtype=torch.float32).to(BF)


def _portions(n_seq: int, n: int, size: int):
    """(portion, first row) of pieces of `size` rows of n_seq portions."""
    i = torch.arange(n_seq, device=DEV, dtype=torch.int32)
    t0 = torch.arange(0, n, size, device=DEV, dtype=torch.int32)
    return i, i.repeat_interleave(len(t0)).contiguous(), t0.repeat(n_seq)


def _rows(reps: int) -> None:
    for T in (64, 8192):
        ys = [rnd(T, W) for _ in range(reps)]
        rs = [torch.randn(T, W, device=DEV) for _ in range(reps)]
        rb = [r.to(BF) for r in rs]
        w, post = rnd(W), rnd(W)
        _report("residual_norm (f32 stream, post and pre norm)", _graph_time(
            [lambda y=y, r=r: D.residual_norm(r, y, w, None, 1e-5,
                                              layer=False, post=post)
             for y, r in zip(ys, rs)]), T * W * 12, 0, shape=[T, W])
        _report("residual_norm (f32 stream, post norm only)", _graph_time(
            [lambda y=y, r=r: D.residual_norm(r, y, None, None, 1e-5,
                                              post=post)
             for y, r in zip(ys, rs)]), T * W * 12, 0, shape=[T, W])
        _report("llama rmsnorm_residual (bf16 stream)", _graph_time(
            [lambda y=y, r=r: D.rmsnorm_residual(y, r, w, 1e-5)
             for y, r in zip(ys, rb)]), T * W * 8, 0, shape=[T, W])
        wf = w.float()
        outs = [torch.empty(T, INNER, device=DEV, dtype=BF)
                for _ in range(reps)]
        _report("part_norm", _graph_time(
            [lambda y=y, o=o: D.part_norm(y, wf, o, 8, 1e-5)
             for y, o in zip(ys, outs)]), T * INNER * 4, 0, shape=[T, INNER])
        _report("llama rmsnorm", _graph_time(
            [lambda y=y: D.rmsnorm(y, w, 1e-5) for y in ys]), T * W * 4, 0,
            shape=[T, W])
        del ys, rs, rb, outs
        gu = [rnd(T, 2 * F) for _ in range(min(reps, 4))]
        _report("glu (gelu)", _graph_time(
            [lambda x=x: D.glu(x[:, :F], x[:, F:], "gelu") for x in gu]),
            T * F * 6, 0, shape=[T, F])
        _report("llama swiglu", _graph_time(
            [lambda x=x: D.swiglu(x[:, :F], x[:, F:]) for x in gu]),
            T * F * 6, 0, shape=[T, F])
        del gu
        table = rnd(32_000, 8 * SIDE)
        ids = torch.randint(0, 32_000, (T,), device=DEV)
        gs = [rnd(T, SIDE) for _ in range(reps)]
        _report("glu_table", _graph_time(
            [lambda g=g: D.glu_table(g, table, ids, 3 * SIDE) for g in gs]),
            T * SIDE * 6, 0, shape=[T, SIDE])


def _convolutions(reps: int) -> None:
    rope = RopeTable(DH, 5e5, DEV)
    rope.ensure(16_384)
    wq, wx = (torch.randn(TAPS, c, device=DEV) for c in (QKV, XBC))
    bias = torch.randn(XBC, device=DEV)
    for n_seq, n in ((64, 1), (1, 8192), (16, 1024)):
        T = n_seq * n
        one = n == 1
        k = reps if one else 3
        xs = [rnd(T, QKV + XBC) for _ in range(k)]
        tails = [(torch.zeros(n_seq, TAPS - 1, QKV, device=DEV, dtype=BF),
                  torch.zeros(n_seq, TAPS - 1, XBC, device=DEV, dtype=BF))
                 for _ in range(k)]
        pages = n_seq * -(-n // 64)
        kc, vc = (torch.zeros(pages, KVH, 64, DH, device=DEV, dtype=BF)
                  for _ in range(2))
        i, item, t0 = _portions(n_seq, n, StepPlan.CONV_ROWS)
        pos = torch.arange(n, device=DEV, dtype=torch.int32)
        slots = (i[:, None] * (64 * -(-n // 64)) + pos).reshape(-1) \
            .contiguous()
        zero = torch.zeros_like(i)
        conv = (None, None, None, zero + 4000, None, i) if one else \
            (item, t0.contiguous(), i * n, zero, zero + n, i)
        extra = n_seq * (TAPS - 1) * 2 * (2 if one else 1)
        _report("conv_qkv (filters, rotation, k and v to pages)", _graph_time(
            [lambda x=x, t=t: D.conv_qkv(
                x[:, :QKV], wq, t[0], rope.cos, rope.sin, DH, slots, kc, vc,
                H, *conv) for x, t in zip(xs, tails)]),
            T * QKV * 4 + QKV * extra + QKV * TAPS * 4 +
            min(n, T) * DH * 4, 0, shape=[n_seq, n, QKV, TAPS])
        _report("conv_silu", _graph_time(
            [lambda x=x, t=t: D.conv_silu(x[:, QKV:], wx, bias, t[1], *conv)
             for x, t in zip(xs, tails)]),
            T * XBC * 4 + XBC * extra + XBC * TAPS * 4, 0,
            shape=[n_seq, n, XBC, TAPS])
        # the Llama decoder's rotation and cache write
        lk = torch.zeros(pages, KVH, DH // 8, 64, 8, device=DEV, dtype=BF)
        lv = torch.zeros(pages, KVH, DH, 64, device=DEV, dtype=BF)
        qkv = [x[:, :QKV].reshape(T, H + 2 * KVH, DH) for x in xs]
        q, kk, v = ([t[:, a:b] for t in qkv] for a, b in (
            (0, H), (H, H + KVH), (H + KVH, H + 2 * KVH)))
        if one:
            bt = i[:, None].contiguous()
            lens = zero + 64
            calls = [lambda a=a, b=b, c=c: ext().rope_kv_append(
                a, b, c, lk, lv, rope.cos, rope.sin, bt, lens)
                for a, b, c in zip(q, kk, v)]
        else:
            q, kk, v = ([t.contiguous() for t in ts] for ts in (q, kk, v))
            p = pos.repeat(n_seq)

            def both(a, b, c):
                ext().rope_inplace(a, b, rope.cos, rope.sin, p)
                ext().kv_scatter(b, c, lk, lv, slots)
            calls = [lambda a=a, b=b, c=c: both(a, b, c)
                     for a, b, c in zip(q, kk, v)]
        _report("llama rope + cache write", _graph_time(calls),
                T * QKV * 4 + min(n, T) * DH * 4, 0, shape=[n_seq, n, QKV])
        del xs, tails, qkv, q, kk, v, calls


def _attention() -> None:
    sink = torch.randn(H, device=DEV)
    for B, ctx in ((8, 4096), (64, 4096)):
        np_ = ctx // 64
        n = max(2, min(6, 256 // B))
        bt = torch.arange(B * np_, device=DEV, dtype=torch.int32) \
            .view(B, np_).contiguous()
        lens = _i32(*[ctx] * B)
        q, gate = rnd(B, H * DH), rnd(B, H * DH)
        out = torch.empty(B, H * DH, device=DEV, dtype=BF)
        size = B * (ctx * KVH * DH * 4 + 4 * H * DH)
        kv = [(rnd(B * np_, KVH, 64, DH), rnd(B * np_, KVH, 64, DH))
              for _ in range(n)]
        _report("gqa_rows (sink, gate, with merge)", _graph_time(
            [lambda c=c: D.gqa_rows(q, c[0], c[1], bt, None, lens, sink,
                                    gate, out, H, 0.1) for c in kv]),
            size + B * H * DH * 2, 4.0 * B * H * ctx * DH,
            shape=[B, ctx, H, KVH, DH])
        kv = [(k.view(-1, KVH, DH // 8, 64, 8), v.view(-1, KVH, DH, 64))
              for k, v in kv]
        q3 = q.view(B, H, DH)
        _report("llama paged_attn_decode (with merge)", _graph_time(
            [lambda c=c: D.paged_attn_decode(q3, c[0], c[1], bt, lens, 0.1)
             for c in kv]), size, 4.0 * B * H * ctx * DH,
            shape=[B, ctx, H, KVH, DH])
        del kv
    for n_seq, n in ((1, 8192), (4, 2048), (16, 1024)):
        T, np_ = n_seq * n, n // 64
        q, gate = rnd(T, H * DH), rnd(T, H * DH)
        out = torch.empty(T, H * DH, device=DEV, dtype=BF)
        k, v = rnd(n_seq * np_, KVH, 64, DH), rnd(n_seq * np_, KVH, 64, DH)
        bt = torch.arange(n_seq * np_, device=DEV, dtype=torch.int32) \
            .view(n_seq, np_).contiguous()
        i, item, t0 = _portions(n_seq, n, D.gqa_portion_rows(DH, DH))
        order = torch.argsort(t0, descending=True, stable=True)
        item, t0 = item[order].contiguous(), t0[order].contiguous()
        zero, lens = torch.zeros_like(i), torch.full_like(i, n)
        flops = 4.0 * n_seq * (n * (n + 1) / 2) * H * DH
        _report("gqa_portions (sink, gate)", _graph_time([
            lambda: D.gqa_portions(q, k, v, bt, sink, gate, item, t0, i * n,
                                   zero, lens, out, H, 0.1)] * 2),
            T * (3 * H + 2 * KVH) * DH * 2, flops,
            shape=[n_seq, n, H, KVH, DH])
        kc, vc = k.view(-1, KVH, DH // 8, 64, 8), v.view(-1, KVH, DH, 64)
        q3 = q.view(T, H, DH)
        _, item16, t16 = _portions(n_seq, n, 16)
        t16 = t16.contiguous()
        _report("llama paged_attn_prefill", _graph_time([
            lambda: ext().paged_attn_prefill(q3, kc, vc, bt, item16, t16,
                                             i * n, zero, lens, 0.1,
                                             True)] * 2),
            T * (2 * H + 2 * KVH) * DH * 2, flops,
            shape=[n_seq, n, H, KVH, DH])


def _state_space(reps: int) -> None:
    A = torch.linspace(1, 16, SH, device=DEV)
    bias = torch.linspace(-6, -2, SH, device=DEV)
    skip = torch.ones(SH, device=DEV)
    cols = INNER + SH                       # z | dt
    # Luzalorn's recurrence of the same state: 32 heads of 128 x 128
    RH, RD = 32, 128
    rope = RopeTable(RD, 1e4, DEV)
    rope.ensure(16_384)
    decay = torch.linspace(0.97, 0.999, RH, device=DEV)
    l2 = torch.log2(decay)
    rwidth = 4 * RH * RD
    for B in (8, 64):
        k = max(2, reps * 8 // B)
        states = [torch.randn(B, SH, N, P, device=DEV) for _ in range(k)]
        u, xbc = rnd(B, cols), rnd(B, XBC)
        slots, lens = _i32(*range(B)), _i32(*[4000] * B)
        _report("ssd_decode", _graph_time(
            [lambda s=s: D.ssd_decode(u, 0, INNER, xbc, A, bias, skip, s, G,
                                      slots, lens) for s in states]),
            B * (SH * N * P * 8 + (XBC + cols + INNER) * 2), 0,
            shape=[B, SH, N, P])
        states = [s.view(B, RH, RD, -1) for s in states]
        x = rnd(B, rwidth)
        _report("luzalorn retention_decode", _graph_time(
            [lambda s=s: D.retention_decode(x, rope.cos, rope.sin, decay, s,
                                            slots, lens, RD, RD ** -0.5,
                                            1e-5) for s in states]),
            B * (RH * RD * RD * 8 + rwidth * 2 + RH * RD * 2), 0,
            shape=[B, RH, RD, RD])
        del states
    for n_seq, n in ((1, 8192), (4, 2048), (32, 1024)):
        T = n_seq * n
        us, xs = [rnd(T, cols) for _ in range(2)], [rnd(T, XBC)
                                                    for _ in range(2)]
        st = torch.zeros(n_seq, SH, N, P, device=DEV)
        out = torch.empty(T, INNER, device=DEV, dtype=BF)
        nch = -(-n // 64)
        i, item, t0 = _portions(n_seq, n, 64)
        t0 = t0.contiguous()
        zero, lens = torch.zeros_like(i), torch.full_like(i, n)
        # chunks of 64: B x^T and S^T C (2 each per state element), per group
        # C B^T over half a chunk, per head the weighted sum of x
        flops = T * (SH * (4 * N * P + 64 * P) + G * 64 * N)
        _report("ssd_chunked (3 kernels)", _graph_time(
            [lambda u=u, x=x: D.ssd_chunked(
                u, 0, INNER, x, A, bias, skip, st, G, i, i * n, zero, lens,
                i * nch, item, t0, out) for u, x in zip(us, xs)]),
            T * (XBC + cols + INNER) * 2, flops, shape=[n_seq, n, SH, N, P])
        del us, xs
        st = st.view(n_seq, RH, RD, RD)
        xs = [rnd(T, rwidth) for _ in range(2)]
        pos = (torch.arange(T, device=DEV, dtype=torch.int32) % n) \
            .contiguous()
        flops = T * RH * (4 * RD * RD + 64 * 2 * RD)
        _report("luzalorn retention_chunked (3 kernels)", _graph_time(
            [lambda x=x: D.retention_chunked(
                x, rope.cos, rope.sin, l2, st, i, i * n, zero, lens, pos,
                i * nch, item, t0, out, RD, RD ** -0.5, 1e-5) for x in xs]),
            T * (rwidth + RH * RD) * 2, flops, shape=[n_seq, n, RH, RD, RD])
        del xs, out


def bench_kernels(reps: int = 8) -> None:
    torch.manual_seed(0)
    _rows(reps)
    _convolutions(reps)
    _attention()
    _state_space(reps)
