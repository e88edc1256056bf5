"""Throughput of the mixer decoders beside the Llama decoder at equal width,
feed-forward and depth, and kernel by kernel against the roofline.

    python bench.py --workload luzalorn     (or lunulix)

Random weights, synthetic tokens.  One JSON line per measurement:
  {"kind": "model", ...}   prefill and decode tokens/s of the models
  {"kind": "kernel", ...}  time of a kernel (launched back to back inside a
                           graph, operands rotated so that they do not stay
                           in cache), its roofline time max(bytes / 8 TB/s,
                           flops / 2.5 PFLOP/s) and the fraction reached,
                           beside the like kernel of the Llama decoder
"""

from __future__ import annotations

import json
import time

import torch

from ..ops import dispatch as D
from ..ops import ext

HBM, MFMA = 8.0e12, 2.5e15


def _graph_time(calls, rounds=5):
    """Seconds per call of the callables, replayed from one graph."""
    for c in calls[:2]:
        c()
    torch.cuda.synchronize()
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        for c in calls:
            c()
    g.replay()
    torch.cuda.synchronize()
    best = 1e9
    for _ in range(rounds):
        a, b = (torch.cuda.Event(enable_timing=True) for _ in range(2))
        a.record()
        g.replay()
        b.record()
        torch.cuda.synchronize()
        best = min(best, a.elapsed_time(b) * 1e-3 / len(calls))
    return best


def _report(name, secs, bytes_, flops, **extra):
    roof = max(bytes_ / HBM, flops / MFMA)
    print(json.dumps({
        "kind": "kernel", "kernel": name, "us": round(secs * 1e6, 2),
        "roofline_us": round(roof * 1e6, 2),
        "fraction": round(roof / secs, 3),
        "bound": "hbm" if bytes_ / HBM >= flops / MFMA else "mfma",
        **extra}), flush=True)


def _i32(*v):
    return torch.tensor(v, dtype=torch.int32, device="cuda:0")


def bench_kernels(reps: int = 8) -> None:
    dev, bf = "cuda:0", torch.bfloat16
    torch.manual_seed(0)

    def rnd(*s):
        return torch.randn(*s, device=dev, dtype=torch.float32).to(bf)

    # ---- norms and gated activation --------------------------------------
    for T, W in ((64, 4096), (8192, 4096)):
        ys = [rnd(T, W) for _ in range(reps)]
        rs = [torch.randn(T, W, device=dev) for _ in range(reps)]
        rb = [r.to(bf) for r in rs]
        w, b = rnd(W), rnd(W)
        _report("residual_norm (f32 stream, layer norm)", _graph_time(
            [lambda y=y, r=r: D.residual_norm(r, y, w, b, 1e-5)
             for y, r in zip(ys, rs)]), T * W * 12, 0, shape=[T, W])
        _report("llama rmsnorm_residual (bf16 stream)", _graph_time(
            [lambda y=y, r=r: D.rmsnorm_residual(y, r, w, 1e-5)
             for y, r in zip(ys, rb)]), T * W * 8, 0, shape=[T, W])
    for T, F in ((64, 14336), (8192, 14336)):
        gu = [rnd(T, 2 * F) for _ in range(min(reps, 4))]
        _report("glu", _graph_time([lambda x=x: D.glu(x[:, :F], x[:, F:])
                                    for x in gu]), T * F * 6, 0, shape=[T, F])
        _report("llama swiglu", _graph_time(
            [lambda x=x: D.swiglu(x[:, :F], x[:, F:]) for x in gu]),
            T * F * 6, 0, shape=[T, F])
        del gu

    # ---- retention --------------------------------------------------------
    from .layers import RopeTable
    H, Dm, E = 16, 128, 256
    rope = RopeTable(Dm, 1e4, dev)
    rope.ensure(16384)
    decay = torch.linspace(0.97, 0.999, H, device=dev)
    l2 = torch.log2(decay)
    width = 2 * H * (Dm + E)
    for B in (8, 64):
        states = [torch.randn(B, H, Dm, E, device=dev)
                  for _ in range(max(2, reps * 8 // B))]
        x = rnd(B, width)
        slots, lens = _i32(*range(B)), _i32(*[4000] * B)
        _report("retention_decode", _graph_time(
            [lambda s=s: D.retention_decode(x, rope.cos, rope.sin, decay, s,
                                            slots, lens, Dm, Dm ** -0.5,
                                            1e-5) for s in states]),
            B * (H * Dm * E * 8 + width * 2 + H * E * 2), 0,
            shape=[B, H, Dm, E])
        del states
    for n_seq, n in ((1, 8192), (4, 2048), (32, 1024)):
        T = n_seq * n
        xs = [rnd(T, width) for _ in range(2)]
        st = torch.zeros(n_seq, H, Dm, E, device=dev)
        out = torch.empty(T, H * E, device=dev, dtype=bf)
        nch = -(-n // 64)
        i = torch.arange(n_seq, device=dev, dtype=torch.int32)
        pos = (torch.arange(T, device=dev, dtype=torch.int32) % n).contiguous()
        ch_item = i.repeat_interleave(nch).contiguous()
        ch_t0 = (torch.arange(nch, device=dev, dtype=torch.int32) * 64) \
            .repeat(n_seq).contiguous()
        lens = torch.full_like(i, n)
        zero = torch.zeros_like(i)
        # recurrent form's work in chunks of 64: k v^T and S^T q (2 each per
        # state element), q k^T and P v over half a chunk
        flops = T * H * (4 * Dm * E + 64 * (Dm + E))
        _report("retention_chunked (3 kernels)", _graph_time(
            [lambda x=x: D.retention_chunked(
                x, rope.cos, rope.sin, l2, st, i, i * n, zero, lens, pos,
                i * nch, ch_item, ch_t0, out, Dm, Dm ** -0.5, 1e-5)
             for x in xs]),
            T * (width + H * E) * 2, flops, shape=[n_seq, n, H, Dm, E])
        del xs, out

    # ---- latent attention beside paged GQA attention -----------------------
    H, Dm, E, R, KVH = 32, 128, 128, 512, 8
    sink = rnd(H)
    for B, ctx in ((8, 4096), (64, 4096)):
        np_ = ctx // 64
        n = max(2, min(6, 256 // B))
        caches = [rnd(B * np_, 64, R) for _ in range(n)]
        bt = torch.arange(B * np_, device=dev, dtype=torch.int32) \
            .view(B, np_).contiguous()
        lens = _i32(*[ctx] * B)
        qa = rnd(B, H * R)
        _report("latent_rows (absorbed decode, with merge)", _graph_time(
            [lambda c=c: D.latent_rows(qa, c, bt, None, lens, sink, 0, 0.1)
             for c in caches]),
            B * (ctx * R * 2 + 4 * H * R), 4.0 * B * H * ctx * R,
            shape=[B, ctx, H, R])
        del caches
        kcs = [(rnd(B * np_, KVH, Dm // 8, 64, 8), rnd(B * np_, KVH, Dm, 64))
               for _ in range(n)]
        q = rnd(B, H, Dm)
        _report("llama paged_attn_decode (with merge)", _graph_time(
            [lambda k=k: D.paged_attn_decode(q, k[0], k[1], bt, lens, 0.1)
             for k in kcs]),
            B * (ctx * KVH * Dm * 4 + 4 * H * Dm), 4.0 * B * H * ctx * Dm,
            shape=[B, ctx, H, KVH, Dm])
        del kcs
        for name, N, K in (("absorb", R, Dm), ("expand", E, R)):
            w = [rnd(H, N, K) for _ in range(reps)]
            x = rnd(B, H * K)
            _report(f"head_matmul {name}", _graph_time(
                [lambda v=v: D.head_matmul(x, v) for v in w]),
                H * N * K * 2 + B * H * (N + K) * 2, 2.0 * B * H * N * K,
                shape=[B, H, N, K])
        w = [rnd(H * Dm, 4096) for _ in range(reps)]
        x = rnd(B, 4096)
        _report("vendor GEMM of the same class (decode q projection)",
                _graph_time([lambda v=v: torch.nn.functional.linear(x, v)
                             for v in w]),
                H * Dm * 4096 * 2 + B * (4096 + H * Dm) * 2,
                2.0 * B * H * Dm * 4096, shape=[B, H * Dm, 4096])
    for n_seq, n, window in ((1, 8192, 0), (1, 8192, 4096), (4, 2048, 0)):
        T = n_seq * n
        q, gate = rnd(T, H * Dm), rnd(T, H * E)
        kvx = rnd(T, H * (Dm + E))
        out = torch.empty(T, H * E, device=dev, dtype=bf)
        i = torch.arange(n_seq, device=dev, dtype=torch.int32)
        nqb = -(-n // 64)
        item = i.repeat_interleave(nqb).contiguous()
        t0 = (torch.arange(nqb, device=dev, dtype=torch.int32) * 64) \
            .repeat(n_seq).contiguous()
        zero, lens = torch.zeros_like(i), torch.full_like(i, n)
        w = window or n
        pairs = n_seq * (w * (w + 1) / 2 + (n - w) * w)
        _report("window_attn_prefill (sink, gate)", _graph_time([
            lambda: D.window_attn_prefill(
                q, kvx, gate, sink, item, t0, i * n, zero, lens, i * n, zero,
                out, Dm, E, window, 0.1)] * 2),
            T * H * (2 * Dm + 3 * E) * 2, 2.0 * pairs * H * (Dm + E),
            shape=[n_seq, n, H, Dm, E], window=window)
        if window:
            continue
        np_ = n // 64
        kc = rnd(n_seq * np_, KVH, Dm // 8, 64, 8)
        vc = rnd(n_seq * np_, KVH, Dm, 64)
        bt = torch.arange(n_seq * np_, device=dev, dtype=torch.int32) \
            .view(n_seq, np_).contiguous()
        q3 = q.view(T, H, Dm)
        item16 = i.repeat_interleave(n // 16).contiguous()
        t16 = (torch.arange(n // 16, device=dev, dtype=torch.int32) * 16) \
            .repeat(n_seq).contiguous()
        _report("llama paged_attn_prefill", _graph_time([
            lambda: ext().paged_attn_prefill(q3, kc, vc, bt, item16, t16,
                                             i * n, zero, lens, 0.1,
                                             True)] * 2),
            T * (2 * H + 2 * KVH) * Dm * 2, 4.0 * pairs * H * Dm,
            shape=[n_seq, n, H, KVH, Dm])


def _models(width: int, ff: int, layers: int, names: tuple):
    """(name, class, configuration) of decoders of equal size."""
    from .llama import LlamaConfig, LlamaModel
    from .lunulix import LunulixConfig, LunulixModel
    from .luzalorn import LuzalornConfig, LuzalornModel
    heads = width // 128
    mlp = {"kind": "dense", "ff": ff}
    ret = {"type": "retention", "mixer": {
        "heads": heads // 2, "dim": 128, "vdim": 256,
        "decay": [1 - 2.0 ** (-5 - i % 6) for i in range(heads // 2)],
        "rot": {"dims": 128, "base": 1e4}}}
    lat = {"type": "latent_attention", "mixer": {
        "heads": heads, "dim": 128, "vdim": 128, "q_rank": width * 3 // 8,
        "kv_rank": 512, "scale": 128 ** -0.5, "mask": {"size": 4096}}}
    par = {"type": "parallel", "mixer": {
        "left": {"heads": heads, "kv_heads": 8, "dim": 128, "vdim": 128,
                 "conv": 4, "scale": 128 ** -0.5,
                 "rot": {"dims": 128, "base": 5e5}}, "left_scale": 0.7,
        "right": {"heads": width // 64, "vdim": 64, "state": 128,
                  "groups": 8, "conv": 4, "norm_groups": 8},
        "right_scale": 0.7}}
    found = {
        "luzalorn": (LuzalornModel, LuzalornConfig(
            layers=[dict(lat if i % 4 == 3 else ret, mlp=mlp)
                    for i in range(layers)], vocab_size=32_000,
            hidden=width)),
        "lunulix": (LunulixModel, LunulixConfig(
            layers=[dict(par, mlp=mlp)] * layers, vocab_size=32_000,
            hidden=width, side_dim=width // 16)),
        "llama": (LlamaModel, LlamaConfig(
            name="bench", vocab_size=32_000, hidden=width, n_layers=layers,
            n_q_heads=heads, n_kv_heads=8, d_head=128, ffn=ff,
            max_pos=16_384))}
    for name in names:
        yield name, *found[name]


def bench_models(names: tuple, layers: int = 8) -> None:
    from .serve import Engine
    for width, ff in ((2048, 8192), (4096, 14_336)):
        for name, cls, cfg in _models(width, ff, layers, names):
            model = cls(cfg, device="cuda:0")
            for n_seq, n in ((1, 8192), (16, 1024)):
                kv = model.new_kv_cache(n_seq * n // 64, state_slots=n_seq)
                for s in range(n_seq):
                    kv.allocate(s, n)
                items = [(torch.randint(0, 32_000, (n,), device="cuda:0"), s,
                          0) for s in range(n_seq)]
                best = 1e9
                for _ in range(4):
                    torch.cuda.synchronize()
                    t = time.perf_counter()
                    model.forward_prefill_batch(items, kv)
                    torch.cuda.synchronize()
                    best = min(best, time.perf_counter() - t)
                print(json.dumps({
                    "kind": "model", "model": name, "width": width, "ff": ff,
                    "layers": layers, "phase": "prefill",
                    "batch": [n_seq, n], "ms": round(best * 1e3, 3),
                    "tokens_per_s": round(n_seq * n / best)}), flush=True)
                del kv, items
            for B in (1, 16, 64):
                eng = Engine(model, max_batch=B, max_seq_len=2560)
                prompts = [[(i * 7 + j) % 30_000 for j in range(2048)]
                           for i in range(B)]
                seqs = [eng.submit(p, 260) for p in prompts]
                while eng.pending:
                    eng._admit()
                eng._decode_run_graph(seqs, 2)        # capture and warm up
                torch.cuda.synchronize()
                t = time.perf_counter()
                eng._decode_run_graph(seqs, 128)
                torch.cuda.synchronize()
                t = (time.perf_counter() - t) / 128
                assert eng.use_graph
                print(json.dumps({
                    "kind": "model", "model": name, "width": width, "ff": ff,
                    "layers": layers, "phase": "decode", "batch": B,
                    "context": 2048, "ms_per_step": round(t * 1e3, 4),
                    "tokens_per_s": round(B / t)}), flush=True)
                del eng, seqs
            del model
            torch.cuda.empty_cache()


def main(workload: str) -> None:
    """workload: <design>[-kernels | -models]"""
    design, _, part = workload.partition("-")
    if part in ("", "kernels"):
        with torch.no_grad():
            if design == "lunulix":
                from .bench_lunulix import bench_kernels as kernels
                kernels()
            else:
                bench_kernels()
    if part in ("", "models"):
        bench_models((design, "llama") if design == "luzalorn" else
                     (design, "luzalorn", "llama"))
