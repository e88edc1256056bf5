"""Token mixers of the config-driven decoders.

A mixer owns its weights and constants and maps normed rows h [T, width] to
[T, width] for one step (layers.StepPlan), reading and writing its own cache
or state of the given run (kv_cache.HybridCache).  Its output is this rank's
partial sum under tensor parallelism: heads are sharded, the output
projection is row-parallel.

Storage is bf16 or f32; whatever is sensitive (angles, scores, softmax,
norms, decays, states) is f32 inside the kernels for both.
"""

from __future__ import annotations

import math
from typing import Callable

import torch

from ..ops import dispatch as D
from .layers import Linear, RopeTable, StepPlan

Getter = Callable[[str], torch.Tensor]


class Shard:
    """This rank's slice of per-head weights."""

    def __init__(self, rank: int, size: int):
        self.rank, self.size = rank, size

    def heads(self, n: int) -> int:
        if n % self.size:
            raise ValueError(f"{n} heads do not divide over {self.size} ranks")
        return n // self.size

    def rows(self, t: torch.Tensor) -> torch.Tensor:
        n = t.shape[0] // self.size
        return t[self.rank * n:(self.rank + 1) * n].contiguous()

    def cols(self, t: torch.Tensor) -> torch.Tensor:
        n = t.shape[1] // self.size
        return t[:, self.rank * n:(self.rank + 1) * n].contiguous()


class Retention:
    """Linear attention with one fixed decay per head, rotated q and k, and
    a per-head rms norm gated by silu(W_g h)."""

    def __init__(self, m: dict, eps: float, get: Getter, shard: Shard,
                 rope: Callable[[int, float], RopeTable],
                 dtype: torch.dtype):
        self.H = shard.heads(m["heads"])
        self.D, self.E = m["dim"], m["vdim"]
        self.eps = eps
        rot = m.get("rot") or {"dims": 0, "base": 1.0}
        self.rot = int(rot["dims"])
        self.rope = rope(self.rot, float(rot["base"]))
        self.kscale = self.D ** -0.5
        self.proj = Linear(torch.cat([shard.rows(get(n))
                                      for n in ("q", "k", "v", "g")]))
        self.out = Linear(shard.cols(get("o")))
        dev = self.proj.w.device
        decay = shard.rows(torch.tensor(m["decay"], dtype=torch.float64))
        self.decay = decay.float().to(dev)
        self.log2_decay = torch.log2(decay.clamp(min=1e-37)).float().to(dev)
        self.chunked = self.proj.w.is_cuda and dtype == torch.bfloat16 and \
            D.retention_chunked_ok(self.H, self.D, self.E)

    @staticmethod
    def shapes(m: dict, width: int) -> dict[str, tuple[int, ...]]:
        hd, he = m["heads"] * m["dim"], m["heads"] * m["vdim"]
        return {"q": (hd, width), "k": (hd, width), "v": (he, width),
                "g": (he, width), "o": (width, he)}

    @staticmethod
    def state_shape(m: dict, shard: Shard) -> tuple[int, int, int]:
        return shard.heads(m["heads"]), m["dim"], m["vdim"]

    def __call__(self, h: torch.Tensor, plan: StepPlan, kv,
                 run: int) -> torch.Tensor:
        x = self.proj(h)
        state = kv.states[run]
        cos, sin = self.rope.cos, self.rope.sin
        n1 = plan.n_one
        one = None
        if n1:
            one = D.retention_decode(x[:n1], cos, sin, self.decay, state,
                                     plan.one_slots, plan.one_lens, self.rot,
                                     self.kscale, self.eps)
            if n1 == plan.n_rows:
                return self.out(one)
        y = torch.empty(plan.n_rows, self.H * self.E, dtype=h.dtype,
                        device=h.device)
        if one is not None:
            y[:n1] = one
        xs, ys = x[n1:], y[n1:]
        if self.chunked:
            D.retention_chunked(xs, cos, sin, self.log2_decay, state,
                                plan.p_slots, plan.p_off, plan.p_start,
                                plan.p_len, plan.p_pos, plan.chunk0,
                                plan.chunk_item, plan.chunk_t0, ys, self.rot,
                                self.kscale, self.eps)
        else:
            D.retention_seq(xs, cos, sin, self.decay, state, plan.p_slots,
                            plan.p_off, plan.p_start, plan.p_len, ys,
                            self.rot, self.kscale, self.eps)
        return self.out(y)


class LatentAttention:
    """Attention over one cached latent per token: low-rank queries, keys
    and values expanded from the latent, sliding window, per-head softmax
    sink, sigmoid output gate.  No positions.

    Two routes with the same result: `absorbed` (queries folded through W_uk,
    read-out through W_uv; touches only latents) for single tokens and
    portions of at most `absorb_max` tokens, and `expanded` (keys and values
    of the visible context by one GEMM, flash attention) for longer ones.
    """

    absorb_max = 16

    def __init__(self, m: dict, eps: float, get: Getter, shard: Shard,
                 rope, dtype: torch.dtype):
        self.H = H = shard.heads(m["heads"])
        self.D, self.E, self.R = m["dim"], m["vdim"], m["kv_rank"]
        self.Q = m["q_rank"]
        self.eps = eps
        self.scale = float(m["scale"])
        self.window = int((m.get("mask") or {}).get("size") or 0)
        self.proj = Linear(torch.cat([get("dq"), get("dkv"),
                                      shard.rows(get("g"))]))
        self.q_norm, self.kv_norm = get("dq.norm"), get("dkv.norm")
        self.uq = Linear(shard.rows(get("uq")))
        uk, uv = shard.rows(get("uk")), shard.rows(get("uv"))
        self.uk_t = uk.view(H, self.D, self.R).transpose(1, 2).contiguous()
        self.uv = uv.view(H, self.E, self.R).contiguous()
        self.sink = shard.rows(get("sink"))
        self.out = Linear(shard.cols(get("o")))
        self.longest = None
        # sizes of the flash kernel, and a gate slice it can read in words
        if uk.is_cuda and dtype == torch.bfloat16 and \
                (self.Q + self.R) % 4 == 0 and self.R % 8 == 0 and \
                D.window_attn_ok(H, self.D, self.E):
            self.longest = self.absorb_max
            self.ukv = Linear(torch.cat([uk, uv]))

    @staticmethod
    def shapes(m: dict, width: int) -> dict[str, tuple[int, ...]]:
        H, q, r = m["heads"], m["q_rank"], m["kv_rank"]
        return {"dq": (q, width), "dq.norm": (q,),
                "uq": (H * m["dim"], q), "dkv": (r, width),
                "dkv.norm": (r,), "uk": (H * m["dim"], r),
                "uv": (H * m["vdim"], r), "sink": (H,),
                "g": (H * m["vdim"], width), "o": (width, H * m["vdim"])}

    def __call__(self, h: torch.Tensor, plan: StepPlan, kv,
                 run: int) -> torch.Tensor:
        cache = kv.latents[run]
        x = self.proj(h)
        gate = x[:, self.Q + self.R:]
        cq = D.latent_norm_store(x, self.q_norm, self.kv_norm, cache,
                                 plan.cache_slots, self.eps)
        q = self.uq(cq)
        rows = plan.attn_rows(self.longest)
        n, part = rows.n, None
        if n < plan.n_rows:
            part = plan.attn_portions(self.longest, self.window)
        y = None
        if n:
            qa = D.head_matmul(q[:n], self.uk_t)
            lat = D.latent_rows(qa, cache, rows.table, rows.item, rows.length,
                                self.sink, self.window, self.scale)
            y = D.head_matmul(lat, self.uv, gate[:n])
        if part is not None:
            full = torch.empty(plan.n_rows, self.H * self.E, dtype=h.dtype,
                               device=h.device)
            if y is not None:
                full[:n] = y
            c = cache.view(-1, self.R).index_select(0, part.ctx_slots)
            D.window_attn_prefill(q[n:], self.ukv(c), gate[n:], self.sink,
                                  part.qb_item, part.qb_t0, part.off,
                                  part.start, part.length, part.ctx_off,
                                  part.ctx_pos, full[n:], self.D, self.E,
                                  self.window, self.scale)
            y = full
        return self.out(y)


MIXERS = {"retention": Retention, "latent_attention": LatentAttention}
