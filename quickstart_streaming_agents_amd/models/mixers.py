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

    storage = "state"            # which of the cache's lists a run indexes

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
    def cache(m: dict, shard: Shard) -> dict:
        return {"state": (shard.heads(m["heads"]), m["dim"], m["vdim"])}

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

    storage = "latent"
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

    @staticmethod
    def cache(m: dict, shard: Shard) -> dict:
        return {"latent": m["kv_rank"]}

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


class ConvAttention:
    """Branch: grouped-query attention whose q, k and v pass a short causal
    convolution, then the rotation; per-head softmax sink, sigmoid output
    gate.  Columns of the projection row: [q | k | v | gate].

    Rows of portions of at most `rows_max` tokens are attended one by one (a
    wave per share of a row's pages), longer portions block by block."""

    rows_max = 16

    def __init__(self, m: dict, out_scale: float, get: Getter, shard: Shard,
                 rope: Callable[..., RopeTable], dtype: torch.dtype):
        self.H, self.G = shard.heads(m["heads"]), shard.heads(m["kv_heads"])
        self.D, self.E = m["dim"], m["vdim"]
        if self.H % self.G:
            raise ValueError("query heads do not divide over kv heads")
        self.scale, self.out_scale = float(m["scale"]), float(out_scale)
        rot = m.get("rot") or {"dims": 0, "base": 1.0}
        self.rot = int(rot["dims"])
        self.rope = rope(self.rot, float(rot["base"]), rot.get("scaling"))
        self.channels = (self.H + self.G) * self.D + self.G * self.E
        self.width = self.H * self.E
        self.rows = torch.cat([shard.rows(get(n))
                               for n in ("q", "k", "v", "g")])
        self.out = shard.cols(get("o"))
        self.filters = torch.cat(
            [shard.rows(get(n + ".conv")) for n in ("q", "k", "v")]) \
            .float().t().contiguous()
        self.sink = shard.rows(get("sink")).float()
        self.longest = None
        if self.rows.is_cuda and dtype == torch.bfloat16 and \
                D.gqa_mfma_ok(self.D, self.E):
            self.longest = self.rows_max
            self.block = D.gqa_portion_rows(self.D, self.E)

    @staticmethod
    def shapes(m: dict, width: int) -> dict[str, tuple[int, ...]]:
        q, k = m["heads"] * m["dim"], m["kv_heads"] * m["dim"]
        v, o = m["kv_heads"] * m["vdim"], m["heads"] * m["vdim"]
        return {"q": (q, width), "k": (k, width), "v": (v, width),
                "q.conv": (q, m["conv"]), "k.conv": (k, m["conv"]),
                "v.conv": (v, m["conv"]), "sink": (m["heads"],),
                "g": (o, width), "o": (width, o)}

    @staticmethod
    def cache(m: dict, shard: Shard) -> dict:
        g = shard.heads(m["kv_heads"])
        c = (shard.heads(m["heads"]) + g) * m["dim"] + g * m["vdim"]
        return {"kv": (g, m["dim"], m["vdim"]), "tail": (m["conv"] - 1, c)}

    def __call__(self, x: torch.Tensor, plan: StepPlan, kv, run: int,
                 tails: torch.Tensor, y: torch.Tensor) -> None:
        c = self.channels
        k, v = kv.keys[run], kv.values[run]
        gate = x[:, c:c + self.width]
        q = D.conv_qkv(x[:, :c], self.filters, tails, self.rope.cos,
                       self.rope.sin, self.rot, plan.cache_slots, k, v,
                       self.H, *plan.conv)
        rows = plan.attn_rows(self.longest)
        n = rows.n
        if n:
            D.gqa_rows(q[:n], k, v, rows.table, rows.item, rows.length,
                       self.sink, gate[:n], y[:n], self.H, self.scale,
                       self.out_scale)
        if n < plan.n_rows:
            p = plan.paged_portions(self.longest, self.block)
            D.gqa_portions(q[n:], k, v, p.table, self.sink, gate[n:],
                           p.qb_item, p.qb_t0, p.off, p.start, p.length,
                           y[n:], self.H, self.scale, self.out_scale)


class StateSpace:
    """Branch: state-space duality (Mamba-2).  x, B and C pass a short causal
    convolution and silu, the state decays by exp(-A dt) per head and token,
    the gated read-out is rms-normed in equal parts.  Columns of the
    projection row: [z | x | B | C | dt]."""

    def __init__(self, m: dict, out_scale: float, eps: float, get: Getter,
                 shard: Shard, dtype: torch.dtype):
        self.H, self.P = shard.heads(m["heads"]), m["vdim"]
        self.N, self.G = m["state"], shard.heads(m["groups"])
        if self.H % self.G:
            raise ValueError("heads do not divide over groups")
        self.parts = shard.heads(m["norm_groups"])
        self.eps = eps
        self.width = self.H * self.P
        if self.width % self.parts:
            raise ValueError("inner width does not divide over norm groups")
        inner, gn = m["heads"] * m["vdim"], m["groups"] * m["state"]
        xbc = (inner, gn, gn)

        def pieces(t, sizes):
            return torch.cat([shard.rows(p) for p in t.split(sizes)])

        self.rows = pieces(get("in"), (inner, *xbc, m["heads"]))
        self.filters = pieces(get("conv"), xbc).float().t().contiguous()
        self.bias = pieces(get("conv.b"), xbc).float()
        self.dt_bias = shard.rows(get("dt_bias")).float()
        self.A = torch.exp(shard.rows(get("A_log")).float())
        self.skip = shard.rows(get("D")).float()
        self.norm = shard.rows(get("norm")).float() * float(out_scale)
        self.out = shard.cols(get("o"))
        self.channels = self.filters.shape[1]
        self.chunked = self.rows.is_cuda and dtype == torch.bfloat16 and \
            D.ssd_chunked_ok(self.H, self.N, self.P, self.G)

    @staticmethod
    def shapes(m: dict, width: int) -> dict[str, tuple[int, ...]]:
        h, inner = m["heads"], m["heads"] * m["vdim"]
        c = inner + 2 * m["groups"] * m["state"]
        return {"in": (inner + c + h, width), "conv": (c, m["conv"]),
                "conv.b": (c,), "dt_bias": (h,), "A_log": (h,), "D": (h,),
                "norm": (inner,), "o": (width, inner)}

    @staticmethod
    def cache(m: dict, shard: Shard) -> dict:
        h = shard.heads(m["heads"])
        c = h * m["vdim"] + 2 * shard.heads(m["groups"]) * m["state"]
        return {"state": (h, m["state"], m["vdim"]),
                "tail": (m["conv"] - 1, c)}

    def __call__(self, u: torch.Tensor, plan: StepPlan, kv, run: int,
                 tails: torch.Tensor, y: torch.Tensor) -> None:
        w, state = self.width, kv.states[run]
        dt = w + self.channels
        xbc = D.conv_silu(u[:, w:dt], self.filters, self.bias, tails,
                          *plan.conv)
        const = (self.A, self.dt_bias, self.skip, state, self.G)
        n1 = plan.n_one
        one = None
        if n1:
            one = D.ssd_decode(u[:n1], 0, dt, xbc[:n1], *const,
                               plan.one_slots, plan.one_lens)
        s = one
        if n1 < plan.n_rows:
            s = torch.empty(plan.n_rows, w, dtype=u.dtype, device=u.device)
            if one is not None:
                s[:n1] = one
            args = (u[n1:], 0, dt, xbc[n1:], *const, plan.p_slots,
                    plan.p_off, plan.p_start, plan.p_len)
            if self.chunked:
                D.ssd_chunked(*args, plan.chunk0, plan.chunk_item,
                              plan.chunk_t0, s[n1:])
            else:
                D.ssd_seq(*args, s[n1:])
        D.part_norm(s, self.norm, y, self.parts, self.eps)


class Parallel:
    """Attention and a state-space layer side by side on the same input:
    left_scale * left + right_scale * right.  One GEMM projects for both, one
    sums both: each branch writes its scaled columns of a common row."""

    storage = "state"

    def __init__(self, m: dict, eps: float, get: Getter, shard: Shard,
                 rope, dtype: torch.dtype):
        self.left = ConvAttention(m["left"], m["left_scale"],
                                  lambda k: get("left." + k), shard, rope,
                                  dtype)
        self.right = StateSpace(m["right"], m["right_scale"], eps,
                                lambda k: get("right." + k), shard, dtype)
        # zero rows keep the branches' columns and the row stride aligned
        rows, at = [], []
        for part, unit in ((self.left, 8), (self.right, 16)):
            at.append(sum(r.shape[0] for r in rows))
            w = part.rows
            del part.rows
            rows += [w, w.new_zeros(-(at[-1] + w.shape[0]) % unit,
                                    w.shape[1])]
        self.at = at[1]
        self.proj = Linear(torch.cat(rows))
        self.out = Linear(torch.cat([self.left.out, self.right.out], 1))
        del self.left.out, self.right.out

    @staticmethod
    def shapes(m: dict, width: int) -> dict[str, tuple[int, ...]]:
        return {f"{side}.{k}": s for side, branch in
                (("left", ConvAttention), ("right", StateSpace))
                for k, s in branch.shapes(m[side], width).items()}

    @staticmethod
    def cache(m: dict, shard: Shard) -> dict:
        a = ConvAttention.cache(m["left"], shard)
        b = StateSpace.cache(m["right"], shard)
        return {"state": b["state"], "kv": a["kv"],
                "tails": (a["tail"], b["tail"])}

    def __call__(self, h: torch.Tensor, plan: StepPlan, kv,
                 run: int) -> torch.Tensor:
        x = self.proj(h)
        wl, wr = self.left.width, self.right.width
        y = torch.empty(plan.n_rows, wl + wr, dtype=h.dtype, device=h.device)
        tails = kv.tails[run]
        self.left(x[:, :self.at], plan, kv, run, tails[0], y[:, :wl])
        self.right(x[:, self.at:], plan, kv, run, tails[1], y[:, wl:])
        return self.out(y)


MIXERS = {"retention": Retention, "latent_attention": LatentAttention,
          "parallel": Parallel}


def cache_args(shapes: list[dict]) -> dict:
    """Arguments of HybridCache for the runs of a model, each given by its
    mixer's cache()."""
    rec = [s for s in shapes if "state" in s]
    return {"latent_ranks": [s["latent"] for s in shapes if "latent" in s],
            "state_shapes": [s["state"] for s in rec],
            "kv_shapes": [s.get("kv") for s in rec],
            "tail_shapes": [s.get("tails", ()) for s in rec]}
