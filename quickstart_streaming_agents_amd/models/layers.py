"""Building blocks shared by the mixer decoders: projections, rotation
tables, feed-forwards and the device-side description of a step."""

from __future__ import annotations

import math

import numpy as np
import torch
import torch.nn.functional as F

from ..ops import dispatch as D


class Linear:
    """y = x W^T.  On the GPU in bf16, decode-sized batches of the small
    shapes stream a packed copy of W (ops/hip/skinny_gemm.hip, the measured
    winner there); everything else is a vendor GEMM."""

    SKINNY_ROWS = 32
    SKINNY_MAX = 6144 * 4096

    def __init__(self, w: torch.Tensor):
        self.w = w
        n, k = w.shape
        self.packed = None
        if w.is_cuda and w.dtype == torch.bfloat16 and \
                D.can_pack_weight(n, k) and n * k <= self.SKINNY_MAX:
            self.packed = D.pack_weight_frag(w)

    def __call__(self, x: torch.Tensor) -> torch.Tensor:
        n, k = self.w.shape
        if self.packed is not None and 1 <= x.shape[0] <= self.SKINNY_ROWS \
                and x.stride(0) % 8 == 0:
            return D.skinny_linear(x, self.packed, n, k)
        return F.linear(x, self.w)


def rope_frequencies(dims: int, base: float,
                     scaling: dict | None = None) -> torch.Tensor:
    """Angle per position of each rotated pair, base^(-2i/dims) in f64.
    `scaling` (factor, low, high, original) stretches a model's context as
    Llama 3.1 does: wavelengths beyond original/low are slowed down by factor,
    those under original/high kept, and the ones between blended."""
    f = base ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64)
                 / max(dims, 1))
    if not scaling:
        return f
    n, low, high = (float(scaling[k]) for k in ("original", "low", "high"))
    slow = f / float(scaling["factor"])
    wave = 2.0 * math.pi / f
    s = (n / wave - low) / (high - low) if high != low \
        else torch.zeros_like(f)
    out = (1.0 - s) * slow + s * f
    out = torch.where(wave > n / low, slow, out)
    return torch.where(wave < n / high, f, out)


class RopeTable:
    """cos/sin of p * frequency, [positions, dims/2] f32, evaluated in f64.
    Grows on demand; earlier tables stay alive because a captured graph may
    still read them."""

    def __init__(self, dims: int, base: float, device: str,
                 scaling: dict | None = None):
        self.dims, self.base, self.device = dims, base, device
        self.freq = rope_frequencies(dims, base, scaling)
        self._kept: list[torch.Tensor] = []
        self.cos = self.sin = torch.zeros(0, dims // 2, device=device)

    def ensure(self, n: int) -> None:
        if n <= self.cos.shape[0]:
            return
        n = max(256, 1 << (n - 1).bit_length())
        ang = torch.outer(torch.arange(n, dtype=torch.float64), self.freq)
        self._kept += [self.cos, self.sin]
        self.cos = ang.cos().float().to(self.device)
        self.sin = ang.sin().float().to(self.device)


class DenseGLU:
    """W_down(act(W_gate h) * (W_up h)); gate and up share one GEMM."""

    def __init__(self, gate: torch.Tensor, up: torch.Tensor,
                 down: torch.Tensor, act: str = "silu"):
        self.ff, self.act = gate.shape[0], act
        self.gate_up = Linear(torch.cat([gate, up]).contiguous())
        self.down = Linear(down)

    def __call__(self, h: torch.Tensor) -> torch.Tensor:
        gu = self.gate_up(h)
        return self.down(D.glu(gu[:, :self.ff], gu[:, self.ff:], self.act))


class TokenSide:
    """Per-layer input of the token itself: W_proj(act(W_gate x) * e), e the
    layer's columns of the token's row in a table that all layers share."""

    def __init__(self, gate: torch.Tensor, proj: torch.Tensor,
                 table: torch.Tensor, layer: int, act: str = "gelu"):
        self.table, self.act = table, act
        self.col0 = layer * gate.shape[0]
        self.gate, self.proj = Linear(gate), Linear(proj)

    def __call__(self, x: torch.Tensor, ids: torch.Tensor) -> torch.Tensor:
        return self.proj(D.glu_table(self.gate(x), self.table, ids,
                                     self.col0, self.act))


def ints_to_device(device, *arrays: np.ndarray) -> list[torch.Tensor]:
    """Several int32 arrays in one host-to-device copy."""
    sizes = [len(a) for a in arrays]
    flat = np.concatenate([np.asarray(a, dtype=np.int32) for a in arrays]) \
        if arrays else np.zeros(0, np.int32)
    return list(torch.from_numpy(flat).to(device).split(sizes))


class AttnRows:
    """Rows whose attention goes through the latents directly."""

    def __init__(self, n, table, item, length):
        self.n, self.table, self.item, self.length = n, table, item, length


class AttnPortions:
    """Portions whose visible context is expanded to keys and values."""

    def __init__(self, qb_item, qb_t0, off, start, length, ctx_off, ctx_pos,
                 ctx_slots):
        self.qb_item, self.qb_t0 = qb_item, qb_t0
        self.off, self.start, self.length = off, start, length
        self.ctx_off, self.ctx_pos = ctx_off, ctx_pos
        self.ctx_slots = ctx_slots


class PagedPortions:
    """Portions whose queries go over the pages block by block."""

    def __init__(self, qb_item, qb_t0, off, start, length, table):
        self.qb_item, self.qb_t0 = qb_item, qb_t0
        self.off, self.start, self.length = off, start, length
        self.table = table


class StepPlan:
    """Device-side description of one engine step.

    Rows of all entries are concatenated, single tokens first, then portions
    by length, so every kernel family works on one contiguous row range:
    rows [0, n_one) advance a sequence by one token, the rest are portions
    of at least two tokens.  `order` maps the plan's entries back to the
    caller's.  `conv` describes all rows to the short convolutions: portions
    in chunks of CONV_ROWS rows, or single tokens (ops.dispatch.conv_qkv).
    """

    CONV_ROWS = 16

    def __init__(self):
        self._rows: dict = {}
        self._portions: dict = {}

    # ---- a pure decode step (graph-capturable: device tensors only) ------
    @classmethod
    def decode(cls, tokens, block_table, seq_lens, state_slots):
        p = cls()
        p.tokens = tokens
        p.n_rows = p.n_one = tokens.shape[0]
        p.block_table = block_table
        p.one_lens = seq_lens
        p.one_slots = state_slots
        p.cache_slots = D.decode_slots(block_table, seq_lens)
        p.conv = (None, None, None, seq_lens, None, state_slots)
        p.items = None
        return p

    # ---- any mixture of single tokens and portions -----------------------
    @classmethod
    def build(cls, items, kv):
        """items: (tokens [n] i64 on the device, seq_id, start)."""
        p = cls()
        dev, page = kv.device, kv.PAGE
        p.device, p.page = dev, page
        lens = np.array([int(t.shape[0]) for t, _, _ in items])
        p.order = np.argsort(lens, kind="stable")
        items = [items[i] for i in p.order]
        lens = lens[p.order]
        starts = np.array([int(s) for _, _, s in items])
        p.items, p.lens, p.starts = items, lens, starts
        p.offs = np.concatenate([[0], np.cumsum(lens)])
        p.n_rows = T = int(p.offs[-1])
        p.n_one = n1 = int((lens == 1).sum())
        p.tokens = torch.cat([t for t, _, _ in items])
        p.pages = [np.array(kv._seq_pages[sid]) for _, sid, _ in items]
        cap = max(len(g) for g in p.pages)
        table = np.zeros((len(items), cap), dtype=np.int32)
        for i, g in enumerate(p.pages):
            table[i, :len(g)] = g
        row_item = np.repeat(np.arange(len(items)), lens)
        pos = starts[row_item] + np.arange(T) - p.offs[row_item]
        p.row_item, p.pos = row_item, pos
        slot_ids = table[row_item, pos // page] * page + pos % page
        state = np.array([kv.slot(sid) for _, sid, _ in items])
        nch = -(-lens[n1:] // 64)
        chunk0 = np.cumsum(nch) - nch
        ch_item = np.repeat(np.arange(len(nch)), nch)
        ch_t0 = (np.arange(int(nch.sum())) - chunk0[ch_item]) * 64 \
            if len(nch) else np.zeros(0)
        cv_item, cv_t0 = cls._cut(lens, cls.CONV_ROWS)
        (bt, p.cache_slots, p.one_slots, p.one_lens, p.p_slots, p.p_off,
         p.p_start, p.p_len, p.p_pos, p.chunk0, p.chunk_item,
         p.chunk_t0, *conv) = ints_to_device(
            dev, table.reshape(-1), slot_ids, state[:n1], starts[:n1] + 1,
            state[n1:], p.offs[n1:-1] - n1, starts[n1:], lens[n1:], pos[n1:],
            chunk0, ch_item, ch_t0, cv_item, cv_t0, p.offs[:-1], starts, lens,
            state)
        p.conv = tuple(conv)
        p.block_table = bt.view(len(items), cap)
        return p

    @staticmethod
    def _cut(lens, size: int):
        """(entry, first token) of pieces of at most `size` tokens."""
        n = -(-lens // size)
        item = np.repeat(np.arange(len(lens)), n)
        return item, (np.arange(int(n.sum()))
                      - (np.cumsum(n) - n)[item]) * size

    # ---- attention routes ------------------------------------------------
    def attn_rows(self, longest: int | None) -> AttnRows:
        """Rows of entries of at most `longest` tokens (None: all rows)."""
        if self.items is None:
            return AttnRows(self.n_rows, self.block_table, None,
                            self.one_lens)
        if longest not in self._rows:
            k = len(self.lens) if longest is None else \
                int((self.lens <= longest).sum())
            n = int(self.offs[k])
            item, length = ints_to_device(self.device, self.row_item[:n],
                                          self.pos[:n] + 1)
            self._rows[longest] = AttnRows(n, self.block_table, item, length)
        return self._rows[longest]

    def attn_portions(self, longest: int | None,
                      window: int) -> AttnPortions | None:
        """Entries of more than `longest` tokens, row offsets counted from
        the first of their rows, and the context a window leaves visible."""
        if self.items is None or longest is None:
            return None
        key = (longest, window)
        if key not in self._portions:
            k = int((self.lens <= longest).sum())
            lens, starts = self.lens[k:], self.starts[k:]
            if not len(lens):
                self._portions[key] = None
                return None
            first = np.maximum(0, starts - window + 1) if window > 0 \
                else np.zeros_like(starts)
            n_ctx = starts + lens - first
            ctx_off = np.cumsum(n_ctx) - n_ctx
            ctx = [g[q // self.page] * self.page + q % self.page
                   for g, q in ((self.pages[k + i],
                                 np.arange(first[i], first[i] + n_ctx[i]))
                                for i in range(len(lens)))]
            nqb = -(-lens // 64)
            qb_item = np.repeat(np.arange(len(lens)), nqb)
            qb_t0 = (np.arange(int(nqb.sum()))
                     - (np.cumsum(nqb) - nqb)[qb_item]) * 64
            self._portions[key] = AttnPortions(*ints_to_device(
                self.device, qb_item, qb_t0, self.offs[k:-1] - self.offs[k],
                starts, lens, ctx_off, first, np.concatenate(ctx)))
        return self._portions[key]

    def paged_portions(self, longest: int | None,
                       rows: int) -> PagedPortions | None:
        """Entries of more than `longest` tokens in blocks of `rows` query
        rows, the ones with most keys first; row offsets count from the first
        of their rows."""
        if self.items is None or longest is None:
            return None
        key = ("paged", longest, rows)
        if key not in self._portions:
            k = int((self.lens <= longest).sum())
            lens, starts = self.lens[k:], self.starts[k:]
            if not len(lens):
                self._portions[key] = None
                return None
            item, t0 = self._cut(lens, rows)
            heavy = np.argsort(-(starts[item] + t0), kind="stable")
            self._portions[key] = PagedPortions(*ints_to_device(
                self.device, item[heavy], t0[heavy],
                self.offs[k:-1] - self.offs[k], starts, lens),
                self.block_table[k:])
        return self._portions[key]
