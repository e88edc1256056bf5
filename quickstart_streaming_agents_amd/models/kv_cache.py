"""Caches of the decode engine: page pools, and pages + state slots.

`PageAllocator` hands out 64-position pages; one page-id space spans all
layers, so a sequence has ONE page list used by every layer.

`PagedKVCache` (Llama, Mixtral) stores keys and values in the layouts of
ops/hip/paged_attn.hip:
  K: [pages, KVH, D/8, 64, 8]  (d-major x8 -> coalesced MFMA A-frag reads)
  V: [pages, KVH, D, 64]       (transposed, pos minor -> coalesced MFMA
                                B-frag reads in the PV pass)

`HybridCache` serves decoders that mix attention with recurrent layers:
  latents: [pages, 64, rank] per attention run (ops/hip/latent_attn.hip)
  states:  [slots, heads, dim, vdim] f32 per recurrent run
           (ops/hip/retention.hip, ssd.hip), one slot per live sequence
A recurrent run may also hold, at the same index,
  keys:    [pages, kv heads, 64, dim] and values [pages, kv heads, 64, vdim]
           (ops/hip/gqa_attn.hip), for a mixer that attends beside its state
  tails:   [slots, taps - 1, channels] per short convolution, its last inputs
           (ops/hip/short_conv.hip); they share the sequence's slot
A "run" is one execution of a layer: a layer that a loop repeats has a cache
or state of its own for every pass.
"""

from __future__ import annotations

import torch


class PageAllocator:
    PAGE = 64

    def __init__(self, n_pages: int, device: str):
        self.n_pages = n_pages
        self.device = device
        self._free = list(range(n_pages - 1, -1, -1))
        self._seq_pages: dict[int, list[int]] = {}
        self._seq_len: dict[int, int] = {}

    # ---- allocator -------------------------------------------------------
    @property
    def free_pages(self) -> int:
        return len(self._free)

    def pages_for(self, n_tokens: int) -> int:
        return (n_tokens + self.PAGE - 1) // self.PAGE

    def allocate(self, seq_id: int, n_tokens: int) -> None:
        need = self.pages_for(n_tokens)
        if need > len(self._free):
            raise MemoryError("KV cache out of pages")
        self._seq_pages[seq_id] = [self._free.pop() for _ in range(need)]
        self._seq_len[seq_id] = n_tokens

    def extend(self, seq_id: int, new_len: int) -> None:
        pages = self._seq_pages[seq_id]
        need = self.pages_for(new_len)
        while len(pages) < need:
            if not self._free:
                raise MemoryError("KV cache out of pages")
            pages.append(self._free.pop())
        self._seq_len[seq_id] = new_len

    def truncate(self, seq_id: int, new_len: int) -> None:
        """Roll a sequence back to new_len positions (prefix reuse across
        agent turns: decode-token KV beyond the shared prompt is discarded)."""
        pages = self._seq_pages[seq_id]
        keep = max(self.pages_for(new_len), 1)
        while len(pages) > keep:
            self._free.append(pages.pop())
        self._seq_len[seq_id] = new_len

    def free(self, seq_id: int) -> None:
        pages = self._seq_pages.pop(seq_id, [])
        self._free.extend(reversed(pages))
        self._seq_len.pop(seq_id, None)

    # ---- per-sequence state surface (page-only caches hold none) ---------
    has_state = False

    def can_admit(self, seq_id: int, new_pages: int) -> bool:
        return new_pages <= self.free_pages

    def reusable_prefix(self, seq_id: int, n: int) -> int:
        """How many of the first n positions a later turn can build on."""
        return n

    def snapshot(self, seq_id: int) -> None:
        """Remember the sequence as it is now, for truncate() to return to."""

    def claim(self, seq_id: int) -> None:
        """A queued turn builds on this idle sequence: keep what it holds."""

    def seq_len(self, seq_id: int) -> int:
        return self._seq_len.get(seq_id, 0)

    # ---- tensors for a step ---------------------------------------------
    def block_table(self, seq_ids: list[int]) -> torch.Tensor:
        max_pages = max(len(self._seq_pages[s]) for s in seq_ids)
        bt = torch.zeros(len(seq_ids), max_pages, dtype=torch.int32)
        for i, s in enumerate(seq_ids):
            pages = self._seq_pages[s]
            bt[i, :len(pages)] = torch.tensor(pages, dtype=torch.int32)
        return bt.to(self.device)

    def seq_lens_tensor(self, seq_ids: list[int]) -> torch.Tensor:
        return torch.tensor([self._seq_len[s] for s in seq_ids],
                            dtype=torch.int32, device=self.device)

    def slot_ids(self, seq_id: int, start_pos: int, n: int) -> torch.Tensor:
        """Global slot id (page*64 + offset) for positions start..start+n."""
        pages = self._seq_pages[seq_id]
        slots = [pages[(start_pos + i) // self.PAGE] * self.PAGE +
                 (start_pos + i) % self.PAGE for i in range(n)]
        return torch.tensor(slots, dtype=torch.int32, device=self.device)


class PagedKVCache(PageAllocator):
    def __init__(self, n_layers: int, kvh: int, d_head: int, n_pages: int,
                 device: str = "cuda", dtype=torch.bfloat16):
        super().__init__(n_pages, device)
        self.n_layers = n_layers
        self.kvh = kvh
        self.d_head = d_head
        self.k = [torch.zeros(n_pages, kvh, d_head // 8, self.PAGE, 8,
                              dtype=dtype, device=device)
                  for _ in range(n_layers)]
        self.v = [torch.zeros(n_pages, kvh, d_head, self.PAGE, dtype=dtype,
                              device=device)
                  for _ in range(n_layers)]


class HybridCache(PageAllocator):
    """Pages of latents or keys and values, plus state slots.

    Unlike pages, a recurrent state cannot be rolled back to an arbitrary
    earlier position.  A conversation therefore takes a snapshot() when its
    prompt has been read: a copy of its state in a second slot.  truncate()
    to that position swaps the snapshot in; any other rollback leaves the
    sequence without a usable state (reusable_prefix() then answers 0 and
    the caller starts the sequence afresh).  Rolled-back sequences are
    "parked": when slots run out, the longest parked one gives up its slot.

    Slots are not cleared when they change owner: the kernels take the state
    before position 0 as zero.
    """

    has_state = True

    def __init__(self, n_pages: int, n_slots: int,
                 latent_ranks: list[int],
                 state_shapes: list[tuple[int, int, int]],
                 device: str = "cuda", dtype=torch.bfloat16,
                 kv_shapes: list[tuple[int, int, int] | None] = (),
                 tail_shapes: list[tuple[tuple[int, int], ...]] = ()):
        """kv_shapes (kv heads, dim, vdim) or None, and tail_shapes, one
        (taps - 1, channels) per convolution, go with state_shapes."""
        super().__init__(n_pages, device)
        self.n_slots = n_slots
        self.latents = [torch.zeros(n_pages, self.PAGE, r, dtype=dtype,
                                    device=device) for r in latent_ranks]
        self.states = [torch.zeros(n_slots, *s, dtype=torch.float32,
                                   device=device) for s in state_shapes]
        paged = [s and [torch.zeros(n_pages, s[0], self.PAGE, d, dtype=dtype,
                                    device=device) for d in s[1:]]
                 for s in kv_shapes]
        self.keys = [p and p[0] for p in paged]
        self.values = [p and p[1] for p in paged]
        self.tails = [tuple(torch.zeros(n_slots, *t, dtype=dtype,
                                        device=device) for t in ts)
                      for ts in tail_shapes]
        self._free_slots = list(range(n_slots - 1, -1, -1))
        self._slot: dict[int, int] = {}
        self._snap: dict[int, tuple[int, int]] = {}    # seq -> (slot, len)
        self._parked: dict[int, int] = {}              # seq -> state position

    # ---- slots -----------------------------------------------------------
    @property
    def free_slots(self) -> int:
        return len(self._free_slots)

    def _take_slot(self) -> int:
        if not self._free_slots and self._parked:
            victim = next(iter(self._parked))
            del self._parked[victim]
            self._free_slots.append(self._slot.pop(victim))
        if not self._free_slots:
            raise MemoryError("out of state slots")
        return self._free_slots.pop()

    def _drop_snapshot(self, seq_id: int) -> None:
        snap = self._snap.pop(seq_id, None)
        if snap is not None:
            self._free_slots.append(snap[0])

    def slot(self, seq_id: int) -> int:
        return self._slot[seq_id]

    def slots_tensor(self, seq_ids: list[int]) -> torch.Tensor:
        return torch.tensor([self._slot[s] for s in seq_ids],
                            dtype=torch.int32, device=self.device)

    # ---- allocator overrides ---------------------------------------------
    def can_admit(self, seq_id: int, new_pages: int) -> bool:
        return super().can_admit(seq_id, new_pages) and bool(
            seq_id in self._slot or self._free_slots or self._parked)

    def allocate(self, seq_id: int, n_tokens: int) -> None:
        if self.pages_for(n_tokens) > self.free_pages:
            raise MemoryError("KV cache out of pages")
        slot = self._take_slot()
        super().allocate(seq_id, n_tokens)
        self._slot[seq_id] = slot

    def extend(self, seq_id: int, new_len: int) -> None:
        super().extend(seq_id, new_len)
        self._parked.pop(seq_id, None)     # it is running again

    def free(self, seq_id: int) -> None:
        self._drop_snapshot(seq_id)
        self._parked.pop(seq_id, None)
        slot = self._slot.pop(seq_id, None)
        if slot is not None:
            self._free_slots.append(slot)
        super().free(seq_id)

    def snapshot(self, seq_id: int) -> None:
        self._drop_snapshot(seq_id)
        if not self._free_slots and not self._parked:
            return                         # no room: the next turn re-reads
        dst, src = self._take_slot(), self._slot[seq_id]
        for s in (*self.states, *(t for ts in self.tails for t in ts)):
            s[dst].copy_(s[src])
        self._snap[seq_id] = (dst, self._seq_len[seq_id])

    def truncate(self, seq_id: int, new_len: int) -> None:
        super().truncate(seq_id, new_len)
        if self._parked.get(seq_id) == new_len:
            return
        snap = self._snap.pop(seq_id, None)
        if snap is not None and snap[1] == new_len:
            self._free_slots.append(self._slot[seq_id])
            self._slot[seq_id] = snap[0]
            self._parked[seq_id] = new_len
            return
        if snap is not None:
            self._free_slots.append(snap[0])
        self._parked.pop(seq_id, None)
        slot = self._slot.pop(seq_id, None)
        if slot is not None:               # the state is past new_len
            self._free_slots.append(slot)

    def reusable_prefix(self, seq_id: int, n: int) -> int:
        at = self._parked.get(seq_id, 0)
        return at if at <= n else 0

    def claim(self, seq_id: int) -> None:
        self._parked.pop(seq_id, None)
