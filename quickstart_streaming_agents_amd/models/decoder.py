"""What the config-driven mixer decoders share: weights from a mapping checked
against the configuration, rotation tables, the cache their mixers ask for,
and the step functions that the engine calls.

A design subclasses MixerDecoder with its configuration class, its checkpoint
layout (`shapes`, `random`), the order of its layer runs, `build` (take the
weights) and `_forward` (one step over all rows of a StepPlan).
"""

from __future__ import annotations

import os
from dataclasses import dataclass

import torch

from .kv_cache import HybridCache
from .layers import RopeTable, StepPlan
from .mixers import MIXERS, Shard, cache_args
from .weights import SafetensorsFile


@dataclass
class LayerRun:
    """One execution of a layer."""
    layer: int
    cache: int                   # index among the runs of its kind of storage
    step: int | None = None      # first layer of pass t: add loop.step[t]
    re_embed: bool = False       # ... and the embedding output


def number_runs(layers: list[dict],
                order: list[tuple[int, int | None]]) -> list[LayerRun]:
    """Layer runs with their cache indices; order: (layer, pass begun)."""
    count: dict[str, int] = {}
    runs = []
    for i, t in order:
        kind = MIXERS[layers[i]["type"]].storage
        k = count.get(kind, 0)
        count[kind] = k + 1
        runs.append(LayerRun(i, k, step=t, re_embed=t is not None and t > 0))
    return runs


def check_layers(layers: list[dict]) -> None:
    for i, L in enumerate(layers):
        if L["type"] not in MIXERS:
            raise ValueError(f"layer {i}: unknown mixer {L['type']!r}")
        if L.get("mlp") and L["mlp"].get("kind", "dense") != "dense":
            raise ValueError(f"layer {i}: unknown feed-forward "
                             f"{L['mlp']['kind']!r}")


class MixerDecoder:
    Config: type

    def __init__(self, cfg, device: str = "cuda", dtype=torch.bfloat16,
                 seed: int = 0, weights=None, tp_rank: int = 0,
                 tp_size: int = 1, tp_group=None):
        """weights: name -> tensor mapping (a dict or SafetensorsFile);
        without it, random weights from `seed`."""
        self.cfg, self.device, self.dtype = cfg, device, dtype
        self.tp_rank, self.tp_size, self.tp_group = tp_rank, tp_size, tp_group
        self.runs = self.layer_runs(cfg)
        self.shard = Shard(tp_rank, tp_size)
        self._ropes: dict[tuple, RopeTable] = {}
        shapes = self.shapes(cfg)
        if weights is None:
            weights = dict(self.random(cfg, device, dtype, seed))

        def get(name: str) -> torch.Tensor:
            t = weights.get(name)
            if t is None:
                raise KeyError(f"checkpoint has no tensor {name!r}")
            if tuple(t.shape) != shapes[name]:
                raise ValueError(f"{name}: shape {tuple(t.shape)}, the "
                                 f"configuration asks for {shapes[name]}")
            return t.to(device=device, dtype=dtype).contiguous()

        self.build(get)
        self.ensure_positions(256)

    @classmethod
    def from_folder(cls, folder: str, config: dict, device: str = "cuda",
                    dtype=torch.bfloat16, **kw) -> "MixerDecoder":
        f = SafetensorsFile(os.path.join(folder, "model.safetensors"))
        try:
            return cls(cls.Config.from_dict(config), device=device,
                       dtype=dtype, weights=f, **kw)
        finally:
            f.close()

    # ---- what a design provides --------------------------------------------
    def build(self, get) -> None:
        raise NotImplementedError

    def _forward(self, plan: StepPlan, kv: HybridCache,
                 rows: torch.Tensor | None,
                 trail: list | None = None) -> torch.Tensor:
        """One step over all rows; logits of `rows` (None: every row).
        trail collects the residual stream after every layer run."""
        raise NotImplementedError

    # ---- positions, cache --------------------------------------------------
    def _rope(self, dims: int, base: float,
              scaling: dict | None = None) -> RopeTable:
        key = (dims, base, tuple(sorted((scaling or {}).items())))
        if key not in self._ropes:
            self._ropes[key] = RopeTable(dims, base, self.device, scaling)
        return self._ropes[key]

    def ensure_positions(self, n: int) -> None:
        for r in self._ropes.values():
            r.ensure(n)

    def new_kv_cache(self, n_pages: int,
                     state_slots: int | None = None) -> HybridCache:
        layers = [self.cfg.layers[r.layer] for r in self.runs]
        return HybridCache(
            n_pages, state_slots or 64, device=self.device, dtype=self.dtype,
            **cache_args([MIXERS[L["type"]].cache(L["mixer"], self.shard)
                          for L in layers]))

    def _reduce(self, y: torch.Tensor) -> torch.Tensor:
        if self.tp_size > 1:
            import torch.distributed as dist
            dist.all_reduce(y, group=self.tp_group)
        return y

    # ---- steps -------------------------------------------------------------
    @torch.no_grad()
    def forward_decode(self, tokens: torch.Tensor, kv: HybridCache,
                       block_table: torch.Tensor, seq_lens: torch.Tensor,
                       positions: torch.Tensor,
                       state_slots: torch.Tensor) -> torch.Tensor:
        """tokens [B] i64 -> logits [B, vocab]; seq_lens INCLUDE the new
        token.  Rows with seq_len 0 and slot -1 are padding."""
        plan = StepPlan.decode(tokens, block_table, seq_lens, state_slots)
        return self._forward(plan, kv, None)

    @torch.no_grad()
    def forward_prefill_batch(self, items, kv: HybridCache,
                              want: list[list[int]] | None = None,
                              trail: list | None = None) -> torch.Tensor:
        """One step over entries (tokens [n] i64, seq_id, start): portions of
        prompts of any length beside single tokens.  Returns the logits at
        the places `want` of every entry (default: its last), in order."""
        self.ensure_positions(max(int(s) + int(t.shape[0])
                                  for t, _, s in items))
        plan = StepPlan.build(items, kv)
        first = {int(e): int(plan.offs[i]) for i, e in enumerate(plan.order)}
        if want is None:
            want = [[int(t.shape[0]) - 1] for t, _, _ in items]
        rows = [first[e] + w for e, ws in enumerate(want) for w in ws]
        # with nothing wanted the caches still have to advance: one row's
        # logits are computed and dropped
        idx = torch.tensor(rows or [0], dtype=torch.int64, device=self.device)
        return self._forward(plan, kv, idx, trail)[:len(rows)]

    @torch.no_grad()
    def forward_prefill(self, tokens: torch.Tensor, kv: HybridCache,
                        seq_id: int) -> torch.Tensor:
        return self.forward_prefill_batch([(tokens, seq_id, 0)], kv)[0]
