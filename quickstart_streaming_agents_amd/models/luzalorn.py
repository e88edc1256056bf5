"""Luzalorn: a small decoder that mixes retention layers with windowed latent
attention and may run a stretch of its layers several times.

  x = embed[token]
  layer: x <- x + mixer(norm1(x)); x <- x + ff(norm2(x))    layer norms
  loop:  layers start..stop-1 run `times` times with the same weights; each
         pass has its own cache or state.  Before a pass, loop.step[t] is
         added to x, and from the second pass on also the embedding output.
  out:   final norm, logits through the embedding table

The residual stream is f32.  Its update, the loop's additions and the next
norm are one kernel per half layer (ops.dispatch.residual_norm): a mixer's
or feed-forward's output is added by the norm that follows it.

The layer list comes from config.json ('layers', each with 'type', 'mixer'
sizes and 'mlp'); the mixers are models/mixers.py.
"""

from __future__ import annotations

from dataclasses import dataclass

import torch

from ..ops import dispatch as D
from .decoder import LayerRun, MixerDecoder, check_layers, number_runs
from .kv_cache import HybridCache
from .layers import DenseGLU, Linear, StepPlan
from .mixers import MIXERS


@dataclass
class LuzalornConfig:
    layers: list[dict]
    vocab_size: int
    hidden: int
    norm_eps: float = 1e-5
    loop: dict | None = None
    name: str = "luzalorn"
    max_pos: int = 1 << 20       # nothing in the design bounds positions

    def __post_init__(self):
        n = len(self.layers)
        check_layers(self.layers)
        if self.loop:
            a, b = self.loop["start"], self.loop["stop"]
            if not (0 <= a < b <= n and self.loop["times"] >= 1):
                raise ValueError(f"loop {self.loop} does not fit {n} layers")

    @classmethod
    def from_dict(cls, d: dict, name: str = "luzalorn") -> "LuzalornConfig":
        return cls(layers=d["layers"], vocab_size=d["vocab"],
                   hidden=d["width"], norm_eps=d["norm"]["eps"],
                   loop=d.get("loop"), name=name)

    def to_dict(self) -> dict:
        return {"architecture": "Luzalorn", "vocab": self.vocab_size,
                "width": self.hidden, "norm": {"eps": self.norm_eps},
                "loop": self.loop, "layers": self.layers}

    @classmethod
    def preset(cls, name: str) -> "LuzalornConfig":
        def decays(n):
            return [1.0 - 2.0 ** (-5 - 5 * i / max(n - 1, 1))
                    for i in range(n)]

        def ret(heads, dim, vdim, base=10_000.0):
            return {"type": "retention",
                    "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                              "decay": decays(heads),
                              "rot": {"dims": dim, "base": base}}}

        def lat(heads, dim, vdim, q_rank, kv_rank, window):
            return {"type": "latent_attention",
                    "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                              "q_rank": q_rank, "kv_rank": kv_rank,
                              "scale": dim ** -0.5,
                              "mask": {"size": window}}}

        def stack(pattern, repeat, ff):
            return [dict(L, mlp={"kind": "dense", "ff": ff})
                    for _ in range(repeat) for L in pattern]

        if name == "tiny-luzalorn":
            return cls(layers=stack([ret(3, 32, 48), lat(5, 24, 40, 72, 48,
                                                          100)], 2, 320),
                       vocab_size=2048, hidden=192, name=name,
                       loop={"start": 1, "stop": 3, "times": 2})
        if name == "luzalorn-1b":
            return cls(layers=stack([ret(8, 128, 256)] * 3 +
                                    [lat(16, 128, 128, 768, 256, 2048)],
                                    4, 8192),
                       vocab_size=128_256, hidden=2048, name=name,
                       loop={"start": 4, "stop": 12, "times": 2})
        if name == "luzalorn-8b":
            return cls(layers=stack([ret(16, 128, 256)] * 3 +
                                    [lat(32, 128, 128, 1536, 512, 4096)],
                                    6, 14_336),
                       vocab_size=128_256, hidden=4096, name=name,
                       loop={"start": 8, "stop": 16, "times": 2})
        raise ValueError(f"unknown preset {name}")


def tensor_shapes(c: LuzalornConfig) -> dict[str, tuple[int, ...]]:
    """Every tensor of a checkpoint, in storage order."""
    w = c.hidden
    out: dict[str, tuple[int, ...]] = {"embed": (c.vocab_size, w)}
    if c.loop:
        out["loop.step"] = (c.loop["times"], w)
    for i, L in enumerate(c.layers):
        p = f"l{i}."
        norms = ["norm1"] + (["norm2"] if L.get("mlp") else [])
        for n in norms:
            out[p + n] = (w,)
            out[p + n + ".b"] = (w,)
        for k, s in MIXERS[L["type"]].shapes(L["mixer"], w).items():
            out[p + "mix." + k] = s
        if L.get("mlp"):
            ff = L["mlp"]["ff"]
            out[p + "mlp.gate"] = (ff, w)
            out[p + "mlp.up"] = (ff, w)
            out[p + "mlp.down"] = (w, ff)
    out["final.norm"] = (w,)
    out["final.norm.b"] = (w,)
    return out


def random_weights(c: LuzalornConfig, device: str, dtype: torch.dtype,
                   seed: int):
    """name -> tensor, generated on the device one at a time (the same
    stream on every rank)."""
    dev = device if str(device).startswith("cuda") else "cpu"
    g = torch.Generator(device=dev).manual_seed(seed)
    for name, shape in tensor_shapes(c).items():
        if name.endswith("norm.b") or name.endswith(("norm1.b", "norm2.b")) \
                or name.endswith("sink"):
            t = torch.zeros(shape, device=dev)
        elif len(shape) == 1:
            t = torch.ones(shape, device=dev)
        else:
            t = torch.randn(shape, generator=g, device=dev) * 0.02
        yield name, t.to(device=device, dtype=dtype)


@dataclass
class _Layer:
    norm1: tuple[torch.Tensor, torch.Tensor]
    mixer: object
    norm2: tuple[torch.Tensor, torch.Tensor] | None = None
    ff: DenseGLU | None = None


def layer_runs(c: LuzalornConfig) -> list[LayerRun]:
    n = len(c.layers)
    seq: list[tuple[int, int | None]] = []
    if c.loop:
        a, b = c.loop["start"], c.loop["stop"]
        seq += [(i, None) for i in range(a)]
        for t in range(c.loop["times"]):
            seq += [(i, t if i == a else None) for i in range(a, b)]
        seq += [(i, None) for i in range(b, n)]
    else:
        seq = [(i, None) for i in range(n)]
    return number_runs(c.layers, seq)


class LuzalornModel(MixerDecoder):
    Config = LuzalornConfig
    shapes = staticmethod(tensor_shapes)
    random = staticmethod(random_weights)
    layer_runs = staticmethod(layer_runs)

    def build(self, get) -> None:
        cfg, shard = self.cfg, self.shard
        self.embed = get("embed")
        self.head = Linear(self.embed)
        self.loop_step = get("loop.step") if cfg.loop else None
        self.final = (get("final.norm"), get("final.norm.b"))
        self.layers = []
        for i, L in enumerate(cfg.layers):
            p = f"l{i}."
            layer = _Layer(
                (get(p + "norm1"), get(p + "norm1.b")),
                MIXERS[L["type"]](L["mixer"], cfg.norm_eps,
                                  lambda k, p=p: get(p + "mix." + k), shard,
                                  self._rope, self.dtype))
            if L.get("mlp"):
                layer.norm2 = (get(p + "norm2"), get(p + "norm2.b"))
                layer.ff = DenseGLU(shard.rows(get(p + "mlp.gate")),
                                    shard.rows(get(p + "mlp.up")),
                                    shard.cols(get(p + "mlp.down")))
            self.layers.append(layer)

    # ---- forward -----------------------------------------------------------
    def _forward(self, plan: StepPlan, kv: HybridCache,
                 rows: torch.Tensor | None,
                 trail: list | None = None) -> torch.Tensor:
        eps = self.cfg.norm_eps
        res = torch.empty(plan.n_rows, self.cfg.hidden, dtype=torch.float32,
                          device=self.device)
        y, init = None, True
        for r in self.runs:
            L = self.layers[r.layer]
            embed = init or r.re_embed
            h = D.residual_norm(
                res, y, *L.norm1, eps, init=init,
                table=self.embed if embed else None,
                ids=plan.tokens if embed else None,
                vec=None if r.step is None else self.loop_step[r.step])
            init = False
            y = self._reduce(L.mixer(h, plan, kv, r.cache))
            if L.ff is not None:
                h = D.residual_norm(res, y, *L.norm2, eps)
                y = self._reduce(L.ff(h))
            if trail is not None:
                trail.append(res + y.float())
        if rows is not None:
            res, y = res.index_select(0, rows), y.index_select(0, rows)
        return self.head(D.residual_norm(res, y, *self.final, eps))
