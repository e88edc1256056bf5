"""Lunulix: a small decoder whose layers run attention and a state-space layer
side by side, with norms on both ends of every sublayer and an input of the
token itself in every layer.

  x = embed[token] * embedding.scale
  layer: x <- x + norm1b(mixer(norm1(x))); x <- x + norm2b(ff(norm2(x)))
         x <- x + side.norm(W_proj(gelu(W_gate x) * e)), e the layer's columns
         of side.embed[token]                            all norms rms norms
  out:   final norm, logits through a head of its own

The residual stream is f32.  A sublayer's output enters it through the norm
that ends the sublayer, in the same kernel that computes the norm which
begins the next one (ops.dispatch.residual_norm with `post`); the token's
input reads the stream itself, so there the kernel hands it on unnormed.

The layer list comes from config.json ('layers', each with 'type', 'mixer'
sizes and 'mlp', null for none); the mixers are models/mixers.py.
"""

from __future__ import annotations

import math
from dataclasses import dataclass

import torch

from ..ops import dispatch as D
from .decoder import MixerDecoder, check_layers, number_runs
from .kv_cache import HybridCache
from .layers import DenseGLU, Linear, StepPlan, TokenSide
from .mixers import MIXERS


@dataclass
class LunulixConfig:
    layers: list[dict]
    vocab_size: int
    hidden: int
    side_dim: int
    embed_scale: float = 1.0
    norm_eps: float = 1e-5
    name: str = "lunulix"
    max_pos: int = 1 << 20       # nothing in the design bounds positions

    def __post_init__(self):
        check_layers(self.layers)

    @classmethod
    def from_dict(cls, d: dict, name: str = "lunulix") -> "LunulixConfig":
        return cls(layers=d["layers"], vocab_size=d["vocab"],
                   hidden=d["width"], side_dim=d["token_side"]["dim"],
                   embed_scale=float(d["embedding"]["scale"]),
                   norm_eps=d["norm"]["eps"], name=name)

    def to_dict(self) -> dict:
        return {"architecture": "Lunulix", "vocab": self.vocab_size,
                "width": self.hidden, "norm": {"eps": self.norm_eps},
                "embedding": {"scale": self.embed_scale},
                "token_side": {"dim": self.side_dim}, "layers": self.layers}

    @classmethod
    def preset(cls, name: str) -> "LunulixConfig":
        def layers(n, ff, left, right):
            heads, kv, dim, base = left
            sh, vdim, state, groups = right
            return [{"type": "parallel", "mlp": {"kind": "dense", "ff": ff},
                     "mixer": {
                         "left": {"heads": heads, "kv_heads": kv, "dim": dim,
                                  "vdim": dim, "conv": 4,
                                  "scale": dim ** -0.5,
                                  "rot": {"dims": dim, "base": base,
                                          "scaling": {"factor": 8.0,
                                                      "low": 1.0, "high": 4.0,
                                                      "original": 8192}}},
                         "left_scale": 0.7,
                         "right": {"heads": sh, "vdim": vdim, "state": state,
                                   "groups": groups, "conv": 4,
                                   "norm_groups": groups},
                         "right_scale": 0.7}} for _ in range(n)]

        def make(vocab, width, n, ff, left, right, side):
            return cls(layers=layers(n, ff, left, right), vocab_size=vocab,
                       hidden=width, side_dim=side, norm_eps=1e-6,
                       embed_scale=width ** 0.5, name=name)

        if name == "tiny-lunulix":
            return make(2048, 192, 3, 320, (6, 2, 32, 1e4), (5, 24, 40, 1),
                        24)
        if name == "lunulix-1b":
            return make(128_256, 2048, 12, 6144, (16, 4, 128, 5e5),
                        (32, 64, 128, 4), 128)
        if name == "lunulix-8b":
            return make(128_256, 4096, 28, 14_336, (32, 8, 128, 5e5),
                        (64, 64, 128, 8), 256)
        raise ValueError(f"unknown preset {name}")


def tensor_shapes(c: LunulixConfig) -> dict[str, tuple[int, ...]]:
    """Every tensor of a checkpoint, in storage order."""
    w, s = c.hidden, c.side_dim
    out: dict[str, tuple[int, ...]] = {
        "embed": (c.vocab_size, w),
        "side.embed": (c.vocab_size, len(c.layers) * s)}
    for i, L in enumerate(c.layers):
        p = f"l{i}."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b")
                                        if L.get("mlp") else ()):
            out[p + n] = (w,)
        for k, shape in MIXERS[L["type"]].shapes(L["mixer"], w).items():
            out[p + "mix." + k] = shape
        if L.get("mlp"):
            ff = L["mlp"]["ff"]
            out[p + "mlp.gate"] = (ff, w)
            out[p + "mlp.up"] = (ff, w)
            out[p + "mlp.down"] = (w, ff)
        out[p + "side.gate"] = (s, w)
        out[p + "side.proj"] = (w, s)
        out[p + "side.norm"] = (w,)
    out["final.norm"] = (w,)
    out["head"] = (c.vocab_size, w)
    return out


def random_weights(c: LunulixConfig, device: str, dtype: torch.dtype,
                   seed: int):
    """name -> tensor, generated on the device one at a time (the same
    stream on every rank).  Step sizes start between 0.001 and 0.1, decay
    rates between 1 and 16."""
    dev = device if str(device).startswith("cuda") else "cpu"
    g = torch.Generator(device=dev).manual_seed(seed)
    for name, shape in tensor_shapes(c).items():
        leaf = name.rsplit(".", 1)[-1]
        if leaf == "A_log":
            t = torch.log(1 + 15 * torch.rand(shape, generator=g, device=dev))
        elif leaf == "dt_bias":
            t = torch.exp(math.log(1e-3) + math.log(100.0)
                          * torch.rand(shape, generator=g, device=dev))
            t = t + torch.log(-torch.expm1(-t))      # softplus(bias) = step
        elif leaf in ("sink", "b"):
            t = torch.zeros(shape, device=dev)
        elif leaf == "conv":
            t = torch.randn(shape, generator=g, device=dev) \
                * shape[1] ** -0.5
        elif len(shape) == 1:
            t = torch.ones(shape, device=dev)
        else:
            t = torch.randn(shape, generator=g, device=dev) * 0.02
        yield name, t.to(device=device, dtype=dtype)


def layer_runs(c: LunulixConfig):
    return number_runs(c.layers, [(i, None) for i in range(len(c.layers))])


@dataclass
class _Layer:
    norm1: torch.Tensor
    mixer: object
    norm1b: torch.Tensor
    side: TokenSide
    side_norm: torch.Tensor
    norm2: torch.Tensor | None = None
    ff: DenseGLU | None = None
    norm2b: torch.Tensor | None = None


class LunulixModel(MixerDecoder):
    Config = LunulixConfig
    shapes = staticmethod(tensor_shapes)
    random = staticmethod(random_weights)
    layer_runs = staticmethod(layer_runs)

    def build(self, get) -> None:
        cfg, shard = self.cfg, self.shard
        self.embed, table = get("embed"), get("side.embed")
        self.head = Linear(get("head"))
        self.final = get("final.norm")
        self.layers = []
        for i, L in enumerate(cfg.layers):
            p = f"l{i}."
            layer = _Layer(
                get(p + "norm1"),
                MIXERS[L["type"]](L["mixer"], cfg.norm_eps,
                                  lambda k, p=p: get(p + "mix." + k), shard,
                                  self._rope, self.dtype),
                get(p + "norm1b"),
                TokenSide(get(p + "side.gate"), get(p + "side.proj"), table,
                          i), get(p + "side.norm"))
            if L.get("mlp"):
                layer.norm2 = get(p + "norm2")
                layer.ff = DenseGLU(shard.rows(get(p + "mlp.gate")),
                                    shard.rows(get(p + "mlp.up")),
                                    shard.cols(get(p + "mlp.down")), "gelu")
                layer.norm2b = get(p + "norm2b")
            self.layers.append(layer)

    def _forward(self, plan: StepPlan, kv: HybridCache,
                 rows: torch.Tensor | None,
                 trail: list | None = None) -> torch.Tensor:
        eps, ids = self.cfg.norm_eps, plan.tokens
        res = torch.empty(plan.n_rows, self.cfg.hidden, dtype=torch.float32,
                          device=self.device)
        y = post = None
        for r in self.runs:
            L = self.layers[r.layer]
            first = y is None
            h = D.residual_norm(res, y, L.norm1, None, eps, layer=False,
                                post=post, init=first,
                                table=self.embed if first else None,
                                ids=ids if first else None,
                                tscale=self.cfg.embed_scale)
            y, post = self._reduce(L.mixer(h, plan, kv, r.cache)), L.norm1b
            if L.ff is not None:
                h = D.residual_norm(res, y, L.norm2, None, eps, layer=False,
                                    post=post)
                y, post = self._reduce(L.ff(h)), L.norm2b
            x = D.residual_norm(res, y, None, None, eps, post=post)
            y, post = L.side(x, ids), L.side_norm
            if trail is not None:
                e = y.float()
                trail.append(res + e * torch.rsqrt(
                    e.pow(2).mean(-1, keepdim=True) + eps) * post.float())
        if rows is not None:
            res, y = res.index_select(0, rows), y.index_select(0, rows)
        return self.head(D.residual_norm(res, y, self.final, None, eps,
                                         layer=False, post=post))
