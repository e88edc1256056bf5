"""Cases shared by the CPU and GPU tests of the Lunulix decoder: small
configurations with random weights, compared with tests/lunulix_oracle.py."""

from __future__ import annotations

import functools

import lunulix_oracle as O
import torch
from mixer_scenarios import (CUTS, TOL, MixerCase, alone, check, greedy_check,
                             portions, row_errors, run_steps,
                             scenario_conversation, scenario_cuts,
                             scenario_generate, scenario_mixed,
                             scenario_reuse)

from quickstart_streaming_agents_amd.models.lunulix import (LunulixConfig,
                                                            LunulixModel,
                                                            tensor_shapes)

__all__ = ["CUTS", "TOL", "alone", "check", "greedy_check", "portions",
           "row_errors", "run_steps", "scenario_conversation",
           "scenario_cuts", "scenario_generate", "scenario_mixed",
           "scenario_reuse"]

STRETCH = {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 64}


def left(heads, kv, dim, vdim, conv, rot, scale, base=10_000.0,
         scaling=None):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
            "conv": conv, "scale": scale,
            "rot": {"dims": rot, "base": base, "scaling": scaling}}


def right(heads, vdim, state, groups, conv, parts):
    return {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
            "conv": conv, "norm_groups": parts}


def par(a, b, ff=None, left_scale=0.8, right_scale=1.3):
    return {"type": "parallel",
            "mixer": {"left": a, "left_scale": left_scale, "right": b,
                      "right_scale": right_scale},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def model(vocab, width, side, *layers, eps=1e-5, scale=3.0):
    return {"architecture": "Lunulix", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "embedding": {"scale": scale},
            "token_side": {"dim": side}, "layers": list(layers)}


CONFIGS = {
    # no size a multiple of 8, a layer without feed-forward, key heads equal
    # to query heads, norm parts that cut through heads
    "odd": model(301, 100, 37,
                 par(left(3, 3, 20, 18, 2, 12, 0.31, 500.0, STRETCH),
                     right(6, 7, 13, 3, 5, 2), 90, 0.4, 1.0),
                 par(left(4, 2, 13, 20, 5, 6, 0.3), right(1, 10, 6, 1, 2, 5)),
                 par(left(2, 1, 6, 30, 1, 6, 0.5), right(4, 4, 20, 4, 3, 1),
                     34, 1.5, 0.2), eps=2e-5),
    # matrix-core sizes that are not powers of two, layers of unlike sizes
    "tiles": model(512, 192, 56,
                   par(left(6, 2, 40, 72, 4, 32, 0.16, 1e5, STRETCH),
                       right(5, 40, 48, 1, 4, 1), 160, 0.6, 0.9),
                   par(left(5, 5, 64, 32, 3, 64, 0.2), right(6, 16, 24, 2, 2,
                                                            3), 224),
                   par(left(4, 1, 96, 128, 2, 24, 0.1, 3e4),
                       right(4, 72, 128, 4, 3, 8), 128), eps=1e-6,
                   scale=0.7),
    # one branch fits its matrix-core form, the other does not
    "uneven": model(130, 72, 40,
                    par(left(6, 3, 16, 24, 4, 8, 0.3),
                        right(3, 12, 10, 1, 4, 1), 50),
                    par(left(3, 1, 18, 10, 4, 4, 0.3, 1e3, STRETCH),
                        right(2, 24, 32, 2, 4, 4), 44)),
    # one of everything: no taps beyond the current token, nothing rotated
    "ones": model(96, 64, 48,
                  par(left(1, 1, 32, 16, 1, 0, 0.2), right(1, 32, 16, 1, 1,
                                                           1), 64, 1.0, 1.0),
                  par(left(1, 1, 16, 32, 2, 2, 0.5), right(1, 8, 8, 1, 2, 1),
                      72, 1.0, 1.0), scale=1.0),
    # wide heads and states, more query heads per key head than one tile has
    "wide": model(200, 256, 40,
                  par(left(17, 1, 256, 136, 4, 128, 0.05, 1e6),
                      right(2, 200, 256, 1, 4, 2), 264)),
}


def make_weights(cfg: LunulixConfig, seed=0, peak=3.0, fast=0.0):
    """bf16-exact random weights: activations of order one, norms, biases
    and sinks away from their neutral values, attention scores peaked, decays
    from slow to fast (`fast` shifts them)."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(shape, generator=g)
        leaf = name.rsplit(".", 1)[-1]
        if leaf == "sink":
            t = t + 1.0
        elif leaf == "A_log":
            t = t * 0.7 + fast
        elif leaf == "dt_bias":
            t = t * 1.5 - 2.0 + fast
        elif leaf in ("D", "b"):
            t = t * 0.5
        elif name in ("embed", "side.embed"):
            pass
        elif len(shape) == 1:
            t = t * 0.2 + 1.0
        elif leaf == "conv":
            t = t * shape[1] ** -0.5
        else:
            t = t * shape[1] ** -0.5
            if leaf == "q":
                t = t * peak
        out[name] = t.to(torch.bfloat16)
    return out


class Case(MixerCase):
    def __init__(self, name, device="cpu", dtype=torch.float32, seed=0,
                 config=None, peak=3.0, fast=0.0):
        d = config or CONFIGS[name]
        cfg = LunulixConfig.from_dict(d)
        super().__init__(d, cfg, LunulixModel,
                         make_weights(cfg, seed, peak, fast), O.forward,
                         device, dtype)
        self._shaken = {}

    def limits(self, want):
        """Where a sublayer's output nearly cancels, the norm at its end blows
        its rounding up: a bf16 row may be off by a little more than what errors
        of the weights as large as bf16's rounding do to it."""
        plain = super().limits(want)
        toks = next((k for k, v in self._oracle.items() if v is want), None)
        if self.dtype != torch.bfloat16 or toks is None:
            return plain
        if toks not in self._shaken:
            err = []
            for seed in range(3):
                g = torch.Generator().manual_seed(seed)
                w = {k: t.double() * (1 + 2 ** -8 * torch.randn(
                    t.shape, generator=g)) for k, t in self.weights.items()}
                err.append(row_errors(self.forward(self.raw, w,
                                                   list(toks))[0], want))
            self._shaken[toks] = torch.stack(err).max(0).values
        return torch.maximum(plain, 2 * self._shaken[toks])


# ---- keys far away ----------------------------------------------------------

def far_case(device, dtype):
    """One layer whose state forgets within a few tokens: a token acts at a
    distance only through attention."""
    return Case(None, device, dtype, peak=6.0, fast=2.5, config=model(
        128, 64, 32, par(left(4, 2, 32, 32, 3, 16, 0.6, 1e4, STRETCH),
                        right(2, 16, 16, 1, 2, 1), 64, 1.0, 0.1)))


@functools.cache
def _far_prompts(spot, n):
    """Two prompts that differ at `spot` only, picked so that the last rows'
    logits differ most, and the oracle's difference there."""
    case = far_case("cpu", torch.float32)
    toks = [t % 5 for t in case.tokens(n, seed=spot)]
    last = {}
    for t in range(5, 37):
        toks[spot] = t
        last[t] = case.oracle(list(toks))[-8:]
    scale = float(torch.stack(list(last.values())).pow(2).mean().sqrt())
    dist, a, b = max((float((last[x] - last[y]).pow(2).mean().sqrt()), x, y)
                     for x in last for y in last if x < y)
    assert dist > 3 * TOL[torch.bfloat16] * scale, dist / scale
    return [toks[:spot] + [t] + toks[spot + 1:] for t in (a, b)], \
        last[a] - last[b], scale


def scenario_far_key(spot, n, device, dtype, cuts):
    """A token far back, at a page's edge, moves the last rows by as much as
    it should."""
    case = far_case(device, dtype)
    prompts, want, scale = _far_prompts(spot, n)
    got = []
    for toks in prompts:
        got.append(run_steps(case, {"a": toks},
                             alone("a", cuts(len(toks))))["a"])
        check(case, got[-1], case.oracle(toks))
    moved = (got[0][-8:] - got[1][-8:]).double()
    assert float((moved - want).pow(2).mean().sqrt()) <= \
        2 * TOL[case.dtype] * scale
