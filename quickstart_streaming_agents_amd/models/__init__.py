"""Model registry: preset names and checkpoint folders -> decoder instances.

Decoder families: Llama (Llama-3-8B is the flagship agent LLM, the Qwen2
geometry shares its class), Mixtral MoE, and the config-driven mixer decoders:
Luzalorn (retention and latent-attention layers) and Lunulix (attention and a
state-space layer side by side).

`build_model(name)` takes a preset name (random weights) or a folder with
config.json + model.safetensors; a folder's class is chosen by the
'architecture' its config.json names (ARCHITECTURES).
"""

from __future__ import annotations

import json
import os


def _luzalorn():
    from .luzalorn import LuzalornModel
    return LuzalornModel


def _lunulix():
    from .lunulix import LunulixModel
    return LunulixModel


# config.json 'architecture' -> loader of the model class; a preset of the
# family is named after it ("luzalorn-8b", "tiny-lunulix")
ARCHITECTURES = {"Luzalorn": _luzalorn, "Lunulix": _lunulix}


def load_model(folder: str, device: str = "cuda", dtype=None, **kw):
    """A model with the weights of `folder`."""
    with open(os.path.join(folder, "config.json"), encoding="utf-8") as fh:
        config = json.load(fh)
    arch = config.get("architecture")
    if arch not in ARCHITECTURES:
        raise ValueError(f"{folder}: unknown architecture {arch!r} "
                         f"(known: {', '.join(sorted(ARCHITECTURES))})")
    return ARCHITECTURES[arch]().from_folder(
        folder, config, device=device, dtype=dtype or _dtype(device), **kw)


def _dtype(device):
    import torch
    return torch.bfloat16 if str(device).startswith("cuda") \
        else torch.float32


def build_model(name: str, device: str = "cuda", dtype=None, seed: int = 0,
                tp_rank: int = 0, tp_size: int = 1, tp_group=None,
                ep_size: int | None = None):
    dtype = dtype or _dtype(device)
    tp = dict(tp_rank=tp_rank, tp_size=tp_size, tp_group=tp_group)
    if os.path.isfile(os.path.join(name, "config.json")):
        return load_model(name, device=device, dtype=dtype, **tp)
    for arch, cls in ARCHITECTURES.items():
        if arch.lower() in name.split("-"):
            model = cls()
            return model(model.Config.preset(name), device=device,
                         dtype=dtype, seed=seed, **tp)
    if name.startswith("mixtral") or name == "tiny-moe":
        from .mixtral import MixtralConfig, MixtralModel
        return MixtralModel(MixtralConfig.preset(name), device=device,
                            dtype=dtype, seed=seed, ep_size=ep_size, **tp)
    from .llama import LlamaConfig, LlamaModel
    return LlamaModel(LlamaConfig.preset(name), device=device, dtype=dtype,
                      seed=seed, **tp)
