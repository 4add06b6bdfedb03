"""Model architectures the engine serves, by name and by checkpoint.

A checkpoint directory names its architecture in config.json (``architecture``,
or the Hugging Face ``architectures`` / ``model_type``); a bare name is a
random-init configuration of one of the families below.
"""
from __future__ import annotations

import json
from pathlib import Path
from typing import Optional

import torch

from . import dozazen, llama, topelorn

_FAMILIES = {"llama": llama.CONFIGS, "dozazen": dozazen.CONFIGS, "topelorn": topelorn.CONFIGS}
# families on one GPU per replica, with a 32-bit mode on the GPU
_ONE_GPU = {"dozazen": (dozazen.load, dozazen.DozazenModel), "topelorn": (topelorn.load, topelorn.TopelornModel)}
FLOAT32_FAMILIES = tuple(_ONE_GPU)


def architecture_of(path) -> str:
    """The family of the checkpoint directory ``path``."""
    c = json.loads((Path(path) / "config.json").read_text())
    names = [c.get("architecture"), *(c.get("architectures") or ()), c.get("model_type")]
    for n in (str(n).lower() for n in names if n):
        for fam in _FAMILIES:
            if n == fam or n == fam + "forcausallm":
                return fam
    if not any(names):
        return "llama"                     # a config.json of bare Llama sizes
    raise NotImplementedError(f"{path}: architecture {next(n for n in names if n)!r} "
                              f"(served: {', '.join(sorted(_FAMILIES))})")


def load_model(path, device, tp_rank: int = 0, tp: int = 1, tp_group=None, dtype=torch.bfloat16,
               max_pos: Optional[int] = None):
    """The model over a checkpoint directory.  ``dtype`` float32 needs a family
    with a 32-bit mode; ``max_pos`` bounds the position tables."""
    fam = architecture_of(path)
    if fam in _ONE_GPU:
        if tp > 1:
            raise NotImplementedError(f"{fam} runs on one GPU per replica (tp = 1)")
        return _ONE_GPU[fam][0](path, device, dtype=dtype, max_pos=max_pos)
    if dtype != torch.bfloat16 and fam not in FLOAT32_FAMILIES:
        raise NotImplementedError(f"{fam} runs in bfloat16")
    from .weights import llama_from_checkpoint
    return llama_from_checkpoint(path, device, tp_rank, tp, tp_group)


def get_config(name: str):
    for cfgs in _FAMILIES.values():
        if name in cfgs:
            return cfgs[name]
    raise KeyError(f"unknown model config {name!r}; have "
                   f"{sorted(n for cfgs in _FAMILIES.values() for n in cfgs)}")


def random_model(name: str, device, seed: int = 0):
    """A named configuration with random-init weights, one GPU."""
    for fam, (_, model) in _ONE_GPU.items():
        if name in _FAMILIES[fam]:
            return model.random(name, device, seed=seed)
    get_config(name)
    return llama.LlamaModel.random(name, device, seed=seed)
