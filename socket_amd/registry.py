"""Which model class a configuration names, and how its weights are read.

A model folder holds config.json, whose "architecture" is a key of ARCHITECTURES, and
model.safetensors.  `load_model` is what generate.py and bin/trace_run use.
"""
from __future__ import annotations

import json
import math
import os
from dataclasses import fields
from typing import Callable, Dict

import torch

from . import guselix, morasun
from .checkpoint import Checkpoint
from .hybrid import HybridArgs, HybridTransformer
from .mixers import GatedRecurrence
from .model import ModelArgs, Transformer


def _load_hybrid(config: dict, ckpt: Checkpoint, device, dtype, design) -> HybridTransformer:
    args = design.args_from_config(config, ckpt.shapes)
    with torch.device("meta"):
        model = HybridTransformer(args)
    model = model.to_empty(device=device).cast(device, dtype)
    design.load_tensors(model, ckpt.take, ckpt.ignore)
    return model.eval()


def _load_llama(config: dict, ckpt: Checkpoint, device, dtype) -> Transformer:
    known = {f.name for f in fields(ModelArgs)}
    args = ModelArgs(**{k: v for k, v in config.items() if k in known})
    with torch.device("meta"):
        model = Transformer(args)
    model = model.to_empty(device=device).to(dtype=dtype)
    with torch.no_grad():
        for name, p in list(model.named_parameters()) + list(model.named_buffers()):
            if p is not None:
                src = ckpt.take(name)
                if tuple(src.shape) != tuple(p.shape):
                    raise ValueError(f"tensor {name} has shape {tuple(src.shape)}, expected {tuple(p.shape)}")
                p.copy_(src)
    return model.eval()


# architecture -> loader(config, checkpoint, device, dtype)
ARCHITECTURES: Dict[str, Callable] = {
    "Transformer": _load_llama,      # the Llama-style decoder: config.json holds ModelArgs' fields
    morasun.ARCHITECTURE: lambda config, ckpt, device, dtype: _load_hybrid(config, ckpt, device, dtype, morasun),
    guselix.ARCHITECTURE: lambda config, ckpt, device, dtype: _load_hybrid(config, ckpt, device, dtype, guselix),
}


def needs_full_library(architecture: str) -> bool:
    """False for designs whose kernels are all in libsocket_core.so."""
    return architecture == "Transformer"


def read_config(path: str) -> dict:
    with open(os.path.join(path, "config.json")) as f:
        config = json.load(f)
    if config.get("architecture") not in ARCHITECTURES:
        raise ValueError(f"unknown architecture {config.get('architecture')!r}; known: {sorted(ARCHITECTURES)}")
    return config


@torch.no_grad()
def load_model(path: str, device, dtype=torch.bfloat16) -> Transformer:
    """The model in folder `path` on `device`, its matrices in `dtype`."""
    config = read_config(path)
    if dtype == torch.float32:
        torch.set_float32_matmul_precision("highest")     # (32-bit means 32-bit: no reduced-precision products)
    ckpt = Checkpoint(os.path.join(path, "model.safetensors"))
    model = ARCHITECTURES[config["architecture"]](config, ckpt, torch.device(device), dtype)
    ckpt.finish()
    return model


@torch.no_grad()
def random_model(args: HybridArgs, device, dtype=torch.bfloat16, seed: int = 1234) -> HybridTransformer:
    """A hybrid model with weights ~ N(0, 0.02), norms at one and decays spread over time
    constants of some to some thousand tokens."""
    with torch.device("meta"):
        model = HybridTransformer(args)
    model = model.to_empty(device=device).cast(device, dtype)
    gen = torch.Generator(device=device).manual_seed(seed)
    for m in model.modules():
        for name, p in m._parameters.items():
            if p is None:
                continue
            if name.startswith("norm") or name.endswith("norm"):
                p.fill_(1.0)
            elif name == "dwa":          # mostly the layer's own result
                p.fill_(0.25 / max(p.numel() - 1, 1))
                p[-1] = 0.75
            else:
                p.normal_(mean=0.0, std=0.02, generator=gen)
        if isinstance(m, GatedRecurrence):
            if m.a_log is not None:
                m.a_log.uniform_(0.0, math.log(16.0), generator=gen)
                m.decay_bias.uniform_(-7.0, -2.0, generator=gen)
            if m.conv_w is not None:
                m.conv_w.uniform_(-0.5, 0.5, generator=gen)
    return model.eval()
