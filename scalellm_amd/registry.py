"""Model registry: config.json's "architecture" -> the class that serves it.

A registered class has
    from_checkpoint(config: dict, checkpoint: Checkpoint, limits: ModelLimits) -> step model
and a step model has
    forward(tokens, positions, params: InputParameters, return_logits: bool) -> next ids | logits
    max_positions, vocab, and optionally portion_min (see engine.StepBuilder) and n_states (recurrent state slots: one per
    live sequence, see engine.BlockAllocator).
The class names the kernel libraries it runs on (`libraries`); load_model() compiles those that are not built yet.
"""
from __future__ import annotations

import importlib
import os
from dataclasses import dataclass
from typing import Dict

import torch

from . import build
from .checkpoint import Checkpoint, load_config

# modules that register models when imported
_MODULES = ("dagupel", "vebusun")
_MODELS: Dict[str, type] = {}


@dataclass
class ModelLimits:
    """What the engine sizes a model for."""
    n_blocks: int            # cache blocks of the pool
    block_size: int
    dtype: torch.dtype = torch.bfloat16
    device: str = "cuda"
    n_states: int = 64       # live sequences a recurrent model keeps state for
    max_positions: int = 0   # longest sequence of a model without a limit of its own; 0 = what the pool holds


def register_model(name: str):
    def add(cls):
        if name in _MODELS:
            raise ValueError(f"model {name} is registered twice")
        _MODELS[name] = cls
        return cls
    return add


def model_class(architecture: str) -> type:
    for m in _MODULES:
        importlib.import_module(f"{__package__}.{m}")
    if architecture not in _MODELS:
        raise ValueError(f"unknown architecture {architecture!r}; known: {', '.join(sorted(_MODELS))}")
    return _MODELS[architecture]


def architecture_of(config: dict) -> str:
    arch = config.get("architecture")
    if not isinstance(arch, str):
        raise ValueError("config.json names no architecture")
    return arch


def load_model(path: str, limits: ModelLimits):
    config = load_config(path)
    cls = model_class(architecture_of(config))
    for library in cls.libraries:
        build.ensure(library)
    return cls.from_checkpoint(config, Checkpoint.open(os.path.join(path, "model.safetensors")), limits)
