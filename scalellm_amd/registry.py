"""Model registry: config.json's "architecture" -> the class that serves it.

A registered class has
    from_checkpoint(config: dict, checkpoint: Checkpoint, limits: ModelLimits) -> step model
and a step model has
    forward(tokens, positions, params: InputParameters, return_logits: bool) -> next ids | logits
    max_positions, vocab, and optionally portion_min (see engine.StepBuilder).
"""
from __future__ import annotations

import importlib
import os
from dataclasses import dataclass
from typing import Dict

import torch

from .checkpoint import Checkpoint, load_config

# modules that register models when imported
_MODULES = ("dagupel",)
_MODELS: Dict[str, type] = {}


@dataclass
class ModelLimits:
    """What the engine sizes a model for."""
    n_blocks: int            # cache blocks of the pool
    block_size: int
    dtype: torch.dtype = torch.bfloat16
    device: str = "cuda"


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
    return cls.from_checkpoint(config, Checkpoint.open(os.path.join(path, "model.safetensors")), limits)
