"""Reading a model folder: config.json and model.safetensors.

A safetensors file is an 8-byte little-endian length, that many bytes of JSON (name -> dtype, shape, data_offsets) and
the data.  The file is mapped, not read: a tensor is copied when its layer takes it.
"""
from __future__ import annotations

import json
import os
import struct
from typing import Dict, Iterable, Optional

import numpy as np
import torch

_DTYPES = {"BF16": torch.bfloat16, "F16": torch.float16, "F32": torch.float32, "I32": torch.int32, "I64": torch.int64}


class CheckpointError(RuntimeError):
    pass


def load_config(path: str) -> dict:
    with open(os.path.join(path, "config.json")) as f:
        return json.load(f)


class Checkpoint:
    """Named tensors of one safetensors file.  take() hands a tensor out and checks its shape; finish() complains
    about tensors nobody took."""

    def __init__(self, tensors: Dict[str, torch.Tensor]):
        self._tensors = tensors
        self._taken = set()

    @staticmethod
    def open(path: str) -> "Checkpoint":
        data = np.memmap(path, dtype=np.uint8, mode="c")   # (copy on write: torch wants writable memory)
        if data.size < 8:
            raise CheckpointError(f"{path}: not a safetensors file")
        n = struct.unpack("<Q", data[:8].tobytes())[0]
        if n > data.size - 8:
            raise CheckpointError(f"{path}: header of {n} bytes in a file of {data.size}")
        header = json.loads(data[8:8 + n].tobytes())
        out = {}
        for name, info in header.items():
            if name == "__metadata__":
                continue
            dtype = _DTYPES.get(info["dtype"])
            if dtype is None:
                raise CheckpointError(f"{name}: dtype {info['dtype']} is not supported")
            a, b = info["data_offsets"]
            count = int(np.prod(info["shape"], dtype=np.int64)) if info["shape"] else 1
            size = torch.empty(0, dtype=dtype).element_size()
            if not 0 <= a <= b <= data.size - 8 - n or b - a != count * size:
                raise CheckpointError(f"{name}: data_offsets do not fit its shape or the file")
            raw = data[8 + n + a:8 + n + b]
            if raw.ctypes.data % size:
                raw = raw.copy()
            out[name] = torch.from_numpy(raw).view(dtype).view(info["shape"]) if count else torch.empty(info["shape"], dtype=dtype)
        return Checkpoint(out)

    def names(self) -> Iterable[str]:
        return self._tensors.keys()

    def take(self, name: str, shape: Optional[tuple] = None) -> torch.Tensor:
        t = self._tensors.get(name)
        if t is None:
            raise CheckpointError(f"weight is not in the checkpoint: {name}")
        if shape is not None and tuple(t.shape) != tuple(shape):
            raise CheckpointError(f"{name}: shape {tuple(t.shape)}, expected {tuple(shape)}")
        self._taken.add(name)
        return t

    def finish(self) -> None:
        left = sorted(set(self._tensors) - self._taken)
        if left:
            raise CheckpointError(f"tensors the model does not use: {', '.join(left[:8])}{' ...' if len(left) > 8 else ''}")
