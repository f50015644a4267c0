"""Where a model's weights come from: a safetensors file or a seed.

A model asks its source for every tensor by name and shape.  A source checks
the shape against what the configuration says, so a file that does not fit
is refused with the tensor's name instead of failing inside a kernel.
"""
from __future__ import annotations

import json
import math
import os
from typing import Optional, Sequence

import torch

CONFIG_FILE = "config.json"
WEIGHTS_FILE = "model.safetensors"


def read_config(path: str) -> dict:
    with open(os.path.join(path, CONFIG_FILE)) as f:
        return json.load(f)


class CheckpointSource:
    """Tensors of DIR/model.safetensors."""

    def __init__(self, path: str):
        from safetensors import safe_open
        self.path = os.path.join(path, WEIGHTS_FILE)
        self._file = safe_open(self.path, framework="pt", device="cpu")
        self._names = set(self._file.keys())

    def __call__(self, name: str, shape: Sequence[Optional[int]],
                 **_) -> torch.Tensor:
        """The tensor `name`; None in `shape` leaves that size to the file."""
        if name not in self._names:
            raise KeyError(f"{self.path}: no tensor {name}")
        t = self._file.get_tensor(name)
        if len(t.shape) != len(shape) or any(
                want is not None and want != have
                for want, have in zip(shape, t.shape)):
            raise ValueError(f"{self.path}: {name} has shape "
                             f"{tuple(t.shape)}, expected {tuple(shape)}")
        return t


class RandomSource:
    """Seeded random weights.  mean/spread describe vectors; matrices are
    scaled by their input width.  `free` is the size of an open dimension."""

    def __init__(self, seed: int, device: str = "cpu", free: int = 16):
        self.gen = torch.Generator(device=device)
        self.gen.manual_seed(seed)
        self.free = free

    def __call__(self, name, shape, mean=0.0, spread=None):
        shape = [self.free if s is None else s for s in shape]
        if spread is None:
            spread = 1.0 / math.sqrt(shape[-1]) if shape else 1.0
        t = torch.empty(shape, device=self.gen.device, dtype=torch.float32)
        t.normal_(mean, spread, generator=self.gen)
        return t.to(torch.bfloat16)
