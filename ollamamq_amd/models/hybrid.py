"""What the models over a HybridCache share: the source of their weights, the
packed copies that the weight-streaming decode products read, and the tables
of rotary positions.

A layer lists its weight matrices in `matrices()` and finds the packed copy
of each in `packs` (empty on the CPU, in fp32 and where memory is short); so
does a model for matrices that belong to no layer.
"""
from __future__ import annotations

import math
import os
from dataclasses import dataclass
from typing import Dict, Optional, Tuple

import torch

from ..ops import interface as ops
from .checkpoint import CheckpointSource, RandomSource


@dataclass(frozen=True)
class RopeSpec:
    """Rotary positions over the first `dims` dimensions of a head, pair i
    turning by base^(-2i/dims) per token: dimensions (2i, 2i+1), or
    (i, i + dims/2) with `halves`.  scaling = (factor,
    original, fast, slow) is YaRN's: pairs that turn more than `fast` times
    over the original context keep their frequency, those below `slow` have
    it divided by `factor`, a linear ramp over the pairs between, and the
    rotation is scaled by 0.1 ln(factor) + 1."""
    dims: int
    base: float
    scaling: Optional[Tuple[float, float, float, float]] = None
    halves: bool = False

    def __post_init__(self):
        if self.dims < 0 or self.dims % 2:
            raise ValueError(f"{self.dims} rotated dimensions")

    @classmethod
    def from_json(cls, d: dict, halves: bool = False) -> "RopeSpec":
        sc = d.get("scaling")
        return cls(int(d["dims"]), float(d["base"]), sc and tuple(
            float(sc[k]) for k in ("factor", "original", "fast", "slow")),
            halves)

    def frequencies(self) -> torch.Tensor:
        """Angle per token of every pair, float64."""
        n = self.dims
        i = torch.arange(n // 2, dtype=torch.float64)
        f = self.base ** (-2.0 * i / n)
        if self.scaling is None or not n:
            return f
        factor, original, fast, slow = self.scaling

        def pair(turns):
            return n * math.log(original / (2 * math.pi * turns)) \
                / (2 * math.log(self.base))

        lo = max(math.floor(pair(fast)), 0)
        hi = min(math.ceil(pair(slow)), n - 1)
        ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
        return f / factor * ramp + f * (1.0 - ramp)

    @property
    def magnitude(self) -> float:
        return 1.0 if self.scaling is None \
            else 0.1 * math.log(self.scaling[0]) + 1.0


class RopeTables:
    """ops.Rope of a RopeSpec, one table for all layers that share it.
    Angles are taken in float64, the table is fp32."""

    def __init__(self, positions: int, device):
        self.positions, self.device = positions, device
        self._made: Dict[RopeSpec, ops.Rope] = {}

    def __call__(self, spec: RopeSpec) -> ops.Rope:
        if spec not in self._made:
            p = torch.arange(self.positions, dtype=torch.float64,
                             device=self.device)
            a = torch.outer(p, spec.frequencies().to(self.device))
            cs = torch.stack([a.cos(), a.sin()], -1) * spec.magnitude
            self._made[spec] = ops.Rope(cs.flatten(1).float().contiguous(),
                                        spec.dims, spec.halves)
        return self._made[spec]


class HybridLayer:
    """One layer's resident weights."""

    packs: Dict[str, torch.Tensor]

    def matrices(self) -> Dict[str, torch.Tensor]:
        raise NotImplementedError

    def pack(self, name: str, w: torch.Tensor):
        """Packed copy of a matrix."""
        return ops.pack_weight(w)

    @staticmethod
    def fused_rows(mats, put) -> torch.Tensor:
        """Input projections as one matrix; zero rows fill it up to the
        32-row tiles of the packed form."""
        fill = -sum(m.shape[0] for m in mats) % 32
        if fill:
            mats = mats + [torch.zeros(fill, mats[0].shape[1],
                                       dtype=mats[0].dtype,
                                       device=mats[0].device)]
        return put(torch.cat(mats)).contiguous()


class HybridModel:
    """Holds weights only: caches and states live in engine.HybridCache."""

    layers: list
    embed: torch.Tensor           # [vocab, width]
    head: torch.Tensor            # [vocab, width], may be the embedding
    packs: Dict[str, torch.Tensor]

    def __init__(self, cfg, device: str, dtype: torch.dtype, tp_size: int,
                 process_group):
        if tp_size != 1 or process_group is not None:
            raise ValueError(f"{cfg.name}: no tensor parallelism")
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype
        self.tp_rank, self.tp_size, self.group = 0, 1, None
        self.head_pk, self.frag_decode = None, False

    def _source(self, seed: int, fast_init: bool, free: int = 16):
        """Where the tensors come from; see checkpoint.py."""
        if self.cfg.checkpoint:
            return CheckpointSource(self.cfg.checkpoint)
        on_gpu = fast_init and self.device.type == "cuda"
        return RandomSource(seed, "cuda" if on_gpu else "cpu", free)

    def _put(self, t: torch.Tensor) -> torch.Tensor:
        return t.to(device=self.device, dtype=self.dtype)

    def matrices(self) -> Dict[str, torch.Tensor]:
        """Matrices that belong to no layer, besides embedding and head."""
        return {}

    def _pack_weights(self):
        """Packed copies for the weight-streaming decode products.  When
        every layer matrix has one, a decode step keeps its activations in
        the fragment layout those products read (frag_decode)."""
        self.packs = {}
        for layer in self.layers:
            layer.packs = {}
        if self.device.type != "cuda" or self.dtype != torch.bfloat16 \
                or os.environ.get("OLLAMAMQ_NO_PACK") == "1":
            return
        free, _ = torch.cuda.mem_get_info(self.device)
        if self.weight_bytes() > free * 0.45:
            return
        for layer in self.layers:
            layer.packs = {n: layer.pack(n, w)
                           for n, w in layer.matrices().items()}
        self.packs = {n: ops.pack_weight(w)
                      for n, w in self.matrices().items()}
        self.head_pk = ops.pack_weight(self.head)
        self.frag_decode = self.cfg.width % 64 == 0 and all(
            p is not None for owner in (self, *self.layers)
            for p in owner.packs.values())

    def weight_bytes(self) -> int:
        n = self.embed.numel()
        if self.head is not self.embed:
            n += self.head.numel()
        for owner in (self, *self.layers):
            n += sum(w.numel() for w in owner.matrices().values())
        return n * self.embed.element_size()
