"""NeoX rotary embedding on the first rotary_dim dims of each head — reference:
layers/rotary_embedding.py:17-71.  The cos/sin table is built on the host with the same torch
ops as the reference (so the table is bit-identical); the rotation is glm_rope_neox.

StepRotation, PairRotary, HalfRotary: rotations of neighbouring columns (with YaRN's scaling) or of columns half the rotated part apart,
for models that run step batches (no counterpart in the reference)."""
from __future__ import annotations

import math
from functools import lru_cache

import torch
from torch import nn

from nanovllm import hip_ops


class RotaryEmbedding(nn.Module):

    def __init__(self, head_size: int, rotary_dim: int, max_position_embeddings: int,
                 base: float) -> None:
        super().__init__()
        self.head_size = head_size
        self.rotary_dim = rotary_dim
        expo = torch.arange(0, rotary_dim, 2, dtype=torch.float) / rotary_dim
        inv_freq = 1.0 / (base ** expo)
        t = torch.arange(max_position_embeddings, dtype=torch.float)
        freqs = torch.outer(t, inv_freq)
        cache = torch.cat((freqs.cos(), freqs.sin()), dim=-1).unsqueeze(1)
        self.register_buffer("cos_sin_cache", cache, persistent=False)

    def forward(self, positions: torch.Tensor, query: torch.Tensor, key: torch.Tensor):
        return hip_ops.rope_neox(positions, query, key, self.cos_sin_cache, self.rotary_dim)


@lru_cache(1)
def get_rope(head_size: int, rotary_dim: int, max_position: int, base: float,
             rope_scaling: dict | None = None, partial_rotary_factor: float = 1.0):
    assert rope_scaling is None
    if partial_rotary_factor < 1.0:
        rotary_dim = int(head_size * partial_rotary_factor)
    return RotaryEmbedding(head_size, rotary_dim, max_position, base)


def yarn_frequencies(base: float, dims: int, factor: float, original: float, fast: float, slow: float) -> list[float]:
    """Frequencies of dims / 2 pairs with YaRN's interpolation: pairs that turn more than `fast` times over the original length keep
    theirs, those that turn less than `slow` times are slowed down by `factor`, with a linear ramp over the pair index between."""
    def pair_of(turns):
        return dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))

    lo, hi = max(math.floor(pair_of(fast)), 0), min(math.ceil(pair_of(slow)), dims - 1)
    width = max(hi - lo, 0.001)
    freq = []
    for i in range(dims // 2):
        f, ramp = base ** (-2.0 * i / dims), min(max((i - lo) / width, 0.0), 1.0)
        freq.append(f / factor * ramp + f * (1.0 - ramp))
    return freq


class StepRotation:
    """A rotation whose table is made on the device from a step's positions, so no length is built in; layers with the same rotation share
    it (`key`).  freq: frequency of every pair that turns; pairs: pairs of the table."""

    def __init__(self, freq: tuple, mscale: float, pairs: int):
        self.freq, self.mscale, self.pairs = freq, mscale, pairs
        self.key = (pairs, freq, mscale)
        self._dev = {}

    def prepare(self, device) -> None:
        """The frequencies on the device (at load time: a captured step only reads them)."""
        if device not in self._dev:
            self._dev[device] = torch.tensor(self.freq, dtype=torch.float64, device="cpu").to(device)

    def table(self, pos: torch.Tensor) -> torch.Tensor:
        """cos, sin [T, pairs, 2] at the positions of a step."""
        return hip_ops.rope_pairs(pos, self._dev[pos.device], self.mscale, self.pairs)

    def shared_table(self, pos: torch.Tensor, tables: dict) -> torch.Tensor:
        """The table of a step, made once for all layers with this rotation (`tables`: of the step)."""
        if self.key not in tables:
            tables[self.key] = self.table(pos)
        return tables[self.key]


class PairRotary(StepRotation):
    """Rotation of the column pairs (2i, 2i+1), i < dims / 2, of a head's rotated part of rot_dim columns (the rest do not turn)."""

    def __init__(self, rot_dim: int, dims: int, base: float, scaling: dict | None = None):
        if dims % 2 or rot_dim % 2 or not 0 < dims <= rot_dim:
            raise ValueError(f"a rotation of {dims} of {rot_dim} columns")
        if scaling is None:
            freq, mscale = tuple(base ** (-2.0 * i / dims) for i in range(dims // 2)), 1.0
        else:
            freq = tuple(yarn_frequencies(base, dims, *(scaling[k] for k in ("factor", "original", "fast", "slow"))))
            mscale = 0.1 * math.log(scaling["factor"]) + 1.0
        super().__init__(freq, mscale, hip_ops.round8(rot_dim) // 2)


class HalfRotary(StepRotation):
    """Rotation of the column pairs (i, i + dims / 2), i < dims / 2, of a head of dim columns (those from dims on do not turn)."""

    def __init__(self, dim: int, dims: int, base: float):
        if dims % 2 or not 0 < dims <= dim:
            raise ValueError(f"a rotation of {dims} of {dim} columns")
        self.dims = dims
        super().__init__(tuple(base ** (-2.0 * i / dims) for i in range(dims // 2)), 1.0, dims // 2)
