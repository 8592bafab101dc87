"""Feed-forwards W_down act(W_up h) and W_down unit(W_gate h, W_up h), the activation in the epilogue of the first projection."""
from __future__ import annotations

import torch
import torch.nn.functional as F
from torch import nn

from nanovllm import hip_ops
from nanovllm.distributed.parallel_state import get_tp_group
from nanovllm.layers.linear import PaddedLinear


def xielu_constants(p: torch.Tensor) -> tuple:
    """Epilogue constants of xIELU from its two learned numbers: quadratic coefficient softplus(p) for z > 0, exponential
    coefficient 1/2 + softplus(q) for z <= 0 (evaluated in fp32)."""
    v = p.detach().to(device="cpu", dtype=torch.float32)
    return (hip_ops.ACT_XIELU, float(F.softplus(v[0])), float(0.5 + F.softplus(v[1])))


class DenseMLP(nn.Module):

    def __init__(self, width: int, ff: int, dtype):
        super().__init__()
        tp = get_tp_group()
        if ff % tp.world_size:
            raise ValueError(f"a feed-forward of {ff} does not split over {tp.world_size} ranks")
        self.tp_size, self.tp_rank, self.ff = tp.world_size, tp.rank, ff // tp.world_size
        self.up = PaddedLinear(width, [hip_ops.round8(self.ff)], dtype)
        self.down = PaddedLinear(self.ff, [hip_ops.round8(width)], dtype)
        self.act = hip_ops.NO_ACT

    def load(self, w: dict, device) -> None:
        """w: up, down, act."""
        lo = self.tp_rank * self.ff
        self.up.load([w["up"][lo: lo + self.ff]], device)
        self.down.load([w["down"][:, lo: lo + self.ff]], device)
        self.act = xielu_constants(w["act"])

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        y = self.down(self.up(h, act=self.act))
        if self.tp_size > 1:
            get_tp_group().all_reduce(y)
        return y


class GatedMLP(nn.Module):
    """Clamped gated unit: g sigmoid(slope g) (u + 1) with g = min(gate, limit), u = up within +-limit."""

    def __init__(self, width: int, ff: int, limit: float, dtype):
        super().__init__()
        tp = get_tp_group()
        if ff % tp.world_size:
            raise ValueError(f"a feed-forward of {ff} does not split over {tp.world_size} ranks")
        self.tp_size, self.tp_rank, self.ff, self.limit = tp.world_size, tp.rank, ff // tp.world_size, limit
        self.gate_up = PaddedLinear(width, [hip_ops.round8(self.ff)] * 2, dtype)
        self.down = PaddedLinear(self.ff, [hip_ops.round8(width)], dtype)

    def load(self, w: dict, device) -> None:
        """w: gate, up, down."""
        lo = self.tp_rank * self.ff
        self.gate_up.load([w["gate"][lo: lo + self.ff], w["up"][lo: lo + self.ff]], device)
        self.down.load([w["down"][:, lo: lo + self.ff]], device)

    def forward(self, h: torch.Tensor) -> torch.Tensor:
        y = self.down(hip_ops.gated_glu(h, self.gate_up.weight, self.limit))
        if self.tp_size > 1:
            get_tp_group().all_reduce(y)
        return y
