"""A layer whose mixer and feed-forward read the same rows and are added up: x <- x + mixer(h) + W_down act(W_up h).

Both sublayers share their two ends, so a layer is two projections however many parts it has: up, queries, keys, values and gates are one
(activations per column in its epilogue), and W_o and W_down are one, over the mixer's output and the unit's side by side in one buffer.
Across ranks that is one all-reduce per layer."""
from __future__ import annotations

import torch
from torch import nn

from nanovllm import hip_ops
from nanovllm.distributed.parallel_state import get_tp_group
from nanovllm.layers.group_attention import GroupAttention
from nanovllm.layers.linear import PaddedLinear

NO_COLUMN = 1 << 24     # behind every column (epilogue constants are floats)
PARTIAL_ROWS = 32       # up to as many rows the output projection leaves its K slices to the next norm
PARTIAL_SLICES = 8
PARTIAL_MIN_K = 4096


class ParallelBlock(nn.Module):

    def __init__(self, width: int, mixer: GroupAttention, ff: int, dtype):
        """mixer: made with joint=True; ff: columns of the feed-forward (square of relu), 0: none."""
        super().__init__()
        tp = get_tp_group()
        if ff % tp.world_size:
            raise ValueError(f"a feed-forward of {ff} does not split over {tp.world_size} ranks")
        self.tp_size, self.tp_rank, self.ff, self.mixer = tp.world_size, tp.rank, ff // tp.world_size, mixer
        self.ffp, self.attp, self.wp = hip_ops.round8(self.ff), mixer.heads * mixer.vdimp, hip_ops.round8(width)
        self.in_proj = PaddedLinear(width, ([self.ffp] if ff else []) + mixer.in_sizes, dtype)
        self.out_proj = PaddedLinear(mixer.out_sizes + ([self.ff] if ff else []), [self.wp], dtype)
        gates = self.ffp + mixer.g_off if mixer.gate else NO_COLUMN
        self.act = (hip_ops.ACT_RELU2_GATE, float(self.ffp), float(gates)) if ff or mixer.gate else hip_ops.NO_ACT

    def load(self, mix: dict, mlp: dict, device) -> None:
        """mix: the mixer's tensors; mlp: up, down."""
        lo, hi = self.tp_rank * self.ff, (self.tp_rank + 1) * self.ff
        self.mixer.load_small(mix, device)
        self.in_proj.load(([mlp["up"][lo: hi]] if self.ff else []) + self.mixer.in_blocks(mix, device), device)
        o = self.mixer.out_block(mix)
        self.out_proj.load([torch.cat([o, mlp["down"][:, lo: hi].to(o.device)], 1) if self.ff else o], device)

    def slices(self, T: int) -> int:
        """K slices of the output projection, summed up by the next norm (few rows, or few output tiles; not across ranks)."""
        if self.tp_size > 1 or T == 1 or self.out_proj.K < PARTIAL_MIN_K:
            return 1
        return PARTIAL_SLICES if T <= PARTIAL_ROWS else hip_ops.gemm_slices(T, self.wp, self.out_proj.K)

    def forward(self, h: torch.Tensor, meta, run: int = 0, cs: torch.Tensor | None = None):
        """What the layer adds to the residual, [T, wp] (or its K-slice partial sums)."""
        T, n = h.shape[0], self.attp + self.ffp
        rows = torch.empty((T, self.attp + self.in_proj.N), dtype=h.dtype, device=h.device)   # mixer's output | unit | queries, keys, values, gates
        self.in_proj(h, act=self.act, out=rows[:, self.attp:])
        self.mixer.attend(rows[:, n:], rows[:, : self.attp], meta, run=run, cs=cs)
        slices = self.slices(T) if h.dtype == torch.bfloat16 else 1
        if slices > 1:
            return hip_ops.gemm_bf16_partial(rows[:, :n], self.out_proj.weight, slices)
        y = self.out_proj(rows[:, :n])
        if self.tp_size > 1:
            get_tp_group().all_reduce(y)
        return y
