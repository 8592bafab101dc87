"""Feed-forward of many small gated experts behind a softmax router, without a shared one: sum over a token's `top` experts of score x
W_down (silu(W_gate h) W_up h).

Logits, scores and the weighted sum are fp32; the sum itself belongs to the launch that closes the sublayer (hip_ops.ExpertRows)."""
from __future__ import annotations

import torch
from torch import nn

from nanovllm import hip_ops
from nanovllm.distributed.parallel_state import get_tp_group
from nanovllm.layers.linear import PaddedLinear


class ExpertMLP(nn.Module):

    def __init__(self, width: int, ff: int, experts: int, top: int, dtype):
        super().__init__()
        tp = get_tp_group()
        if ff % tp.world_size:
            raise ValueError(f"experts of {ff} do not split over {tp.world_size} ranks")
        if not 0 < top <= experts:
            raise ValueError(f"{top} of {experts} experts")
        self.tp_size, self.tp_rank, self.ff = tp.world_size, tp.rank, ff // tp.world_size
        self.width, self.wp, self.ffp, self.experts, self.top, self.dtype = width, hip_ops.round8(width), hip_ops.round8(self.ff), experts, top, dtype
        self.router = PaddedLinear(width, [hip_ops.round8(experts)], dtype)
        self.w13 = self.w2 = None      # [experts, gate | up rows, width], [experts, width, ff]

    def load(self, w: dict, device) -> None:
        """w: router; e<i>.gate, e<i>.up, e<i>.down for every expert."""
        lo, f = self.tp_rank * self.ff, self.ff
        self.router.load([w["router"]], device)
        self.w13 = hip_ops.padded_weight(2 * self.ffp, self.wp, self.experts, dtype=self.dtype, device=device)
        self.w2 = hip_ops.padded_weight(self.wp, self.ffp, self.experts, dtype=self.dtype, device=device)
        self.w13.zero_()
        self.w2.zero_()
        for e in range(self.experts):
            self.w13[e, :f, : self.width] = w[f"e{e}.gate"][lo: lo + f].to(device=device, dtype=self.dtype)
            self.w13[e, self.ffp: self.ffp + f, : self.width] = w[f"e{e}.up"][lo: lo + f].to(device=device, dtype=self.dtype)
            self.w2[e, : self.width, :f] = w[f"e{e}.down"][:, lo: lo + f].to(device=device, dtype=self.dtype)

    def forward(self, h: torch.Tensor):
        w, offs, tok, pos = hip_ops.softmax_router_align(self.router(h, out_f32=True), self.experts, self.top)
        act = hip_ops.grouped_swiglu(h, self.w13, offs, tok)
        # (a token's experts are distinct: no group holds more rows than there are tokens)
        y = hip_ops.ExpertRows(hip_ops.grouped_down(act, self.w2, offs, h.shape[0]), pos, w)
        if self.tp_size > 1:
            y = hip_ops.combine_weighted(y)
            get_tp_group().all_reduce(y)
        return y
