"""Gated matrix memory (mLSTM) as a mixer: one projection for queries, keys, values and output gate, the recurrence over a state per
sequence, the output projection (csrc/matrix_memory.hip).

Short portions (decoded tokens above all) go token by token with the state in registers, long ones 64 tokens at a time on the matrix
cores; fp32 always goes token by token.  The step's batch says which rows are which (StepBatch.Ta)."""
from __future__ import annotations

import torch
from torch import nn

from nanovllm import hip_ops
from nanovllm.distributed.parallel_state import get_tp_group
from nanovllm.layers.linear import PaddedLinear


class MatrixMemory(nn.Module):

    def __init__(self, width: int, heads: int, dim: int, vdim: int, gate_cap: float, eps: float, dtype):
        super().__init__()
        tp = get_tp_group()
        if heads % tp.world_size:
            raise ValueError(f"{heads} heads do not split over {tp.world_size} ranks")
        self.tp_size, self.tp_rank, self.heads = tp.world_size, tp.rank, heads // tp.world_size
        self.dim, self.vdim, self.cap, self.eps, self.dtype = dim, vdim, gate_cap, eps, dtype
        self.dimp, self.vdimp, self.wp = hip_ops.round8(dim), hip_ops.round8(vdim), hip_ops.round8(width)
        H = self.heads
        self.in_proj = PaddedLinear(width, [self.dimp] * (2 * H) + [self.vdimp] * (2 * H), dtype)
        self.gates = PaddedLinear(width, [hip_ops.round8(2 * H)], dtype)   # rows i | f; projected where the recurrence needs them
        self.o_proj = PaddedLinear([vdim] * H, [hip_ops.round8(width)], dtype)
        self.chunkwise = dtype == torch.bfloat16 and self.dimp <= hip_ops.MEMORY_CHUNK_MAX_DIM
        self.gate_bias = self.norm = self.state = None

    def load(self, w: dict, device) -> None:
        """w: q, k, v, g, o, norm, i, i.b, f, f.b."""
        H, h0 = self.heads, self.tp_rank * self.heads

        def heads_of(t, size):  # this rank's heads of a head-by-head layout
            return t.view(H * self.tp_size, size, -1)[h0: h0 + H].to(device)

        d, v = self.dim, self.vdim
        self.in_proj.load(list(heads_of(w["q"], d)) + list(heads_of(w["k"], d)) + list(heads_of(w["v"], v)) + list(heads_of(w["g"], v)), device)
        self.gates.load([torch.cat([w["i"][h0: h0 + H], w["f"][h0: h0 + H]])], device)
        self.gate_bias = torch.cat([w["i.b"][h0: h0 + H], w["f.b"][h0: h0 + H]]).to(device=device, dtype=torch.float32)
        norm = torch.zeros(H, self.vdimp, dtype=torch.float32, device=device)
        norm[:, :v] = heads_of(w["norm"], v)[..., 0].to(torch.float32)
        self.norm = norm.reshape(-1)
        self.o_proj.load([w["o"][:, h0 * v: (h0 + H) * v]], device)

    def state_bytes(self) -> int:
        """Bytes per state row (a sequence holds two: one read, one written by a step)."""
        return 4 * self.heads * (self.dimp * self.vdimp + self.dimp + 1)

    def allocate_state(self, rows: int, device) -> None:
        H = self.heads
        self.state = tuple(torch.empty(rows, H, *s, dtype=torch.float32, device=device) for s in ((self.dimp, self.vdimp), (self.dimp,), ()))

    def forward(self, h: torch.Tensor, meta) -> torch.Tensor:
        H, T, Ta, ns = self.heads, h.shape[0], meta.Ta, meta.n_short
        x = self.in_proj(h)
        y = torch.empty((T, H * self.vdimp), dtype=h.dtype, device=h.device)
        gates = (self.gates.weight[: 2 * H], self.gate_bias, self.norm)
        form = (H, self.dim, self.vdim, self.cap, self.eps)
        if not self.chunkwise:
            Ta, ns = T, meta.q_start.numel() - 1
        if Ta:
            hip_ops.memory_recurrent(x[:Ta], h[:Ta], *gates, y[:Ta], self.state, meta.pos, meta.q_start[: ns + 1], meta.state_in, meta.state_out, *form)
        if Ta < T:
            hip_ops.memory_chunkwise(x[Ta:], h[Ta:], *gates, y[Ta:], self.state, meta.pos[Ta:], meta.long_q_start, meta.state_in[ns:], meta.state_out[ns:],
                                     meta.long_tile_seq, meta.long_tile_off, *form)
        y = self.o_proj(y)
        if self.tp_size > 1:
            get_tp_group().all_reduce(y)
        return y
