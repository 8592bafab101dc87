"""Linear attention with a constant decay per head as a mixer: one projection for queries, keys, values (through SiLU) and output gate
(through the sigmoid), the recurrence over a state per sequence, one RMS norm over all heads, the output projection
(csrc/matrix_memory.hip).

Short portions (decoded tokens above all) go token by token with the state in registers, long ones 64 tokens at a time on the matrix
cores; fp32 always goes token by token.  The step's batch says which rows are which (StepBatch.Ta)."""
from __future__ import annotations

import torch
from torch import nn

from nanovllm import hip_ops
from nanovllm.layers.linear import PaddedLinear


class LinearAttention(nn.Module):
    """The norm runs over the heads of all ranks, so every rank of a tensor-parallel group holds the whole mixer."""

    def __init__(self, width: int, heads: int, dim: int, vdim: int, decay: list[float], eps: float, dtype):
        super().__init__()
        if len(decay) != heads:
            raise ValueError(f"{len(decay)} decays for {heads} heads")
        self.heads, self.dim, self.vdim, self.eps, self.dtype = heads, dim, vdim, eps, dtype
        self.dimp, self.vdimp = hip_ops.round8(dim), hip_ops.round8(vdim)
        self.powers = torch.tensor([[float(d) ** j for j in range(65)] for d in decay], dtype=torch.float64, device="cpu").to(torch.float32)
        self.in_proj = PaddedLinear(width, [self.dimp] * (2 * heads) + [self.vdimp] * (2 * heads), dtype)
        self.g_off = heads * (2 * self.dimp + self.vdimp)
        self.o_proj = PaddedLinear([vdim] * heads, [hip_ops.round8(width)], dtype)
        self.chunkwise = dtype == torch.bfloat16 and self.dimp <= hip_ops.MEMORY_CHUNK_MAX_DIM
        self.norm = self.decay = self.state = None

    def load(self, w: dict, device) -> None:
        """w: q, k, v, g, norm, o."""
        H, d, v = self.heads, self.dim, self.vdim
        by_head = lambda t, size: list(t.view(H, size, -1))  # noqa: E731
        self.in_proj.load(by_head(w["q"], d) + by_head(w["k"], d) + by_head(w["v"], v) + by_head(w["g"], v), device)
        norm = torch.zeros(H, self.vdimp, dtype=torch.float32, device=device)
        norm[:, :v] = w["norm"].to(device=device, dtype=torch.float32).view(H, v)
        self.norm = norm.reshape(-1)
        self.o_proj.load([w["o"]], device)
        self.powers = self.powers.to(device)
        self.decay = self.powers[:, 1].contiguous()

    def state_bytes(self) -> int:
        """Bytes per state row (a sequence holds two: one read, one written by a step)."""
        return 4 * self.heads * self.dimp * self.vdimp

    def allocate_state(self, rows: int, device) -> None:
        self.state = torch.empty(rows, self.heads, self.dimp, self.vdimp, dtype=torch.float32, device=device)

    def forward(self, h: torch.Tensor, meta) -> torch.Tensor:
        H, T, Ta, ns = self.heads, h.shape[0], meta.Ta, meta.n_short
        x = self.in_proj(h, act=(hip_ops.ACT_SILU_GATE, float(self.g_off), 0.0))
        gate = x[:, self.g_off:]
        y = torch.empty((T, H * self.vdimp), dtype=h.dtype, device=h.device)
        if not self.chunkwise:
            Ta, ns = T, meta.q_start.numel() - 1
        form = (H, self.dimp, self.vdimp)
        if Ta:
            o = hip_ops.linear_recurrent(x[:Ta], self.decay, self.state, meta.pos, meta.q_start[: ns + 1], meta.state_in, meta.state_out, *form)
            hip_ops.row_norm_gate(o, gate[:Ta], self.norm, H * self.vdim, self.eps, y[:Ta])
        if Ta < T:
            o = hip_ops.linear_chunkwise(x[Ta:], self.powers, self.state, meta.pos[Ta:], meta.long_q_start, meta.state_in[ns:], meta.state_out[ns:], *form)
            hip_ops.row_norm_gate(o, gate[Ta:], self.norm, H * self.vdim, self.eps, y[Ta:])
        return self.o_proj(y)
