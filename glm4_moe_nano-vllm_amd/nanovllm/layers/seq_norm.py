"""Norms around a sublayer and the causal convolution on what it reads (csrc/seq_norm.hip).

A sublayer computes x <- x + rms(f(h)) * g_post with h = n + conv(n), n = rms(x) * g_pre.  The closing norm of one sublayer and
the opening norm + convolution of the next are one launch; `SublayerEntry.forward` is that launch."""
from __future__ import annotations

import torch
from torch import nn

from nanovllm import hip_ops


def norm_gain(w: torch.Tensor, size: int, device, zero_centred: bool = True) -> torch.Tensor:
    """fp32 gain of an RMS norm, padded with zeros; zero_centred: the stored weight is the deviation from one."""
    g = torch.zeros(size, dtype=torch.float32, device=device)
    g[: w.numel()] = w.to(device=device, dtype=torch.float32) + (1.0 if zero_centred else 0.0)
    return g


class SublayerEntry(nn.Module):
    """Everything between the end of one sublayer and the input of the next.  `runs`: how often the sublayer runs in a step
    with the same weights — every run keeps its own convolution state."""

    def __init__(self, width: int, taps: int, eps: float, runs: int = 1):
        super().__init__()
        self.width, self.wp, self.eps = width, hip_ops.round8(width), eps
        self.taps = hip_ops.seq_norm_taps(taps)
        self.runs = runs
        self.g_pre = self.conv_w = None
        self.state: list = [None] * runs

    def load(self, norm_w: torch.Tensor, conv_w: torch.Tensor, device) -> None:
        self.g_pre = norm_gain(norm_w, self.wp, device)
        assert conv_w.shape[0] == self.width and conv_w.shape[1] <= self.taps
        w = torch.zeros(self.taps, self.wp, dtype=torch.bfloat16, device=device)
        w[self.taps - conv_w.shape[1]:, : self.width] = conv_w.to(device=device, dtype=torch.bfloat16).t()
        self.conv_w = w

    def state_bytes(self) -> int:
        """Bytes per state row set (a sequence holds two: one read, one written by a step)."""
        return self.runs * (self.taps - 1) * self.wp * 4

    def allocate_state(self, rows: int, device) -> None:
        self.state = [torch.empty(rows, self.taps - 1, self.wp, dtype=torch.float32, device=device) for _ in range(self.runs)]

    def forward(self, x, y, g_post, meta, run: int, act_dtype):
        return hip_ops.seq_norm(x, self.width, self.eps, y=y, g_post=g_post, g_pre=self.g_pre, conv=(self.conv_w, self.state[run]),
                                meta=meta, act_dtype=act_dtype)
