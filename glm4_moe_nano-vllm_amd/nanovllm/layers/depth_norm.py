"""Sublayers that read the fp32 residual as it is and are closed by an RMS norm in groups, with a short causal convolution on what a
mixer reads and a learned average over the results of all layers so far (csrc/depth_norm.hip).

    x <- x + norm(mixer(x + conv(x)));  x <- x + norm(mlp(x));  what the next layer reads: sum_j a_j X_j

X_0 is the embedding output, X_(i+1) the result of layer i.  The end of one sublayer, the average and the beginning of the next are one
launch."""
from __future__ import annotations

import torch
from torch import nn

from nanovllm import hip_ops
from nanovllm.layers.seq_norm import norm_gain


class CausalTaps(nn.Module):
    """h + conv(h) in front of a mixer: taps and the last inputs of every sequence."""

    def __init__(self, width: int, taps: int):
        super().__init__()
        self.width, self.wp = width, hip_ops.round8(width)
        self.taps = hip_ops.depth_norm_taps(max(taps, 2))
        self.weight = self.state = None

    def load(self, w: torch.Tensor, device) -> None:
        assert w.shape[0] == self.width and w.shape[1] <= self.taps
        t = torch.zeros(self.taps, self.wp, dtype=torch.bfloat16, device=device)
        t[self.taps - w.shape[1]:, : self.width] = w.to(device=device, dtype=torch.bfloat16).t()
        self.weight = t

    def state_bytes(self) -> int:
        """Bytes per state row (a sequence holds two: one read, one written by a step)."""
        return (self.taps - 1) * self.wp * 4

    def allocate_state(self, rows: int, device) -> None:
        self.state = torch.empty(rows, self.taps - 1, self.wp, dtype=torch.float32, device=device)


class DepthResidual(nn.Module):
    """The residual of a step and its planes X_0 .. X_(L-1); every method is one launch."""

    def __init__(self, width: int, layers: int, groups: int, eps: float, dtype):
        super().__init__()
        if width % groups:
            raise ValueError(f"a width of {width} in {groups} groups")
        self.width, self.wp, self.layers, self.groups, self.eps, self.dtype = width, hip_ops.round8(width), layers, groups, eps, dtype
        self.coef: list = [None] * layers        # of the average behind layer i, over X_0 .. X_(i+1)
        self.g_final = None

    def load(self, final: torch.Tensor, coef: list, device) -> None:
        self.g_final = norm_gain(final, self.wp, device, zero_centred=False)
        for i, a in enumerate(coef):
            assert a.numel() == i + 2
            self.coef[i] = a.to(device=device, dtype=torch.float32).contiguous()

    def planes(self, T: int, device) -> torch.Tensor:
        return torch.empty((self.layers, T, self.wp), dtype=torch.float32, device=device)

    def _run(self, x, **kw):
        return hip_ops.depth_norm(x, self.width, self.groups, self.eps, act_dtype=self.dtype, **kw)

    def first(self, planes, taps: CausalTaps, meta):
        """What the first mixer reads."""
        return planes[0], self._run(planes[0], conv=(taps.weight, taps.state), meta=meta)[1]

    def inside(self, x, y, g_post):
        """Behind a mixer, in front of its layer's feed-forward: (residual, its rows in the activation dtype)."""
        out = torch.empty_like(x)
        return out, self._run(x, y=y, g_post=g_post, x_out=out, cast=True)[0]

    def behind(self, i: int, planes, x, y, g_post, taps: CausalTaps, meta):
        """Behind layer i's last sublayer, in front of layer i + 1: (averaged residual, what the next mixer reads)."""
        out = torch.empty_like(x)
        _, h = self._run(x, y=y, g_post=g_post, x_out=planes[i + 1], depth=(planes[: i + 1], self.coef[i]), x_next=out, conv=(taps.weight, taps.state), meta=meta)
        return out, h

    def last(self, planes, x, y, g_post, rows):
        """Behind the last layer: rows of the closing norm."""
        return self._run(x, y=y, g_post=g_post, depth=(planes, self.coef[-1]), g_pre=self.g_final, rows=rows)[1]

    def result(self, i: int, planes, x, y, g_post):
        """What layer i hands on, nothing else."""
        out = torch.empty_like(x)
        self._run(x, y=y, g_post=g_post, depth=(planes[: i + 1], self.coef[i]), x_next=out)
        return out
