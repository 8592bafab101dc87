"""Sublayers around a residual of several parallel streams (csrc/stream_norm.hip).

A sublayer reads u = sum_s in[s] x_s through an RMS norm with one gain (and, for a mixer, a token shift) and, when it is finished,
x_t <- sum_s mix[s, t] x_s + mult out[t] (scale . y).  The end of one sublayer and the beginning of the next are one launch;
`StreamSublayer.enter` is that launch."""
from __future__ import annotations

import torch
from torch import nn

from nanovllm import hip_ops


def _vector(w: torch.Tensor, size: int, device) -> torch.Tensor:
    v = torch.zeros(size, dtype=torch.float32, device=device)
    v[: w.numel()] = w.reshape(-1).to(device=device, dtype=torch.float32)
    return v


class StreamSublayer(nn.Module):

    def __init__(self, width: int, streams: int, eps: float, residual_mult: float, shifted: bool):
        super().__init__()
        self.width, self.wp, self.streams, self.eps, self.mult, self.shifted = width, hip_ops.round8(width), streams, eps, residual_mult, shifted
        self.gain = 1.0
        self.w_in = self.mix_out = self.y_scale = self.shift = self.state = None

    def load(self, norm: torch.Tensor, scale: torch.Tensor, hc_in: torch.Tensor, hc_out: torch.Tensor, hc_mix: torch.Tensor, shift: torch.Tensor | None,
             device) -> None:
        S = self.streams
        assert hc_mix.shape == (S, S) and hc_in.numel() == hc_out.numel() == S and scale.numel() == self.width and (shift is not None) is self.shifted
        self.gain = float(norm.float())
        self.w_in = _vector(hc_in, S, device)
        self.mix_out = torch.cat([_vector(hc_mix, S * S, device), self.mult * _vector(hc_out, S, device)])
        self.y_scale = _vector(scale, self.wp, device)
        if shift is not None:
            assert shift.numel() == self.width
            self.shift = _vector(shift, self.wp, device)

    def state_bytes(self) -> int:
        """Bytes per state row (a sequence holds two: one read, one written by a step)."""
        return self.wp * 4 if self.shifted else 0

    def allocate_state(self, rows: int, device) -> None:
        if self.shifted:
            self.state = torch.empty(rows, self.wp, dtype=torch.float32, device=device)

    def enter(self, x, finished: "StreamSublayer | None", y, meta, act_dtype):
        """x: streams in front of the sublayer `finished` whose output is y (None: nothing is outstanding).  Returns the streams
        behind it and what this sublayer reads."""
        f = finished
        return hip_ops.stream_norm(x, self.streams, self.width, self.eps, y=y, y_scale=f.y_scale if f else None, mix_out=f.mix_out if f else None, w_in=self.w_in,
                                   gain=self.gain, shift=self.shift, state=self.state, meta=meta, act_dtype=act_dtype)

    def leave(self, x, y):
        """The streams behind this sublayer."""
        return hip_ops.stream_norm(x, self.streams, self.width, self.eps, y=y, y_scale=self.y_scale, mix_out=self.mix_out)[0]


class StreamHead(nn.Module):
    """Sum of the streams and the closing norm, on the rows that are asked for."""

    def __init__(self, width: int, streams: int, eps: float):
        super().__init__()
        self.width, self.streams, self.eps, self.gain, self.ones = width, streams, eps, 1.0, None

    def load(self, norm: torch.Tensor, device) -> None:
        self.gain, self.ones = float(norm.float()), torch.ones(self.streams, dtype=torch.float32, device=device)

    def forward(self, x, finished: StreamSublayer | None, y, rows, act_dtype):
        f = finished
        return hip_ops.stream_norm(x, self.streams, self.width, self.eps, y=y, y_scale=f.y_scale if f else None, mix_out=f.mix_out if f else None, w_in=self.ones,
                                   gain=self.gain, rows=rows, act_dtype=act_dtype, keep_x=False)[1]
