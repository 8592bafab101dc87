"""Shared pieces of the Napadra tests: small configurations of deliberately odd sizes and random models."""
import copy

import torch

from dafolorn_util import distance, run_cut, session, tokens  # noqa: F401
from oracle import napadra_oracle as O


def _mlp(ff, limit):
    return None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}


def attn(heads, kv_heads, dim, vdim, chunk, ff=None, limit=2.0, scale=None, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk}, "scale": scale if scale is not None else dim ** -0.5}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": _mlp(ff, limit)}


def mlstm(heads, dim, vdim, ff=None, limit=2.0, cap=9.0):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": _mlp(ff, limit)}


def config(width, vocab, streams, layers, mult=0.5, eps=1e-5):
    return {"architecture": "Napadra", "width": width, "vocab": vocab, "streams": streams, "layers": layers, "residual_mult": mult, "norm": {"eps": eps}}


CONFIGS = {
    # nothing a multiple of 8; a borrowed cache with a longer chunk than its owner's; one layer of each mixer with and without feed-forward
    "odd": config(76, 203, 3, [attn(5, 5, 20, 12, 33, 100), mlstm(3, 20, 44), attn(5, 5, 20, 12, 150, None, kv_from=0), mlstm(2, 36, 28, 60, 0.7, 4.0)], 0.4),
    # one stream, sixteen heads on one key/value head, chunks of one token, several value tiles, a scale that is not dim^-1/2
    "wide": config(136, 320, 1, [mlstm(2, 72, 136, 72), attn(16, 1, 136, 200, 1, 264, 0.5, 0.02), attn(16, 1, 136, 200, 65, None, scale=0.05)], 1.0, 1e-3),
    # four streams, twenty heads per key/value head (two row groups), tiny heads, chunks longer than most portions
    "tall": config(64, 128, 4, [attn(40, 2, 8, 16, 300, 128, 5.0), attn(9, 3, 16, 8, 24, 40), mlstm(5, 136, 72, None)], 0.3),
    # heads beyond the tiled kernels: keys of 264 in both mixers, values of 328
    "huge": config(72, 64, 2, [attn(2, 1, 264, 24, 40, 48, scale=0.05), mlstm(2, 264, 24, 48), attn(1, 1, 16, 328, 77, None), mlstm(1, 64, 328, None)], 0.5),
    # no attention at all, many streams (no kernel of their own)
    "memory": config(200, 96, 7, [mlstm(4, 32, 64, 136), mlstm(6, 8, 8, None, cap=15.0)], 0.2),
}


def make_model(path, name_or_cfg, seed=0):
    cfg = copy.deepcopy(CONFIGS[name_or_cfg]) if isinstance(name_or_cfg, str) else name_or_cfg
    t = O.random_tensors(cfg, seed)
    O.write_model(str(path), cfg, t)
    return cfg, t


LIMIT = {"float32": 2e-5, "bfloat16": 4e-2}


def errors(got, want, scale):
    """Per position: rms of the difference over the vocabulary, relative to `scale`."""
    return (got.double() - want.double()).pow(2).mean(-1).sqrt() / scale


class Reference:
    """Plain evaluation of one sequence, with the limit of every position: in fp32 a constant; in bf16 at least a constant, more where
    disturbing the projections by their rounding moves the logits further (a memory that holds almost nothing yet, divided by its own
    norm, amplifies whatever is in it)."""

    def __init__(self, cfg, t, toks):
        self.logits = O.forward(cfg, t, toks)
        self.scale = float(self.logits.pow(2).mean().sqrt())
        moved = torch.stack([errors(O.forward(cfg, t, toks, noise=i), self.logits, self.scale) for i in range(3)]).amax(0)
        self.limit = {"float32": torch.full_like(moved, LIMIT["float32"]), "bfloat16": torch.clamp(4 * moved, min=LIMIT["bfloat16"])}

    def check(self, got, dtype, what=None):
        n = got.shape[0]
        e = errors(got, self.logits[:n], self.scale) / self.limit[dtype][:n]
        assert float(e.max()) < 1, (what, int(e.argmax()), float(e.max()), float(self.limit[dtype][int(e.argmax())]))

    def check_one(self, got, pos, dtype):
        e = float(errors(got[None], self.logits[pos: pos + 1], self.scale)[0] / self.limit[dtype][pos])
        assert e < 1, (pos, e)
