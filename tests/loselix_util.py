"""Shared pieces of the Loselix tests: small configurations of deliberately odd sizes, random models, and a reference with limits."""
import copy

import torch

from dafolorn_util import distance, run_cut, session, tokens  # noqa: F401
from gulozen_util import errors
from oracle import loselix_oracle as O


def _layer(kind, heads, kv, dim, vdim, ff, scale, **extra):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5, **extra}
    return {"type": kind, "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def two_maps(heads, kv, dim, vdim, ff=None, dims=4, base=10000.0, diff=0.7, cap=9.0, scale=None):
    return _layer("attention", heads, kv, dim, vdim, ff, scale, rot={"base": base, "dims": dims}, diff=diff, softcap=cap)


def gated(heads, kv, dim, vdim, ff=None, dims=4, base=10000.0, scale=None):
    return _layer("attention_2", heads, kv, dim, vdim, ff, scale, rot={"base": base, "dims": dims})


def sigmoid(heads, kv, dim, ff=None, coef=0.4, every=10, scale=None):
    return _layer("attention_3", heads, kv, dim, dim, ff, scale, q_temp={"coef": coef, "every": every})


def config(width, vocab, layers, loop=None, eps=1e-5):
    return {"architecture": "Loselix", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps},
            "loop": None if loop is None else dict(zip(("start", "stop", "times"), loop))}


CONFIGS = {
    # nothing a multiple of 8, a layer without feed-forward, the loop behind the first layer
    "odd": config(76, 203, [two_maps(4, 2, 20, 12, 100, dims=6), sigmoid(6, 3, 20, None, 0.7, 7), gated(3, 1, 12, 28, 60, dims=12)], (1, 3, 2)),
    # no loop, heads of 136 and 200 columns, scales that are not dim^-1/2, more than one row of a decode tile, whole eights rotated, a large eps
    "wide": config(136, 320, [gated(17, 1, 136, 200, 264, dims=32, scale=0.04), two_maps(2, 2, 72, 136, 72, dims=64, base=500.0, cap=30.0, scale=0.3), sigmoid(2, 1, 136, 40, 0.1, 100, 0.05)],
                   None, 1e-3),
    # many heads (several groups of rows per tile), all layers three times, a head of eight columns that turn whole
    "tall": config(64, 128, [sigmoid(40, 2, 8, 128, 1.5, 3), two_maps(12, 1, 24, 64, 40, dims=16, diff=0.2), gated(24, 8, 8, 72, 56, dims=8, base=100.0)], (0, 3, 3)),
    # heads beyond the tiled kernels: keys of 264, two maps of 136, values of 328; the loop once only
    "huge": config(72, 64, [gated(2, 1, 264, 24, 48, dims=2, scale=0.05), two_maps(2, 1, 136, 24, None, dims=136, cap=50.0), sigmoid(2, 2, 264, 24, 0.3, 50, 0.03), gated(1, 1, 16, 328, 40)],
                   (1, 2, 1)),
    # the loop up to the last layer; a temperature that grows at every position, equal sizes everywhere, no feed-forward at all
    "tail": config(200, 96, [two_maps(4, 4, 32, 64, None, dims=32, diff=0.0), sigmoid(8, 2, 64, None, 0.25, 1), gated(8, 4, 64, 64, None, dims=48)], (1, 3, 2)),
}


def make_model(path, name_or_cfg, seed=0):
    cfg = copy.deepcopy(CONFIGS[name_or_cfg]) if isinstance(name_or_cfg, str) else name_or_cfg
    t = O.random_tensors(cfg, seed)
    O.write_model(str(path), cfg, t)
    return cfg, t


LIMIT = {"float32": 3e-5, "bfloat16": 4e-2}


class Reference:
    """Plain evaluation of one sequence, with the limit of every position: in fp32 a constant; in bf16 at least a constant, more where
    disturbing the projections by their rounding moves the logits further."""

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
