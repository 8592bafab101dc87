"""Shared pieces of the Gulozen tests: small configurations of deliberately odd sizes, random models, and a reference with limits."""
import copy

import torch

from dafolorn_util import distance, run_cut, session  # noqa: F401
from oracle import gulozen_oracle as O

YARN = {"factor": 3.0, "original": 128, "fast": 16.0, "slow": 1.0}


def moe(ff, experts, top):
    return None if ff is None else {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, mlp=None, scale=None, base=10000.0, dims=None, scaling=None):
    rot = {"base": base, "dims": rot_dim if dims is None else dims}
    if scaling is not None:
        rot["scaling"] = dict(scaling)
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "rot": rot,
         "scale": scale if scale is not None else (dim + rot_dim) ** -0.5}
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def lightning(heads, dim, vdim, mlp=None, decay=None):
    if decay is None:
        decay = [1 - 2.0 ** -(1 + 1.7 * h) for h in range(heads)]
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, "mlp": mlp}


def config(width, vocab, groups, taps, layers, scale=3.0, eps=1e-5):
    return {"architecture": "Gulozen", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps, "groups": groups}, "canon": {"taps": taps},
            "embedding": {"scale": scale}}


CONFIGS = {
    # nothing a multiple of 8 (norm groups of 19 columns, six rotated ones of which four turn), layers without feed-forward, all experts chosen
    "odd": config(76, 203, 4, 3, [latent(5, 20, 6, 12, 44, 36, moe(20, 5, 2), dims=4, scaling=YARN), lightning(3, 20, 44),
                                  latent(3, 12, 10, 20, 28, 44, moe(36, 3, 3))]),
    # one norm group, five taps, one expert of many chosen, heads of 200 columns, a scale that is not dim^-1/2, two rotations
    "wide": config(136, 320, 1, 5, [lightning(2, 72, 136, moe(72, 9, 1)), latent(17, 136, 64, 200, 264, 264, moe(40, 6, 4), 0.03, 500.0, scaling=YARN),
                                    latent(2, 16, 8, 64, 24, 72)], 1.0, 1e-3),
    # many heads (several groups per tile), a cache row of 552 columns, many small norm groups, more than 64 experts
    "tall": config(64, 128, 8, 2, [latent(40, 8, 16, 8, 16, 536, moe(8, 70, 6), scaling=YARN), lightning(5, 136, 72), latent(70, 16, 8, 8, 40, 24, moe(24, 16, 3))], 12.0),
    # heads beyond the tiled kernels: keys of 264 columns in both mixers, values of 328; hundreds of experts
    "huge": config(72, 64, 2, 4, [latent(2, 264, 24, 24, 56, 64, moe(8, 300, 2), 0.05), lightning(1, 264, 24, moe(24, 4, 2), [0.97]), lightning(1, 64, 328, None, [0.9]),
                                  latent(1, 16, 8, 328, 16, 48)], 0.5),
    # no attention; a convolution over one token; a memory that never forgets and one that forgets at once
    "memory": config(200, 96, 5, 1, [lightning(4, 32, 64, moe(56, 8, 3), [1.0, 0.0, 0.5, 0.995]), lightning(6, 8, 8)]),
}


def make_model(path, name_or_cfg, seed=0):
    cfg = copy.deepcopy(CONFIGS[name_or_cfg]) if isinstance(name_or_cfg, str) else name_or_cfg
    t = O.random_tensors(cfg, seed)
    O.write_model(str(path), cfg, t)
    return cfg, t


def tokens(cfg, t, n, seed):
    """Random tokens among those whose experts do not hang on a rounding."""
    ok = O.steady_tokens(cfg, t)
    assert ok.numel() >= 8
    return ok[torch.randint(0, ok.numel(), (n,), generator=torch.Generator().manual_seed(seed))].tolist()


LIMIT = {"float32": 2e-5, "bfloat16": 4e-2}


def errors(got, want, scale):
    """Per position: rms of the difference over the vocabulary, relative to `scale`."""
    return (got.double() - want.double()).pow(2).mean(-1).sqrt() / scale


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
