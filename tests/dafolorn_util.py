"""Shared pieces of the Dafolorn tests: small configurations of deliberately odd sizes, random models, and running them."""
import contextlib
import copy
import os

import torch

from oracle import dafolorn_oracle as O


def layer(heads, dim, vdim, rank, window, ff, scale=None):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "mask": {"size": window},
            "scale": scale if scale is not None else dim ** -0.5}, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(width, vocab, taps, layers, loop=None, cap=None, eps=1e-5):
    return {"architecture": "Dafolorn", "width": width, "vocab": vocab, "canon": {"taps": taps}, "norm": {"eps": eps}, "layers": layers,
            "loop": None if loop is None else dict(zip(("start", "stop", "times"), loop)), "logit_softcap": cap}


CONFIGS = {
    # nothing a multiple of 8, a layer without feed-forward, the loop from the first layer, no soft cap
    "odd": config(76, 203, 3, [layer(5, 20, 12, 44, 33, 100), layer(3, 24, 44, 72, 7, None), layer(2, 68, 72, 136, 150, 60)], (0, 2, 3)),
    # one token windows, five taps, loop in the middle and once only, large heads, a scale that is not dim^-1/2
    "wide": config(136, 320, 5, [layer(1, 136, 200, 264, 1, 264, 0.02), layer(17, 16, 16, 64, 65, 72), layer(4, 32, 64, 320, 129, 64, 0.3)],
                   (1, 2, 1), 5.0, 1e-3),
    # many heads (several groups per tile), a latent of 536 columns, no loop
    "tall": config(64, 128, 2, [layer(40, 8, 8, 536, 48, 128), layer(70, 16, 8, 24, 300, 40)], None, 20.0),
    # value heads beyond the expanded kernel: prompts attend in the absorbed form
    "huge": config(72, 64, 3, [layer(2, 264, 24, 64, 40, 48, 0.05), layer(1, 16, 328, 48, 77, 48)], (0, 1, 2), 8.0),
    # loop up to the last layer, twice two layers
    "tail": config(200, 96, 4, [layer(6, 40, 24, 88, 64, 136), layer(4, 48, 32, 104, 64, 136), layer(6, 40, 24, 88, 31, 136)], (1, 3, 2), 12.0),
}


def make_model(path, name_or_cfg, seed=0):
    cfg = copy.deepcopy(CONFIGS[name_or_cfg]) if isinstance(name_or_cfg, str) else name_or_cfg
    t = O.random_tensors(cfg, seed)
    O.write_model(str(path), cfg, t)
    return cfg, t


@contextlib.contextmanager
def session(path, dtype, max_tokens, eager=True):
    from nanovllm.trace import TraceSession
    s = TraceSession(str(path), dtype, max_tokens, enforce_eager=eager)
    try:
        yield s
    finally:
        s.close()
        torch.cuda.empty_cache()


def tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def run_cut(s, toks, cuts, name="a", end=True):
    """The sequence in portions of the given sizes (the last size repeats); logits of every position."""
    out, at, i = [], 0, 0
    while at < len(toks):
        n = min(cuts[min(i, len(cuts) - 1)], len(toks) - at)
        last = at + n == len(toks)
        out.append(s.step([{"id": name, "tokens": toks[at: at + n], "want": list(range(n))}], [name] if last and end else []))
        at, i = at + n, i + 1
    return torch.cat(out)


def distance(got, want):
    """Worst position: rms of the difference over the vocabulary, relative to the rms of all logits."""
    want = want.double()
    return float(((got.double() - want).pow(2).mean(-1).sqrt()).max() / want.pow(2).mean().sqrt())


LIMIT = {"float32": 3e-5, "bfloat16": 4e-2}
HERE = os.path.dirname(os.path.abspath(__file__))
