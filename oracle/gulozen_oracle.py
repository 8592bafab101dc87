"""TEST INFRASTRUCTURE ONLY.  Plain, slow evaluation of the Gulozen design in one dtype on the CPU (float64 by default), one function
per mechanism, written from its equations and sharing no code with the product.  A sequence is always evaluated as a whole; caches,
pages, portions and batches do not exist here.

    x      residual [T, width]
    h      what a mixer reads
    weights: dict name -> tensor (any dtype; converted on use)
    noise  (a seed): projections disturbed by the rounding of bfloat16, to see how far rounding alone moves the logits"""
from __future__ import annotations

import math

import torch

from .dafolorn_oracle import Weights, canon, norm_plain, sink_softmax, unit_rms, write_model  # noqa: F401


# ---- norms ----------------------------------------------------------------------------------------------------------------
def norm_groups(x, w, groups, eps):
    """Each of `groups` equal parts of the vector divided by its own root mean square; one gain over the whole."""
    parts = x.view(*x.shape[:-1], groups, -1)
    return unit_rms(parts, eps).reshape(x.shape) * w


def silu(z):
    return z / (1.0 + torch.exp(-z))


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


class Project:
    """x W^T; with noise, the result off by a random relative 2^-9."""

    def __init__(self, noise=None):
        self.g = None if noise is None else torch.Generator().manual_seed(noise)

    def __call__(self, x, w):
        y = x @ w.T
        return y if self.g is None else y * (1.0 + (torch.rand(y.shape, generator=self.g, dtype=y.dtype) * 2 - 1) * 2.0 ** -9)


# ---- positions ------------------------------------------------------------------------------------------------------------
def yarn_frequencies(base, dims, scaling):
    """(frequency of every pair, factor on cos and sin): slow pairs are interpolated by `factor`, fast ones are not, a ramp between."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return f, 1.0
    factor, original = scaling["factor"], scaling["original"]

    def turns_at(t):   # pair index (times two) that makes t turns over the original length
        return dims * math.log(original / (2 * math.pi * t)) / (2 * math.log(base))

    lo, hi = max(math.floor(turns_at(scaling["fast"])), 0), min(math.ceil(turns_at(scaling["slow"])), dims - 1)
    out = []
    for i, v in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(v / factor * r + v * (1 - r))
    return out, 0.1 * math.log(factor) + 1.0


def rotate(x, rot):
    """x [T, ..., n]: neighbouring columns of the first rot.dims are pairs, turned by position x frequency."""
    f, m = yarn_frequencies(rot["base"], rot["dims"], rot.get("scaling"))
    a = torch.arange(x.shape[0], dtype=x.dtype)[:, None] * torch.tensor(f, dtype=x.dtype)
    a = a.view(a.shape[0], *(1,) * (x.dim() - 2), len(f))
    c, s, n = m * torch.cos(a), m * torch.sin(a), 2 * len(f)
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out = x.clone()
    out[..., 0:n:2], out[..., 1:n:2] = u * c - v * s, v * c + u * s
    return out


# ---- mixers ---------------------------------------------------------------------------------------------------------------
def latent_attention(h, W, pre, spec, eps, proj):
    H, dim, rd, vdim, rank = spec["heads"], spec["dim"], spec["rot_dim"], spec["vdim"], spec["kv_rank"]
    T = h.shape[0]
    cq = norm_plain(proj(h, W[pre + "dq"]), W[pre + "dq.norm"], eps)
    q = proj(cq, W[pre + "uq"]).view(T, H, dim + rd)
    both = proj(h, W[pre + "dkv"])
    assert both.shape[1] == rank + rd
    c, kr = norm_plain(both[:, :rank], W[pre + "dkv.norm"], eps), rotate(both[:, rank:], spec["rot"])
    k, v = proj(c, W[pre + "uk"]).view(T, H, dim), proj(c, W[pre + "uv"]).view(T, H, vdim)
    qr = rotate(q[..., dim:], spec["rot"])
    sink, visible = W[pre + "sink"], torch.tril(torch.ones(T, T, dtype=torch.bool))
    out = torch.empty(T, H, vdim, dtype=h.dtype)
    for i in range(H):
        s = (q[:, i, :dim] @ k[:, i].T + qr[:, i] @ kr.T) * spec["scale"]
        out[:, i] = sink_softmax(s, visible, sink[i]) @ v[:, i]
    return proj(out.reshape(T, H * vdim) * sigmoid(proj(h, W[pre + "g"])), W[pre + "o"])


def lightning(h, W, pre, spec, eps, proj):
    """S_t = decay S_(t-1) + k v^T, read by q, one state per head."""
    H, dim, vdim = spec["heads"], spec["dim"], spec["vdim"]
    T = h.shape[0]
    q, k = silu(proj(h, W[pre + "q"])).view(T, H, dim), silu(proj(h, W[pre + "k"])).view(T, H, dim)
    v = silu(proj(h, W[pre + "v"])).view(T, H, vdim)
    decay = torch.tensor(spec["decay"], dtype=h.dtype)
    S, out = torch.zeros(H, dim, vdim, dtype=h.dtype), torch.empty(T, H, vdim, dtype=h.dtype)
    for t in range(T):
        S = decay[:, None, None] * S + k[t, :, :, None] * v[t, :, None, :]
        out[t] = (S * q[t, :, :, None]).sum(1)
    return proj(norm_plain(out.reshape(T, H * vdim), W[pre + "norm"], eps) * sigmoid(proj(h, W[pre + "g"])), W[pre + "o"])


# ---- feed-forward ---------------------------------------------------------------------------------------------------------
def moe(x, W, pre, spec, proj, gaps=None):
    """gaps (a list) receives how far the last chosen expert's logit is above the first one that is not chosen, per token."""
    E, top = spec["router"]["experts"], spec["router"]["top"]
    z = x @ W[pre + "router"].T
    if gaps is not None and top < E:
        o = z.sort(-1, descending=True).values
        gaps.append(o[:, top - 1] - o[:, top])
    s = torch.exp(z - z.max(-1, keepdim=True).values)
    s = s / s.sum(-1, keepdim=True)
    best = s.topk(top, dim=-1).indices
    out = torch.zeros_like(x)
    for e in range(E):
        rows = (best == e).any(-1).nonzero().flatten()
        if rows.numel():
            p = f"{pre}e{e}."
            y = proj(silu(proj(x[rows], W[p + "gate"])) * proj(x[rows], W[p + "up"]), W[p + "down"])
            out[rows] += s[rows, e, None] * y
    return out


# ---- layers and model -----------------------------------------------------------------------------------------------------
def layer_forward(x, W, i, entry, cfg, proj, gaps=None):
    p, eps, groups = f"l{i}.", cfg["norm"]["eps"], cfg["norm"]["groups"]
    h = canon(x, W[p + "canon1"])
    mixer = {"latent_attention": latent_attention, "lightning": lightning}[entry["type"]]
    x = x + norm_groups(mixer(h, W, p + "mix.", entry["mixer"], eps, proj), W[p + "norm1"], groups, eps)
    if entry.get("mlp") is not None:
        x = x + norm_groups(moe(x, W, p + "mlp.", entry["mlp"], proj, gaps), W[p + "norm2"], groups, eps)
    return x


def forward(cfg: dict, tensors: dict, tokens, dtype=torch.float64, layers_out: list | None = None, noise=None, gaps: list | None = None):
    """Logits [T, vocab] of one sequence; layers_out (a list) receives what every layer hands on."""
    W, proj = Weights(tensors, dtype), Project(noise)
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.int64)] * cfg["embedding"]["scale"]
    X = [x]
    for i, e in enumerate(cfg["layers"]):
        X.append(layer_forward(x, W, i, e, cfg, proj, gaps))
        a = W[f"l{i}.dwa"]
        assert a.numel() == len(X)
        x = sum(a[j] * X[j] for j in range(len(X)))
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm_groups(x, W["final.norm"], groups, eps) @ W["head"].T


# ---- random models for tests ----------------------------------------------------------------------------------------------
FLAGS = 6      # columns that carry a token's signs through the model


def random_tensors(cfg: dict, seed: int) -> dict:
    """bfloat16 weights of the right names and shapes; sizes chosen so that every mechanism matters.

    Which expert is the last one chosen is a jump: a rounding decides close calls.  The last FLAGS columns of the embedding are large signs
    that no sublayer changes (their norm gains and taps are zero) and that the routers read above all; tokens whose choice is close in any
    layer are left out of the vocabulary (steady_tokens) and have zero rows in the head."""
    g = torch.Generator().manual_seed(seed)

    def n(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16)

    w, V, taps, F = cfg["width"], cfg["vocab"], cfg["canon"]["taps"], FLAGS
    t = {"embed": n(V, w, std=1.0 / cfg["embedding"]["scale"]), "final.norm": n(w, std=0.1, mean=1.0), "head": n(V, w, std=w ** -0.5)}
    t["embed"][:, -F:] = (torch.randint(0, 2, (V, F), generator=g) * 4 - 2) / cfg["embedding"]["scale"]
    for i, e in enumerate(cfg["layers"]):
        m, p = e["mixer"], f"l{i}."
        t[p + "norm1"] = n(w, std=0.1, mean=0.8)
        t[p + "norm1"][-F:] = 0
        t[p + "canon1"] = n(w, taps, std=0.4)
        t[p + "canon1"][-F:] = 0
        t[p + "dwa"] = n(i + 2, std=0.2)
        t[p + "dwa"][-1], t[p + "dwa"][0] = 0.7, 0.4
        if e["type"] == "lightning":
            H, d, dv = m["heads"], m["dim"], m["vdim"]
            t[p + "mix.q"], t[p + "mix.k"] = n(H * d, w, std=w ** -0.5), n(H * d, w, std=w ** -0.5)
            t[p + "mix.v"], t[p + "mix.g"] = n(H * dv, w, std=w ** -0.5), n(H * dv, w, std=w ** -0.5)
            t[p + "mix.norm"], t[p + "mix.o"] = n(H * dv, std=0.1, mean=1.0), n(w, H * dv, std=(H * dv) ** -0.5)
        else:
            H, d, rd, dv, r, qr = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"]
            t[p + "mix.dq"], t[p + "mix.dq.norm"], t[p + "mix.uq"] = n(qr, w, std=w ** -0.5), n(qr, std=0.1, mean=1.0), n(H * (d + rd), qr, std=1.5 * qr ** -0.5)
            t[p + "mix.dkv"], t[p + "mix.dkv.norm"] = n(r + rd, w, std=w ** -0.5), n(r, std=0.1, mean=1.0)
            t[p + "mix.uk"], t[p + "mix.uv"] = n(H * d, r, std=1.5 * r ** -0.5), n(H * dv, r, std=r ** -0.5)
            t[p + "mix.sink"], t[p + "mix.g"], t[p + "mix.o"] = n(H), n(H * dv, w, std=w ** -0.5), n(w, H * dv, std=(H * dv) ** -0.5)
        if e.get("mlp") is not None:
            E, ff = e["mlp"]["router"]["experts"], e["mlp"]["expert"]["ff"]
            t[p + "norm2"], t[p + "mlp.router"] = n(w, std=0.1, mean=0.8), n(E, w, std=0.02 * w ** -0.5)
            t[p + "norm2"][-F:] = 0
            t[p + "mlp.router"][:, -F:] = n(E, F, std=0.4)
            for k in range(E):
                q = f"{p}mlp.e{k}."
                t[q + "gate"], t[q + "up"], t[q + "down"] = n(ff, w, std=w ** -0.5), n(ff, w, std=w ** -0.5), n(w, ff, std=ff ** -0.5)
    keep = torch.zeros(V, dtype=torch.bool)
    keep[steady_tokens(cfg, t)] = True
    t["head"][~keep] = 0
    return t


def steady_tokens(cfg: dict, tensors: dict, margin: float = 0.06) -> torch.Tensor:
    """Tokens whose experts do not hang on a rounding."""
    gaps: list = []
    forward(cfg, tensors, list(range(cfg["vocab"])), dtype=torch.float32, gaps=gaps)
    ok = torch.ones(cfg["vocab"], dtype=torch.bool)
    for z in gaps:
        ok &= z > margin
    return ok.nonzero().flatten()
