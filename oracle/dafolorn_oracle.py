"""TEST INFRASTRUCTURE ONLY.  Plain, slow evaluation of the Dafolorn design in one dtype on the CPU (float64 by default),
one function per mechanism, written from its equations and sharing no code with the product.  A sequence is always
evaluated as a whole; caches, pages, portions and batches do not exist here.

    x      residual stream [T, width]
    h      what a sublayer reads
    weights: dict name -> tensor (any dtype; converted on use)"""
from __future__ import annotations

import math

import torch


class Weights:
    def __init__(self, tensors: dict, dtype=torch.float64):
        self.t, self.dtype = tensors, dtype

    def __getitem__(self, name: str) -> torch.Tensor:
        return self.t[name].to(self.dtype)

    def __contains__(self, name: str) -> bool:
        return name in self.t


# ---- norms and activations ------------------------------------------------------------------------------------------------
def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_zero_centred(x, w, eps):
    """RMS norm whose stored weight is the deviation from one."""
    return unit_rms(x, eps) * (1.0 + w)


def norm_plain(x, w, eps):
    return unit_rms(x, eps) * w


def softplus(v):
    return torch.log1p(torch.exp(-v.abs())) + torch.clamp(v, min=0)


def xielu(z, p, q):
    """Quadratic for z > 0, exponential-linear for z <= 0, both with slope one half at the origin."""
    pos = softplus(p) * z * z + 0.5 * z
    zn = torch.clamp(z, max=0)
    neg = (0.5 + softplus(q)) * (torch.exp(zn) - 1.0 - zn) + 0.5 * zn
    return torch.where(z > 0, pos, neg)


def soft_cap(z, cap):
    return z if cap is None else cap * torch.tanh(z / cap)


# ---- convolution over time ------------------------------------------------------------------------------------------------
def canon(h, w):
    """h + depthwise causal convolution; w [width, taps], the last tap multiplies the current token."""
    taps = w.shape[1]
    out = h.clone()
    for t in range(h.shape[0]):
        for j in range(taps):
            s = t - (taps - 1 - j)
            if s >= 0:
                out[t] += w[:, j] * h[s]
    return out


# ---- attention ------------------------------------------------------------------------------------------------------------
def sink_softmax(scores, visible, sink):
    """scores [T, T], visible bool [T, T]; one extra unit of mass exp(sink) in every denominator."""
    s = scores.masked_fill(~visible, -math.inf)
    m = torch.maximum(s.max(-1, keepdim=True).values, sink)
    e = torch.exp(s - m)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - m))


def window_mask(T, size):
    d = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (d >= 0) & (d < size)


def latent_attention(h, W, pre, spec, eps):
    H, dim, vdim, rank = spec["heads"], spec["dim"], spec["vdim"], spec["kv_rank"]
    T = h.shape[0]
    q = (h @ W[pre + "q"].T).view(T, H, dim)
    c = norm_plain(h @ W[pre + "dkv"].T, W[pre + "dkv.norm"], eps)
    assert c.shape[1] == rank
    k = (c @ W[pre + "uk"].T).view(T, H, dim)
    v = (c @ W[pre + "uv"].T).view(T, H, vdim)
    visible = window_mask(T, spec["mask"]["size"])
    sink = W[pre + "sink"]
    out = torch.empty(T, H, vdim, dtype=h.dtype)
    for i in range(H):
        a = sink_softmax((q[:, i] @ k[:, i].T) * spec["scale"], visible, sink[i])
        out[:, i] = a @ v[:, i]
    return out.reshape(T, H * vdim) @ W[pre + "o"].T


# ---- feed-forward ---------------------------------------------------------------------------------------------------------
def dense_mlp(h, W, pre):
    act = W[pre + "act"]
    return xielu(h @ W[pre + "up"].T, act[0], act[1]) @ W[pre + "down"].T


# ---- layers and model -----------------------------------------------------------------------------------------------------
def layer_forward(x, W, i, entry, eps):
    p = f"l{i}."
    h = canon(norm_zero_centred(x, W[p + "norm1"], eps), W[p + "canon1"])
    assert entry["type"] == "latent_attention"
    x = x + norm_zero_centred(latent_attention(h, W, p + "mix.", entry["mixer"], eps), W[p + "norm1b"], eps)
    if entry.get("mlp") is not None:
        h = canon(norm_zero_centred(x, W[p + "norm2"], eps), W[p + "canon2"])
        x = x + norm_zero_centred(dense_mlp(h, W, p + "mlp."), W[p + "norm2b"], eps)
    return x


def pass_entry(x, x0, W, t):
    """Ahead of pass t of the looped layers: mix the embedding output back in, then add the pass's vector."""
    return torch.cat([x, x0], -1) @ W["loop.in"].T + W["loop.step"][t]


def forward(cfg: dict, tensors: dict, tokens, dtype=torch.float64, layers_out: list | None = None):
    """Logits [T, vocab] of one sequence; layers_out (a list) receives the residual stream after every layer run."""
    W = Weights(tensors, dtype)
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.int64)]
    x0 = x
    L = cfg["layers"]
    loop = cfg.get("loop")

    def run(i, x):
        x = layer_forward(x, W, i, L[i], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
        return x

    lo, hi, times = (loop["start"], loop["stop"], loop["times"]) if loop else (len(L), len(L), 0)
    for i in range(lo):
        x = run(i, x)
    for t in range(times):
        x = pass_entry(x, x0, W, t)
        for i in range(lo, hi):
            x = run(i, x)
    for i in range(hi, len(L)):
        x = run(i, x)
    x = norm_zero_centred(x, W["final.norm"], eps)
    return soft_cap(x @ W["embed"].T, cfg.get("logit_softcap"))


# ---- random models for tests ----------------------------------------------------------------------------------------------
def random_tensors(cfg: dict, seed: int, scale: float = 1.0) -> dict:
    """bfloat16 weights of the right names and shapes; gains chosen so that every mechanism matters."""
    g = torch.Generator().manual_seed(seed)

    def n(*shape, std=1.0):
        return (torch.randn(*shape, generator=g) * std).to(torch.bfloat16)

    w, V, taps = cfg["width"], cfg["vocab"], cfg["canon"]["taps"]
    t = {"embed": n(V, w, std=0.7), "final.norm": n(w, std=0.1)}
    loop = cfg.get("loop")
    if loop:
        t["loop.in"] = n(w, 2 * w, std=(2 * w) ** -0.5)
        t["loop.step"] = n(loop["times"], w, std=0.3)
    for i, e in enumerate(cfg["layers"]):
        m, p = e["mixer"], f"l{i}."
        H, d, dv, r = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
        t[p + "norm1"], t[p + "norm1b"] = n(w, std=0.1), n(w, std=0.1)
        t[p + "canon1"] = n(w, taps, std=0.4)
        t[p + "mix.q"] = n(H * d, w, std=scale * 1.5 * w ** -0.5)
        t[p + "mix.dkv"], t[p + "mix.dkv.norm"] = n(r, w, std=w ** -0.5), (1 + 0.1 * n(r).float()).to(torch.bfloat16)
        t[p + "mix.uk"], t[p + "mix.uv"] = n(H * d, r, std=1.5 * r ** -0.5), n(H * dv, r, std=r ** -0.5)
        t[p + "mix.sink"] = n(H, std=1.0)
        t[p + "mix.o"] = n(w, H * dv, std=(H * dv) ** -0.5)
        if e.get("mlp") is not None:
            ff = e["mlp"]["ff"]
            t[p + "norm2"], t[p + "norm2b"] = n(w, std=0.1), n(w, std=0.1)
            t[p + "canon2"] = n(w, taps, std=0.4)
            t[p + "mlp.up"], t[p + "mlp.down"] = n(ff, w, std=w ** -0.5), n(w, ff, std=ff ** -0.5)
            t[p + "mlp.act"] = n(2, std=0.7)
    return t


def write_model(path: str, cfg: dict, tensors: dict) -> None:
    import json
    import os

    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in tensors.items()}, os.path.join(path, "model.safetensors"))
