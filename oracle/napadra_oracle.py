"""TEST INFRASTRUCTURE ONLY.  Plain, slow evaluation of the Napadra design in one dtype on the CPU (float64 by default),
one function per mechanism, written from its equations and sharing no code with the product.  A sequence is always
evaluated as a whole, the recurrence token by token; caches, pages, portions and batches do not exist here.

    x      residual streams [T, streams, width]
    h      what a sublayer reads [T, width]
    weights: dict name -> tensor (any dtype; converted on use)"""
from __future__ import annotations

import math

import torch


class Weights:
    """noise: seed of a relative disturbance of every projection's result by up to 2^-8, about what 16-bit activations do (None: none)."""

    def __init__(self, tensors: dict, dtype=torch.float64, noise: int | None = None):
        self.t, self.dtype = tensors, dtype
        self.gen = None if noise is None else torch.Generator().manual_seed(noise)

    def __getitem__(self, name: str) -> torch.Tensor:
        return self.t[name].to(self.dtype)

    def linear(self, h: torch.Tensor, name: str) -> torch.Tensor:
        z = h @ self[name].T
        return z if self.gen is None else z * (1 + 2.0 ** -8 * (2 * torch.rand(z.shape, generator=self.gen, dtype=z.dtype) - 1))


# ---- embedding --------------------------------------------------------------------------------------------------------------
def sinusoid(T: int, width: int) -> torch.Tensor:
    """[T, width] fp64: angle p * 10000^(-2i / width), sine at the even entries, cosine at the odd ones."""
    out = torch.zeros(T, width, dtype=torch.float64)
    p = torch.arange(T, dtype=torch.float64)
    for j in range(width):
        a = p * 10000.0 ** (-2.0 * (j // 2) / width)
        out[:, j] = torch.sin(a) if j % 2 == 0 else torch.cos(a)
    return out


# ---- norms and activations ----------------------------------------------------------------------------------------------------
def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def clamped_glu(gate, up, limit):
    g = torch.clamp(gate, max=limit)
    u = torch.clamp(up, min=-limit, max=limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def log_sigmoid(z):
    return -(torch.log1p(torch.exp(-z.abs())) + torch.clamp(-z, min=0))


def soft_cap(z, cap):
    return cap * torch.tanh(z / cap)


# ---- streams --------------------------------------------------------------------------------------------------------------------
def collapse(x, w_in):
    return sum(w_in[s] * x[:, s] for s in range(x.shape[1]))


def spread(x, mix, w_out, y):
    """mix [from, to]; y: the finished sublayer's (scaled) output."""
    n = x.shape[1]
    return torch.stack([sum(mix[s, t] * x[:, s] for s in range(n)) + w_out[t] * y for t in range(n)], 1)


def token_shift(h, w):
    prev = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (prev - h) * w


# ---- attention --------------------------------------------------------------------------------------------------------------------
def chunk_mask(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & (i // size == j // size)


def sink_softmax(scores, visible, sink):
    """scores [T, T], visible bool [T, T]; one extra unit of mass exp(sink) in every denominator."""
    s = scores.masked_fill(~visible, -math.inf)
    m = torch.maximum(s.max(-1, keepdim=True).values, sink)
    e = torch.exp(s - m)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - m))


def slope(h: int, heads: int) -> float:
    return 2.0 ** (-8.0 * (h + 1) / heads)


def keys_values(h, W, pre, spec):
    T, G = h.shape[0], spec["kv_heads"]
    return (W.linear(h, pre + "k")).view(T, G, spec["dim"]), (W.linear(h, pre + "v")).view(T, G, spec["vdim"])


def attention(h, W, pre, spec, kv):
    H, G, T = spec["heads"], spec["kv_heads"], h.shape[0]
    q = (W.linear(h, pre + "q")).view(T, H, spec["dim"])
    k, v = kv
    dist = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(h.dtype)
    visible, sink = chunk_mask(T, spec["mask"]["size"]), W[pre + "sink"]
    out = torch.empty(T, H, spec["vdim"], dtype=h.dtype)
    for i in range(H):
        g = i // (H // G)
        a = sink_softmax((q[:, i] @ k[:, g].T) * spec["scale"] - slope(i, H) * dist, visible, sink[i])
        out[:, i] = a @ v[:, g]
    return W.linear(out.reshape(T, -1), pre + "o")


# ---- matrix memory ------------------------------------------------------------------------------------------------------------------
def mlstm_cell(q, k, v, i, f):
    """One head: q, k [T, dim], v [T, vdim], log gates i, f [T] -> [T, vdim]."""
    T = q.shape[0]
    S, n, m = torch.zeros(q.shape[1], v.shape[1], dtype=q.dtype), torch.zeros(q.shape[1], dtype=q.dtype), torch.zeros((), dtype=q.dtype)
    out = torch.empty(T, v.shape[1], dtype=q.dtype)
    for t in range(T):
        m_new = torch.maximum(f[t] + m, i[t])
        keep, add = torch.exp(f[t] + m - m_new), torch.exp(i[t] - m_new)
        S = keep * S + add * torch.outer(k[t], v[t])
        n = keep * n + add * k[t]
        m = m_new
        out[t] = (S.T @ q[t]) / (torch.maximum((n @ q[t]).abs(), torch.exp(-m)) + 1e-6)
    return out


def mlstm(h, W, pre, spec, eps):
    H, d, dv, cap, T = spec["heads"], spec["dim"], spec["vdim"], spec["gate_cap"], h.shape[0]
    q = (W.linear(h, pre + "q")).view(T, H, d) * d ** -0.5
    k, v = (W.linear(h, pre + "k")).view(T, H, d), (W.linear(h, pre + "v")).view(T, H, dv)
    i = soft_cap(W.linear(h, pre + "i") + W[pre + "i.b"], cap)
    f = log_sigmoid(soft_cap(W.linear(h, pre + "f") + W[pre + "f.b"], cap))
    o = torch.stack([unit_rms(mlstm_cell(q[:, a], k[:, a], v[:, a], i[:, a], f[:, a]), eps) for a in range(H)], 1)
    y = o.reshape(T, -1) * W[pre + "norm"] * torch.sigmoid(W.linear(h, pre + "g"))
    return W.linear(y, pre + "o")


# ---- feed-forward -------------------------------------------------------------------------------------------------------------------
def dense_mlp(h, W, pre, limit):
    return W.linear(clamped_glu(W.linear(h, pre + "gate"), W.linear(h, pre + "up"), limit), pre + "down")


# ---- layers and model ---------------------------------------------------------------------------------------------------------------
def sublayer(x, W, p, q, m, eps, shift, f):
    """x: streams; q: 1 or 2; f: h -> output of the mixer or the feed-forward."""
    h = unit_rms(collapse(x, W[p + f"hc{q}.in"]), eps) * W[p + f"norm{q}"]
    if shift is not None:
        h = token_shift(h, shift)
    return spread(x, W[p + f"hc{q}.mix"], m * W[p + f"hc{q}.out"], W[p + f"ls{q}"] * f(h))


def forward(cfg: dict, tensors: dict, tokens, dtype=torch.float64, layers_out: list | None = None, noise: int | None = None):
    """Logits [T, vocab] of one sequence; layers_out (a list) receives the sum of the streams after every layer."""
    W = Weights(tensors, dtype, noise)
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    T = len(tokens)
    e = W["embed"][torch.as_tensor(tokens, dtype=torch.int64)] + sinusoid(T, cfg["width"]).to(dtype)
    x = torch.stack([e] * cfg["streams"], 1)
    kv = {}
    for i, entry in enumerate(cfg["layers"]):
        p, spec = f"l{i}.", entry["mixer"]

        def mixer(h):
            if entry["type"] == "mlstm":
                return mlstm(h, W, p + "mix.", spec, eps)
            kv[i] = kv[spec["kv_from"]] if spec.get("kv_from") is not None else keys_values(h, W, p + "mix.", spec)
            return attention(h, W, p + "mix.", spec, kv[i])

        x = sublayer(x, W, p, 1, m, eps, W[p + "shift"], mixer)
        if entry.get("mlp") is not None:
            x = sublayer(x, W, p, 2, m, eps, None, lambda h: dense_mlp(h, W, p + "mlp.", entry["mlp"]["limit"]))
        if layers_out is not None:
            layers_out.append(x.sum(1))
    return (unit_rms(x.sum(1), eps) * W["final.norm"]) @ W["head"].T


# ---- random models for tests --------------------------------------------------------------------------------------------------------
def random_tensors(cfg: dict, seed: int) -> dict:
    """bfloat16 weights of the right names and shapes; sizes chosen so that every mechanism matters."""
    g = torch.Generator().manual_seed(seed)

    def n(*shape, std=1.0, mean=0.0):
        return (torch.randn(shape, generator=g) * std + mean).to(torch.bfloat16)

    w, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    t = {"embed": n(V, w, std=0.7), "head": n(V, w, std=w ** -0.5), "final.norm": n(std=0.1, mean=1.0)}
    for i, e in enumerate(cfg["layers"]):
        s, p = e["mixer"], f"l{i}."
        H, d, dv = s["heads"], s["dim"], s["vdim"]
        for q in (1, 2) if e.get("mlp") is not None else (1,):
            t[p + f"norm{q}"], t[p + f"ls{q}"] = n(std=0.1, mean=1.0), n(w, std=0.3, mean=1.0)
            t[p + f"hc{q}.in"], t[p + f"hc{q}.out"] = n(S, std=0.3, mean=0.7), n(S, std=0.4, mean=1.0)
            t[p + f"hc{q}.mix"] = (torch.eye(S) + 0.2 * torch.randn(S, S, generator=g)).to(torch.bfloat16)
        t[p + "shift"] = n(w, std=0.3, mean=0.4)
        t[p + "mix.o"] = n(w, H * dv, std=1.5 * (H * dv) ** -0.5)
        if e["type"] == "attention":
            G = s["kv_heads"]
            t[p + "mix.q"], t[p + "mix.sink"] = n(H * d, w, std=2.0 * w ** -0.5), n(H)
            if s.get("kv_from") is None:
                t[p + "mix.k"], t[p + "mix.v"] = n(G * d, w, std=2.0 * w ** -0.5), n(G * dv, w, std=w ** -0.5)
        else:
            t[p + "mix.q"], t[p + "mix.k"] = n(H * d, w, std=w ** -0.5), n(H * d, w, std=w ** -0.5)
            t[p + "mix.v"], t[p + "mix.g"] = n(H * dv, w, std=w ** -0.5), n(H * dv, w, std=w ** -0.5)
            t[p + "mix.norm"] = n(H * dv, std=0.2, mean=1.0)
            t[p + "mix.i"], t[p + "mix.i.b"] = n(H, w, std=1.5 * w ** -0.5), n(H, std=1.0)
            t[p + "mix.f"], t[p + "mix.f.b"] = n(H, w, std=1.5 * w ** -0.5), n(H, std=1.0, mean=3.0)
        if e.get("mlp") is not None:
            ff = e["mlp"]["ff"]
            t[p + "mlp.gate"], t[p + "mlp.up"], t[p + "mlp.down"] = n(ff, w, std=w ** -0.5), n(ff, w, std=w ** -0.5), n(w, ff, std=ff ** -0.5)
    return t


def write_model(path: str, cfg: dict, tensors: dict) -> None:
    import json
    import os

    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in tensors.items()}, os.path.join(path, "model.safetensors"))
