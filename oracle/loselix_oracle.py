"""TEST INFRASTRUCTURE ONLY.  Plain, slow evaluation of the Loselix design in one dtype on the CPU (float64 by default), one function
per mechanism, written from its equations and sharing no code with the product.  A sequence is always evaluated as a whole; caches,
pages, portions and batches do not exist here.

    x      residual [T, width]
    h      what both sublayers of a layer read
    weights: dict name -> tensor (any dtype; converted on use)
    noise  (a seed): projections disturbed by the rounding of bfloat16, to see how far rounding alone moves the logits"""
from __future__ import annotations

import math

import torch

from .dafolorn_oracle import Weights, norm_plain, unit_rms, write_model  # noqa: F401
from .gulozen_oracle import Project, sigmoid


# ---- mechanisms -----------------------------------------------------------------------------------------------------------
def rotate_half(x, rot):
    """x [T, ..., n]: column i of the first rot.dims turns with column i + rot.dims / 2, by position x frequency i."""
    n = rot["dims"]
    f = torch.tensor([rot["base"] ** (-2.0 * i / n) for i in range(n // 2)], dtype=x.dtype)
    a = (torch.arange(x.shape[0], dtype=x.dtype)[:, None] * f).view(x.shape[0], *(1,) * (x.dim() - 2), n // 2)
    u, v = x[..., : n // 2], x[..., n // 2: n]
    return torch.cat([u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a), x[..., n:]], -1)


def soft_cap(s, cap):
    return cap * torch.tanh(s / cap)


def causal(T):
    return torch.tril(torch.ones(T, T, dtype=torch.bool))


def causal_softmax(s):
    """Rows of scores [T, T] -> weights over the keys up to each row's own."""
    s = s.masked_fill(~causal(s.shape[0]), -math.inf)
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def sigmoid_weights(s, bias):
    """Every visible key by itself; nothing is normalised."""
    return torch.where(causal(s.shape[0]), sigmoid(s + bias), torch.zeros_like(s))


def query_temperature(T, spec, dtype):
    """Factor on the queries of every position: grows with the logarithm of how many blocks of `every` positions are complete."""
    p = torch.arange(T)
    return 1.0 + spec["coef"] * torch.log((p + 1).div(spec["every"], rounding_mode="floor").to(dtype) + 1.0)


def relu_squared(z):
    return torch.clamp(z, min=0) ** 2


def map_weight(W, pre, diff):
    """lambda of the differential attention: what the second map's output is multiplied with before it is taken off the first's."""
    return torch.exp((W[pre + "lq1"] * W[pre + "lk1"]).sum()) - torch.exp((W[pre + "lq2"] * W[pre + "lk2"]).sum()) + diff


# ---- mixers ---------------------------------------------------------------------------------------------------------------
def differential(h, W, pre, spec, eps, proj):
    H, G, d, dv, T = spec["heads"], spec["kv_heads"], spec["dim"], spec["vdim"], h.shape[0]
    q = rotate_half(proj(h, W[pre + "q"]).view(T, H, 2, d), spec["rot"])
    k = rotate_half(proj(h, W[pre + "k"]).view(T, G, 2, d), spec["rot"])
    v = proj(h, W[pre + "v"]).view(T, G, dv)
    lam, out = map_weight(W, pre, spec["diff"]), torch.empty(T, H, dv, dtype=h.dtype)
    for i in range(H):
        j = i // (H // G)
        a = [causal_softmax(soft_cap(q[:, i, m] @ k[:, j, m].T * spec["scale"], spec["softcap"])) @ v[:, j] for m in (0, 1)]
        out[:, i] = unit_rms(a[0] - lam * a[1], eps) * (1.0 - spec["diff"])
    return proj(out.reshape(T, H * dv), W[pre + "o"])


def gated_heads(h, W, pre, spec, eps, proj):
    H, G, d, dv, T = spec["heads"], spec["kv_heads"], spec["dim"], spec["vdim"], h.shape[0]
    q = rotate_half(proj(h, W[pre + "q"]).view(T, H, d), spec["rot"])
    k = rotate_half(proj(h, W[pre + "k"]).view(T, G, d), spec["rot"])
    v, g = proj(h, W[pre + "v"]).view(T, G, dv), sigmoid(proj(h, W[pre + "g"]))
    out = torch.empty(T, H, dv, dtype=h.dtype)
    for i in range(H):
        j = i // (H // G)
        out[:, i] = causal_softmax(q[:, i] @ k[:, j].T * spec["scale"]) @ v[:, j] * g[:, i, None]
    return proj(out.reshape(T, H * dv), W[pre + "o"])


def sigmoid_attention(h, W, pre, spec, eps, proj):
    H, G, d, T = spec["heads"], spec["kv_heads"], spec["dim"], h.shape[0]
    assert spec["vdim"] == d
    raw = proj(h, W[pre + "k"])
    q = norm_plain(proj(h, W[pre + "q"]), W[pre + "q.norm"], eps) * query_temperature(T, spec["q_temp"], h.dtype)[:, None]
    q, k, v = q.view(T, H, d), norm_plain(raw, W[pre + "k.norm"], eps).view(T, G, d), raw.view(T, G, d)
    out = torch.empty(T, H, d, dtype=h.dtype)
    for i in range(H):
        j = i // (H // G)
        out[:, i] = sigmoid_weights(q[:, i] @ k[:, j].T * spec["scale"], W[pre + "pb"][i]) @ v[:, j]
    return proj(out.reshape(T, H * d) * sigmoid(proj(h, W[pre + "g"])), W[pre + "o"])


MIXERS = {"attention": differential, "attention_2": gated_heads, "attention_3": sigmoid_attention}


# ---- layers and model -----------------------------------------------------------------------------------------------------
def layer_forward(x, W, i, entry, eps, proj):
    p = f"l{i}."
    h = norm_plain(x, W[p + "norm1"], eps)
    y = MIXERS[entry["type"]](h, W, p + "mix.", entry["mixer"], eps, proj)
    if entry.get("mlp") is not None:
        y = y + proj(relu_squared(proj(h, W[p + "mlp.up"])), W[p + "mlp.down"])
    return x + y


def layer_order(cfg):
    """(layer, whether a pass of the loop other than its first begins here), in the order the layers run."""
    n, lo, hi, times = len(cfg["layers"]), 0, 0, 1
    if cfg.get("loop"):
        lo, hi, times = (cfg["loop"][k] for k in ("start", "stop", "times"))
    out = [(i, False) for i in range(lo)]
    for t in range(times):
        out += [(i, t > 0 and i == lo) for i in range(lo, hi)]
    return out + [(i, False) for i in range(hi, n)]


def forward(cfg: dict, tensors: dict, tokens, dtype=torch.float64, layers_out: list | None = None, noise=None):
    """Logits [T, vocab] of one sequence; layers_out (a list) receives the residual stream after every layer run."""
    W, proj, eps = Weights(tensors, dtype), Project(noise), cfg["norm"]["eps"]
    e = W["embed"][torch.as_tensor(tokens, dtype=torch.int64)]
    x = e
    for i, again in layer_order(cfg):
        if again:
            x = x + e
        x = layer_forward(x, W, i, cfg["layers"][i], eps, proj)
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm_plain(x, W["final.norm"], eps) @ W["head"].T


# ---- random models for tests ----------------------------------------------------------------------------------------------
def random_tensors(cfg: dict, seed: int) -> dict:
    """bfloat16 weights of the right names and shapes; sizes chosen so that every mechanism matters."""
    g = torch.Generator().manual_seed(seed)

    def n(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16)

    w, V = cfg["width"], cfg["vocab"]
    t = {"embed": n(V, w), "final.norm": n(w, std=0.1, mean=1.0), "head": n(V, w, std=w ** -0.5)}
    for i, e in enumerate(cfg["layers"]):
        m, p = e["mixer"], f"l{i}."
        H, G, d, dv, maps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], 2 if e["type"] == "attention" else 1
        t[p + "norm1"] = n(w, std=0.1, mean=1.0)
        t[p + "mix.q"], t[p + "mix.k"] = n(H * maps * d, w, std=1.5 * w ** -0.5), n(G * maps * d, w, std=1.5 * w ** -0.5)
        t[p + "mix.o"] = n(w, H * dv, std=(H * dv) ** -0.5)
        if e["type"] != "attention_3":
            t[p + "mix.v"] = n(G * dv, w, std=w ** -0.5)
        if e["type"] == "attention":
            for k in ("lq1", "lk1", "lq2", "lk2"):
                t[p + "mix." + k] = n(d, std=0.6 * d ** -0.5)
        elif e["type"] == "attention_2":
            t[p + "mix.g"] = n(H, w, std=2 * w ** -0.5)
        else:
            t[p + "mix.q.norm"], t[p + "mix.k.norm"] = n(H * d, std=0.2, mean=1.0), n(G * d, std=0.2, mean=1.0)
            t[p + "mix.pb"], t[p + "mix.g"] = n(H, std=1.0, mean=-3.0), n(H * dv, w, std=w ** -0.5)
        if e.get("mlp") is not None:
            ff = e["mlp"]["ff"]
            t[p + "mlp.up"], t[p + "mlp.down"] = n(ff, w, std=w ** -0.5), n(w, ff, std=ff ** -0.5)
    return t
