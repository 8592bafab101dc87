"""Configuration of the Gulozen design: config.json -> the namespace the engine and the model read.  Every size and constant comes
from the file; unknown mixers, feed-forwards and rotations are refused rather than guessed."""
from __future__ import annotations

import types

import torch

from nanovllm.engine.key_reach import EVERYTHING, KeyReach
from nanovllm.hip_ops import round8

MAX_POSITIONS = 1 << 30  # rotations and recurrences go on for ever: nothing limits a sequence but memory


class LayerSpec(types.SimpleNamespace):
    """One entry of `layers`: mixer type and sizes, feed-forward kind and sizes (mlp None: no feed-forward)."""


def _layer(i: int, e: dict) -> LayerSpec:
    m = e["mixer"]
    s = LayerSpec(index=i, type=e["type"], heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), mlp=None)
    if s.type == "latent_attention":
        s.q_rank, s.kv_rank, s.rot_dim, s.scale = int(m["q_rank"]), int(m["kv_rank"]), int(m["rot_dim"]), float(m["scale"])
        rot = m["rot"]
        unknown = set(rot) - {"base", "dims", "scaling"}
        if unknown:
            raise NotImplementedError(f"layer {i}: rotation with {sorted(unknown)}")
        s.rot_base, s.rot_pairs_dim, s.rot_scaling = float(rot["base"]), int(rot["dims"]), None
        if rot.get("scaling") is not None:
            s.rot_scaling = {k: float(rot["scaling"][k]) for k in ("factor", "original", "fast", "slow")}
        if min(s.q_rank, s.kv_rank, s.rot_dim) < 1:
            raise ValueError(f"layer {i}: sizes must be positive")
    elif s.type == "lightning":
        s.decay = [float(d) for d in m["decay"]]
        if len(s.decay) != s.heads:
            raise ValueError(f"layer {i}: {len(s.decay)} decays for {s.heads} heads")
    else:
        raise NotImplementedError(f"layer {i}: mixer {s.type!r}")
    mlp = e.get("mlp")
    if mlp is not None:
        if mlp["kind"] != "moe":
            raise NotImplementedError(f"layer {i}: feed-forward {mlp['kind']!r}")
        s.mlp, s.ff, s.experts, s.top = mlp["kind"], int(mlp["expert"]["ff"]), int(mlp["router"]["experts"]), int(mlp["router"]["top"])
        if s.ff < 1 or not 0 < s.top <= s.experts:
            raise ValueError(f"layer {i}: {s.top} of {s.experts} experts of {s.ff}")
    if min(s.heads, s.dim, s.vdim) < 1:
        raise ValueError(f"layer {i}: sizes must be positive")
    return s


def read_config(raw: dict) -> types.SimpleNamespace:
    d = raw if isinstance(raw, dict) else dict(vars(raw))
    layers = [_layer(i, e) for i, e in enumerate(d["layers"])]
    width, groups = int(d["width"]), int(d["norm"]["groups"])
    if not layers or groups < 1 or width % groups:
        raise ValueError(f"{len(layers)} layers, a width of {width} in {groups} groups")
    attends = any(s.type == "latent_attention" for s in layers)
    return types.SimpleNamespace(
        raw=d, model_type="gulozen", vocab_size=int(d["vocab"]), hidden_size=width, padded_width=round8(width), layers=layers,
        norm_groups=groups, rms_norm_eps=float(d["norm"]["eps"]), conv_taps=int(d["canon"]["taps"]), embedding_scale=float(d["embedding"]["scale"]),
        key_reach=KeyReach(windows=(EVERYTHING,) if attends else ()), num_hidden_layers=len(layers), max_position_embeddings=MAX_POSITIONS,
        torch_dtype=torch.bfloat16)
