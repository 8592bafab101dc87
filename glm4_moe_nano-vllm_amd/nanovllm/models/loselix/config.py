"""Configuration of the Loselix design: config.json -> the namespace the engine and the model read.  Every size and constant comes
from the file; unknown mixers, feed-forwards and rotations are refused rather than guessed."""
from __future__ import annotations

import types

import torch

from nanovllm.engine.key_reach import EVERYTHING, KeyReach
from nanovllm.hip_ops import round8
from nanovllm.models.layer_loop import read_loop

MAX_POSITIONS = 1 << 30  # rotations go on for ever: nothing limits a sequence but memory


class LayerSpec(types.SimpleNamespace):
    """One entry of `layers`: mixer type, sizes and constants, columns of the feed-forward (0: none)."""


def _rotation(s: LayerSpec, rot: dict) -> None:
    unknown = set(rot) - {"base", "dims"}
    if unknown:
        raise NotImplementedError(f"layer {s.index}: rotation with {sorted(unknown)}")
    s.rot_base, s.rot_dims = float(rot["base"]), int(rot["dims"])


def _layer(i: int, e: dict) -> LayerSpec:
    m = e["mixer"]
    s = LayerSpec(index=i, type=e["type"], heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), scale=float(m["scale"]), ff=0)
    if s.type == "attention":
        _rotation(s, m["rot"])
        s.diff, s.softcap = float(m["diff"]), float(m["softcap"])
        if s.softcap <= 0:
            raise ValueError(f"layer {i}: a soft cap of {s.softcap}")
    elif s.type == "attention_2":
        _rotation(s, m["rot"])
    elif s.type == "attention_3":
        s.temp_coef, s.temp_every = float(m["q_temp"]["coef"]), int(m["q_temp"]["every"])
        if s.temp_every < 1 or s.temp_every != m["q_temp"]["every"] or s.dim != s.vdim:
            raise ValueError(f"layer {i}: a temperature every {m['q_temp']['every']} positions, keys of {s.dim} columns that are values of {s.vdim}")
    else:
        raise NotImplementedError(f"layer {i}: mixer {s.type!r}")
    mlp = e.get("mlp")
    if mlp is not None:
        if mlp["kind"] != "dense":
            raise NotImplementedError(f"layer {i}: feed-forward {mlp['kind']!r}")
        s.ff = int(mlp["ff"])
    if min(s.heads, s.kv_heads, s.dim, s.vdim) < 1 or s.heads % s.kv_heads or (mlp is not None and s.ff < 1):
        raise ValueError(f"layer {i}: {s.heads} heads over {s.kv_heads} of {s.dim} and {s.vdim}, a feed-forward of {s.ff}: sizes must be positive and heads group up")
    return s


def read_config(raw: dict) -> types.SimpleNamespace:
    d = raw if isinstance(raw, dict) else dict(vars(raw))
    layers = [_layer(i, e) for i, e in enumerate(d["layers"])]
    if not layers:
        raise ValueError("no layers")
    width = int(d["width"])
    return types.SimpleNamespace(
        raw=d, model_type="loselix", vocab_size=int(d["vocab"]), hidden_size=width, padded_width=round8(width), layers=layers, loop=read_loop(d.get("loop"), len(layers)),
        rms_norm_eps=float(d["norm"]["eps"]), num_hidden_layers=len(layers), max_position_embeddings=MAX_POSITIONS, key_reach=KeyReach(windows=(EVERYTHING,)),
        torch_dtype=torch.bfloat16)
