"""Which model a config.json describes: architecture -> configuration reader, model class and what the engine has to know
about it before the model exists.  Entries are resolved lazily so that a process imports only the model it serves."""
from __future__ import annotations

import importlib
from dataclasses import dataclass


@dataclass(frozen=True)
class ModelEntry:
    name: str
    config_reader: str        # "module:function": dict -> namespace with the attribute names the engine reads
    model_class: str          # "module:class"
    default_block_size: int   # tokens per cache block
    block_multiple: int       # block sizes must be multiples of this
    dtypes: tuple             # activation dtypes the model runs in
    kernel_set: str | None    # build.py kernel set that is enough for this model (None: the whole library)
    step_batches: bool        # True: the model runs StepBatch inputs (portions of prompts beside decoded tokens, recurrent state)

    @staticmethod
    def _resolve(path: str):
        mod, attr = path.split(":")
        return getattr(importlib.import_module(mod), attr)

    def read_config(self, raw: dict):
        return self._resolve(self.config_reader)(raw)

    def load_class(self):
        return self._resolve(self.model_class)


GLM4_MOE = ModelEntry("glm4_moe", "nanovllm.config:normalise_hf_config", "nanovllm.models.glm4_moe.model:Glm4MoeForCausalLM",
                      256, 256, ("bfloat16",), None, False)
DAFOLORN = ModelEntry("dafolorn", "nanovllm.models.dafolorn.config:read_config", "nanovllm.models.dafolorn.model:DafolornForCausalLM",
                      64, 32, ("bfloat16", "float32"), "dafolorn", True)
NAPADRA = ModelEntry("napadra", "nanovllm.models.napadra.config:read_config", "nanovllm.models.napadra.model:NapadraForCausalLM",
                     64, 64, ("bfloat16", "float32"), "napadra", True)
GULOZEN = ModelEntry("gulozen", "nanovllm.models.gulozen.config:read_config", "nanovllm.models.gulozen.model:GulozenForCausalLM",
                     64, 32, ("bfloat16", "float32"), "gulozen", True)
LOSELIX = ModelEntry("loselix", "nanovllm.models.loselix.config:read_config", "nanovllm.models.loselix.model:LoselixForCausalLM",
                     64, 64, ("bfloat16", "float32"), "loselix", True)

_ENTRIES = {e.name: e for e in (GLM4_MOE, DAFOLORN, NAPADRA, GULOZEN, LOSELIX)}


def find_model(cfg) -> ModelEntry:
    """Entry for a config (dict or namespace): `architecture`, then `model_type`, then the first of `architectures`;
    a config that names none is GLM-4-MoE's."""
    get = cfg.get if isinstance(cfg, dict) else (lambda k, d=None: getattr(cfg, k, d))
    name = get("architecture") or get("model_type")
    if not name:
        archs = get("architectures") or ()
        name = {"Glm4MoeForCausalLM": "glm4_moe"}.get(archs[0], archs[0]) if archs else "glm4_moe"
    entry = _ENTRIES.get(str(name).lower())
    if entry is None:
        raise NotImplementedError(f"model {name!r} is not built here; known: {sorted(_ENTRIES)}")
    return entry
