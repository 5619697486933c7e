"""Which class serves a checkpoint directory, by its config.json."""
from __future__ import annotations

import importlib
import json
import os
from typing import Tuple

import torch

# architecture name -> (module, class); every class has ``from_pretrained(path, device=..., dtype=...)`` and ``dtypes``, the formats it computes in
MODELS = {
    "AriaForConditionalGeneration": ("modeling_aria", "AriaForConditionalGeneration"),
    "Duguzen": ("duguzen", "DuguzenForCausalLM"),
    "Kozipel": ("kozipel", "KozipelForCausalLM"),
}
MODEL_TYPES = {"aria": "AriaForConditionalGeneration"}   # Hugging Face configs without an architecture name


def read_config(path: str) -> dict:
    with open(os.path.join(path, "config.json")) as f:
        return json.load(f)


def architecture(config: dict) -> str:
    names = [config.get("architecture")] + list(config.get("architectures") or []) + [MODEL_TYPES.get(config.get("model_type"))]
    for n in names:
        if n in MODELS:
            return n
    raise ValueError(f"no model for architecture {[n for n in names if n]} / model_type {config.get('model_type')!r}; known: {sorted(MODELS)}")


def resolve(config: dict) -> Tuple[str, type]:
    name = architecture(config)
    module, cls = MODELS[name]
    return name, getattr(importlib.import_module(f"{__package__}.{module}"), cls)


def load_model(path: str, device="cuda", dtype: torch.dtype = torch.bfloat16):
    """The model of a checkpoint directory, weights loaded, on ``device``."""
    name, cls = resolve(read_config(path))
    if dtype not in getattr(cls, "dtypes", (torch.bfloat16,)):
        raise TypeError(f"{name} does not compute in {dtype}")
    kwargs = {"dtype": dtype} if hasattr(cls, "dtypes") else {}
    return cls.from_pretrained(path, device=device, **kwargs)


def serving_model(model):
    """The object ``serving.Scheduler`` drives: the model itself, or the decode twin of a Hugging Face-shaped one."""
    if hasattr(model, "step"):
        return model
    if hasattr(model, "to_gptfast"):
        return model.to_gptfast()
    raise TypeError(f"{type(model).__name__} has no serving form")
