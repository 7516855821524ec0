"""Model registry: config.json names an architecture, the registry maps it to the class that reads the configuration, loads the
weights and runs a step.  The classes are imported on first use."""
from __future__ import annotations

import importlib
import json
import os

# architecture name -> (module, class)
_REGISTRY = {
    "Bagedra": ("omniserve_amd.models.bagedra", "Bagedra"),
    "Bobavik": ("omniserve_amd.models.bobavik", "Bobavik"),
    "LlamaForCausalLM": ("omniserve_amd.models.qserve_llama", "QServeLlama"),
}


def register(architecture: str, module: str, cls: str) -> None:
    _REGISTRY[architecture] = (module, cls)


def architectures():
    return sorted(_REGISTRY)


def read_config(model_dir: str) -> dict:
    with open(os.path.join(model_dir, "config.json")) as f:
        return json.load(f)


def architecture_of(config: dict) -> str:
    name = config.get("architecture") or (config.get("architectures") or [None])[0]
    if name is None:
        raise ValueError("config.json names no architecture")
    return name


def model_class(config: dict):
    name = architecture_of(config)
    if name not in _REGISTRY:
        raise ValueError("unknown architecture %r (known: %s)" % (name, ", ".join(architectures())))
    module, cls = _REGISTRY[name]
    return getattr(importlib.import_module(module), cls)


def load_model(model_dir: str, dtype=None, device="cuda"):
    """The model of a checkpoint directory on `device`; dtype None: the class's own default."""
    config = read_config(model_dir)
    return model_class(config).from_pretrained(model_dir, config, dtype, device)
