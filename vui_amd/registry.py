"""Which class serves a checkpoint.  A checkpoint names its design in its configuration (`architecture`); one without
that key is a Vui checkpoint, as the reference writes them (src/vui/model.py:1154-1219)."""
from __future__ import annotations

import json
import os

_MODELS: dict = {}
DEFAULT = "Vui"


def register_model(name: str):
    def put(cls):
        _MODELS[name] = cls
        return cls
    return put


def _import_all() -> None:
    from . import lm, model  # noqa: F401  (each registers its classes)


def registered() -> "list[str]":
    _import_all()
    return sorted(_MODELS)


def model_class(architecture: str):
    _import_all()
    if architecture not in _MODELS:
        raise ValueError(f"unknown architecture {architecture!r} (known: {', '.join(sorted(_MODELS))})")
    return _MODELS[architecture]


def read_architecture(path: "str | dict") -> str:
    """The design a local checkpoint names: a folder with config.json, a .safetensors file with a `config` in its
    metadata, or a dict {"config", "model"}."""
    if isinstance(path, dict):
        return path["config"].get("architecture", DEFAULT)
    if os.path.isdir(path):
        with open(os.path.join(path, "config.json")) as f:
            return json.load(f).get("architecture", DEFAULT)
    if not os.path.exists(path):
        raise FileNotFoundError(f"{path}: only local checkpoints can be loaded")
    if path.endswith(".safetensors"):
        from safetensors import safe_open

        with safe_open(path, framework="pt") as f:
            meta = f.metadata() or {}
        return json.loads(meta.get("config", "{}")).get("architecture", DEFAULT)
    return DEFAULT


def load_model(path: "str | dict", device="cuda", dtype=None, **kw):
    """The model behind a local checkpoint, whatever its design."""
    import torch

    return model_class(read_architecture(path)).from_pretrained(path, device=device, dtype=dtype or torch.bfloat16, **kw)
