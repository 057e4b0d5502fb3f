"""Model folders: `config.json` (its "architecture" key names the model class) + `model.safetensors`.

`register(name)` puts a class beside the others; the class provides
  config_from_dict(d)          the configuration of a config.json, validated (unknown keys are errors)
  from_tensors(config, tensors, dtype, device)   the model with the file's tensors
  HIP_SOURCES                  csrc/ stems its kernels live in (None: the whole library)
"""
from __future__ import annotations

import json
from pathlib import Path

import torch

from . import _hip
from .checkpoint import read_safetensors

_MODELS: dict = {}


def register(name: str):
    def put(cls):
        if name in _MODELS:
            raise ValueError(f"architecture {name} is registered twice")
        _MODELS[name] = cls
        return cls

    return put


def architectures() -> list:
    _load_all()
    return sorted(_MODELS)


def _load_all() -> None:
    from . import bobasun, model, mugivik  # noqa: F401  (they register themselves)


def model_class(name: str):
    _load_all()
    if name not in _MODELS:
        raise ValueError(f"unknown architecture {name!r}; known: {', '.join(sorted(_MODELS))}")
    return _MODELS[name]


def read_config(folder) -> tuple:
    """(model class, configuration) of a model folder."""
    d = json.loads((Path(folder) / "config.json").read_text())
    if not isinstance(d, dict) or "architecture" not in d:
        raise ValueError(f"{folder}/config.json has no 'architecture'")
    cls = model_class(d["architecture"])
    return cls, cls.config_from_dict(d)


def is_model_folder(path) -> bool:
    return (Path(path) / "config.json").is_file() and (Path(path) / "model.safetensors").is_file()


def load_model(folder, dtype: torch.dtype = torch.bfloat16, device="cuda"):
    """The model of a folder on `device`, weights and activations in `dtype` (bfloat16 or float32)."""
    cls, config = read_config(folder)
    if torch.device(device).type == "cuda":
        _hip.require(cls.HIP_SOURCES)
    tensors = read_safetensors(Path(folder) / "model.safetensors")
    return cls.from_tensors(config, tensors, dtype, torch.device(device)).eval()
