"""Models by the name their config.json gives, and loading them from a folder of config.json + model.safetensors
(the role of astrai/factory.py:10-158 and astrai/model/automodel.py:54-81)."""
from __future__ import annotations

import json
import logging
import os
from typing import Any, Callable, Dict, Type

import torch
import torch.nn as nn

logger = logging.getLogger(__name__)

_MODELS: Dict[str, Type[nn.Module]] = {}


def register_model(name: str) -> Callable[[Type[nn.Module]], Type[nn.Module]]:
    """Class decorator.  A registered class has ``config_class.from_dict(config, tensor_shapes)``, takes
    ``(config, dtype=, device=)``, and offers ``tensors()``: checkpoint name -> parameter (or view of one)."""
    def add(cls):
        if name in _MODELS and _MODELS[name] is not cls:
            raise ValueError(f"model {name!r} is registered already")
        _MODELS[name] = cls
        return cls
    return add


def model_names():
    return sorted(_MODELS)


def model_class(config: Dict[str, Any]) -> Type[nn.Module]:
    """By ``architecture``, or by ``model_type`` as the reference's configurations name it."""
    name = config.get("architecture", config.get("model_type"))
    if name not in _MODELS:
        raise ValueError(f"unknown model {name!r}; registered: {', '.join(model_names())}")
    return _MODELS[name]


def load_tensors(model: nn.Module, tensors) -> None:
    """Fill a model from ``name -> tensor``; every name of the model must be there with its shape.  Names the model
    does not know are reported and left out."""
    want = model.tensors()
    missing, extra = sorted(set(want) - set(tensors)), sorted(set(tensors) - set(want))
    if missing:
        raise ValueError(f"checkpoint does not fit the model: missing {', '.join(missing[:5])}")
    if extra:
        logger.warning("checkpoint tensors the model has no place for: %s", ", ".join(extra[:10]))
    with torch.no_grad():
        for name, dst in want.items():
            src = tensors[name]
            if tuple(src.shape) != tuple(dst.shape):
                raise ValueError(f"{name}: checkpoint has {tuple(src.shape)}, the configuration asks for {tuple(dst.shape)}")
            dst.copy_(src)


def load_model(path: str, dtype: torch.dtype = torch.bfloat16, device="cuda:0") -> nn.Module:
    """A model from ``path/config.json`` and ``path/model.safetensors``, in evaluation mode on ``device``."""
    from safetensors.torch import load_file

    with open(os.path.join(path, "config.json")) as f:
        config = json.load(f)
    cls = model_class(config)
    tensors = load_file(os.path.join(path, "model.safetensors"))
    cfg = cls.config_class.from_dict(config, {n: tuple(t.shape) for n, t in tensors.items()})
    model = cls(cfg, dtype=dtype, device=device).eval()
    load_tensors(model, tensors)
    return model
