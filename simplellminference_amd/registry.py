"""Model registry: ``config.json``'s "architecture" -> the class that serves it.

``load_model(folder)`` is how the command line (``__main__.py``) and ``bin/trace_run`` get a model. A Llama folder holds
``config.json`` ({"architecture": "Llama", + any LlamaModelConfig field}) and the reference's flat fp32 weight file
``model.bin``; a block-stack folder holds ``config.json`` and ``model.safetensors``."""
from __future__ import annotations

import os
from dataclasses import fields
from typing import Callable

from .checkpoint import read_config
from .model import LlamaModel, LlamaModelConfig
from .stack import Bokulix, Rugudra

_REGISTRY: dict[str, Callable] = {}


def register(architecture: str):
    def add(build: Callable) -> Callable:
        _REGISTRY[architecture] = build
        return build
    return add


def architectures() -> list[str]:
    return sorted(_REGISTRY)


@register("Llama")
def _llama(cfg: dict, folder: str, dtype: str, max_length: int, batch: int, device: int):
    known = {f.name for f in fields(LlamaModelConfig)}
    config = LlamaModelConfig(**{**{k: v for k, v in cfg.items() if k in known}, "max_length": max_length})
    t = "f32" if dtype in ("float32", "f32", "fp32") else "f16"
    return LlamaModel(model_path=os.path.join(folder, "model.bin"), config=config, w_dtype=t, kv_dtype=t, batch=batch,
                      device=device)


@register("Rugudra")
def _rugudra(cfg: dict, folder: str, dtype: str, max_length: int, batch: int, device: int):
    return Rugudra.from_config(cfg, max_length, model_path=folder, dtype=dtype, batch=batch, device=device)


@register("Bokulix")
def _bokulix(cfg: dict, folder: str, dtype: str, max_length: int, batch: int, device: int):
    return Bokulix.from_config(cfg, max_length, model_path=folder, dtype=dtype, batch=batch, device=device)


def load_model(folder: str, dtype: str = "bfloat16", max_length: int = 1024, batch: int = 1, device: int = 0):
    """The initialised model of a folder, by its config.json."""
    cfg = read_config(folder)
    arch = cfg.get("architecture")
    if arch not in _REGISTRY:
        raise ValueError(f"unknown architecture {arch!r} (known: {', '.join(architectures())})")
    return _REGISTRY[arch](cfg, folder, dtype, max_length, batch, device).init()
