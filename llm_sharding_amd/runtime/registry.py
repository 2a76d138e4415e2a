"""Which classes serve a model: chosen by its configuration, in one place.

    cfg = load_config(folder)                 # config.json -> LlamaConfig | StackConfig
    src = folder_source(folder, cfg)          # or random_source(cfg, seed)
    eng = make_engine(cfg, 0, cfg.num_hidden_layers, device, ..., source=src)
"""
from __future__ import annotations

import json
import os

from ..config import LlamaConfig
from ..models import designs
from ..models.stack import StackConfig
from .engine import RandomSource, ShardFolderSource, StackFolderSource, StackRandomSource, StageEngine


def load_config(path: str):
    """The configuration of a model folder (or of a config.json)."""
    p = os.path.join(path, "config.json") if os.path.isdir(path) else path
    with open(p) as f:
        d = json.load(f)
    if d.get("architecture") in designs.DESIGNS:
        folder = os.path.dirname(os.path.abspath(p))
        have = os.path.exists(os.path.join(folder, "model.safetensors"))
        return designs.DESIGNS[d["architecture"]].config_from_dict(
            d, name=os.path.basename(folder), shapes=designs.CheckpointTensors(folder).shapes() if have else None)
    if "layers" in d and "architecture" in d:
        raise ValueError(f"unknown architecture {d['architecture']!r}")
    return LlamaConfig.from_pretrained(path)


def is_stack(cfg) -> bool:
    return isinstance(cfg, StackConfig)


def engine_class(cfg):
    if is_stack(cfg):
        from .stack_engine import StackEngine
        return StackEngine
    return StageEngine


def make_engine(cfg, start: int, end: int, *args, **kw) -> StageEngine:
    """A stage engine for layers [start, end) of the model."""
    return engine_class(cfg)(cfg, start, end, *args, **kw)


def folder_source(path: str, cfg):
    return StackFolderSource(path, cfg) if is_stack(cfg) else ShardFolderSource(path, cfg)


def random_source(cfg, seed: int = 0):
    return StackRandomSource(cfg, seed) if is_stack(cfg) else RandomSource(cfg, seed)


def compute_dtype(cfg, device, dtype):
    """The type an engine on ``device`` computes in when ``dtype`` is asked for."""
    cls = engine_class(cfg)
    return dtype if device.type != "cuda" or dtype in cls.GPU_DTYPES else cls.GPU_DTYPES[0]


def kernel_family(cfg) -> str:
    """The kernel library that serves this model alone (csrc/build.py FAMILIES; "" = the full one)."""
    if not is_stack(cfg):
        return ""
    return {"deretar": "latent", "gupuvik": "hybrid", "dumizen": "looped", "runidra": "streams"}[cfg.model_type]


__all__ = ["load_config", "is_stack", "engine_class", "make_engine", "folder_source", "random_source",
           "compute_dtype", "kernel_family"]
