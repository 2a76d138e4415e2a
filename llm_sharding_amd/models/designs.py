"""The config-driven stack designs by the ``architecture`` of their config.json, and their checkpoints.

A design module translates config.json into a :class:`.stack.StackConfig` (``config_from_dict``) and
names and draws the tensors (``layer_shapes``, ``random_*``, ``write_random_checkpoint``; ``extra_shapes``
and ``random_extra`` where there are tensors of no layer)."""
from __future__ import annotations

import json
import os
import struct

from . import deretar, dumizen, gupuvik, runidra

DESIGNS = {m.ARCHITECTURE: m for m in (deretar, gupuvik, dumizen, runidra)}
_BY_TYPE = {"deretar": deretar, "gupuvik": gupuvik, "dumizen": dumizen, "runidra": runidra}


def of(cfg):
    """The design module of a stack configuration."""
    return _BY_TYPE[cfg.model_type]


class CheckpointTensors:
    """Named tensors of a checkpoint folder (model.safetensors), read one at a time (memory-mapped)."""

    def __init__(self, path: str):
        self.file = os.path.join(path, "model.safetensors")
        if not os.path.exists(self.file):
            raise FileNotFoundError(self.file)

    def get(self, names: dict, device, dtype) -> dict:
        """{key: tensor name} -> {key: tensor}; shapes are checked by the caller."""
        from safetensors import safe_open
        with safe_open(self.file, framework="pt", device="cpu") as f:
            return {k: f.get_tensor(n).to(device=device, dtype=dtype) for k, n in names.items()}

    def shapes(self) -> dict:
        """Tensor name -> shape, from the file's header alone."""
        with open(self.file, "rb") as f:
            head = json.loads(f.read(struct.unpack("<Q", f.read(8))[0]))
        return {k: tuple(v["shape"]) for k, v in head.items() if k != "__metadata__"}


__all__ = ["DESIGNS", "of", "CheckpointTensors"]
