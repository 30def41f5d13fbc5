"""Weights from the safetensors files of a model folder (role of nanovllm/utils/loader.py)."""
from __future__ import annotations

import glob
import os
from typing import Dict, Iterable, Tuple

import torch
from safetensors import safe_open


class TensorFolder:
    """Every tensor of every ``*.safetensors`` file in a folder, read one at a time.  Tracks what has
    been taken, so that a model can insist on having used everything."""

    def __init__(self, folder: str):
        files = sorted(glob.glob(os.path.join(folder, "*.safetensors")))
        if not files:
            raise FileNotFoundError(f"no *.safetensors file in {folder}")
        self._where: Dict[str, object] = {}
        for path in files:
            handle = safe_open(path, framework="pt", device="cpu")
            for name in handle.keys():
                self._where[name] = handle
        self._taken = set()

    def take(self, name: str, shape: Iterable[int]) -> torch.Tensor:
        if name not in self._where:
            raise KeyError(f"tensor {name!r} is missing")
        t = self._where[name].get_tensor(name)
        if tuple(t.shape) != tuple(shape):
            raise ValueError(f"tensor {name!r} has shape {tuple(t.shape)}, the configuration asks for {tuple(shape)}")
        self._taken.add(name)
        return t

    def unused(self) -> Tuple[str, ...]:
        return tuple(sorted(set(self._where) - self._taken))
