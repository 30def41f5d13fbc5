"""Which model family a ``config.json`` belongs to: its configuration class and its model class.

A family is found by the architecture name of the file (``"architecture"``, or the first entry of
``"architectures"``); a file that names none is a Qwen3 configuration.  A configuration class has
``from_raw(dict)`` and the attributes ``vocab_size``, ``hidden_size``, ``max_position_embeddings``,
``portions`` (the family's steps may cut prompts anywhere and mix portions with single tokens) and
``dtypes`` (element types it runs in).  Model classes are imported when they are built.
"""
from __future__ import annotations

import importlib
import json
import os
from dataclasses import dataclass
from typing import Dict

_DEFAULT = "Qwen3ForCausalLM"


@dataclass(frozen=True)
class Family:
    config: str                  # "module:class", relative to this package
    model: str
    kernels: str = "path"        # the kernel set its steps run on (``_lib.LIBRARIES``)

    @staticmethod
    def _resolve(where: str):
        module, name = where.split(":")
        return getattr(importlib.import_module(module, __package__), name)

    @property
    def config_class(self):
        return self._resolve(self.config)

    @property
    def model_class(self):
        return self._resolve(self.model)


_families: Dict[str, Family] = {}


def register(architecture: str, config: str, model: str, kernels: str = "path") -> None:
    _families[architecture] = Family(config, model, kernels)


register("Qwen3ForCausalLM", ".config:ModelConfig", ".model:Qwen3ForCausalLM")
register("Kaparax", ".kaparax:KaparaxConfig", ".kaparax:Kaparax", "mixers")
register("Pidutar", ".pidutar:PidutarConfig", ".pidutar:Pidutar", "latent")
register("Sokolorn", ".sokolorn:SokolornConfig", ".sokolorn:Sokolorn", "masked")
register("Bedenex", ".bedenex:BedenexConfig", ".bedenex:Bedenex", "parallel")


def family_of_raw(raw: dict) -> Family:
    name = raw.get("architecture") or (raw.get("architectures") or [_DEFAULT])[0]
    if name not in _families:
        raise ValueError(f"unknown architecture {name!r} (known: {', '.join(sorted(_families))})")
    return _families[name]


def _read(model_dir: str) -> dict:
    with open(os.path.join(model_dir, "config.json")) as f:
        return json.load(f)


def load_config(model_dir: str):
    raw = _read(model_dir)
    return family_of_raw(raw).config_class.from_raw(raw)


def kernels_of(model_dir: str) -> str:
    """The kernel set a model folder needs, without importing the family."""
    return family_of_raw(_read(model_dir)).kernels


def is_config(obj) -> bool:
    return any(isinstance(obj, f.config_class) for f in _families.values())


def _family_of(cfg) -> Family:
    for f in _families.values():
        if isinstance(cfg, f.config_class):
            return f
    raise ValueError(f"no model class for {type(cfg).__name__}")


def model_class(cfg):
    return _family_of(cfg).model_class


def kernels_for(cfg) -> str:
    return _family_of(cfg).kernels
