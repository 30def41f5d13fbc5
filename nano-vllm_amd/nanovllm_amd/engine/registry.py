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


def register(architecture: str, config: str, model: str) -> None:
    _families[architecture] = Family(config, model)


register("Qwen3ForCausalLM", ".config:ModelConfig", ".model:Qwen3ForCausalLM")
register("Kaparax", ".kaparax:KaparaxConfig", ".kaparax:Kaparax")


def family_of_raw(raw: dict) -> Family:
    name = raw.get("architecture") or (raw.get("architectures") or [_DEFAULT])[0]
    if name not in _families:
        raise ValueError(f"unknown architecture {name!r} (known: {', '.join(sorted(_families))})")
    return _families[name]


def load_config(model_dir: str):
    with open(os.path.join(model_dir, "config.json")) as f:
        raw = json.load(f)
    return family_of_raw(raw).config_class.from_raw(raw)


def is_config(obj) -> bool:
    return any(isinstance(obj, f.config_class) for f in _families.values())


def model_class(cfg):
    for f in _families.values():
        if isinstance(cfg, f.config_class):
            return f.model_class
    raise ValueError(f"no model class for {type(cfg).__name__}")
