"""Kaparax: a decoder whose layers are chunked softmax attention or retention, in any order.

Every sublayer is normed before and after (layer norm with bias), the residual stream is fp32, a layer
may have no feed-forward, and a layer may run another layer's weights with a cache or state of its own.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional, Tuple, Union

import torch
import torch.nn.functional as F
from torch import nn

from ..context import get_context
from . import mixers
from .layered import LayeredModel
from .mixers import AttentionSpec, MlpSpec, RetentionSpec, RopeTables, Rotary

MixerSpec = Union[AttentionSpec, RetentionSpec]


def _rotary(raw: dict) -> Rotary:
    rot = Rotary(float(raw["base"]), int(raw["dims"]))
    if rot.dims < 0 or rot.dims % 2:
        raise ValueError(f"rotated dimensions must be an even number, not {rot.dims}")
    return rot


def _attention_spec(raw: dict) -> AttentionSpec:
    spec = AttentionSpec(heads=int(raw["heads"]), kv_heads=int(raw["kv_heads"]), dim=int(raw["dim"]), vdim=int(raw["vdim"]),
                         taps=int(raw["conv"]), chunk=int(raw["mask"]["size"]), scale=float(raw["scale"]),
                         softcap=float(raw.get("softcap") or 0.0), rot=_rotary(raw["rot"]))
    if spec.heads % spec.kv_heads or spec.taps < 1 or spec.chunk < 1 or spec.rot.dims > spec.dim:
        raise ValueError(f"inconsistent attention sizes: {spec}")
    return spec


def _retention_spec(raw: dict) -> RetentionSpec:
    spec = RetentionSpec(heads=int(raw["heads"]), dim=int(raw["dim"]), vdim=int(raw["vdim"]),
                         decay=tuple(float(d) for d in raw["decay"]), rot=_rotary(raw["rot"]))
    if len(spec.decay) != spec.heads or spec.rot.dims > spec.dim or not all(0.0 <= d <= 1.0 for d in spec.decay):
        raise ValueError(f"inconsistent retention sizes: {spec}")
    return spec


def _mlp_spec(raw: Optional[dict]) -> Optional[MlpSpec]:
    if raw is None:
        return None
    if raw["kind"] != "dense":
        raise ValueError(f"unknown feed-forward kind {raw['kind']!r}")
    return MlpSpec(ff=int(raw["ff"]), limit=float(raw["limit"]))


_MIXER_PARSERS = {"attention": _attention_spec, "retention": _retention_spec}


@dataclass(frozen=True)
class LayerSpec:
    mixer: MixerSpec
    mlp: Optional[MlpSpec]
    weights_of: int                      # the layer whose tensors this one runs (its own index: its own)


@dataclass(frozen=True)
class KaparaxConfig:
    vocab_size: int
    hidden_size: int
    embed_scale: float
    norm_eps: float
    layers: Tuple[LayerSpec, ...]
    max_position_embeddings: int = 1 << 20     # the design sets no bound; the engine's max_model_len does
    name: str = "kaparax"

    portions = True
    dtypes = ("bfloat16", "float32")

    @classmethod
    def from_raw(cls, raw: dict) -> "KaparaxConfig":
        entries = raw["layers"]
        layers: List[LayerSpec] = []
        for i, entry in enumerate(entries):
            kind = entry["type"]
            if kind not in _MIXER_PARSERS:
                raise ValueError(f"layer {i}: unknown mixer {kind!r}")
            source, seen = i, set()
            while entries[source].get("weights_of") is not None:      # (a shared layer may itself name another)
                seen.add(source)
                source = entries[source]["weights_of"]
                if not 0 <= source < len(entries) or source in seen:
                    raise ValueError(f"layer {i}: weights_of leads to no layer with tensors of its own")
            layers.append(LayerSpec(_MIXER_PARSERS[kind](entry["mixer"]), _mlp_spec(entry.get("mlp")), source))
        for i, spec in enumerate(layers):
            if (spec.mixer, spec.mlp) != (layers[spec.weights_of].mixer, layers[spec.weights_of].mlp):
                raise ValueError(f"layer {i} differs from layer {spec.weights_of}, whose weights it shares")
        if not layers:
            raise ValueError("a model needs at least one layer")
        return cls(int(raw["vocab"]), int(raw["width"]), float(raw["embedding"]["scale"]), float(raw["norm"]["eps"]), tuple(layers))

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)


class _Norm(nn.Module):

    def __init__(self, width: int):
        super().__init__()
        self.w = nn.Parameter(torch.ones(width))
        self.b = nn.Parameter(torch.zeros(width))

    def load(self, width: int, take, name: str) -> None:
        self.w.copy_(take(name, (width,)))
        self.b.copy_(take(name + ".b", (width,)))

    @property
    def pair(self):
        return self.w, self.b


class LayerWeights(nn.Module):

    def __init__(self, spec: LayerSpec, width: int):
        super().__init__()
        self.norm1, self.norm1b = _Norm(width), _Norm(width)
        self.mix = mixers.MIXERS[type(spec.mixer)][0](spec.mixer, width)
        if spec.mlp is not None:
            self.norm2, self.norm2b = _Norm(width), _Norm(width)
            self.mlp = mixers.MlpWeights(spec.mlp, width)

    def load(self, spec: LayerSpec, width: int, take, prefix: str) -> None:
        for name in ("norm1", "norm1b") + (("norm2", "norm2b") if spec.mlp is not None else ()):
            getattr(self, name).load(width, take, prefix + name)
        self.mix.load(spec.mixer, width, take, prefix + "mix.")
        if spec.mlp is not None:
            self.mlp.load(spec.mlp, width, take, prefix + "mlp.")


class _Layer:
    """A layer of the stack: weights (possibly shared) and a mixer runtime of its own."""

    def __init__(self, spec: LayerSpec, weights: LayerWeights, ropes: RopeTables, eps: float):
        self.weights = weights
        self.mixer = mixers.MIXERS[type(spec.mixer)][1](spec.mixer, weights.mix, ropes, eps)
        self.mlp = mixers.ClampedGateMLP(spec.mlp, weights.mlp) if spec.mlp is not None else None


class Kaparax(LayeredModel):

    def __init__(self, cfg: KaparaxConfig, max_position: int, device, seed: int = 0):
        super().__init__(cfg)
        self.final = _Norm(cfg.hidden_size)
        self.layer_weights = nn.ModuleDict({str(i): LayerWeights(s, cfg.hidden_size)
                                            for i, s in enumerate(cfg.layers) if s.weights_of == i})
        ropes = RopeTables(max_position, device)
        self.layers = [_Layer(s, self.layer_weights[str(s.weights_of)], ropes, cfg.norm_eps) for s in cfg.layers]
        self.random_weights(device, seed)

    def load_tensors(self, take) -> None:
        width = self.cfg.hidden_size
        self.final.load(width, take, "final.norm")
        for i, weights in self.layer_weights.items():
            weights.load(self.cfg.layers[int(i)], width, take, f"l{i}.")

    def forward_layers(self, input_ids, positions, hidden, residual, first: int, last: int):
        eps, layers = self.cfg.norm_eps, self.layers
        if first == 0:
            residual, hidden = mixers.embed_norm(input_ids, self.embed, self.cfg.embed_scale, layers[0].weights.norm1.pair, eps)
        for i in range(first, last):
            layer, w = layers[i], layers[i].weights
            nxt, rows = self.final.pair, get_context().logit_rows
            if i + 1 < len(layers):
                nxt, rows = layers[i + 1].weights.norm1.pair, None
            y = layer.mixer(hidden)
            post = w.norm1b.pair
            if layer.mlp is not None:
                hidden = mixers.post_add_norm(y, residual, post, w.norm2.pair, eps)
                y, post = layer.mlp(hidden), w.norm2b.pair
            hidden = mixers.post_add_norm(y, residual, post, nxt, eps, rows)
        return hidden, residual

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden, self.head)
