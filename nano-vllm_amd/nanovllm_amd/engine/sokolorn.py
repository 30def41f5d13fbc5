"""Sokolorn: a decoder of two kinds of attention layers, in any order: one without positions, under a sliding window, with
sinks and a gate per head; one rotated, over all earlier keys, that may read an earlier layer's keys and values.

Sublayers read the fp32 residual stream itself and are normed on their output; a layer's feed-forward is dense (squared
relu), a mixture of experts with an optional shared one, or missing; the embedding is also the head, its logits capped.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional, Tuple, Union

import torch
import torch.nn.functional as F
from torch import nn

from ..context import get_context
from .branches import embed_rms_norms, post_rms_norms
from .experts import Experts, ExpertsSpec, ExpertWeights, GateForm, SharedExpertSpec, project
from .layered import LayeredModel
from .masked import HEAD, WHOLE, MaskedAttention, MaskedSpec, MaskedWeights
from .mixers import RopeTables, Rotary, RotaryScaling, soft_cap_

NORM_OFFSET = 1.0                # norm weights of the stream are stored as the deviation from this
GATE_SLOPE, GATE_SHIFT = 1.702, 1.0


def _rotary(raw: dict, dim: int) -> Rotary:
    scaling = None
    if raw.get("scaling") is not None:
        scaling = RotaryScaling(*(float(raw["scaling"][k]) for k in ("factor", "low", "high", "original")))
        if scaling.factor <= 0.0 or scaling.original <= 0.0 or scaling.high < scaling.low:
            raise ValueError(f"inconsistent scaling of the rotation: {scaling}")
    rot = Rotary(float(raw["base"]), int(raw["dims"]), scaling)
    if rot.dims < 0 or rot.dims % 2 or rot.dims > dim:
        raise ValueError(f"cannot rotate {rot.dims} of {dim} elements")
    return rot


def _sizes(raw: dict) -> dict:
    return dict(heads=int(raw["heads"]), kv_heads=int(raw["kv_heads"]), dim=int(raw["dim"]), vdim=int(raw["vdim"]), scale=float(raw["scale"]),
                kv_from=None if raw.get("kv_from") is None else int(raw["kv_from"]))


def _windowed_spec(raw: dict) -> MaskedSpec:
    spec = MaskedSpec(**_sizes(raw), window=int(raw["mask"]["size"]), qk_norm=WHOLE, sink=True, gate=True)
    if spec.window < 1:
        raise ValueError(f"a window holds at least one key: {spec}")
    return spec


def _rotary_spec(raw: dict) -> MaskedSpec:
    return MaskedSpec(**_sizes(raw), rot=_rotary(raw["rot"], int(raw["dim"])), qk_norm=HEAD, bias=True)


@dataclass(frozen=True)
class DenseSpec:
    ff: int


MlpSpec = Union[DenseSpec, ExpertsSpec]


def _mlp_spec(raw: Optional[dict]) -> Optional[MlpSpec]:
    if raw is None:
        return None
    if raw["kind"] == "dense":
        return DenseSpec(int(raw["ff"]))
    if raw["kind"] != "moe":
        raise ValueError(f"unknown feed-forward kind {raw['kind']!r}")
    gate = lambda part: GateForm(float(part["limit"]), GATE_SLOPE, GATE_SHIFT)
    shared = raw.get("shared")
    spec = ExpertsSpec(experts=int(raw["router"]["experts"]), top=int(raw["router"]["top"]), ff=int(raw["expert"]["ff"]), gate=gate(raw["expert"]),
                       bias=True, shared=None if shared is None else SharedExpertSpec(int(shared["ff"]), gate(shared)))
    if not 1 <= spec.top <= spec.experts:
        raise ValueError(f"inconsistent mixture of experts: {spec}")
    return spec


_MIXER_PARSERS = {"attention": _windowed_spec, "attention_2": _rotary_spec}


@dataclass(frozen=True)
class LayerSpec:
    kind: str
    mixer: MaskedSpec
    mlp: Optional[MlpSpec]


@dataclass(frozen=True)
class SokolornConfig:
    vocab_size: int
    hidden_size: int
    norm_eps: float
    logit_softcap: float                       # 0: none
    layers: Tuple[LayerSpec, ...]
    max_position_embeddings: int = 1 << 20     # the design sets no bound; the engine's max_model_len does
    name: str = "sokolorn"

    portions = True
    dtypes = ("bfloat16", "float32")

    @classmethod
    def from_raw(cls, raw: dict) -> "SokolornConfig":
        layers: List[LayerSpec] = []
        for i, entry in enumerate(raw["layers"]):
            kind = entry["type"]
            if kind not in _MIXER_PARSERS:
                raise ValueError(f"layer {i}: unknown mixer {kind!r}")
            spec = LayerSpec(kind, _MIXER_PARSERS[kind](entry["mixer"]), _mlp_spec(entry.get("mlp")))
            if spec.mixer.heads % spec.mixer.kv_heads:
                raise ValueError(f"layer {i}: query heads do not divide into {spec.mixer.kv_heads} groups")
            layers.append(spec)
        for i, layer in enumerate(layers):
            j = layer.mixer.kv_from
            if j is None:
                continue
            source = layers[j] if 0 <= j < i else None
            if source is None or source.kind != layer.kind or source.mixer.kv_from is not None:
                raise ValueError(f"layer {i}: kv_from leads to no earlier layer of its kind with keys of its own")
            if not layer.mixer.reads_like(source.mixer):
                raise ValueError(f"layer {i} cannot read the keys of layer {j}: sizes or rotation differ")
        if not layers:
            raise ValueError("a model needs at least one layer")
        return cls(int(raw["vocab"]), int(raw["width"]), float(raw["norm"]["eps"]), float(raw.get("logit_softcap") or 0.0), tuple(layers))

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)


class DenseWeights(nn.Module):

    def __init__(self, spec: DenseSpec, width: int):
        super().__init__()
        self.up = nn.Parameter(torch.empty(spec.ff, width))
        self.down = nn.Parameter(torch.empty(width, spec.ff))

    def load(self, spec: DenseSpec, width: int, take, prefix: str) -> None:
        self.up.copy_(take(prefix + "up", self.up.shape))
        self.down.copy_(take(prefix + "down", self.down.shape))


class LayerWeights(nn.Module):

    def __init__(self, spec: LayerSpec, width: int):
        super().__init__()
        self.norm1 = nn.Parameter(torch.zeros(width))
        self.mix = MaskedWeights(spec.mixer, width)
        self.norm2 = self.mlp = None
        if spec.mlp is not None:
            self.norm2 = nn.Parameter(torch.zeros(width))
            self.mlp = (ExpertWeights if isinstance(spec.mlp, ExpertsSpec) else DenseWeights)(spec.mlp, width)

    def load(self, spec: LayerSpec, width: int, take, prefix: str) -> None:
        self.norm1.copy_(take(prefix + "norm1", (width,)))
        self.mix.load(spec.mixer, width, take, prefix + "mix.")
        if spec.mlp is not None:
            self.norm2.copy_(take(prefix + "norm2", (width,)))
            self.mlp.load(spec.mlp, width, take, prefix + "mlp.")


class _Layer:

    def __init__(self, spec: LayerSpec, weights: LayerWeights, ropes: RopeTables, eps: float, earlier: List["_Layer"]):
        self.weights = weights
        source = None if spec.mixer.kv_from is None else earlier[spec.mixer.kv_from].mixer
        self.mixer = MaskedAttention(spec.mixer, weights.mix, ropes, eps, source)
        self.has_mlp = spec.mlp is not None
        self.experts = Experts(spec.mlp, weights.mlp, ropes.device) if isinstance(spec.mlp, ExpertsSpec) else None

    @property
    def counters(self) -> Optional[torch.Tensor]:
        return None if self.experts is None else self.experts.counters

    def feed_forward(self, h: torch.Tensor):
        """Dense or shared branch and its weight, experts' outputs and theirs."""
        w = self.weights.mlp
        if self.experts is None:
            return project(project(h, w.up, squared_relu=True), w.down), None, None, None
        y, shared, weight = self.experts(h)
        top = self.experts.spec.top
        return shared, None if shared is None else weight[:, top], y, weight[:, :top]


class Sokolorn(LayeredModel):

    def __init__(self, cfg: SokolornConfig, max_position: int, device, seed: int = 0):
        super().__init__(cfg, tied=True)
        self.final = nn.Parameter(torch.zeros(cfg.hidden_size))
        self.layer_weights = nn.ModuleList([LayerWeights(s, cfg.hidden_size) for s in cfg.layers])
        ropes = RopeTables(max_position, device)
        for spec, weights in zip(cfg.layers, self.layer_weights):
            self.layers.append(_Layer(spec, weights, ropes, cfg.norm_eps, self.layers))
        self.random_weights(device, seed)

    def load_tensors(self, take) -> None:
        width = self.cfg.hidden_size
        self.final.copy_(take("final.norm", (width,)))
        for i, (spec, weights) in enumerate(zip(self.cfg.layers, self.layer_weights)):
            weights.load(spec, width, take, f"l{i}.")

    def forward_layers(self, input_ids, positions, hidden, residual, first: int, last: int):
        """``hidden`` between layers is the residual stream itself in the model's element type."""
        layers, norm = self.layers, dict(eps=self.cfg.norm_eps, weight_offset=NORM_OFFSET)
        if first == 0:
            residual, hidden, _ = embed_rms_norms(input_ids, self.embed, 1.0, (None, None), self.cfg.norm_eps)
        for i in range(first, last):
            layer, w = layers[i], layers[i].weights
            end = dict(nxt=None)
            if i + 1 == len(layers):
                end = dict(nxt=self.final, rows=get_context().logit_rows)
            y = layer.mixer(hidden)
            if layer.has_mlp:
                hidden = post_rms_norms(residual, y, None, None, None, w.norm1, None, clear=layer.counters, **norm)
                hidden = post_rms_norms(residual, *layer.feed_forward(hidden), w.norm2, **end, **norm)
            else:
                hidden = post_rms_norms(residual, y, None, None, None, w.norm1, **end, **norm)
        return hidden, residual

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        logits = F.linear(hidden, self.head)
        return soft_cap_(logits, self.cfg.logit_softcap) if self.cfg.logit_softcap > 0.0 else logits
