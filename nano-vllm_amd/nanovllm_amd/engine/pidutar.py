"""Pidutar: a decoder whose layers are latent attention or matrix memory, in any order, each beside a mixture of experts.

Mixer and feed-forward of a layer read the same point of the stream through norms of their own and are added
together (scaled per channel and by one constant); the residual stream is fp32, norm weights are stored around
zero, a layer may have no feed-forward, and an attention layer may read an earlier one's cache.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional, Tuple, Union

import torch
from torch import nn

from ..context import get_context
from .branches import branches_rms_norms, embed_rms_norms
from .experts import Experts, ExpertsSpec, ExpertWeights
from .latent import LatentAttention, LatentSpec, LatentWeights
from .layered import LayeredModel
from .mixers import RopeTables, Rotary
from .mlstm import Mlstm, MlstmSpec, MlstmWeights

NORM_OFFSET = 1.0                # norm weights are stored as the deviation from this

MixerSpec = Union[LatentSpec, MlstmSpec]


def _latent_spec(raw: dict) -> LatentSpec:
    spec = LatentSpec(heads=int(raw["heads"]), dim=int(raw["dim"]), rot_dim=int(raw["rot_dim"]), vdim=int(raw["vdim"]),
                      q_rank=int(raw["q_rank"]), kv_rank=int(raw["kv_rank"]), window=int(raw["mask"]["size"]), scale=float(raw["scale"]),
                      rot=Rotary(float(raw["rot"]["base"]), int(raw["rot"]["dims"])),
                      kv_from=None if raw.get("kv_from") is None else int(raw["kv_from"]))
    if spec.window < 1 or spec.rot_dim < 2 or spec.rot_dim % 2 or spec.rot.dims != spec.rot_dim:
        raise ValueError(f"inconsistent latent attention sizes: {spec}")
    return spec


def _mlstm_spec(raw: dict) -> MlstmSpec:
    spec = MlstmSpec(heads=int(raw["heads"]), dim=int(raw["dim"]), vdim=int(raw["vdim"]), gate_cap=float(raw["gate_cap"]))
    if spec.gate_cap <= 0.0:
        raise ValueError(f"the gate cap must be positive: {spec}")
    return spec


def _mlp_spec(raw: Optional[dict]) -> Optional[ExpertsSpec]:
    if raw is None:
        return None
    if raw["kind"] != "moe":
        raise ValueError(f"unknown feed-forward kind {raw['kind']!r}")
    router = raw["router"]
    spec = ExpertsSpec(experts=int(router["experts"]), top=int(router["top"]), ff=int(raw["expert"]["ff"]), scale=float(router["scale"]))
    if not 1 <= spec.top <= spec.experts:
        raise ValueError(f"inconsistent mixture of experts: {spec}")
    return spec


_MIXER_PARSERS = {"latent_attention": _latent_spec, "mlstm": _mlstm_spec}
_MIXER_WEIGHTS = {LatentSpec: LatentWeights, MlstmSpec: MlstmWeights}


@dataclass(frozen=True)
class LayerSpec:
    mixer: MixerSpec
    mlp: Optional[ExpertsSpec]


@dataclass(frozen=True)
class PidutarConfig:
    vocab_size: int
    hidden_size: int
    embed_scale: float
    residual_mult: float
    logit_scale: float
    norm_eps: float
    layers: Tuple[LayerSpec, ...]
    max_position_embeddings: int = 1 << 20     # the design sets no bound; the engine's max_model_len does
    name: str = "pidutar"

    portions = True
    dtypes = ("bfloat16", "float32")

    @classmethod
    def from_raw(cls, raw: dict) -> "PidutarConfig":
        layers: List[LayerSpec] = []
        for i, entry in enumerate(raw["layers"]):
            kind = entry["type"]
            if kind not in _MIXER_PARSERS:
                raise ValueError(f"layer {i}: unknown mixer {kind!r}")
            layers.append(LayerSpec(_MIXER_PARSERS[kind](entry["mixer"]), _mlp_spec(entry.get("mlp"))))
        for i, layer in enumerate(layers):
            j = getattr(layer.mixer, "kv_from", None)
            if j is None:
                continue
            source = layers[j].mixer if 0 <= j < i else None
            if not isinstance(source, LatentSpec) or source.kv_from is not None:
                raise ValueError(f"layer {i}: kv_from leads to no earlier attention layer with a cache of its own")
            if (source.kv_rank, source.rot_dim, source.rot) != (layer.mixer.kv_rank, layer.mixer.rot_dim, layer.mixer.rot):
                raise ValueError(f"layer {i} cannot read the cache of layer {j}: sizes or rotation differ")
        if not layers:
            raise ValueError("a model needs at least one layer")
        return cls(int(raw["vocab"]), int(raw["width"]), float(raw["embedding"]["scale"]), float(raw["residual_mult"]),
                   float(raw["logit_scale"]), float(raw["norm"]["eps"]), tuple(layers))

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)


class LayerWeights(nn.Module):

    def __init__(self, spec: LayerSpec, width: int):
        super().__init__()
        self.norm1, self.ls1 = nn.Parameter(torch.zeros(width)), nn.Parameter(torch.ones(width))
        self.mix = _MIXER_WEIGHTS[type(spec.mixer)](spec.mixer, width)
        self.norm2 = self.ls2 = self.mlp = None
        if spec.mlp is not None:
            self.norm2, self.ls2 = nn.Parameter(torch.zeros(width)), nn.Parameter(torch.ones(width))
            self.mlp = ExpertWeights(spec.mlp, width)

    def load(self, spec: LayerSpec, width: int, take, prefix: str) -> None:
        for name in ("norm1", "ls1") + (("norm2", "ls2") if spec.mlp is not None else ()):
            getattr(self, name).copy_(take(prefix + name, (width,)))
        self.mix.load(spec.mixer, width, take, prefix + "mix.")
        if spec.mlp is not None:
            self.mlp.load(spec.mlp, width, take, prefix + "mlp.")


class _Layer:

    def __init__(self, spec: LayerSpec, weights: LayerWeights, ropes: RopeTables, eps: float, earlier: List["_Layer"]):
        self.weights = weights
        if isinstance(spec.mixer, LatentSpec):
            source = None if spec.mixer.kv_from is None else earlier[spec.mixer.kv_from].mixer
            self.mixer = LatentAttention(spec.mixer, weights.mix, ropes, eps, source)
        else:
            self.mixer = Mlstm(spec.mixer, weights.mix, eps)
        self.mlp = Experts(spec.mlp, weights.mlp, ropes.device) if spec.mlp is not None else None

    @property
    def counters(self) -> Optional[torch.Tensor]:
        return None if self.mlp is None else self.mlp.counters


class Pidutar(LayeredModel):

    def __init__(self, cfg: PidutarConfig, max_position: int, device, seed: int = 0):
        super().__init__(cfg)
        self.final = nn.Parameter(torch.zeros(cfg.hidden_size))
        self.layer_weights = nn.ModuleList([LayerWeights(s, cfg.hidden_size) for s in cfg.layers])
        ropes = RopeTables(max_position, device)
        for spec, weights in zip(cfg.layers, self.layer_weights):
            self.layers.append(_Layer(spec, weights, ropes, cfg.norm_eps, self.layers))
        self.random_weights(device, seed)
        for spec, weights in zip(cfg.layers, self.layer_weights):
            if isinstance(spec.mixer, LatentSpec):
                weights.mix.by_head(spec.mixer)

    def load_tensors(self, take) -> None:
        width = self.cfg.hidden_size
        self.final.copy_(take("final.norm", (width,)))
        for i, (spec, weights) in enumerate(zip(self.cfg.layers, self.layer_weights)):
            weights.load(spec, width, take, f"l{i}.")

    def forward_layers(self, input_ids, positions, hidden, residual, first: int, last: int):
        cfg, layers = self.cfg, self.layers
        norm = dict(eps=cfg.norm_eps, weight_offset=NORM_OFFSET)
        if first == 0:
            w = layers[0].weights
            residual, *hidden = embed_rms_norms(input_ids, self.embed, cfg.embed_scale, (w.norm1, w.norm2), clear=layers[0].counters, **norm)
        for i in range(first, last):
            layer, w = layers[i], layers[i].weights
            y1 = layer.mixer(hidden[0])
            y2, _, weight = layer.mlp(hidden[1]) if layer.mlp is not None else (None, None, None)
            step = (residual, cfg.residual_mult, y1, w.ls1, y2, weight, w.ls2)
            if i + 1 < len(layers):
                nxt = layers[i + 1].weights
                hidden = branches_rms_norms(*step, (nxt.norm1, nxt.norm2), clear=layers[i + 1].counters, **norm)
            else:
                hidden = branches_rms_norms(*step, (self.final, None), rows=get_context().logit_rows, **norm)[0]
        return hidden, residual

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        # (the scale goes into the product, ahead of the rounding of its result)
        return torch.addmm(hidden.new_empty(1), hidden, self.head.t(), beta=0, alpha=self.cfg.logit_scale)
