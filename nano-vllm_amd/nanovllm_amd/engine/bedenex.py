"""Bedenex: a decoder whose layers are chunked attention with a distance bias or latent attention over all earlier keys, in any
order, each beside a dense feed-forward, a mixture of experts or nothing.

Mixer and feed-forward read the same norm of an fp32 stream and are added behind gates of every element that read it too, so one
product serves them all.  Some layers in a row may run several times with the same weights, each pass with caches of its own; a
pass begins from a product of the stream and the embeddings, and a vector of its own.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import List, Optional, Tuple, Union

import torch
import torch.nn.functional as F
from torch import nn

from ..context import get_context
from .branches import embed_rms_norms, entry_rms_norm, gated_rms_norm
from .experts import SIGMOID, Experts, ExpertsSpec, ExpertWeights, project, project_f32
from .latent import LatentAttention, LatentSpec, LatentWeights
from .layered import LayeredModel, load_rows
from .masked import UNIT, MaskedAttention, MaskedSpec, MaskedWeights
from .mixers import RopeTables, Rotary, gelu_gate

MixerSpec = Union[LatentSpec, MaskedSpec]


def _latent_spec(raw: dict) -> LatentSpec:
    spec = LatentSpec(heads=int(raw["heads"]), dim=int(raw["dim"]), rot_dim=int(raw["rot_dim"]), vdim=int(raw["vdim"]), q_rank=0,
                      kv_rank=int(raw["kv_rank"]), window=None, scale=float(raw["scale"]), rot=Rotary(float(raw["rot"]["base"]), int(raw["rot"]["dims"])),
                      gate=False, sink=True, halves=True)
    if spec.rot_dim < 2 or spec.rot_dim % 2 or spec.rot.dims != spec.rot_dim:
        raise ValueError(f"inconsistent latent attention sizes: {spec}")
    return spec


def _chunked_spec(raw: dict) -> MaskedSpec:
    spec = MaskedSpec(heads=int(raw["heads"]), kv_heads=int(raw["kv_heads"]), dim=int(raw["dim"]), vdim=int(raw["vdim"]), scale=float(raw["scale"]),
                      chunk=int(raw["mask"]["size"]), distance_bias=True, qk_norm=UNIT, v_norm=True, gate=True)
    if spec.chunk < 1:
        raise ValueError(f"a chunk holds at least one position: {spec}")
    if spec.heads % spec.kv_heads:
        raise ValueError(f"query heads do not divide into groups: {spec}")
    return spec


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
    spec = ExpertsSpec(experts=int(raw["router"]["experts"]), top=int(raw["router"]["top"]), ff=int(raw["expert"]["ff"]), score=SIGMOID, weigh_input=True)
    if not 1 <= spec.top <= spec.experts:
        raise ValueError(f"inconsistent mixture of experts: {spec}")
    return spec


_MIXERS = {"latent_attention": (_latent_spec, LatentWeights, LatentAttention), "attention": (_chunked_spec, MaskedWeights, MaskedAttention)}


@dataclass(frozen=True)
class LayerSpec:
    kind: str
    mixer: MixerSpec
    mlp: Optional[MlpSpec]


@dataclass(frozen=True)
class LoopSpec:
    """Layers ``[start, stop)`` run ``times`` times in a row."""
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class BedenexConfig:
    vocab_size: int
    hidden_size: int
    norm_eps: float
    layers: Tuple[LayerSpec, ...]
    loop: Optional[LoopSpec]
    max_position_embeddings: int = 1 << 20     # the design sets no bound; the engine's max_model_len does
    name: str = "bedenex"

    portions = True
    dtypes = ("bfloat16", "float32")

    @classmethod
    def from_raw(cls, raw: dict) -> "BedenexConfig":
        layers: List[LayerSpec] = []
        for i, entry in enumerate(raw["layers"]):
            kind = entry["type"]
            if kind not in _MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {kind!r}")
            layers.append(LayerSpec(kind, _MIXERS[kind][0](entry["mixer"]), _mlp_spec(entry.get("mlp"))))
        if not layers:
            raise ValueError("a model needs at least one layer")
        loop = None
        if raw.get("loop") is not None:
            loop = LoopSpec(*(int(raw["loop"][k]) for k in ("start", "stop", "times")))
            if not 0 <= loop.start < loop.stop <= len(layers) or loop.times < 1:
                raise ValueError(f"inconsistent loop: {loop}")
        return cls(int(raw["vocab"]), int(raw["width"]), float(raw["norm"]["eps"]), tuple(layers), loop)

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def runs(self) -> List[Tuple[int, Optional[int]]]:
        """(layer, the pass that begins with it or None) in the order in which layers run."""
        order = range(len(self.layers))
        if self.loop is None:
            return [(i, None) for i in order]
        s = self.loop
        looped = [(i, t if i == s.start else None) for t in range(s.times) for i in range(s.start, s.stop)]
        return [(i, None) for i in order[: s.start]] + looped + [(i, None) for i in order[s.stop:]]


class LayerWeights(nn.Module):
    """The gates' projections, and a dense feed-forward's first two, stand in one weight behind the mixer's own (mixer | gate of the
    mixer | gate of the feed-forward | gate, up)."""

    def __init__(self, spec: LayerSpec, width: int):
        super().__init__()
        branches = 1 if spec.mlp is None else 2
        dense = isinstance(spec.mlp, DenseSpec)
        self.norm1 = nn.Parameter(torch.ones(width))
        self.mix = _MIXERS[spec.kind][1](spec.mixer, width, branches * width + (2 * spec.mlp.ff if dense else 0))
        self.gate_bias = nn.Parameter(torch.zeros(branches * width))
        self.down = nn.Parameter(torch.empty(width, spec.mlp.ff)) if dense else None
        self.mlp = ExpertWeights(spec.mlp, width) if isinstance(spec.mlp, ExpertsSpec) else None
        first = self.mix.own_rows
        self.gates = slice(first, first + branches * width)
        self.gate_up = slice(self.gates.stop, self.gates.stop + 2 * spec.mlp.ff) if dense else None

    def load(self, spec: LayerSpec, width: int, take, prefix: str) -> None:
        self.norm1.copy_(take(prefix + "norm1", (width,)))
        self.mix.load(spec.mixer, width, take, prefix + "mix.")
        names = [prefix + "rg1"] + ([] if spec.mlp is None else [prefix + "rg2"])
        self.gate_bias.copy_(torch.cat([take(n + ".b", (width,)) for n in names]))
        beside = [take(n, (width, width)) for n in names]
        if self.down is not None:
            beside += [take(f"{prefix}mlp.{n}", (spec.mlp.ff, width)) for n in ("gate", "up")]
            self.down.copy_(take(prefix + "mlp.down", self.down.shape))
        if self.mlp is not None:
            self.mlp.load(spec.mlp, width, take, prefix + "mlp.")
        load_rows(self.mix.projections, self.mix.own_rows, beside)


class _Run:
    """One run of a layer: its weights, which other runs may share, and caches of its own."""

    def __init__(self, spec: LayerSpec, weights: LayerWeights, ropes: RopeTables, eps: float, begins: Optional[int]):
        self.weights, self.begins = weights, begins
        self.mixer = _MIXERS[spec.kind][2](spec.mixer, weights.mix, ropes, eps)
        self.experts = Experts(spec.mlp, weights.mlp, ropes.device) if weights.mlp is not None else None

    @property
    def counters(self) -> Optional[torch.Tensor]:
        return None if self.experts is None else self.experts.counters

    def branches(self, h: torch.Tensor):
        """What mixer and feed-forward give, and the gates' logits."""
        w = self.weights
        x = project(h, w.mix.projections)
        y2 = None
        if self.experts is not None:
            y2 = self.experts(h)[0]
        elif w.down is not None:
            y2 = project(gelu_gate(x[:, w.gate_up]), w.down)
        return self.mixer.mix(x), y2, x[:, w.gates]


class Bedenex(LayeredModel):

    def __init__(self, cfg: BedenexConfig, max_position: int, device, seed: int = 0):
        super().__init__(cfg)
        width = cfg.hidden_size
        self.final = nn.Parameter(torch.ones(width))
        self.loop_in = nn.Parameter(torch.empty(width, 2 * width)) if cfg.loop else None
        self.loop_step = nn.Parameter(torch.empty(cfg.loop.times, width)) if cfg.loop else None
        self.layer_weights = nn.ModuleList([LayerWeights(s, width) for s in cfg.layers])
        ropes = RopeTables(max_position, device)
        self.layers = [_Run(cfg.layers[i], self.layer_weights[i], ropes, cfg.norm_eps, begins) for i, begins in cfg.runs()]
        self.random_weights(device, seed)
        for spec, weights in zip(cfg.layers, self.layer_weights):
            if isinstance(spec.mixer, LatentSpec):
                weights.mix.by_head(spec.mixer)

    def load_tensors(self, take) -> None:
        width = self.cfg.hidden_size
        self.final.copy_(take("final.norm", (width,)))
        if self.loop_in is not None:
            self.loop_in.copy_(take("loop.in", self.loop_in.shape))
            self.loop_step.copy_(take("loop.step", self.loop_step.shape))
        for i, (spec, weights) in enumerate(zip(self.cfg.layers, self.layer_weights)):
            weights.load(spec, width, take, f"l{i}.")

    def forward_layers(self, input_ids, positions, hidden, residual, first: int, last: int):
        """``hidden`` between runs is (norm of the stream, or None where a pass begins; what a pass begins from: the stream |
        the embeddings in the model's element type)."""
        runs, eps, width = self.layers, self.cfg.norm_eps, self.cfg.hidden_size
        if first == 0:
            h, both, run = None, None, runs[0]
            if self.loop_in is not None:
                both = torch.empty((input_ids.numel(), 2 * width), dtype=self.embed.dtype, device=self.embed.device)
            if run.begins is None:
                residual, h, _ = embed_rms_norms(input_ids, self.embed, 1.0, (run.weights.norm1, None), eps, clear=run.counters,
                                                 copy=None if both is None else both[:, width:])
            else:
                residual, _, _ = embed_rms_norms(input_ids, self.embed, 1.0, (None, None), eps, out=both[:, :width], copy=both[:, width:])
            hidden = h, both
        h, both = hidden
        for i in range(first, last):
            run, w = runs[i], runs[i].weights
            if run.begins is not None:
                h = entry_rms_norm(project_f32(both, self.loop_in), self.loop_step[run.begins], residual, w.norm1, eps, clear=run.counters)
            y1, y2, gates = run.branches(h)
            if i + 1 == len(runs):
                return gated_rms_norm(residual, y1, y2, gates, w.gate_bias, self.final, eps, rows=get_context().logit_rows), residual
            nxt = runs[i + 1]
            if nxt.begins is None:
                h = gated_rms_norm(residual, y1, y2, gates, w.gate_bias, nxt.weights.norm1, eps, clear=nxt.counters)
            else:
                h = None
                gated_rms_norm(residual, y1, y2, gates, w.gate_bias, None, eps, out=both[:, :width])
        return (h, both), residual

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return F.linear(hidden, self.head)
