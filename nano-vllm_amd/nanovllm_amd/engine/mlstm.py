"""Matrix memory with exponential gates (the mLSTM of xLSTM): recurrent state in slots, gates from fp32 products."""
from __future__ import annotations

from dataclasses import dataclass

import torch
from torch import nn

from .. import _lib
from ..context import RowGroup, get_context
from .experts import linear_f32, project
from .mixers import _DTYPE, _ptr, _stream, scratch


def mlstm(qkvg: torch.Tensor, gate_logits: torch.Tensor, gate_bias: torch.Tensor, norm_weight: torch.Tensor, state: torch.Tensor,
          mass: torch.Tensor, top: torch.Tensor, group: RowGroup, out: torch.Tensor, q_scale: float, gate_cap: float, eps: float) -> None:
    """The recurrence with its gates, head norm and output gate; see ``nva_mlstm``."""
    slots, heads, dim, vdim = state.shape
    assert qkvg.stride(1) == 1 and qkvg.shape == (group.count, 2 * heads * (dim + vdim))
    assert gate_logits.dtype == torch.float32 and gate_logits.is_contiguous() and gate_logits.shape == (group.count, 2 * heads)
    assert gate_bias.dtype == torch.float32 and gate_bias.numel() == 2 * heads and norm_weight.numel() == heads * vdim and norm_weight.dtype == qkvg.dtype
    assert out.shape == (group.count, heads * vdim) and out.is_contiguous() and out.dtype == qkvg.dtype
    for t, shape in ((state, (slots, heads, dim, vdim)), (mass, (slots, heads, dim)), (top, (slots, heads))):
        assert t.shape == shape and t.dtype == torch.float32 and t.is_contiguous()
    lib, ws = _lib.load_latent(), None
    if group.cu is not None:
        nbytes = lib.nva_mlstm_workspace_bytes(group.num_seqs, group.max_q, heads, dim, vdim, _DTYPE[qkvg.dtype])
        ws = scratch(qkvg.device, nbytes) if nbytes else None
    rc = lib.nva_mlstm(
        qkvg.data_ptr(), qkvg.stride(0), gate_logits.data_ptr(), gate_bias.data_ptr(), norm_weight.data_ptr(), state.data_ptr(),
        mass.data_ptr(), top.data_ptr(), group.state_slots.data_ptr(), _ptr(group.cu), group.seq_lens.data_ptr(), out.data_ptr(), _ptr(ws),
        0 if ws is None else ws.numel(), group.count, group.num_seqs, group.max_q, heads, dim, vdim, slots, float(q_scale),
        float(gate_cap), float(eps), _DTYPE[qkvg.dtype], _stream())
    _lib.check(rc, "nva_mlstm")


@dataclass(frozen=True)
class MlstmSpec:
    heads: int
    dim: int
    vdim: int
    gate_cap: float


class MlstmWeights(nn.Module):
    """q, k, v and output gate projections fused along the output; input and forget gates likewise."""

    def __init__(self, spec: MlstmSpec, width: int):
        super().__init__()
        self.qkvg = nn.Parameter(torch.empty(2 * spec.heads * (spec.dim + spec.vdim), width))
        self.gates = nn.Parameter(torch.empty(2 * spec.heads, width))
        self.gate_bias = nn.Parameter(torch.zeros(2 * spec.heads, dtype=torch.float32))
        self.norm = nn.Parameter(torch.ones(spec.heads * spec.vdim))
        self.o = nn.Parameter(torch.empty(width, spec.heads * spec.vdim))

    def load(self, spec: MlstmSpec, width: int, take, prefix: str) -> None:
        qk, v, h = spec.heads * spec.dim, spec.heads * spec.vdim, spec.heads
        self.qkvg.copy_(torch.cat([take(f"{prefix}{n}", (size, width)) for n, size in (("q", qk), ("k", qk), ("v", v), ("g", v))]))
        self.gates.copy_(torch.cat([take(f"{prefix}{n}", (h, width)) for n in "if"]))
        self.gate_bias.copy_(torch.cat([take(f"{prefix}{n}.b", (h,)) for n in "if"]))
        self.norm.copy_(take(f"{prefix}norm", (v,)))
        self.o.copy_(take(f"{prefix}o", self.o.shape))


class Mlstm:
    """One layer's runtime: its recurrent state."""

    def __init__(self, spec: MlstmSpec, weights: MlstmWeights, eps: float):
        self.spec, self.weights, self.eps = spec, weights, eps
        self.state = self.mass = self.top = None

    def kv_elements_per_token(self) -> int:
        return 0

    def state_bytes_per_slot(self, elem_bytes: int) -> int:
        s = self.spec
        return s.heads * (s.dim * s.vdim + s.dim + 1) * 4

    def bind(self, num_blocks: int, block: int, slots: int, dtype: torch.dtype, device) -> None:
        s = self.spec
        zeros = lambda *shape: torch.zeros((slots, s.heads) + shape, dtype=torch.float32, device=device)
        self.state, self.mass, self.top = zeros(s.dim, s.vdim), zeros(s.dim), zeros()

    def unbind(self) -> None:
        self.state = self.mass = self.top = None

    def __call__(self, h: torch.Tensor) -> torch.Tensor:
        s, w = self.spec, self.weights
        qkvg, gates = project(h, w.qkvg), linear_f32(h, w.gates)
        o = torch.empty((h.shape[0], s.heads * s.vdim), dtype=h.dtype, device=h.device)
        for group in get_context().groups:
            rows = slice(group.first, group.first + group.count)
            mlstm(qkvg[rows], gates[rows], w.gate_bias, w.norm, self.state, self.mass, self.top, group, o[rows], s.dim ** -0.5, s.gate_cap, self.eps)
        return project(o, w.o)
