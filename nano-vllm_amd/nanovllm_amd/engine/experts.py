"""Mixture of experts: a router in fp32 (softmax or sigmoids) and small gated feed-forwards of which every row uses the best
few, weighted on their results or on what they read; optionally a shared expert that every row runs, behind a gate of its own.

Nothing depends on the host knowing how many rows an expert has: the router leaves lists of assignments, and the
products walk them, so a step with experts is captured into a graph like any other."""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Optional

import torch
import torch.nn.functional as F
from torch import nn

from .. import _lib
from .mixers import _DTYPE, _need_cuda, _ptr, _stream, clamped_gate, squared_relu_


@dataclass(frozen=True)
class GateForm:
    """``g sigmoid(slope g) (u + shift)`` with ``g = min(gate, limit)``, ``u = clamp(up, -limit, limit)``."""
    limit: float = math.inf
    slope: float = 1.0
    shift: float = 0.0


SILU = GateForm()
SOFTMAX, SIGMOID = "softmax", "sigmoid"       # weights: softmax over the chosen logits; their sigmoids as they are
_SCORES = {SOFTMAX: _lib.SCORE_SOFTMAX, SIGMOID: _lib.SCORE_SIGMOID}
JOIN_ROWS = 256                  # rows up to which a shared expert runs in the launches of the routed ones


def grouped_linear(x: torch.Tensor, weight: torch.Tensor, out: torch.Tensor, squared_relu: bool = False) -> torch.Tensor:
    """``out[r, g] = weight[g] @ x[r, g]``; ``x [n, groups, k]`` and ``out [n, groups, n_out]`` may be strided views."""
    groups, n_out, k = weight.shape
    assert x.shape[1:] == (groups, k) and out.shape == (x.shape[0], groups, n_out) and x.stride(2) == out.stride(2) == 1
    assert weight.is_contiguous() and weight.dtype == x.dtype
    _need_cuda(x, weight)
    rc = _lib.load_shared().nva_grouped_linear(x.data_ptr(), x.stride(0), x.stride(1), weight.data_ptr(), out.data_ptr(), out.stride(0),
                                               out.stride(1), x.shape[0], groups, n_out, k, int(squared_relu), _DTYPE[x.dtype], _DTYPE[out.dtype], _stream())
    _lib.check(rc, "nva_grouped_linear")
    return out


def linear_f32(x: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    """``x @ weight.T`` with few outputs, kept in fp32."""
    out = torch.empty((x.shape[0], weight.shape[0]), dtype=torch.float32, device=x.device)
    grouped_linear(x[:, None], weight[None], out[:, None])
    return out


def streams(x: torch.Tensor, weight: torch.Tensor) -> bool:
    """Whether ``x @ weight.T`` has so few rows that the kernel that streams the weights once is faster than the library's."""
    n, k = x.shape
    return x.dtype == torch.bfloat16 and (n <= 16 and weight.numel() <= 1 << 24 or n <= 64 and k <= 1024)


def project(x: torch.Tensor, weight: torch.Tensor, squared_relu: bool = False) -> torch.Tensor:
    """``x @ weight.T``, or ``max(x @ weight.T, 0)^2``."""
    if not streams(x, weight):
        y = F.linear(x, weight)
        return squared_relu_(y) if squared_relu else y
    out = torch.empty((x.shape[0], weight.shape[0]), dtype=x.dtype, device=x.device)
    grouped_linear(x[:, None], weight[None], out[:, None], squared_relu)
    return out


def project_f32(x: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    """``x @ weight.T`` whose fp32 sums are kept."""
    if x.dtype == torch.float32:
        return F.linear(x, weight)
    if streams(x, weight):
        return linear_f32(x, weight)
    return torch.mm(x, weight.t(), out_dtype=torch.float32)


@dataclass
class Assignments:
    choice: torch.Tensor         # int32 [n, top], best first
    weight: torch.Tensor         # fp32 [n, top + gates]: the choices' weights, the gates' sigmoids
    lists: torch.Tensor          # int32 [experts, n]: row * top + k of every assignment
    counts: torch.Tensor         # int32 [experts]


def route(h: torch.Tensor, router: torch.Tensor, top: int, scale: float, counts: torch.Tensor, bias: Optional[torch.Tensor] = None,
          gates: int = 0, score: str = SOFTMAX) -> Assignments:
    """Router of ``h [n, width]``, ``router [experts + gates, width]``; ``counts`` (int32 ``[experts]``) must be zero."""
    n, width = h.shape
    experts = router.shape[0] - gates
    assert h.stride(1) == 1 and router.is_contiguous() and router.shape[1] == width and router.dtype == h.dtype
    assert counts.dtype == torch.int32 and counts.numel() == experts
    assert bias is None or (bias.dtype == torch.float32 and bias.numel() == router.shape[0] and bias.is_contiguous())
    _need_cuda(h, router)
    i32 = lambda *shape: torch.empty(shape, dtype=torch.int32, device=h.device)
    a = Assignments(i32(n, top), torch.empty((n, top + gates), dtype=torch.float32, device=h.device), i32(experts, n), counts)
    rc = _lib.load_shared().nva_router(h.data_ptr(), h.stride(0), router.data_ptr(), _ptr(bias), a.choice.data_ptr(), a.weight.data_ptr(),
                                       a.lists.data_ptr(), counts.data_ptr(), n, n, width, experts, gates, top, _SCORES[score], float(scale),
                                       _DTYPE[h.dtype], _stream())
    _lib.check(rc, "nva_router")
    return a


def routed_linear(x: torch.Tensor, weight: torch.Tensor, a: Assignments, gate: Optional[GateForm], shared=None, weigh_input: bool = False):
    """One product per assignment, ``[n * top, n_out]``: of row ``p // top`` of ``x [n, k]``, or of row ``p`` of
    ``x [n * top, k]``.  With ``gate`` the weights are (gate | up) and the result has its form.
    ``weigh_input``: as if every assignment's row were multiplied by its weight first (with ``gate``).
    ``shared = (x [n, k'], weight, limit)``: a product of every row with a weight of its own in the same launch (few rows);
    then both results are returned."""
    experts, rows, k = weight.shape
    n, top = a.choice.shape
    assert x.stride(1) == 1 and x.shape[1] == k and x.shape[0] in (n, n * top) and weight.is_contiguous() and weight.dtype == x.dtype
    n_out = rows if gate is None else rows // 2
    out = torch.empty((n * top, n_out), dtype=x.dtype, device=x.device)
    form = gate or SILU
    args = (x.data_ptr(), x.stride(0), weight.data_ptr(), out.data_ptr(), a.lists.data_ptr(), a.counts.data_ptr(), a.lists.stride(0), n, top,
            experts, n_out, k, int(x.shape[0] == n), int(gate is not None), form.limit, form.slope, form.shift)
    assert not weigh_input or (gate is not None and shared is None)
    if shared is None:
        weigh = (a.weight.data_ptr(), a.weight.stride(0)) if weigh_input else (None, 0)
        _lib.check(_lib.load_shared().nva_routed_linear(*args, *weigh, _DTYPE[x.dtype], _stream()), "nva_routed_linear")
        return out
    xs, ws, limit = shared
    assert xs.shape == (n, ws.shape[1]) and xs.stride(1) == 1 and ws.is_contiguous() and xs.dtype == ws.dtype == x.dtype == torch.bfloat16
    beside = torch.empty((n, ws.shape[0] if gate is None else ws.shape[0] // 2), dtype=x.dtype, device=x.device)
    rc = _lib.load_shared().nva_routed_shared_linear(*args, xs.data_ptr(), xs.stride(0), ws.data_ptr(), beside.data_ptr(), beside.shape[1],
                                                     ws.shape[1], limit, _stream())
    _lib.check(rc, "nva_routed_shared_linear")
    return out, beside


@dataclass(frozen=True)
class SharedExpertSpec:
    ff: int
    gate: GateForm


@dataclass(frozen=True)
class ExpertsSpec:
    experts: int
    top: int
    ff: int
    scale: float = 1.0
    gate: GateForm = SILU
    bias: bool = False                            # of the router
    shared: Optional[SharedExpertSpec] = None
    score: str = SOFTMAX
    weigh_input: bool = False                     # the weights belong to what the experts read


class ExpertWeights(nn.Module):
    """The gate of the shared expert is one more row of the router."""

    def __init__(self, spec: ExpertsSpec, width: int):
        super().__init__()
        rows = spec.experts + (spec.shared is not None)
        self.router = nn.Parameter(torch.empty(rows, width))
        self.bias = nn.Parameter(torch.zeros(rows, dtype=torch.float32)) if spec.bias else None
        self.gate_up = nn.Parameter(torch.empty(spec.experts, 2 * spec.ff, width))
        self.down = nn.Parameter(torch.empty(spec.experts, width, spec.ff))
        self.shared_gate_up = self.shared_down = None
        if spec.shared is not None:
            self.shared_gate_up = nn.Parameter(torch.empty(2 * spec.shared.ff, width))
            self.shared_down = nn.Parameter(torch.empty(width, spec.shared.ff))

    def load(self, spec: ExpertsSpec, width: int, take, prefix: str) -> None:
        self.router[: spec.experts].copy_(take(f"{prefix}router", (spec.experts, width)))
        if spec.bias:
            self.bias.zero_()
            self.bias[: spec.experts].copy_(take(f"{prefix}router.b", (spec.experts,)))
        for e in range(spec.experts):
            for part, name in enumerate(("gate", "up")):
                self.gate_up[e, part * spec.ff: (part + 1) * spec.ff].copy_(take(f"{prefix}e{e}.{name}", (spec.ff, width)))
            self.down[e].copy_(take(f"{prefix}e{e}.down", (width, spec.ff)))
        if spec.shared is not None:
            self.router[spec.experts:].copy_(take(f"{prefix}shared.sg", (1, width)))
            self.shared_gate_up.copy_(torch.cat([take(f"{prefix}shared.{name}", (spec.shared.ff, width)) for name in ("gate", "up")]))
            self.shared_down.copy_(take(f"{prefix}shared.down", (width, spec.shared.ff)))


class Experts:
    """One layer's runtime.  ``counters`` have to be zero when it is called (the norm before it sees to that)."""

    def __init__(self, spec: ExpertsSpec, weights: ExpertWeights, device):
        self.spec, self.weights = spec, weights
        self.counters = torch.zeros(spec.experts, dtype=torch.int32, device=device)

    def __call__(self, h: torch.Tensor):
        """The chosen experts' outputs ``[n * top, width]``, the shared one's ``[n, width]`` (or None), and their weights: ``[n, top]``
        and, as one more column, the shared expert's.  (With ``weigh_input`` the outputs are only to be added.)"""
        s, w = self.spec, self.weights
        a = route(h, w.router, s.top, s.scale, self.counters, w.bias, w.router.shape[0] - s.experts, s.score)
        if s.shared is None:
            return routed_linear(routed_linear(h, w.gate_up, a, s.gate, weigh_input=s.weigh_input), w.down, a, None), None, a.weight
        form = s.shared.gate
        assert not s.weigh_input
        assert (form.slope, form.shift) == (s.gate.slope, s.gate.shift) and form.shift == 1.0
        if self._joins(h):
            mid, shared = routed_linear(h, w.gate_up, a, s.gate, (h, w.shared_gate_up, form.limit))
            return (*routed_linear(mid, w.down, a, None, (shared, w.shared_down, 0.0)), a.weight)
        shared = project(clamped_gate(project(h, w.shared_gate_up), form.limit, form.slope), w.shared_down)
        return routed_linear(routed_linear(h, w.gate_up, a, s.gate), w.down, a, None), shared, a.weight

    def _joins(self, h: torch.Tensor) -> bool:
        """Whether the shared expert runs in the launches of the routed ones."""
        n, width = h.shape
        return h.dtype == torch.bfloat16 and n <= JOIN_ROWS and width % 8 == self.spec.ff % 8 == self.spec.shared.ff % 8 == 0
