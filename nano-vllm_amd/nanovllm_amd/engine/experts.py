"""Mixture of experts: a softmax router in fp32 and small gated (SiLU) feed-forwards of which every row uses the best few.

Nothing depends on the host knowing how many rows an expert has: the router leaves lists of assignments, and the
products walk them, so a step with experts is captured into a graph like any other."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Tuple

import torch
import torch.nn.functional as F
from torch import nn

from .. import _lib
from .mixers import _DTYPE, _need_cuda, _stream


def grouped_linear(x: torch.Tensor, weight: torch.Tensor, out: torch.Tensor) -> torch.Tensor:
    """``out[r, g] = weight[g] @ x[r, g]``; ``x [n, groups, k]`` and ``out [n, groups, n_out]`` may be strided views."""
    groups, n_out, k = weight.shape
    assert x.shape[1:] == (groups, k) and out.shape == (x.shape[0], groups, n_out) and x.stride(2) == out.stride(2) == 1
    assert weight.is_contiguous() and weight.dtype == x.dtype
    _need_cuda(x, weight)
    rc = _lib.load_latent().nva_grouped_linear(x.data_ptr(), x.stride(0), x.stride(1), weight.data_ptr(), out.data_ptr(), out.stride(0),
                                               out.stride(1), x.shape[0], groups, n_out, k, _DTYPE[x.dtype], _DTYPE[out.dtype], _stream())
    _lib.check(rc, "nva_grouped_linear")
    return out


def linear_f32(x: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    """``x @ weight.T`` with few outputs, kept in fp32."""
    out = torch.empty((x.shape[0], weight.shape[0]), dtype=torch.float32, device=x.device)
    grouped_linear(x[:, None], weight[None], out[:, None])
    return out


def project(x: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    """``x @ weight.T``: the library's product, or for few rows the kernel that streams the weights once, where it is faster."""
    n, k = x.shape
    few = n <= 16 and weight.numel() <= 1 << 24 or n <= 64 and k <= 1024
    if not few or x.dtype != torch.bfloat16:
        return F.linear(x, weight)
    out = torch.empty((n, weight.shape[0]), dtype=x.dtype, device=x.device)
    grouped_linear(x[:, None], weight[None], out[:, None])
    return out


@dataclass
class Assignments:
    choice: torch.Tensor         # int32 [n, top], best first
    weight: torch.Tensor         # fp32 [n, top]
    lists: torch.Tensor          # int32 [experts, n]: row * top + k of every assignment
    counts: torch.Tensor         # int32 [experts]


def route(h: torch.Tensor, router: torch.Tensor, top: int, scale: float, counts: torch.Tensor) -> Assignments:
    """Router of ``h [n, width]``; ``counts`` (int32 ``[experts]``) must be zero."""
    n, width = h.shape
    experts = router.shape[0]
    assert h.stride(1) == 1 and router.is_contiguous() and router.shape[1] == width and router.dtype == h.dtype
    assert counts.dtype == torch.int32 and counts.numel() == experts
    _need_cuda(h, router)
    i32 = lambda *shape: torch.empty(shape, dtype=torch.int32, device=h.device)
    a = Assignments(i32(n, top), torch.empty((n, top), dtype=torch.float32, device=h.device), i32(experts, n), counts)
    rc = _lib.load_latent().nva_router(h.data_ptr(), h.stride(0), router.data_ptr(), a.choice.data_ptr(), a.weight.data_ptr(),
                                       a.lists.data_ptr(), counts.data_ptr(), n, n, width, experts, top, float(scale), _DTYPE[h.dtype],
                                       _stream())
    _lib.check(rc, "nva_router")
    return a


def routed_linear(x: torch.Tensor, weight: torch.Tensor, a: Assignments, gated: bool) -> torch.Tensor:
    """One product per assignment, ``[n * top, n_out]``: of row ``p // top`` of ``x [n, k]``, or of row ``p`` of
    ``x [n * top, k]``.  ``gated``: the weights are (gate | up), the result is silu(gate) * up."""
    experts, rows, k = weight.shape
    n, top = a.choice.shape
    assert x.stride(1) == 1 and x.shape[1] == k and x.shape[0] in (n, n * top) and weight.is_contiguous() and weight.dtype == x.dtype
    n_out = rows // 2 if gated else rows
    out = torch.empty((n * top, n_out), dtype=x.dtype, device=x.device)
    rc = _lib.load_latent().nva_routed_linear(x.data_ptr(), x.stride(0), weight.data_ptr(), out.data_ptr(), a.lists.data_ptr(),
                                              a.counts.data_ptr(), a.lists.stride(0), n, top, experts, n_out, k, int(x.shape[0] == n), int(gated),
                                              _DTYPE[x.dtype], _stream())
    _lib.check(rc, "nva_routed_linear")
    return out


@dataclass(frozen=True)
class ExpertsSpec:
    experts: int
    top: int
    ff: int
    scale: float


class ExpertWeights(nn.Module):

    def __init__(self, spec: ExpertsSpec, width: int):
        super().__init__()
        self.router = nn.Parameter(torch.empty(spec.experts, width))
        self.gate_up = nn.Parameter(torch.empty(spec.experts, 2 * spec.ff, width))
        self.down = nn.Parameter(torch.empty(spec.experts, width, spec.ff))

    def load(self, spec: ExpertsSpec, width: int, take, prefix: str) -> None:
        self.router.copy_(take(f"{prefix}router", self.router.shape))
        for e in range(spec.experts):
            for part, name in enumerate(("gate", "up")):
                self.gate_up[e, part * spec.ff: (part + 1) * spec.ff].copy_(take(f"{prefix}e{e}.{name}", (spec.ff, width)))
            self.down[e].copy_(take(f"{prefix}e{e}.down", (width, spec.ff)))


class Experts:
    """One layer's runtime.  ``counters`` have to be zero when it is called (the norm before it sees to that)."""

    def __init__(self, spec: ExpertsSpec, weights: ExpertWeights, device):
        self.spec, self.weights = spec, weights
        self.counters = torch.zeros(spec.experts, dtype=torch.int32, device=device)

    def __call__(self, h: torch.Tensor) -> Tuple[torch.Tensor, torch.Tensor]:
        """The chosen experts' outputs ``[n * top, width]`` and their weights ``[n, top]``."""
        w = self.weights
        a = route(h, w.router, self.spec.top, self.spec.scale, self.counters)
        return routed_linear(routed_linear(h, w.gate_up, a, True), w.down, a, False), a.weight
