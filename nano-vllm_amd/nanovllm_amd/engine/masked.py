"""Grouped-query attention over a paged cache with what a design may ask for: a sliding window, chunks of positions or all
earlier keys, biases, norms of queries and keys (of every head, or over a whole projection; with weights or without) and of
values, rotary positions, a bias that grows with the logarithm of the distance, or no positions, a sink and an output gate per
head.  A layer may read another layer's keys and values.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple

import torch
from torch import nn

from .. import _lib
from ..context import RowGroup, get_context
from .experts import project
from .mixers import _DTYPE, Rotary, RopeTables, _ptr, _stream, scratch

ALL_KEYS = 1 << 30               # a window no sequence reaches

HEAD, WHOLE = "head", "whole"    # what a norm of queries and keys is taken over
UNIT = "unit"                    # over every head, without a weight
_NORMS = {None: 0, HEAD: 0, WHOLE: _lib.QKV_NORM_WHOLE, UNIT: _lib.QKV_NORM_UNIT}


def qkv_prepare(x: torch.Tensor, bias: Optional[torch.Tensor], q_norm: Optional[torch.Tensor], k_norm: Optional[torch.Tensor], qk_norm: Optional[str],
                rope: Optional[torch.Tensor], q_out: torch.Tensor, k_cache: Optional[torch.Tensor], v_cache: Optional[torch.Tensor],
                group: RowGroup, heads: int, kv_heads: int, dim: int, vdim: int, eps: float, v_norm: bool = False) -> None:
    """Bias, norms, rotation, cache write; see ``nva_qkv_prepare``."""
    cached, whole = k_cache is not None, qk_norm == WHOLE
    columns = heads * dim + (kv_heads * (dim + vdim) if cached else 0)
    assert x.stride(1) == 1 and x.shape[0] == group.count and x.shape[1] >= columns and q_out.shape == (group.count, heads * dim)
    assert q_out.is_contiguous() and q_out.dtype == x.dtype and (bias is None or (bias.numel() == columns and bias.dtype == x.dtype))
    for w, count in ((q_norm, heads), (k_norm, kv_heads)):
        assert w is None or (w.numel() == (count if whole else 1) * dim and w.dtype == x.dtype)
    if cached:
        assert k_cache.shape[2:] == (kv_heads, dim) and v_cache.shape == k_cache.shape[:3] + (vdim,) and group.slot_mapping.numel() == group.count
        assert k_cache.is_contiguous() and v_cache.is_contiguous() and k_cache.dtype == v_cache.dtype == x.dtype
    rot_dims, positions = (0, 0) if rope is None else (rope.shape[1], rope.shape[0])
    rc = _lib.load_shared().nva_qkv_prepare(
        x.data_ptr(), x.stride(0), _ptr(bias), _ptr(q_norm), _ptr(k_norm), _NORMS[qk_norm] | (_lib.QKV_NORM_VALUES if v_norm else 0), _ptr(rope), q_out.data_ptr(), _ptr(k_cache), _ptr(v_cache),
        group.slot_mapping.data_ptr(), k_cache.shape[0] * k_cache.shape[1] if cached else 0, _ptr(group.cu), group.seq_lens.data_ptr(),
        _ptr(group.token_seq), group.count, group.num_seqs, heads, kv_heads, dim, vdim, rot_dims, positions, float(eps), _DTYPE[x.dtype], _stream())
    _lib.check(rc, "nva_qkv_prepare")


def masked_attention(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, group: RowGroup, out: torch.Tensor, heads: int,
                     window: int, scale: float, sinks: Optional[torch.Tensor] = None, gate: Optional[torch.Tensor] = None,
                     softcap: float = 0.0, chunks: bool = False, bias: Optional[Tuple[torch.Tensor, torch.Tensor]] = None) -> None:
    """Softmax attention over the last ``window`` keys, or inside chunks of as many positions, over the paged cache; ``bias``: slopes
    and rates of a distance bias; see ``nva_masked_attn``."""
    num_blocks, block, kv_heads, dim = k_cache.shape
    vdim = v_cache.shape[3]
    assert q.stride(1) == 1 and q.shape == (group.count, heads * dim) and out.shape == (group.count, heads * vdim)
    assert out.is_contiguous() and q.dtype == out.dtype == k_cache.dtype == v_cache.dtype and k_cache.is_contiguous() and v_cache.is_contiguous()
    slope, rate = bias or (None, None)
    for x in (sinks, slope, rate):
        assert x is None or (x.dtype == torch.float32 and x.numel() == heads and x.is_contiguous())
    assert gate is None or (gate.shape == (group.count, heads) and gate.stride(1) == 1 and gate.dtype == q.dtype)
    table = group.block_tables
    assert table.dtype == torch.int32 and table.shape[0] == group.num_seqs and table.stride(1) == 1
    lib, ws = _lib.load_shared(), None
    if group.cu is None and q.dtype == torch.bfloat16:
        nbytes = lib.nva_chunk_attn_workspace_bytes(group.count, heads, kv_heads, vdim, table.shape[1], block, window)
        ws = scratch(q.device, nbytes) if nbytes else None
    rc = lib.nva_masked_attn(
        q.data_ptr(), q.stride(0), k_cache.data_ptr(), v_cache.data_ptr(), table.data_ptr(), table.stride(0), table.shape[1],
        _ptr(group.cu), group.seq_lens.data_ptr(), _ptr(group.token_seq), out.data_ptr(), _ptr(ws), 0 if ws is None else ws.numel(),
        group.count, group.num_seqs, group.max_q, heads, kv_heads, dim, vdim, block, num_blocks, _lib.MASK_CHUNKS if chunks else _lib.MASK_WINDOW, window, float(scale),
        float(softcap), _ptr(sinks), _ptr(slope), _ptr(rate), _ptr(gate), 0 if gate is None else gate.stride(0), _DTYPE[q.dtype], _stream())
    _lib.check(rc, "nva_masked_attn")


@dataclass(frozen=True)
class MaskedSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int] = None             # keys a query sees, its own included; None: all up to it
    rot: Optional[Rotary] = None             # pairs i, i + dims / 2
    qk_norm: Optional[str] = None            # HEAD, WHOLE, UNIT
    bias: bool = False                       # of the q, k and v projections
    sink: bool = False
    gate: bool = False
    kv_from: Optional[int] = None            # the layer whose keys and values this one reads
    chunk: Optional[int] = None              # positions of a chunk; a query sees no key of another one (excludes a window)
    distance_bias: bool = False              # slope ln(1 + rate d) off the score of a key that lies d back, slope and rate per head
    v_norm: bool = False                     # every head's values divided by their root mean square

    @property
    def qkv_rows(self) -> int:
        return self.heads * self.dim + (self.kv_heads * (self.dim + self.vdim) if self.kv_from is None else 0)

    def reads_like(self, other: "MaskedSpec") -> bool:
        """Whether this layer can read the other one's keys and values."""
        return (self.heads, self.kv_heads, self.dim, self.vdim, self.rot) == (other.heads, other.kv_heads, other.dim, other.vdim, other.rot)


class MaskedWeights(nn.Module):
    """Projections (query | key and value, if the layer has its own | gate) fused along the output, a multiple of 8 rows; and
    behind them ``beside`` rows of others that read the same input."""

    def __init__(self, spec: MaskedSpec, width: int, beside: int = 0):
        super().__init__()
        own, whole = spec.kv_from is None, spec.qk_norm == WHOLE
        rows = spec.qkv_rows + (spec.heads if spec.gate else 0)
        self.own_rows = -(-rows // 8) * 8
        self.qkvg = nn.Parameter(torch.zeros(self.own_rows + -(-beside // 8) * 8, width))
        self.bias = nn.Parameter(torch.zeros(spec.qkv_rows)) if spec.bias else None
        self.q_norm = nn.Parameter(torch.ones(spec.dim * (spec.heads if whole else 1))) if spec.qk_norm in (HEAD, WHOLE) else None
        self.k_norm = nn.Parameter(torch.ones(spec.dim * (spec.kv_heads if whole else 1))) if spec.qk_norm in (HEAD, WHOLE) and own else None
        self.sinks = nn.Parameter(torch.zeros(spec.heads, dtype=torch.float32)) if spec.sink else None
        self.slope, self.rate = (nn.Parameter(torch.zeros(spec.heads, dtype=torch.float32)) if spec.distance_bias else None for _ in range(2))
        self.o = nn.Parameter(torch.empty(width, spec.heads * spec.vdim))

    @property
    def projections(self) -> torch.Tensor:
        """All products of the layer's input; the mixer's own are the first ``own_rows``."""
        return self.qkvg

    def load(self, spec: MaskedSpec, width: int, take, prefix: str) -> None:
        parts = [("q", spec.heads * spec.dim)]
        if spec.kv_from is None:
            parts += [("k", spec.kv_heads * spec.dim), ("v", spec.kv_heads * spec.vdim)]
        rows = parts + ([("g", spec.heads)] if spec.gate else [])
        self.qkvg.zero_()
        self.qkvg[: sum(size for _, size in rows)].copy_(torch.cat([take(prefix + name, (size, width)) for name, size in rows]))
        if spec.bias:
            self.bias.copy_(torch.cat([take(f"{prefix}{name}.b", (size,)) for name, size in parts]))
        for norm, name in ((self.q_norm, "q.norm"), (self.k_norm, "k.norm")):
            if norm is not None:
                norm.copy_(take(prefix + name, norm.shape))
        if spec.sink:
            self.sinks.copy_(take(prefix + "sink", (spec.heads,)))
        if spec.distance_bias:
            self.slope.copy_(take(prefix + "r1", (spec.heads,)))
            self.rate.copy_(take(prefix + "r2", (spec.heads,)))
        self.o.copy_(take(prefix + "o", self.o.shape))


class MaskedAttention:
    """One layer's runtime: its share of the paged cache, or the layer whose share it reads."""

    def __init__(self, spec: MaskedSpec, weights: MaskedWeights, ropes: RopeTables, eps: float, source: Optional["MaskedAttention"] = None):
        self.spec, self.weights, self.eps, self.source = spec, weights, eps, source
        self.rope = None if spec.rot is None else ropes.get(spec.rot)
        self.span = min(spec.chunk or spec.window or ALL_KEYS, ALL_KEYS)
        self.bias = (weights.slope, weights.rate) if spec.distance_bias else None
        self.k_cache = self.v_cache = None

    def kv_elements_per_token(self) -> int:
        return self.spec.kv_heads * (self.spec.dim + self.spec.vdim) if self.source is None else 0

    def state_bytes_per_slot(self, elem_bytes: int) -> int:
        return 0

    def bind(self, num_blocks: int, block: int, slots: int, dtype: torch.dtype, device) -> None:
        s = self.spec
        if self.source is None:
            self.k_cache = torch.zeros((num_blocks, block, s.kv_heads, s.dim), dtype=dtype, device=device)
            self.v_cache = torch.zeros((num_blocks, block, s.kv_heads, s.vdim), dtype=dtype, device=device)

    def unbind(self) -> None:
        self.k_cache = self.v_cache = None

    def __call__(self, h: torch.Tensor) -> torch.Tensor:
        return self.mix(project(h, self.weights.qkvg))

    def mix(self, x: torch.Tensor) -> torch.Tensor:
        """The layer's result from the products of its input, whose first columns are its own."""
        s, w = self.spec, self.weights
        owner = self if self.source is None else self.source
        gate = x[:, s.qkv_rows: s.qkv_rows + s.heads] if s.gate else None
        q = torch.empty((x.shape[0], s.heads * s.dim), dtype=x.dtype, device=x.device)
        o = torch.empty((x.shape[0], s.heads * s.vdim), dtype=x.dtype, device=x.device)
        for group in get_context().groups:
            rows = slice(group.first, group.first + group.count)
            qkv_prepare(x[rows], w.bias, w.q_norm, w.k_norm, s.qk_norm, self.rope, q[rows], self.k_cache, self.v_cache, group,
                        s.heads, s.kv_heads, s.dim, s.vdim, self.eps, s.v_norm)
            masked_attention(q[rows], owner.k_cache, owner.v_cache, group, o[rows], s.heads, self.span, s.scale, w.sinks,
                             None if gate is None else gate[rows], chunks=s.chunk is not None, bias=self.bias)
        return project(o, w.o)
