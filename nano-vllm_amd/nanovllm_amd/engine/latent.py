"""Latent attention: keys and values through a low-rank latent, queries through one of their own or directly, a rotated key
part shared by all heads, a sliding window or all earlier keys, a sink and a sigmoid gate per head where asked for.  The cache
holds one row (latent | rotated part) per token; a layer may read another layer's.

Single tokens and short portions meet the cached latents directly (the query goes through the key product's
transpose, the result through the value product); longer portions gather the visible latents and multiply them
out first.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional

import torch
import torch.nn.functional as F
from torch import nn

from .. import _lib
from ..context import RowGroup, get_context
from .experts import grouped_linear, project
from .mixers import _DTYPE, Rotary, RopeTables, _ptr, _stream, scratch

EXPAND_FROM = 32                 # rows a gathered key has to serve on average before multiplying it out pays
EXPAND_MAX_KEYS = 1 << 17        # keys multiplied out at a time, at most


def latent_prepare(x: torch.Tensor, q_norm: Optional[torch.Tensor], kv_norm: Optional[torch.Tensor], rope: torch.Tensor, q_out: Optional[torch.Tensor],
                   cache: Optional[torch.Tensor], group: RowGroup, rot_dim: int, eps: float) -> None:
    """Query latents (with ``q_out``) and, with a cache, what the rows leave behind in it; see ``nva_latent_prepare``."""
    q_rank = 0 if q_out is None else q_out.shape[1]
    rank = 0 if cache is None else cache.shape[2] - rot_dim
    assert x.stride(1) == 1 and x.shape[0] == group.count and x.shape[1] >= q_rank + (rank + rot_dim if cache is not None else 0)
    assert rope.shape[1] == rot_dim
    assert q_out is None or (q_out.is_contiguous() and q_out.shape[0] == group.count and q_out.dtype == x.dtype == q_norm.dtype)
    if cache is not None:
        assert cache.is_contiguous() and cache.dtype == x.dtype and kv_norm.numel() == rank and group.slot_mapping.numel() == group.count
    rc = _lib.load_shared().nva_latent_prepare(
        x.data_ptr(), x.stride(0), _ptr(q_norm), _ptr(kv_norm), rope.data_ptr(), _ptr(q_out), _ptr(cache),
        group.slot_mapping.data_ptr(), 0 if cache is None else cache.shape[0] * cache.shape[1], _ptr(group.cu), group.seq_lens.data_ptr(),
        _ptr(group.token_seq), group.count, group.num_seqs, q_rank, rank, rot_dim, rope.shape[0], float(eps), _DTYPE[x.dtype], _stream())
    _lib.check(rc, "nva_latent_prepare")


def latent_attention(q_latent: torch.Tensor, q_rot: torch.Tensor, gate: Optional[torch.Tensor], rope: torch.Tensor, cache: torch.Tensor,
                     group: RowGroup, out: torch.Tensor, window: int, scale: float, sinks: Optional[torch.Tensor] = None) -> None:
    """Attention over the cached latents; ``q_latent`` and ``out [n, heads, rank]``; see ``nva_latent_attn``."""
    n, heads, rank = q_latent.shape
    num_blocks, block, width = cache.shape
    rot, table, window = width - rank, group.block_tables, min(window, 1 << 30)
    assert n == group.count and q_latent.is_contiguous() and out.shape == q_latent.shape and out.is_contiguous()
    assert q_rot.shape == (n, heads, rot) and q_rot.stride(2) == 1
    _check_gate_and_sinks(gate, sinks, n, heads, cache.dtype)
    assert q_latent.dtype == q_rot.dtype == cache.dtype == out.dtype and cache.is_contiguous() and rope.shape[1] == rot
    assert table.dtype == torch.int32 and table.shape[0] == group.num_seqs and table.stride(1) == 1
    lib, dtype = _lib.load_shared(), _DTYPE[cache.dtype]
    nbytes = lib.nva_latent_attn_workspace_bytes(n, heads, rank, rot, table.shape[1], block, window, dtype)
    ws = scratch(out.device, nbytes) if nbytes else None
    rc = lib.nva_latent_attn(
        q_latent.data_ptr(), q_rot.data_ptr(), q_rot.stride(0), q_rot.stride(1), _ptr(gate), 0 if gate is None else gate.stride(0), _ptr(sinks),
        rope.data_ptr(), cache.data_ptr(), table.data_ptr(), table.stride(0), table.shape[1], _ptr(group.cu), group.seq_lens.data_ptr(), _ptr(group.token_seq),
        out.data_ptr(), _ptr(ws), 0 if ws is None else ws.numel(), n, group.num_seqs, heads, rank, rot, block, num_blocks, window,
        rope.shape[0], float(scale), dtype, _stream())
    _lib.check(rc, "nva_latent_attn")


def _check_gate_and_sinks(gate: Optional[torch.Tensor], sinks: Optional[torch.Tensor], n: int, heads: int, dtype: torch.dtype) -> None:
    assert gate is None or (gate.shape == (n, heads) and gate.stride(1) == 1 and gate.dtype == dtype)
    assert sinks is None or (sinks.dtype == torch.float32 and sinks.numel() == heads and sinks.is_contiguous())


def latent_gather(cache: torch.Tensor, group: RowGroup, key_cu: torch.Tensor, n_keys: int) -> torch.Tensor:
    """The cache rows of the last ``key_cu[s + 1] - key_cu[s]`` tokens of every sequence, ``[n_keys, width]``."""
    num_blocks, block, width = cache.shape
    out = torch.empty((n_keys, width), dtype=cache.dtype, device=cache.device)
    table = group.block_tables
    assert key_cu.dtype == torch.int32 and key_cu.numel() == group.num_seqs + 1 and cache.is_contiguous()
    rc = _lib.load_shared().nva_latent_gather(cache.data_ptr(), table.data_ptr(), table.stride(0), table.shape[1], key_cu.data_ptr(),
                                              group.seq_lens.data_ptr(), out.data_ptr(), n_keys, group.num_seqs, width, block, num_blocks,
                                              _DTYPE[cache.dtype], _stream())
    _lib.check(rc, "nva_latent_gather")
    return out


def latent_prefill(q: torch.Tensor, kv: torch.Tensor, k_rot: torch.Tensor, gate: Optional[torch.Tensor], rope: torch.Tensor, group: RowGroup,
                   key_cu: torch.Tensor, out: torch.Tensor, dim: int, vdim: int, window: int, scale: float,
                   sinks: Optional[torch.Tensor] = None) -> None:
    """Attention of portions over keys and values multiplied out; see ``nva_latent_prefill``."""
    n, heads = q.shape[0], out.shape[1] // vdim
    _check_gate_and_sinks(gate, sinks, n, heads, q.dtype)
    rot, window = k_rot.shape[1], min(window, 1 << 30)
    assert n == group.count and q.shape == (n, heads * (dim + rot)) and q.stride(1) == 1 and out.shape == (n, heads * vdim) and out.is_contiguous()
    assert kv.shape[1] == heads * (dim + vdim) and kv.stride(1) == 1 and k_rot.shape[0] == kv.shape[0] and k_rot.stride(1) == 1
    assert q.dtype == kv.dtype == k_rot.dtype == out.dtype and rope.shape[1] == rot and group.cu is not None
    rc = _lib.load_shared().nva_latent_prefill(
        q.data_ptr(), q.stride(0), kv.data_ptr(), kv.stride(0), k_rot.data_ptr(), k_rot.stride(0), _ptr(gate), 0 if gate is None else gate.stride(0), _ptr(sinks),
        rope.data_ptr(), group.cu.data_ptr(), group.seq_lens.data_ptr(), key_cu.data_ptr(), out.data_ptr(), n, group.num_seqs, group.max_q,
        heads, dim, rot, vdim, window, rope.shape[0], float(scale), _DTYPE[q.dtype], _stream())
    _lib.check(rc, "nva_latent_prefill")


def visible_keys(group: RowGroup, window: int, device):
    """Keys the group's portions see, as ``(key_cu, n_keys)``, if multiplying them out pays; None otherwise.
    Formed once per step and window."""
    if group.cu is None or group.spans is None:
        return None
    if ("keys", window) not in group.shared:
        counts = [min(start, window - 1) + count for start, count in group.spans]
        n_keys = sum(counts)
        found = None
        if n_keys <= EXPAND_MAX_KEYS and sum(c * k for (_, c), k in zip(group.spans, counts)) >= EXPAND_FROM * n_keys:
            cu = torch.tensor([0] + counts, dtype=torch.int64).cumsum(0).to(torch.int32)
            found = cu.pin_memory().to(device, non_blocking=True), n_keys
        group.shared[("keys", window)] = found
    return group.shared[("keys", window)]


@dataclass(frozen=True)
class LatentSpec:
    heads: int
    dim: int                     # unrotated query / key elements per head
    rot_dim: int                 # rotated ones
    vdim: int
    q_rank: int                  # 0: queries straight from the layer's input
    kv_rank: int
    window: Optional[int]        # None: all earlier keys
    scale: float
    rot: Rotary
    kv_from: Optional[int] = None            # the layer whose cache this one reads
    gate: bool = True
    sink: bool = False
    halves: bool = False         # rotated pairs are i and i + rot_dim / 2 of the given weights (laid side by side when they are loaded)

    @property
    def query_rows(self) -> int:
        """Columns of the query latent, or of the queries, in the first product of the input."""
        return self.q_rank or self.heads * (self.dim + self.rot_dim)

    @property
    def down_rows(self) -> int:
        return self.query_rows + (self.kv_rank + self.rot_dim if self.kv_from is None else 0) + (self.heads if self.gate else 0)

    def paired(self, rows: torch.Tensor) -> torch.Tensor:
        """Rows of a product whose results are rotated: the partners of a pair next to one another.  (Queries and keys are laid out
        alike, so no score changes.)"""
        return torch.stack(rows.chunk(2), 1).flatten(0, 1) if self.halves else rows


class LatentWeights(nn.Module):
    """Down projections (query latent, or queries | latent and rotated key part, if the layer has its own | gate) fused along
    the output and padded to a multiple of 8, behind them ``beside`` rows of others that read the same input; the key and value products stacked for keys multiplied out, and
    head by head for the absorbed form (the key product transposed)."""

    def __init__(self, spec: LatentSpec, width: int, beside: int = 0):
        super().__init__()
        h = spec.heads
        self.own_rows = -(-spec.down_rows // 8) * 8
        self.down = nn.Parameter(torch.zeros(self.own_rows + -(-beside // 8) * 8, width))
        self.q_norm = nn.Parameter(torch.ones(spec.q_rank)) if spec.q_rank else None
        self.uq = nn.Parameter(torch.empty(h * (spec.dim + spec.rot_dim), spec.q_rank)) if spec.q_rank else None
        self.kv_norm = nn.Parameter(torch.ones(spec.kv_rank)) if spec.kv_from is None else None
        self.ukv = nn.Parameter(torch.empty(h * (spec.dim + spec.vdim), spec.kv_rank))
        self.uk_t = nn.Parameter(torch.empty(h, spec.kv_rank, spec.dim))
        self.uv = nn.Parameter(torch.empty(h, spec.vdim, spec.kv_rank))
        self.sinks = nn.Parameter(torch.zeros(h, dtype=torch.float32)) if spec.sink else None
        self.o = nn.Parameter(torch.empty(width, h * spec.vdim))

    @property
    def projections(self) -> torch.Tensor:
        """All products of the layer's input; the mixer's own are the first ``own_rows``."""
        return self.down

    def load(self, spec: LatentSpec, width: int, take, prefix: str) -> None:
        h, own = spec.heads, spec.kv_from is None
        queries = lambda name, size: torch.cat([torch.cat([x[: spec.dim], spec.paired(x[spec.dim:])])
                                                for x in take(prefix + name, (h * (spec.dim + spec.rot_dim), size)).chunk(h)])
        parts = [take(prefix + "dq", (spec.q_rank, width)) if spec.q_rank else queries("q", width)]
        if own:
            dkv = take(prefix + "dkv", (spec.kv_rank + spec.rot_dim, width))
            parts += [dkv[: spec.kv_rank], spec.paired(dkv[spec.kv_rank:])]
            self.kv_norm.copy_(take(prefix + "dkv.norm", (spec.kv_rank,)))
        if spec.gate:
            parts.append(take(prefix + "g", (h, width)))
        self.down.zero_()
        self.down[: spec.down_rows].copy_(torch.cat(parts))
        if spec.q_rank:
            self.q_norm.copy_(take(prefix + "dq.norm", (spec.q_rank,)))
            self.uq.copy_(queries("uq", spec.q_rank))
        if spec.sink:
            self.sinks.copy_(take(prefix + "sink", (h,)))
        self.ukv.copy_(torch.cat([take(prefix + "uk", (h * spec.dim, spec.kv_rank)), take(prefix + "uv", (h * spec.vdim, spec.kv_rank))]))
        self.by_head(spec)
        self.o.copy_(take(prefix + "o", self.o.shape))

    @torch.no_grad()
    def by_head(self, spec: LatentSpec) -> None:
        """The absorbed form's copies of the key and value products."""
        uk, uv = self.ukv.split([spec.heads * spec.dim, spec.heads * spec.vdim])
        self.uk_t.copy_(uk.view(spec.heads, spec.dim, spec.kv_rank).transpose(1, 2))
        self.uv.copy_(uv.view(spec.heads, spec.vdim, spec.kv_rank))


class LatentAttention:
    """One layer's runtime: its share of the paged cache, or the layer whose share it reads."""

    def __init__(self, spec: LatentSpec, weights: LatentWeights, ropes: RopeTables, eps: float, source: Optional["LatentAttention"] = None):
        self.spec, self.weights, self.eps, self.source = spec, weights, eps, source
        self.rope = ropes.get(spec.rot)
        self.window = spec.window or 1 << 30
        self.cache = None

    def kv_elements_per_token(self) -> int:
        return self.spec.kv_rank + self.spec.rot_dim if self.source is None else 0

    def state_bytes_per_slot(self, elem_bytes: int) -> int:
        return 0

    def bind(self, num_blocks: int, block: int, slots: int, dtype: torch.dtype, device) -> None:
        if self.source is None:
            self.cache = torch.zeros((num_blocks, block, self.spec.kv_rank + self.spec.rot_dim), dtype=dtype, device=device)

    def unbind(self) -> None:
        self.cache = None

    def __call__(self, h: torch.Tensor) -> torch.Tensor:
        return self.mix(project(h, self.weights.down))

    def mix(self, down: torch.Tensor) -> torch.Tensor:
        """The layer's result from the products of its input, whose first columns are its own."""
        s, w, n = self.spec, self.weights, down.shape[0]
        cache = self.cache if self.source is None else self.source.cache
        gate = down[:, s.down_rows - s.heads: s.down_rows] if s.gate else None
        empty = lambda *shape: torch.empty(shape, dtype=down.dtype, device=down.device)
        q_latent, o = empty(n, s.q_rank) if s.q_rank else None, empty(n, s.heads * s.vdim)
        groups = [(g, slice(g.first, g.first + g.count)) for g in get_context().groups]
        for group, rows in groups:
            if s.q_rank:
                latent_prepare(down[rows], w.q_norm, w.kv_norm, self.rope, q_latent[rows], self.cache, group, s.rot_dim, self.eps)
            elif self.source is None:
                latent_prepare(down[rows, s.query_rows:], None, w.kv_norm, self.rope, None, self.cache, group, s.rot_dim, self.eps)
        q = project(q_latent, w.uq) if s.q_rank else down[:, : s.query_rows]
        expands = down.dtype == torch.bfloat16 and _lib.load_shared().nva_latent_prefill_supported(s.dim, s.rot_dim, s.vdim, _DTYPE[down.dtype])
        for group, rows in groups:
            keys = visible_keys(group, self.window, down.device) if expands else None
            head_gates = None if gate is None else gate[rows]
            if keys is not None:
                key_cu, n_keys = keys
                latents = latent_gather(cache, group, key_cu, n_keys)
                latent_prefill(q[rows], F.linear(latents[:, : s.kv_rank], w.ukv), latents[:, s.kv_rank:], head_gates, self.rope, group, key_cu,
                               o[rows], s.dim, s.vdim, self.window, s.scale, w.sinks)
                continue
            heads = q[rows].unflatten(1, (s.heads, s.dim + s.rot_dim))
            met = grouped_linear(heads[..., : s.dim], w.uk_t, empty(group.count, s.heads, s.kv_rank))
            mixed = empty(group.count, s.heads, s.kv_rank)
            latent_attention(met, heads[..., s.dim:], head_gates, self.rope, cache, group, mixed, self.window, s.scale, w.sinks)
            grouped_linear(mixed, w.uv, o[rows].view(-1, s.heads, s.vdim))
        return project(o, w.o)
