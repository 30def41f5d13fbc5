"""Mixers and feed-forwards of layered models on the GPU.

``ChunkAttention`` (short convolution, rotary positions, softmax attention inside position chunks,
paged keys and values), ``Retention`` (linear attention with a fixed decay, recurrent state in slots)
and ``ClampedGateMLP``; plus the norms around the fp32 residual stream.  All are thin layers over the
C ABI and run in bf16 or fp32.  A mixer reads the step's rows from the Context as row groups
(``nanovllm_amd.context.RowGroup``): single tokens and portions, each with its own kernels.

Weights and runtime are separate objects: several layers may run the same weights, each with a cache
or state of its own.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Dict, Optional, Sequence, Tuple

import torch
import torch.nn.functional as F
from torch import nn

from .. import _lib
from ..context import RowGroup, get_context

_DTYPE = {torch.bfloat16: _lib.DTYPE_BF16, torch.float32: _lib.DTYPE_F32}


def _stream() -> int:
    return torch.cuda.current_stream().cuda_stream


def _ptr(t: Optional[torch.Tensor]):
    return None if t is None else t.data_ptr()


def _need_cuda(*tensors) -> None:
    for t in tensors:
        if not t.is_cuda:
            raise RuntimeError("nanovllm_amd ops run on the GPU only (there is no CPU fallback)")


_scratch: Dict[torch.device, torch.Tensor] = {}
_retired_scratch: list = []


def scratch(device: torch.device, nbytes: int) -> torch.Tensor:
    """Scratch memory of the mixers' kernels, one buffer per device (their calls are ordered on one
    stream).  It grows outside graph capture only: a captured call is preceded by an eager one of the
    same shape.  A replaced buffer lives on, because graphs captured earlier hold its address."""
    ws = _scratch.get(device)
    if ws is None or ws.numel() < nbytes:
        if torch.cuda.is_current_stream_capturing():
            raise RuntimeError("scratch memory must be sized by an eager call before graph capture")
        if ws is not None:
            _retired_scratch.append(ws)
        ws = _scratch[device] = torch.empty(max(nbytes, 1 << 20), dtype=torch.uint8, device=device)
    return ws


# ---- ops -----------------------------------------------------------------------------------------

def embed_norm(ids: torch.Tensor, table: torch.Tensor, scale: float, norm: Tuple[torch.Tensor, torch.Tensor], eps: float):
    """``residual = table[ids] * scale`` (fp32) and its layer norm."""
    vocab, width = table.shape
    assert ids.dtype == torch.int64 and ids.is_contiguous() and table.is_contiguous()
    _need_cuda(ids, table)
    n = ids.numel()
    residual = torch.empty((n, width), dtype=torch.float32, device=table.device)
    out = torch.empty((n, width), dtype=table.dtype, device=table.device)
    rc = _lib.load_mixers().nva_embed_norm(ids.data_ptr(), table.data_ptr(), float(scale), norm[0].data_ptr(), norm[1].data_ptr(),
                                    residual.data_ptr(), out.data_ptr(), n, width, vocab, float(eps), _DTYPE[table.dtype],
                                    _stream())
    _lib.check(rc, "nva_embed_norm")
    return residual, out


def post_add_norm(y: torch.Tensor, residual: torch.Tensor, post: Tuple[torch.Tensor, torch.Tensor],
                  nxt: Tuple[torch.Tensor, torch.Tensor], eps: float, rows: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``residual += layer_norm(y)`` in place; returns the next layer norm of the new residual.  With
    ``rows`` (int32) only those rows are computed, and the residual stays as it is."""
    n, width = y.shape
    assert residual.shape == y.shape and residual.dtype == torch.float32 and residual.is_contiguous() and y.stride(1) == 1
    _need_cuda(y, residual)
    count = n if rows is None else rows.numel()
    if rows is not None:
        assert rows.dtype == torch.int32 and rows.is_contiguous()
    out = torch.empty((count, width), dtype=y.dtype, device=y.device)
    rc = _lib.load_mixers().nva_post_add_norm(y.data_ptr(), y.stride(0), residual.data_ptr(), post[0].data_ptr(), post[1].data_ptr(),
                                       nxt[0].data_ptr(), nxt[1].data_ptr(), out.data_ptr(), _ptr(rows), count, n, width,
                                       float(eps), _DTYPE[y.dtype], _stream())
    _lib.check(rc, "nva_post_add_norm")
    return out


def clamped_gate(x: torch.Tensor, limit: float, alpha: float, cubic: float = 0.0, shift: float = 1.0) -> torch.Tensor:
    """``g sigmoid(alpha (g + cubic g^3)) (u + shift)`` of a fused ``[gate | up]`` projection, g capped and u clamped at ``limit``."""
    assert x.dim() == 2 and x.stride(1) == 1 and x.shape[1] % 2 == 0
    _need_cuda(x)
    inter = x.shape[1] // 2
    out = torch.empty((x.shape[0], inter), dtype=x.dtype, device=x.device)
    rc = _lib.load_shared().nva_clamped_gate(x.data_ptr(), x.stride(0), out.data_ptr(), x.shape[0], inter, float(limit),
                                      float(alpha), float(cubic), float(shift), _DTYPE[x.dtype], _stream())
    _lib.check(rc, "nva_clamped_gate")
    return out


GELU_SLOPE, GELU_CUBIC = 2.0 * math.sqrt(2.0 / math.pi), 0.044715      # the tanh form: (1 + tanh y) / 2 = sigmoid(2 y)


def gelu_gate(x: torch.Tensor) -> torch.Tensor:
    """``gelu(gate) up`` of a fused ``[gate | up]`` projection, the tanh form of gelu."""
    return clamped_gate(x, math.inf, GELU_SLOPE, GELU_CUBIC, 0.0)


def squared_relu_(x: torch.Tensor) -> torch.Tensor:
    """``max(x, 0)^2`` in place."""
    assert x.dim() == 2 and x.is_contiguous()
    _need_cuda(x)
    rc = _lib.load_shared().nva_squared_relu(x.data_ptr(), x.stride(0), x.data_ptr(), x.shape[0], x.shape[1], _DTYPE[x.dtype], _stream())
    _lib.check(rc, "nva_squared_relu")
    return x


def soft_cap_(x: torch.Tensor, cap: float) -> torch.Tensor:
    """``cap tanh(x / cap)`` in place."""
    assert x.dim() == 2 and x.is_contiguous()
    _need_cuda(x)
    rc = _lib.load_shared().nva_soft_cap(x.data_ptr(), x.shape[0], x.shape[1], float(cap), _DTYPE[x.dtype], _stream())
    _lib.check(rc, "nva_soft_cap")
    return x


def conv_rope_store(qkv: torch.Tensor, conv_weight: torch.Tensor, conv_state: Optional[torch.Tensor], group: RowGroup,
                    rope: Optional[torch.Tensor], q_out: torch.Tensor, k_cache: torch.Tensor,
                    v_cache: torch.Tensor, heads: int, rot_dims: int) -> None:
    """Short convolution of q, k and v, rotation of q and k, cache write; see ``nva_conv_rope_store``."""
    taps = conv_weight.shape[0]
    _, _, kv_heads, dim = k_cache.shape
    vdim = v_cache.shape[3]
    assert qkv.stride(1) == 1 and qkv.shape[1] == (heads + kv_heads) * dim + kv_heads * vdim == conv_weight.shape[1]
    assert q_out.shape == (qkv.shape[0], heads * dim) and q_out.is_contiguous() and qkv.dtype == q_out.dtype == k_cache.dtype
    assert k_cache.is_contiguous() and v_cache.is_contiguous() and conv_weight.is_contiguous()
    assert group.slot_mapping.numel() == qkv.shape[0] == group.count
    slots = k_cache.shape[0] * k_cache.shape[1]
    state_slots = 0 if conv_state is None else conv_state.shape[0]
    rc = _lib.load_mixers().nva_conv_rope_store(
        qkv.data_ptr(), qkv.stride(0), conv_weight.data_ptr(), _ptr(conv_state), _ptr(group.state_slots), _ptr(group.cu),
        group.seq_lens.data_ptr(), _ptr(group.token_seq), _ptr(rope), q_out.data_ptr(),
        k_cache.data_ptr(), v_cache.data_ptr(), group.slot_mapping.data_ptr(), slots, group.count, group.num_seqs, heads,
        kv_heads, dim, vdim, rot_dims, taps, 1 if rope is None else rope.shape[0], state_slots, _DTYPE[qkv.dtype], _stream())
    _lib.check(rc, "nva_conv_rope_store")


def chunk_attention(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, group: RowGroup, out: torch.Tensor,
                    heads: int, chunk: int, scale: float, softcap: float) -> None:
    """Softmax attention inside position chunks over the paged cache; see ``nva_chunk_attn``."""
    num_blocks, block, kv_heads, dim = k_cache.shape
    vdim = v_cache.shape[3]
    assert q.stride(1) == 1 and q.shape == (group.count, heads * dim) and out.shape == (group.count, heads * vdim)
    assert out.is_contiguous() and q.dtype == out.dtype == k_cache.dtype == v_cache.dtype
    table = group.block_tables
    assert table.dtype == torch.int32 and table.shape[0] == group.num_seqs and table.stride(1) == 1
    chunk, lib, ws = min(chunk, 1 << 30), _lib.load_mixers(), None
    if group.cu is None and q.dtype == torch.bfloat16:
        nbytes = lib.nva_chunk_attn_workspace_bytes(group.count, heads, kv_heads, vdim, table.shape[1], block, chunk)
        ws = scratch(q.device, nbytes) if nbytes else None
    rc = lib.nva_chunk_attn(
        q.data_ptr(), q.stride(0), k_cache.data_ptr(), v_cache.data_ptr(), table.data_ptr(), table.stride(0), table.shape[1],
        _ptr(group.cu), group.seq_lens.data_ptr(), _ptr(group.token_seq), out.data_ptr(), _ptr(ws), 0 if ws is None else ws.numel(),
        group.count, group.num_seqs, group.max_q, heads, kv_heads, dim, vdim, block, num_blocks, chunk, float(scale), float(softcap or 0.0),
        _DTYPE[q.dtype], _stream())
    _lib.check(rc, "nva_chunk_attn")


def retention(qkvg: torch.Tensor, state: torch.Tensor, group: RowGroup, rope: Optional[torch.Tensor],
              log2_decay: torch.Tensor, out: torch.Tensor, rot_dims: int, k_scale: float, eps: float) -> None:
    """Retention with its rotation, head norm and output gate; see ``nva_retention``."""
    slots, heads, dim, vdim = state.shape
    assert qkvg.stride(1) == 1 and qkvg.shape == (group.count, 2 * heads * (dim + vdim))
    assert out.shape == (group.count, heads * vdim) and out.is_contiguous() and out.dtype == qkvg.dtype
    assert state.dtype == torch.float32 and state.is_contiguous() and log2_decay.dtype == torch.float32
    lib, ws = _lib.load_mixers(), None
    if group.cu is not None:
        nbytes = lib.nva_retention_workspace_bytes(group.num_seqs, group.max_q, heads, dim, vdim, rot_dims, _DTYPE[qkvg.dtype])
        ws = scratch(qkvg.device, nbytes) if nbytes else None
    rc = lib.nva_retention(
        qkvg.data_ptr(), qkvg.stride(0), state.data_ptr(), group.state_slots.data_ptr(), _ptr(group.cu),
        group.seq_lens.data_ptr(), _ptr(rope), log2_decay.data_ptr(), out.data_ptr(), _ptr(ws),
        0 if ws is None else ws.numel(), group.count, group.num_seqs, group.max_q, heads, dim, vdim, rot_dims, 1 if rope is None else rope.shape[0], slots, float(k_scale),
        float(eps), _DTYPE[qkvg.dtype], _stream())
    _lib.check(rc, "nva_retention")


# ---- rotary tables -------------------------------------------------------------------------------

@dataclass(frozen=True)
class RotaryScaling:
    """Frequencies stretched to longer contexts than ``original``: those that turn less than ``low`` times over it are
    divided by ``factor``, those that turn more than ``high`` times stay, the ones between are blended."""
    factor: float
    low: float
    high: float
    original: float

    def __call__(self, freq: torch.Tensor) -> torch.Tensor:
        turns = self.original * freq / (2.0 * math.pi)
        keep = ((turns - self.low) / (self.high - self.low) if self.high > self.low else (turns >= self.high).to(freq.dtype)).clamp(0.0, 1.0)
        return freq * (keep + (1.0 - keep) / self.factor)


@dataclass(frozen=True)
class Rotary:
    """Rotation of the first ``dims`` elements of a head by position * base^(-2i/dims), the frequencies possibly scaled;
    which elements make pair i (i and i + dims / 2, or neighbours) is the mixer's affair."""
    base: float
    dims: int
    scaling: Optional[RotaryScaling] = None


class RopeTables:
    """``[max_position, dims]`` fp32 tables (cos | sin), one per distinct rotation of a model.  Angles
    are formed in double precision and rounded once."""

    def __init__(self, max_position: int, device):
        self.max_position, self.device = max_position, device
        self._tables: Dict[Rotary, Optional[torch.Tensor]] = {}

    def get(self, rot: Rotary) -> Optional[torch.Tensor]:
        if rot not in self._tables:
            table = None
            if rot.dims > 0:
                i = torch.arange(rot.dims // 2, dtype=torch.float64)
                freq = torch.exp(-2.0 * i / rot.dims * math.log(rot.base))
                if rot.scaling is not None:
                    freq = rot.scaling(freq)
                angle = torch.outer(torch.arange(self.max_position, dtype=torch.float64), freq)
                table = torch.cat([angle.cos(), angle.sin()], dim=-1).float().contiguous().to(self.device)
            self._tables[rot] = table
        return self._tables[rot]


# ---- specifications, weights and layers ------------------------------------------------------------

@dataclass(frozen=True)
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int
    chunk: int
    scale: float
    softcap: float
    rot: Rotary

    @property
    def channels(self) -> int:
        return (self.heads + self.kv_heads) * self.dim + self.kv_heads * self.vdim


@dataclass(frozen=True)
class RetentionSpec:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]
    rot: Rotary


@dataclass(frozen=True)
class MlpSpec:
    ff: int
    limit: float
    alpha: float = 1.702


class AttentionWeights(nn.Module):
    """q, k and v projections and convolutions fused along the channels; convolution taps first."""

    def __init__(self, spec: AttentionSpec, width: int):
        super().__init__()
        self.qkv = nn.Parameter(torch.empty(spec.channels, width))
        self.conv = nn.Parameter(torch.empty(spec.taps, spec.channels))
        self.o = nn.Parameter(torch.empty(width, spec.heads * spec.vdim))

    def load(self, spec: AttentionSpec, width: int, take, prefix: str) -> None:
        sizes = (("q", spec.heads * spec.dim), ("k", spec.kv_heads * spec.dim), ("v", spec.kv_heads * spec.vdim))
        self.qkv.copy_(torch.cat([take(f"{prefix}{n}", (size, width)) for n, size in sizes]))
        self.conv.copy_(torch.cat([take(f"{prefix}{n}.conv", (size, spec.taps)) for n, size in sizes]).t())
        self.o.copy_(take(f"{prefix}o", self.o.shape))


class RetentionWeights(nn.Module):
    """q, k, v and gate projections fused along the output."""

    def __init__(self, spec: RetentionSpec, width: int):
        super().__init__()
        self.qkvg = nn.Parameter(torch.empty(2 * spec.heads * (spec.dim + spec.vdim), width))
        self.o = nn.Parameter(torch.empty(width, spec.heads * spec.vdim))

    def load(self, spec: RetentionSpec, width: int, take, prefix: str) -> None:
        qk, v = spec.heads * spec.dim, spec.heads * spec.vdim
        self.qkvg.copy_(torch.cat([take(f"{prefix}{n}", (size, width)) for n, size in (("q", qk), ("k", qk), ("v", v), ("g", v))]))
        self.o.copy_(take(f"{prefix}o", self.o.shape))


class MlpWeights(nn.Module):

    def __init__(self, spec: MlpSpec, width: int):
        super().__init__()
        self.gate_up = nn.Parameter(torch.empty(2 * spec.ff, width))
        self.down = nn.Parameter(torch.empty(width, spec.ff))

    def load(self, spec: MlpSpec, width: int, take, prefix: str) -> None:
        self.gate_up.copy_(torch.cat([take(f"{prefix}{n}", (spec.ff, width)) for n in ("gate", "up")]))
        self.down.copy_(take(f"{prefix}down", self.down.shape))


class ChunkAttention:
    """One attention layer's runtime: its share of the paged cache and of the carried rows."""

    def __init__(self, spec: AttentionSpec, weights: AttentionWeights, ropes: RopeTables, eps: float):
        self.spec, self.weights, self.rope = spec, weights, ropes.get(spec.rot)
        self.k_cache = self.v_cache = self.conv_state = None

    def kv_elements_per_token(self) -> int:
        return self.spec.kv_heads * (self.spec.dim + self.spec.vdim)

    def state_bytes_per_slot(self, elem_bytes: int) -> int:
        return (self.spec.taps - 1) * self.spec.channels * elem_bytes

    def bind(self, num_blocks: int, block: int, slots: int, dtype: torch.dtype, device) -> None:
        s = self.spec
        self.k_cache = torch.zeros((num_blocks, block, s.kv_heads, s.dim), dtype=dtype, device=device)
        self.v_cache = torch.zeros((num_blocks, block, s.kv_heads, s.vdim), dtype=dtype, device=device)
        self.conv_state = torch.zeros((slots, s.taps - 1, s.channels), dtype=dtype, device=device) if s.taps > 1 else None

    def unbind(self) -> None:
        self.k_cache = self.v_cache = self.conv_state = None

    def __call__(self, h: torch.Tensor) -> torch.Tensor:
        s, w = self.spec, self.weights
        qkv = F.linear(h, w.qkv)
        q = torch.empty((h.shape[0], s.heads * s.dim), dtype=h.dtype, device=h.device)
        o = torch.empty((h.shape[0], s.heads * s.vdim), dtype=h.dtype, device=h.device)
        for group in get_context().groups:
            rows = slice(group.first, group.first + group.count)
            conv_rope_store(qkv[rows], w.conv, self.conv_state, group, self.rope, q[rows], self.k_cache,
                            self.v_cache, s.heads, s.rot.dims)
            chunk_attention(q[rows], self.k_cache, self.v_cache, group, o[rows], s.heads, s.chunk, s.scale, s.softcap)
        return F.linear(o, w.o)


class Retention:
    """One retention layer's runtime: its recurrent state."""

    def __init__(self, spec: RetentionSpec, weights: RetentionWeights, ropes: RopeTables, eps: float):
        self.spec, self.weights, self.rope, self.eps = spec, weights, ropes.get(spec.rot), eps
        # (a decay of 0 as 2^-1000: its zeroth power stays 1)
        logs = [max(math.log2(d), -1000.0) if d > 0.0 else -1000.0 for d in spec.decay]
        self.log2_decay = torch.tensor(logs, dtype=torch.float32, device=ropes.device)
        self.state = None

    def kv_elements_per_token(self) -> int:
        return 0

    def state_bytes_per_slot(self, elem_bytes: int) -> int:
        return self.spec.heads * self.spec.dim * self.spec.vdim * 4

    def bind(self, num_blocks: int, block: int, slots: int, dtype: torch.dtype, device) -> None:
        s = self.spec
        self.state = torch.zeros((slots, s.heads, s.dim, s.vdim), dtype=torch.float32, device=device)

    def unbind(self) -> None:
        self.state = None

    def __call__(self, h: torch.Tensor) -> torch.Tensor:
        s, w = self.spec, self.weights
        qkvg = F.linear(h, w.qkvg)
        o = torch.empty((h.shape[0], s.heads * s.vdim), dtype=h.dtype, device=h.device)
        for group in get_context().groups:
            rows = slice(group.first, group.first + group.count)
            retention(qkvg[rows], self.state, group, self.rope, self.log2_decay, o[rows], s.rot.dims,
                      s.dim ** -0.5, self.eps)
        return F.linear(o, w.o)


class ClampedGateMLP:

    def __init__(self, spec: MlpSpec, weights: MlpWeights):
        self.spec, self.weights = spec, weights

    def __call__(self, h: torch.Tensor) -> torch.Tensor:
        return F.linear(clamped_gate(F.linear(h, self.weights.gate_up), self.spec.limit, self.spec.alpha), self.weights.down)


MIXERS = {AttentionSpec: (AttentionWeights, ChunkAttention), RetentionSpec: (RetentionWeights, Retention)}
