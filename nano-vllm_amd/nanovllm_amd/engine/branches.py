"""The residual step of layers whose mixer and feed-forward read the same point of the stream: both branches'
results are added at once (scaled per channel, or behind gates of every element) and the next layer's norms are taken in the same
pass over the row; of layers that norm what a sublayer gives, where the next sublayer reads the stream itself; and of a stream
that begins anew."""
from __future__ import annotations

from typing import Optional, Tuple

import torch

from .. import _lib
from .mixers import _DTYPE, _need_cuda, _ptr, _stream


def _outputs(rows: int, table: torch.Tensor, second: Optional[torch.Tensor]):
    width = table.shape[-1]
    out1 = torch.empty((rows, width), dtype=table.dtype, device=table.device)
    return out1, None if second is None else torch.empty_like(out1)


def embed_rms_norms(ids: torch.Tensor, table: torch.Tensor, scale: float, weights: Tuple[Optional[torch.Tensor], Optional[torch.Tensor]],
                    eps: float, weight_offset: float = 0.0, clear: Optional[torch.Tensor] = None, out: Optional[torch.Tensor] = None,
                    copy: Optional[torch.Tensor] = None):
    """``residual = table[ids] * scale`` (fp32) and its RMS norms with one or two weights (stored as the
    deviation from ``weight_offset``; without weights: the residual itself, rounded); ``clear``: int32 counters to zero.  ``out``: where the
    first goes; ``copy``: where the residual itself, rounded, goes as well (row strides of their own).  Returns (residual, out1, out2)."""
    vocab, width = table.shape
    assert ids.dtype == torch.int64 and ids.is_contiguous() and table.is_contiguous()
    _need_cuda(ids, table)
    n = ids.numel()
    residual = torch.empty((n, width), dtype=torch.float32, device=table.device)
    out1, out2 = _outputs(n, table, weights[1]) if out is None else (out, None)
    for t in (out1, copy):
        assert t is None or (t.shape == (n, width) and t.stride(1) == 1 and t.dtype == table.dtype)
    assert out is None or weights[1] is None
    rc = _lib.load_shared().nva_embed_rms_norms(
        ids.data_ptr(), table.data_ptr(), float(scale), _ptr(weights[0]), _ptr(weights[1]), float(weight_offset),
        residual.data_ptr(), out1.data_ptr(), out1.stride(0), _ptr(out2), _ptr(copy), 0 if copy is None else copy.stride(0),
        _ptr(clear), 0 if clear is None else clear.numel(), n, width, vocab,
        float(eps), _DTYPE[table.dtype], _stream())
    _lib.check(rc, "nva_embed_rms_norms")
    return residual, out1, out2


def branches_rms_norms(residual: torch.Tensor, mult: float, y1: Optional[torch.Tensor], gain1: Optional[torch.Tensor],
                       y2: Optional[torch.Tensor], term_weight: Optional[torch.Tensor], gain2: Optional[torch.Tensor],
                       weights: Tuple[torch.Tensor, Optional[torch.Tensor]], eps: float, weight_offset: float = 0.0,
                       rows: Optional[torch.Tensor] = None, clear: Optional[torch.Tensor] = None):
    """``residual += mult * (gain1 * y1 + gain2 * sum_k term_weight[:, k] * y2[:, k])`` in place (``y2 [n * terms,
    width]``), then the norms.  With ``rows`` (int32) only those rows are computed and the residual stays as it is."""
    n, width = residual.shape
    assert residual.dtype == torch.float32 and residual.is_contiguous()
    _need_cuda(residual, weights[0])
    terms = 0
    if y1 is not None:
        assert y1.shape == residual.shape and y1.stride(1) == 1 and y1.dtype == weights[0].dtype
    if y2 is not None:
        terms = y2.shape[0] // max(n, 1)
        assert y2.shape == (n * terms, width) and y2.is_contiguous() and y2.dtype == weights[0].dtype
        assert term_weight is None or (term_weight.shape == (n, terms) and term_weight.dtype == torch.float32 and term_weight.is_contiguous())
    count = n if rows is None else rows.numel()
    if rows is not None:
        assert rows.dtype == torch.int32 and rows.is_contiguous()
    out1, out2 = _outputs(count, weights[0], weights[1])
    rc = _lib.load_shared().nva_branches_rms_norms(
        _ptr(y1), 0 if y1 is None else y1.stride(0), _ptr(gain1), _ptr(y2), _ptr(term_weight), terms, _ptr(gain2), float(mult),
        residual.data_ptr(), weights[0].data_ptr(), _ptr(weights[1]), float(weight_offset), out1.data_ptr(), _ptr(out2), _ptr(rows),
        _ptr(clear), 0 if clear is None else clear.numel(), count, n, width, float(eps), _DTYPE[weights[0].dtype], _stream())
    _lib.check(rc, "nva_branches_rms_norms")
    return out1, out2


def post_rms_norms(residual: torch.Tensor, y1: Optional[torch.Tensor], y1_weight: Optional[torch.Tensor], y2: Optional[torch.Tensor],
                   term_weight: Optional[torch.Tensor], post: torch.Tensor, nxt: Optional[torch.Tensor], eps: float, weight_offset: float = 0.0,
                   rows: Optional[torch.Tensor] = None, clear: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``residual += rms_norm(y1_weight * y1 + sum_k term_weight[:, k] * y2[:, k])`` in place; returns the residual, rounded, or with
    ``nxt`` its norm.  ``y1_weight [n]`` and ``term_weight [n, terms]`` may be columns of one tensor.  With ``rows`` (int32) only
    those rows are computed and the residual stays as it is."""
    n, width = residual.shape
    assert residual.dtype == torch.float32 and residual.is_contiguous() and (y1 is not None or y2 is not None)
    _need_cuda(residual, post)
    terms = stride = 0
    if y1 is not None:
        assert y1.shape == residual.shape and y1.stride(1) == 1 and y1.dtype == post.dtype
    if y2 is not None:
        terms = y2.shape[0] // max(n, 1)
        assert y2.shape == (n * terms, width) and y2.is_contiguous() and y2.dtype == post.dtype
    for w, shape in ((y1_weight, (n,)), (term_weight, (n, terms))):
        if w is not None:
            assert w.shape == shape and w.dtype == torch.float32 and stride in (0, w.stride(0)) and (w.dim() == 1 or w.stride(1) == 1)
            stride = w.stride(0)
    count = n if rows is None else rows.numel()
    assert rows is None or (rows.dtype == torch.int32 and rows.is_contiguous())
    out, _ = _outputs(count, post, None)
    rc = _lib.load_shared().nva_post_rms_norms(
        _ptr(y1), 0 if y1 is None else y1.stride(0), _ptr(y1_weight), _ptr(y2), _ptr(term_weight), stride, terms, post.data_ptr(),
        residual.data_ptr(), _ptr(nxt), float(weight_offset), out.data_ptr(), _ptr(rows), _ptr(clear), 0 if clear is None else clear.numel(),
        count, n, width, float(eps), _DTYPE[post.dtype], _stream())
    _lib.check(rc, "nva_post_rms_norms")
    return out


def gated_rms_norm(residual: torch.Tensor, y1: torch.Tensor, y2: Optional[torch.Tensor], gate: torch.Tensor, gate_bias: torch.Tensor,
                   weight: Optional[torch.Tensor], eps: float, weight_offset: float = 0.0, rows: Optional[torch.Tensor] = None,
                   clear: Optional[torch.Tensor] = None, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``residual += sigmoid(z1 + b1) * y1 + sigmoid(z2 + b2) * sum_k y2[:, k]`` in place, ``gate = (z1 | z2)`` and ``gate_bias = (b1 |
    b2)`` (without ``y2 [n * terms, width]`` the first halves only); returns the norm, or without ``weight`` the residual, rounded, in ``out``
    if given.  With ``rows`` (int32) only those rows are computed and the residual stays as it is."""
    n, width = residual.shape
    assert residual.dtype == torch.float32 and residual.is_contiguous()
    _need_cuda(residual, y1)
    terms = 0 if y2 is None else y2.shape[0] // max(n, 1)
    assert y1.shape == residual.shape and y1.stride(1) == 1 and gate.shape == (n, (1 if y2 is None else 2) * width) and gate.stride(1) == 1
    assert y2 is None or (y2.shape == (n * terms, width) and y2.is_contiguous() and y2.dtype == y1.dtype)
    assert gate_bias.numel() >= gate.shape[1] and gate_bias.dtype == gate.dtype == y1.dtype and (weight is None or weight.dtype == y1.dtype)
    count = n if rows is None else rows.numel()
    assert rows is None or (rows.dtype == torch.int32 and rows.is_contiguous())
    if out is None:
        out = torch.empty((count, width), dtype=y1.dtype, device=y1.device)
    assert out.shape == (count, width) and out.stride(1) == 1 and out.dtype == y1.dtype
    rc = _lib.load_shared().nva_gated_rms_norm(
        y1.data_ptr(), y1.stride(0), _ptr(y2), terms, gate.data_ptr(), gate.stride(0), gate_bias.data_ptr(), residual.data_ptr(), _ptr(weight),
        float(weight_offset), out.data_ptr(), out.stride(0), _ptr(rows), _ptr(clear), 0 if clear is None else clear.numel(), count, n, width,
        float(eps), _DTYPE[y1.dtype], _stream())
    _lib.check(rc, "nva_gated_rms_norm")
    return out


def entry_rms_norm(product: torch.Tensor, step: torch.Tensor, residual: torch.Tensor, weight: torch.Tensor, eps: float,
                   weight_offset: float = 0.0, clear: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``residual = product + step`` (fp32) and its norm."""
    n, width = residual.shape
    assert product.shape == residual.shape and product.dtype == residual.dtype == torch.float32 and product.is_contiguous() and residual.is_contiguous()
    assert step.numel() == width and step.dtype == weight.dtype
    _need_cuda(product, step)
    out = torch.empty((n, width), dtype=weight.dtype, device=weight.device)
    rc = _lib.load_shared().nva_entry_rms_norm(product.data_ptr(), step.data_ptr(), residual.data_ptr(), weight.data_ptr(), float(weight_offset),
                                               out.data_ptr(), _ptr(clear), 0 if clear is None else clear.numel(), n, width, float(eps),
                                               _DTYPE[weight.dtype], _stream())
    _lib.check(rc, "nva_entry_rms_norm")
    return out
