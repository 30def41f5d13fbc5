"""Plain restatement of the Pidutar decoder on the CPU.  TEST INFRASTRUCTURE ONLY.

One function per mechanism, written from the equations, token by token where that is the
definition; nothing here is shared with the product package.  A whole sequence is run at once
from position 0, so there is no cache, no state hand-over, no batch and no portion: what the
engine computes for any cut and any mix has to agree with this.

``config`` is the parsed ``config.json`` (a dict), ``weights`` maps tensor names to tensors.
Everything is evaluated in ``dtype`` (float64 by default).  The optional ``record`` list of
``forward`` receives the residual stream after every layer.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

EXPERT_SUM_GUARD = 1e-20
MEMORY_GUARD = 1e-6


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """Division by the root mean square of the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def centred_weight_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """RMS norm whose stored weight is the deviation from one."""
    return unit_rms(x, eps) * (1.0 + w)


def rotate_neighbours(x: torch.Tensor, base: float, dims: int) -> torch.Tensor:
    """``x [T, heads, d]`` at positions 0..T-1: elements 2i and 2i + 1 turn by position * base^(-2i/dims);
    elements from ``dims`` on stay."""
    t = x.shape[0]
    out = x.clone()
    for i in range(dims // 2):
        angle = torch.arange(t, dtype=x.dtype) * base ** (-2.0 * i / dims)
        c, s = angle.cos()[:, None], angle.sin()[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def window_visible(t: int, size: int) -> torch.Tensor:
    """``[T, T]`` bool: query i sees itself and the size - 1 keys before it."""
    lag = torch.arange(t)[:, None] - torch.arange(t)[None]
    return (lag >= 0) & (lag < size)


def softmax_attention(q, k, v, scale: float, visible: torch.Tensor) -> torch.Tensor:
    """``q, k [T, H, d]``, ``v [T, H, dv]`` -> ``[T, H, dv]``."""
    out = torch.zeros(q.shape[0], q.shape[1], v.shape[2], dtype=q.dtype)
    for h in range(q.shape[1]):
        s = (q[:, h] @ k[:, h].T * scale).masked_fill(~visible, -math.inf)
        out[:, h] = torch.softmax(s, dim=-1) @ v[:, h]
    return out


def soft_cap(z: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(z / cap)


def log_sigmoid(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, max=0.0) - torch.log1p(torch.exp(-z.abs()))


def matrix_memory(q, k, v, log_in, log_keep) -> torch.Tensor:
    """``q, k [T, H, d]``, ``v [T, H, dv]``, gates ``[T, H]``: the stabilised recurrence, one token at a time."""
    t, heads, d = q.shape
    memory = torch.zeros(heads, d, v.shape[2], dtype=q.dtype)
    mass = torch.zeros(heads, d, dtype=q.dtype)
    top = torch.zeros(heads, dtype=q.dtype)
    out = torch.zeros(t, heads, v.shape[2], dtype=q.dtype)
    for i in range(t):
        new_top = torch.maximum(log_keep[i] + top, log_in[i])
        keep, take = torch.exp(log_keep[i] + top - new_top), torch.exp(log_in[i] - new_top)
        top = new_top
        memory = keep[:, None, None] * memory + take[:, None, None] * k[i][:, :, None] * v[i][:, None, :]
        mass = keep[:, None] * mass + take[:, None] * k[i]
        size = torch.maximum((mass * q[i]).sum(-1).abs(), torch.exp(-top)) + MEMORY_GUARD
        out[i] = (memory * q[i][:, :, None]).sum(1) / size[:, None]
    return out


def route(z: torch.Tensor, top: int, scale: float) -> Tuple[torch.Tensor, torch.Tensor]:
    """Router logits ``[T, E]`` -> chosen experts and their weights, ``[T, top]`` each."""
    s, chosen = torch.topk(torch.softmax(z, dim=-1), top, dim=-1)
    return chosen, s / (s.sum(-1, keepdim=True) + EXPERT_SUM_GUARD) * scale


def gated_mlp(h, gate, up, down) -> torch.Tensor:
    g = h @ gate.T
    return (g * torch.sigmoid(g) * (h @ up.T)) @ down.T


def expert_mixture(h: torch.Tensor, w, m: dict) -> torch.Tensor:
    chosen, weight = route(h @ w("router").T, m["router"]["top"], m["router"]["scale"])
    out = torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        rows, which = (chosen == e).nonzero(as_tuple=True)
        if len(rows):
            y = gated_mlp(h[rows], w(f"e{e}.gate"), w(f"e{e}.up"), w(f"e{e}.down"))
            out[rows] += weight[rows, which][:, None] * y
    return out


def latent_keys(h: torch.Tensor, w, m: dict, eps: float) -> Tuple[torch.Tensor, torch.Tensor]:
    """What a token leaves behind: its normed latent ``[T, kv_rank]`` and its rotated key part ``[T, rot_dim]``."""
    down = h @ w("dkv").T
    latent = unit_rms(down[:, : m["kv_rank"]], eps) * w("dkv.norm")
    return latent, rotate_neighbours(down[:, None, m["kv_rank"]:], m["rot"]["base"], m["rot"]["dims"])[:, 0]


def latent_attention(h: torch.Tensor, keys, w, m: dict, eps: float) -> torch.Tensor:
    t, heads, dim, rot, vdim = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    latent, turned = keys
    q = ((unit_rms(h @ w("dq").T, eps) * w("dq.norm")) @ w("uq").T).view(t, heads, dim + rot)
    q = torch.cat([q[..., :dim], rotate_neighbours(q[..., dim:], m["rot"]["base"], m["rot"]["dims"])], dim=-1)
    k = torch.cat([(latent @ w("uk").T).view(t, heads, dim), turned[:, None].expand(t, heads, rot)], dim=-1)
    v = (latent @ w("uv").T).view(t, heads, vdim)
    o = softmax_attention(q, k, v, m["scale"], window_visible(t, m["mask"]["size"]))
    return (o * torch.sigmoid(h @ w("g").T)[..., None]).reshape(t, -1) @ w("o").T


def mlstm(h: torch.Tensor, w, m: dict, eps: float) -> torch.Tensor:
    t, heads, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w("q").T).view(t, heads, d) * d ** -0.5
    k, v = (h @ w("k").T).view(t, heads, d), (h @ w("v").T).view(t, heads, dv)
    log_in = soft_cap(h @ w("i").T + w("i.b"), m["gate_cap"])
    log_keep = log_sigmoid(soft_cap(h @ w("f").T + w("f.b"), m["gate_cap"]))
    o = unit_rms(matrix_memory(q, k, v, log_in, log_keep), eps).reshape(t, -1)
    return (o * w("norm") * torch.sigmoid(h @ w("g").T)) @ w("o").T


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64,
            record: Optional[list] = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one sequence."""
    eps, mult = config["norm"]["eps"], config["residual_mult"]
    get = lambda name: weights[name].to(dtype)
    norm = lambda x, name: centred_weight_norm(x, get(name), eps)
    x = get("embed")[torch.as_tensor(tokens)] * config["embedding"]["scale"]
    kept: Dict[int, tuple] = {}
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        mix, ff = lambda name: get(p + "mix." + name), lambda name: get(p + "mlp." + name)
        h = norm(x, p + "norm1")
        if layer["type"] == "mlstm":
            y = mlstm(h, mix, m, eps)
        else:
            source = m.get("kv_from")
            if source is None:
                kept[i] = latent_keys(h, mix, m, eps)
            y = latent_attention(h, kept[i if source is None else source], mix, m, eps)
        y = y * get(p + "ls1")
        if layer["mlp"] is not None:
            y = y + expert_mixture(norm(x, p + "norm2"), ff, layer["mlp"]) * get(p + "ls2")
        x = x + mult * y
        if record is not None:
            record.append(x.clone())
    return norm(x, "final.norm") @ get("head").T * config["logit_scale"]
