"""Plain restatement of the Sokolorn decoder on the CPU.  TEST INFRASTRUCTURE ONLY.

One function per mechanism, written from the equations; nothing here is shared with the product
package.  A whole sequence is run at once from position 0, so there is no cache, no batch and no
portion: what the engine computes for any cut and any mix has to agree with this.

``config`` is the parsed ``config.json`` (a dict), ``weights`` maps tensor names to tensors.
Everything is evaluated in ``dtype`` (float64 by default).  The optional ``record`` list of
``forward`` receives the residual stream after every layer.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

SWISH_SLOPE = 1.702


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """Division by the root mean square of the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def centred_weight_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """RMS norm whose stored weight is the deviation from one."""
    return unit_rms(x, eps) * (1.0 + w)


def whole_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """RMS norm over everything a projection gives, before it is taken apart into heads."""
    return unit_rms(x, eps) * w


def head_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """``x [T, heads, d]``: RMS norm of every head by itself, one weight for all of them."""
    return unit_rms(x, eps) * w


def rotation_frequencies(dims: int, base: float, scaling: Optional[dict]) -> List[float]:
    """base^(-2i/dims); with scaling, slow turns are slowed further by ``factor``, fast ones stay, and between
    the two thresholds (in turns over ``original`` positions) the two are blended."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling is not None:
            turns = scaling["original"] * f / (2.0 * math.pi)          # over the original context
            if turns < scaling["low"]:
                f = f / scaling["factor"]
            elif turns <= scaling["high"]:
                s = (turns - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return out


def rotate_halves(x: torch.Tensor, frequencies: List[float]) -> torch.Tensor:
    """``x [T, heads, d]`` at positions 0..T-1: elements i and i + half turn by position * frequency i; elements
    beyond both halves stay."""
    half = len(frequencies)
    out = x.clone()
    for i, f in enumerate(frequencies):
        angle = torch.arange(x.shape[0], dtype=x.dtype) * f
        c, s = angle.cos()[:, None], angle.sin()[:, None]
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def visible(t: int, window: Optional[int]) -> torch.Tensor:
    """``[T, T]`` bool: query i sees itself and what came before it, at most ``window`` keys in all."""
    lag = torch.arange(t)[:, None] - torch.arange(t)[None]
    return (lag >= 0) if window is None else (lag >= 0) & (lag < window)


def softmax_attention(q, k, v, scale: float, seen: torch.Tensor, sink: Optional[torch.Tensor] = None) -> torch.Tensor:
    """``q [T, H, d]``, ``k [T, G, d]``, ``v [T, G, dv]`` -> ``[T, H, dv]``; ``sink [H]`` is one more score per head that
    belongs to no key."""
    group = q.shape[1] // k.shape[1]
    out = torch.zeros(q.shape[0], q.shape[1], v.shape[2], dtype=q.dtype)
    for h in range(q.shape[1]):
        s = (q[:, h] @ k[:, h // group].T * scale).masked_fill(~seen, -math.inf)
        if sink is not None:
            s = torch.cat([s, sink[h].expand(len(s), 1)], 1)
        out[:, h] = torch.softmax(s, dim=-1)[:, : k.shape[0]] @ v[:, h // group]
    return out


def head_gates(h: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    return torch.sigmoid(h @ w.T)


def windowed_attention(h: torch.Tensor, w, m: dict, eps: float) -> torch.Tensor:
    """No positions in the scores; norms over whole projections; a window, sinks, a gate per head."""
    t, heads, groups = h.shape[0], m["heads"], m["kv_heads"]
    q = whole_norm(h @ w("q").T, w("q.norm"), eps).view(t, heads, m["dim"])
    k = whole_norm(h @ w("k").T, w("k.norm"), eps).view(t, groups, m["dim"])
    v = (h @ w("v").T).view(t, groups, m["vdim"])
    o = softmax_attention(q, k, v, m["scale"], visible(t, m["mask"]["size"]), w("sink"))
    return (o * head_gates(h, w("g"))[..., None]).reshape(t, -1) @ w("o").T


def turned(x: torch.Tensor, m: dict) -> torch.Tensor:
    return rotate_halves(x, rotation_frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling")))


def keys_and_values(h: torch.Tensor, w, m: dict, eps: float) -> Tuple[torch.Tensor, torch.Tensor]:
    """What a token leaves behind in a layer with positions: normed and rotated keys, values."""
    t = h.shape[0]
    k = (h @ w("k").T + w("k.b")).view(t, m["kv_heads"], m["dim"])
    v = (h @ w("v").T + w("v.b")).view(t, m["kv_heads"], m["vdim"])
    return turned(head_norm(k, w("k.norm"), eps), m), v


def rotary_attention(h: torch.Tensor, kv, w, m: dict, eps: float) -> torch.Tensor:
    """Biases, norms per head, rotation, all earlier keys (possibly another layer's)."""
    t = h.shape[0]
    q = (h @ w("q").T + w("q.b")).view(t, m["heads"], m["dim"])
    q = turned(head_norm(q, w("q.norm"), eps), m)
    return softmax_attention(q, *kv, m["scale"], visible(t, None)).reshape(t, -1) @ w("o").T


def squared_relu_mlp(h, up, down) -> torch.Tensor:
    return torch.relu(h @ up.T) ** 2 @ down.T


def clamped_mlp(h, gate, up, down, limit: float) -> torch.Tensor:
    g = torch.clamp(h @ gate.T, max=limit)
    u = torch.clamp(h @ up.T, -limit, limit)
    return (g * torch.sigmoid(SWISH_SLOPE * g) * (u + 1.0)) @ down.T


def route(z: torch.Tensor, top: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """Router logits ``[T, E]`` -> chosen experts and the softmax over their logits, ``[T, top]`` each."""
    best, chosen = torch.topk(z, top, dim=-1)
    return chosen, torch.softmax(best, dim=-1)


def shared_part(h: torch.Tensor, w, limit: float) -> torch.Tensor:
    return torch.sigmoid(h @ w("shared.sg").T) * clamped_mlp(h, w("shared.gate"), w("shared.up"), w("shared.down"), limit)


def expert_mixture(h: torch.Tensor, w, m: dict) -> torch.Tensor:
    chosen, weight = route(h @ w("router").T + w("router.b"), m["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        rows, which = (chosen == e).nonzero(as_tuple=True)
        if len(rows):
            y = clamped_mlp(h[rows], w(f"e{e}.gate"), w(f"e{e}.up"), w(f"e{e}.down"), m["expert"]["limit"])
            out[rows] += weight[rows, which][:, None] * y
    if m.get("shared") is not None:
        out = out + shared_part(h, w, m["shared"]["limit"])
    return out


def soft_cap(z: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(z / cap)


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64,
            record: Optional[list] = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one sequence."""
    eps = config["norm"]["eps"]
    get = lambda name: weights[name].to(dtype)
    norm = lambda x, name: centred_weight_norm(x, get(name), eps)
    x = get("embed")[torch.as_tensor(tokens)]
    kept: Dict[int, tuple] = {}
    for i, layer in enumerate(config["layers"]):
        p, m, ff = f"l{i}.", layer["mixer"], layer.get("mlp")
        mix, mlp = lambda name: get(p + "mix." + name), lambda name: get(p + "mlp." + name)
        if layer["type"] == "attention":
            y = windowed_attention(x, mix, m, eps)
        else:
            source = m.get("kv_from")
            if source is None:
                kept[i] = keys_and_values(x, mix, m, eps)
            y = rotary_attention(x, kept[i if source is None else source], mix, m, eps)
        x = x + norm(y, p + "norm1")
        if ff is not None:
            y = squared_relu_mlp(x, mlp("up"), mlp("down")) if ff["kind"] == "dense" else expert_mixture(x, mlp, ff)
            x = x + norm(y, p + "norm2")
        if record is not None:
            record.append(x.clone())
    return soft_cap(norm(x, "final.norm") @ get("embed").T, config["logit_softcap"])
