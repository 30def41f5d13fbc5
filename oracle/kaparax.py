"""Plain restatement of the Kaparax decoder on the CPU.  TEST INFRASTRUCTURE ONLY.

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
from typing import Dict, List, Optional

import torch


def layer_norm(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor, eps: float) -> torch.Tensor:
    """Mean and (biased) variance over the last axis, eps inside the root, then scale and shift."""
    centred = x - x.mean(-1, keepdim=True)
    return centred / torch.sqrt((centred * centred).mean(-1, keepdim=True) + eps) * w + b


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """Division by the root mean square of the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rotate(x: torch.Tensor, base: float, dims: int) -> torch.Tensor:
    """``x [T, heads, d]`` at positions 0..T-1: elements i and i + dims/2 turn by position * base^(-2i/dims);
    elements from ``dims`` on stay."""
    t, half = x.shape[0], dims // 2
    if half == 0:
        return x
    freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=x.dtype)
    angle = torch.arange(t, dtype=x.dtype)[:, None] * freq[None]
    c, s = angle.cos()[:, None], angle.sin()[:, None]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], dim=-1)


def short_conv(u: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """``u [T, channels]``, ``w [channels, taps]``: tap ``taps - 1`` meets the present value, tap 0 the
    oldest; values before the start of the sequence are zero."""
    t, taps = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for j in range(taps):
        shift = taps - 1 - j
        if shift < t:
            y[shift:] += u[: t - shift] * w[:, j]
    return y


def capped(score: torch.Tensor, cap: Optional[float]) -> torch.Tensor:
    return score if not cap else cap * torch.tanh(score / cap)


def chunk_visible(t: int, size: int) -> torch.Tensor:
    """``[T, T]`` bool: query i sees key j <= i of its own chunk of ``size`` positions."""
    pos = torch.arange(t)
    return (pos[None] <= pos[:, None]) & (pos[None] // size == pos[:, None] // size)


def softmax_attention(q, k, v, scale: float, cap, visible: torch.Tensor) -> torch.Tensor:
    """``q [T, H, d]``, ``k [T, G, d]``, ``v [T, G, dv]`` -> ``[T, H, dv]``; query head h reads kv head h // (H/G)."""
    t, heads, _ = q.shape
    group = heads // k.shape[1]
    out = torch.zeros(t, heads, v.shape[2], dtype=q.dtype)
    for h in range(heads):
        s = capped(q[:, h] @ k[:, h // group].T * scale, cap)
        p = torch.softmax(s.masked_fill(~visible, -math.inf), dim=-1)
        out[:, h] = p @ v[:, h // group]
    return out


def retention(q, k, v, decay) -> torch.Tensor:
    """``q, k [T, H, d]``, ``v [T, H, dv]``: the recurrence itself, one token at a time."""
    t, heads, d = q.shape
    state = torch.zeros(heads, d, v.shape[2], dtype=q.dtype)
    gamma = torch.as_tensor(decay, dtype=q.dtype)[:, None, None]
    out = torch.zeros(t, heads, v.shape[2], dtype=q.dtype)
    for i in range(t):
        state = gamma * state + k[i][:, :, None] * v[i][:, None, :]
        out[i] = (state * q[i][:, :, None]).sum(1)
    return out


def gated_mlp(h: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor, limit: float) -> torch.Tensor:
    """Gate capped from above, up clamped on both sides and shifted by one, sigmoid of slope 1.702."""
    g = torch.clamp(h @ gate.T, max=limit)
    u = torch.clamp(h @ up.T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def attention_mixer(h: torch.Tensor, w, m: dict) -> torch.Tensor:
    t = h.shape[0]
    proj = {}
    for name, heads, size in (("q", m["heads"], m["dim"]), ("k", m["kv_heads"], m["dim"]), ("v", m["kv_heads"], m["vdim"])):
        proj[name] = short_conv(h @ w(name).T, w(name + ".conv")).view(t, heads, size)
    q = rotate(proj["q"], m["rot"]["base"], m["rot"]["dims"])
    k = rotate(proj["k"], m["rot"]["base"], m["rot"]["dims"])
    o = softmax_attention(q, k, proj["v"], m["scale"], m["softcap"], chunk_visible(t, m["mask"]["size"]))
    return o.reshape(t, -1) @ w("o").T


def retention_mixer(h: torch.Tensor, w, m: dict, eps: float) -> torch.Tensor:
    t = h.shape[0]
    heads, d, dv = m["heads"], m["dim"], m["vdim"]
    q = rotate((h @ w("q").T).view(t, heads, d), m["rot"]["base"], m["rot"]["dims"])
    k = rotate((h @ w("k").T).view(t, heads, d), m["rot"]["base"], m["rot"]["dims"]) * d ** -0.5
    o = unit_rms(retention(q, k, (h @ w("v").T).view(t, heads, dv), m["decay"]), eps).reshape(t, -1)
    gate = h @ w("g").T
    return (o * gate * torch.sigmoid(gate)) @ w("o").T


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64,
            record: Optional[list] = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one sequence."""
    eps = config["norm"]["eps"]
    get = lambda name: weights[name].to(dtype)
    norm = lambda x, name: layer_norm(x, get(name), get(name + ".b"), eps)
    x = get("embed")[torch.as_tensor(tokens)] * config["embedding"]["scale"]
    for i, layer in enumerate(config["layers"]):
        p = f"l{layer.get('weights_of', i)}."
        mix = lambda name: get(p + "mix." + name)
        h = norm(x, p + "norm1")
        y = attention_mixer(h, mix, layer["mixer"]) if layer["type"] == "attention" else \
            retention_mixer(h, mix, layer["mixer"], eps)
        x = x + norm(y, p + "norm1b")
        if layer["mlp"] is not None:
            y = gated_mlp(norm(x, p + "norm2"), get(p + "mlp.gate"), get(p + "mlp.up"), get(p + "mlp.down"),
                          layer["mlp"]["limit"])
            x = x + norm(y, p + "norm2b")
        if record is not None:
            record.append(x.clone())
    return norm(x, "final.norm") @ get("head").T
