"""Plain restatement of the Bedenex decoder on the CPU.  TEST INFRASTRUCTURE ONLY.

One function per mechanism, written from the equations; nothing here is shared with the product
package.  A whole sequence is run at once from position 0, so there is no cache, no batch and no
portion: what the engine computes for any cut and any mix has to agree with this.

``config`` is the parsed ``config.json`` (a dict), ``weights`` maps tensor names to tensors.
Everything is evaluated in ``dtype`` (float64 by default).  The optional ``record`` list of
``forward`` receives the residual stream after every layer, a looped one each time.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """Division by the root mean square of the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def weighted_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(x, eps) * w


def turned(x: torch.Tensor, base: float, dims: int) -> torch.Tensor:
    """``x [T, ..., dims]`` at positions 0..T-1: elements i and i + dims / 2 turn by position * base^(-2i/dims)."""
    half = dims // 2
    out = x.clone()
    for i in range(half):
        angle = torch.arange(x.shape[0], dtype=x.dtype) * base ** (-2.0 * i / dims)
        c, s = (f(angle).view(-1, *[1] * (x.dim() - 2)) for f in (torch.cos, torch.sin))
        u, v = x[..., i], x[..., i + half]
        out[..., i], out[..., i + half] = u * c - v * s, v * c + u * s
    return out


def causal(t: int) -> torch.Tensor:
    return torch.ones(t, t, dtype=torch.bool).tril()


def in_chunk(t: int, size: int) -> torch.Tensor:
    """``[T, T]`` bool: what came before a query inside its own chunk of positions, and itself."""
    at = torch.arange(t) // size
    return causal(t) & (at[:, None] == at[None])


def distance_bias(t: int, r1: torch.Tensor, r2: torch.Tensor) -> torch.Tensor:
    """``[T, T]``: what one head takes off the score of a key that lies i - j back."""
    lag = (torch.arange(t)[:, None] - torch.arange(t)[None]).clamp(min=0).to(r1.dtype)
    return r1 * torch.log1p(r2 * lag)


def softmax_with_sink(s: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """Weights of the scores ``[T, T]``, whose sum also holds exp(sink)."""
    return torch.softmax(torch.cat([s, sink.expand(len(s), 1)], 1), -1)[:, :-1]


def latent_attention(h: torch.Tensor, w, m: dict, eps: float) -> torch.Tensor:
    t, heads, d, r, dv, rank = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (h @ w("q").T).view(t, heads, d + r)
    down = h @ w("dkv").T
    c = weighted_norm(down[:, :rank], w("dkv.norm"), eps)
    k_rot = turned(down[:, rank:], m["rot"]["base"], r)
    q_rot = turned(q[..., d:], m["rot"]["base"], r)
    k, v = (c @ w("uk").T).view(t, heads, d), (c @ w("uv").T).view(t, heads, dv)
    out = torch.zeros(t, heads, dv, dtype=h.dtype)
    for n in range(heads):
        s = (q[:, n, :d] @ k[:, n].T + q_rot[:, n] @ k_rot.T) * m["scale"]
        out[:, n] = softmax_with_sink(s.masked_fill(~causal(t), -math.inf), w("sink")[n]) @ v[:, n]
    return out.reshape(t, -1) @ w("o").T


def head_norm(x: torch.Tensor, eps: float) -> torch.Tensor:
    """Queries and keys, every head by itself."""
    return unit_rms(x, eps)


def value_norm(v: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(v, eps)


def head_gates(h: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    return torch.sigmoid(h @ w.T)


def biased_attention(h: torch.Tensor, w, m: dict, eps: float) -> torch.Tensor:
    """Queries, keys and values of unit root mean square, a bias that grows with the logarithm of the distance, chunks,
    a gate per head."""
    t, heads, groups = h.shape[0], m["heads"], m["kv_heads"]
    q = head_norm((h @ w("q").T).view(t, heads, m["dim"]), eps)
    k = head_norm((h @ w("k").T).view(t, groups, m["dim"]), eps)
    v = value_norm((h @ w("v").T).view(t, groups, m["vdim"]), eps)
    out = torch.zeros(t, heads, m["vdim"], dtype=h.dtype)
    for n in range(heads):
        g = n // (heads // groups)
        s = q[:, n] @ k[:, g].T * m["scale"] - distance_bias(t, w("r1")[n], w("r2")[n])
        out[:, n] = torch.softmax(s.masked_fill(~in_chunk(t, m["mask"]["size"]), -math.inf), -1) @ v[:, g]
    return (out * head_gates(h, w("g"))[..., None]).reshape(t, -1) @ w("o").T


def gelu(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def gelu_mlp(h, gate, up, down) -> torch.Tensor:
    return (gelu(h @ gate.T) * (h @ up.T)) @ down.T


def silu_mlp(h, gate, up, down) -> torch.Tensor:
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def route(z: torch.Tensor, top: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """Router logits ``[T, E]`` -> chosen experts and their sigmoids as they are, ``[T, top]`` each."""
    best, chosen = torch.topk(z, top, dim=-1)
    return chosen, torch.sigmoid(best)


def weighted_expert(h, weight, gate, up, down) -> torch.Tensor:
    """The weight belongs to what the expert reads."""
    return silu_mlp(weight[:, None] * h, gate, up, down)


def expert_mixture(h: torch.Tensor, w, m: dict) -> torch.Tensor:
    chosen, weight = route(h @ w("router").T, m["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        rows, which = (chosen == e).nonzero(as_tuple=True)
        if len(rows):
            out[rows] += weighted_expert(h[rows], weight[rows, which], w(f"e{e}.gate"), w(f"e{e}.up"), w(f"e{e}.down"))
    return out


def channel_gate(h: torch.Tensor, w: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    return torch.sigmoid(h @ w.T + b)


def entry(x: torch.Tensor, x0: torch.Tensor, w: torch.Tensor, step: torch.Tensor) -> torch.Tensor:
    """What a pass begins with."""
    return torch.cat([x, x0], -1) @ w.T + step


def layer_order(layers: int, loop: Optional[dict]) -> List[Tuple[int, Optional[int]]]:
    """(layer, number of the pass that begins with it or None) in the order in which layers run."""
    if loop is None:
        return [(i, None) for i in range(layers)]
    start, stop = loop["start"], loop["stop"]
    out = [(i, None) for i in range(start)]
    for t in range(loop["times"]):
        out += [(i, t if i == start else None) for i in range(start, stop)]
    return out + [(i, None) for i in range(stop, layers)]


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64,
            record: Optional[list] = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one sequence."""
    eps = config["norm"]["eps"]
    get = lambda name: weights[name].to(dtype)
    x0 = x = get("embed")[torch.as_tensor(tokens)]
    for i, begins in layer_order(len(config["layers"]), config.get("loop")):
        layer = config["layers"][i]
        p, ff = f"l{i}.", layer.get("mlp")
        mix, mlp = lambda name: get(p + "mix." + name), lambda name: get(p + "mlp." + name)
        if begins is not None:
            x = entry(x, x0, get("loop.in"), get("loop.step")[begins])
        h = weighted_norm(x, get(p + "norm1"), eps)
        mixer = latent_attention if layer["type"] == "latent_attention" else biased_attention
        y = mixer(h, mix, layer["mixer"], eps) * channel_gate(h, get(p + "rg1"), get(p + "rg1.b"))
        if ff is not None:
            z = gelu_mlp(h, mlp("gate"), mlp("up"), mlp("down")) if ff["kind"] == "dense" else expert_mixture(h, mlp, ff)
            y = y + z * channel_gate(h, get(p + "rg2"), get(p + "rg2.b"))
        x = x + y
        if record is not None:
            record.append(x.clone())
    return weighted_norm(x, get("final.norm"), eps) @ get("head").T
