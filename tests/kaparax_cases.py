"""Small random Kaparax models and row groups for the tests (sizes and values made here)."""
import json
import os
import random

import torch
from safetensors.torch import save_file

BLOCK = 256


def attention(heads, kv, dim, vdim, conv, chunk, rot, scale=0.3, cap=20.0, base=5000.0):
    return dict(type="attention", mixer=dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, conv=conv, mask=dict(size=chunk),
                                             scale=scale, softcap=cap, rot=dict(base=base, dims=rot)))


def retention(heads, dim, vdim, rot, decay=None, base=300.0):
    decay = decay or [1.0 - 2.0 ** -(2 + 1.7 * h) for h in range(heads)]
    return dict(type="retention", mixer=dict(heads=heads, dim=dim, vdim=vdim, decay=decay, rot=dict(base=base, dims=rot)))


def mlp(ff, limit=1.1):
    return dict(kind="dense", ff=ff, limit=limit)


def model(width, vocab, layers, scale=3.5, eps=1e-5):
    out = []
    for entry in layers:
        mixer, ff, *shared = entry
        layer = dict(mixer, mlp=ff)
        if shared:
            layer["weights_of"] = shared[0]
        out.append(layer)
    return dict(architecture="Kaparax", vocab=vocab, width=width, embedding=dict(scale=scale), norm=dict(eps=eps), layers=out)


def configs():
    """name -> configuration.  Together: one and several kv heads and a group of 1, equal and unequal
    key and value sizes, whole, part and no rotation, 1 to 11 taps, chunks shorter and longer than a
    page, any pattern of feed-forwards, shared weights of both mixers, a score cap beyond what an
    unreferenced exponential could hold, sizes off every vector width."""
    a1 = attention(6, 2, 48, 40, 3, 37, 32, cap=2.5)
    r1 = retention(3, 32, 48, 16)
    a2 = attention(8, 2, 128, 128, 4, 300, 128, scale=0.15)
    r2 = retention(2, 128, 128, 128)
    a3 = attention(3, 3, 20, 12, 2, 64, 12, cap=150.0, scale=0.5)
    r3 = retention(2, 12, 20, 0, decay=[0.4, 1.0])
    a4 = attention(5, 1, 64, 96, 6, 500, 0)
    r4 = retention(4, 64, 160, 64, decay=[0.2, 0.9, 0.99, 0.9999])
    a5 = attention(4, 4, 96, 64, 1, 129, 64, cap=5.0)
    a6 = attention(4, 2, 32, 24, 11, 90, 20)
    r5 = retention(2, 192, 64, 96)
    return {
        "mixed": model(104, 320, [(r1, mlp(72)), (a1, None), (a1, mlp(56)), (r1, None), (a1, None, 1), (r1, mlp(72), 0), (a1, mlp(56), 2)]),
        "wide": model(256, 512, [(a2, mlp(384)), (r2, None), (a2, mlp(384), 0), (r2, None, 1)], eps=1e-6),
        "odd": model(50, 301, [(a3, mlp(27)), (r3, mlp(31)), (a3, None), (r3, None)], scale=0.7),
        "deep_state": model(128, 256, [(r4, None), (a4, mlp(96)), (r4, mlp(64)), (a4, None)]),
        "taps": model(192, 256, [(a5, mlp(128, limit=0.4)), (r5, mlp(128)), (a5, None), (a6, mlp(64))]),
    }


def random_weights(cfg, seed=0):
    """bf16 tensors with the names a checkpoint of the family has; norm scales and shifts are not trivial."""
    g = torch.Generator().manual_seed(seed)
    n = lambda *s, std=1.0: torch.randn(*s, generator=g) * std
    width, out = cfg["width"], {}

    def norm(name):
        out[name], out[name + ".b"] = 1.0 + n(width, std=0.2), n(width, std=0.2)

    def linear(name, rows, cols, gain=1.0):
        out[name] = n(rows, cols, std=gain * cols ** -0.5)

    linear("embed", cfg["vocab"], width, gain=width ** 0.5)
    for i, layer in enumerate(cfg["layers"]):
        if "weights_of" in layer:
            continue
        p, m = f"l{i}.", layer["mixer"]
        norm(p + "norm1"), norm(p + "norm1b")
        if layer["type"] == "attention":
            for name, rows in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                linear(p + "mix." + name, rows, width)
                out[p + "mix." + name + ".conv"] = n(rows, m["conv"], std=m["conv"] ** -0.5)
        else:
            for name, rows in (("q", m["heads"] * m["dim"]), ("k", m["heads"] * m["dim"]), ("v", m["heads"] * m["vdim"]),
                               ("g", m["heads"] * m["vdim"])):
                linear(p + "mix." + name, rows, width)
        linear(p + "mix.o", width, m["heads"] * m["vdim"])
        if layer["mlp"] is not None:
            norm(p + "norm2"), norm(p + "norm2b")
            linear(p + "mlp.gate", layer["mlp"]["ff"], width)
            linear(p + "mlp.up", layer["mlp"]["ff"], width)
            linear(p + "mlp.down", width, layer["mlp"]["ff"])
    norm("final.norm")
    linear("head", cfg["vocab"], width)
    return {k: v.to(torch.bfloat16).contiguous() for k, v in out.items()}


def write_model(folder, cfg, weights):
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file(weights, os.path.join(folder, "model.safetensors"))
    return str(folder)


def row_error(got, want):
    """Root mean square of the difference over the vocabulary (means taken off) over the spread of the
    expected logits, per row."""
    d = got.double() - want.double()
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.double().std(-1).mean()


def cut(total, sizes, rng):
    """Portion lengths from ``sizes`` that add up to ``total``."""
    out = []
    while total:
        out.append(min(total, rng.choice(sizes)))
        total -= out[-1]
    return out


def tokens(n, vocab, seed):
    rng = random.Random(seed)
    return [rng.randrange(vocab) for _ in range(n)]
