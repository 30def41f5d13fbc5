"""Small random Sokolorn models for the tests (sizes and values made here)."""
import torch

from kaparax_cases import cut, row_error, tokens, write_model  # noqa: F401


def windowed(heads, kv_heads, dim, vdim, window, scale=None):
    return dict(type="attention", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=window),
                                             scale=scale or 1.3 * dim ** -0.5))


def rotary(heads, kv_heads, dim, vdim, rot, scale=None, base=4000.0, scaling=None, kv_from=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale or 1.7 * dim ** -0.5, rot=dict(base=base, dims=rot))
    if scaling is not None:
        m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type="attention_2", mixer=m)


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff, limit=1.2, shared=None):
    out = dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=experts, top=top))
    if shared is not None:
        out["shared"] = dict(ff=shared[0], limit=shared[1])
    return out


def model(width, vocab, layers, cap=20.0, eps=1e-5):
    return dict(architecture="Sokolorn", vocab=vocab, width=width, norm=dict(eps=eps), logit_softcap=cap,
                layers=[dict(mixer, mlp=ff) for mixer, ff in layers])


def configs():
    """name -> configuration.  Together: windows of 1, below, at and above a page, one and many heads and groups, keys and
    values read by one and by two later layers, partial, whole and no rotation, with and without scaling, layers without
    a feed-forward, shared experts of other sizes and limits and none, one expert and many, every expert chosen, both
    kinds of layer first and last, sizes off every vector width."""
    slow = (6.0, 1.5, 5.0, 300)
    return {
        "mixed": model(104, 320, [(windowed(6, 2, 32, 48, 37), moe(6, 2, 40, 0.9, shared=(56, 1.6))), (rotary(6, 3, 48, 40, 32, scaling=slow), dense(200)),
                                  (windowed(4, 4, 64, 24, 300), None), (rotary(6, 3, 48, 40, 32, scale=0.11, scaling=slow, kv_from=1), moe(5, 3, 48, 1.4)),
                                  (windowed(5, 1, 40, 56, 90), dense(88)), (rotary(4, 2, 64, 64, 64, base=900.0), None),
                                  (rotary(6, 3, 48, 40, 32, scaling=slow, kv_from=1), moe(7, 1, 24, 2.0, shared=(32, 0.5))),
                                  (windowed(3, 3, 24, 32, 256), dense(64))]),
        "wide": model(256, 512, [(rotary(8, 2, 128, 128, 64, scaling=(8.0, 1.0, 4.0, 512)), dense(512)), (windowed(8, 8, 64, 64, 129), moe(16, 4, 128, shared=(128, 1.2))),
                                 (windowed(16, 2, 128, 128, 300), dense(384)), (rotary(8, 2, 128, 128, 64, scaling=(8.0, 1.0, 4.0, 512), kv_from=0), moe(8, 2, 192, shared=(320, 3.0))),
                                 (windowed(8, 8, 64, 64, 257), dense(512))], eps=1e-6, cap=30.0),
        "odd": model(50, 301, [(rotary(3, 1, 20, 9, 6), moe(3, 3, 27, shared=(13, 0.8))), (windowed(3, 3, 17, 20, 64), None), (windowed(6, 2, 12, 20, 5), moe(6, 2, 31)),
                               (rotary(3, 1, 20, 9, 6, kv_from=0), dense(75)), (rotary(2, 2, 30, 14, 0), dense(19))], cap=8.0),
        "ones": model(64, 128, [(windowed(1, 1, 8, 8, 1), moe(1, 1, 16, shared=(8, 1.0))), (rotary(1, 1, 16, 16, 16), dense(8)), (rotary(1, 1, 16, 16, 16, kv_from=1), None),
                                (windowed(1, 1, 16, 8, 2), moe(2, 2, 8, shared=(16, 1.0)))], cap=50.0),
        "many_heads": model(192, 256, [(windowed(40, 2, 72, 96, 500), moe(40, 6, 48, shared=(96, 1.1))), (rotary(33, 1, 24, 16, 16, scaling=(3.0, 2.0, 2.5, 100)), moe(24, 5, 32)),
                                       (rotary(20, 5, 96, 160, 80), dense(600)), (windowed(12, 12, 160, 32, 256), None), (rotary(33, 1, 24, 16, 16, scaling=(3.0, 2.0, 2.5, 100), kv_from=1), dense(96))]),
    }


def random_weights(cfg, seed=0):
    """bf16 tensors with the names a checkpoint of the family has; norm weights, sinks and biases are not trivial."""
    g = torch.Generator().manual_seed(seed)
    n = lambda *s, std=1.0: torch.randn(*s, generator=g) * std
    width, out = cfg["width"], {}

    def linear(name, rows, cols, gain=1.0):
        out[name] = n(rows, cols, std=gain * cols ** -0.5)

    def gated(name, ff):
        linear(name + ".gate", ff, width, 1.5), linear(name + ".up", ff, width, 1.5), linear(name + ".down", width, ff, 2.0)

    linear("embed", cfg["vocab"], width, gain=width ** 0.5)
    for i, layer in enumerate(cfg["layers"]):
        p, m, ff = f"l{i}.", layer["mixer"], layer["mlp"]
        x, h, kv = p + "mix.", m["heads"], m["kv_heads"]
        out[p + "norm1"] = n(width, std=0.3)
        parts = [("q", h * m["dim"])] + ([] if "kv_from" in m else [("k", kv * m["dim"]), ("v", kv * m["vdim"])])
        for name, rows in parts:
            linear(x + name, rows, width)
        if layer["type"] == "attention":
            out[x + "q.norm"], out[x + "k.norm"] = 1.0 + n(h * m["dim"], std=0.3), 1.0 + n(kv * m["dim"], std=0.3)
            out[x + "sink"] = 2.0 + n(h)
            linear(x + "g", h, width)
        else:
            for name, rows in parts:
                out[f"{x}{name}.b"] = n(rows, std=0.7)
                if name != "v":
                    out[f"{x}{name}.norm"] = 1.0 + n(m["dim"], std=0.3)
        linear(x + "o", width, h * m["vdim"])
        if ff is None:
            continue
        out[p + "norm2"] = n(width, std=0.3)
        if ff["kind"] == "dense":
            linear(p + "mlp.up", ff["ff"], width), linear(p + "mlp.down", width, ff["ff"], 2.0)
            continue
        linear(p + "mlp.router", ff["router"]["experts"], width, 2.0)
        out[p + "mlp.router.b"] = n(ff["router"]["experts"])
        for e in range(ff["router"]["experts"]):
            gated(f"{p}mlp.e{e}", ff["expert"]["ff"])
        if "shared" in ff:
            gated(p + "mlp.shared", ff["shared"]["ff"])
            linear(p + "mlp.shared.sg", 1, width)
    out["final.norm"] = n(width, std=0.3)
    return {k: v.to(torch.bfloat16).contiguous() for k, v in out.items()}
