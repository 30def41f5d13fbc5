"""Small random Bedenex models for the tests (sizes and values made here)."""
import torch

from kaparax_cases import cut, row_error, tokens, write_model  # noqa: F401


def latent(heads, dim, rot, vdim, rank, scale=None, base=3000.0):
    return dict(type="latent_attention", mixer=dict(heads=heads, dim=dim, rot_dim=rot, vdim=vdim, kv_rank=rank, scale=scale or 1.6 * (dim + rot) ** -0.5,
                                                    rot=dict(base=base, dims=rot)))


def chunked(heads, kv_heads, dim, vdim, chunk, scale=None):
    return dict(type="attention", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=chunk), scale=scale or 1.5 * dim ** -0.5))


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))


def model(width, vocab, layers, loop, eps=1e-5):
    out = dict(architecture="Bedenex", vocab=vocab, width=width, norm=dict(eps=eps), layers=[dict(mixer, mlp=ff) for mixer, ff in layers])
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


def configs():
    """name -> configuration.  Together: loops at the beginning, in the middle and at the end, over one layer and over all, run
    once, twice and more often, and none; chunks of 1, below, at and above a page and beyond every sequence; one and many heads
    and groups, key and value sizes that differ, rotated parts smaller and larger than the others, layers without a
    feed-forward, one expert and many, one chosen and all, sizes off every vector width."""
    return {
        "mixed": model(104, 320, [(chunked(6, 2, 32, 48, 37), dense(200)), (latent(5, 24, 16, 40, 72), moe(6, 2, 40)), (chunked(4, 4, 64, 24, 300), None),
                                  (latent(3, 40, 48, 16, 96, base=500.0), dense(88)), (chunked(5, 1, 40, 56, 90), moe(5, 1, 48))], (1, 4, 2)),
        "wide": model(256, 512, [(latent(8, 128, 64, 128, 512), moe(16, 4, 128)), (chunked(16, 2, 128, 128, 256), dense(512)),
                                 (chunked(8, 8, 64, 64, 130), moe(8, 3, 192)), (latent(20, 64, 32, 64, 256), dense(384))], (0, 2, 3), eps=1e-6),
        "odd": model(50, 301, [(chunked(3, 3, 17, 20, 64), moe(3, 3, 27)), (latent(3, 9, 6, 13, 21), dense(75)), (chunked(6, 2, 12, 9, 5), None),
                               (latent(2, 30, 10, 14, 50), moe(6, 2, 31))], (1, 4, 2)),
        "ones": model(64, 128, [(chunked(1, 1, 8, 8, 1), moe(1, 1, 16)), (latent(1, 8, 2, 8, 8), dense(8)), (chunked(1, 1, 16, 8, 2), moe(2, 2, 8)),
                                (latent(1, 16, 16, 8, 16), None)], (2, 3, 4)),
        "many_heads": model(192, 256, [(chunked(40, 2, 72, 96, 5000), dense(600)), (latent(33, 32, 128, 48, 200), moe(40, 6, 48)),
                                       (chunked(20, 5, 96, 160, 513), moe(24, 5, 32)), (latent(18, 160, 64, 136, 520), dense(96)), (chunked(12, 12, 160, 32, 80), None)], (3, 5, 1)),
        "straight": model(128, 200, [(chunked(4, 2, 32, 32, 64), dense(128)), (latent(4, 32, 32, 32, 64), moe(4, 1, 64))], None),
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
    if "loop" in cfg:
        linear("loop.in", width, 2 * width, 1.2)
        out["loop.step"] = n(cfg["loop"]["times"], width, std=0.5)
    for i, layer in enumerate(cfg["layers"]):
        p, m, ff = f"l{i}.", layer["mixer"], layer["mlp"]
        x, h = p + "mix.", m["heads"]
        out[p + "norm1"] = 1.0 + n(width, std=0.3)
        if layer["type"] == "attention":
            for name, rows in (("q", h * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"]), ("g", h)):
                linear(x + name, rows, width)
            out[x + "r1"], out[x + "r2"] = 0.2 + 1.5 * torch.rand(h, generator=g), 0.05 + torch.rand(h, generator=g)
        else:
            for name, rows, cols in (("q", h * (m["dim"] + m["rot_dim"]), width), ("dkv", m["kv_rank"] + m["rot_dim"], width),
                                     ("uk", h * m["dim"], m["kv_rank"]), ("uv", h * m["vdim"], m["kv_rank"])):
                linear(x + name, rows, cols)
            out[x + "dkv.norm"] = 1.0 + n(m["kv_rank"], std=0.3)
            out[x + "sink"] = 3.0 + n(h)
        linear(x + "o", width, h * m["vdim"], 1.5)
        for name in ("rg1",) + (("rg2",) if ff is not None else ()):
            linear(p + name, width, width)
            out[f"{p}{name}.b"] = 0.5 + n(width, std=0.7)
        if ff is None:
            continue
        if ff["kind"] == "dense":
            linear(p + "mlp.gate", ff["ff"], width, 1.5), linear(p + "mlp.up", ff["ff"], width, 1.5), linear(p + "mlp.down", width, ff["ff"], 2.0)
            continue
        linear(p + "mlp.router", ff["router"]["experts"], width, 2.0)
        for e in range(ff["router"]["experts"]):
            gated(f"{p}mlp.e{e}", ff["expert"]["ff"])
    out["final.norm"] = 1.0 + n(width, std=0.3)
    linear("head", cfg["vocab"], width)
    return {k: v.to(torch.bfloat16).contiguous() for k, v in out.items()}
