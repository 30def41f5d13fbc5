"""Small random Pidutar models for the tests (sizes and values made here)."""
import torch

from kaparax_cases import cut, row_error, tokens, write_model  # noqa: F401


def latent(heads, dim, rot, vdim, q_rank, kv_rank, window, scale=None, base=3000.0, kv_from=None):
    m = dict(heads=heads, dim=dim, rot_dim=rot, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, mask=dict(size=window),
             scale=scale or 1.7 * (dim + rot) ** -0.5, rot=dict(base=base, dims=rot))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type="latent_attention", mixer=m)


def mlstm(heads, dim, vdim, cap=6.0):
    return dict(type="mlstm", mixer=dict(heads=heads, dim=dim, vdim=vdim, gate_cap=cap))


def moe(experts, top, ff, scale=1.3):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top, scale=scale))


def model(width, vocab, layers, embed=0.9, mult=0.6, logit=1.4, eps=1e-5):
    return dict(architecture="Pidutar", vocab=vocab, width=width, embedding=dict(scale=embed), residual_mult=mult, logit_scale=logit,
                norm=dict(eps=eps), layers=[dict(mixer, mlp=ff) for mixer, ff in layers])


def configs():
    """name -> configuration.  Together: windows of 1, below, at and above a page, one and many heads, caches read
    by one and by two later layers with other heads, sizes and windows, layers without a feed-forward, one expert
    and many, every expert chosen, both mixers first and last, sizes off every vector width."""
    return {
        "mixed": model(104, 320, [(mlstm(3, 32, 48), moe(5, 2, 40)), (latent(6, 48, 24, 40, 56, 72, 37), None), (mlstm(2, 64, 24, cap=11.0), None),
                                  (latent(3, 32, 24, 64, 40, 72, 300, kv_from=1), moe(7, 3, 24, scale=0.8)), (latent(4, 40, 8, 32, 24, 40, 90), moe(4, 1, 56)),
                                  (latent(5, 24, 8, 16, 32, 40, 20, kv_from=4), moe(5, 2, 40)), (latent(2, 16, 24, 24, 16, 72, 256, kv_from=1), None)]),
        "wide": model(256, 512, [(latent(8, 128, 64, 128, 192, 512, 300), moe(16, 4, 128)), (mlstm(2, 128, 128, cap=15.0), moe(16, 4, 128)),
                                 (latent(8, 128, 64, 128, 192, 512, 129, kv_from=0), moe(8, 2, 192))], eps=1e-6, mult=1.0, logit=1.0),
        "odd": model(50, 301, [(latent(3, 20, 6, 12, 22, 18, 64), moe(3, 3, 27)), (mlstm(2, 12, 20), None), (mlstm(3, 20, 9, cap=3.0), moe(6, 2, 31)),
                               (latent(2, 9, 6, 7, 10, 18, 5, kv_from=0), moe(3, 2, 13))], embed=2.5),
        "ones": model(64, 128, [(latent(1, 8, 2, 8, 8, 8, 1), moe(1, 1, 16, scale=1.0)), (mlstm(1, 16, 16), moe(2, 1, 8)),
                                (latent(1, 16, 16, 8, 16, 16, 2), moe(2, 2, 8))], embed=1.0, mult=1.0, logit=1.0),
        "many_heads": model(192, 256, [(latent(20, 72, 32, 96, 120, 192, 500), moe(40, 6, 48)), (mlstm(2, 192, 64, cap=9.0), moe(24, 5, 32)),
                                       (latent(33, 24, 32, 16, 64, 192, 256, kv_from=0), None), (mlstm(4, 64, 160), moe(40, 6, 48))]),
    }


def random_weights(cfg, seed=0):
    """bf16 tensors with the names a checkpoint of the family has; norm weights, gains and biases are not trivial."""
    g = torch.Generator().manual_seed(seed)
    n = lambda *s, std=1.0: torch.randn(*s, generator=g) * std
    width, out = cfg["width"], {}

    def linear(name, rows, cols, gain=1.0):
        out[name] = n(rows, cols, std=gain * cols ** -0.5)

    linear("embed", cfg["vocab"], width, gain=width ** 0.5)
    for i, layer in enumerate(cfg["layers"]):
        p, m, ff = f"l{i}.", layer["mixer"], layer["mlp"]
        x = p + "mix."
        out[p + "norm1"], out[p + "ls1"] = n(width, std=0.3), 0.8 + n(width, std=0.3)
        h = m["heads"]
        if layer["type"] == "mlstm":
            for name, rows in (("q", h * m["dim"]), ("k", h * m["dim"]), ("v", h * m["vdim"]), ("g", h * m["vdim"])):
                linear(x + name, rows, width)
            linear(x + "i", h, width, 2.0), linear(x + "f", h, width, 2.0)
            out[x + "i.b"], out[x + "f.b"] = n(h), 4.0 + n(h)
            out[x + "norm"] = 1.0 + n(h * m["vdim"], std=0.3)
        else:
            linear(x + "dq", m["q_rank"], width), linear(x + "uq", h * (m["dim"] + m["rot_dim"]), m["q_rank"])
            out[x + "dq.norm"] = 1.0 + n(m["q_rank"], std=0.3)
            if "kv_from" not in m:
                linear(x + "dkv", m["kv_rank"] + m["rot_dim"], width)
                out[x + "dkv.norm"] = 1.0 + n(m["kv_rank"], std=0.3)
            linear(x + "uk", h * m["dim"], m["kv_rank"]), linear(x + "uv", h * m["vdim"], m["kv_rank"])
            linear(x + "g", h, width)
        linear(x + "o", width, h * m["vdim"])
        if ff is not None:
            out[p + "norm2"], out[p + "ls2"] = n(width, std=0.3), 0.8 + n(width, std=0.3)
            linear(p + "mlp.router", ff["router"]["experts"], width, 2.0)
            for e in range(ff["router"]["experts"]):
                linear(f"{p}mlp.e{e}.gate", ff["expert"]["ff"], width), linear(f"{p}mlp.e{e}.up", ff["expert"]["ff"], width)
                linear(f"{p}mlp.e{e}.down", width, ff["expert"]["ff"], 2.0)
    out["final.norm"] = n(width, std=0.3)
    linear("head", cfg["vocab"], width)
    return {k: v.to(torch.bfloat16).contiguous() for k, v in out.items()}
