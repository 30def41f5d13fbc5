"""Sokolorn on the host: configuration, weight files, the cache it asks for, and the oracle against itself and
against mistakes planted in it."""
import json
import math

import pytest
import torch

from oracle import sokolorn as plain
from nanovllm_amd.engine import EngineConfig, Scheduler, registry
from nanovllm_amd.engine.experts import ExpertsSpec
from nanovllm_amd.engine.masked import ALL_KEYS, HEAD, WHOLE
from nanovllm_amd.engine.mixers import RopeTables, Rotary, RotaryScaling
from nanovllm_amd.engine.sokolorn import DenseSpec, Sokolorn, SokolornConfig
import sokolorn_cases as cases

F64 = torch.float64


# ---- the oracle against itself and against hand-made values -----------------------------------------

def test_oracle_rotation_turns_halves():
    g = torch.Generator().manual_seed(0)
    q = torch.randn(1, 1, 10, generator=g, dtype=F64).expand(9, 1, 10)
    freq = plain.rotation_frequencies(6, 50.0, None)
    r = plain.rotate_halves(q, freq)
    assert torch.equal(r[..., 6:], q[..., 6:]) and torch.equal(r[0], q[0])
    gram = r[:, 0, :6] @ r[:, 0, :6].T                        # depends on the distance only
    for d in range(9):
        assert torch.allclose(torch.diagonal(gram, d), gram[0, d].expand(9 - d))
    u, v, a = float(q[0, 0, 1]), float(q[0, 0, 4]), 3.0 * 50.0 ** (-2 / 6)
    assert float(r[3, 0, 1]) == pytest.approx(u * math.cos(a) - v * math.sin(a)) and float(r[3, 0, 4]) == pytest.approx(v * math.cos(a) + u * math.sin(a))


def test_oracle_scaled_frequencies():
    """Wavelengths below original / high stay, beyond original / low they are stretched, and the blend meets both ends."""
    base, dims, scaling = 1000.0, 64, dict(factor=5.0, low=2.0, high=8.0, original=400)
    plainly, scaled = plain.rotation_frequencies(dims, base, None), plain.rotation_frequencies(dims, base, scaling)
    kinds = set()
    for f, s in zip(plainly, scaled):
        wave = 2 * math.pi / f
        if wave < 400 / 8:
            kinds.add("fast")
            assert s == f
        elif wave > 400 / 2:
            kinds.add("slow")
            assert s == pytest.approx(f / 5)
        else:
            kinds.add("between")
            part = (400 / wave - 2.0) / 6.0
            assert s == pytest.approx((1 - part) * f / 5 + part * f) and f / 5 <= s <= f
    assert kinds == {"fast", "slow", "between"}


def test_oracle_window_and_sink():
    vis = plain.visible(6, 3)
    assert [int(r.sum()) for r in vis] == [1, 2, 3, 3, 3, 3] and bool(vis[5, 3]) and not bool(vis[5, 2]) and not bool(vis[2, 3])
    assert torch.equal(plain.visible(4, 1), torch.eye(4, dtype=torch.bool)) and int(plain.visible(5, None).sum()) == 15
    q, k, v = torch.zeros(2, 2, 3, dtype=F64), torch.zeros(2, 1, 3, dtype=F64), torch.ones(2, 1, 1, dtype=F64)
    o = plain.softmax_attention(q, k, v, 1.0, plain.visible(2, None), torch.tensor([0.0, math.log(6.0)], dtype=F64))
    assert o[:, 0, 0].tolist() == pytest.approx([1 / 2, 2 / 3]) and o[:, 1, 0].tolist() == pytest.approx([1 / 7, 2 / 8])


def test_oracle_router_and_gates():
    chosen, weight = plain.route(torch.tensor([[0.0, math.log(3.0), -9.0, math.log(2.0)]], dtype=F64), 2)
    assert chosen.tolist() == [[1, 3]] and weight[0].tolist() == pytest.approx([0.6, 0.4])
    one = lambda v: torch.tensor([[v]], dtype=F64)
    act = lambda g, u: float(plain.clamped_mlp(one(1.0), one(g), one(u), one(1.0), 1.5))
    sig = lambda z: 1 / (1 + math.exp(-1.702 * z))
    assert act(9.0, -9.0) == pytest.approx(1.5 * sig(1.5) * -0.5) and act(-9.0, 9.0) == pytest.approx(-9.0 * sig(-9.0) * 2.5)
    assert float(plain.squared_relu_mlp(one(-2.0), one(3.0), one(1.0))) == 0.0 and float(plain.squared_relu_mlp(one(2.0), one(3.0), one(0.5))) == 18.0
    assert float(plain.soft_cap(one(1e9), 7.0)) == pytest.approx(7.0)


# ---- configuration, registry, weight files ---------------------------------------------------------

def _bad(raw, path, value):
    bad = json.loads(json.dumps(raw))
    at = bad
    for p in path[:-1]:
        at = at[p]
    at[path[-1]] = value
    return bad


def test_config_is_read_and_checked(tmp_path):
    raw = cases.configs()["mixed"]
    cfg = SokolornConfig.from_raw(raw)
    first, second, fourth = cfg.layers[0].mixer, cfg.layers[1].mixer, cfg.layers[3].mixer
    assert (first.window, first.rot, first.qk_norm, first.bias, first.sink, first.gate) == (37, None, WHOLE, False, True, True)
    assert (second.window, second.qk_norm, second.bias, second.sink, second.gate) == (None, HEAD, True, False, False)
    assert second.rot == Rotary(4000.0, 32, RotaryScaling(6.0, 1.5, 5.0, 300.0)) and fourth.kv_from == 1 and fourth.scale == 0.11
    assert cfg.layers[2].mlp is None and cfg.layers[1].mlp == DenseSpec(200) and isinstance(cfg.layers[3].mlp, ExpertsSpec)
    moe = cfg.layers[0].mlp
    assert (moe.experts, moe.top, moe.ff, moe.gate.limit, moe.shared.ff, moe.shared.gate.limit) == (6, 2, 40, 0.9, 56, 1.6) and cfg.layers[3].mlp.shared is None
    assert cfg.num_hidden_layers == 8 and cfg.logit_softcap == 20.0
    (tmp_path / "config.json").write_text(json.dumps(raw))
    assert registry.load_config(str(tmp_path)) == cfg and registry.model_class(cfg) is Sokolorn
    assert registry.kernels_of(str(tmp_path)) == registry.kernels_for(cfg) == "masked"
    mixer = ("layers", 3, "mixer")
    for path, value in ((("layers", 0, "type"), "other"), (("layers", 0, "mlp", "kind"), "gated"), (("layers", 0, "mlp", "router", "top"), 7),
                        (mixer + ("kv_from",), 3), (mixer + ("kv_from",), 0), (mixer + ("kv_from",), 5), (mixer + ("kv_from",), 70), (mixer + ("kv_from",), -1),
                        (mixer + ("kv_heads",), 2), (mixer + ("rot", "base"), 9.0), (mixer + ("rot", "scaling", "factor"), 7.0), (mixer + ("dim",), 56),
                        (("layers", 6, "mixer", "kv_from"), 3), (("layers", 5, "mixer", "rot", "dims"), 72), (("layers", 5, "mixer", "rot", "dims"), 31),
                        (("layers", 0, "mixer", "mask", "size"), 0), (("layers", 0, "mixer", "kv_heads"), 4),
                        (("layers", 1, "mixer", "rot", "scaling", "high"), 1.0), (("layers",), [])):
        with pytest.raises(ValueError):
            SokolornConfig.from_raw(_bad(raw, path, value))
    assert EngineConfig(cfg, dtype="float32", max_num_batched_tokens=600, max_model_len=4096).torch_dtype is torch.float32


def test_weights_land_where_they_belong(tmp_path):
    raw = cases.configs()["mixed"]
    w = cases.random_weights(raw, 3)
    m = Sokolorn(SokolornConfig.from_raw(raw), 64, torch.device("cpu"))
    m.load_weights(cases.write_model(tmp_path, raw, w))
    f = {k: v.float() for k, v in w.items()}
    assert m.head is m.embed and torch.equal(m.embed, f["embed"]) and sum(p is m.embed for p in m.parameters()) == 1
    win, rot, reads = (m.layer_weights[i].mix for i in (0, 1, 3))
    rows = 6 * 32 + 2 * (32 + 48) + 6
    assert win.qkvg.shape[0] % 8 == 0 and torch.equal(win.qkvg[:rows], torch.cat([f[f"l0.mix.{n}"] for n in "qkvg"])) and not win.qkvg[rows:].any()
    assert torch.equal(win.sinks, f["l0.mix.sink"]) and win.sinks.dtype == torch.float32 and win.bias is None and win.k_norm.shape == (64,)
    assert torch.equal(rot.bias, torch.cat([f[f"l1.mix.{n}.b"] for n in "qkv"])) and rot.sinks is None and rot.q_norm.shape == (48,)
    assert torch.equal(reads.qkvg, f["l3.mix.q"]) and torch.equal(reads.bias, f["l3.mix.q.b"]) and reads.k_norm is None
    moe = m.layer_weights[0].mlp
    assert torch.equal(moe.router, torch.cat([f["l0.mlp.router"], f["l0.mlp.shared.sg"]])) and torch.equal(moe.bias[:6], f["l0.mlp.router.b"]) and moe.bias[6] == 0
    assert torch.equal(moe.gate_up[4], torch.cat([f["l0.mlp.e4.gate"], f["l0.mlp.e4.up"]])) and torch.equal(moe.down[2], f["l0.mlp.e2.down"])
    assert torch.equal(moe.shared_gate_up, torch.cat([f["l0.mlp.shared.gate"], f["l0.mlp.shared.up"]])) and torch.equal(moe.shared_down, f["l0.mlp.shared.down"])
    assert m.layer_weights[3].mlp.router.shape[0] == 5 and m.layer_weights[3].mlp.shared_down is None and m.layer_weights[2].norm2 is None
    assert m.layers[3].mixer.source is m.layers[1].mixer and m.layers[6].mixer.source is m.layers[1].mixer and m.layers[1].mixer.span == ALL_KEYS
    del w["l3.norm1"]
    with pytest.raises(KeyError, match="l3.norm1"):
        m.load_weights(cases.write_model(tmp_path / "b", raw, w))
    w = cases.random_weights(raw, 3)
    w["l3.mix.k"] = w["l1.mix.k"].clone()
    with pytest.raises(ValueError, match="l3.mix.k"):
        m.load_weights(cases.write_model(tmp_path / "c", raw, w))


def test_cache_is_kept_by_layers_with_keys_of_their_own():
    cfg = SokolornConfig.from_raw(cases.configs()["mixed"])
    m = Sokolorn(cfg, 64, torch.device("cpu"))
    assert m.kv_bytes_per_token() == 4 * (2 * (32 + 48) + 3 * (48 + 40) + 4 * (64 + 24) + 1 * (40 + 56) + 2 * (64 + 64) + 3 * (24 + 32))
    assert m.state_bytes_per_slot() == 0
    m.bind_cache(3, 256, 2)
    assert m.layers[0].mixer.k_cache.shape == (3, 256, 2, 32) and m.layers[0].mixer.v_cache.shape == (3, 256, 2, 48) and m.layers[3].mixer.k_cache is None
    m.unbind_cache()
    assert m.layers[0].mixer.k_cache is None and m.layers[1].mixer.v_cache is None
    s = Scheduler(EngineConfig(cfg, max_num_seqs=3, max_num_batched_tokens=512, num_kvcache_blocks=4, max_model_len=2048))
    assert s.portions and s.block_manager.num_state_slots == 3


@pytest.mark.parametrize("scaling", [None, (6.0, 1.5, 5.0, 300), (2.0, 1.0, 1.0, 64), (8.0, 0.5, 30.0, 4096)])
def test_rotary_tables_follow_the_scaled_frequencies(scaling):
    rot = Rotary(4000.0, 48, None if scaling is None else RotaryScaling(*map(float, scaling)))
    table = RopeTables(900, torch.device("cpu")).get(rot).double()
    raw = None if scaling is None else dict(zip(("factor", "low", "high", "original"), scaling))
    if scaling is not None and scaling[1] == scaling[2]:
        raw["high"] = raw["low"] * (1 + 1e-12)               # (the blend's width is nothing)
    freq = torch.tensor(plain.rotation_frequencies(48, 4000.0, raw), dtype=F64)
    angle = torch.outer(torch.arange(900, dtype=F64), freq)
    assert float((table - torch.cat([angle.cos(), angle.sin()], 1)).abs().max()) < 1e-6


# ---- the engine tests' models show a planted mistake ---------------------------------------------------

_true = {n: getattr(plain, n) for n in ("visible", "rotate_halves", "rotation_frequencies", "route", "unit_rms", "whole_norm", "head_norm", "centred_weight_norm",
                                        "windowed_attention", "rotary_attention", "keys_and_values", "softmax_attention", "clamped_mlp", "shared_part", "soft_cap",
                                        "head_gates", "squared_relu_mlp", "expert_mixture")}


def _without(name, value):
    """The function with one of its tensors replaced."""
    def swap(fn):
        def run(*a):
            i = next(j for j, x in enumerate(a) if callable(x))
            w = a[i]
            return fn(*a[:i], lambda n: value(w(n)) if n == name else w(n), *a[i + 1:])
        return run
    return swap


def _in_pages(fn):
    return lambda t, size: fn(t, size) & ((torch.arange(t)[:, None] // 256) == (torch.arange(t)[None] // 256))


MISTAKES = {
    "a window one key longer": dict(visible=lambda t, size: _true["visible"](t, None if size is None else size + 1)),
    "a window one key shorter": dict(visible=lambda t, size: _true["visible"](t, None if size is None else max(1, size - 1))),
    "a window over all keys": dict(visible=lambda t, size: _true["visible"](t, None)),
    "keys of the page before unseen": dict(visible=_in_pages(_true["visible"])),
    "no sink": dict(softmax_attention=lambda q, k, v, scale, seen, sink=None: _true["softmax_attention"](q, k, v, scale, seen)),
    "a sink that is scaled": dict(softmax_attention=lambda q, k, v, scale, seen, sink=None: _true["softmax_attention"](q, k, v, scale, seen, None if sink is None else sink * scale)),
    "rotation of neighbours": dict(rotate_halves=lambda x, f: torch.cat(
        [_true["rotate_halves"](x[..., : 2 * len(f)].unflatten(-1, (len(f), 2)).transpose(-1, -2).flatten(-2), f).unflatten(-1, (2, len(f))).transpose(-1, -2).flatten(-2),
         x[..., 2 * len(f):]], -1)),
    "no rotation": dict(rotate_halves=lambda x, f: x),
    "frequencies that are not scaled": dict(rotation_frequencies=lambda dims, base, scaling: _true["rotation_frequencies"](dims, base, None)),
    "frequencies all divided": dict(rotation_frequencies=lambda dims, base, scaling: [f / (scaling["factor"] if scaling else 1) for f in _true["rotation_frequencies"](dims, base, None)]),
    "queries and keys normed by head": dict(whole_norm=lambda x, w, eps: plain.unit_rms(x.unflatten(-1, (-1, 8)), eps).flatten(-2) * w),
    "queries and keys not normed": dict(whole_norm=lambda x, w, eps: x * w),
    "heads not normed": dict(head_norm=lambda x, w, eps: x * w),
    "heads normed without their weight": dict(head_norm=lambda x, w, eps: plain.unit_rms(x, eps)),
    "values without their bias": dict(keys_and_values=_without("v.b", lambda t: 0 * t)(_true["keys_and_values"])),
    "keys without their bias": dict(keys_and_values=_without("k.b", lambda t: 0 * t)(_true["keys_and_values"])),
    "queries without their bias": dict(rotary_attention=_without("q.b", lambda t: 0 * t)(_true["rotary_attention"])),
    "no gate per head": dict(head_gates=lambda h, w: torch.ones(h.shape[0], w.shape[0], dtype=h.dtype)),
    "one expert fewer": dict(route=lambda z, top: _true["route"](z, max(1, top - 1))),
    "expert weights from all logits": dict(route=lambda z, top: (_true["route"](z, top)[0], torch.topk(torch.softmax(z, -1), top, -1)[0])),
    "a router without its bias": dict(expert_mixture=_without("router.b", lambda t: 0 * t)(_true["expert_mixture"])),
    "no shared expert": dict(shared_part=lambda h, w, limit: 0 * h),
    "a shared expert without its gate": dict(shared_part=lambda h, w, limit: 2 * _without("shared.sg", lambda t: 0 * t)(_true["shared_part"])(h, w, limit)),
    "experts without limits": dict(clamped_mlp=lambda h, g, u, d, limit: _true["clamped_mlp"](h, g, u, d, 1e9)),
    "relu that is not squared": dict(squared_relu_mlp=lambda h, up, down: torch.relu(h @ up.T) @ down.T),
    "norm weights without the one": dict(centred_weight_norm=lambda x, w, eps: plain.unit_rms(x, eps) * w),
    "logits that are not capped": dict(soft_cap=lambda z, cap: z),
}


@pytest.mark.parametrize("mistake", sorted(MISTAKES))
def test_planted_mistakes_show_in_the_logits(monkeypatch, mistake):
    cfg = cases.configs()["mixed"]
    weights = cases.random_weights(cfg, 1)
    ids = cases.tokens(300, cfg["vocab"], 5)
    want = plain.forward(cfg, weights, ids)
    for name, wrong in MISTAKES[mistake].items():
        monkeypatch.setattr(plain, name, wrong)
    err = cases.row_error(plain.forward(cfg, weights, ids), want)
    # far beyond the fp32 limit everywhere it acts, and beyond the bf16 one
    assert float(err.max()) > 0.15, (mistake, float(err.max()), float(err.mean()))


def test_planted_sources_and_limits_show_in_the_logits():
    """Another layer's keys instead of the named one's; the experts' limit for the shared one."""
    layers = [(cases.rotary(4, 2, 16, 16, 16), cases.dense(64)), (cases.rotary(4, 2, 16, 16, 16), cases.moe(4, 2, 32, 0.5, shared=(32, 3.0))),
              (cases.rotary(4, 2, 16, 16, 16, kv_from=0), cases.dense(64))]
    cfg = cases.model(64, 200, layers)
    weights = cases.random_weights(cfg, 2)
    ids = cases.tokens(60, 200, 3)
    want = plain.forward(cfg, weights, ids)
    for path, value in ((("layers", 2, "mixer", "kv_from"), 1), (("layers", 1, "mlp", "shared", "limit"), 0.5), (("layers", 1, "mlp", "expert", "limit"), 3.0)):
        assert float(cases.row_error(plain.forward(_bad(cfg, path, value), weights, ids), want).max()) > 0.15, path
