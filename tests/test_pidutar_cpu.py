"""Pidutar on the host: configuration, weight files, the cache it asks for, and the oracle against itself and
against mistakes planted in it."""
import json
import math

import pytest
import torch

from oracle import pidutar as plain
from nanovllm_amd.context import RowGroup
from nanovllm_amd.engine import EngineConfig, Scheduler, registry
from nanovllm_amd.engine import latent as latent_module
from nanovllm_amd.engine.latent import LatentSpec
from nanovllm_amd.engine.mlstm import MlstmSpec
from nanovllm_amd.engine.pidutar import Pidutar, PidutarConfig
import pidutar_cases as cases

F64 = torch.float64


# ---- the oracle against itself and against hand-made values -----------------------------------------

def test_oracle_rotation_turns_neighbours():
    g = torch.Generator().manual_seed(0)
    q = torch.randn(1, 1, 10, generator=g, dtype=F64).expand(9, 1, 10)
    r = plain.rotate_neighbours(q, 50.0, 6)
    assert torch.equal(r[..., 6:], q[..., 6:]) and torch.equal(r[0], q[0])
    gram = r[:, 0, :6] @ r[:, 0, :6].T                        # depends on the distance only
    for d in range(9):
        assert torch.allclose(torch.diagonal(gram, d), gram[0, d].expand(9 - d))
    u, v, a = float(q[0, 0, 2]), float(q[0, 0, 3]), 3.0 * 50.0 ** (-2 / 6)
    assert float(r[3, 0, 2]) == pytest.approx(u * math.cos(a) - v * math.sin(a)) and float(r[3, 0, 3]) == pytest.approx(v * math.cos(a) + u * math.sin(a))


def test_oracle_window():
    vis = plain.window_visible(6, 3)
    assert [int(r.sum()) for r in vis] == [1, 2, 3, 3, 3, 3] and bool(vis[5, 3]) and not bool(vis[5, 2]) and not bool(vis[2, 3])
    assert torch.equal(plain.window_visible(4, 1), torch.eye(4, dtype=torch.bool))


def test_oracle_memory_is_the_weighted_sum():
    """Without its reference m the recurrence is a plain weighted sum; m only decides where the two floors lie."""
    g = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(12, 2, 5, generator=g, dtype=F64) for _ in range(3))
    log_in, log_keep = 2.0 * torch.randn(12, 2, generator=g, dtype=F64), -torch.rand(12, 2, generator=g, dtype=F64)
    got = plain.matrix_memory(q, k, v, log_in, log_keep)
    for h in range(2):
        run = log_keep[:, h].cumsum(0)
        for t in range(12):
            w = torch.exp(run[t] - run[: t + 1] + log_in[: t + 1, h]) * (k[: t + 1, h] @ q[t, h])
            top = max([float(run[t])] + [float(run[t] - run[s] + log_in[s, h]) for s in range(t + 1)])
            want = (w @ v[: t + 1, h]) / (max(abs(float(w.sum())), 1.0) + 1e-6 * math.exp(top))
            assert torch.allclose(got[t, h], want), (h, t)


def test_oracle_gates_and_router():
    assert float(plain.soft_cap(torch.tensor(1e9, dtype=F64), 7.0)) == pytest.approx(7.0)
    for z in (-800.0, -3.0, 0.0, 40.0):
        assert float(plain.log_sigmoid(torch.tensor(z, dtype=F64))) == pytest.approx(z if z < -700 else -math.log1p(math.exp(-z)), abs=1e-12)
    chosen, weight = plain.route(torch.tensor([[0.0, math.log(3.0), math.log(2.0)]], dtype=F64), 2, 5.0)
    assert chosen.tolist() == [[1, 2]] and weight[0].tolist() == pytest.approx([3.0, 2.0])


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
    cfg = PidutarConfig.from_raw(raw)
    assert isinstance(cfg.layers[0].mixer, MlstmSpec) and isinstance(cfg.layers[1].mixer, LatentSpec) and cfg.num_hidden_layers == 7
    assert cfg.layers[1].mlp is None and cfg.layers[3].mixer.kv_from == 1 and cfg.layers[3].mixer.window == 300 and cfg.layers[3].mlp.top == 3
    assert (cfg.residual_mult, cfg.logit_scale, cfg.embed_scale) == (0.6, 1.4, 0.9) and cfg.layers[2].mixer.gate_cap == 11.0
    (tmp_path / "config.json").write_text(json.dumps(raw))
    assert registry.load_config(str(tmp_path)) == cfg and registry.model_class(cfg) is Pidutar
    assert registry.kernels_of(str(tmp_path)) == registry.kernels_for(cfg) == "latent"
    mixer = ("layers", 3, "mixer")
    for path, value in ((("layers", 0, "type"), "other"), (("layers", 0, "mlp", "kind"), "dense"), (("layers", 0, "mlp", "router", "top"), 6),
                        (mixer + ("kv_from",), 3), (mixer + ("kv_from",), 0), (mixer + ("kv_from",), 4), (mixer + ("kv_from",), 70),
                        (mixer + ("kv_rank",), 80), (mixer + ("rot", "base"), 9.0), (("layers", 6, "mixer", "kv_from"), 3),
                        (mixer + ("rot", "dims"), 16), (mixer + ("mask", "size"), 0), (("layers", 2, "mixer", "gate_cap"), 0.0), (("layers",), [])):
        with pytest.raises(ValueError):
            PidutarConfig.from_raw(_bad(raw, path, value))
    assert EngineConfig(cfg, dtype="float32", max_num_batched_tokens=600, max_model_len=4096).torch_dtype is torch.float32


def test_weights_land_where_they_belong(tmp_path):
    raw = cases.configs()["mixed"]
    w = cases.random_weights(raw, 3)
    folder = cases.write_model(tmp_path, raw, w)
    m = Pidutar(PidutarConfig.from_raw(raw), 64, torch.device("cpu"))
    m.load_weights(folder)
    f = {k: v.float() for k, v in w.items()}
    own, reads, mem = m.layer_weights[1].mix, m.layer_weights[3].mix, m.layer_weights[0]
    assert own.down.shape[0] % 8 == 0 and torch.equal(own.down[: 56 + 96 + 6], torch.cat([f["l1.mix.dq"], f["l1.mix.dkv"], f["l1.mix.g"]]))
    assert not own.down[56 + 96 + 6:].any() and torch.equal(reads.down[: 40 + 3], torch.cat([f["l3.mix.dq"], f["l3.mix.g"]])) and reads.kv_norm is None
    x, c = torch.randn(6, 48), torch.randn(72)
    assert torch.allclose(torch.einsum("hd,hrd,r->h", x, own.uk_t, c), (x * (f["l1.mix.uk"] @ c).view(6, 48)).sum(1), rtol=1e-4, atol=1e-4)
    assert torch.equal(own.uv.reshape(240, 72), f["l1.mix.uv"]) and torch.equal(own.ukv, torch.cat([f["l1.mix.uk"], f["l1.mix.uv"]]))
    assert torch.equal(mem.mix.gates, torch.cat([f["l0.mix.i"], f["l0.mix.f"]])) and torch.equal(mem.mix.gate_bias, torch.cat([f["l0.mix.i.b"], f["l0.mix.f.b"]]))
    assert mem.mix.gate_bias.dtype == torch.float32 and torch.equal(mem.ls2, f["l0.ls2"])
    assert torch.equal(mem.mlp.gate_up[4], torch.cat([f["l0.mlp.e4.gate"], f["l0.mlp.e4.up"]])) and torch.equal(mem.mlp.down[2], f["l0.mlp.e2.down"])
    assert m.layer_weights[1].mlp is None and m.layers[3].mixer.source is m.layers[1].mixer and m.layers[6].mixer.source is m.layers[1].mixer
    del w["l3.ls1"]
    with pytest.raises(KeyError, match="l3.ls1"):
        m.load_weights(cases.write_model(tmp_path / "b", raw, w))
    w = cases.random_weights(raw, 3)
    w["l3.mix.dkv"] = w["l1.mix.dkv"].clone()
    with pytest.raises(ValueError, match="l3.mix.dkv"):
        m.load_weights(cases.write_model(tmp_path / "c", raw, w))


def test_cache_is_one_row_per_token_and_source_layer():
    cfg = PidutarConfig.from_raw(cases.configs()["mixed"])
    m = Pidutar(cfg, 64, torch.device("cpu"))
    assert m.kv_bytes_per_token() == 4 * (72 + 24 + 40 + 8)
    assert m.state_bytes_per_slot() == 4 * (3 * (32 * 48 + 32 + 1) + 2 * (64 * 24 + 64 + 1))
    m.bind_cache(3, 256, 2)
    assert m.layers[1].mixer.cache.shape == (3, 256, 96) and m.layers[3].mixer.cache is None and m.layers[0].mixer.state.shape == (2, 3, 32, 48)
    m.unbind_cache()
    assert m.layers[1].mixer.cache is None and m.layers[0].mixer.top is None
    s = Scheduler(EngineConfig(cfg, max_num_seqs=3, max_num_batched_tokens=512, num_kvcache_blocks=4, max_model_len=2048))
    assert s.portions and s.block_manager.num_state_slots == 3


def test_which_portions_are_multiplied_out(monkeypatch):
    monkeypatch.setattr(torch.Tensor, "pin_memory", lambda self: self)
    none = torch.zeros(0, dtype=torch.int32)
    group = lambda spans: RowGroup(0, sum(c for _, c in spans), len(spans), none, none, none, none, none, none, max(c for _, c in spans), spans)
    cpu = torch.device("cpu")
    cu, n = latent_module.visible_keys(group([(0, 300), (1000, 500)]), 100, cpu)
    assert cu.tolist() == [0, 300, 899] and n == 899              # 99 tokens before the second portion are in its window
    g = group([(4000, 2)])
    assert latent_module.visible_keys(g, 5000, cpu) is None and g.shared == {("keys", 5000): None}
    assert latent_module.visible_keys(group([(0, 8)]), 100, cpu) is None
    assert latent_module.visible_keys(RowGroup(0, 1, 1, none, none, none, none), 100, cpu) is None     # single tokens
    assert latent_module.visible_keys(group([(0, latent_module.EXPAND_MAX_KEYS + 1)]), 100, cpu) is None


# ---- the engine tests' models show a planted mistake ---------------------------------------------------

_true = {n: getattr(plain, n) for n in ("window_visible", "rotate_neighbours", "matrix_memory", "soft_cap", "log_sigmoid", "route", "unit_rms",
                                        "centred_weight_norm", "latent_keys", "latent_attention", "mlstm", "softmax_attention", "gated_mlp")}


def _restart(at):
    return lambda *x: torch.cat([_true["matrix_memory"](*(t[:at] for t in x)), _true["matrix_memory"](*(t[at:] for t in x))])


def _unrotated_cache(h, w, m, eps):
    latent, _ = _true["latent_keys"](h, w, m, eps)
    return latent, (h @ w("dkv").T)[:, m["kv_rank"]:]


def _unnormed_cache(h, w, m, eps):
    _, turned = _true["latent_keys"](h, w, m, eps)
    return (h @ w("dkv").T)[:, : m["kv_rank"]], turned


def _without(name, value):
    """The mixer with one of its tensors replaced."""
    def swap(fn):
        def run(*a):
            i = next(j for j, x in enumerate(a) if callable(x))
            w = a[i]
            return fn(*a[:i], lambda n: value(w(n)) if n == name else w(n), *a[i + 1:])
        return run
    return swap


MISTAKES = {
    "a window one key longer": dict(window_visible=lambda t, size: _true["window_visible"](t, size + 1)),
    "a window one key shorter": dict(window_visible=lambda t, size: _true["window_visible"](t, max(1, size - 1))),
    "keys of the page before unseen": dict(window_visible=lambda t, size: _true["window_visible"](t, size) & ((torch.arange(t)[:, None] // 256) == (torch.arange(t)[None] // 256))),
    "a memory lost at token 256": dict(matrix_memory=_restart(256)),
    "a forget gate that is not capped": dict(soft_cap=lambda z, cap: z),
    "a forget gate without its logarithm": dict(log_sigmoid=lambda z: -torch.sigmoid(-z)),
    "rotation of halves": dict(rotate_neighbours=lambda x, base, dims: torch.cat(
        [_true["rotate_neighbours"](torch.stack([x[..., : dims // 2], x[..., dims // 2: dims]], -1).flatten(-2), base, dims).unflatten(-1, (dims // 2, 2)).transpose(-1, -2).flatten(-2),
         x[..., dims:]], -1)),
    "a cached key part that is not rotated": dict(latent_keys=_unrotated_cache),
    "a latent that is not normed": dict(latent_keys=_unnormed_cache),
    "one expert fewer": dict(route=lambda z, top, scale: _true["route"](z, max(1, top - 1), scale)),
    "expert weights that are not normalised": dict(route=lambda z, top, scale: (_true["route"](z, top, scale)[0], torch.topk(torch.softmax(z, -1), top, -1)[0] * scale)),
    "expert weights without their scale": dict(route=lambda z, top, scale: _true["route"](z, top, 1.0)),
    "norm weights without the one": dict(centred_weight_norm=lambda x, w, eps: plain.unit_rms(x, eps) * w),
    "no gate per head": dict(latent_attention=_without("g", lambda t: 0 * t)(_true["latent_attention"])),
    "no output gate": dict(mlstm=_without("g", lambda t: 0 * t)(_true["mlstm"])),
    "gates without their bias": dict(mlstm=_without("f.b", lambda t: 0 * t)(_true["mlstm"])),
    "a head norm without its weight": dict(mlstm=_without("norm", lambda t: 0 * t + 1)(_true["mlstm"])),
    "a query latent that is not normed": dict(latent_attention=_without("dq.norm", lambda t: 0 * t + 1)(_true["latent_attention"])),
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


@pytest.mark.parametrize("part", ["embedding", "residual_mult", "logit_scale", "window"])
def test_planted_constants_show_in_the_logits(part):
    cfg = cases.configs()["mixed"]
    weights = cases.random_weights(cfg, 1)
    ids = cases.tokens(80, cfg["vocab"], 5)
    want = plain.forward(cfg, weights, ids)
    bad = json.loads(json.dumps(cfg))
    if part == "embedding":
        bad["embedding"]["scale"] = 1.0
    elif part == "window":                                    # a layer with the window of the one whose cache it reads
        bad["layers"][3]["mixer"]["mask"]["size"] = 37
    else:
        bad[part] = 1.0
    assert float(cases.row_error(plain.forward(bad, weights, ids), want).max()) > 0.15
