"""Bedenex on the host: configuration, weight files, the caches it asks for, and the oracle against itself and
against mistakes planted in it."""
import json
import math

import pytest
import torch

from oracle import bedenex as plain
from nanovllm_amd.engine import EngineConfig, Scheduler, registry
from nanovllm_amd.engine.bedenex import Bedenex, BedenexConfig, DenseSpec, LoopSpec
from nanovllm_amd.engine.experts import SIGMOID, ExpertsSpec
from nanovllm_amd.engine.latent import LatentSpec
from nanovllm_amd.engine.masked import UNIT
from nanovllm_amd.engine.mixers import GELU_CUBIC, GELU_SLOPE, Rotary
import bedenex_cases as cases

F64 = torch.float64


# ---- the oracle against itself and against hand-made values -----------------------------------------

def test_oracle_rotation_turns_halves():
    g = torch.Generator().manual_seed(0)
    q = torch.randn(1, 2, 6, generator=g, dtype=F64).expand(9, 2, 6)
    r = plain.turned(q, 50.0, 6)
    assert torch.equal(r[0], q[0]) and torch.equal(plain.turned(q[:, 1], 50.0, 6), r[:, 1])
    gram = r[:, 0] @ r[:, 0].T                                # depends on the distance only
    for d in range(9):
        assert torch.allclose(torch.diagonal(gram, d), gram[0, d].expand(9 - d))
    u, v, a = float(q[0, 0, 1]), float(q[0, 0, 4]), 3.0 * 50.0 ** (-2 / 6)
    assert float(r[3, 0, 1]) == pytest.approx(u * math.cos(a) - v * math.sin(a)) and float(r[3, 0, 4]) == pytest.approx(v * math.cos(a) + u * math.sin(a))


def test_oracle_chunks_bias_and_sink():
    vis = plain.in_chunk(7, 3)
    assert [int(r.sum()) for r in vis] == [1, 2, 3, 1, 2, 3, 1] and bool(vis[5, 3]) and not bool(vis[3, 2]) and not bool(vis[3, 4])
    assert torch.equal(plain.in_chunk(4, 1), torch.eye(4, dtype=torch.bool)) and int(plain.in_chunk(5, 9).sum()) == 15
    b = plain.distance_bias(4, torch.tensor(2.0, dtype=F64), torch.tensor(0.5, dtype=F64))
    assert [float(b[3, j]) for j in range(4)] == pytest.approx([2 * math.log(2.5), 2 * math.log(2.0), 2 * math.log(1.5), 0.0])
    w = plain.softmax_with_sink(torch.zeros(1, 2, dtype=F64), torch.tensor(math.log(6.0), dtype=F64))
    assert w[0].tolist() == pytest.approx([1 / 8, 1 / 8])


def test_oracle_router_gates_and_activations():
    chosen, weight = plain.route(torch.tensor([[0.0, math.log(3.0), -9.0, math.log(2.0)]], dtype=F64), 2)
    assert chosen.tolist() == [[1, 3]] and weight[0].tolist() == pytest.approx([0.75, 2 / 3])
    one = lambda v: torch.tensor([[v]], dtype=F64)
    sig = lambda z: 1 / (1 + math.exp(-z))
    assert float(plain.weighted_expert(one(2.0), torch.tensor([0.5], dtype=F64), one(3.0), one(4.0), one(1.0))) == pytest.approx(3.0 * sig(3.0) * 4.0)
    assert float(plain.channel_gate(one(2.0), one(0.5), torch.tensor([1.0], dtype=F64))) == pytest.approx(sig(2.0))
    for z in (-5.0, -0.7, 0.0, 0.3, 4.0):                     # (the form that the kernel takes)
        assert float(plain.gelu(torch.tensor(z, dtype=F64))) == pytest.approx(z * sig(GELU_SLOPE * (z + GELU_CUBIC * z ** 3)), abs=1e-12)
    assert abs(float(plain.gelu(torch.tensor(1.3, dtype=F64))) - 1.3 * 0.5 * (1 + math.erf(1.3 / math.sqrt(2)))) < 1e-3


def test_oracle_order_of_looped_layers():
    assert plain.layer_order(5, dict(start=1, stop=3, times=2)) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None), (4, None)]
    assert plain.layer_order(2, dict(start=0, stop=2, times=1)) == [(0, 0), (1, None)] and plain.layer_order(2, None) == [(0, None), (1, None)]
    x, x0 = torch.tensor([[1.0, 2.0]], dtype=F64), torch.tensor([[3.0, 4.0]], dtype=F64)
    w = torch.tensor([[1.0, 0.0, 10.0, 0.0], [0.0, 1.0, 0.0, 100.0]], dtype=F64)
    assert plain.entry(x, x0, w, torch.tensor([0.5, 0.25], dtype=F64)).tolist() == [[31.5, 402.25]]


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
    cfg = BedenexConfig.from_raw(raw)
    first, second = cfg.layers[0].mixer, cfg.layers[1].mixer
    assert (first.chunk, first.window, first.rot, first.qk_norm, first.v_norm, first.distance_bias, first.bias, first.sink, first.gate) == (37, None, None, UNIT, True, True, False, False, True)
    assert (second.q_rank, second.window, second.gate, second.sink, second.halves, second.kv_from) == (0, None, False, True, True, None)
    assert second.rot == Rotary(3000.0, 16) and cfg.layers[3].mixer.rot.base == 500.0
    moe = cfg.layers[1].mlp
    assert isinstance(moe, ExpertsSpec) and (moe.experts, moe.top, moe.ff, moe.score, moe.weigh_input, moe.bias, moe.shared) == (6, 2, 40, SIGMOID, True, False, None)
    assert cfg.layers[0].mlp == DenseSpec(200) and cfg.layers[2].mlp is None and cfg.loop == LoopSpec(1, 4, 2) and cfg.num_hidden_layers == 5
    assert cfg.runs() == plain.layer_order(5, raw["loop"])
    (tmp_path / "config.json").write_text(json.dumps(raw))
    assert registry.load_config(str(tmp_path)) == cfg and registry.model_class(cfg) is Bedenex
    assert registry.kernels_of(str(tmp_path)) == registry.kernels_for(cfg) == "parallel"
    for path, value in ((("layers", 0, "type"), "other"), (("layers", 0, "mlp", "kind"), "gated"), (("layers", 1, "mlp", "router", "top"), 7), (("layers",), []),
                        (("layers", 1, "mixer", "rot", "dims"), 14), (("layers", 1, "mixer", "rot_dim"), 15), (("layers", 0, "mixer", "mask", "size"), 0),
                        (("layers", 0, "mixer", "kv_heads"), 4), (("loop", "start"), -1), (("loop", "start"), 4), (("loop", "stop"), 6), (("loop", "times"), 0)):
        with pytest.raises(ValueError):
            BedenexConfig.from_raw(_bad(raw, path, value))
    for name, other in cases.configs().items():
        assert BedenexConfig.from_raw(other).runs() == plain.layer_order(len(other["layers"]), other.get("loop")), name
    assert EngineConfig(cfg, dtype="float32", max_num_batched_tokens=600, max_model_len=4096).torch_dtype is torch.float32


def test_weights_land_where_they_belong(tmp_path):
    raw = cases.configs()["mixed"]
    w = cases.random_weights(raw, 3)
    m = Bedenex(BedenexConfig.from_raw(raw), 64, torch.device("cpu"))
    m.load_weights(cases.write_model(tmp_path, raw, w))
    f, width = {k: v.float() for k, v in w.items()}, 104
    assert torch.equal(m.head, f["head"]) and torch.equal(m.loop_in, f["loop.in"]) and torch.equal(m.loop_step, f["loop.step"]) and torch.equal(m.final, f["final.norm"])
    # a chunked layer beside a dense feed-forward: one product for everything that reads the norm
    first = m.layer_weights[0]
    rows = 6 * 32 + 2 * (32 + 48) + 6
    assert first.mix.own_rows == -(-rows // 8) * 8 and torch.equal(first.mix.qkvg[:rows], torch.cat([f[f"l0.mix.{n}"] for n in "qkvg"]))
    assert torch.equal(first.mix.qkvg[first.gates], torch.cat([f["l0.rg1"], f["l0.rg2"]])) and torch.equal(first.gate_bias, torch.cat([f["l0.rg1.b"], f["l0.rg2.b"]]))
    assert torch.equal(first.mix.qkvg[first.gate_up], torch.cat([f["l0.mlp.gate"], f["l0.mlp.up"]])) and torch.equal(first.down, f["l0.mlp.down"])
    assert first.mix.qkvg.shape[0] == first.gate_up.stop and torch.equal(first.mix.slope, f["l0.mix.r1"]) and torch.equal(first.mix.rate, f["l0.mix.r2"])
    assert first.mix.q_norm is None and first.mix.sinks is None and first.mix.slope.dtype == torch.float32
    # a latent layer: rotated partners side by side, queries and keys alike
    second = m.layer_weights[1]
    heads, dim, rot, rank = 5, 24, 16, 72
    q, dkv = f["l1.mix.q"].view(heads, dim + rot, width), f["l1.mix.dkv"]
    got_q, got_dkv = second.mix.down[: heads * (dim + rot)].view(heads, dim + rot, width), second.mix.down[heads * (dim + rot): heads * (dim + rot) + rank + rot]
    assert torch.equal(got_q[:, :dim], q[:, :dim]) and torch.equal(got_dkv[:rank], dkv[:rank])
    for i in range(rot // 2):
        for got, want, at in ((got_q, q, dim), (got_dkv[None], dkv[None], rank)):
            assert torch.equal(got[:, at + 2 * i], want[:, at + i]) and torch.equal(got[:, at + 2 * i + 1], want[:, at + i + rot // 2])
    assert second.mix.q_norm is None and second.mix.uq is None and torch.equal(second.mix.sinks, f["l1.mix.sink"]) and second.down is None
    assert torch.equal(second.mix.uk_t[2], f["l1.mix.uk"].view(heads, dim, rank)[2].t()) and torch.equal(second.mlp.gate_up[4], torch.cat([f["l1.mlp.e4.gate"], f["l1.mlp.e4.up"]]))
    third = m.layer_weights[2]                                # no feed-forward: one gate
    assert third.gates.stop - third.gates.start == width and third.gate_bias.shape == (width,) and third.mlp is third.down is None
    # runs of one layer share weights and nothing else
    assert [r.weights for r in m.layers] == [m.layer_weights[i] for i in (0, 1, 2, 3, 1, 2, 3, 4)] and [r.begins for r in m.layers] == [None, 0, None, None, 1, None, None, None]
    assert m.layers[1].mixer is not m.layers[4].mixer and m.layers[1].experts.counters is not m.layers[4].experts.counters
    del w["l2.rg1.b"]
    with pytest.raises(KeyError, match="l2.rg1.b"):
        m.load_weights(cases.write_model(tmp_path / "b", raw, w))
    w = cases.random_weights(raw, 3)
    w["l2.rg2"] = w["l2.rg1"].clone()
    with pytest.raises(ValueError, match="l2.rg2"):
        m.load_weights(cases.write_model(tmp_path / "c", raw, w))
    straight = Bedenex(BedenexConfig.from_raw(cases.configs()["straight"]), 64, torch.device("cpu"))
    assert straight.loop_in is None and straight.loop_step is None


def test_latent_weights_of_both_layouts():
    """Pairs given as halves or as neighbours, queries direct or through a latent, gate or none: the sizes of the first product."""
    base = dict(heads=3, dim=8, rot_dim=4, vdim=8, kv_rank=16, window=None, scale=1.0, rot=Rotary(10.0, 4))
    direct, through = LatentSpec(q_rank=0, gate=False, halves=True, **base), LatentSpec(q_rank=24, **base)
    assert direct.down_rows == 3 * 12 + 20 and through.down_rows == 24 + 20 + 3 and through.query_rows == 24 and direct.query_rows == 36
    rows = torch.arange(6.0)[:, None]
    assert direct.paired(rows)[:, 0].tolist() == [0, 3, 1, 4, 2, 5] and torch.equal(through.paired(rows), rows)


def test_every_pass_keeps_its_own_cache():
    cfg = BedenexConfig.from_raw(cases.configs()["mixed"])
    m = Bedenex(cfg, 64, torch.device("cpu"))
    looped = (72 + 16) + 4 * (64 + 24) + (96 + 48)
    assert m.kv_bytes_per_token() == 4 * (2 * (32 + 48) + 2 * looped + 1 * (40 + 56)) and m.state_bytes_per_slot() == 0
    m.bind_cache(3, 256, 2)
    assert m.layers[1].mixer.cache.shape == m.layers[4].mixer.cache.shape == (3, 256, 88) and m.layers[1].mixer.cache is not m.layers[4].mixer.cache
    assert m.layers[2].mixer.k_cache.shape == (3, 256, 4, 64) and m.layers[5].mixer.v_cache.shape == (3, 256, 4, 24)
    m.unbind_cache()
    assert m.layers[1].mixer.cache is None and m.layers[5].mixer.v_cache is None
    s = Scheduler(EngineConfig(cfg, max_num_seqs=3, max_num_batched_tokens=512, num_kvcache_blocks=4, max_model_len=2048))
    assert s.portions and s.block_manager.num_state_slots == 3


# ---- the engine tests' models show a planted mistake ---------------------------------------------------

_NAMES = ("unit_rms", "weighted_norm", "turned", "causal", "in_chunk", "distance_bias", "softmax_with_sink", "latent_attention", "head_gates", "head_norm", "value_norm",
          "gelu", "route", "weighted_expert", "silu_mlp", "expert_mixture", "channel_gate", "entry", "layer_order", "biased_attention")
_true = {n: getattr(plain, n) for n in _NAMES}


def _in_pages(fn):
    return lambda t, *a: fn(t, *a) & ((torch.arange(t)[:, None] // 256) == (torch.arange(t)[None] // 256))


def _neighbours(x, base, dims):
    there = x.unflatten(-1, (dims // 2, 2)).transpose(-1, -2).flatten(-2)
    return _true["turned"](there, base, dims).unflatten(-1, (2, dims // 2)).transpose(-1, -2).flatten(-2)


def _reading(**renamed):
    """The mixer with one of its tensors taken for another, or changed."""
    def swap(fn):
        return lambda h, w, m, eps: fn(h, lambda n: renamed[n](w) if n in renamed else w(n), m, eps)
    return swap


def _lag(shift):
    return lambda t, r1, r2: r1 * torch.log1p(r2 * ((torch.arange(t)[:, None] - torch.arange(t)[None]).clamp(min=0).to(r1.dtype) + shift).clamp(min=0))


MISTAKES = {
    "a chunk one position longer": dict(in_chunk=lambda t, size: _true["in_chunk"](t, size + 1)),
    "a chunk one position shorter": dict(in_chunk=lambda t, size: _true["in_chunk"](t, max(1, size - 1))),
    "chunks counted from position 1": dict(in_chunk=lambda t, size: _true["in_chunk"](t + 1, size)[1:, 1:]),
    "no chunks": dict(in_chunk=lambda t, size: _true["causal"](t)),
    "a window instead of chunks": dict(in_chunk=lambda t, size: _true["causal"](t) & ~torch.ones(t, t, dtype=torch.bool).tril(-size)),
    "latents of the page before unseen": dict(causal=_in_pages(_true["causal"])),
    "no distance bias": dict(distance_bias=lambda t, r1, r2: 0.0),
    "a distance bias that is linear": dict(distance_bias=lambda t, r1, r2: r1 * r2 * (torch.arange(t)[:, None] - torch.arange(t)[None]).clamp(min=0).to(r1.dtype)),
    "a distance bias in base 2": dict(distance_bias=lambda t, r1, r2: _true["distance_bias"](t, r1, r2) / math.log(2.0)),
    "a distance one longer": dict(distance_bias=_lag(1)),
    "a distance one shorter": dict(distance_bias=_lag(-1)),
    "slopes for rates": dict(biased_attention=_reading(r1=lambda w: w("r2"), r2=lambda w: w("r1"))(_true["biased_attention"])),
    "every head the first one's bias": dict(biased_attention=_reading(r1=lambda w: w("r1")[:1].expand(99), r2=lambda w: w("r2")[:1].expand(99))(_true["biased_attention"])),
    "queries and keys not normed": dict(head_norm=lambda x, eps: x),
    "values not normed": dict(value_norm=lambda v, eps: v),
    "no gate per head": dict(head_gates=lambda h, w: torch.ones(h.shape[0], w.shape[0], dtype=h.dtype)),
    "no sink": dict(softmax_with_sink=lambda s, sink: torch.softmax(s, -1)),
    "a sink that is halved": dict(softmax_with_sink=lambda s, sink: _true["softmax_with_sink"](s, 0.5 * sink)),
    "rotation of neighbours": dict(turned=_neighbours),
    "no rotation": dict(turned=lambda x, base, dims: x),
    "positions from 1 for keys alone": dict(turned=lambda x, base, dims: _true["turned"](x, base, dims) if x.dim() == 3
                                            else _true["turned"](torch.cat([x[:1], x]), base, dims)[1:]),
    "the latent not normed": dict(latent_attention=lambda h, w, m, eps: _true["latent_attention"](h, lambda n: w(n) * (1.0 if n != "dkv.norm" else 3.0), m, eps)),
    "norms without their weights": dict(weighted_norm=lambda x, w, eps: plain.unit_rms(x, eps)),
    "silu for gelu": dict(gelu=plain.silu),
    "one expert fewer": dict(route=lambda z, top: _true["route"](z, max(1, top - 1))),
    "expert weights that sum to one": dict(route=lambda z, top: (lambda c, s: (c, s / s.sum(-1, keepdim=True)))(*_true["route"](z, top))),
    "expert weights from a softmax": dict(route=lambda z, top: (_true["route"](z, top)[0], torch.topk(torch.softmax(z, -1), top, -1)[0])),
    "weights on what the experts give": dict(weighted_expert=lambda h, weight, *w: weight[:, None] * plain.silu_mlp(h, *w)),
    "no gates on the residual": dict(channel_gate=lambda h, w, b: torch.ones_like(h)),
    "residual gates without their bias": dict(channel_gate=lambda h, w, b: _true["channel_gate"](h, w, 0 * b)),
    "a pass without its vector": dict(entry=lambda x, x0, w, step: _true["entry"](x, x0, w, 0 * step)),
    "a pass without the embeddings": dict(entry=lambda x, x0, w, step: _true["entry"](x, 0 * x0, w, step)),
    "stream and embeddings exchanged": dict(entry=lambda x, x0, w, step: _true["entry"](x0, x, w, step)),
    "a pass that adds to the stream": dict(entry=lambda x, x0, w, step: x + _true["entry"](x, x0, w, step)),
    "the first pass' vector for all": dict(layer_order=lambda n, loop: [(i, None if t is None else 0) for i, t in _true["layer_order"](n, loop)]),
    "one pass fewer": dict(layer_order=lambda n, loop: _true["layer_order"](n, dict(loop, times=loop["times"] - 1))),
    "only the first pass begins anew": dict(layer_order=lambda n, loop: [(i, t if t == 0 else None) for i, t in _true["layer_order"](n, loop)]),
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


def test_planted_exchange_of_tensors_shows_in_the_logits():
    cfg = cases.configs()["mixed"]
    weights = cases.random_weights(cfg, 1)
    ids = cases.tokens(120, cfg["vocab"], 5)
    want = plain.forward(cfg, weights, ids)
    for a, b in (("l0.rg1", "l0.rg2"), ("l1.rg1.b", "l1.rg2.b"), ("l0.mlp.gate", "l0.mlp.up"), ("l1.mlp.e0.gate", "l1.mlp.e0.up"), ("embed", "head"), ("l0.norm1", "final.norm")):
        other = dict(weights, **{a: weights[b], b: weights[a]})
        assert float(cases.row_error(plain.forward(cfg, other, ids), want).max()) > 0.1, (a, b)
