"""Kaparax on the host: configuration, weight files, state slots, mixed scheduling, row-group inputs,
and the oracle against itself."""
import json
import math
import random

import numpy as np
import pytest
import torch

from oracle import kaparax as plain
from nanovllm_amd.engine import BlockManager, EngineConfig, SamplingParams, Scheduler, Sequence
from nanovllm_amd.engine import registry
from nanovllm_amd.engine.kaparax import Kaparax, KaparaxConfig
from nanovllm_amd.engine.config import ModelConfig
from nanovllm_amd.engine.loader import TensorFolder
from nanovllm_amd.engine.mixers import AttentionSpec, RetentionSpec, RopeTables, Rotary
from nanovllm_amd.engine.model_runner import Span, build_span_inputs
import kaparax_cases as cases


# ---- the oracle against itself and against hand-made values -----------------------------------------

def test_oracle_rotation_is_relative_and_leaves_the_rest():
    g = torch.Generator().manual_seed(0)
    q = torch.randn(1, 1, 10, generator=g, dtype=torch.float64).expand(9, 1, 10)
    r = plain.rotate(q, 50.0, 6)
    assert torch.equal(r[..., 6:], q[..., 6:]) and torch.equal(r[0], q[0])
    gram = r[:, 0, :6] @ r[:, 0, :6].T                        # depends on the distance only
    for d in range(9):
        assert torch.allclose(torch.diagonal(gram, d), gram[0, d].expand(9 - d))
    u, v, a = q[0, 0, 1], q[0, 0, 4], 3.0 * 50.0 ** (-2 / 6)
    assert math.isclose(float(r[3, 0, 1]), float(u * math.cos(a) - v * math.sin(a)), rel_tol=1e-12)
    assert math.isclose(float(r[3, 0, 4]), float(v * math.cos(a) + u * math.sin(a)), rel_tol=1e-12)


def test_oracle_convolution_taps():
    u = torch.arange(1.0, 6.0, dtype=torch.float64)[:, None]
    w = torch.tensor([[100.0, 10.0, 1.0]], dtype=torch.float64)
    assert plain.short_conv(u, w)[:, 0].tolist() == [1.0, 12.0, 123.0, 234.0, 345.0]
    assert plain.short_conv(u[:1], w)[:, 0].tolist() == [1.0]


def test_oracle_retention_is_the_decayed_sum():
    g = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(12, 2, 5, generator=g, dtype=torch.float64) for _ in range(3))
    decay = [0.9, 0.5]
    got = plain.retention(q, k, v, decay)
    for h in range(2):
        i, j = torch.arange(12)[:, None], torch.arange(12)[None]
        weight = torch.where(j <= i, decay[h] ** (i - j).clamp_min(0).double(), torch.zeros(()).double())
        assert torch.allclose(got[:, h], (q[:, h] @ k[:, h].T * weight) @ v[:, h])


def test_oracle_chunks_and_cap():
    vis = plain.chunk_visible(7, 3)
    assert [int(r.sum()) for r in vis] == [1, 2, 3, 1, 2, 3, 1] and bool(vis[5, 3]) and not bool(vis[3, 2])
    assert float(plain.capped(torch.tensor(1e9), 7.0)) == pytest.approx(7.0) and float(plain.capped(torch.tensor(3.0), None)) == 3.0


def test_oracle_gate_limits():
    eye = torch.eye(1, dtype=torch.float64)
    for h, want in ((10.0, 2.0 / (1 + math.exp(-3.404)) * 3.0), (-10.0, -10.0 / (1 + math.exp(17.02)) * -1.0)):
        assert float(plain.gated_mlp(torch.full((1, 1), h, dtype=torch.float64), eye, eye, eye, 2.0)) == pytest.approx(want)


# ---- configuration, registry, weight files ---------------------------------------------------------

def test_config_is_read_and_checked(tmp_path):
    raw = cases.configs()["mixed"]
    cfg = KaparaxConfig.from_raw(raw)
    assert [l.weights_of for l in cfg.layers] == [0, 1, 2, 3, 1, 0, 2] and cfg.layers[1].mlp is None
    assert isinstance(cfg.layers[0].mixer, RetentionSpec) and isinstance(cfg.layers[1].mixer, AttentionSpec)
    assert cfg.layers[1].mixer.rot == Rotary(5000.0, 32) and cfg.layers[1].mixer.chunk == 37 and cfg.layers[0].mlp.ff == 72
    (tmp_path / "config.json").write_text(json.dumps(raw))
    assert registry.load_config(str(tmp_path)) == cfg and registry.model_class(cfg) is Kaparax
    (tmp_path / "config.json").write_text(json.dumps({"hidden_size": 64, "num_attention_heads": 4}))
    assert isinstance(registry.load_config(str(tmp_path)), ModelConfig)
    chain = json.loads(json.dumps(raw))
    chain["layers"][1]["weights_of"], chain["layers"][1]["mlp"] = 4, None     # towards a later layer, which has tensors then
    del chain["layers"][4]["weights_of"]
    assert [l.weights_of for l in KaparaxConfig.from_raw(chain).layers][1] == 4
    bad = json.loads(json.dumps(raw))
    bad["layers"][4]["mixer"]["dim"] = 64
    with pytest.raises(ValueError, match="shares"):
        KaparaxConfig.from_raw(bad)
    for path, value in ((("layers", 0, "type"), "other"), (("layers", 0, "mlp", "kind"), "routed"), (("layers", 4, "weights_of"), 4), (("layers", 4, "weights_of"), 70)):
        bad = json.loads(json.dumps(raw))
        at = bad
        for p in path[:-1]:
            at = at[p]
        at[path[-1]] = value
        with pytest.raises(ValueError):
            KaparaxConfig.from_raw(bad)
    with pytest.raises(ValueError, match="unknown architecture"):
        registry.family_of_raw({"architecture": "Unheard"})
    with pytest.raises(ValueError, match="float32"):
        EngineConfig(ModelConfig(), dtype="float32")
    assert EngineConfig(cfg, dtype="float32", max_num_batched_tokens=600, max_model_len=4096).torch_dtype is torch.float32


def test_weights_land_where_they_belong(tmp_path):
    raw = cases.configs()["mixed"]
    w = cases.random_weights(raw, 3)
    folder = cases.write_model(tmp_path, raw, w)
    cfg = KaparaxConfig.from_raw(raw)
    m = Kaparax(cfg, 64, torch.device("cpu"))
    m.load_weights(folder)
    a = m.layer_weights["1"].mix
    assert torch.equal(a.qkv, torch.cat([w["l1.mix.q"], w["l1.mix.k"], w["l1.mix.v"]]).float())
    assert torch.equal(a.conv[2], torch.cat([w[f"l1.mix.{n}.conv"] for n in "qkv"])[:, 2].float())
    r = m.layer_weights["0"]
    assert torch.equal(r.mix.qkvg, torch.cat([w[f"l0.mix.{n}"] for n in "qkvg"]).float())
    assert torch.equal(r.mlp.gate_up, torch.cat([w["l0.mlp.gate"], w["l0.mlp.up"]]).float()) and torch.equal(r.norm2b.b, w["l0.norm2b.b"].float())
    assert m.layers[4].weights is m.layers[1].weights and m.layers[4].mixer is not m.layers[1].mixer
    assert not hasattr(m.layer_weights["1"], "mlp") and "4" not in m.layer_weights
    del w["l2.norm1b.b"]
    with pytest.raises(KeyError, match="l2.norm1b.b"):
        m.load_weights(cases.write_model(tmp_path / "b", raw, w))
    w = cases.random_weights(raw, 3)
    w["l9.norm1"] = w["l2.norm1"].clone()
    with pytest.raises(ValueError, match="l9.norm1"):
        m.load_weights(cases.write_model(tmp_path / "c", raw, w))
    with pytest.raises(ValueError, match="shape"):
        TensorFolder(folder).take("head", (1, 2))


def test_rope_tables_are_shared_and_precise():
    t = RopeTables(5000, torch.device("cpu"))
    a = t.get(Rotary(1e4, 8))
    assert t.get(Rotary(1e4, 8)) is a and t.get(Rotary(1e4, 0)) is None and a.shape == (5000, 8)
    angle = 4999 * 1e4 ** (-2 * 1 / 8)
    assert float(a[4999, 1]) == pytest.approx(math.cos(angle), abs=1e-7) and float(a[4999, 5]) == pytest.approx(math.sin(angle), abs=1e-7)


# ---- blocks, slots, scheduling ---------------------------------------------------------------------

def _scheduler(blocks=16, seqs=3, budget=512):
    cfg = EngineConfig(KaparaxConfig.from_raw(cases.configs()["mixed"]), max_num_seqs=seqs, max_num_batched_tokens=budget,
                       num_kvcache_blocks=blocks, max_model_len=2048)
    return Scheduler(cfg)


def test_state_slots_travel_with_the_blocks():
    bm = BlockManager(6, 256, prefix_cache=False, num_state_slots=2)
    a, b, c = (Sequence(list(range(300))) for _ in range(3))
    bm.allocate(a), bm.allocate(b)
    assert (a.state_slot, b.state_slot) == (0, 1) and not set(a.block_table) & set(b.block_table) and b.num_cached_tokens == 0
    assert not bm.can_allocate(c)                            # blocks are left, slots are not
    bm.deallocate(a)
    assert a.state_slot == -1 and bm.can_allocate(c)
    bm.allocate(c)
    assert c.state_slot == 0
    c.token_ids += [1] * 300
    bm.extend(c)
    assert len(c.block_table) == 3
    c.token_ids += [1] * 600
    with pytest.raises(RuntimeError):
        bm.extend(c)


def test_mixed_steps_decode_first_then_portions():
    s = _scheduler(seqs=3, budget=256)
    a, b, c, d = (Sequence([1] * n, SamplingParams(max_tokens=8)) for n in (100, 400, 30, 10))
    for q in (a, b, c, d):
        s.add(q)
    seqs, mixed = s.schedule()
    assert mixed and seqs == [a, b] and [q.num_scheduled_tokens for q in seqs] == [100, 156] and s.needs_tokens()
    s.postprocess(seqs, [7, -1])
    assert len(a) == 101 and len(b) == 400 and b.num_cached_tokens == 156 and a.is_prefilled and not b.is_prefilled
    seqs, mixed = s.schedule()                                # a decodes beside the rest of b; c fits the budget, d has no slot
    assert mixed and seqs == [a, b, c] and [q.num_scheduled_tokens for q in seqs] == [1, 244, 11]
    s.postprocess(seqs, [7, 8, -1])
    seqs, mixed = s.schedule()
    assert mixed and seqs == [a, b, c] and c.num_scheduled_tokens == 19
    s.postprocess(seqs, [7, 8, 9])
    seqs, mixed = s.schedule()
    assert not mixed and seqs == [a, b, c] and s.waiting[0] is d
    for _ in range(8):
        s.postprocess(seqs, [7] * len(seqs))
        seqs, _ = s.schedule()
        if d in seqs:
            break
    assert d in seqs and a.is_finished and d.state_slot == 0 and d.block_table


def test_preempted_sequences_start_over():
    s = _scheduler(blocks=3, seqs=3, budget=1024)
    a, b = Sequence([1] * 256, SamplingParams(max_tokens=40)), Sequence([2] * 256, SamplingParams(max_tokens=40))
    s.add(a), s.add(b)
    seqs, _ = s.schedule()
    s.postprocess(seqs, [5, 6])                               # both now need a second block, one is left
    seqs, mixed = s.schedule()
    assert seqs == [a] and not mixed and b.state_slot == -1 and b.num_cached_tokens == 0 and s.waiting[0] is b
    for _ in range(39):
        s.postprocess(seqs, [5])
        if a.is_finished:
            break
        seqs, mixed = s.schedule()
        assert seqs == [a]
    seqs, mixed = s.schedule()
    assert mixed and seqs == [b] and b.prefill_target == 257 and b.num_scheduled_tokens == 257


def test_step_inputs_of_single_tokens_and_portions():
    def seq(n, table, slot):
        q = Sequence(list(range(100, 100 + n)))
        q.block_table, q.state_slot = table, slot
        return q
    a, b, c = seq(700, [4, 1, 3], 2), seq(258, [0, 5], 0), seq(5, [2], 1)
    h = build_span_inputs([Span(a, 250, 20, [19, 0]), Span(b, 257, 1, [0]), Span(c, 0, 5, [])], 256)
    assert h["input_ids"].tolist() == [357] + list(range(350, 370)) + list(range(100, 105))
    assert h["positions"].tolist() == [257] + list(range(250, 270)) + list(range(5))
    assert h["slot_mapping"].tolist() == [5 * 256 + 1] + [4 * 256 + p for p in range(250, 256)] + [256 + p for p in range(14)] + [512 + p for p in range(5)]
    assert h["logit_rows"].tolist() == [20, 1, 0]
    one, many = h["singles"], h["portions"]
    assert one["seq_lens"].tolist() == [258] and one["state_slots"].tolist() == [0] and one["block_tables"].tolist() == [[0, 5]]
    assert many["seq_lens"].tolist() == [270, 5] and many["cu"].tolist() == [0, 20, 25] and many["state_slots"].tolist() == [2, 1]
    assert many["token_seq"].tolist() == [0] * 20 + [1] * 5 and many["block_tables"].tolist() == [[4, 1, 3], [2, -1, -1]] and many["max_q"] == 20
    assert build_span_inputs([Span(b, 257, 1, [])], 256)["portions"] is None


def test_trace_command_refuses_what_no_model_does(tmp_path):
    from nanovllm_amd.engine import trace
    (tmp_path / "config.json").write_text(json.dumps({"hidden_size": 64, "num_attention_heads": 4}))
    assert trace.main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"]) == 3


# ---- the engine tests' models show a planted mistake ---------------------------------------------------

def _reset_state_at(at):
    true = plain.retention
    return lambda q, k, v, decay: torch.cat([true(q[:at], k[:at], v[:at], decay), true(q[at:], k[at:], v[at:], decay)])


def _forget_rows_before(at):
    true = plain.short_conv
    return lambda u, w: torch.cat([true(u[:at], w), true(u[at:], w)])


_true = {n: getattr(plain, n) for n in ("chunk_visible", "rotate", "short_conv", "capped", "gated_mlp", "layer_norm", "unit_rms")}
MISTAKES = {
    "a chunk one key longer": dict(chunk_visible=lambda t, size: _true["chunk_visible"](t, size + 1)),
    "keys of the page before unseen": dict(chunk_visible=lambda t, size: _true["chunk_visible"](t, size) & _true["chunk_visible"](t, 256)),
    "a state lost at token 256": dict(retention=_reset_state_at(256)),
    "carried rows lost at token 256": dict(short_conv=_forget_rows_before(256)),
    "rotation of neighbours": dict(rotate=lambda x, base, dims: _true["rotate"](x.flip(-1), base, dims).flip(-1) if dims else x),
    "taps in the wrong order": dict(short_conv=lambda u, w: _true["short_conv"](u, w.flip(1))),
    "no score cap": dict(capped=lambda s, cap: s),
    "no limit in the feed-forward": dict(gated_mlp=lambda h, g, u, d, limit: _true["gated_mlp"](h, g, u, d, 1e9)),
    "a norm without its shift": dict(layer_norm=lambda x, w, b, eps: _true["layer_norm"](x, w, 0 * b, eps)),
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
    assert float(err.max()) > 0.12, (mistake, float(err.max()), float(err.mean()))     # beyond the bf16 limit, far beyond the fp32 one
