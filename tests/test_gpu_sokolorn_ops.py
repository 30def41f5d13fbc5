"""Every mechanism of the Sokolorn layers alone, on the GPU, against the plain implementation: ragged batches of
portions and of single tokens, pages in random order, unwritten pages full of NaN."""
import math

import pytest
import torch

from oracle import sokolorn as plain
from nanovllm_amd.engine import branches, experts, masked, mixers
from nanovllm_amd.engine.mixers import RopeTables, Rotary, RotaryScaling

from row_batches import BF16, BLOCK, F32, Batch, batches, close, rand, tol

pytestmark = pytest.mark.gpu
F64 = torch.float64


# ---- the residual step ---------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("width", [8, 50, 104, 512, 1544, 4096, 5000])
@pytest.mark.parametrize("n", [37, 1100])
def test_norm_of_what_a_sublayer_gives(dev, dtype, width, n):
    if n > 1024 and width > 1544:
        n = 1030
    g = torch.Generator().manual_seed(width)
    vocab, eps = 90, 1e-5
    table, y1 = rand(g, vocab, width, dtype=dtype), rand(g, n, width, dtype=dtype)
    post, nxt = (0.3 * rand(g, width, dtype=dtype) for _ in range(2))
    ids = torch.randint(0, vocab, (n,), generator=g)
    res, out, none = branches.embed_rms_norms(ids.to(dev), table.to(dev), 1.0, (None, None), eps)
    t = tol(dtype, 6e-3, 3e-6)
    assert none is None and res.dtype == F32 and torch.equal(out.cpu(), table[ids]) and torch.equal(res.cpu(), table[ids].float())
    counters = torch.full((700,), 9, dtype=torch.int32, device=dev)
    for terms, shared in ((0, True), (0, False), (1, False), (3, True), (8, True), (6, False)):
        y2 = rand(g, n * terms, width, dtype=dtype) if terms else None
        weight = torch.rand(n, terms + 1, generator=g)
        y = torch.zeros(n, width, dtype=F64)
        if terms:
            y = (weight[:, :terms].double()[..., None] * y2.double().view(n, terms, width)).sum(1)
        if shared or not terms:
            y = y + y1.double() * (weight[:, terms:].double() if shared else 1.0)
        want = res.double().cpu() + plain.centred_weight_norm(y, post.double(), eps)
        w = weight.to(dev)
        args = (y1.to(dev) if shared or not terms else None, w[:, terms] if shared else None, y2.to(dev) if terms else None,
                w[:, :terms] if terms else None, post.to(dev))
        rows, before = torch.tensor([5, 36, 0, 5], dtype=torch.int32), res.clone()
        picked = branches.post_rms_norms(res, *args, nxt.to(dev), eps, 1.0, rows=rows.to(dev))
        assert torch.equal(res, before)
        other = res.clone()
        normed = branches.post_rms_norms(other, *args, nxt.to(dev), eps, 1.0)
        counters.fill_(9)
        out = branches.post_rms_norms(res, *args, None, eps, 1.0, clear=counters[:600])
        assert torch.equal(other, res) and torch.equal(out, res.to(dtype))
        close(picked, normed[rows.long().to(dev)], tol(dtype, 8e-3, 2e-6), "picked rows")       # (few rows: sums in another order)
        assert not counters[:600].any() and bool((counters[600:] == 9).all())
        close(res, want, 3e-6, f"residual, {terms} terms")
        close(normed, plain.centred_weight_norm(want, nxt.double(), eps), t, f"next norm, {terms} terms")


# ---- activations, experts -----------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("width", [8, 27, 1536])
def test_squared_relu_and_soft_cap(dev, dtype, width):
    g = torch.Generator().manual_seed(width)
    x = 3.0 * rand(g, 19, width, dtype=dtype)
    close(mixers.squared_relu_(x.to(dev)), torch.relu(x.double()) ** 2, tol(dtype, 5e-3, 1e-6))
    for cap in (0.7, 30.0):
        close(mixers.soft_cap_(x.to(dev), cap), plain.soft_cap(x.double(), cap), tol(dtype, 5e-3, 2e-6))


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", [(16, 40, 64), (9, 20, 50), (600, 264, 1032), (5, 8, 2048)])
def test_dense_feed_forward_with_its_activation(dev, dtype, shape):
    ff, width, k = shape
    g = torch.Generator().manual_seed(ff)
    w = rand(g, ff, k, dtype=F32).mul(k ** -0.5).to(dtype)
    for n in (1, 7, 16, 33, 64, 150):
        x = rand(g, n, k, dtype=dtype)
        close(experts.project(x.to(dev), w.to(dev), squared_relu=True), torch.relu(x.double() @ w.double().T) ** 2, tol(dtype, 1e-2, 5e-6), f"{n} rows")


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", [(8, 3, 64), (5, 5, 50), (1, 1, 16), (64, 8, 256), (63, 8, 128), (130, 6, 96), (16, 1, 1032)])
def test_router_with_bias_and_gate(dev, dtype, shape):
    n_experts, top, width = shape
    g = torch.Generator().manual_seed(n_experts)
    for n in (1, 16, 45, 5000):
        h, w = rand(g, n, width, dtype=dtype), (rand(g, n_experts + 1, width, dtype=F32) * width ** -0.5).to(dtype)
        bias = torch.cat([2.0 * torch.randn(n_experts, generator=g), torch.zeros(1)])
        z = h.double() @ w.double().T
        want_gate, z = torch.sigmoid(z[:, n_experts]), z[:, :n_experts] + bias[:n_experts].double()
        chosen, weight = plain.route(z, top)
        a = experts.route(h.to(dev), w.to(dev), top, 1.0, torch.zeros(n_experts, dtype=torch.int32, device=dev), bias.to(dev), 1)
        got = a.choice.cpu().long()
        near = (z.gather(1, got) - z.gather(1, chosen)).abs()         # (two logits a rounding apart may trade places)
        assert float(near.max()) < 1e-5 and float((got == chosen).double().mean()) > 0.99
        assert a.weight.shape == (n, top + 1) and int(a.counts.sum()) == n * top
        close(a.weight[:, :top], weight, 2e-5, "weights")
        close(a.weight[:, top], want_gate, 2e-5, "gate")
        for e, c in enumerate(a.counts.cpu().tolist()):
            assert torch.equal(a.lists.cpu()[e, :c].sort().values.long(), (got.flatten() == e).nonzero()[:, 0])


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", [  # experts, best, width, ff, the shared one's ff
    (6, 2, 64, 40, 56), (3, 3, 50, 27, 13), (16, 4, 256, 128, 128), (1, 1, 16, 24, 8), (40, 6, 192, 48, 320), (4, 2, 520, 200, 8), (8, 2, 1024, 768, 1536), (5, 2, 256, 88, None)])
@pytest.mark.parametrize("n", [1, 7, 17, 64, 65, 700, 1500])
def test_experts_with_a_shared_one(dev, dtype, shape, n):
    n_experts, top, width, ff, sff = shape
    g = torch.Generator().manual_seed(n)
    limit, slimit = 0.8, 1.7
    h = rand(g, n, width, dtype=dtype)
    lin = lambda rows, cols, gain=1.5: rand(g, rows, cols, dtype=F32).mul(gain * cols ** -0.5).to(dtype)
    w = {"router": lin(n_experts, width, 2.0), "router.b": torch.randn(n_experts, generator=g).to(dtype)}
    for name, size in [(f"e{e}", ff) for e in range(n_experts)] + ([("shared", sff)] if sff else []):
        w[name + ".gate"], w[name + ".up"], w[name + ".down"] = lin(size, width), lin(size, width), lin(width, size, 1.0)
    if sff:
        w["shared.sg"] = lin(1, width)
    form = lambda x: experts.GateForm(x, 1.702, 1.0)
    spec = experts.ExpertsSpec(n_experts, top, ff, gate=form(limit), bias=True, shared=experts.SharedExpertSpec(sff, form(slimit)) if sff else None)
    with torch.device(dev):
        weights = experts.ExpertWeights(spec, width).requires_grad_(False)
    for p in weights.parameters():
        if p is not weights.bias:
            p.data = p.data.to(dtype)
    weights.load(spec, width, lambda name, size: w[name], "")
    run = experts.Experts(spec, weights, dev)
    y, shared, weight = run(h.to(dev))
    got = (y.double().view(n, top, width) * weight[:, :top].double()[..., None]).sum(1)
    m = dict(router=dict(experts=n_experts, top=top), expert=dict(limit=limit))
    if sff:
        m["shared"] = dict(limit=slimit)
        got = got + shared.double() * weight[:, top:].double()
        close(shared, plain.clamped_mlp(h.double(), *(w[f"shared.{x}"].double() for x in ("gate", "up", "down")), slimit), tol(dtype, 1.5e-2, 1e-5), "shared alone")
    want = plain.expert_mixture(h.double(), lambda name: w[name].double(), m)
    err = ((got.cpu() - want).abs().amax(1) / want.abs().max())
    z = (h.double() @ w["router"].double().T + w["router.b"].double()).sort(-1, descending=True).values
    clear = z[:, top - 1] - z[:, top] > 1e-4 if top < n_experts else torch.ones(n, dtype=torch.bool)
    assert torch.isfinite(got).all() and float(err[clear].max()) < tol(dtype, 1.5e-2, 1e-5), float(err[clear].max())


# ---- what attention reads: bias, norms, rotation, cache ---------------------------------------------------------

SHAPES = [  # heads, key heads, key size, value size, rotated
    (6, 2, 32, 48, 16), (8, 8, 64, 64, 64), (3, 1, 20, 9, 6), (1, 1, 8, 8, 8), (40, 2, 72, 96, 0), (33, 1, 24, 16, 16), (32, 8, 128, 128, 64), (12, 4, 160, 32, 48),
    (5, 5, 17, 20, 16), (16, 2, 256, 200, 128), (64, 64, 128, 64, 96), (70, 7, 200, 8, 8), (4, 2, 96, 96, 20)]


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("kind", ["whole", "head with bias", "nothing"])
def test_bias_norms_rotation_and_cache_write(dev, dtype, shape, kind):
    heads, kv, dim, vdim, rot = shape
    rot = 0 if kind == "whole" else rot
    rotary = Rotary(300.0, rot, RotaryScaling(4.0, 1.0, 6.0, 90.0))
    rope = RopeTables(1024, dev).get(rotary)
    freq = plain.rotation_frequencies(rot, 300.0, dict(factor=4.0, low=1.0, high=6.0, original=90.0))
    queries, keys = heads * dim, kv * dim
    columns = queries + keys + kv * vdim
    for batch in batches(dev):
        g = torch.Generator().manual_seed(7)
        full = [rand(g, n, columns, dtype=dtype) for n, _ in batch.spans]
        whole, bias = kind == "whole", rand(g, columns, dtype=dtype) if kind == "head with bias" else None
        wq = 1 + 0.3 * rand(g, queries if whole else dim, dtype=dtype) if kind != "nothing" else None
        wk = 1 + 0.3 * rand(g, keys if whole else dim, dtype=dtype) if kind != "nothing" else None
        on = lambda t: None if t is None else t.to(dev)
        wide = lambda x: torch.cat([x, torch.full((x.shape[0], 8 + -x.shape[1] % 8), 5.0, dtype=dtype)], 1).to(dev)
        x = wide(batch.rows(full))
        kc = torch.full((batch.num_blocks, BLOCK, kv, dim), 7.0, dtype=dtype, device=dev)
        vc = torch.full((batch.num_blocks, BLOCK, kv, vdim), 7.0, dtype=dtype, device=dev)
        q = torch.full((x.shape[0], queries), 9.0, dtype=dtype, device=dev)
        masked.qkv_prepare(x, on(bias), on(wq), on(wk), masked.WHOLE if whole else masked.HEAD, rope, q, kc, vc, batch.group, heads, kv, dim, vdim, 1e-5)

        def normed(t, w):
            if w is None:
                return t.unflatten(-1, (-1, dim))
            if whole:
                return plain.whole_norm(t, w.double(), 1e-5).unflatten(-1, (-1, dim))
            return plain.head_norm(t.unflatten(-1, (-1, dim)), w.double(), 1e-5)
        wanted = []
        for f in full:
            f = f.double() + (0 if bias is None else bias.double())
            wanted.append(torch.cat([plain.rotate_halves(normed(f[:, :queries], wq), freq).flatten(1),
                                     plain.rotate_halves(normed(f[:, queries: queries + keys], wk), freq).flatten(1), f[:, queries + keys:]], 1))
        n, t = x.shape[0] - batch.pad, tol(dtype, 6e-3, 5e-6)
        want = batch.rows(wanted)[:n]
        close(q[:n], want[:, :queries], t, "queries")
        assert not q[n:].any()
        close(batch.gather(kc).flatten(1), want[:, queries: queries + keys], t, "keys")
        close(batch.gather(vc).flatten(1), want[:, queries + keys:], t, "values")
        untouched = torch.ones(batch.num_blocks * BLOCK, dtype=torch.bool)
        slots = batch.group.slot_mapping.long().cpu()
        untouched[slots[slots >= 0]] = False
        assert bool((kc.view(-1, keys).cpu()[untouched] == 7).all()) and bool((vc.view(-1, kv * vdim).cpu()[untouched] == 7).all())
        again = torch.full_like(q, 9.0)                       # a layer that reads another one's keys: queries only
        masked.qkv_prepare(wide(batch.rows(full)[:, :queries]), on(None if bias is None else bias[:queries]), on(wq), None, masked.WHOLE if whole else masked.HEAD, rope, again, None, None,
                           batch.group, heads, kv, dim, vdim, 1e-5)
        close(again, q, tol(dtype, 8e-3, 1e-6), "queries alone")


# ---- attention --------------------------------------------------------------------------------------------------

ATTN = [  # heads, key heads, key size, value size
    (6, 2, 32, 48), (8, 8, 64, 64), (3, 1, 20, 9), (1, 1, 8, 8), (40, 2, 72, 96), (33, 1, 24, 16), (8, 2, 128, 128), (4, 4, 160, 32), (10, 5, 96, 96), (2, 1, 256, 200),
    (2, 2, 64, 128), (2, 1, 128, 64), (4, 1, 128, 256), (5, 5, 17, 20)]


def _attention_case(dev, dtype, batch, shape, window, scale, extras=True, edit=None, cap=0.0):
    heads, kv, dim, vdim = shape
    g = torch.Generator().manual_seed(3)
    q = [rand(g, n, heads, dim, dtype=dtype) for n, _ in batch.spans]
    k = [rand(g, n, kv, dim, dtype=dtype) for n, _ in batch.spans]
    v = [rand(g, n, kv, vdim, dtype=dtype) for n, _ in batch.spans]
    gate = [rand(g, n, heads, dtype=dtype) for n, _ in batch.spans] if extras else None
    sinks = 3.0 * torch.randn(heads, generator=g) if extras else None
    if edit is not None:
        edit(q, k, v, gate, sinks)
    kc, vc = (torch.full((batch.num_blocks, BLOCK, kv, d), float("nan"), dtype=dtype) for d in (dim, vdim))
    batch.fill(kc, k, upto_start=False), batch.fill(vc, v, upto_start=False)
    qs = batch.rows(q).to(dev)
    gates = None
    if extras:                                                # (a strided view, as the fused projection leaves it)
        gates = torch.cat([torch.zeros(len(qs), 3, dtype=dtype), batch.rows(gate)], 1).to(dev)[:, 3:]
    out = torch.full((qs.shape[0], heads * vdim), 9.0, dtype=dtype, device=dev)
    masked.masked_attention(qs.flatten(1), kc.to(dev), vc.to(dev), batch.group, out, heads, window or masked.ALL_KEYS, scale,
                            None if sinks is None else sinks.to(dev), gates, cap)
    want = []
    for i, (a, b, c) in enumerate(zip(q, k, v)):
        o = plain.softmax_attention(a.double(), b.double(), c.double(), scale, plain.visible(len(a), window), None if sinks is None else sinks.double())
        want.append(o * torch.sigmoid(gate[i].double())[..., None] if extras else o)
    return out.view(-1, heads, vdim), batch.rows(want)


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", ATTN)
@pytest.mark.parametrize("window", [1, 37, 64, 256, 300, None])
def test_attention_under_windows(dev, dtype, shape, window):
    for batch in batches(dev) + [Batch(dev, [(600, 2), (256, 3), (40, 7), (513, 400)], seed=4)]:
        for extras in (True, False):
            # (pages that no row has been written to hold NaN: what is not seen must not reach the result)
            got, want = _attention_case(dev, dtype, batch, shape, window, 1.2 * shape[2] ** -0.5, extras)
            close(got, want, tol(dtype, 1e-2, 1e-5), f"window {window} single {batch.single} extras {extras}")


@pytest.mark.parametrize("dtype", [BF16, F32])
def test_long_contexts_in_many_ranges(dev, dtype):
    """Contexts over several key ranges of a decode step, windows that begin inside one."""
    for shape in ((8, 2, 128, 128), (4, 4, 64, 64)):
        for window in (700, 1500, None):
            got, want = _attention_case(dev, dtype, Batch(dev, [(2100, 1), (1537, 1), (512, 1), (3, 1)], single=True, seed=2), shape, window, 0.1)
            close(got, want, tol(dtype, 1e-2, 1e-5), f"{shape} window {window}")


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", [(4, 2, 64, 64), (2, 1, 128, 128), (2, 2, 96, 64), (3, 1, 20, 12)])
@pytest.mark.parametrize("window", [48, 256, 300, None])
def test_one_loud_key_at_the_edges(dev, dtype, shape, window):
    """Key j answers every query far above the rest: the queries that see it, and only those, return its value."""
    n = 2 * (window or 200) + 70
    for loud in sorted({0, 1, (window or 9) - 1, window or 9, 255, 256, n - 2}):
        def edit(q, k, v, gate, sinks):
            sinks.fill_(-30.0)
            for a, b, c, z in zip(q, k, v, gate):
                a[..., 0], b[..., 0], c[..., 3] = 8.0, 0.0, 1.0
                a[..., 1:], b[..., 1:] = 0.0, 0.0
                z.fill_(20.0)
                if loud < len(b):
                    b[loud, :, 0], c[loud, :, 3] = 16.0, 3.0
        ends = [e for e in (loud + 1, min(loud + (window or n), n), min(loud + (window or n) + 1, n), n) if e > 0]
        for batch in (Batch(dev, [(n, n), (n, 70), (n, 2)], seed=loud), Batch(dev, [(e, 1) for e in ends], single=True, seed=loud)):
            got, want = _attention_case(dev, dtype, batch, shape, window, 0.25, edit=edit)
            close(got, want, tol(dtype, 1e-2, 1e-5), f"loud key {loud}")
            pos = batch.positions.cpu()[: len(got)]
            sees = (pos >= loud) & (pos - loud < (window or n))
            assert bool(((got.cpu()[..., 3] - 3.0).abs().amax(1) < 0.1).eq(sees).all()), loud


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("scores", ["rising", "falling", "far below the sink", "far above the sink", "jumps"])
def test_running_maximum(dev, dtype, scores):
    """Scores that grow or fall by hundreds along the keys, far above and below the sinks."""
    shape, n = (4, 2, 64, 64), 700

    def edit(q, k, v, gate, sinks):
        sinks.copy_(torch.tensor([-2.0, 0.0, 3.0, 8.0]))
        for a, b in zip(q, k):
            a.zero_(), b.zero_()
            a[..., 0] = 4.0
            x = torch.arange(len(b)).float()
            level = {"rising": x, "falling": -x, "far below the sink": -40.0 - x % 3, "far above the sink": 60.0 + x % 3, "jumps": (x // 64 * 37 % 11) * 12.0}[scores]
            b[..., 0] = (level / 4.0)[:, None].to(dtype)
    for batch in (Batch(dev, [(n, n), (n, 90), (n, 2)], seed=1), Batch(dev, [(n, 1), (300, 1), (64, 1), (1, 1)], single=True, seed=2)):
        for window in (100, None):
            got, want = _attention_case(dev, dtype, batch, shape, window, 1.0, edit=edit)
            assert torch.isfinite(got).all() and float((got.double().cpu() - want).abs().max()) < tol(dtype, 2e-2, 2e-5), (window, batch.single)


def test_chunks_with_sinks_gates_and_caps(dev):
    """The other mask, and scores that are capped, through the same entry point."""
    from nanovllm_amd import _lib
    heads, kv, dim = 4, 2, 64
    for dtype in (BF16, F32):
        for batch in batches(dev):
            g = torch.Generator().manual_seed(5)
            q, k, v = ([rand(g, n, x, dim, dtype=dtype) for n, _ in batch.spans] for x in (heads, kv, kv))
            sinks, gate = torch.randn(heads, generator=g), [rand(g, n, heads, dtype=dtype) for n, _ in batch.spans]
            kc, vc = (torch.full((batch.num_blocks, BLOCK, kv, dim), float("nan"), dtype=dtype) for _ in range(2))
            batch.fill(kc, k, upto_start=False), batch.fill(vc, v, upto_start=False)
            kc, vc, qs, gs, sk = kc.to(dev), vc.to(dev), batch.rows(q).to(dev).flatten(1), batch.rows(gate).to(dev), sinks.to(dev)
            out = torch.empty(len(qs), heads * dim, dtype=dtype, device=dev)
            grp, chunk, cap = batch.group, 100, 5.0
            ptr = lambda t: None if t is None else t.data_ptr()
            rc = _lib.load_masked().nva_masked_attn(
                qs.data_ptr(), qs.stride(0), kc.data_ptr(), vc.data_ptr(), grp.block_tables.data_ptr(), grp.block_tables.stride(0), grp.block_tables.shape[1],
                ptr(grp.cu), grp.seq_lens.data_ptr(), ptr(grp.token_seq), out.data_ptr(), None, 0, grp.count, grp.num_seqs, grp.max_q, heads, kv, dim, dim,
                BLOCK, batch.num_blocks, 0, chunk, 0.3, cap, sk.data_ptr(), None, None, gs.data_ptr(), heads, _lib.DTYPE_BF16 if dtype is BF16 else _lib.DTYPE_F32,
                torch.cuda.current_stream().cuda_stream)
            _lib.check(rc, "nva_masked_attn")
            want = []
            for a, b, c, z in zip(q, k, v, gate):
                i = torch.arange(len(a))
                seen = (i[:, None] >= i[None]) & (i[:, None] // chunk == i[None] // chunk)
                o = torch.zeros(len(a), heads, dim, dtype=F64)
                for h in range(heads):
                    s = plain.soft_cap(a[:, h].double() @ b[:, h // 2].double().T * 0.3, cap).masked_fill(~seen, -math.inf)
                    p = torch.softmax(torch.cat([s, sinks[h].double().expand(len(a), 1)], 1), -1)[:, :-1]
                    o[:, h] = p @ c[:, h // 2].double()
                want.append(o * torch.sigmoid(z.double())[..., None])
            close(out.view(-1, heads, dim), batch.rows(want), tol(dtype, 1e-2, 1e-5), f"single {batch.single}")
