"""Every mechanism of the Bedenex layers alone, on the GPU, against the plain implementation: ragged batches of
portions and of single tokens, pages in random order, unwritten pages full of NaN."""
import math

import pytest
import torch

from oracle import bedenex as plain
from nanovllm_amd.engine import branches, experts, latent, masked, mixers
from nanovllm_amd.engine.latent import LatentSpec
from nanovllm_amd.engine.mixers import RopeTables, Rotary

from row_batches import BF16, BLOCK, F32, Batch, batches, close, rand, tol

pytestmark = pytest.mark.gpu
F64 = torch.float64


# ---- the stream ----------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("width", [8, 50, 104, 512, 1544, 4096, 5000])
@pytest.mark.parametrize("n", [37, 1100])
def test_gated_branches_and_beginnings(dev, dtype, width, n):
    g = torch.Generator().manual_seed(width)
    vocab, eps, t = 90, 1e-5, tol(dtype, 6e-3, 3e-6)
    table, y1 = rand(g, vocab, width, dtype=dtype), rand(g, n, width, dtype=dtype)
    w, step = 1 + 0.3 * rand(g, width, dtype=dtype), rand(g, width, dtype=dtype)
    logits, bias = rand(g, n, 2 * width + 8 + -2 * width % 8, dtype=dtype), rand(g, 2 * width, dtype=dtype)
    ids = torch.randint(0, vocab, (n,), generator=g)
    counters = torch.full((700,), 9, dtype=torch.int32, device=dev)
    both = torch.full((n, 2 * width), 7.0, dtype=dtype, device=dev)
    # embeddings beside their norm, or on both sides of what a pass begins from
    res, h, none = branches.embed_rms_norms(ids.to(dev), table.to(dev), 1.0, (w.to(dev), None), eps, clear=counters[:600], copy=both[:, width:])
    assert none is None and torch.equal(res.cpu(), table[ids].float()) and torch.equal(both[:, width:].cpu(), table[ids]) and bool((both[:, :width] == 7).all())
    close(h, plain.weighted_norm(table[ids].double(), w.double(), eps), t, "embedding norm")
    again, _, _ = branches.embed_rms_norms(ids.to(dev), table.to(dev), 1.0, (None, None), eps, out=both[:, :width], copy=both[:, width:])
    assert torch.equal(again, res) and torch.equal(both[:, :width], both[:, width:]) and not counters[:600].any() and bool((counters[600:] == 9).all())
    z = logits[:, 8: 8 + 2 * width]
    gates = torch.sigmoid(z.double() + bias.double())
    for terms in (0, 1, 3, 8):
        y2 = rand(g, n * terms, width, dtype=dtype) if terms else None
        want = res.double().cpu() + gates[:, :width] * y1.double()
        if terms:
            want = want + gates[:, width:] * y2.double().view(n, terms, width).sum(1)
        args = (y1.to(dev), None if y2 is None else y2.to(dev), logits.to(dev)[:, 8: 8 + (2 if terms else 1) * width], bias.to(dev))
        rows, before = torch.tensor([5, 36, 0, 5], dtype=torch.int32), res.clone()
        picked = branches.gated_rms_norm(res, *args, w.to(dev), eps, rows=rows.to(dev))
        assert torch.equal(res, before)
        other = res.clone()
        normed = branches.gated_rms_norm(other, *args, w.to(dev), eps)
        counters.fill_(9)
        branches.gated_rms_norm(res, *args, None, eps, clear=counters[:600], out=both[:, :width])
        assert torch.equal(other, res) and torch.equal(both[:, :width], res.to(dtype)) and torch.equal(both[:, width:].cpu(), table[ids])
        assert not counters[:600].any() and bool((counters[600:] == 9).all())
        close(picked, normed[rows.long().to(dev)], tol(dtype, 8e-3, 2e-6), "picked rows")       # (few rows: sums in another order)
        close(res, want, 3e-6, f"residual, {terms} terms")
        close(normed, plain.weighted_norm(want, w.double(), eps), t, f"norm, {terms} terms")
    product = torch.randn(n, width, generator=g)
    counters.fill_(9)
    out = branches.entry_rms_norm(product.to(dev), step.to(dev), res, w.to(dev), eps, clear=counters[:600])
    want = product.double() + step.double()
    close(res, want, 1e-6, "begun anew")
    close(out, plain.weighted_norm(want, w.double(), eps), t, "its norm")
    assert not counters[:600].any() and bool((counters[600:] == 9).all())


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", [(16, 32), (50, 100), (1024, 2048), (104, 208), (1536, 3072)])
def test_product_whose_sums_stay_fp32(dev, dtype, shape):
    rows_out, k = shape
    g = torch.Generator().manual_seed(k)
    w = rand(g, rows_out, k, dtype=F32).mul(k ** -0.5).to(dtype)
    for n in (1, 16, 65, 700):
        x = rand(g, n, k, dtype=dtype)
        got = experts.project_f32(x.to(dev), w.to(dev))
        assert got.dtype == F32 and got.is_contiguous()
        close(got, x.double() @ w.double().T, 3e-6, f"{n} rows")


def test_product_in_a_replayed_graph(dev):
    """The library's form of it, several replays with other work between them."""
    g = torch.Generator().manual_seed(1)
    x, w = rand(g, 130, 2048, dtype=BF16).to(dev), rand(g, 1024, 2048, dtype=BF16).to(dev)
    held = x.clone()
    experts.project_f32(held, w)
    torch.cuda.synchronize()
    graph = torch.cuda.CUDAGraph()
    with torch.cuda.graph(graph):
        out = experts.project_f32(held, w)
    for i in range(5):
        held.copy_(x.roll(i, 0))
        graph.replay()
        want = experts.project_f32(x.roll(i, 0), w)
        torch.cuda.synchronize()
        assert torch.equal(out, want), i


# ---- feed-forwards -----------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("ff", [8, 27, 1536])
def test_gelu_gate(dev, dtype, ff):
    g = torch.Generator().manual_seed(ff)
    x = 3.0 * rand(g, 19, 2 * ff, dtype=dtype)
    x[0, :8] = torch.tensor([-60.0, -9.0, -4.0, -0.01, 0.0, 0.01, 9.0, 60.0]).to(dtype)
    want = plain.gelu(x[:, :ff].double()) * x[:, ff:].double()
    close(mixers.gelu_gate(x.to(dev)), want, tol(dtype, 5e-3, 1e-6))
    strided = torch.cat([x, x], 1).to(dev)[:, 2 * ff:]
    close(mixers.gelu_gate(strided), want, tol(dtype, 5e-3, 1e-6), "behind other columns")


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", [(8, 3, 64), (5, 5, 50), (1, 1, 16), (64, 8, 256), (130, 6, 96), (16, 1, 1032)])
def test_router_of_sigmoids(dev, dtype, shape):
    n_experts, top, width = shape
    g = torch.Generator().manual_seed(n_experts)
    for n in (1, 16, 45, 5000):
        h, w = rand(g, n, width, dtype=dtype), (rand(g, n_experts, width, dtype=F32) * 2.0 * width ** -0.5).to(dtype)
        z = h.double() @ w.double().T
        chosen, weight = plain.route(z, top)
        a = experts.route(h.to(dev), w.to(dev), top, 1.0, torch.zeros(n_experts, dtype=torch.int32, device=dev), score=experts.SIGMOID)
        got = a.choice.cpu().long()
        near = (z.gather(1, got) - z.gather(1, chosen)).abs()         # (two logits a rounding apart may trade places)
        assert float(near.max()) < 1e-5 and float((got == chosen).double().mean()) > 0.99
        close(a.weight, weight, 2e-5, "weights")
        for e, c in enumerate(a.counts.cpu().tolist()):
            assert torch.equal(a.lists.cpu()[e, :c].sort().values.long(), (got.flatten() == e).nonzero()[:, 0])


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", [  # experts, best, width, ff
    (6, 2, 64, 40), (3, 3, 50, 27), (16, 4, 256, 128), (1, 1, 16, 24), (40, 6, 192, 48), (4, 2, 520, 200), (5, 1, 256, 88), (2, 1, 1536, 136), (2, 2, 256, 96)])
@pytest.mark.parametrize("n", [1, 7, 17, 64, 65, 700, 1500])
def test_experts_that_read_weighted_rows(dev, dtype, shape, n):
    n_experts, top, width, ff = shape
    g = torch.Generator().manual_seed(n)
    h = rand(g, n, width, dtype=dtype)
    lin = lambda rows, cols, gain=1.5: rand(g, rows, cols, dtype=F32).mul(gain * cols ** -0.5).to(dtype)
    w = {"router": lin(n_experts, width, 2.0)}
    for e in range(n_experts):
        w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"] = lin(ff, width), lin(ff, width), lin(width, ff, 1.0)
    spec = experts.ExpertsSpec(n_experts, top, ff, score=experts.SIGMOID, weigh_input=True)
    with torch.device(dev):
        weights = experts.ExpertWeights(spec, width).requires_grad_(False)
    for p in weights.parameters():
        p.data = p.data.to(dtype)
    weights.load(spec, width, lambda name, size: w[name], "")
    y, shared, _ = experts.Experts(spec, weights, dev)(h.to(dev))
    assert shared is None
    got = y.double().view(n, top, width).sum(1).cpu()
    want = plain.expert_mixture(h.double(), lambda name: w[name].double(), dict(router=dict(experts=n_experts, top=top)))
    z = (h.double() @ w["router"].double().T).sort(-1, descending=True).values
    clear = z[:, top - 1] - z[:, top] > 1e-4 if top < n_experts else torch.ones(n, dtype=torch.bool)
    err = (got - want).abs().amax(1) / want.abs().max()
    assert torch.isfinite(got).all() and float(err[clear].max()) < tol(dtype, 1.5e-2, 1e-5), float(err[clear].max())


# ---- what attention reads -----------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", [  # heads, key heads, key size, value size
    (6, 2, 32, 48), (8, 8, 64, 64), (3, 1, 20, 9), (1, 1, 8, 8), (40, 2, 72, 96), (33, 1, 24, 16), (32, 8, 128, 128), (5, 5, 17, 20), (16, 2, 256, 200), (70, 7, 200, 8), (4, 2, 8, 512)])
def test_norms_without_weights_and_of_values(dev, dtype, shape):
    heads, kv, dim, vdim = shape
    queries, keys = heads * dim, kv * dim
    columns = queries + keys + kv * vdim
    for batch in batches(dev):
        g = torch.Generator().manual_seed(7)
        full = [rand(g, n, columns, dtype=dtype) * (0.1 + torch.rand(n, 1, generator=g)).to(dtype) for n, _ in batch.spans]
        for qk_norm, v_norm in ((masked.UNIT, True), (masked.UNIT, False), (None, True)):
            x = batch.rows(full)
            x = torch.cat([x, torch.full((x.shape[0], 8 + -x.shape[1] % 8), 5.0, dtype=dtype)], 1).to(dev)
            kc = torch.full((batch.num_blocks, BLOCK, kv, dim), 7.0, dtype=dtype, device=dev)
            vc = torch.full((batch.num_blocks, BLOCK, kv, vdim), 7.0, dtype=dtype, device=dev)
            q = torch.full((x.shape[0], queries), 9.0, dtype=dtype, device=dev)
            masked.qkv_prepare(x, None, None, None, qk_norm, None, q, kc, vc, batch.group, heads, kv, dim, vdim, 1e-3, v_norm)
            n, t = x.shape[0] - batch.pad, tol(dtype, 6e-3, 5e-6)
            rows = batch.rows([f.double() for f in full])[:n]
            parts = rows[:, :queries].reshape(n, heads, dim), rows[:, queries: queries + keys].reshape(n, kv, dim), rows[:, queries + keys:].reshape(n, kv, vdim)
            norm_qk = (lambda y: plain.head_norm(y, 1e-3)) if qk_norm else (lambda y: y)
            close(q[:n].view(n, heads, dim), norm_qk(parts[0]), t, "queries")
            assert not q[n:].any()
            close(batch.gather(kc), norm_qk(parts[1]), t, "keys")
            close(batch.gather(vc), plain.value_norm(parts[2], 1e-3) if v_norm else parts[2], t, "values")
            untouched = torch.ones(batch.num_blocks * BLOCK, dtype=torch.bool)
            slots = batch.group.slot_mapping.long().cpu()
            untouched[slots[slots >= 0]] = False
            assert bool((kc.view(-1, keys).cpu()[untouched] == 7).all()) and bool((vc.view(-1, kv * vdim).cpu()[untouched] == 7).all())


# ---- attention in chunks with a distance bias -------------------------------------------------------------------

ATTN = [  # heads, key heads, key size, value size
    (6, 2, 32, 48), (8, 8, 64, 64), (3, 1, 20, 9), (1, 1, 8, 8), (40, 2, 72, 96), (33, 1, 24, 16), (8, 2, 128, 128), (4, 4, 160, 32), (10, 5, 96, 96), (2, 1, 256, 200),
    (2, 2, 64, 128), (2, 1, 128, 64), (4, 1, 128, 256), (5, 5, 17, 20)]


def _chunk_case(dev, dtype, batch, shape, chunk, scale, edit=None):
    heads, kv, dim, vdim = shape
    g = torch.Generator().manual_seed(3)
    q = [rand(g, n, heads, dim, dtype=dtype) for n, _ in batch.spans]
    k = [rand(g, n, kv, dim, dtype=dtype) for n, _ in batch.spans]
    v = [rand(g, n, kv, vdim, dtype=dtype) for n, _ in batch.spans]
    gate = [rand(g, n, heads, dtype=dtype) for n, _ in batch.spans]
    r1, r2 = 2.5 * torch.rand(heads, generator=g), 0.02 + torch.rand(heads, generator=g)
    r1[0] = 0.0
    if edit is not None:
        edit(q, k, v, gate, r1, r2)
    kc, vc = (torch.full((batch.num_blocks, BLOCK, kv, d), float("nan"), dtype=dtype) for d in (dim, vdim))
    batch.fill(kc, k, upto_start=False), batch.fill(vc, v, upto_start=False)
    qs = batch.rows(q).to(dev)
    gates = torch.cat([torch.zeros(len(qs), 3, dtype=dtype), batch.rows(gate)], 1).to(dev)[:, 3:]     # (a strided view, as the fused projection leaves it)
    out = torch.full((qs.shape[0], heads * vdim), 9.0, dtype=dtype, device=dev)
    masked.masked_attention(qs.flatten(1), kc.to(dev), vc.to(dev), batch.group, out, heads, chunk, scale, None, gates, chunks=True, bias=(r1.to(dev), r2.to(dev)))
    want = []
    for a, b, c, z in zip(q, k, v, gate):
        t, o = len(a), torch.zeros(len(a), heads, vdim, dtype=F64)
        seen = plain.in_chunk(t, chunk)
        for h in range(heads):
            s = a[:, h].double() @ b[:, h // (heads // kv)].double().T * scale - plain.distance_bias(t, r1[h].double(), r2[h].double())
            o[:, h] = torch.softmax(s.masked_fill(~seen, -math.inf), -1) @ c[:, h // (heads // kv)].double()
        want.append(o * torch.sigmoid(z.double())[..., None])
    return out.view(-1, heads, vdim), batch.rows(want)


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", ATTN)
@pytest.mark.parametrize("chunk", [1, 37, 64, 256, 300, 5000])
def test_chunked_attention_with_a_distance_bias(dev, dtype, shape, chunk):
    for batch in batches(dev) + [Batch(dev, [(600, 2), (256, 3), (40, 7), (513, 400)], seed=4)]:
        # (pages that no row has been written to hold NaN: what is not seen must not reach the result)
        got, want = _chunk_case(dev, dtype, batch, shape, chunk, 1.2 * shape[2] ** -0.5)
        close(got, want, tol(dtype, 1e-2, 1e-5), f"chunk {chunk} single {batch.single}")


@pytest.mark.parametrize("dtype", [BF16, F32])
def test_long_chunks_in_many_ranges(dev, dtype):
    """Chunks over several key ranges of a decode step."""
    for shape in ((8, 2, 128, 128), (4, 4, 64, 64)):
        for chunk in (700, 1500, 4096):
            got, want = _chunk_case(dev, dtype, Batch(dev, [(2100, 1), (1537, 1), (512, 1), (3, 1)], single=True, seed=2), shape, chunk, 0.1)
            close(got, want, tol(dtype, 1e-2, 1e-5), f"{shape} chunk {chunk}")


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", [(4, 2, 64, 64), (2, 1, 128, 128), (2, 2, 96, 64), (3, 1, 20, 12)])
@pytest.mark.parametrize("chunk", [48, 256, 300])
def test_one_loud_key_at_the_edges(dev, dtype, shape, chunk):
    """Key j answers every query far above the rest: the queries of its chunk that come after it, and only those, return its value."""
    n = 2 * chunk + 70
    for loud in sorted({0, 1, chunk - 1, chunk, chunk + 1, 2 * chunk - 1, 255, 256, n - 2}):
        def edit(q, k, v, gate, r1, r2):
            for a, b, c, z in zip(q, k, v, gate):
                a[..., 0], b[..., 0], c[..., 3] = 8.0, 0.0, 1.0
                a[..., 1:], b[..., 1:] = 0.0, 0.0
                z.fill_(20.0)
                if loud < len(b):
                    b[loud, :, 0], c[loud, :, 3] = 16.0, 3.0
        edge = (loud // chunk + 1) * chunk
        ends = sorted({e for e in (loud, loud + 1, min(edge, n), min(edge + 1, n), n) if e > 0})
        for batch in (Batch(dev, [(n, n), (n, 70), (n, 2)], seed=loud), Batch(dev, [(e, 1) for e in ends], single=True, seed=loud)):
            got, want = _chunk_case(dev, dtype, batch, shape, chunk, 0.25, edit=edit)
            close(got, want, tol(dtype, 1e-2, 1e-5), f"loud key {loud}")
            pos = batch.positions.cpu()[: len(got)]
            sees = (pos >= loud) & (pos // chunk == loud // chunk)
            assert bool(((got.cpu()[..., 3] - 3.0).abs().amax(1) < 0.1).eq(sees).all()), loud


@pytest.mark.parametrize("dtype", [BF16, F32])
def test_the_bias_alone(dev, dtype):
    """Equal scores: the weights are (1 + rate d)^-slope, up to steep ones, and the values tell the distances."""
    shape, n = (4, 2, 64, 64), 700

    def edit(q, k, v, gate, r1, r2):
        r1.copy_(torch.tensor([0.0, 1.0, 6.0, 90.0])), r2.copy_(torch.tensor([0.3, 0.01, 2.0, 50.0]))
        for a, b, c, z in zip(q, k, v, gate):
            a.zero_(), b.zero_(), z.fill_(30.0)
            c[..., 0] = (torch.arange(len(c)) % 13).to(dtype)[:, None]
    for batch in (Batch(dev, [(n, n), (n, 90), (n, 2)], seed=1), Batch(dev, [(n, 1), (300, 1), (64, 1), (1, 1)], single=True, seed=2)):
        for chunk in (100, 4096):
            got, want = _chunk_case(dev, dtype, batch, shape, chunk, 1.0, edit=edit)
            close(got, want, tol(dtype, 6e-3, 1e-5), f"chunk {chunk}")
            last = got.cpu()[..., 3, 0].double()
            assert torch.isfinite(got).all() and float((last - batch.positions.cpu()[: len(got)] % 13).abs().max()) < 0.05    # the steepest sees itself alone


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("scores", ["rising", "falling", "jumps"])
def test_running_maximum_beside_a_bias(dev, dtype, scores):
    """Scores that grow or fall by hundreds along the keys."""
    shape, n = (4, 2, 64, 64), 700

    def edit(q, k, v, gate, r1, r2):
        for a, b in zip(q, k):
            a.zero_(), b.zero_()
            a[..., 0] = 4.0
            x = torch.arange(len(b)).float()
            level = {"rising": x, "falling": -x, "jumps": (x // 64 * 37 % 11) * 12.0}[scores]
            b[..., 0] = (level / 4.0)[:, None].to(dtype)
    for batch in (Batch(dev, [(n, n), (n, 90), (n, 2)], seed=1), Batch(dev, [(n, 1), (300, 1), (64, 1), (1, 1)], single=True, seed=2)):
        for chunk in (100, 4096):
            got, want = _chunk_case(dev, dtype, batch, shape, chunk, 1.0, edit=edit)
            assert torch.isfinite(got).all() and float((got.double().cpu() - want).abs().max()) < tol(dtype, 2e-2, 5e-5), (chunk, batch.single)


# ---- latent attention with direct queries and sinks ------------------------------------------------------------

LATENT = [  # heads, unrotated, rotated, value size, latent rank
    (6, 48, 24, 40, 72), (8, 128, 64, 128, 512), (3, 20, 6, 12, 18), (1, 8, 2, 8, 8), (20, 72, 32, 96, 192), (33, 24, 32, 16, 256), (2, 200, 96, 144, 128), (17, 64, 64, 64, 384), (4, 32, 16, 48, 600)]


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", LATENT)
def test_latents_without_a_query_latent(dev, dtype, shape):
    """Cache rows of weights whose pairs were given as halves."""
    heads, dim, rot, vdim, rank = shape
    spec = LatentSpec(heads, dim, rot, vdim, 0, rank, None, 1.0, Rotary(200.0, rot), gate=False, sink=True, halves=True)
    rope = RopeTables(1024, dev).get(spec.rot)
    for batch in batches(dev):
        g = torch.Generator().manual_seed(7)
        full = [rand(g, n, rank + rot, dtype=dtype) for n, _ in batch.spans]
        weight = 1 + 0.3 * rand(g, rank, dtype=dtype)
        lead = -(-(heads * (dim + rot)) // 8) * 8                       # (the queries' columns before them)
        laid = [torch.cat([f[:, :rank], spec.paired(f[:, rank:].t()).t()], 1) for f in full]
        x = batch.rows(laid)
        x = torch.cat([torch.full((x.shape[0], lead), 3.0, dtype=dtype), x, torch.zeros(x.shape[0], -(rank + rot) % 8, dtype=dtype)], 1).to(dev)
        cache = torch.full((batch.num_blocks, BLOCK, rank + rot), 7.0, dtype=dtype, device=dev)
        latent.latent_prepare(x[:, lead:], None, weight.to(dev), rope, None, cache, batch.group, rot, 1e-5)
        t = tol(dtype, 6e-3, 3e-6)
        wanted = [torch.cat([plain.weighted_norm(f[:, :rank].double(), weight.double(), 1e-5), spec.paired(plain.turned(f[:, rank:].double(), 200.0, rot).t()).t()], 1) for f in full]
        got, want = batch.gather(cache), batch.rows(wanted)[: x.shape[0] - batch.pad]
        close(got[:, :rank], want[:, :rank], t, "latent")
        close(got[:, rank:], want[:, rank:], t, "rotated part")
        untouched = torch.ones(batch.num_blocks * BLOCK, dtype=torch.bool)
        slots = batch.group.slot_mapping.long().cpu()
        untouched[slots[slots >= 0]] = False
        assert bool((cache.view(-1, rank + rot).cpu()[untouched] == 7).all())


def _latent_case(dev, dtype, batch, shape, scale, expanded, edit=None):
    """Absorbed form: queries that have met the key product; expanded: keys and values multiplied out by torch."""
    heads, dim, rot, vdim, rank = shape
    g = torch.Generator().manual_seed(3)
    spec = LatentSpec(heads, dim, rot, vdim, 0, rank, None, scale, Rotary(200.0, rot), gate=False, sink=True, halves=True)
    q = [rand(g, n, heads, dim + rot, dtype=dtype) for n, _ in batch.spans]
    rows = [rand(g, n, rank + rot, dtype=dtype) for n, _ in batch.spans]        # (latents normed, rotated parts turned, as halves)
    uk, uv = (rand(g, heads, s, rank, dtype=F32).mul(rank ** -0.5).to(dtype) for s in (dim, vdim))
    sinks = 3.0 + 2.0 * torch.randn(heads, generator=g)
    if edit is not None:
        edit(q, rows, uk, uv, sinks)
    pair = lambda x: spec.paired(x.movedim(-1, 0)).movedim(0, -1)
    laid = [torch.cat([r[:, :rank], pair(r[:, rank:])], 1) for r in rows]
    cache = torch.full((batch.num_blocks, BLOCK, rank + rot), float("nan"), dtype=dtype)
    batch.fill(cache, laid, upto_start=False)
    cache = cache.to(dev)
    rope = RopeTables(4096, dev).get(spec.rot)
    qs = batch.rows([torch.cat([a[..., :dim], pair(a[..., dim:])], -1) for a in q]).to(dev)
    want = []
    for a, c in zip(q, rows):
        a, c, o = a.double(), c.double(), torch.zeros(len(a), heads, vdim, dtype=F64)
        turned = plain.turned(a[..., dim:], 200.0, rot)
        for h in range(heads):
            s = (a[:, h, :dim] @ (c[:, :rank] @ uk[h].double().T).T + turned[:, h] @ c[:, rank:].T) * scale
            o[:, h] = plain.softmax_with_sink(s.masked_fill(~plain.causal(len(a)), -math.inf), sinks[h].double()) @ (c[:, :rank] @ uv[h].double().T)
        want.append(o)
    want = batch.rows(want)
    if expanded:
        key_cu = torch.tensor([0] + [n for n, _ in batch.spans]).cumsum(0).to(torch.int32).to(dev)
        keys = latent.latent_gather(cache, batch.group, key_cu, sum(n for n, _ in batch.spans))
        c = torch.cat(rows)[:, :rank].double()
        kv = torch.cat([torch.stack([c @ u[h].double().T for h in range(heads)], 1).flatten(1) for u in (uk, uv)], 1).to(dtype).to(dev)
        out = torch.full((qs.shape[0], heads * vdim), 9.0, dtype=dtype, device=dev)
        latent.latent_prefill(qs.flatten(1), kv, keys[:, rank:], None, rope, batch.group, key_cu, out, dim, vdim, 1 << 30, scale, sinks.to(dev))
        return out.view(-1, heads, vdim), want
    a = batch.rows(q)[..., :dim].double()
    met = torch.stack([a[:, h] @ uk[h].double() for h in range(heads)], 1).to(dtype).to(dev).contiguous()
    out = torch.full((qs.shape[0], heads, rank), 9.0, dtype=dtype, device=dev)
    latent.latent_attention(met, qs[..., dim:], None, rope, cache, batch.group, out, 1 << 30, scale, sinks.to(dev))
    o = out.double().cpu()
    return torch.stack([o[:, h] @ uv[h].double().T for h in range(heads)], 1), want


LONG = [(300, 300), (2, 2), (257, 3), (600, 90), (40, 2), (130, 65), (1, 1), (70, 69), (513, 400)]


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", LATENT)
def test_attention_over_cached_latents_with_sinks(dev, dtype, shape):
    more = [Batch(dev, [(600, 2), (256, 3), (40, 7)], seed=4), Batch(dev, [(2100, 1), (1537, 1), (512, 1), (3, 1)], single=True, seed=2)]
    for batch in batches(dev) + more:
        got, want = _latent_case(dev, dtype, batch, shape, 0.7 * (shape[1] + shape[2]) ** -0.5, False)
        close(got, want, tol(dtype, 1.5e-2, 1e-5), f"spans {batch.spans}")


@pytest.mark.parametrize("shape", [s for s in LATENT if s[1] % 8 == 0 and s[2] % 8 == 0])
def test_attention_over_keys_multiplied_out_with_sinks(dev, shape):
    for batch in (Batch(dev, LONG, seed=1), Batch(dev, [(2, 2), (600, 3), (1, 1)], seed=2)):
        got, want = _latent_case(dev, BF16, batch, shape, 0.7 * (shape[1] + shape[2]) ** -0.5, True)
        close(got, want, 1.5e-2)


@pytest.mark.parametrize("form", ["absorbed", "expanded", "plain"])
@pytest.mark.parametrize("level", [-40.0, 0.0, 60.0])
def test_sinks_far_below_and_above_the_scores(dev, form, level):
    """Equal scores at a level: n keys of weight e^level beside e^sink; a far key that stands out is found."""
    shape = (4, 64, 32, 64, 128)
    dtype, n = (F32 if form == "plain" else BF16), 700

    def edit(q, rows, uk, uv, sinks):
        sinks.copy_(level + torch.tensor([-30.0, 0.0, 6.0, 200.0]))
        uk.zero_(), uv.zero_()
        uk[:, 0, 0] = uv[:, 3, 1] = 1.0
        for a, c in zip(q, rows):
            a.zero_()
            a[..., 0] = 4.0
            c[:, 0], c[:, 1] = level / 4.0, 1.0
            if len(c) > 300:
                c[17, 0], c[17, 1] = level / 4.0 + 4.0, 5.0
    bs = [Batch(dev, [(n, n), (n, 90), (n, 2)], seed=1)]
    if form != "expanded":
        bs.append(Batch(dev, [(n, 1), (300, 1), (64, 1), (1, 1)], single=True, seed=2))
    for batch in bs:
        got, want = _latent_case(dev, dtype, batch, shape, 1.0, form == "expanded", edit=edit)
        close(got, want, tol(dtype, 1e-2, 3e-5))                     # (up to 700 equal terms in a row)
        assert float(got[..., 3, :].abs().max()) < 1e-3 and float(want[:, 0, 3].min()) > 0.9
