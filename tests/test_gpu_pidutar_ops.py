"""Every mechanism of the Pidutar layers alone, on the GPU, against the plain implementation: ragged batches of
portions and of single tokens, pages in random order, state left by earlier rows."""
import pytest
import torch

from oracle import pidutar as plain
from nanovllm_amd.engine import branches, experts, latent
from nanovllm_amd.engine.mixers import RopeTables, Rotary
from nanovllm_amd.engine.mlstm import mlstm

from row_batches import BF16, BLOCK, F32, Batch, batches, close, rand, tol

pytestmark = pytest.mark.gpu
F64 = torch.float64


# ---- the residual step ---------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("width", [8, 50, 104, 512, 1544, 4096, 5000])
def test_branches_and_their_norms(dev, dtype, width):
    g = torch.Generator().manual_seed(width)
    n, vocab, eps = 37, 90, 1e-5
    table, y1 = rand(g, vocab, width, dtype=dtype), rand(g, n, width, dtype=dtype)
    w1, w2, g1, g2 = (0.3 * rand(g, width, dtype=dtype) for _ in range(4))
    ids = torch.randint(0, vocab, (n,), generator=g)
    on = lambda *t: [x.to(dev) for x in t]
    counters = torch.full((700,), 9, dtype=torch.int32, device=dev)
    res, a, b = branches.embed_rms_norms(ids.to(dev), table.to(dev), 2.5, on(w1, w2), eps, 1.0, counters[:600])
    x = table[ids].double() * 2.5
    t = tol(dtype, 6e-3, 3e-6)
    assert res.dtype == F32 and a.dtype == dtype and not counters[:600].any() and bool((counters[600:] == 9).all())
    close(res, x, 1e-6, "residual")
    close(a, plain.centred_weight_norm(x, w1.double(), eps), t, "first norm")
    close(b, plain.centred_weight_norm(x, w2.double(), eps), t, "second norm")
    for terms in (0, 1, 3, 8):
        y2 = rand(g, n * terms, width, dtype=dtype) if terms else None
        weight = torch.rand(n, terms, generator=g) if terms else None
        add = g1.double() * y1.double()
        if terms:
            add = add + g2.double() * (weight.double()[..., None] * y2.double().view(n, terms, width)).sum(1)
        want = res.double().cpu() + 0.7 * add
        args = (0.7, y1.to(dev), g1.to(dev)) + ((y2.to(dev), weight.to(dev), g2.to(dev)) if terms else (None, None, None))
        rows, before = torch.tensor([5, 36, 0, 5], dtype=torch.int32), res.clone()
        picked = branches.branches_rms_norms(res, *args, on(w1) + [None], eps, 1.0, rows=rows.to(dev))
        assert torch.equal(res, before) and picked[1] is None
        a, b = branches.branches_rms_norms(res, *args, on(w1, w2), eps, 1.0, clear=counters)
        assert torch.equal(picked[0], a[rows.long().to(dev)]) and not counters.any()
        close(res, want, 2e-6, "residual after the add")
        close(a, plain.centred_weight_norm(want, w1.double(), eps), t, "first norm")
        close(b, plain.centred_weight_norm(want, w2.double(), eps), t, "second norm")
    plain_weight = branches.branches_rms_norms(res, 1.0, None, None, y1.to(dev), None, None, on(w1) + [None], eps, 0.0)[0]
    close(plain_weight, plain.unit_rms(want + y1.double(), eps) * w1.double(), t, "dense second branch, weight stored plainly")


# ---- products of groups, the router, experts -----------------------------------------------------------

@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", [(1, 8, 16), (3, 20, 9), (5, 72, 40), (2, 1, 520), (16, 128, 512), (4, 513, 128), (1, 30, 1032)])
def test_grouped_linear(dev, dtype, shape):
    groups, n_out, k = shape
    g = torch.Generator().manual_seed(n_out)
    for n in (1, 5, 17, 40, 150):
        x, w = rand(g, n, groups, k + 8, dtype=dtype), rand(g, groups, n_out, k, dtype=dtype)
        want = torch.einsum("ngk,gok->ngo", x[..., :k].double(), w.double())
        out = torch.full((n, groups, n_out + 4), 9.0, dtype=dtype, device=dev)
        experts.grouped_linear(x.to(dev)[..., :k], w.to(dev), out[..., :n_out])
        close(out[..., :n_out], want, tol(dtype, 5e-3, 3e-6), f"{n} rows")
        assert bool((out[..., n_out:] == 9).all())
        if groups == 1:
            got = experts.linear_f32(x[:, 0, :k].contiguous().to(dev), w[0].to(dev))
            assert got.dtype == F32
            close(got, want[:, 0], 3e-6, "kept in fp32")


def _assignments_are_whole(a, n, top):
    """Every assignment is in exactly its expert's list."""
    choice, lists, counts = a.choice.cpu(), a.lists.cpu(), a.counts.cpu()
    assert int(counts.sum()) == n * top
    for e, c in enumerate(counts.tolist()):
        mine = lists[e, :c].sort().values
        assert torch.equal(mine.long(), (choice.flatten() == e).nonzero()[:, 0])


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", [(8, 3, 64), (5, 5, 50), (1, 1, 16), (64, 8, 256), (130, 6, 96), (1000, 40, 40), (16, 1, 1032)])
def test_router(dev, dtype, shape):
    n_experts, top, width = shape
    g = torch.Generator().manual_seed(n_experts)
    for n in (1, 16, 45) + ((5000,) if n_experts <= 128 else ()):
        h, w = rand(g, n, width, dtype=dtype), rand(g, n_experts, width, dtype=dtype) * width ** -0.5
        w = w.to(dtype)
        z = h.double() @ w.double().T
        chosen, weight = plain.route(z, top, 1.7)
        counts = torch.zeros(n_experts, dtype=torch.int32, device=dev)
        a = experts.route(h.to(dev), w.to(dev), top, 1.7, counts)
        got = a.choice.cpu().long()
        # (two logits a rounding apart may trade places)
        near = (z.gather(1, got) - z.gather(1, chosen)).abs()
        assert float(near.max()) < 1e-5 and float((got == chosen).double().mean()) > 0.99
        assert bool((got.sort(1).values.diff(dim=1) > 0).all())
        close(a.weight, weight, 2e-5, "weights")
        _assignments_are_whole(a, n, top)


def test_router_prefers_the_lower_index_of_equals(dev):
    h, w = torch.ones(3, 16, dtype=BF16, device=dev), torch.zeros(70, 16, dtype=BF16, device=dev)
    w[69], w[4] = 0.5, 0.5
    a = experts.route(h, w, 4, 1.0, torch.zeros(70, dtype=torch.int32, device=dev))
    assert a.choice.cpu().tolist() == [[4, 69, 0, 1]] * 3


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", [(6, 2, 64, 40), (3, 3, 50, 27), (16, 4, 256, 128), (1, 1, 16, 24), (40, 6, 192, 48), (4, 2, 520, 200), (8, 2, 1024, 768), (5, 2, 256, 96), (70, 35, 64, 36)])
@pytest.mark.parametrize("n", [1, 7, 60, 700, 1500, 4100])
def test_experts(dev, dtype, shape, n):
    """Both products and the weighted sum, with rows spread evenly and with (nearly) all of them at one expert."""
    n_experts, top, width, ff = shape
    if width * ff * n > 2 ** 28:
        n = 330
    for skewed in (False, True):
        g = torch.Generator().manual_seed(n)
        h = rand(g, n, width, dtype=dtype)
        w = {"router": rand(g, n_experts, width, dtype=F32).mul(2 * width ** -0.5).to(dtype)}
        if skewed:                                            # one expert wins everywhere, the others share the rest
            h[:, 0] = 4.0
            w["router"][n_experts // 2, 0] = 2.0
        for e in range(n_experts):
            w[f"e{e}.gate"], w[f"e{e}.up"] = (rand(g, ff, width, dtype=F32).mul(width ** -0.5).to(dtype) for _ in range(2))
            w[f"e{e}.down"] = rand(g, width, ff, dtype=F32).mul(ff ** -0.5).to(dtype)
        spec = experts.ExpertsSpec(n_experts, top, ff, 0.9)
        with torch.device(dev):
            weights = experts.ExpertWeights(spec, width).to(dtype).requires_grad_(False)
        weights.load(spec, width, lambda name, size: w[name], "")
        run = experts.Experts(spec, weights, dev)
        y, shared, weight = run(h.to(dev))
        assert shared is None
        got = (y.double().view(n, top, width) * weight.double()[..., None]).sum(1)
        want = plain.expert_mixture(h.double(), lambda name: w[name].double(), dict(router=dict(experts=n_experts, top=top, scale=0.9)))
        err = ((got.cpu() - want).abs().amax(1) / want.abs().max())
        # (rows whose last choice is a rounding away from the next one may differ by an expert)
        z = (h.double() @ w["router"].double().T).sort(-1, descending=True).values
        clear = z[:, top - 1] - z[:, top] > 1e-4 if top < n_experts else torch.ones(n, dtype=torch.bool)
        assert torch.isfinite(got).all() and float(err[clear].max()) < tol(dtype, 1.5e-2, 1e-5), (skewed, float(err[clear].max()))


@pytest.mark.parametrize("shape", [  # experts, top, inner size, outputs, rows
    (3, 2, 1536, 264, 1500), (2, 1, 1568, 96, 1100), (70, 2, 1600, 520, 20000), (4, 3, 96, 200, 900), (3, 2, 736, 72, 1300), (9, 2, 128, 520, 330)])
@pytest.mark.parametrize("gated", [True, False])
def test_tiles_of_experts(dev, shape, gated):
    """Products with many rows per expert, whole and ragged tiles of every form, an expert without rows, against fp32 products."""
    n_experts, top, k, n_out, n = shape
    g = torch.Generator(device=dev).manual_seed(k)
    rnd = lambda *s: torch.randn(*s, generator=g, device=dev)
    x = rnd(n if gated else n * top, k).bfloat16()
    w = rnd(n_experts, 2 * n_out if gated else n_out, k).mul(k ** -0.5).bfloat16()
    router = rnd(n_experts, 64).bfloat16()
    router[0] = 0.0                                          # (with all-positive rows below: never among the best)
    h = rnd(n, 64).bfloat16()
    h[:, 0], router[:, 0] = 8.0, 8.0
    router[0, 0] = -8.0
    a = experts.route(h, router, top, 1.0, torch.zeros(n_experts, dtype=torch.int32, device=dev))
    assert n_experts == 1 or top == n_experts or int(a.counts[0]) == 0
    got = experts.routed_linear(x, w, a, experts.SILU if gated else None)
    for e in range(n_experts):
        rows = (a.choice.flatten() == e).nonzero()[:, 0]
        y = x[rows // top if gated else rows].float() @ w[e].float().T
        if gated:
            y = torch.nn.functional.silu(y[:, :n_out]) * y[:, n_out:]
        if len(rows):
            err = (got[rows].float() - y).abs().max() / y.abs().max()
            assert float(err) < 6e-3, (e, len(rows), float(err))


# ---- latent attention --------------------------------------------------------------------------------------

LATENT = [  # heads, unrotated, rotated, value size, query rank, latent rank
    (6, 48, 24, 40, 56, 72), (8, 128, 64, 128, 192, 512), (3, 20, 6, 12, 22, 18), (1, 8, 2, 8, 8, 8), (20, 72, 32, 96, 120, 192),
    (33, 24, 32, 16, 64, 256), (2, 200, 96, 144, 40, 128), (17, 64, 64, 64, 96, 384), (4, 32, 16, 48, 30, 600)]


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", LATENT)
def test_what_a_token_leaves_behind(dev, dtype, shape):
    heads, dim, rot, vdim, q_rank, rank = shape
    rope = RopeTables(1024, dev).get(Rotary(200.0, rot))
    m = dict(kv_rank=rank, rot=dict(base=200.0, dims=rot))
    for batch in batches(dev):
        g = torch.Generator().manual_seed(7)
        columns = q_rank + rank + rot + heads
        full = [rand(g, n, columns, dtype=dtype) for n, _ in batch.spans]
        wq, wkv = 1 + 0.3 * rand(g, q_rank, dtype=dtype), 1 + 0.3 * rand(g, rank, dtype=dtype)
        x = batch.rows(full)
        pad = torch.zeros(x.shape[0], -columns % 8, dtype=dtype)
        x = torch.cat([x, pad], 1).to(dev)
        cache = torch.full((batch.num_blocks, BLOCK, rank + rot), 7.0, dtype=dtype, device=dev)
        q = torch.empty((x.shape[0], q_rank), dtype=dtype, device=dev)
        latent.latent_prepare(x, wq.to(dev), wkv.to(dev), rope, q, cache, batch.group, rot, 1e-5)
        n = x.shape[0] - batch.pad
        t = tol(dtype, 6e-3, 3e-6)
        close(q[:n], plain.unit_rms(batch.rows(full)[:n, :q_rank].double(), 1e-5) * wq.double(), t, "query latent")
        keys = []
        for f in full:
            h = f.double()[:, q_rank: q_rank + rank + rot]
            keys.append(torch.cat(plain.latent_keys(h, lambda name: torch.eye(rank + rot, dtype=F64) if name == "dkv" else wkv.double(), m, 1e-5), 1))
        got, want = batch.gather(cache), batch.rows(keys)[:n]
        close(got[:, :rank], want[:, :rank], t, "latent")
        close(got[:, rank:], want[:, rank:], t, "rotated part")
        untouched = torch.ones(batch.num_blocks * BLOCK, dtype=torch.bool)
        slots = batch.group.slot_mapping.long().cpu()
        untouched[slots[slots >= 0]] = False
        assert bool((cache.view(-1, rank + rot).cpu()[untouched] == 7).all())
        again = torch.empty_like(q)                           # a layer that reads another one's cache
        latent.latent_prepare(x, wq.to(dev), None, rope, again, None, batch.group, rot, 1e-5)
        close(again[:n], q[:n], tol(dtype, 8e-3, 1e-6), "query latent alone")


def _latent_case(dev, dtype, batch, shape, window, scale, expanded, edit=None):
    """Absorbed form: queries that have met the key product; expanded: keys and values multiplied out by torch."""
    heads, dim, rot, vdim, _, rank = shape
    g = torch.Generator().manual_seed(3)
    q = [rand(g, n, heads, dim + rot, dtype=dtype) for n, _ in batch.spans]
    rows = [rand(g, n, rank + rot, dtype=dtype) for n, _ in batch.spans]
    gate = [rand(g, n, heads, dtype=dtype) for n, _ in batch.spans]
    uk, uv = (rand(g, heads, s, rank, dtype=F32).mul(rank ** -0.5).to(dtype) for s in (dim, vdim))
    if edit is not None:
        edit(q, rows, gate, uk, uv)
    cache = torch.full((batch.num_blocks, BLOCK, rank + rot), float("nan"), dtype=dtype)
    batch.fill(cache, rows, upto_start=False)
    cache = cache.to(dev)
    rope = RopeTables(2048, dev).get(Rotary(200.0, rot))
    qs, gates = batch.rows(q).to(dev), batch.rows(gate).to(dev)
    want = []
    for a, c, z in zip(q, rows, gate):
        a, c, z = a.double(), c.double(), z.double()
        turned = torch.cat([a[..., :dim], plain.rotate_neighbours(a[..., dim:], 200.0, rot)], -1)
        k = torch.cat([torch.einsum("tr,hdr->thd", c[:, :rank], uk.double()), c[:, None, rank:].expand(-1, heads, -1)], -1)
        v = torch.einsum("tr,hvr->thv", c[:, :rank], uv.double())
        want.append(plain.softmax_attention(turned, k, v, scale, plain.window_visible(len(a), window)) * torch.sigmoid(z)[..., None])
    want = batch.rows(want)
    if expanded:
        counts = [min(n - c, window - 1) + c for n, c in batch.spans]
        key_cu = torch.tensor([0] + counts).cumsum(0).to(torch.int32).to(dev)
        keys = latent.latent_gather(cache, batch.group, key_cu, sum(counts))
        wanted = torch.cat([r[len(r) - c:] for r, c in zip(rows, counts)])
        assert torch.equal(keys.cpu(), wanted)
        kv = torch.cat([torch.einsum("tr,hdr->thd", wanted[:, :rank].double(), u.double()).flatten(1) for u in (uk, uv)], 1).to(dtype).to(dev)
        out = torch.full((qs.shape[0], heads * vdim), 9.0, dtype=dtype, device=dev)
        latent.latent_prefill(qs.flatten(1), kv, keys[:, rank:], gates, rope, batch.group, key_cu, out, dim, vdim, window, scale)
        return out.view(-1, heads, vdim), want
    met = torch.einsum("thd,hdr->thr", batch.rows(q)[..., :dim].double(), uk.double()).to(dtype).to(dev).contiguous()
    out = torch.full((qs.shape[0], heads, rank), 9.0, dtype=dtype, device=dev)
    latent.latent_attention(met, qs[..., dim:], gates, rope, cache, batch.group, out, window, scale)
    return torch.einsum("thr,hvr->thv", out.double().cpu(), uv.double()), want


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", LATENT)
@pytest.mark.parametrize("window", [1, 37, 256, 300, 4096])
def test_attention_over_cached_latents(dev, dtype, shape, window):
    for batch in batches(dev) + [Batch(dev, [(600, 2), (256, 3), (40, 7)], seed=4)]:
        # (pages that no row has been written to hold NaN: what is not seen must not reach the result)
        got, want = _latent_case(dev, dtype, batch, shape, window, 0.7 * (shape[1] + shape[2]) ** -0.5, False)
        close(got, want, tol(dtype, 1.5e-2, 1e-5), f"window {window} single {batch.single}")


@pytest.mark.parametrize("shape", [s for s in LATENT if s[1] % 8 == 0 and s[2] % 8 == 0])
@pytest.mark.parametrize("window", [1, 37, 64, 256, 300, 4096])
def test_attention_over_keys_multiplied_out(dev, shape, window):
    for batch in (Batch(dev, PORTIONS_LONG, seed=1), Batch(dev, [(2, 2), (600, 3), (1, 1)], seed=2)):
        got, want = _latent_case(dev, BF16, batch, shape, window, 0.7 * (shape[1] + shape[2]) ** -0.5, True)
        close(got, want, 1.5e-2, f"window {window}")


PORTIONS_LONG = [(300, 300), (2, 2), (257, 3), (600, 90), (40, 2), (130, 65), (1, 1), (70, 69), (513, 400)]


@pytest.mark.parametrize("form", ["absorbed", "expanded", "plain"])
@pytest.mark.parametrize("window", [48, 256, 300])
def test_one_loud_key_at_the_edges(dev, form, window):
    """Key j answers every query far above the rest: the queries that see it, and only those, return its value."""
    shape = (4, 64, 32, 64, 0, 128)
    dtype, rank = (F32 if form == "plain" else BF16), 128
    n = 2 * window + 70
    for loud in (0, 1, window - 1, window, 255, 256, n - 2):
        def edit(q, rows, gate, uk, uv):
            uk.zero_(), uv.zero_()
            uk[:, 0, 0] = uv[:, 3, 1] = 1.0
            for a, c, z in zip(q, rows, gate):
                a[..., 0], a[..., 64:] = 8.0, 0.0
                z.fill_(20.0)
                c[:, 0], c[:, 1] = 0.0, 1.0
                if loud < len(c):
                    c[loud, 0], c[loud, 1] = 16.0, 3.0
        ends = [e for e in (loud + 1, min(loud + window, n), min(loud + window + 1, n), n) if e > 0]
        bs = [Batch(dev, [(n, n), (n, 70), (n, 2)], seed=loud)]
        if form != "expanded":
            bs.append(Batch(dev, [(e, 1) for e in ends], single=True, seed=loud))
        for batch in bs:
            got, want = _latent_case(dev, dtype, batch, shape, window, 0.25, form == "expanded", edit=edit)
            close(got, want, tol(dtype, 1e-2, 1e-5), f"loud key {loud}")
            pos = batch.positions.cpu()[: len(got)]
            sees = (pos >= loud) & (pos - loud < window)
            assert bool(((got.cpu()[..., 3] - 3.0).abs().amax(1) < 0.1).eq(sees).all()), loud


# ---- matrix memory ---------------------------------------------------------------------------------------------

MEMORY = [  # heads, key size, value size
    (3, 32, 48), (3, 64, 24), (2, 128, 128), (2, 12, 20), (2, 20, 9), (4, 64, 160), (2, 192, 64), (1, 256, 128), (2, 128, 256), (2, 320, 64), (1, 8, 512)]


def _memory_after(k, v, log_in, log_keep):
    """State, mass and reference after all rows, as weighted sums."""
    t = k.shape[0]
    run = log_keep.cumsum(0)
    score = run[-1] - run + log_in                             # [T, H]
    top = torch.maximum(score.amax(0), run[-1])                # (m_0 = 0 decays like everything else)
    w = torch.exp(score - top)
    return torch.einsum("th,thd,thv->hdv", w, k, v), torch.einsum("th,thd->hd", w, k), top


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", MEMORY)
@pytest.mark.parametrize("gates", [(0.0, 4.0, 6.0), (-6.0, -2.0, 8.0), (8.0, 9.0, 15.0)])
def test_matrix_memory(dev, dtype, shape, gates):
    heads, dim, vdim = shape
    in_bias, keep_bias, cap = gates
    sizes = [heads * dim, heads * dim, heads * vdim, heads * vdim]
    many = batches(dev) + [Batch(dev, [(900, 900), (700, 640)], seed=5)]
    for batch in many if dim * vdim <= 128 * 128 else many[:2]:
        g = torch.Generator().manual_seed(11)
        full = [rand(g, n, sum(sizes), dtype=dtype) for n, _ in batch.spans]
        z = [2.0 * torch.randn(n, 2 * heads, generator=g) for n, _ in batch.spans]
        bias = torch.randn(2 * heads, generator=g) + torch.tensor([in_bias] * heads + [keep_bias] * heads)
        weight = 1 + 0.3 * rand(g, heads * vdim, dtype=dtype)
        state, mass, top = (torch.full((batch.num_state_slots, heads) + s, 1e6) for s in ((dim, vdim), (dim,), ()))
        want, last = [], []
        for x, zz, (n, c), slot in zip(full, z, batch.spans, batch.state_slots):
            q, k, v, gate = x.double().split(sizes, dim=1)
            q, k, v = q.view(n, heads, dim) * dim ** -0.5, k.view(n, heads, dim), v.view(n, heads, vdim)
            both = plain.soft_cap(zz.double() + bias.double(), cap)
            log_in, log_keep = both[:, :heads], plain.log_sigmoid(both[:, heads:])
            o = plain.matrix_memory(q, k, v, log_in, log_keep)
            want.append(plain.unit_rms(o, 1e-5).reshape(n, -1) * weight.double() * torch.sigmoid(gate))
            if n - c > 0:
                state[slot], mass[slot], top[slot] = (t.float() for t in _memory_after(k[: n - c], v[: n - c], log_in[: n - c], log_keep[: n - c]))
            last.append(_memory_after(k, v, log_in, log_keep))
        held = [t.clone() for t in (state, mass, top)]
        state, mass, top = (t.to(dev) for t in (state, mass, top))
        x, zz = batch.rows(full).to(dev), batch.rows(z).to(dev).contiguous()
        out = torch.full((x.shape[0], heads * vdim), 9.0, dtype=dtype, device=dev)
        mlstm(x, zz, bias.to(dev), weight.to(dev), state, mass, top, batch.group, out, dim ** -0.5, cap, 1e-5)
        what = f"{shape} {gates} single {batch.single} spans {batch.spans}"
        close(out, batch.rows(want), tol(dtype, 1e-2, 1e-4), what)
        for name, got, before, part in (("state", state, held[0], 0), ("mass", mass, held[1], 1), ("reference", top, held[2], 2)):
            got = got.cpu()
            for after, slot in zip(last, batch.state_slots):  # fp32 whatever the projections are
                close(got[slot], after[part], 1e-4, name + " " + what)
                before[slot] = got[slot]
            assert torch.equal(got, before), "a slot of no sequence was written"
