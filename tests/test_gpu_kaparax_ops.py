"""Every mechanism of the Kaparax layers alone, on the GPU, against the plain implementation: ragged
batches of portions and of single tokens, pages in random order, state left by earlier rows."""
import pytest
import torch

from oracle import kaparax as plain
from nanovllm_amd.engine import mixers
from nanovllm_amd.engine.mixers import RopeTables, Rotary

from row_batches import BF16, BLOCK, F32, Batch
from row_batches import batches as _batches, close as _close, rand as _rand, tol as _tol

pytestmark = pytest.mark.gpu


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("width", [8, 50, 104, 512, 1544, 4096, 5000])
def test_norms_around_the_residual(dev, dtype, width):
    g = torch.Generator().manual_seed(width)
    n, vocab, eps = 37, 90, 1e-5
    table, y = _rand(g, vocab, width, dtype=dtype), 3.0 * _rand(g, n, width, dtype=dtype) + 0.5
    w = [1 + 0.3 * _rand(g, width, dtype=dtype) if i % 2 == 0 else 0.3 * _rand(g, width, dtype=dtype) for i in range(4)]
    ids = torch.randint(0, vocab, (n,), generator=g)
    d = [x.to(dev) for x in w]
    res, out = mixers.embed_norm(ids.to(dev), table.to(dev), 2.5, (d[0], d[1]), eps)
    x = table[ids].double() * 2.5
    assert res.dtype == F32 and out.dtype == dtype
    _close(res, x, 1e-6, "residual")
    _close(out, plain.layer_norm(x, w[0].double(), w[1].double(), eps), _tol(dtype, 6e-3, 3e-6), "norm of the embedding")
    x2 = res.double().cpu() + plain.layer_norm(y.double(), w[2].double(), w[3].double(), eps)
    want = plain.layer_norm(x2, w[0].double(), w[1].double(), eps)
    rows = torch.tensor([5, 36, 0, 5], dtype=torch.int32)
    before = res.clone()
    picked = mixers.post_add_norm(y.to(dev), res, (d[2], d[3]), (d[0], d[1]), eps, rows.to(dev))
    assert torch.equal(res, before)
    got = mixers.post_add_norm(y.to(dev), res, (d[2], d[3]), (d[0], d[1]), eps)
    assert torch.equal(picked, got[rows.long().to(dev)])
    _close(res, x2, 2e-6, "residual after the add")
    _close(got, want, _tol(dtype, 6e-3, 5e-6), "next norm")


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("ff", [8, 27, 96, 3072])
def test_clamped_gate(dev, dtype, ff):
    g = torch.Generator().manual_seed(ff)
    x = 3.0 * _rand(g, 19, 2 * ff, dtype=dtype)
    limit = 1.25
    gate, up = x[:, :ff].double().clamp(max=limit), x[:, ff:].double().clamp(-limit, limit)
    want = gate * torch.sigmoid(1.702 * gate) * (up + 1)
    _close(mixers.clamped_gate(x.to(dev), limit, 1.702), want, _tol(dtype, 5e-3, 1e-6))


ATTN = [  # heads, kv heads, key size, value size, rotated, taps
    (6, 2, 48, 40, 32, 3), (6, 1, 64, 24, 64, 4), (8, 2, 128, 128, 128, 4), (3, 3, 20, 12, 12, 2), (5, 1, 64, 96, 0, 6),
    (4, 4, 96, 64, 64, 1), (2, 1, 256, 192, 128, 8), (4, 2, 32, 24, 20, 11)]


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", ATTN)
def test_convolution_rotation_and_cache_write(dev, dtype, shape):
    heads, kv, dim, vdim, rot, taps = shape
    channels = (heads + kv) * dim + kv * vdim
    table = RopeTables(4096, dev).get(Rotary(200.0, rot))
    batches = _batches(dev)
    if shape is ATTN[0]:                                     # enough rows for the form that walks longer runs
        batches.append(Batch(dev, [(2203, 2203), (1500, 40), (2100, 2001), (1, 1), (700, 17)], seed=3))
    for batch in batches:
        g = torch.Generator().manual_seed(7)
        full = [_rand(g, n, channels, dtype=dtype) for n, _ in batch.spans]
        weight = _rand(g, taps, channels, dtype=dtype)
        state = _rand(g, batch.num_state_slots, taps - 1, channels, dtype=dtype) * 100 if taps > 1 else None
        for x, (n, c), slot in zip(full, batch.spans, batch.state_slots):
            for r in range(taps - 1):                        # rows before the portion; garbage where the sequence starts
                at = n - c - (taps - 1) + r
                if n - c > 0:
                    state[slot, r] = x[at] if at >= 0 else 0
        before = state.clone() if taps > 1 else None
        state = state.to(dev) if taps > 1 else None
        kc = torch.full((batch.num_blocks, BLOCK, kv, dim), 7.0, dtype=dtype, device=dev)
        vc = torch.full((batch.num_blocks, BLOCK, kv, vdim), 7.0, dtype=dtype, device=dev)
        x = batch.rows(full).to(dev)
        q = torch.empty((x.shape[0], heads * dim), dtype=dtype, device=dev)
        mixers.conv_rope_store(x, weight.to(dev), state, batch.group, table, q, kc, vc, heads, rot)
        ref = [plain.short_conv(f.double(), weight.t().double()) for f in full]
        n = x.shape[0] - batch.pad
        split = [r.split([heads * dim, kv * dim, kv * vdim], dim=1) for r in ref]
        want_q = batch.rows([plain.rotate(a.view(-1, heads, dim), 200.0, rot) for a, _, _ in split])
        want_k = batch.rows([plain.rotate(b.view(-1, kv, dim), 200.0, rot) for _, b, _ in split])[:n]
        want_v = batch.rows([c.view(-1, kv, vdim) for _, _, c in split])[:n]
        tol = _tol(dtype, 5e-3, 2e-6)
        _close(q.view(-1, heads, dim), want_q, tol, "q")
        _close(batch.gather(kc), want_k, tol, "k")
        _close(batch.gather(vc), want_v, tol, "v")
        written = batch.group.slot_mapping.long().cpu()
        untouched = torch.ones(batch.num_blocks * BLOCK, dtype=torch.bool)
        untouched[written[written >= 0]] = False
        assert bool((kc.view(-1, kv * dim).cpu()[untouched] == 7).all()) and bool((vc.view(-1, kv * vdim).cpu()[untouched] == 7).all())
        if taps > 1:                                         # the carried rows are the last projected ones, the other slots as they were
            after = state.cpu()
            for f, (n, _), slot in zip(full, batch.spans, batch.state_slots):
                for r in range(taps - 1):
                    at = n - (taps - 1) + r
                    assert torch.equal(after[slot, r], f[at] if at >= 0 else torch.zeros_like(f[0])), (n, slot, r)
                before[slot] = after[slot]
            assert torch.equal(after, before)


def _attention_case(dev, dtype, batch, shape, chunk, scale, cap, seed=3, edit=None):
    heads, kv, dim, vdim = shape
    g = torch.Generator().manual_seed(seed)
    q = [_rand(g, n, heads, dim, dtype=dtype) for n, _ in batch.spans]
    k = [_rand(g, n, kv, dim, dtype=dtype) for n, _ in batch.spans]
    v = [_rand(g, n, kv, vdim, dtype=dtype) for n, _ in batch.spans]
    if edit is not None:
        edit(q, k, v)
    kc = torch.full((batch.num_blocks, BLOCK, kv, dim), float("nan"), dtype=dtype)
    vc = torch.full((batch.num_blocks, BLOCK, kv, vdim), float("nan"), dtype=dtype)
    batch.fill(kc, k, upto_start=False), batch.fill(vc, v, upto_start=False)
    rows = batch.rows(q).to(dev).view(-1, heads * dim)
    out = torch.full((rows.shape[0], heads * vdim), 9.0, dtype=dtype, device=dev)
    mixers.chunk_attention(rows, kc.to(dev), vc.to(dev), batch.group, out, heads, chunk, scale, cap)
    want = batch.rows([plain.softmax_attention(a.double(), b.double(), c.double(), scale, cap, plain.chunk_visible(len(a), chunk))
                       for a, b, c in zip(q, k, v)])
    return out.view(-1, heads, vdim), want


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", [s[:4] for s in ATTN] + [(16, 1, 64, 64), (40, 2, 32, 32)])
@pytest.mark.parametrize("chunk,cap", [(1, 20.0), (37, 20.0), (64, 100.0), (210, 0.0), (256, 30.0), (4096, 50.0)])
def test_attention_in_chunks(dev, dtype, shape, chunk, cap):
    for batch in _batches(dev):
        # (pages that no row has been written to hold NaN: what is not seen must not reach the result)
        got, want = _attention_case(dev, dtype, batch, shape, chunk, 2.5 * shape[2] ** -0.5, cap)
        _close(got, want, _tol(dtype, 1e-2, 1e-5), f"chunk {chunk} cap {cap} single {batch.single}")


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("chunk", [48, 256, 300])
def test_one_loud_key_at_the_edges(dev, dtype, chunk):
    """Key j answers every query far above the rest: the queries that see it, and only those, return its value."""
    heads, kv, dim, vdim = 4, 2, 64, 64
    n = 2 * chunk + 70
    for loud in (0, 1, chunk - 1, chunk, chunk + 1, 2 * chunk - 1, 255, 256, n - 2):
        def edit(q, k, v):
            for a, b, c in zip(q, k, v):
                a[:, :, 0] = 8.0
                b *= 0.1
                b[:, :, 0] = 0.0
                if loud < len(b):
                    b[loud, :, 0] = 16.0
                    c[loud] = 3.0
        ends = [e for e in (loud + 1, min(chunk * (loud // chunk + 1), n), min(chunk * (loud // chunk + 1) + 1, n), n) if e > 0]
        batches = [Batch(dev, [(n, n), (n, 70)], seed=loud), Batch(dev, [(e, 1) for e in ends], single=True, seed=loud)]
        for batch in batches:
            got, want = _attention_case(dev, dtype, batch, (heads, kv, dim, vdim), chunk, 0.125, 30.0, edit=edit)
            _close(got, want, _tol(dtype, 1e-2, 1e-5), f"loud key {loud}")
            pos = batch.positions.cpu()[: len(got)]
            sees = (pos >= loud) & (pos // chunk == loud // chunk)
            assert bool(((got.cpu() - 3.0).abs().amax((1, 2)) < 0.1).eq(sees).all()), loud


RET = [  # heads, key size, value size, rotated
    (3, 32, 48, 16), (3, 64, 24, 64), (2, 128, 128, 128), (2, 12, 20, 0), (2, 20, 9, 4), (4, 64, 160, 64), (2, 192, 64, 96), (2, 256, 256, 256)]


@pytest.mark.parametrize("dtype", [BF16, F32])
@pytest.mark.parametrize("shape", RET)
@pytest.mark.parametrize("decays", [(0.9, 0.999), (0.2, 1.0), (0.0, 0.97)])
def test_retention_with_norm_and_gate(dev, dtype, shape, decays):
    heads, dim, vdim, rot = shape
    decay = [decays[h % 2] for h in range(heads)]
    log2 = mixers.Retention(mixers.RetentionSpec(heads, dim, vdim, tuple(decay), Rotary(90.0, rot)), None, RopeTables(1024, dev), 1e-5).log2_decay
    table = RopeTables(1024, dev).get(Rotary(90.0, rot))
    sizes = [heads * dim, heads * dim, heads * vdim, heads * vdim]
    for batch in _batches(dev) + [Batch(dev, [(900, 900), (700, 640)], seed=5)]:
        g = torch.Generator().manual_seed(11)
        full = [_rand(g, n, sum(sizes), dtype=dtype) for n, _ in batch.spans]
        split = [f.double().split(sizes, dim=1) for f in full]
        state = torch.full((batch.num_state_slots, heads, dim, vdim), 1e6)
        want, last = [], []
        for (q, k, v, z), (n, c), slot in zip(split, batch.spans, batch.state_slots):
            q = plain.rotate(q.view(n, heads, dim), 90.0, rot)
            k = plain.rotate(k.view(n, heads, dim), 90.0, rot) * dim ** -0.5
            v = v.view(n, heads, vdim)
            i = torch.arange(n, dtype=torch.float64)
            gamma = torch.tensor(decay, dtype=torch.float64)

            def carried(end):                                # state after the first ``end`` tokens, as a weighted sum
                w = gamma[None] ** (end - 1 - i[:end])[:, None]
                return torch.einsum("th,thd,thv->hdv", w, k[:end], v[:end])
            if n - c > 0:
                state[slot] = carried(n - c).float()
            o = plain.unit_rms(plain.retention(q, k, v, decay), 1e-5).reshape(n, -1)
            want.append(o * z * torch.sigmoid(z))
            last.append(carried(n))
        before, state = state.clone(), state.to(dev)
        rows = batch.rows(full).to(dev)
        out = torch.full((rows.shape[0], heads * vdim), 9.0, dtype=dtype, device=dev)
        mixers.retention(rows, state, batch.group, table, log2, out, rot, dim ** -0.5, 1e-5)
        what = f"{shape} {decays} single {batch.single} spans {batch.spans}"
        # (without any memory o is (q . k) v, and dividing by its size magnifies rounding where q . k is near 0)
        _close(out, batch.rows(want), _tol(dtype, 8e-3, 2e-5 if min(decay) > 0 else 1e-4), what)
        after = state.cpu()
        for s, slot in zip(last, batch.state_slots):         # the state is fp32 whatever the projections are
            _close(after[slot], s, 6e-5, "state " + what)
            before[slot] = after[slot]
        assert torch.equal(after, before), "a slot of no sequence was written"
