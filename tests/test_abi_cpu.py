"""Host-side checks of the C ABI that need no GPU: the library loads, exports every symbol
the header declares, and rejects bad arguments before any launch."""
import ctypes as C
import os
import re

import pytest
import torch

from nanovllm_amd import _lib

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
HEADER = os.path.join(ROOT, "include", "nanovllm_amd.h")


def _declared_symbols():
    text = open(HEADER).read()
    text = re.sub(r"/\*.*?\*/", "", text, flags=re.S)
    return sorted(set(re.findall(r"\b(nva_[a-z_0-9]+)\s*\(", text)))


def test_library_exports_every_declared_symbol():
    lib = _lib.load()
    names = _declared_symbols()
    assert len(names) >= 9
    for n in names:
        assert hasattr(lib, n), f"{n} declared in the header but not exported"
        assert n in _lib.SIGNATURES, f"{n} has no ctypes signature"
    assert sorted(_lib.SIGNATURES) == names


def test_version_and_status_strings():
    lib = _lib.load()
    assert lib.nva_version() >= 1
    seen = {_lib.status_string(c) for c in range(10)}
    assert len(seen) == 10 and _lib.status_string(0) == "ok"
    assert _lib.status_string(1234) == "unknown status"


def test_device_count_reports_no_device_cleanly():
    lib = _lib.load()
    n = C.c_int(-1)
    rc = lib.nva_device_count(C.byref(n))
    if torch.cuda.is_available():
        assert rc == _lib.OK and n.value >= 1
    else:
        assert rc == _lib.ERR_NO_DEVICE and n.value == 0
    assert lib.nva_device_count(None) == _lib.ERR_NULL_POINTER


A = 0x1000   # a fake, 16-byte aligned address: validation fails before anything dereferences it


def test_store_kvcache_validation():
    f = _lib.load().nva_store_kvcache
    assert f(None, 1024, A, 1024, A, A, A, 4, 8, 128, 512, None) == _lib.ERR_NULL_POINTER
    assert f(A, 1024, A, 1024, A, A, None, 4, 8, 128, 512, None) == _lib.ERR_NULL_POINTER
    assert f(A, 1024, A, 1024, A, A, A, -1, 8, 128, 512, None) == _lib.ERR_BAD_SHAPE
    assert f(A, 1000, A, 1024, A, A, A, 4, 8, 128, 512, None) == _lib.ERR_BAD_STRIDE     # stride < row
    assert f(A, 1024, A, 4100, A, A, A, 4, 8, 128, 512, None) == _lib.ERR_BAD_STRIDE     # not 16-byte rows
    assert f(A + 2, 1024, A, 1024, A, A, A, 4, 8, 128, 512, None) == _lib.ERR_MISALIGNED
    assert f(A, 1024, A, 1024, A, A, A, 4, 8, 100, 512, None) == _lib.ERR_UNSUPPORTED_GEOMETRY
    assert f(None, 0, None, 0, None, None, None, 0, 8, 128, 512, None) == _lib.OK        # empty batch


def test_decode_validation_and_workspace_size():
    lib = _lib.load()
    ws = lib.nva_paged_decode_workspace_bytes
    # prefix sums and context lengths (each 256-byte aligned) + a 32-byte record per worker + 8 bytes per
    # (sequence, head) pair (256-byte aligned) + (2048 wavefronts * min(heads, 8) + 4 * batch * heads) partial rows of 130 floats
    assert ws(64, 16, 128, 8) == 512 + 256 + 2048 * 32 + 64 * 16 * 8 + (2048 * 8 + 4 * 64 * 16) * 130 * 4
    assert ws(3, 2, 128, 1) == 256 + 256 + 2048 * 32 + 256 + (2048 * 2 + 4 * 3 * 2) * 130 * 4
    assert ws(0, 16, 128, 8) == 0
    f = lib.nva_paged_decode_attn
    ok = dict(q=A, qs=2048, kc=A, vc=A, bt=A, bts=8, mb=8, cl=A, out=A, ws=A, wsb=ws(4, 16, 128, 8),
              b=4, hq=16, hkv=8, dh=128, bs=256, nb=64, scale=0.088, stream=None)

    def call(**kw):
        a = dict(ok, **kw)
        return f(a["q"], a["qs"], a["kc"], a["vc"], a["bt"], a["bts"], a["mb"], a["cl"], a["out"], a["ws"],
                 a["wsb"], a["b"], a["hq"], a["hkv"], a["dh"], a["bs"], a["nb"], a["scale"], a["stream"])

    assert call(q=None) == _lib.ERR_NULL_POINTER
    assert call(bt=None) == _lib.ERR_NULL_POINTER
    assert call(dh=64) == _lib.ERR_UNSUPPORTED_GEOMETRY
    assert call(bs=128) == _lib.ERR_UNSUPPORTED_GEOMETRY
    assert call(bs=768) == _lib.ERR_UNSUPPORTED_GEOMETRY             # blocks of 256 * 2^k tokens only
    assert call(hq=72, hkv=8) == _lib.ERR_UNSUPPORTED_GEOMETRY        # group 9 (1 to 8 are built)
    assert call(hq=16, hkv=3) == _lib.ERR_UNSUPPORTED_GEOMETRY
    assert call(qs=1024) == _lib.ERR_BAD_STRIDE
    assert call(bts=4) == _lib.ERR_BAD_STRIDE
    assert call(ws=A + 4) == _lib.ERR_MISALIGNED
    assert call(wsb=ok["wsb"] - 1) == _lib.ERR_WORKSPACE_TOO_SMALL
    assert call(b=-2) == _lib.ERR_BAD_SHAPE
    assert call(b=0) == _lib.OK
    g = lib.nva_paged_decode_attn_planned
    a = ok
    args = [a["q"], a["qs"], a["kc"], a["vc"], a["bt"], a["bts"], a["mb"], a["cl"], a["out"], a["ws"], a["wsb"],
            a["b"], a["hq"], a["hkv"], a["dh"], a["bs"], a["nb"], a["scale"]]
    assert g(*args, 2, None) == _lib.ERR_BAD_SHAPE                    # neither build nor reuse
    assert g(*(args[:11] + [0] + args[12:]), 1, None) == _lib.OK      # empty batch
    assert g(*(args[:9] + [A + 4] + args[10:]), 1, None) == _lib.ERR_MISALIGNED


def test_prefill_validation():
    f = _lib.load().nva_varlen_prefill_attn
    ok = dict(q=A, qs=2048, k=A, ks=1024, v=A, vs=4096, kc=None, vc=None, bt=None, bts=0, mb=0, cq=A, ck=A,
              b=2, mq=100, mk=100, out=A, hq=16, hkv=8, dh=128, bs=256, nb=0, scale=0.088, stream=None)

    def call(**kw):
        a = dict(ok, **kw)
        return f(a["q"], a["qs"], a["k"], a["ks"], a["v"], a["vs"], a["kc"], a["vc"], a["bt"], a["bts"], a["mb"],
                 a["cq"], a["ck"], a["b"], a["mq"], a["mk"], a["out"], a["hq"], a["hkv"], a["dh"], a["bs"],
                 a["nb"], a["scale"], a["stream"])

    assert call(q=None) == _lib.ERR_NULL_POINTER
    assert call(k=None) == _lib.ERR_NULL_POINTER                       # packed mode needs k/v
    assert call(cq=None) == _lib.ERR_NULL_POINTER
    assert call(dh=256) == _lib.ERR_UNSUPPORTED_GEOMETRY
    assert call(vs=1000) == _lib.ERR_BAD_STRIDE
    assert call(out=A + 8) == _lib.ERR_MISALIGNED
    paged = dict(k=None, v=None, kc=A, vc=A, bt=A, bts=4, mb=4, nb=32)
    assert call(**dict(paged, kc=None)) == _lib.ERR_NULL_POINTER
    assert call(**dict(paged, bs=768)) == _lib.ERR_UNSUPPORTED_GEOMETRY   # blocks of 256 * 2^k tokens only
    assert call(**dict(paged, bts=2)) == _lib.ERR_BAD_STRIDE
    assert call(**dict(paged, mk=4 * 256 + 1)) == _lib.ERR_BAD_SHAPE   # table too narrow for max_seqlen_k
    assert call(b=0) == _lib.OK and call(mq=0) == _lib.OK


def test_sampler_validation_and_workspace_size():
    lib = _lib.load()
    ws = lib.nva_sample_workspace_bytes
    assert ws(256, 151936) == 256 * 75 * 16 and ws(1, 1) == 16 and ws(2, 2049) == 64 and ws(0, 10) == 0   # one 16-byte record per 2048-column chunk
    f = lib.nva_sample
    assert f(None, 100, A, None, 0, 0, 0, A, A, 1 << 20, 4, 100, None) == _lib.ERR_NULL_POINTER
    assert f(A, 100, A, None, 0, 0, 0, A, None, 1 << 20, 4, 100, None) == _lib.ERR_NULL_POINTER
    assert f(A, 99, A, None, 0, 0, 0, A, A, 1 << 20, 4, 100, None) == _lib.ERR_BAD_STRIDE
    assert f(A, 100, A, A, 50, 0, 0, A, A, 1 << 20, 4, 100, None) == _lib.ERR_BAD_STRIDE
    assert f(A, 100, A, None, 0, 0, 0, A, A, 8, 4, 100, None) == _lib.ERR_WORKSPACE_TOO_SMALL
    assert f(A, 100, A, None, 0, 0, 0, A, A, 1 << 20, 4, 0, None) == _lib.ERR_BAD_SHAPE
    assert f(A, 100, A, None, 0, 0, 0, A, A, 1 << 20, 0, 100, None) == _lib.OK


def test_gather_last_rms_norm_validation():
    f = _lib.load().nva_gather_last_rms_norm
    assert f(None, 1024, A, 1024, A, A, A, 4, 100, 1024, 1e-6, None) == _lib.ERR_NULL_POINTER
    assert f(A, 1024, A, 1024, None, A, A, 4, 100, 1024, 1e-6, None) == _lib.ERR_NULL_POINTER    # cu_seqlens_q
    assert f(A, 1024, A, 1024, A, A, None, 4, 100, 1024, 1e-6, None) == _lib.ERR_NULL_POINTER    # out
    assert f(A, 1024, A, 1024, A, A, A, -1, 100, 1024, 1e-6, None) == _lib.ERR_BAD_SHAPE
    assert f(A, 1024, A, 1024, A, A, A, 4, 0, 1024, 1e-6, None) == _lib.ERR_BAD_SHAPE            # rows to pick from nothing
    assert f(A, 1000, A, 1024, A, A, A, 4, 100, 1024, 1e-6, None) == _lib.ERR_BAD_STRIDE
    assert f(A, 1024, A, 1028, A, A, A, 4, 100, 1024, 1e-6, None) == _lib.ERR_BAD_STRIDE
    assert f(A + 4, 1024, A, 1024, A, A, A, 4, 100, 1024, 1e-6, None) == _lib.ERR_MISALIGNED
    assert f(A, 1024, A, 1024, A, A, A, 4, 100, 1020, 1e-6, None) == _lib.ERR_UNSUPPORTED_GEOMETRY
    assert f(A, 8192, A, 8192, A, A, A, 4, 100, 8192, 1e-6, None) == _lib.ERR_UNSUPPORTED_GEOMETRY
    assert f(None, 0, None, 0, None, None, None, 0, 0, 1024, 1e-6, None) == _lib.OK               # empty batch


def test_stage_decode_inputs_validation():
    f = _lib.load().nva_stage_decode_inputs
    # (dst, src_host, nbytes, ids_offset, index_offset, n, prev_tokens, n_prev, stream)
    assert f(None, A, 4096, 0, 2048, 16, None, 0, None) == _lib.ERR_NULL_POINTER
    assert f(A, A, 4096, 0, 2048, 16, None, 4, None) == _lib.ERR_NULL_POINTER               # tokens announced, none given
    assert f(A, A, 4100, 0, 2048, 16, None, 0, None) == _lib.ERR_MISALIGNED                 # whole 16-byte chunks only
    assert f(A, A, 4096, 8, 2048, 16, None, 0, None) == _lib.ERR_MISALIGNED
    assert f(A + 8, A, 4096, 0, 2048, 16, None, 0, None) == _lib.ERR_MISALIGNED
    assert f(A, A, 4096, 0, 2048, 1024, None, 0, None) == _lib.ERR_BAD_SHAPE                # ids run past the buffer
    assert f(A, A, 4096, 0, 4090, 16, None, 0, None) == _lib.ERR_MISALIGNED
    assert f(A, A, 4096, 0, 4092, 16, None, 0, None) == _lib.ERR_BAD_SHAPE                  # index runs past the buffer
    assert f(A, A, -16, 0, 0, 0, None, 0, None) == _lib.ERR_BAD_SHAPE
    assert f(None, None, 0, 0, 0, 0, None, 0, None) == _lib.OK                              # nothing to move


def test_python_wrappers_refuse_cpu_tensors_and_keep_reference_asserts():
    import nanovllm_amd as nva
    k = torch.zeros(4, 8, 128, dtype=torch.bfloat16)
    cache = torch.zeros(2, 256, 8, 128, dtype=torch.bfloat16)
    slots = torch.arange(4, dtype=torch.int32)
    with pytest.raises(RuntimeError, match="GPU only"):
        nva.store_kvcache(k, k, cache, cache, slots)
    with pytest.raises(AssertionError):                                # slot_mapping.numel() == N
        nva.store_kvcache(k, k, cache, cache, slots[:3])
    with pytest.raises(AssertionError):                                # stride(1) == head_dim
        nva.store_kvcache(k.transpose(1, 2).contiguous().transpose(1, 2), k, cache, cache, slots)
    with pytest.raises(RuntimeError, match="GPU only"):
        nva.sample(torch.zeros(2, 10, dtype=torch.bfloat16), torch.ones(2))


def test_missing_library_fails_loudly(monkeypatch):
    monkeypatch.setattr(_lib, "_lib", None)
    monkeypatch.setattr(_lib, "LIB_PATH", "/nonexistent/libnanovllm_amd.so")
    with pytest.raises(_lib.HipLibraryMissing, match="no CPU fallback"):
        _lib.load()
    fresh = _lib._Symbols()                                            # the mixers' library alone serves its own and the common symbols
    assert fresh.nva_version() >= 1 and fresh.nva_retention_workspace_bytes(0, 0, 1, 8, 8, 0, 0) == 0
    with pytest.raises(_lib.HipLibraryMissing, match="no CPU fallback"):
        fresh.nva_rms_norm
    monkeypatch.setattr(_lib, "MIXERS_LIB_PATH", "/nonexistent/libnanovllm_mixers.so")
    with pytest.raises(_lib.HipLibraryMissing, match="no CPU fallback"):
        _lib.load_mixers()


def test_sample_static_validation():
    """The allocation-free sampler rejects bad arguments and problems beyond its built-in scratch
    array before it touches a device."""
    f = _lib.load().nva_sample_static
    # (logits, row_stride, temperatures, noise, noise_stride, seed, offset, out_tokens, batch, vocab, stream)
    assert f(None, 100, A, None, 0, 0, 0, A, 4, 100, None) == _lib.ERR_NULL_POINTER
    assert f(A, 99, A, None, 0, 0, 0, A, 4, 100, None) == _lib.ERR_BAD_STRIDE
    assert f(A, 100, A, None, 0, 0, 0, A, 4, 0, None) == _lib.ERR_BAD_SHAPE
    assert f(A, 100, A, None, 0, 0, 0, A, 0, 100, None) == _lib.OK
    assert f(A, 151936, A, None, 0, 0, 0, A, 1748, 151936, None) == _lib.ERR_SCRATCH_TOO_SMALL    # 1748 * 75 records > 131072
    assert f(A, 1 << 29, A, None, 0, 0, 0, A, 1, 1 << 29, None) == _lib.ERR_SCRATCH_TOO_SMALL     # 262144 records


def test_probe_validation():
    """The calibration read rejects bad arguments before any launch."""
    f = _lib.load().nva_probe_stream_read
    # (src, nbytes, sink, stream)
    assert f(None, 1024, A, None) == _lib.ERR_NULL_POINTER
    assert f(A, 1024, None, None) == _lib.ERR_NULL_POINTER
    assert f(A + 8, 1024, A, None) == _lib.ERR_MISALIGNED
    assert f(A, 1000, A, None) == _lib.ERR_MISALIGNED               # not a multiple of 16
    assert f(A, -16, A, None) == _lib.ERR_BAD_SHAPE
    assert f(A, 0, A, None) == _lib.OK                               # nothing to read


def _with(ok, f, **kw):
    """Calls ``f`` with the values of ``ok`` (in order), some of them replaced."""
    assert not set(kw) - set(ok), set(kw) - set(ok)
    return f(*dict(ok, **kw).values())


def test_norms_and_gate_of_layered_models_validation():
    lib = _lib.load()
    ok = dict(ids=A, table=A, scale=1.0, w=A, b=A, res=A, out=A, rows=4, width=64, vocab=10, eps=1e-5, dtype=0, stream=None)
    for kw, rc in ((dict(ids=None), _lib.ERR_NULL_POINTER), (dict(res=None), _lib.ERR_NULL_POINTER), (dict(width=0), _lib.ERR_BAD_SHAPE),
                   (dict(vocab=0), _lib.ERR_BAD_SHAPE), (dict(dtype=2), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(rows=0, ids=None), _lib.OK)):
        assert _with(ok, lib.nva_embed_norm, **kw) == rc, kw
    ok = dict(y=A, ys=64, res=A, pw=A, pb=A, nw=A, nb=A, out=A, rows_of=None, rows=4, src=4, width=64, eps=1e-5, dtype=1, stream=None)
    for kw, rc in ((dict(y=None), _lib.ERR_NULL_POINTER), (dict(nb=None), _lib.ERR_NULL_POINTER), (dict(ys=63), _lib.ERR_BAD_STRIDE),
                   (dict(rows=3), _lib.ERR_BAD_SHAPE), (dict(rows_of=A, src=0), _lib.ERR_BAD_SHAPE), (dict(rows=0, src=0), _lib.OK),
                   (dict(dtype=-1), _lib.ERR_UNSUPPORTED_GEOMETRY)):
        assert _with(ok, lib.nva_post_add_norm, **kw) == rc, kw
    ok = dict(x=A, xs=128, out=A, rows=4, inter=64, limit=1.0, alpha=1.7, cubic=0.0, shift=1.0, dtype=0, stream=None)
    for kw, rc in ((dict(x=None), _lib.ERR_NULL_POINTER), (dict(xs=127), _lib.ERR_BAD_STRIDE), (dict(inter=0), _lib.ERR_BAD_SHAPE),
                   (dict(rows=-1), _lib.ERR_BAD_SHAPE), (dict(rows=0, x=None), _lib.OK)):
        assert _with(ok, lib.nva_clamped_gate, **kw) == rc, kw


def test_conv_rope_store_validation():
    f = _lib.load().nva_conv_rope_store
    ok = dict(qkv=A, stride=192, w=A, state=A, slots=A, cu=A, lens=A, tseq=A, rope=A, q=A, kc=A, vc=A, sm=A, num_slots=512, n=9, seqs=2,
              heads=4, kv=1, dim=32, vdim=32, rot=32, taps=4, max_pos=64, state_slots=4, dtype=0, stream=None)
    for kw, rc in ((dict(qkv=None), _lib.ERR_NULL_POINTER), (dict(state=None), _lib.ERR_NULL_POINTER), (dict(slots=None), _lib.ERR_NULL_POINTER),
                   (dict(tseq=None), _lib.ERR_NULL_POINTER), (dict(rope=None), _lib.ERR_NULL_POINTER), (dict(vc=None), _lib.ERR_NULL_POINTER),
                   (dict(stride=191), _lib.ERR_BAD_STRIDE), (dict(rot=34), _lib.ERR_BAD_SHAPE), (dict(rot=31), _lib.ERR_UNSUPPORTED_GEOMETRY),
                   (dict(taps=17), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(taps=0), _lib.ERR_BAD_SHAPE), (dict(cu=None), _lib.ERR_BAD_SHAPE),
                   (dict(dtype=7), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(n=0, qkv=None), _lib.OK)):
        assert _with(ok, f, **kw) == rc, kw


def test_chunk_attention_validation_and_workspace():
    lib = _lib.load()
    ws = lib.nva_chunk_attn_workspace_bytes
    assert ws(8, 16, 8, 128, 2, 256, 400) == 0                       # one range of keys holds them all
    assert ws(8, 16, 8, 128, 16, 256, 1 << 20) == 8 * 9 * 16 * 130 * 4   # 4096 keys and up to 31 before a multiple of 32, ranges of 512
    assert ws(0, 16, 8, 128, 16, 256, 100) == 0
    ok = dict(q=A, qs=2048, kc=A, vc=A, bt=A, bts=16, mb=16, cu=None, lens=A, tseq=None, out=A, ws=A, wsb=1 << 30, n=8, seqs=8, mq=1,
              heads=16, kv=8, dim=128, vdim=128, bs=256, nb=64, chunk=8192, scale=0.1, cap=30.0, dtype=0, stream=None)
    for kw, rc in ((dict(q=None), _lib.ERR_NULL_POINTER), (dict(ws=None), _lib.ERR_NULL_POINTER), (dict(ws=A + 8), _lib.ERR_MISALIGNED),
                   (dict(wsb=100), _lib.ERR_WORKSPACE_TOO_SMALL), (dict(heads=12), _lib.ERR_BAD_SHAPE), (dict(chunk=0), _lib.ERR_BAD_SHAPE),
                   (dict(bs=64), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(dim=520), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(qs=2047), _lib.ERR_BAD_STRIDE),
                   (dict(bts=15), _lib.ERR_BAD_STRIDE), (dict(cu=A), _lib.ERR_NULL_POINTER), (dict(seqs=7), _lib.ERR_BAD_SHAPE),
                   (dict(dtype=3), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(n=0, q=None), _lib.OK)):
        assert _with(ok, lib.nva_chunk_attn, **kw) == rc, kw


def test_retention_validation_and_workspace():
    lib = _lib.load()
    ws = lib.nva_retention_workspace_bytes
    assert ws(1, 200, 8, 128, 128, 128, 0) == 0 and ws(600, 4096, 8, 128, 128, 128, 0) == 0       # short, or enough sequences
    assert ws(1, 4096, 8, 128, 128, 128, 0) == 16 * 8 * 128 * 128 * 4                             # segments of 256 tokens
    assert ws(1, 4096, 8, 128, 128, 128, 1) == 0 and ws(1, 4096, 8, 100, 128, 0, 0) == 0          # sizes that walk token by token
    ok = dict(x=A, xs=4096, state=A, slots=A, cu=A, lens=A, rope=A, decay=A, out=A, ws=A, wsb=1 << 30, n=4096, seqs=1, mq=4096, heads=8,
              dim=128, vdim=128, rot=128, max_pos=64, state_slots=4, ks=0.1, eps=1e-6, dtype=0, stream=None)
    for kw, rc in ((dict(x=None), _lib.ERR_NULL_POINTER), (dict(state=None), _lib.ERR_NULL_POINTER), (dict(rope=None), _lib.ERR_NULL_POINTER),
                   (dict(decay=None), _lib.ERR_NULL_POINTER), (dict(ws=None), _lib.ERR_NULL_POINTER), (dict(ws=A + 4), _lib.ERR_MISALIGNED),
                   (dict(wsb=1000), _lib.ERR_WORKSPACE_TOO_SMALL), (dict(xs=4095), _lib.ERR_BAD_STRIDE), (dict(rot=130), _lib.ERR_BAD_SHAPE),
                   (dict(rot=127), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(dim=1024, xs=1 << 20), _lib.ERR_UNSUPPORTED_GEOMETRY),
                   (dict(cu=None), _lib.ERR_BAD_SHAPE), (dict(n=0, x=None), _lib.OK)):
        assert _with(ok, lib.nva_retention, **kw) == rc, kw


def test_branches_and_experts_validation():
    lib = _lib.load()
    ok = dict(ids=A, table=A, scale=1.0, w1=A, w2=A, off=1.0, res=A, o1=A, o1s=64, o2=A, copy=A, cs=128, clear=None, nclear=0, rows=4, width=64, vocab=10, eps=1e-5, dtype=0, stream=None)
    for kw, rc in ((dict(ids=None), _lib.ERR_NULL_POINTER), (dict(o2=None), _lib.ERR_NULL_POINTER), (dict(width=0), _lib.ERR_BAD_SHAPE),
                   (dict(nclear=-1), _lib.ERR_BAD_SHAPE), (dict(o1s=63), _lib.ERR_BAD_STRIDE), (dict(cs=63), _lib.ERR_BAD_STRIDE),
                   (dict(dtype=2), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(rows=0, ids=None), _lib.OK)):
        assert _with(ok, lib.nva_embed_rms_norms, **kw) == rc, kw
    ok = dict(y1=A, ys=64, y2=A, terms=2, gate=A, gs=128, gb=A, res=A, w=A, off=0.0, out=A, os=64, rows_of=None, clear=None, nclear=0, rows=4, src=4, width=64,
              eps=1e-5, dtype=0, stream=None)
    for kw, rc in ((dict(y1=None), _lib.ERR_NULL_POINTER), (dict(gate=None), _lib.ERR_NULL_POINTER), (dict(gb=None), _lib.ERR_NULL_POINTER),
                   (dict(out=None), _lib.ERR_NULL_POINTER), (dict(ys=63), _lib.ERR_BAD_STRIDE), (dict(gs=127), _lib.ERR_BAD_STRIDE),
                   (dict(y2=None, gs=63), _lib.ERR_BAD_STRIDE), (dict(os=63), _lib.ERR_BAD_STRIDE), (dict(terms=0), _lib.ERR_BAD_SHAPE),
                   (dict(rows=3), _lib.ERR_BAD_SHAPE), (dict(rows_of=A, src=0), _lib.ERR_BAD_SHAPE), (dict(dtype=2), _lib.ERR_UNSUPPORTED_GEOMETRY),
                   (dict(rows=0, src=0), _lib.OK)):
        assert _with(ok, lib.nva_gated_rms_norm, **kw) == rc, kw
    ok = dict(p=A, step=A, res=A, w=A, off=0.0, out=A, clear=None, nclear=0, rows=4, width=64, eps=1e-5, dtype=0, stream=None)
    for kw, rc in ((dict(p=None), _lib.ERR_NULL_POINTER), (dict(step=None), _lib.ERR_NULL_POINTER), (dict(w=None), _lib.ERR_NULL_POINTER),
                   (dict(width=0), _lib.ERR_BAD_SHAPE), (dict(dtype=2), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(rows=0, p=None), _lib.OK)):
        assert _with(ok, lib.nva_entry_rms_norm, **kw) == rc, kw
    ok = dict(y1=A, ys=64, g1=A, y2=A, tw=A, terms=2, g2=A, mult=1.0, res=A, w1=A, w2=A, off=1.0, o1=A, o2=A, rows_of=None, clear=None, nclear=0,
              rows=4, src=4, width=64, eps=1e-5, dtype=1, stream=None)
    for kw, rc in ((dict(res=None), _lib.ERR_NULL_POINTER), (dict(w1=None), _lib.ERR_NULL_POINTER), (dict(o2=None), _lib.ERR_NULL_POINTER),
                   (dict(ys=63), _lib.ERR_BAD_STRIDE), (dict(terms=0), _lib.ERR_BAD_SHAPE), (dict(rows=3), _lib.ERR_BAD_SHAPE),
                   (dict(rows_of=A, src=0), _lib.ERR_BAD_SHAPE), (dict(rows=0, src=0), _lib.OK), (dict(dtype=-1), _lib.ERR_UNSUPPORTED_GEOMETRY)):
        assert _with(ok, lib.nva_branches_rms_norms, **kw) == rc, kw
    ok = dict(x=A, xs=256, xg=64, w=A, out=A, os=256, og=64, rows=4, groups=4, n_out=64, k=64, relu=0, dtype=0, odt=0, stream=None)
    for kw, rc in ((dict(x=None), _lib.ERR_NULL_POINTER), (dict(w=None), _lib.ERR_NULL_POINTER), (dict(xs=63), _lib.ERR_BAD_STRIDE),
                   (dict(og=63), _lib.ERR_BAD_STRIDE), (dict(k=0), _lib.ERR_BAD_SHAPE), (dict(groups=70000), _lib.ERR_BAD_SHAPE),
                   (dict(dtype=1, odt=0), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(rows=0, x=None), _lib.OK), (dict(groups=0, x=None), _lib.OK)):
        assert _with(ok, lib.nva_grouped_linear, **kw) == rc, kw
    ok = dict(x=A, xs=64, w=A, b=None, choice=A, cw=A, lists=A, counts=A, ls=16, rows=16, width=64, experts=8, gates=0, top=2, score=1, scale=1.0, dtype=0, stream=None)
    for kw, rc in ((dict(counts=None), _lib.ERR_NULL_POINTER), (dict(cw=None), _lib.ERR_NULL_POINTER), (dict(top=9), _lib.ERR_BAD_SHAPE),
                   (dict(ls=15), _lib.ERR_BAD_SHAPE), (dict(xs=63), _lib.ERR_BAD_STRIDE), (dict(experts=1025), _lib.ERR_UNSUPPORTED_GEOMETRY),
                   (dict(experts=512, top=129), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(gates=-1), _lib.ERR_BAD_SHAPE),
                   (dict(gates=65), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(score=2), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(rows=0, x=None), _lib.OK)):
        assert _with(ok, lib.nva_router, **kw) == rc, kw
    ok = dict(x=A, xs=64, w=A, out=A, lists=A, counts=A, ls=16, rows=16, terms=2, experts=8, n_out=32, k=64, per_row=1, gated=1, limit=1.0, slope=1.7, shift=1.0, iw=A, iws=2, dtype=0, stream=None)
    for kw, rc in ((dict(lists=None), _lib.ERR_NULL_POINTER), (dict(out=None), _lib.ERR_NULL_POINTER), (dict(terms=9), _lib.ERR_BAD_SHAPE),
                   (dict(ls=15), _lib.ERR_BAD_SHAPE), (dict(xs=63), _lib.ERR_BAD_STRIDE), (dict(dtype=5), _lib.ERR_UNSUPPORTED_GEOMETRY),
                   (dict(iws=1), _lib.ERR_BAD_STRIDE), (dict(gated=0), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(rows=0, x=None), _lib.OK)):
        assert _with(ok, lib.nva_routed_linear, **kw) == rc, kw
    del ok["dtype"], ok["stream"], ok["iw"], ok["iws"]
    ok.update(sx=A, sxs=64, sw=A, so=A, sn=24, sk=64, sl=1.0, stream=None)
    for kw, rc in ((dict(lists=None), _lib.ERR_NULL_POINTER), (dict(so=None), _lib.ERR_NULL_POINTER), (dict(terms=9), _lib.ERR_BAD_SHAPE),
                   (dict(sn=0), _lib.ERR_BAD_SHAPE), (dict(sxs=63), _lib.ERR_BAD_STRIDE), (dict(sk=60), _lib.ERR_UNSUPPORTED_GEOMETRY),
                   (dict(k=60), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(rows=0, sx=None), _lib.OK)):
        assert _with(ok, lib.nva_routed_shared_linear, **kw) == rc, kw


def test_post_norm_prepare_and_masks_validation():
    lib = _lib.load_masked()
    ok = dict(y1=A, ys=64, yw=A, y2=A, tw=A, ws=3, terms=2, post=A, res=A, nxt=None, off=1.0, out=A, rows_of=None, clear=None, nclear=0, rows=4, src=4,
              width=64, eps=1e-5, dtype=0, stream=None)
    for kw, rc in ((dict(post=None), _lib.ERR_NULL_POINTER), (dict(out=None), _lib.ERR_NULL_POINTER), (dict(y1=None, y2=None), _lib.ERR_NULL_POINTER),
                   (dict(ys=63), _lib.ERR_BAD_STRIDE), (dict(ws=1), _lib.ERR_BAD_STRIDE), (dict(ws=0, tw=None), _lib.ERR_BAD_STRIDE),
                   (dict(terms=0), _lib.ERR_BAD_SHAPE), (dict(rows=3), _lib.ERR_BAD_SHAPE), (dict(dtype=2), _lib.ERR_UNSUPPORTED_GEOMETRY),
                   (dict(rows=0, src=0), _lib.OK)):
        assert _with(ok, lib.nva_post_rms_norms, **kw) == rc, kw
    ok = dict(x=A, xs=256, b=A, qn=A, kn=A, norms=5, rope=A, q=A, kc=A, vc=A, sm=A, slots=512, cu=A, lens=A, tseq=A, n=9, seqs=2, heads=4, kv=2, dim=32,
              vdim=32, rot=16, maxp=64, eps=1e-5, dtype=0, stream=None)
    for kw, rc in ((dict(x=None), _lib.ERR_NULL_POINTER), (dict(vc=None), _lib.ERR_NULL_POINTER), (dict(sm=None), _lib.ERR_NULL_POINTER),
                   (dict(rope=None), _lib.ERR_NULL_POINTER), (dict(tseq=None), _lib.ERR_NULL_POINTER), (dict(xs=255), _lib.ERR_BAD_STRIDE),
                   (dict(rot=15), _lib.ERR_BAD_SHAPE), (dict(rot=34), _lib.ERR_BAD_SHAPE), (dict(maxp=0), _lib.ERR_BAD_SHAPE), (dict(cu=None), _lib.ERR_BAD_SHAPE),
                   (dict(dtype=7), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(heads=5000, kv=1, dim=9, vdim=9, rot=0, xs=1 << 20), _lib.ERR_UNSUPPORTED_GEOMETRY),
                   (dict(norms=8), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(n=0, x=None), _lib.OK)):
        assert _with(ok, lib.nva_qkv_prepare, **kw) == rc, kw
    ok = dict(q=A, qs=2048, kc=A, vc=A, bt=A, bts=16, mb=16, cu=None, lens=A, tseq=None, out=A, ws=A, wsb=1 << 30, n=8, seqs=8, mq=1, heads=16, kv=8,
              dim=128, vdim=128, bs=256, nb=64, mask=1, span=8192, scale=0.1, cap=0.0, sinks=A, slope=A, rate=A, gate=A, gs=16, dtype=0, stream=None)
    for kw, rc in ((dict(q=None), _lib.ERR_NULL_POINTER), (dict(ws=None), _lib.ERR_NULL_POINTER), (dict(mask=2), _lib.ERR_UNSUPPORTED_GEOMETRY),
                   (dict(slope=None), _lib.ERR_NULL_POINTER), (dict(rate=None), _lib.ERR_NULL_POINTER), (dict(cap=1.0), _lib.ERR_UNSUPPORTED_GEOMETRY),
                   (dict(gs=15), _lib.ERR_BAD_STRIDE), (dict(span=0), _lib.ERR_BAD_SHAPE), (dict(wsb=100), _lib.ERR_WORKSPACE_TOO_SMALL),
                   (dict(n=0, q=None), _lib.OK)):
        assert _with(ok, lib.nva_masked_attn, **kw) == rc, kw
    ok = dict(x=A, xs=64, out=A, rows=4, width=64, dtype=0, stream=None)
    for kw, rc in ((dict(x=None), _lib.ERR_NULL_POINTER), (dict(xs=63), _lib.ERR_BAD_STRIDE), (dict(xs=72), _lib.ERR_BAD_STRIDE), (dict(width=0), _lib.ERR_BAD_SHAPE),
                   (dict(dtype=3), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(rows=0, x=None), _lib.OK)):
        assert _with(ok, lib.nva_squared_relu, **kw) == rc, kw
    ok = dict(x=A, rows=4, width=64, cap=30.0, dtype=0, stream=None)
    for kw, rc in ((dict(x=None), _lib.ERR_NULL_POINTER), (dict(cap=0.0), _lib.ERR_BAD_SHAPE), (dict(cap=float("nan")), _lib.ERR_BAD_SHAPE),
                   (dict(dtype=3), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(rows=0, x=None), _lib.OK)):
        assert _with(ok, lib.nva_soft_cap, **kw) == rc, kw


def test_symbols_of_several_libraries_come_from_one_that_is_there(monkeypatch):
    monkeypatch.setattr(_lib, "LATENT_LIB_PATH", "/nonexistent/libnanovllm_latent.so")
    monkeypatch.setattr(_lib, "MIXERS_LIB_PATH", "/nonexistent/libnanovllm_mixers.so")
    fresh = _lib._Symbols()
    assert fresh.nva_chunk_attn_workspace_bytes(0, 16, 8, 128, 16, 256, 100) == 0 and fresh.nva_router is not None
    assert fresh.nva_latent_prefill_supported(128, 64, 128, 0) == 1
    with pytest.raises(_lib.HipLibraryMissing, match="no CPU fallback"):
        fresh.nva_mlstm
    with pytest.raises(_lib.HipLibraryMissing, match="no CPU fallback"):
        fresh.nva_retention


def test_latent_attention_validation_and_workspace():
    lib = _lib.load()
    ok = dict(x=A, xs=400, wq=A, wkv=A, rope=A, q=A, cache=A, sm=A, slots=512, cu=A, lens=A, tseq=A, n=9, seqs=2, q_rank=96, rank=128, rot=32, max_pos=64,
              eps=1e-5, dtype=0, stream=None)
    for kw, rc in ((dict(x=None), _lib.ERR_NULL_POINTER), (dict(wkv=None), _lib.ERR_NULL_POINTER), (dict(rope=None), _lib.ERR_NULL_POINTER),
                   (dict(tseq=None), _lib.ERR_NULL_POINTER), (dict(cu=None), _lib.ERR_BAD_SHAPE), (dict(xs=255), _lib.ERR_BAD_STRIDE),
                   (dict(rot=31), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(rank=0), _lib.ERR_BAD_SHAPE), (dict(q_rank=-1), _lib.ERR_BAD_SHAPE),
                   (dict(q=None), _lib.ERR_NULL_POINTER), (dict(n=0, x=None), _lib.OK)):
        assert _with(ok, lib.nva_latent_prepare, **kw) == rc, kw
    ws = lib.nva_latent_attn_workspace_bytes
    assert ws(2000, 16, 512, 64, 16, 256, 4096, 0) == 0               # enough rows for the machine: one range of keys each
    assert ws(1, 16, 512, 64, 16, 256, 1 << 20, 0) == 33 * 16 * 516 * 4   # 4096 keys and up to 63 before a multiple of 64, ranges of 128
    assert ws(40, 16, 512, 64, 16, 256, 1 << 20, 0) == 40 * 17 * 16 * 516 * 4
    assert ws(1, 16, 512, 64, 16, 256, 60, 0) == 0 and ws(1, 16, 512, 64, 16, 256, 4096, 1) == 0 and ws(1, 16, 516, 64, 16, 256, 4096, 0) == 0
    ok = dict(ql=A, qr=A, qrs=3072, qrh=192, gate=A, gs=16, sinks=A, rope=A, cache=A, bt=A, bts=16, mb=16, cu=None, lens=A, tseq=None, out=A, ws=A, wsb=1 << 30,
              n=8, seqs=8, heads=16, rank=512, rot=64, bs=256, nb=64, window=4096, max_pos=4096, scale=0.1, dtype=0, stream=None)
    for kw, rc in ((dict(ql=None), _lib.ERR_NULL_POINTER), (dict(qr=None), _lib.ERR_NULL_POINTER), (dict(ws=None), _lib.ERR_NULL_POINTER),
                   (dict(ws=A + 8), _lib.ERR_MISALIGNED), (dict(wsb=100), _lib.ERR_WORKSPACE_TOO_SMALL), (dict(window=0), _lib.ERR_BAD_SHAPE),
                   (dict(bs=64), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(rank=1000), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(gs=15), _lib.ERR_BAD_STRIDE),
                   (dict(qrs=2000), _lib.ERR_BAD_STRIDE), (dict(bts=15), _lib.ERR_BAD_STRIDE), (dict(cu=A), _lib.ERR_NULL_POINTER),
                   (dict(seqs=7), _lib.ERR_BAD_SHAPE), (dict(n=0, ql=None), _lib.OK)):
        assert _with(ok, lib.nva_latent_attn, **kw) == rc, kw
    ok = dict(cache=A, bt=A, bts=16, mb=16, kcu=A, lens=A, out=A, keys=90, seqs=2, width=576, bs=256, nb=64, dtype=0, stream=None)
    for kw, rc in ((dict(kcu=None), _lib.ERR_NULL_POINTER), (dict(bts=15), _lib.ERR_BAD_STRIDE), (dict(nb=0), _lib.ERR_BAD_SHAPE),
                   (dict(bs=100), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(keys=0, cache=None), _lib.OK)):
        assert _with(ok, lib.nva_latent_gather, **kw) == rc, kw
    fits = lib.nva_latent_prefill_supported
    assert fits(128, 64, 128, 0) == 1 and fits(128, 64, 128, 1) == 0 and fits(100, 64, 128, 0) == 0 and fits(264, 64, 128, 0) == 0 and fits(8, 136, 8, 0) == 0
    ok = dict(q=A, qs=3072, kv=A, kvs=4096, kr=A, krs=576, gate=A, gs=16, sinks=A, rope=A, cu=A, lens=A, kcu=A, out=A, n=9, seqs=2, mq=7, heads=16, dim=128, rot=64,
              vdim=128, window=100, max_pos=4096, scale=0.1, dtype=0, stream=None)
    for kw, rc in ((dict(q=None), _lib.ERR_NULL_POINTER), (dict(kr=None), _lib.ERR_NULL_POINTER), (dict(kcu=None), _lib.ERR_NULL_POINTER),
                   (dict(kvs=4088), _lib.ERR_BAD_STRIDE), (dict(qs=3076), _lib.ERR_BAD_STRIDE), (dict(kv=A + 2), _lib.ERR_MISALIGNED),
                   (dict(dtype=1), _lib.ERR_UNSUPPORTED_GEOMETRY), (dict(window=0), _lib.ERR_BAD_SHAPE), (dict(n=0, q=None), _lib.OK)):
        assert _with(ok, lib.nva_latent_prefill, **kw) == rc, kw


def test_matrix_memory_validation_and_workspace():
    lib = _lib.load()
    ws = lib.nva_mlstm_workspace_bytes
    assert ws(1, 200, 8, 128, 128, 0) == 0 and ws(600, 4096, 8, 128, 128, 0) == 0                 # short, or enough sequences
    assert ws(1, 4096, 8, 128, 128, 0) == 16 * 8 * (128 * 129 + 4) * 4                            # segments of 256 tokens
    assert ws(1, 4096, 8, 128, 128, 1) == 0 and ws(1, 4096, 8, 100, 128, 0) == 0                  # sizes that walk token by token
    ok = dict(x=A, xs=4096, z=A, bias=A, nw=A, state=A, mass=A, top=A, slots=A, cu=A, lens=A, out=A, ws=A, wsb=1 << 30, n=4096, seqs=1, mq=4096, heads=8,
              dim=128, vdim=128, state_slots=4, qs=0.1, cap=5.0, eps=1e-6, dtype=0, stream=None)
    for kw, rc in ((dict(x=None), _lib.ERR_NULL_POINTER), (dict(z=None), _lib.ERR_NULL_POINTER), (dict(mass=None), _lib.ERR_NULL_POINTER),
                   (dict(ws=None), _lib.ERR_NULL_POINTER), (dict(ws=A + 4), _lib.ERR_MISALIGNED), (dict(wsb=1000), _lib.ERR_WORKSPACE_TOO_SMALL),
                   (dict(xs=4095), _lib.ERR_BAD_STRIDE), (dict(cap=0.0), _lib.ERR_BAD_SHAPE), (dict(dim=1024, xs=1 << 20), _lib.ERR_UNSUPPORTED_GEOMETRY),
                   (dict(cu=None), _lib.ERR_BAD_SHAPE), (dict(n=0, x=None), _lib.OK)):
        assert _with(ok, lib.nva_mlstm, **kw) == rc, kw
