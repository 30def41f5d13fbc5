"""ctypes binding of the C ABI declared in include/nanovllm_amd.h.

Shared libraries are built in-tree, next to this file, by ``csrc/Makefile``: ``libnanovllm_amd.so``
(the attention hot path), ``libnanovllm_mixers.so`` (chunked attention and retention of layered models),
``libnanovllm_latent.so`` (latent attention, matrix memory, routed experts), ``libnanovllm_masked.so``
(attention under masks with sinks and gates, routed experts) and ``libnanovllm_parallel.so`` (attention under masks and
latent attention, routed experts).  Each is opened when one of its symbols is first
used, so a model needs only its own; a kernel that several kinds of model need is in several, and comes from
the first that is there.  There is no fallback: an op whose library is missing raises.
"""
from __future__ import annotations

import ctypes as C
import os

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(_HERE, "libnanovllm_amd.so")
MIXERS_LIB_PATH = os.path.join(_HERE, "libnanovllm_mixers.so")
LATENT_LIB_PATH = os.path.join(_HERE, "libnanovllm_latent.so")
MASKED_LIB_PATH = os.path.join(_HERE, "libnanovllm_masked.so")
PARALLEL_LIB_PATH = os.path.join(_HERE, "libnanovllm_parallel.so")

# status codes of enum nva_status
OK = 0
ERR_NULL_POINTER = 1
ERR_BAD_SHAPE = 2
ERR_UNSUPPORTED_GEOMETRY = 3
ERR_BAD_STRIDE = 4
ERR_MISALIGNED = 5
ERR_WORKSPACE_TOO_SMALL = 6
ERR_LAUNCH_FAILED = 7
ERR_NO_DEVICE = 8
ERR_SCRATCH_TOO_SMALL = 9

# element types of enum nva_dtype
DTYPE_BF16, DTYPE_F32 = 0, 1
# enum nva_mask, nva_qkv_norms, nva_score
MASK_CHUNKS, MASK_WINDOW = 0, 1
QKV_NORM_WHOLE, QKV_NORM_UNIT, QKV_NORM_VALUES = 1, 2, 4
SCORE_SOFTMAX, SCORE_SIGMOID = 0, 1

_vp, _i32, _i64, _u64, _f32, _sz = C.c_void_p, C.c_int32, C.c_int64, C.c_uint64, C.c_float, C.c_size_t

# name -> (restype, argtypes); must list every symbol the header declares
SIGNATURES = {
    "nva_version": (C.c_int, []),
    "nva_status_string": (C.c_char_p, [C.c_int]),
    "nva_device_count": (C.c_int, [C.POINTER(C.c_int)]),
    "nva_store_kvcache": (C.c_int, [_vp, _i64, _vp, _i64, _vp, _vp, _vp, _i32, _i32, _i32, _i64, _vp]),
    "nva_paged_decode_workspace_bytes": (_sz, [_i32, _i32, _i32, _i32]),
    "nva_paged_decode_attn": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _i32, _i32, _vp, _vp, _vp, _sz,
                                        _i32, _i32, _i32, _i32, _i32, _i32, _f32, _vp]),
    "nva_paged_decode_attn_planned": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _i32, _i32, _vp, _vp, _vp, _sz,
                                                _i32, _i32, _i32, _i32, _i32, _i32, _f32, _i32, _vp]),
    "nva_varlen_prefill_attn": (C.c_int, [_vp, _i64, _vp, _i64, _vp, _i64, _vp, _vp, _vp, _i32, _i32,
                                          _vp, _vp, _i32, _i32, _i32, _vp, _i32, _i32, _i32, _i32, _i32,
                                          _f32, _vp]),
    "nva_sample_workspace_bytes": (_sz, [_i32, _i32]),
    "nva_rms_norm": (C.c_int, [_vp, _i64, _vp, _i64, _vp, _vp, _vp, _i32, _i32, _f32, _vp]),
    "nva_gather_last_rms_norm": (C.c_int, [_vp, _i64, _vp, _i64, _vp, _vp, _vp, _i32, _i32, _i32, _f32, _vp]),
    "nva_qk_norm_rope": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _vp, _i32, _vp, _vp, _vp, _vp, _vp, _i64,
                                   _i32, _i32, _i32, _i32, _f32, _vp]),
    "nva_silu_and_mul": (C.c_int, [_vp, _i64, _vp, _i32, _i32, _vp]),
    "nva_stage_decode_inputs": (C.c_int, [_vp, _vp, _i64, _i64, _i64, _i32, _vp, _i32, _vp]),
    "nva_sample": (C.c_int, [_vp, _i64, _vp, _vp, _i64, _u64, _u64, _vp, _vp, _sz, _i32, _i32, _vp]),
    "nva_sample_static": (C.c_int, [_vp, _i64, _vp, _vp, _i64, _u64, _u64, _vp, _i32, _i32, _vp]),
    "nva_embed_norm": (C.c_int, [_vp, _vp, _f32, _vp, _vp, _vp, _vp, _i32, _i32, _i32, _f32, _i32, _vp]),
    "nva_post_add_norm": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _i32, _i32, _i32, _f32, _i32, _vp]),
    "nva_clamped_gate": (C.c_int, [_vp, _i64, _vp, _i32, _i32, _f32, _f32, _f32, _f32, _i32, _vp]),
    "nva_conv_rope_store": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp,
                                      _i64, _i32, _i32, _i32, _i32, _i32, _i32, _i32, _i32, _i32, _i32, _i32, _vp]),
    "nva_chunk_attn_workspace_bytes": (_sz, [_i32, _i32, _i32, _i32, _i32, _i32, _i32]),
    "nva_chunk_attn": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _i64, _i32, _vp, _vp, _vp, _vp, _vp, _sz, _i32, _i32, _i32, _i32,
                                 _i32, _i32, _i32, _i32, _i32, _i32, _f32, _f32, _i32, _vp]),
    "nva_masked_attn": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _i64, _i32, _vp, _vp, _vp, _vp, _vp, _sz, _i32, _i32, _i32, _i32,
                                  _i32, _i32, _i32, _i32, _i32, _i32, _i32, _f32, _f32, _vp, _vp, _vp, _vp, _i64, _i32, _vp]),
    "nva_qkv_prepare": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _i32, _vp, _vp, _vp, _vp, _vp, _i64, _vp, _vp, _vp, _i32, _i32, _i32,
                                  _i32, _i32, _i32, _i32, _i32, _f32, _i32, _vp]),
    "nva_squared_relu": (C.c_int, [_vp, _i64, _vp, _i32, _i32, _i32, _vp]),
    "nva_soft_cap": (C.c_int, [_vp, _i32, _i32, _f32, _i32, _vp]),
    "nva_retention_workspace_bytes": (_sz, [_i32, _i32, _i32, _i32, _i32, _i32, _i32]),
    "nva_retention": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _sz, _i32, _i32, _i32, _i32, _i32,
                                _i32, _i32, _i32, _i32, _f32, _f32, _i32, _vp]),
    "nva_embed_rms_norms": (C.c_int, [_vp, _vp, _f32, _vp, _vp, _f32, _vp, _vp, _i64, _vp, _vp, _i64, _vp, _i32, _i32, _i32, _i32, _f32, _i32,
                                      _vp]),
    "nva_gated_rms_norm": (C.c_int, [_vp, _i64, _vp, _i32, _vp, _i64, _vp, _vp, _vp, _f32, _vp, _i64, _vp, _vp, _i32, _i32, _i32, _i32, _f32, _i32,
                                     _vp]),
    "nva_entry_rms_norm": (C.c_int, [_vp, _vp, _vp, _vp, _f32, _vp, _vp, _i32, _i32, _i32, _f32, _i32, _vp]),
    "nva_branches_rms_norms": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _i32, _vp, _f32, _vp, _vp, _vp, _f32, _vp, _vp, _vp, _vp, _i32,
                                         _i32, _i32, _i32, _f32, _i32, _vp]),
    "nva_grouped_linear": (C.c_int, [_vp, _i64, _i64, _vp, _vp, _i64, _i64, _i32, _i32, _i32, _i32, _i32, _i32, _i32, _vp]),
    "nva_router": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _vp, _vp, _vp, _i64, _i32, _i32, _i32, _i32, _i32, _i32, _f32, _i32, _vp]),
    "nva_routed_linear": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _vp, _i64, _i32, _i32, _i32, _i32, _i32, _i32, _i32, _f32, _f32, _f32, _vp, _i64,
                                    _i32, _vp]),
    "nva_routed_shared_linear": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _vp, _i64, _i32, _i32, _i32, _i32, _i32, _i32, _i32, _f32, _f32, _f32,
                                           _vp, _i64, _vp, _vp, _i32, _i32, _f32, _vp]),
    "nva_post_rms_norms": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _i64, _i32, _vp, _vp, _vp, _f32, _vp, _vp, _vp, _i32, _i32, _i32, _i32,
                                     _f32, _i32, _vp]),
    "nva_latent_prepare": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _vp, _vp, _vp, _i64, _vp, _vp, _vp, _i32, _i32, _i32, _i32, _i32,
                                     _i32, _f32, _i32, _vp]),
    "nva_latent_attn_workspace_bytes": (_sz, [_i32] * 8),
    "nva_latent_attn": (C.c_int, [_vp, _vp, _i64, _i64, _vp, _i64, _vp, _vp, _vp, _vp, _i64, _i32, _vp, _vp, _vp, _vp, _vp, _sz,
                                  _i32, _i32, _i32, _i32, _i32, _i32, _i32, _i32, _i32, _f32, _i32, _vp]),
    "nva_latent_gather": (C.c_int, [_vp, _vp, _i64, _i32, _vp, _vp, _vp, _i32, _i32, _i32, _i32, _i32, _i32, _vp]),
    "nva_latent_prefill_supported": (C.c_int, [_i32, _i32, _i32, _i32]),
    "nva_latent_prefill": (C.c_int, [_vp, _i64, _vp, _i64, _vp, _i64, _vp, _i64, _vp, _vp, _vp, _vp, _vp, _vp, _i32, _i32, _i32, _i32,
                                     _i32, _i32, _i32, _i32, _i32, _f32, _i32, _vp]),
    "nva_mlstm_workspace_bytes": (_sz, [_i32] * 6),
    "nva_mlstm": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _sz, _i32, _i32, _i32, _i32, _i32,
                            _i32, _i32, _f32, _f32, _f32, _i32, _vp]),
    "nva_probe_stream_read": (C.c_int, [_vp, _i64, _vp, _vp]),
}

# which libraries of layered models hold a symbol; the common ones are in every library, all others in libnanovllm_amd.so
_NORM_SYMBOLS = {"nva_embed_rms_norms", "nva_branches_rms_norms", "nva_post_rms_norms", "nva_gated_rms_norm", "nva_entry_rms_norm"}
_EXPERT_SYMBOLS = {"nva_grouped_linear", "nva_router", "nva_routed_linear", "nva_routed_shared_linear"}
_ACTIVATION_SYMBOLS = {"nva_clamped_gate", "nva_squared_relu", "nva_soft_cap"}
_ATTN_SYMBOLS = {"nva_chunk_attn", "nva_chunk_attn_workspace_bytes", "nva_masked_attn"}
MIXER_SYMBOLS = {"nva_embed_norm", "nva_post_add_norm", "nva_conv_rope_store", "nva_retention",
                 "nva_retention_workspace_bytes"} | _ATTN_SYMBOLS | _ACTIVATION_SYMBOLS
_LATENT_ATTN_SYMBOLS = {"nva_latent_prepare", "nva_latent_attn", "nva_latent_attn_workspace_bytes", "nva_latent_gather",
                        "nva_latent_prefill", "nva_latent_prefill_supported"}
LATENT_SYMBOLS = {"nva_mlstm", "nva_mlstm_workspace_bytes"} | _LATENT_ATTN_SYMBOLS | _NORM_SYMBOLS | _EXPERT_SYMBOLS
MASKED_SYMBOLS = {"nva_qkv_prepare"} | _ATTN_SYMBOLS | _ACTIVATION_SYMBOLS | _NORM_SYMBOLS | _EXPERT_SYMBOLS
PARALLEL_SYMBOLS = MASKED_SYMBOLS | _LATENT_ATTN_SYMBOLS
COMMON_SYMBOLS = {"nva_version", "nva_status_string", "nva_device_count", "nva_stage_decode_inputs"}


class HipLibraryMissing(RuntimeError):
    pass


class _Symbols:
    """The entry points as attributes, bound (with their signatures) on first use."""

    def __init__(self):
        self._opened = {}

    def __getattr__(self, name: str):
        if name not in SIGNATURES:
            raise AttributeError(name)
        layered = ((MIXER_SYMBOLS, MIXERS_LIB_PATH), (LATENT_SYMBOLS, LATENT_LIB_PATH), (MASKED_SYMBOLS, MASKED_LIB_PATH),
                   (PARALLEL_SYMBOLS, PARALLEL_LIB_PATH))
        if name in COMMON_SYMBOLS:
            paths = [LIB_PATH] + [path for _, path in layered]
        else:
            paths = [path for names, path in layered if name in names] or [LIB_PATH]
        path = next((p for p in paths if os.path.exists(p)), None)
        if path is None:
            raise _missing(paths[0])
        if path not in self._opened:
            self._opened[path] = C.CDLL(path)
        fn = getattr(self._opened[path], name)
        fn.restype, fn.argtypes = SIGNATURES[name]
        setattr(self, name, fn)
        return fn


_lib = None
_symbols = _Symbols()


def _missing(path: str) -> HipLibraryMissing:
    return HipLibraryMissing(f"{path} not found: build it with `make -C nano-vllm_amd/csrc` "
                             "(or __graft_entry__.build()); there is no CPU fallback")


def load():
    """The entry points of the attention hot path (and, where it is built, of the mixers); raises loudly
    when the library has not been built."""
    global _lib
    if _lib is None:
        if not os.path.exists(LIB_PATH):
            raise _missing(LIB_PATH)
        _lib = _symbols
    return _lib


def load_mixers():
    """The entry points of the mixers' library and the common ones; needs that library only."""
    if not os.path.exists(MIXERS_LIB_PATH):
        raise _missing(MIXERS_LIB_PATH)
    return _symbols


def load_latent():
    """The entry points of the library of latent attention, matrix memory and experts, and the common ones."""
    if not os.path.exists(LATENT_LIB_PATH):
        raise _missing(LATENT_LIB_PATH)
    return _symbols


def load_masked():
    """The entry points of the library of masked attention and experts, and the common ones."""
    if not os.path.exists(MASKED_LIB_PATH):
        raise _missing(MASKED_LIB_PATH)
    return _symbols


def load_parallel():
    """The entry points of the library of masked and latent attention side by side, and the common ones."""
    if not os.path.exists(PARALLEL_LIB_PATH):
        raise _missing(PARALLEL_LIB_PATH)
    return _symbols


def load_shared():
    """Entry points that several libraries hold: each comes from the first that is there."""
    return _symbols


# kernel sets by name: the make target that builds one, its library and its loader
LIBRARIES = {"path": (LIB_PATH, load), "mixers": (MIXERS_LIB_PATH, load_mixers), "latent": (LATENT_LIB_PATH, load_latent),
             "masked": (MASKED_LIB_PATH, load_masked), "parallel": (PARALLEL_LIB_PATH, load_parallel)}


def load_set(name: str):
    return LIBRARIES[name][1]()


def status_string(code: int) -> str:
    return _symbols.nva_status_string(int(code)).decode()


def check(code: int, what: str) -> None:
    if code != OK:
        raise RuntimeError(f"{what}: {status_string(code)} (nva_status {code})")
