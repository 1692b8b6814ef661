"""ctypes binding of libmimir_mi355x.so, the C ABI of include/mimir_mi355x.h.

This is the same binding a Go host makes with purego (Dlopen + RegisterFunc):
symbols are looked up by name and called with plain pointers and integers.
The library is built ahead of time by mimir_amd.build; loading fails loudly
when it is missing, and there is no fallback path.
"""
from __future__ import annotations

import ctypes as C
import os

HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(HERE, "lib", "libmimir_mi355x.so")

OK = 0
ERR_OUT_OF_MEMORY, ERR_SHAPE, ERR_DTYPE, ERR_INDEX, ERR_INTERNAL = 2, 0x1001, 0x1002, 0x1003, 0x1005
F32, I32, BF16, F16, Q8_0, Q4_K, Q6_K, Q4_0 = 1, 2, 3, 4, 5, 6, 7, 8

_vp, _i64, _int, _sz = C.c_void_p, C.c_int64, C.c_int, C.c_size_t

# name -> (restype, argtypes): every symbol include/mimir_mi355x.h declares.
SYMBOLS = {
    "mi355x_init": (C.c_uint32, [_int]),
    "mi355x_last_error": (_sz, [C.c_char_p, _sz]),
    "mi355x_block_size": (_int, [_int]),
    "mi355x_block_bytes": (_int, [_int]),
    "mi355x_bytes": (_i64, [_int, _i64]),
    "mi355x_alloc": (C.c_uint32, [C.POINTER(_vp), _sz]),
    "mi355x_free": (C.c_uint32, [_vp]),
    "mi355x_upload": (C.c_uint32, [_vp, _vp, _sz, _vp]),
    "mi355x_download": (C.c_uint32, [_vp, _vp, _sz, _vp]),
    "mi355x_sync": (C.c_uint32, [_vp]),
    "mi355x_qgemv": (C.c_uint32, [_int, _vp, _vp, _vp, _i64, _i64, _i64, _i64, _vp]),
    "mi355x_qgemv_noalloc": (C.c_uint32, [_int, _vp, _vp, _vp, _i64, _i64, _i64, _i64, _vp]),
    "mi355x_act_bytes": (_sz, [_int, _i64]),
    "mi355x_convert_act": (C.c_uint32, [_int, _vp, _i64, _i64, _i64, _vp, _vp]),
    "mi355x_qgemv_act": (C.c_uint32, [_int, _vp, _vp, _vp, _i64, _i64, _i64, _vp]),
    "mi355x_qgemv_act_add": (C.c_uint32, [_int, _vp, _vp, _vp, _vp, _i64, _i64, _i64, _vp]),
    "mi355x_qgemv_act_multi": (C.c_uint32, [_int, _vp, _vp, _vp, _i64, _i64, _i64, _vp, _vp, _i64, _i64, _vp]),
    "mi355x_qgemv_act_swiglu": (C.c_uint32, [_int, _vp, _vp, _vp, _vp, _i64, _i64, _i64, _vp]),
    "mi355x_dequant": (C.c_uint32, [_int, _vp, _i64, _i64, _vp, _int, _vp]),
    "mi355x_gather_rows": (C.c_uint32, [_int, _vp, _i64, _i64, _vp, _i64, _vp, _vp]),
    "mi355x_rmsnorm": (C.c_uint32, [_vp, _vp, _vp, _i64, _i64, C.c_double, _vp]),
    "mi355x_rope": (C.c_uint32, [_vp, _vp, _i64, _i64, _int, _int, _int, _i64, _i64, _i64, _i64, _vp, _vp, _i64, _i64, _vp]),
    "mi355x_kv_write": (C.c_uint32, [_vp, _vp, _int, _i64, _int, _i64, _int, _i64, _i64, _i64, _i64, _i64, _vp]),
    "mi355x_attention": (C.c_uint32, [_vp, _vp, _vp, _vp, _vp, _vp, _int, _vp, _vp, _vp, _vp, _vp, _i64, _int, _int, _i64, _i64, _int, _int,
                                      C.c_double, _int, _i64, _vp]),
    "mi355x_swiglu": (C.c_uint32, [_vp, _vp, _vp, _i64, _i64, _i64, _vp]),
    "mi355x_add": (C.c_uint32, [_vp, _vp, _vp, _i64, _vp]),
    "mi355x_argmax": (C.c_uint32, [_vp, _i64, _i64, _vp, _vp]),
    "mi355x_model_destroy": (C.c_uint32, [_vp]),
    "mi355x_model_set_tensor": (C.c_uint32, [_vp, C.c_char_p, _int, _vp, _i64]),
    "mi355x_model_finalize": (C.c_uint32, [_vp, _i64]),
    "mi355x_model_reset": (C.c_uint32, [_vp]),
    "mi355x_model_cache_len": (_i64, [_vp]),
    "mi355x_model_logits": (C.c_uint32, [_vp, _vp, _i64, _int, _vp]),
    "mi355x_model_logits_at": (C.c_uint32, [_vp, _vp, _i64, _vp, _i64, _vp]),
    "mi355x_model_generate": (C.c_uint32, [_vp, _vp, _i64, _i64, _vp, _vp]),
    "mi355x_stack_create": (C.c_uint32, [_vp, _vp, C.POINTER(_vp)]),
    "mi355x_stack_tensor": (C.c_uint32, [_vp, _i64, _vp, _sz, _vp, _vp]),
    "mi355x_llama_create": (C.c_uint32, [_vp, C.POINTER(_vp)]),
    "mi355x_llama_destroy": (C.c_uint32, [_vp]),
    "mi355x_llama_set_tensor": (C.c_uint32, [_vp, C.c_char_p, _int, _vp, _i64]),
    "mi355x_llama_set_rope_factors": (C.c_uint32, [_vp, _vp, C.c_int32]),
    "mi355x_llama_finalize": (C.c_uint32, [_vp, _i64]),
    "mi355x_llama_reset": (C.c_uint32, [_vp]),
    "mi355x_llama_set_cache": (C.c_uint32, [_vp, C.c_int32, _vp, _vp, _i64]),
    "mi355x_llama_cache_len": (_i64, [_vp]),
    "mi355x_llama_logits": (C.c_uint32, [_vp, _vp, _i64, _int, _vp]),
    "mi355x_llama_generate": (C.c_uint32, [_vp, _vp, _i64, _i64, _vp, _vp]),
    "mi355x_tune": (C.c_uint32, [C.c_char_p, _int]),
    "mi355x_backend_last_error": (_sz, [C.c_char_p, _sz]),
    "mi355x_backend_open": (C.c_uint32, [_int, _vp]),
    "mi355x_backend_close": (C.c_uint32, [_vp]),
    "mi355x_backend_alloc": (C.c_uint32, [_vp, _int, _i64, _vp]),
    "mi355x_backend_free": (C.c_uint32, [_vp, _vp]),
    "mi355x_backend_upload": (C.c_uint32, [_vp, _vp, _vp, _sz]),
    "mi355x_backend_download": (C.c_uint32, [_vp, _vp, _sz, _vp]),
    "mi355x_backend_sync": (C.c_uint32, [_vp]),
    "mi355x_backend_run": (C.c_uint32, [_vp, _vp, _vp, _int, _vp, _int]),
    "mi355x_batch_new": (C.c_uint32, [_vp, _int, _vp, _vp, _vp, _vp, _vp]),
    "mi355x_batch_free": (C.c_uint32, [_vp]),
    "mi355x_backend_run_batch": (C.c_uint32, [_vp, _vp]),
    "mi355x_backend_graph_replays": (_i64, [_vp]),
    "mi355x_qgemm_bf16": (C.c_uint32, [_int, _vp, _vp, _vp, _i64, _i64, _i64, _i64, _int, _vp]),
    "mi355x_attention_d": (C.c_uint32, [_vp, _vp]),
    "mi355x_stream_release": (C.c_uint32, [_vp]),
    "mi355x_last_kernel": (C.c_uint32, [_vp, _sz]),
    "mi355x_timed_begin": (C.c_uint32, [_int]),
    "mi355x_timed_end": (C.c_uint32, [_vp, _vp]),
    "mi355x_gemv_stamps": (C.c_uint32, [_vp]),
    "mi355x_stream_read": (C.c_uint32, [_vp, _sz, _vp, _int, _int, _vp]),
}


class LlamaConfig(C.Structure):
    """mi355x_llama_config."""
    _fields_ = [(n, C.c_int32) for n in ("embed", "hidden", "layers", "heads", "kv_heads", "head_dim", "rope_dim", "vocab", "context",
                                          "interleaved", "cache_dtype", "batch")] + [(n, C.c_double) for n in ("rope_base", "rope_scale", "eps")]


MIXER_LATENT, MIXER_MLSTM, MIXER_LIGHTNING, MIXER_ATTENTION = 1, 2, 3, 4
MLP_RELU2, MLP_SWIGLU = 0, 1
STACK_EMBED_NORM, STACK_POST_NORMS, STACK_DEPTH_AVERAGE, STACK_PARALLEL, STACK_LAYER_SCALE, STACK_OUTPUT_MATRIX = 1, 2, 4, 8, 16, 32


class StackConfig(C.Structure):
    """mi355x_stack_config."""
    _fields_ = [(n, C.c_int32) for n in ("width", "vocab", "layers", "context", "batch", "taps", "norm_groups", "dtype", "flags", "reserved")] + \
               [(n, C.c_int64) for n in ("pair_buckets", "pair_mul_prev", "pair_mul_cur")] + [("eps", C.c_double), ("logit_scale", C.c_double)]


class StackLayer(C.Structure):
    """mi355x_stack_layer."""
    _fields_ = [(n, C.c_int32) for n in ("mixer", "heads", "kv_heads", "dim", "vdim", "rot_dim", "kv_rank", "ff", "mlp", "unit_qk", "value_mix", "head_gate")] + \
               [(n, C.c_double) for n in ("scale", "softcap", "rot_base", "rot_factor", "rot_low", "rot_high", "rot_original", "gate_cap")] + \
               [("decay", C.POINTER(C.c_double))]


class AttentionDesc(C.Structure):
    """mi355x_attention_desc."""
    _fields_ = [(n, C.c_void_p) for n in ("q", "k", "v", "mask", "out", "lse")] + \
               [("q_strides", C.c_int64 * 3), ("k_strides", C.c_int64 * 3), ("v_strides", C.c_int64 * 3), ("out_strides", C.c_int64 * 3),
                ("mask_strides", C.c_int64 * 4)] + [(n, C.c_int64) for n in ("B", "Q", "K", "causal_offset")] + [("scale", C.c_double)] + \
               [(n, C.c_int32) for n in ("kv_dtype", "H", "HK", "D", "DV", "causal")]


class Mi355xError(RuntimeError):
    def __init__(self, status: int, message: str):
        super().__init__(f"[{status:#x}] {message}")
        self.status = status


_lib = None
_lib_part = None  # the part that _lib holds, None: all of it


def load(part: str | None = None) -> C.CDLL:
    """Loads the library and declares every symbol; raises if it is not built. With `part` (a name of
    mimir_amd.build.PARTS) the library of that part alone will do where the whole one is not built: it
    exports the entry points of the part's sources."""
    global _lib, _lib_part
    if _lib is not None and (_lib_part is None or _lib_part == part):
        return _lib
    path = os.environ.get("MIMIR_MI355X_LIB") or LIB_PATH  # as the reference's loaders take a path from the environment
    whole = os.path.exists(path)
    if not whole and part is not None:
        path = os.path.join(HERE, "lib", f"libmimir_mi355x_{part}.so")
    if not os.path.exists(path):
        raise FileNotFoundError(f"{path} is not built: run `python -m mimir_amd.build{' ' + part if part else ''}`")
    lib = C.CDLL(path)
    for name, (res, args) in SYMBOLS.items():
        try:
            fn = getattr(lib, name)  # AttributeError if the symbol is missing
        except AttributeError:
            if whole:
                raise
            continue
        fn.restype, fn.argtypes = res, args
    _lib, _lib_part = lib, (None if whole else part)
    return _lib


def last_error() -> str:
    buf = C.create_string_buffer(1024)
    (_lib or load()).mi355x_last_error(buf, 1024)
    return buf.value.decode(errors="replace")


def check(status: int) -> None:
    if status != OK:
        raise Mi355xError(status, last_error())
