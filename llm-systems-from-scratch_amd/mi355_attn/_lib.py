"""ctypes binding of libmi355attn.so (declarations mirror include/mi355_attn.h)."""
from __future__ import annotations

import ctypes as C
import os

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(_HERE, "libmi355attn.so")
# the same library without the training kernels: what a served model needs, built by the command line tools in a fresh checkout
SERVING_LIB_PATH = os.path.join(_HERE, "libmi355attn_serving.so")
TRAINING_ONLY = ("mi355_prefill_bwd", "mi355_prefill_bwd_mask")

MI355_BF16 = 0
MI355_FP8_E4M3 = 1
MI355_FP32 = 2
MASK_NONE, MASK_CAUSAL, MASK_BOOL = 0, 1, 2
STATIC_SCRATCH_BYTES = 16 << 20          # MI355_STATIC_SCRATCH_BYTES

SCANS = {"auto": 0, "serial": 1, "chunked": 2}
TILINGS = {"auto": 0, "skinny": 1, "large": 2}

_i64x3 = C.c_int64 * 3
_i64x2 = C.c_int64 * 2
_lib = None

EXPORTS = (
    "mi355_prefill_fwd",
    "mi355_prefill_fwd_lse",
    "mi355_prefill_bwd",
    "mi355_prefill_fwd_mask_lse",
    "mi355_prefill_bwd_mask",
    "mi355_paged_decode_fwd",
    "mi355_paged_decode_fwd_static",
    "mi355_paged_decode_workspace_bytes",
    "mi355_paged_decode_chunk_tokens",
    "mi355_prefill_paged_fwd",
    "mi355_gather_kv_fp8",
    "mi355_prefill_fwd_splitkv",
    "mi355_prefill_splitkv_workspace_bytes",
    "mi355_prefill_suggest_kv_splits",
    "mi355_rope_and_cache",
    "mi355_rope_and_cache_fp8",
    "mi355_quantize_kv_fp8",
    "mi355_rms_norm_fwd",
    "mi355_silu_mul_fwd",
    "mi355_prefill_fwd_headwise",
    "mi355_prefill_paged_fwd_headwise",
    "mi355_paged_decode_fwd_headwise",
    "mi355_paged_attn_any_fwd",
    "mi355_kv_cache_write",
    "mi355_dyt_residual_fwd",
    "mi355_polynorm_fwd",
    "mi355_embed_pos_fwd",
    "mi355_prefill_fwd_window",
    "mi355_prefill_paged_fwd_window",
    "mi355_paged_decode_fwd_window",
    "mi355_paged_attn_any_fwd_window",
    "mi355_rope_any",
    "mi355_residual_rms_fwd",
    "mi355_ff_act_fwd",
    "mi355_gated_norm_fwd",
    "mi355_ssm_prefill",
    "mi355_ssm_decode",
    "mi355_moe_route",
    "mi355_moe_group",
    "mi355_moe_gate_up",
    "mi355_moe_down",
    "mi355_calib_copy",
    "mi355_last_error",
    "mi355_version",
)


class SsmArgs(C.Structure):
    """mi355_ssm_args"""
    _fields_ = ([(n, C.c_void_p) for n in ("proj", "conv_weight", "conv_bias", "dt_bias", "neg_a", "d_skip", "conv_state", "ssm_state",
                                           "slots", "positions", "cu_seqlens", "xbc", "y")] +
                [(n, C.c_int64) for n in ("proj_row_stride", "xbc_col", "dt_col", "y_row_stride", "n_rows")] +
                [(n, C.c_int) for n in ("batch", "heads", "vdim", "state", "groups", "taps", "n_slots", "dtype")] +
                [("seg_state", C.c_void_p), ("seg_decay", C.c_void_p), ("seg_len", C.c_int)])


class LibraryMissing(RuntimeError):
    pass


def built():
    """Path of the library to load: the full one, else the serving one, else None."""
    return next((p for p in (LIB_PATH, SERVING_LIB_PATH) if os.path.exists(p)), None)


class _ServingLib:
    """The serving library under the full one's interface: an entry point that it lacks is an error when it is called."""

    class _Missing:
        def __init__(self, name):
            self.name = name

        def __call__(self, *args):
            raise LibraryMissing(f"{self.name} is not in {SERVING_LIB_PATH}; run `python llm-systems-from-scratch_amd/build.py`")

    def __init__(self, lib):
        self._lib = lib
        for name in TRAINING_ONLY:
            setattr(self, name, self._Missing(name))

    def __getattr__(self, name):
        return getattr(self._lib, name)


def load():
    """Loads the HIP library once.  There is no fallback: a missing library is an error."""
    global _lib
    if _lib is not None:
        return _lib
    path = built()
    if path is None:
        raise LibraryMissing(
            f"{LIB_PATH} is not built; run `python llm-systems-from-scratch_amd/build.py` "
            "(needs hipcc, cross-compiles for gfx950 without a GPU)")
    lib = C.CDLL(path) if path == LIB_PATH else _ServingLib(C.CDLL(path))
    vp, i32, i64, f32, sz = C.c_void_p, C.c_int, C.c_int64, C.c_float, C.c_size_t
    lib.mi355_prefill_fwd.restype = i32
    lib.mi355_prefill_fwd.argtypes = [vp, vp, vp, vp, _i64x3, _i64x3, _i64x3, _i64x3, vp, vp, vp, _i64x3,
                                      i32, i32, i32, i32, i32, i32, f32, i32, i32, vp]
    lib.mi355_prefill_fwd_lse.restype = i32
    lib.mi355_prefill_fwd_lse.argtypes = [vp, vp, vp, vp, vp, _i64x3, _i64x3, _i64x3, _i64x3, _i64x2, vp, vp,
                                          i32, i32, i32, i32, i32, i32, f32, i32, i32, vp]
    lib.mi355_prefill_bwd.restype = i32
    lib.mi355_prefill_bwd.argtypes = [vp] * 10 + [_i64x3] * 8 + [_i64x2, vp, vp,
                                                                 i32, i32, i32, i32, i32, i32, f32, i32, i32, vp]
    lib.mi355_prefill_fwd_mask_lse.restype = i32
    lib.mi355_prefill_fwd_mask_lse.argtypes = [vp, vp, vp, vp, vp, _i64x3, _i64x3, _i64x3, _i64x3, _i64x2, vp, _i64x3,
                                               i32, i32, i32, i32, i32, i32, f32, i32, vp]
    lib.mi355_prefill_bwd_mask.restype = i32
    lib.mi355_prefill_bwd_mask.argtypes = [vp] * 10 + [_i64x3] * 8 + [_i64x2, vp, _i64x3,
                                                                      i32, i32, i32, i32, i32, i32, f32, i32, vp]
    lib.mi355_prefill_paged_fwd.restype = i32
    lib.mi355_prefill_paged_fwd.argtypes = [vp, vp, vp, vp, i64, i64, vp, vp, i64, i64, vp,
                                            i32, i32, i32, i32, i32, i32, i64, f32, i32, i32, i64, vp, sz, vp]
    lib.mi355_gather_kv_fp8.restype = i32
    lib.mi355_gather_kv_fp8.argtypes = [vp, vp, vp, vp, vp, i64, i64, vp, vp, vp, vp, i64, i64, i32, i32, i32, i32, i64, vp]
    lib.mi355_prefill_fwd_splitkv.restype = i32
    lib.mi355_prefill_fwd_splitkv.argtypes = [vp, vp, vp, vp, _i64x3, _i64x3, _i64x3, _i64x3, vp, vp,
                                              i32, i32, i32, i32, i32, i32, f32, i32, i32, i32, i64, vp, sz, vp]
    lib.mi355_prefill_splitkv_workspace_bytes.restype = sz
    lib.mi355_prefill_splitkv_workspace_bytes.argtypes = [i64, i32, i32, i32]
    lib.mi355_prefill_suggest_kv_splits.restype = i32
    lib.mi355_prefill_suggest_kv_splits.argtypes = [i32, i32, i32, i32, i32, i64, i32, i32]
    lib.mi355_paged_decode_fwd.restype = i32
    lib.mi355_paged_decode_fwd.argtypes = [vp, vp, vp, vp, vp, i64, vp, vp, vp, vp, sz,
                                           i32, i32, i32, i32, i32, i64, i32, f32, i32, vp]
    lib.mi355_paged_decode_fwd_static.restype = i32
    lib.mi355_paged_decode_fwd_static.argtypes = [vp, vp, vp, vp, vp, i64, vp, vp, vp,
                                                  i32, i32, i32, i32, i32, i64, i32, f32, i32, vp]
    lib.mi355_paged_decode_workspace_bytes.restype = sz
    lib.mi355_paged_decode_workspace_bytes.argtypes = [i32, i32, i32, i32]
    lib.mi355_paged_decode_chunk_tokens.restype = i32
    lib.mi355_paged_decode_chunk_tokens.argtypes = [i32, i32, i32, i32]
    lib.mi355_rope_and_cache.restype = i32
    lib.mi355_rope_and_cache.argtypes = [vp, vp, vp, vp, vp, vp, vp, vp, vp, i64, i32, i32, i32, i32, i32,
                                         i64, i64, i64, i64, vp, i64, vp]
    lib.mi355_rope_and_cache_fp8.restype = i32
    lib.mi355_rope_and_cache_fp8.argtypes = [vp] * 11 + [i64, i32, i32, i32, i32, i32, i64, i64, i64, i64, vp, i64, vp]
    lib.mi355_quantize_kv_fp8.restype = i32
    lib.mi355_quantize_kv_fp8.argtypes = [vp, vp, vp, i64, i32, i32, i32, vp]
    lib.mi355_rms_norm_fwd.restype = i32
    lib.mi355_rms_norm_fwd.argtypes = [vp, vp, vp, vp, vp, vp, i64, i32, i64, i64, i64, i64, f32, i32, vp]
    lib.mi355_silu_mul_fwd.restype = i32
    lib.mi355_silu_mul_fwd.argtypes = [vp, vp, vp, i64, i32, i64, i64, i64, vp]
    lib.mi355_prefill_fwd_headwise.restype = i32
    lib.mi355_prefill_fwd_headwise.argtypes = [vp, vp, vp, vp, _i64x3, _i64x3, _i64x3, _i64x3, vp, vp, vp, vp,
                                               i32, i32, i32, i32, i32, i32, f32, i32, i32, i32, i64, vp, sz, vp]
    lib.mi355_prefill_paged_fwd_headwise.restype = i32
    lib.mi355_prefill_paged_fwd_headwise.argtypes = [vp, vp, vp, vp, i64, i64, vp, vp, i64, i64, vp, vp, vp,
                                                     i32, i32, i32, i32, i32, i32, i64, f32, i32, i32, i64, vp, sz, vp]
    lib.mi355_paged_decode_fwd_headwise.restype = i32
    lib.mi355_paged_decode_fwd_headwise.argtypes = [vp, i64, vp, vp, vp, vp, i64, vp, vp, vp, vp, vp, vp, sz,
                                                    i32, i32, i32, i32, i32, i64, i32, f32, i32, vp]
    lib.mi355_paged_attn_any_fwd.restype = i32
    lib.mi355_paged_attn_any_fwd.argtypes = [vp, vp, vp, vp, i64, i64, i64, vp, vp, i64, i64, vp, vp, vp,
                                             i32, i32, i32, i32, i32, i32, i64, f32, i32, vp]
    lib.mi355_kv_cache_write.restype = i32
    lib.mi355_kv_cache_write.argtypes = [vp, vp, vp, vp, vp, i64, i64, i32, i32, i32, i64, i64, i32, vp]
    lib.mi355_dyt_residual_fwd.restype = i32
    lib.mi355_dyt_residual_fwd.argtypes = [vp, vp, vp, vp, f32, vp, vp, vp, vp, f32, vp, vp, vp, i64, i32, i64, i64, i64,
                                           i32, vp]
    lib.mi355_polynorm_fwd.restype = i32
    lib.mi355_polynorm_fwd.argtypes = [vp, vp, i64, i32, i64, i64, C.c_float * 4, f32, i32, vp]
    lib.mi355_embed_pos_fwd.restype = i32
    lib.mi355_embed_pos_fwd.argtypes = [vp, vp, vp, vp, vp, i64, i32, i64, i64, i32, vp]
    lib.mi355_prefill_fwd_window.restype = i32
    lib.mi355_prefill_fwd_window.argtypes = [vp, vp, vp, vp, _i64x3, _i64x3, _i64x3, _i64x3, vp, vp, vp, vp,
                                             i32, i32, i32, i32, i32, i32, f32, i32, i32, i32, vp]
    lib.mi355_prefill_paged_fwd_window.restype = i32
    lib.mi355_prefill_paged_fwd_window.argtypes = [vp, vp, vp, vp, i64, i64, vp, vp, i64, i64, vp, vp, vp,
                                                   i32, i32, i32, i32, i32, i32, i64, f32, i32, i32, i32, vp]
    lib.mi355_paged_decode_fwd_window.restype = i32
    lib.mi355_paged_decode_fwd_window.argtypes = [vp, i64, vp, vp, vp, i64, vp, i64, vp, vp, vp, vp, vp, vp, sz,
                                                  i32, i32, i32, i32, i32, i64, i32, f32, i32, i32, i32, vp]
    lib.mi355_paged_attn_any_fwd_window.restype = i32
    lib.mi355_paged_attn_any_fwd_window.argtypes = [vp, vp, vp, vp, i64, i64, i64, vp, vp, i64, i64, vp, vp, vp,
                                                    i32, i32, i32, i32, i32, i32, i64, f32, i32, i32, i32, vp]
    lib.mi355_rope_any.restype = i32
    lib.mi355_rope_any.argtypes = [vp, vp, vp, vp, i64, i32, i32, i32, i32, i64, i64, i32, vp]
    lib.mi355_residual_rms_fwd.restype = i32
    lib.mi355_residual_rms_fwd.argtypes = [vp, vp, vp, vp, i32, vp, vp, i64, vp, f32, f32, vp, i64, i32, i32, i64, i64, i64,
                                           i32, vp]
    lib.mi355_ff_act_fwd.restype = i32
    lib.mi355_ff_act_fwd.argtypes = [vp, vp, vp, vp, i64, i32, i64, i64, i64, i32, vp]
    lib.mi355_gated_norm_fwd.restype = i32
    lib.mi355_gated_norm_fwd.argtypes = [vp, vp, vp, vp, i64, i32, i32, i64, i64, i64, f32, i32, vp]
    lib.mi355_ssm_prefill.restype = i32
    lib.mi355_ssm_prefill.argtypes = [C.POINTER(SsmArgs), i32, vp]
    lib.mi355_ssm_decode.restype = i32
    lib.mi355_ssm_decode.argtypes = [C.POINTER(SsmArgs), vp]
    lib.mi355_moe_route.restype = i32
    lib.mi355_moe_route.argtypes = [vp, vp, vp, vp, vp, vp, i64, i64, i64, i32, i32, i32, i32, vp]
    lib.mi355_moe_group.restype = i32
    lib.mi355_moe_group.argtypes = [vp, i64, i32, vp, vp, vp]
    lib.mi355_moe_gate_up.restype = i32
    lib.mi355_moe_gate_up.argtypes = [vp, vp, vp, vp, vp, i64, i64, i64, i32, i32, i32, i32, i32, i32, vp]
    lib.mi355_moe_down.restype = i32
    lib.mi355_moe_down.argtypes = [vp, vp, vp, vp, vp, vp, i64, i64, i64, i32, i32, i32, i32, i32, i32, vp]
    lib.mi355_calib_copy.restype = i32
    lib.mi355_calib_copy.argtypes = [vp, vp, sz, vp]
    lib.mi355_last_error.restype = C.c_char_p
    lib.mi355_version.restype = C.c_char_p
    _lib = lib
    return lib


def strides3(values):
    return _i64x3(*[int(v) for v in values])


def strides2(values):
    return _i64x2(*[int(v) for v in values])


def floats4(values):
    return (C.c_float * 4)(*[float(v) for v in values])


def check(rc: int, what: str):
    if rc != 0:
        msg = load().mi355_last_error().decode()
        if rc < 0:
            raise ValueError(f"{what}: {msg} (code {rc})")
        raise RuntimeError(f"{what}: HIP error {rc}: {msg}")
