"""ctypes bindings of libw4a16_hip.so (include/w4a16.h) and libdense_lm_hip.so (include/dense_lm.h)."""

import ctypes
import os

_HERE = os.path.dirname(os.path.abspath(__file__))
_LIB_PATH = os.path.join(os.path.dirname(_HERE), "lib", "libw4a16_hip.so")
DENSE_ABI = 2
_DENSE_PATH = os.path.join(os.path.dirname(_HERE), "lib", "libdense_lm_hip.so")

OK = 0
ERR_NULL, ERR_SHAPE, ERR_GROUP, ERR_ALIGN, ERR_WORKSPACE, ERR_HIP, ERR_TUNE, ERR_TIMEOUT, ERR_TOO_LARGE, ERR_NOT_PREPARED = -1, -2, -3, -4, -5, -6, -7, -8, -9, -10

# every symbol include/w4a16.h declares: name -> (restype, argtypes)
_vp, _ci, _sz, _cf = ctypes.c_void_p, ctypes.c_int, ctypes.c_size_t, ctypes.c_float
SYMBOLS = {
    "w4a16_abi_version": (_ci, []),
    "w4a16_strerror": (ctypes.c_char_p, [_ci]),
    "w4a16_last_hip_error": (ctypes.c_char_p, []),
    "awq_dequant_bf16": (_ci, [_vp, _vp, _vp, _vp, _ci, _ci, _ci, _vp]),
    "awq_dequant_1d_tile_bytes": (_sz, [_ci, _ci, _ci]),
    "awq_dequant_1d_bf16": (_ci, [_vp, _vp, _ci, _ci, _ci, _vp]),
    "w4a16_gemm_workspace_bytes": (_sz, [_ci, _ci, _ci]),
    "w4a16_ffn_workspace_bytes": (_sz, [_ci, _ci]),
    "w4a16_workspace_init": (_ci, [_vp, _sz, _vp]),
    "w4a16_workspace_check": (_ci, [_vp, _vp]),
    "w4a16_gemv_bf16": (_ci, [_vp, _vp, _vp, _vp, _vp, _ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_gemm_bf16": (_ci, [_vp, _vp, _vp, _vp, _vp, _ci, _ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_gemv_swiglu_bf16": (_ci, [_vp] * 8 + [_ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_ffn_swiglu_bf16": (_ci, [_vp] * 12 + [_ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_gemv_add_bf16": (_ci, [_vp] * 6 + [_ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_rms_gemv_bf16": (_ci, [_vp, _vp, _cf] + [_vp] * 4 + [_ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_rms_gemv_swiglu_bf16": (_ci, [_vp, _vp, _cf] + [_vp] * 7 + [_ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_block_workspace_bytes": (_sz, [_ci, _ci]),
    "w4a16_o_gemv_ffn_bf16": (_ci, [_vp, _vp, _vp, _cf] + [_vp] * 15 + [_ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_attention_workspace_bytes": (_sz, [_ci, _ci]),
    "w4a16_decode_attention_bf16": (_ci, [_vp] * 5 + [_ci] * 5 + [_vp, _sz, _vp]),
    "w4a16_prefill_block_workspace_bytes": (_sz, [_ci, _ci, _ci]),
    "rms_norm_rows_bf16": (_ci, [_vp, _vp, _cf, _vp, _ci, _ci, _vp]),
    "w4a16_prefill_o_ffn_bf16": (_ci, [_vp, _vp, _vp, _cf] + [_vp] * 15 + [_ci, _ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_prefill_qkv_workspace_bytes": (_sz, [_ci, _ci]),
    "w4a16_prefill_rms_qkv_rope_bf16": (_ci, [_vp, _vp, _cf, _vp, _vp, _vp, _vp, _ci, _ci, _vp] + [_ci] * 6 + [_vp, _sz, _vp]),
    "w4a16_prefill_rms_qkv_rope_stream_bf16": (_ci, [_vp, _vp, _cf, _vp, _vp, _ci, _ci, _vp] + [_ci] * 6 + [_vp, _sz, _vp]),
    "w4a16_prefill_o_ffn_stream_bf16": (_ci, [_vp, _vp, _vp, _cf] + [_vp] * 7 + [_ci, _ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_q4nx_prefill_rms_qkv_rope_stream_bf16": (_ci, [_vp, _vp, _cf, _vp, _vp, _ci, _ci, _vp] + [_ci] * 5 + [_vp, _sz, _vp]),
    "w4a16_q4nx_prefill_o_ffn_stream_bf16": (_ci, [_vp, _vp, _vp, _cf] + [_vp] * 7 + [_ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_prefill_attention_bf16": (_ci, [_vp, _vp, _ci, _ci, _ci, _ci, _vp]),
    "lm_head_workspace_bytes": (_sz, [_ci]),
    "w4a16_decode_attn_o_gemv_ffn_bf16": (_ci, [_vp] * 5 + [_ci] * 5 + [_vp, _sz, _vp, _vp, _cf] + [_vp] * 12 + [_vp, _vp, _ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_rms_gemv_sumsq_bf16": (_ci, [_vp, _vp, _ci, _vp, _cf, _vp, _vp, _vp, _vp, _ci, _ci, _ci, _vp, _sz, _vp]),
    "rope_halfsplit_bf16": (_ci, [_vp, _vp, _vp, _ci, _ci, _vp]),
    "lm_head_gemv_bf16": (_ci, [_vp, _vp, _cf, _vp, _vp, _vp, _ci, _ci, _vp, _sz, _vp]),
    "q4nx_dequant_bf16": (_ci, [_vp, _vp, _ci, _ci, _ci, _vp]),
    "q4nx_repack": (_ci, [_vp, _vp, _vp, _vp, _ci, _ci, _ci, _vp]),
    "w4a16_q4nx_stream_bytes": (_sz, [_ci, _ci]),
    "w4a16_q4nx_blocks_to_stream": (_ci, [_vp, _vp, _ci, _ci, _ci, _vp]),
    "w4a16_q4nx_repack_stream": (_ci, [_vp, _vp, _vp, _vp, _ci, _ci, _vp]),
    "w4a16_q4nx_gemv_stream_bf16": (_ci, [_vp, _vp, _vp, _vp, _ci, _ci, _vp]),
    "w4a16_q4nx_gemm_stream_bf16": (_ci, [_vp, _vp, _vp, _vp, _ci, _ci, _ci, _vp]),
    "w4a16_q4nx_rms_gemv_stream_bf16": (_ci, [_vp, _vp, _ci, _vp, _cf, _vp, _vp, _ci, _ci, _vp]),
    "w4a16_q4nx_o_gemv_ffn_stream_bf16": (_ci, [_vp, _vp, _vp, _cf] + [_vp] * 8 + [_ci, _ci, _vp, _sz, _vp]),
    "w4a16_stream_bytes": (_sz, [_ci, _ci]),
    "w4a16_repack_stream": (_ci, [_vp, _vp, _vp, _vp, _ci, _ci, _ci, _vp]),
    "w4a16_gemv_stream_bf16": (_ci, [_vp, _vp, _vp, _ci, _ci, _ci, _vp]),
    "w4a16_probe_stream_read": (_ci, [_vp, _vp, _ci, _ci, _vp]),
    "w4a16_gemm_stream_bf16": (_ci, [_vp, _vp, _vp, _ci, _ci, _ci, _ci, _vp]),
    "w4a16_gemm_stream_scratch_bytes": (_sz, [_ci, _ci, _ci]),
    "w4a16_gemm_stream_scratch_bf16": (_ci, [_vp, _vp, _vp, _ci, _ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_gemv_add_stream_bf16": (_ci, [_vp, _vp, _vp, _vp, _ci, _ci, _ci, _vp]),
    "w4a16_gemv_swiglu_stream_bf16": (_ci, [_vp, _vp, _vp, _vp, _ci, _ci, _ci, _vp]),
    "w4a16_rms_gemv_stream_bf16": (_ci, [_vp, _vp, _ci, _vp, _cf, _vp, _vp, _ci, _ci, _ci, _vp]),
    "w4a16_rms_gemv_swiglu_stream_bf16": (_ci, [_vp, _vp, _cf, _vp, _vp, _vp, _ci, _ci, _ci, _vp]),
    "w4a16_ffn_swiglu_stream_bf16": (_ci, [_vp] * 6 + [_ci, _ci, _ci, _vp]),
    "w4a16_block_stream_workspace_bytes": (_sz, [_ci, _ci]),
    "w4a16_o_gemv_ffn_stream_bf16": (_ci, [_vp, _vp, _vp, _cf] + [_vp] * 8 + [_ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_decode_attn_o_gemv_ffn_stream_bf16": (_ci, [_vp] * 5 + [_ci] * 5 + [_vp, _sz, _vp, _vp, _cf] + [_vp] * 6 + [_ci, _ci, _ci, _vp, _sz, _vp]),
    "w4a16_gemv_noalloc_bf16": (_ci, [_vp, _vp, _vp, _vp, _vp, _ci, _ci, _ci, _vp]),
    "w4a16_noalloc_check": (_ci, [_vp]),
    "w4a16_tune": (_ci, [ctypes.c_char_p, _ci]),
}


# ---- libdense_lm_hip.so: descriptor structs and symbols of include/dense_lm.h
_i32, _i64 = ctypes.c_int32, ctypes.c_int64


class Intake(ctypes.Structure):
    _fields_ = [("mode", _i32), ("width", _i32), ("eps", _cf), ("scale", _cf), ("x", _vp), ("res", _vp), ("y", _vp), ("norm_w", _vp),
                ("final_w", _vp), ("res_out", _vp), ("h_out", _vp), ("embed", _vp), ("token", _vp)]


class Router(ctypes.Structure):
    _fields_ = [("logits", _vp), ("correction", _vp), ("ld", _i32), ("experts", _i32), ("top", _i32), ("groups", _i32), ("keep", _i32)]


class GemmArgs(ctypes.Structure):
    _fields_ = [("a", _vp), ("w", _vp), ("out", _vp), ("lda", _i64), ("ldo", _i64), ("w_stride", _i64), ("tiles", _vp), ("order", _vp),
                ("M", _i32), ("N", _i32), ("K", _i32), ("epilogue", _i32), ("n_tiles", _i32), ("gather", _i32), ("tile_rows", _i32),
                ("silu_begin", _i32), ("silu_end", _i32)]


class LatentShape(ctypes.Structure):
    _fields_ = [("heads", _i32), ("dim", _i32), ("rot", _i32), ("vdim", _i32), ("rank", _i32), ("rot_pairs", _i32), ("true_rank", _i32),
                ("scale", _cf)]


class LatentRows(ctypes.Structure):
    _fields_ = [("proj", _vp), ("lut", _vp), ("kv_norm", _vp), ("cache", _vp), ("pos_dev", _vp), ("ld", _i64), ("kv_off", _i32),
                ("gate_off", _i32), ("M", _i32), ("pos", _i32), ("eps", _cf)]


class RowOutput(ctypes.Structure):
    _fields_ = [("silu_begin", _i32), ("silu_end", _i32), ("gate", _i32)]


class HeadShape(ctypes.Structure):
    _fields_ = [("heads", _i32), ("kv_heads", _i32), ("dim", _i32), ("vdim", _i32), ("true_dim", _i32), ("window", _i32), ("ring", _i32),
                ("scale", _cf), ("out_scale", _cf)]


class HeadRows(ctypes.Structure):
    _fields_ = [("proj", _vp), ("q_norm", _vp), ("k_norm", _vp), ("cache", _vp), ("pos_dev", _vp), ("ld", _i64), ("off", _i32), ("M", _i32),
                ("pos", _i32), ("eps", _cf)]


class ShortConvArgs(ctypes.Structure):
    _fields_ = [("proj", _vp), ("w", _vp), ("history", _vp), ("factors", _vp), ("pos_dev", _vp), ("ld", _i64), ("k_heads", _i32), ("heads", _i32),
                ("dim", _i32), ("vdim", _i32), ("taps", _i32), ("off", _i32), ("M", _i32), ("pos", _i32), ("q_scale", _cf), ("unit_eps", _cf)]


class ShortProduct(ctypes.Structure):
    _fields_ = [("w", _vp), ("x", _vp), ("out", _vp), ("K", _i32), ("N", _i32)]


class RecurrenceArgs(ctypes.Structure):
    _fields_ = [("qkv", _vp), ("log2_decay", _vp), ("z", _vp), ("a_log", _vp), ("dt_bias", _vp), ("factors", _vp), ("beta", _vp), ("state", _vp),
                ("pos_dev", _vp), ("ld", _i64), ("ld_beta", _i64), ("k_heads", _i32), ("heads", _i32), ("dim", _i32), ("vdim", _i32),
                ("q_off", _i32), ("k_off", _i32), ("v_off", _i32), ("M", _i32), ("pos", _i32)]


DENSE_SYMBOLS = {
    "dlm_abi_version": (_ci, []),
    "dlm_strerror": (ctypes.c_char_p, [_ci]),
    "dlm_last_hip_error": (ctypes.c_char_p, []),
    "dlm_gemv_keys": (_ci, [_ci, _ci]),
    "dlm_gemv": (_ci, [_ci] + [_vp] * 5 + [_ci] * 3 + [_vp]),
    "dlm_argmax": (_ci, [_vp, _ci] + [_vp] * 4),
    "dlm_moe_gate_up_gemv": (_ci, [_ci] + [_vp] * 6 + [_ci, _ci, _vp]),
    "dlm_moe_down_gemv": (_ci, [_ci] + [_vp] * 5 + [_ci] * 4 + [_vp]),
    "dlm_moe_select": (_ci, [_vp, _ci, _vp, _vp, _vp]),
    "dlm_moe_max_tiles": (_ci, [_ci] * 3),
    "dlm_moe_plan": (_ci, [_vp] + [_ci] * 3 + [_vp] * 3),
    "dlm_gemm_tile_rows": (_ci, [_ci] * 4),
    "dlm_gemm": (_ci, [_ci, _vp, _vp]),
    "dlm_embed_rows": (_ci, [_ci, _vp, _vp, _cf, _vp, _vp, _ci, _ci, _vp]),
    "dlm_residual_norm_rows": (_ci, [_ci, _vp, _vp, _vp, _ci, _vp, _cf, _ci, _vp, _ci, _ci, _vp]),
    "dlm_norm_rows": (_ci, [_ci, _vp, _vp, _vp, _cf, _ci, _vp, _ci, _ci, _vp]),
    "dlm_gemv_act": (_ci, [_ci] + [_vp] * 4 + [_ci, _ci, _vp]),
    "dlm_add_norm_rows": (_ci, [_ci] + [_vp] * 4 + [_cf, _vp, _cf, _ci, _vp, _ci, _ci, _vp]),
    "dlm_head_decode_supported": (_ci, [_ci, _vp]),
    "dlm_head_prefill_supported": (_ci, [_ci, _vp]),
    "dlm_head_prepare": (_ci, [_ci] + [_vp] * 4),
    "dlm_head_prefill": (_ci, [_ci] + [_vp] * 4 + [_i64, _vp]),
    "dlm_head_decode": (_ci, [_ci] + [_vp] * 3 + [_ci] + [_vp] * 3),
    "dlm_head_merge": (_ci, [_ci, _vp, _vp, _ci] + [_vp] * 3 + [_i64, _vp]),
    "dlm_short_conv": (_ci, [_ci] + [_vp] * 3),
    "dlm_recurrence_steps": (_ci, [_ci] + [_vp] * 3),
    "dlm_recurrence_chunk_bytes": (_sz, [_vp]),
    "dlm_recurrence_chunks": (_ci, [_ci] + [_vp] * 4),
    "dlm_head_state_begin": (_ci, [_ci] + [_vp] * 6),
    "dlm_head_state_end": (_ci, [_ci, _vp, _vp, _ci] + [_vp] * 6 + [_ci, _ci, _cf, _vp, _vp]),
    "dlm_conv_products": (_ci, [_ci] + [_vp] * 5),
    "dlm_gated_norm": (_ci, [_ci, _vp, _vp, _vp, _i64, _vp, _i64] + [_ci] * 4 + [_cf, _vp]),
    "dlm_latent_decode_supported": (_ci, [_ci, _vp]),
    "dlm_latent_prefill_supported": (_ci, [_ci, _vp]),
    "dlm_latent_prepare": (_ci, [_ci, _vp, _vp, _vp]),
    "dlm_latent_prefill": (_ci, [_ci, _vp, _vp, _vp, _i64, _vp, _vp, _i64, _vp]),
    "dlm_latent_absorb": (_ci, [_ci] + [_vp] * 5),
    "dlm_latent_decode": (_ci, [_ci, _vp, _vp, _vp, _ci, _vp, _vp, _vp]),
    "dlm_latent_combine": (_ci, [_ci, _vp, _vp, _ci] + [_vp] * 5 + [_i64, _vp]),
}


class LibraryNotBuiltError(RuntimeError):
    pass


class W4A16Error(RuntimeError):
    """A C-ABI call returned a negative code."""

    library = "w4a16"

    def __init__(self, code, message):
        super().__init__(f"{self.library} error {code}: {message}")
        self.code = code


class DenseLmError(W4A16Error):
    """The same from libdense_lm_hip.so."""

    library = "dense_lm"


_lib = None
_dense = None


def library_path():
    return _LIB_PATH


def _bind(path, symbols):
    lib = ctypes.CDLL(path)
    for name, (restype, argtypes) in symbols.items():
        fn = getattr(lib, name)
        fn.restype = restype
        fn.argtypes = argtypes
    return lib


def load_dense_library():
    """Load the library of the dense-weight models; raises LibraryNotBuiltError when it is missing."""
    global _dense
    if _dense is None:
        if not os.path.exists(_DENSE_PATH):
            raise LibraryNotBuiltError(f"{_DENSE_PATH} is missing: build it with `python mlir-air_amd/build.py --only dense_lm` "
                                       "(there is no CPU fallback)")
        lib = _bind(_DENSE_PATH, DENSE_SYMBOLS)
        if lib.dlm_abi_version() != DENSE_ABI:
            raise LibraryNotBuiltError(f"{_DENSE_PATH}: ABI version {lib.dlm_abi_version()} != {DENSE_ABI}, rebuild")
        _dense = lib
    return _dense


def check_dense(code):
    """Raise DenseLmError for a negative return code of a dlm_ call."""
    if code != OK:
        lib = load_dense_library()
        msg = lib.dlm_strerror(code).decode()
        if code == ERR_HIP:
            msg += ": " + lib.dlm_last_hip_error().decode()
        raise DenseLmError(code, msg)


def load_library():
    """Load the HIP library; raises LibraryNotBuiltError when it is missing."""
    global _lib
    if _lib is not None:
        return _lib
    if not os.path.exists(_LIB_PATH):
        raise LibraryNotBuiltError(
            f"{_LIB_PATH} is missing: build it with `python mlir-air_amd/build.py` "
            "(there is no CPU fallback for the W4A16 kernels)"
        )
    lib = _bind(_LIB_PATH, SYMBOLS)
    if lib.w4a16_abi_version() != 1:
        raise LibraryNotBuiltError(f"{_LIB_PATH}: ABI version {lib.w4a16_abi_version()} != 1, rebuild")
    _lib = lib
    return lib


def check(code):
    """Raise W4A16Error for a negative return code."""
    if code != OK:
        lib = load_library()
        msg = lib.w4a16_strerror(code).decode()
        if code == ERR_HIP:
            msg += ": " + lib.w4a16_last_hip_error().decode()
        raise W4A16Error(code, msg)
