"""ctypes binding of the libraries in ``csrc/`` (the C ABI in ``include/a81w41.h`` and ``include/a81w41_model.h``).

``lib()`` is the A81W41 layer with the Qwen3 model, ``core()`` what all models share.  A library is loaded from the source tree; if it has not been built the call
fails with instructions -- there is no fallback path.
"""
from __future__ import annotations

import ctypes as C
import os

_HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(_HERE, "csrc")
LIB_PATH = os.path.join(CSRC, "liba81w41.so")
DENSE_PATH = os.path.join(CSRC, "liba81w41_dense.so")
CORE_PATH = os.path.join(CSRC, "liba81w41_core.so")

OK = 0
ERR_UNSUPPORTED = 5
_vp, _i, _i64, _sz = C.c_void_p, C.c_int, C.c_int64, C.c_size_t

# name -> (restype, argtypes): every symbol include/a81w41.h declares
SIGNATURES = {
    "a81w41_status_string": (C.c_char_p, [_i]),
    "a81w41_last_error": (C.c_char_p, []),
    "a81w41_weight_blob_bytes": (_sz, [_i, _i, _i]),
    "a81w41_act_blob_bytes": (_sz, [_i64, _i]),
    "a81w41_repack_w81_weight_fp16": (_i, [_i, _i, _i, _vp, _vp, _vp, _vp]),
    "a81w41_repack_w81_weight_fp32": (_i, [_i, _i, _i, _vp, _vp, _vp, _vp]),
    "a81w41_quantize_weight_q41": (_i, [_vp, _i, _i, _vp, _vp, _vp]),
    "a81w41_quantize_row_q8_1_repack_fp16": (_i, [_vp, _vp, _i64, _vp]),
    "a81w41_quantize_row_q8_1_repack_fp32": (_i, [_vp, _vp, _i64, _vp]),
    "a81w41_gemv_repack_A81W41_fp16": (_i, [_vp, _vp, _vp, _i, _i, _i, _vp]),
    "a81w41_gemm_repack_A81W41_fp32": (_i, [_vp, _vp, _vp, _i, _i, _i, _vp]),
    "a81w41_gemm_repack_A81W41_fp32_static": (_i, [_vp, _vp, _vp, _i, _i, _i, _vp]),
    "a81w41_gemm_schedule_selfcheck": (_i, [_i, _i, _i, _i, _i]),
    "a81w41_gemm_fp6_plan_selfcheck": (_i, [_i, _i, _i, _i]),
    "a81w41_block_idot": (_i, [_vp, _i, _vp, _i, _vp, _i, _i, _i, _vp]),
    "a81w41_repack_w80_weight": (_i, [_i, _i, _i, _vp, _vp, _vp]),
    "a81w41_quantize_weight_q40": (_i, [_vp, _i, _i, _vp, _vp]),
    "a81w41_quantize_row_q8_0_repack": (_i, [_vp, _vp, _i64, _vp]),
    "a81w41_gemv_repack_A80W40": (_i, [_vp, _vp, _vp, _i, _i, _i, _vp]),
    "a81w41_gemm_repack_A80W40_workspace_bytes": (_sz, [_i, _i, _i]),
    "a81w41_gemm_repack_A80W40": (_i, [_vp, _vp, _vp, _i, _i, _i, _vp, _sz, _vp]),
    "a81w41_block_idot_A80W40": (_i, [_vp, _vp, _vp, _i, _i, _i, _vp]),
    "a81w41_context_create": (_i, [_i, _i, C.POINTER(_vp)]),
    "a81w41_context_destroy": (None, [_vp]),
    "a81w41_context_activation_scratch_dev": (_vp, [_vp]),
    "a81w41_linear_create": (_i, [_vp, _i, _i, _vp, _vp, _vp, C.POINTER(_vp)]),
    "a81w41_linear_create_from_blobs": (_i, [_vp, _i, _i, _vp, _vp, C.POINTER(_vp)]),
    "a81w41_linear_load": (_i, [_vp, C.c_char_p, _i, _i, _i, C.POINTER(_vp)]),
    "a81w41_linear_destroy": (None, [_vp]),
    "a81w41_linear_resident_bytes": (_sz, [_vp, C.POINTER(_sz), C.POINTER(_sz), C.POINTER(_sz)]),
    "a81w41_linear_kernel_name": (C.c_char_p, [_vp, _i]),
    "a81w41_linear_in_features": (_i, [_vp]),
    "a81w41_linear_out_features": (_i, [_vp]),
    "a81w41_linear_weight_fp16_dev": (_vp, [_vp]),
    "a81w41_linear_weight_fp32_dev": (_vp, [_vp]),
    "a81w41_linear_forward": (_i, [_vp, _vp, _i, _vp, _vp]),
    "a81w41_linear_forward_quantized": (_i, [_vp, _vp, _i, _vp, _vp]),
    "a81w41_linear_set_kernel": (_i, [_vp, _i]),
    "a81w41_linear_forward_multi": (_i, [_i, C.POINTER(_vp), _vp, _i, C.POINTER(_vp), _vp]),
    "a81w41_linear_forward_host": (_i, [_vp, _vp, _i, _vp]),
    "a81w41_context_chain_begin": (_i, [_vp, _vp]),
    "a81w41_context_chain_end": (_i, [_vp]),
    "a81w41_context_chain_status": (_i, [_vp, C.POINTER(_i)]),
    "a81w41_context_chain_set_spin_limit": (_i, [_vp, C.c_uint]),
    "a81w41_context_chain_selfcheck_stuck_wait": (_i, [_vp, _vp, _vp, C.c_uint, _vp]),
    "a81w41_qwen3_create": (_i, [_vp, C.POINTER(_vp)]),
    "a81w41_qwen3_load": (_i, [C.c_char_p, _vp, C.POINTER(_vp)]),
    "a81w41_qwen3_destroy": (None, [_vp]),
    "a81w41_qwen3_set_linear": (_i, [_vp, _i, _i, _vp, _vp, _vp]),
    "a81w41_qwen3_set_linear_blobs": (_i, [_vp, _i, _i, _vp, _vp]),
    "a81w41_qwen3_set_norm": (_i, [_vp, _i, _i, _vp]),
    "a81w41_qwen3_set_embedding": (_i, [_vp, _vp]),
    "a81w41_qwen3_set_option": (_i, [_vp, _i, _i]),
    "a81w41_qwen3_chain_status": (_i, [_vp, C.POINTER(_i)]),
    "a81w41_qwen3_resident_bytes": (_sz, [_vp, C.POINTER(_sz), C.POINTER(_sz), C.POINTER(_sz), C.POINTER(_sz)]),
    "a81w41_qwen3_read_buffer": (_i, [_vp, _i, _vp, _sz]),
    "a81w41_qwen3_reset": (_i, [_vp]),
    "a81w41_qwen3_forward": (_i, [_vp, _vp, _i, _vp]),
    "a81w41_qwen3_attention": (_i, [_vp, _i, _vp, _vp, _vp, _vp, _i, _i, _i, _i, _i, C.c_float, _i, _vp]),
    "a81w41_qwen3_attention_one_token": (_i, [_vp, _i, _i, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _i, C.c_float, C.c_float,
                                              _i, _vp]),
    "a81w41_qwen3_generate_greedy": (_i, [_vp, _vp, _i, _i, _vp, C.POINTER(C.c_double), C.POINTER(C.c_double)]),
}

# every symbol include/a81w41_model.h declares, and the status functions
CORE_SIGNATURES = {
    "a81w41_status_string": (C.c_char_p, [_i]),
    "a81w41_last_error": (C.c_char_p, []),
    "a81w41_model_load": (_i, [C.c_char_p, C.c_char_p, _i, C.POINTER(_vp)]),
    "a81w41_model_create_random": (_i, [C.c_char_p, C.c_char_p, _i, C.c_uint64, C.POINTER(_vp)]),
    "a81w41_model_destroy": (None, [_vp]),
    "a81w41_model_vocab": (_i, [_vp]),
    "a81w41_model_max_seq": (_i, [_vp]),
    "a81w41_model_position": (_i, [_vp]),
    "a81w41_model_reset": (_i, [_vp]),
    "a81w41_model_forward": (_i, [_vp, _vp, _i, _vp, _i, _vp]),
    "a81w41_model_generate_greedy": (_i, [_vp, _vp, _i, _i, _vp, C.POINTER(C.c_double), C.POINTER(C.c_double)]),
    "a81w41_model_set_option": (_i, [_vp, C.c_char_p, _i]),
    "a81w41_model_read_buffer": (_i, [_vp, C.c_char_p, _vp, _sz]),
    "a81w41_model_resident_bytes": (_sz, [_vp, C.POINTER(_sz), C.POINTER(_sz)]),
}

# every symbol include/a81w41_dense.h declares
DENSE_SIGNATURES = {
    "a81w41_dense_gemm": (_i, [_vp, _i, _vp, _i, _vp, _i, _i, _i, _i, _i, _vp]),
    "a81w41_latent_attention": (_i, [_vp, _vp, _i, _i, _i, _i, _vp, _i, _i, C.c_float, _vp, _i, _i, _i, _vp, _vp, _vp]),
    "a81w41_formed_attention": (_i, [_vp, _vp, _vp, _i, _vp, _i, _vp, _i, _i, _i, _i, _vp, _i, _i, C.c_float, _vp, _vp]),
    "a81w41_grouped_attention": (_i, [_vp, _vp, _i, _i, _i, _i, _i, _i, _vp, _i, _i, C.c_float, _i, _i, _vp, _i, _i, _i, _vp, _vp, _vp]),
    "a81w41_matrix_memory_state": (_sz, [_i, _i, _i]),
    "a81w41_matrix_memory_scratch": (_sz, [_i, _i, _i, _i]),
    "a81w41_matrix_memory": (_i, [_vp, _i, _i, _i, _i, _i, C.c_float, C.c_float, _vp, _vp, _vp, _vp, _vp, _i, _vp, _vp, _vp]),
    "a81w41_router": (_i, [_vp, _i, _vp, _i, _i, _i, _vp, _vp, _vp]),
}


class Qwen3Config(C.Structure):
    """a81w41_qwen3_config"""
    _fields_ = [("n_layers", _i), ("hidden", _i), ("n_q_heads", _i), ("n_kv_heads", _i), ("intermediate", _i),
                ("vocab", _i), ("max_seq", _i), ("rope_theta", C.c_float), ("rms_eps", C.c_float)]

_libs = {}


class A81W41Error(RuntimeError):
    def __init__(self, status: int, message: str):
        super().__init__(f"a81w41 status {status}: {message}")
        self.status = status


def load(path: str, signatures: dict):
    """Load a library of ``csrc/`` (once) and bind the named symbols."""
    if path not in _libs:
        if not os.path.exists(path):
            raise ImportError(
                f"{path} is missing: build it with `make -C {CSRC}` "
                "(or __graft_entry__.build()); this package has no CPU fallback")
        L = C.CDLL(path)
        for name, (res, args) in signatures.items():
            fn = getattr(L, name)  # AttributeError if the library lacks a declared symbol
            fn.restype = res
            fn.argtypes = args
        _libs[path] = L
    return _libs[path]


def lib():
    """The A81W41 layer and the Qwen3 model, every exported symbol bound."""
    return load(LIB_PATH, SIGNATURES)


def dense():
    """The models with dense weights and their parity hooks."""
    return load(DENSE_PATH, DENSE_SIGNATURES)


def core():
    """The model interface; a model's own library registers with it when it is loaded."""
    return load(CORE_PATH, CORE_SIGNATURES)


def check(status: int) -> None:
    if status != OK:
        raise A81W41Error(status, core().a81w41_last_error().decode())
