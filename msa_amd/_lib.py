"""ctypes binding of the C ABIs declared in ``include/msa_amd.h`` and ``include/msa_seq.h``.

There is no fallback: if the HIP library is missing or a call fails, an exception is raised.
"""
from __future__ import annotations

import ctypes as C
import os
from typing import Optional

HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.environ.get("MSA_AMD_LIB", os.path.join(HERE, "libmsa_amd.so"))   # override: an alternative build

SEQ_LIB_PATH = os.path.join(HERE, "libmsa_seq.so")

MSA_BF16, MSA_F32 = 0, 1
MODE_COSINE, MODE_SCALED_DOT = 0, 1

_vp, _i32, _i64, _f32, _sz = C.c_void_p, C.c_int32, C.c_int64, C.c_float, C.c_size_t

# name -> (restype, argtypes); mirrors include/msa_amd.h one to one
SIGNATURES = {
    "msa_last_error": (C.c_char_p, []),
    "msa_abi_version": (C.c_int, []),
    "msa_chunk_table": (C.c_int, [_vp, _i32, _i32, _i64, _vp, _vp, _vp, _vp, _vp, _vp]),
    "msa_pool_chunks": (C.c_int, [_vp, _vp, _vp, _i32, _i64, _i32, _i32, _vp, _vp, _vp, _i64, _vp, _vp, _vp, _i32,
                                  _i32, _i32, _vp, _vp, _vp, _vp]),
    "msa_bank_create": (C.c_int, [C.POINTER(_vp), _i32, _i64, _i32, _i32, _i32, _vp, _vp, _i64]),
    "msa_bank_set_layer": (C.c_int, [_vp, _i32, _vp, _vp, _vp]),
    "msa_bank_destroy": (C.c_int, [_vp]),
    "msa_route_workspace_bytes": (_sz, [_i32, _i32, _i32, _i32, _i32, _i64, _i64, _i32]),
    "msa_route_topk_workspace_bytes": (_sz, [_i32, _i32, _i32, _i32, _i32, _i64, _i32]),
    "msa_chunk_scores": (C.c_int, [_vp, _i32, _vp, _vp, _i32, _i32, _i32, _i32, _f32, _vp, _vp, _sz, _vp]),
    "msa_route_topk": (C.c_int, [_vp, _i32, _vp, _vp, _i32, _i32, _i32, _i32, _f32, _i32, _vp, _vp, _vp, _vp, _sz,
                                 _vp]),
    "msa_route_topk_reduce": (C.c_int, [_vp, _i32, _vp, _vp, _i32, _i32, _i32, _i32, _f32, _i32, _i32, _i32, _vp, _vp, _vp,
                                        _vp, _sz, _vp]),
    "msa_route_topk_static": (C.c_int, [_vp, _i32, _vp, _vp, _i32, _i32, _i32, _i32, _f32, _i32, _vp, _vp, _vp, _vp]),
    "msa_profile_enable": (C.c_int, [_i32]),
    "msa_profile_collect": (C.c_int, [_vp, _i32, _vp]),
    "msa_diag_mfma_loop": (C.c_int, [_i32, _i32, _i32, _vp, _vp, _vp]),
    "msa_diag_fill_lds": (C.c_int, [C.c_uint32, _vp, _i32, _vp]),
    "msa_diag_read_stream": (C.c_int, [_vp, C.c_int64, _vp, _i32, _vp]),
    "msa_diag_scan_walk": (C.c_int, [_i32, _i32, _i32, _i32, _i32, _vp]),
    "msa_route_set_tile_pool": (C.c_int, [_i32]),
    "msa_gather_plan": (C.c_int, [_vp, _vp, _i32, _i32, _vp]),
    "msa_gather_kv": (C.c_int, [_vp, _i32, _vp, _i32, _i32, _vp, _vp, _i64, _vp]),
    "msa_gather_device_workspace_bytes": (_sz, [_i32, _i32]),
    "msa_gather_kv_device": (C.c_int, [_vp, _i32, _vp, _i32, _i32, _vp, _vp, _i64, _vp, _vp, _sz, _vp]),
    "msa_route_topk_gather": (C.c_int, [_vp, _i32, _vp, _vp, _i32, _i32, _i32, _i32, _f32, _i32, _vp, _vp, _vp, _vp, _sz,
                                        _i32, _vp, _i32, _i32, _vp, _vp, _i64, _vp, _vp, _sz, _vp]),
    "msa_assemble_context": (C.c_int, [_vp, _vp, _i32, _vp, _vp, _vp, _vp, _vp, _vp, _i32, _i32, _i32, _i32, _vp,
                                       _vp, _i32, _vp, _vp]),
    "msa_cache_append": (C.c_int, [_vp, _vp, _i32, _i32, _i32, _i32, _vp, _vp, _i32, _vp, _vp]),
    "msa_cache_append_rows": (C.c_int, [_vp, _vp, _vp, _i32, _i32, _i32, _i32, _i32, _vp, _vp, _i32, _vp, _vp]),
    "msa_attn_workspace_bytes": (_sz, [_i32, _i32, _i32, _i32, _i32]),
    "msa_flash_attn": (C.c_int, [_vp, _vp, _vp, _vp, _vp, _vp, _i32, _i32, _i32, _i32, _i32, _f32, _i32, _vp, _vp]),
    "msa_flash_set_form": (C.c_int, [_i32]),
    "msa_diag_asm_kernel_resources": (C.c_int, [_i32, _vp, _vp]),
    "msa_flash_attn_hint": (C.c_int, [_vp, _vp, _vp, _vp, _vp, _vp, _i32, _i32, _i32, _i32, _i32, _f32, _i32, _vp, _i32, _vp]),
    "msa_qk_norm_rope": (C.c_int, [_vp, _vp, _vp, _i64, _i64, _i64, _vp, _vp, _vp, _f32, _vp, _vp, _i32, _i32, _i64, _i32,
                                   _i32, _i32, _vp, _vp, _vp, _vp]),
    "msa_qkv_proj": (C.c_int, [_vp, _i64, _i32, _vp, _i32, _i32, _i32, _i32, _vp, _vp, _vp, _f32, _vp, _vp, _i32, _vp, _vp, _vp,
                               _vp, _vp]),
    "msa_qk_norm_rope_append": (C.c_int, [_vp, _vp, _vp, _i64, _i64, _i64, _vp, _vp, _vp, _f32, _vp, _vp, _i32, _i32, _i32,
                                          _i32, _i32, _i32, _vp, _vp, _vp, _i32, _vp, _vp]),
    "msa_rmsnorm": (C.c_int, [_vp, _vp, _vp, _i32, _i64, _i32, _f32, _vp, _vp]),
    "msa_silu_mul": (C.c_int, [_vp, _i32, _i64, _i32, _vp, _vp]),
    "msa_decode_attn_fused": (C.c_int, [_vp, _i64, _vp, _vp, _vp, _f32, _vp, _vp, _i32, _i32, _i32, _i32, _i32, _vp, _vp,
                                        _i32, _vp, _f32, _vp, _vp, _sz, _vp]),
    "msa_greedy_sample": (C.c_int, [_vp, _i32, _i32, _i64, _vp, _vp, _vp, _vp, _i64, _vp, _i32, _vp]),
    "msa_skinny_linear": (C.c_int, [_vp, _vp, _vp, _vp, _f32, _i32, _i32, _i32, _i32, _i32, _vp, _vp]),
    "msa_skinny_linear_workspace_bytes": (_sz, [_i32, _i32, _i32]),
    "msa_skinny_linear_ws": (C.c_int, [_vp, _vp, _vp, _vp, _f32, _i32, _i32, _i32, _i32, _i32, _vp, _vp, _sz, _vp]),
    "msa_sparse_attn": (C.c_int, [_vp, _vp, _vp, _vp, _vp, _vp, _i32, _i32, _i32, _i32, _i32, _i32, _i32, _i32, _f32,
                                  _i32, _vp, _vp, _sz, _vp]),
}


class SeqBatch(C.Structure):
    """``msa_seq_batch``."""
    _fields_ = [("cu", _vp), ("row_seq", _vp), ("slot", _vp), ("pos", _vp), ("n_seq", _i32), ("rows", _i32),
                ("max_rows", _i32), ("reserved", _i32)]


class DynTanh(C.Structure):
    """``msa_dyn_tanh``."""
    _fields_ = [("w", _vp), ("b", _vp), ("alpha", _f32), ("reserved", _i32)]


class RowsArgs(C.Structure):
    """``msa_rows_args``."""
    _fields_ = [("x", _vp), ("x_b", _vp), ("w", _vp), ("out", _vp), ("x_stride", _i64), ("x_b_stride", _i64),
                ("out_stride", _i64), ("M", _i32), ("N", _i32), ("K", _i32), ("groups", _i32), ("n_b", _i32), ("gelu_n", _i32),
                ("cap", _f32), ("reserved", _i32), ("add", _vp),
                ("x_in", _vp), ("x_out", _vp), ("gate", _vp), ("gate_stride", _i64), ("gate_bias", _vp), ("norm", DynTanh),
                ("h", _vp), ("shift", _vp), ("prev", _vp), ("h_shift", _vp),
                ("taps", _vp), ("conv_bias", _vp), ("conv_state", _vp), ("conv_lo", _i32), ("conv_n", _i32), ("conv_k", _i32),
                ("reserved2", _i32),
                ("z_bias", _vp), ("u_bias", _vp), ("gru_state", _vp), ("out2", _vp), ("gru_n", _i32), ("reserved3", _i32),
                ("slot", _vp), ("glu_limit", _f32), ("glu_alpha", _f32), ("glu_shift", _f32), ("reserved4", _i32)]


class QKRopeArgs(C.Structure):
    """``msa_qk_rope_args``."""
    _fields_ = [("q", _vp), ("k", _vp), ("v", _vp), ("q_stride", _i64), ("k_stride", _i64), ("v_stride", _i64), ("q_norm", _vp),
                ("k_norm", _vp), ("freqs", _vp), ("q_out", _vp), ("k_cache", _vp), ("v_cache", _vp), ("Lcap", _i64), ("H", _i32),
                ("G", _i32), ("D", _i32), ("E", _i32), ("n_pairs", _i32), ("eps", _f32)]


class KVAttnArgs(C.Structure):
    """``msa_kv_attn_args``."""
    _fields_ = [("q", _vp), ("k_cache", _vp), ("v_cache", _vp), ("gate", _vp), ("out", _vp), ("Lcap", _i64), ("gate_stride", _i64),
                ("max_keys", _i64), ("H", _i32), ("G", _i32), ("D", _i32), ("E", _i32), ("chunk", _i32), ("scale", _f32)]


class DeltaArgs(C.Structure):
    """``msa_delta_args``."""
    _fields_ = [("qkv", _vp), ("a", _vp), ("b", _vp), ("gate", _vp), ("qkv_stride", _i64), ("a_stride", _i64), ("b_stride", _i64),
                ("gate_stride", _i64), ("A_log", _vp), ("dt_bias", _vp), ("norm", _vp), ("state", _vp), ("out", _vp), ("H", _i32),
                ("G", _i32), ("D", _i32), ("E", _i32), ("eps", _f32), ("reserved", _i32)]


ROWS_PLAIN, ROWS_F32, ROWS_RESIDUAL, ROWS_MAMBA, ROWS_GRU, ROWS_GLU = range(6)
_batch = C.POINTER(SeqBatch)

# include/msa_seq.h
SEQ_SIGNATURES = {
    "msa_seq_residual_norm": (C.c_int, [_vp, _vp, _i64, _vp, _i64, _vp, _vp, _i32, _i32, C.POINTER(DynTanh), _vp, _vp, _vp, _vp,
                                        _batch, _vp]),
    "msa_seq_gelu": (C.c_int, [_vp, _i64, _i32, _i32, _i32, _vp]),
    "msa_seq_softcap": (C.c_int, [_vp, _i32, _i64, _f32, _vp, _vp]),
    "msa_seq_join": (C.c_int, [_vp, _vp, _i32, _i32, _i32, _vp, _vp]),
    "msa_seq_conv_silu": (C.c_int, [_vp, _i64, _vp, _vp, _i32, _i32, _i32, _vp, _vp, _i64, _batch, _vp]),
    "msa_seq_ssd_scan": (C.c_int, [_vp, _i64, _vp, _i64, _vp, _i64, _vp, _vp, _vp, _i32, _i32, _i32, _i32, _i32, _vp, _vp, _batch,
                                   _vp]),
    "msa_seq_ssd_chunked_workspace_bytes": (_sz, [_i32, _i32, _i32, _i32, _i32]),
    "msa_seq_ssd_chunked": (C.c_int, [_vp, _i64, _vp, _i64, _vp, _i64, _vp, _vp, _vp, _i32, _i32, _i32, _i32, _i32, _vp, _vp, _batch,
                                      _vp, _sz, _vp]),
    "msa_seq_group_rmsnorm": (C.c_int, [_vp, _i32, _i32, _i32, _i32, _vp, _f32, _vp, _vp]),
    "msa_seq_min_gru_workspace_bytes": (_sz, [_i32, _i32, _i32, _i32]),
    "msa_seq_min_gru": (C.c_int, [_vp, _i64, _vp, _vp, _i32, _i32, _vp, _vp, _batch, _vp, _sz, _vp]),
    "msa_seq_latent_append": (C.c_int, [_vp, _i64, _vp, _f32, _i32, _i32, _vp, _i64, _batch, _vp]),
    "msa_seq_latent_attn": (C.c_int, [_vp, _vp, _i64, _vp, _f32, _i32, _i32, _i32, _vp, _batch, _vp]),
    "msa_seq_latent_decode_workspace_bytes": (_sz, [_i32, _i32, _i32, _i64]),
    "msa_seq_latent_decode": (C.c_int, [_vp, _vp, _i64, _vp, _f32, _i32, _i32, _i32, _i64, _vp, _batch, _vp, _sz, _vp]),
    "msa_seq_flash": (C.c_int, [_vp, _i64, _vp, _i64, _vp, _i64, _vp, _vp, _f32, _i32, _i32, _i32, _i32, _i32, _i32, _vp, _i64, _vp,
                                _batch, _vp]),
    "msa_seq_qk_rope_append": (C.c_int, [C.POINTER(QKRopeArgs), _i32, _batch, _vp]),
    "msa_seq_kv_attn": (C.c_int, [C.POINTER(KVAttnArgs), _i32, _batch, _vp]),
    "msa_seq_kv_decode_workspace_bytes": (_sz, [C.POINTER(KVAttnArgs), _i32]),
    "msa_seq_kv_decode": (C.c_int, [C.POINTER(KVAttnArgs), _batch, _vp, _sz, _vp]),
    "msa_seq_delta_scan": (C.c_int, [C.POINTER(DeltaArgs), _i32, _batch, _vp]),
    "msa_seq_delta_chunked_workspace_bytes": (_sz, [C.POINTER(DeltaArgs), _i32, _i32]),
    "msa_seq_delta_chunked": (C.c_int, [C.POINTER(DeltaArgs), _batch, _vp, _sz, _vp]),
    "msa_seq_head_norm_gate": (C.c_int, [_vp, _vp, _i64, _vp, _f32, _i32, _i32, _i32, _i32, _vp]),
    "msa_seq_rms_residual": (C.c_int, [_vp, _vp, _i64, _vp, _f32, _vp, _vp, _vp, _i32, _i32, _i32, _vp]),
    "msa_seq_clamped_glu": (C.c_int, [_vp, _i64, _i32, _i32, _i32, _f32, _f32, _f32, _vp, _vp]),
    "msa_rows_linear": (C.c_int, [C.POINTER(RowsArgs), _i32, _vp]),
}
# entry points of include/msa_amd.h that libmsa_seq.so holds too (the error text is per library)
SEQ_SHARED = ("msa_last_error", "msa_abi_version", "msa_greedy_sample")


class MsaError(RuntimeError):
    def __init__(self, code: int, where: str, message: str):
        super().__init__(f"{where} failed with code {code}: {message}")
        self.code = code


_libs = {}


def _open(path: str, table) -> C.CDLL:
    if path in _libs:
        return _libs[path]
    if not os.path.exists(path):
        raise ImportError(f"{path} is missing: build it with `python -m msa_amd.build` "
                          "(there is no CPU or PyTorch fallback for this path)")
    lib = C.CDLL(path)
    for name, (res, args) in table.items():
        fn = getattr(lib, name)          # AttributeError if the library lacks a declared symbol
        fn.restype, fn.argtypes = res, args
    _libs[path] = lib
    return lib


def load() -> C.CDLL:
    """Loads the library and declares every entry point; raises if it is missing."""
    return _open(LIB_PATH, SIGNATURES)


def load_seq() -> C.CDLL:
    """The same for the library of the recurrent / latent-attention layers."""
    return _open(SEQ_LIB_PATH, {**SEQ_SIGNATURES, **{n: SIGNATURES[n] for n in SEQ_SHARED}})


def check(code: int, where: str, lib: Optional[C.CDLL] = None) -> None:
    if code != 0:
        raise MsaError(code, where, (lib or load()).msa_last_error().decode("utf-8", "replace"))


def ptr(t) -> Optional[int]:
    """Device/host address of a torch tensor (None passes NULL)."""
    return None if t is None else t.data_ptr()


def dtype_code(torch_dtype) -> int:
    import torch
    if torch_dtype == torch.bfloat16:
        return MSA_BF16
    if torch_dtype == torch.float32:
        return MSA_F32
    raise TypeError(f"unsupported dtype {torch_dtype}: the kernels take bfloat16 or float32")
