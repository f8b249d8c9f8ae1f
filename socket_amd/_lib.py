"""ctypes binding of libsocket_hip.so and of libsocket_core.so, which it depends on
(the C ABI declared in include/socket_hip.h).

There is no CPU route: importing works anywhere (so the package can be
inspected and the library's exports checked without a GPU), but the library
must be present, and any compute call needs a HIP device.  A missing library
raises at first use with the build command to run.
"""
from __future__ import annotations

import ctypes
import os
from ctypes import c_char_p, c_float, c_int, c_int64, c_size_t, c_void_p, POINTER

import torch

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(_HERE, "libsocket_hip.so")
CORE_PATH = os.path.join(_HERE, "libsocket_core.so")

SOCKET_OK = 0
SOCKET_ERR_NULL = -1
SOCKET_ERR_SHAPE = -2
SOCKET_ERR_UNSUPPORTED = -3
SOCKET_ERR_ALIGN = -4
SOCKET_ERR_WORKSPACE = -5
SOCKET_ERR_LAUNCH = -6

SOCKET_F32, SOCKET_BF16, SOCKET_F16 = 0, 1, 2
SOCKET_TOPK_MAX_M = 16384

_DTYPE_ENUM = {torch.float32: SOCKET_F32, torch.bfloat16: SOCKET_BF16, torch.float16: SOCKET_F16}

_P, _I, _L, _Z = c_void_p, c_int, c_int64, c_size_t
_F = c_float


class DepthMix(ctypes.Structure):
    """socket_depth_mix"""
    _fields_ = [("past", _P), ("past_stride", _L), ("w", _P), ("n", _I), ("result", _P)]


class Residual(ctypes.Structure):
    """socket_residual"""
    _fields_ = [("x", _P), ("embed", _P), ("ids", _P), ("ids64", _I), ("vocab", _I), ("a", _P), ("b", _P),
                ("scale_a", _F), ("scale_b", _F), ("pending_f32", _I), ("post_w", _P), ("pre_w", _P), ("eps", _F),
                ("dtype", _I), ("dim", _I), ("x_out", _P), ("h_out", _P), ("embed_scale", _F), ("x_stride", _L),
                ("depth", DepthMix)]


class RowsLinear(ctypes.Structure):
    """socket_rows_linear"""
    _fields_ = [("norm", POINTER(Residual)), ("x1", _P), ("x2", _P), ("w1", _P), ("w2", _P), ("s1", _F), ("s2", _F),
                ("K1", _I), ("K2", _I), ("kind", _I), ("limit", _F), ("y", _P), ("y_f32", _I), ("M", _I), ("N", _I),
                ("b1", _P), ("b2", _P), ("res", _P), ("depth", DepthMix)]


class RopeHalf(ctypes.Structure):
    """socket_rope_half"""
    _fields_ = [("proj", _P), ("dtype", _I), ("proj_stride_b", _L), ("proj_stride_t", _L), ("q_off", _I), ("k_off", _I),
                ("H", _I), ("G", _I), ("D", _I), ("rot_dims", _I), ("cos_sin", _P), ("n_pos", _L), ("pos0", _L),
                ("pos", _P), ("q_out", _P), ("q_pitch", _I), ("k_out", _P), ("k_ring", _P), ("v_ring", _P),
                ("ring_stride_b", _L), ("ring_stride_g", _L), ("ring_stride_s", _L), ("chunk", _I), ("ring_len", _P),
                ("B", _I), ("T", _I)]


class ChunkAttention(ctypes.Structure):
    """socket_chunk_attention"""
    _fields_ = [("q", _P), ("q_stride_b", _L), ("q_stride_t", _L), ("q_stride_h", _L),
                ("k_new", _P), ("k_stride_b", _L), ("k_stride_t", _L), ("k_stride_g", _L),
                ("v_new", _P), ("v_stride_b", _L), ("v_stride_t", _L), ("v_stride_g", _L),
                ("k_ring", _P), ("v_ring", _P), ("ring_stride_b", _L), ("ring_stride_g", _L), ("ring_stride_s", _L),
                ("dtype", _I), ("B", _I), ("T", _I), ("H", _I), ("G", _I), ("D", _I), ("chunk", _I), ("pos0", _L),
                ("pos", _P), ("scale", _F), ("softcap", _F), ("out", _P), ("force_simple", _I),
                ("Dv", _I), ("k_from", _L), ("k2", _P), ("k2_stride_b", _L), ("k2_stride_t", _L), ("D2", _I),
                ("gate", _P), ("gate_stride_b", _L), ("gate_stride_t", _L)]


class Recurrence(ctypes.Structure):
    """socket_recurrence"""
    _fields_ = [("dtype", _I), ("B", _I), ("T", _I), ("H", _I), ("Hk", _I), ("dk", _I), ("dv", _I),
                ("proj", _P), ("proj_stride_b", _L), ("proj_stride_t", _L),
                ("q_off", _I), ("k_off", _I), ("v_off", _I), ("beta_off", _I), ("decay_off", _I), ("gate_off", _I),
                ("taps", _I), ("conv_w", _P), ("conv_state", _P), ("unit_qk", _I), ("q_scale", _F),
                ("decay_kind", _I), ("a_log", _P), ("decay_bias", _P), ("inv_tau", _F),
                ("decay_w", _P), ("decay_rank", _I), ("decay_z", _P), ("decay_z_f32", _I),
                ("gate_kind", _I), ("gate_w", _P), ("gate_rank", _I), ("gate_z", _P), ("norm_w", _P), ("eps", _F),
                ("state", _P), ("fresh", _I), ("pos", _P), ("pos0", _L), ("t0", _I), ("n", _I), ("o_buf", _P),
                ("workspace", _P), ("workspace_bytes", _Z), ("out", _P),
                ("rule", _I), ("rate_off", _I), ("rate_bias", _P), ("decay_tanh", _I), ("decay_rate", _F),
                ("norm_per_head", _I)]


class Latent(ctypes.Structure):
    """socket_latent"""
    _fields_ = [("dtype", _I), ("B", _I), ("T", _I), ("H", _I), ("dim", _I), ("rot", _I), ("q_rank", _I), ("rank", _I),
                ("in_", _P), ("in_f32", _I), ("in_stride_b", _L), ("in_stride_t", _L),
                ("cq_off", _I), ("c_off", _I), ("rot_off", _I), ("q_norm", _P), ("c_norm", _P), ("eps", _F),
                ("cos_sin", _P), ("n_pos", _L), ("pos0", _L), ("pos", _P),
                ("cache", _P), ("cache_stride_b", _L), ("cache_stride_t", _L), ("cq_out", _P), ("append", _I),
                ("q", _P), ("w_uk", _P), ("q_lat", _P)]


class LatentAttend(ctypes.Structure):
    """socket_latent_attention"""
    _fields_ = [("dtype", _I), ("B", _I), ("T", _I), ("H", _I), ("rank", _I), ("rot", _I), ("vdim", _I),
                ("q_lat", _P), ("cache", _P), ("cache_stride_b", _L), ("cache_stride_t", _L), ("n_pos", _L), ("pos0", _L),
                ("pos", _P), ("scale", _F), ("splits", _I), ("o", _P), ("ml", _P),
                ("w_uv", _P), ("gate", _P), ("gate_f32", _I), ("gate_stride_b", _L), ("gate_stride_t", _L), ("out", _P)]


# name -> (restype, argtypes); one entry per declaration in include/socket_hip.h.
# What libsocket_core.so exports:
CORE_SIGNATURES = {
    "socket_residual_norm": (_I, [POINTER(Residual), _L, _P]),
    "socket_rows_linear_bf16": (_I, [POINTER(RowsLinear), _P]),
    "socket_gated_unit": (_I, [_P, _P, _I, _L, _I, _I, _F, _P]),
    "socket_rope_half_rows": (_I, [POINTER(RopeHalf), _P]),
    "socket_chunk_ring_store": (_I, [_P, _L, _L, _L, _P, _L, _L, _L, _P, _P, _L, _L, _L, _I, _I, _I, _I, _I, _I, _L, _P]),
    "socket_chunk_attend": (_I, [POINTER(ChunkAttention), _P]),
    "socket_dense_decode_capped_workspace_bytes": (_Z, [_I, _I, _I]),
    "socket_dense_decode_capped": (_I, [_P, _P, _P, _I] + [_L] * 8 + [_P, _P, _L, _L, _P, _Z, _I, _I, _I, _I, _I, _F, _F, _P]),
    "socket_recurrence_step": (_I, [POINTER(Recurrence), _P]),
    "socket_recurrence_chunk": (_I, [_I, _I]),
    "socket_recurrence_workspace_bytes": (_Z, [_I, _I, _I, _I, _I, _I]),
    "socket_tanh_rows": (_I, [_P, _L, _P, _I, _L, _I, _P]),
    "socket_latent_rows": (_I, [POINTER(Latent), _P]),
    "socket_latent_absorb": (_I, [POINTER(Latent), _P]),
    "socket_rotate_tail": (_I, [_P, _I, _I, _I, _I, _I, _I, _P, _L, _L, _P]),
    "socket_latent_attend": (_I, [POINTER(LatentAttend), _P]),
    "socket_latent_values": (_I, [POINTER(LatentAttend), _P]),
    "socket_recurrence_scan": (_I, [POINTER(Recurrence), _P]),
    "socket_recurrence_conv_tail": (_I, [POINTER(Recurrence), _P]),
    "socket_abi_version": (_I, []),
    "socket_status_string": (c_char_p, [_I]),
    "socket_device_query": (_I, [POINTER(c_int), POINTER(c_int)]),
    "socket_rope_append": (_I, [_P, _I, _L, _P, _I, _L, _P, _I, _P, _P, _P, _L, _L, _L, _P, _P, _P, _I, _I, _I, _I,
                                _L, _P]),
    "socket_add_rmsnorm": (_I, [_P, _P, _P, _P, _P, _I, _L, _I, c_float, _P]),
    "socket_silu_mul": (_I, [_P, _P, _P, _I, _L, _P]),
    "socket_gemv_bf16": (_I, [_P, _L, _P, _P, _P, _L, _I, _I, _I, _P]),
    "socket_norm_gemv_bf16": (_I, [_P, _P, _P, c_float, _P, _P, _P, _P, _I, _I, _I, _P]),
    "socket_attend_stage1": (_I, [_P, _P, _P, _I, _L, _L, _L, _L, _L, _L, _L, _L,
                                  _P, _L, _L, _P, _L, _L, _P, _P,
                                  _I, _I, _I, _I, _I, _I, _I, _I, _P]),
    "socket_attend_stage2": (_I, [_P, _P, _P, _L, _L, _P, _I, _L, _L, _I, _I, _I, _I, _I, _P]),
    "socket_sparse_attention_block_seq": (_I, [_I, _I, _I]),
    "socket_sparse_attention_workspace_bytes": (_Z, [_I, _I, _I, _I]),
    "socket_sparse_attention": (_I, [_P, _P, _P, _I, _L, _L, _L, _L, _L, _L, _L, _L,
                                     _P, _L, _L, _P, _L, _L, _P, _L, _L, _P, _Z,
                                     _I, _I, _I, _I, _I, _I, _P]),
    "socket_static_scratch_bytes": (_Z, []),
    "socket_static_scratch_init": (_I, []),
    "socket_sparse_attention_static": (_I, [_P, _P, _P, _I, _L, _L, _L, _L, _L, _L, _L, _L,
                                            _P, _L, _L, _P, _L, _L, _P, _L, _L,
                                            _I, _I, _I, _I, _I, _I, _P]),
    "socket_dense_decode_workspace_bytes": (_Z, [_I, _I, _I, _I]),
    "socket_dense_decode": (_I, [_P, _P, _P, _I, _L, _L, _L, _L, _L, _L, _L, _L,
                                 _P, _P, _L, _L, _P, _Z, _I, _I, _I, _I, _I, _P]),
}

# All of it (libsocket_hip.so resolves the core's names through its dependency):
SIGNATURES = {
    **CORE_SIGNATURES,
    "socket_words_per_key": (_I, [_I, _I]),
    "socket_permute_planes": (_I, [_P, _I, _I, _I, _I, _P, _P]),
    "socket_hash_keys": (_I, [_P, _P, _I, _L, _L, _L, _L, _L, _L, _P, _P, _P, _P, _I,
                              _I, _I, _I, _I, _I, _I, _L, _P]),
    "socket_unpack_codes": (_I, [_P, _P, _I, _I, _I, _I, _I, _I, _L, _L, _L, _L, _L, _P]),
    "socket_pack_codes": (_I, [_P, _L, _L, _L, _L, _P, _I, _I, _I, _I, _I, _I, _L, _P]),
    "socket_score_range_parts": (_I, [_I, _I, _I, _I, _I, _I, _I, _I]),
    "socket_score_packed": (_I, [_P, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _L, _L, _I, _P]),
    "socket_soft_hash_collision": (_I, [_P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _P]),
    "socket_soft_hash_score_f16": (_I, [_P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _P]),
    "socket_score_plan_query": (_I, [_I, _I, _I, _I, _I, _I, _I, _I, _I, POINTER(c_int), POINTER(c_int),
                                     POINTER(c_int), POINTER(c_float)]),
    "socket_score_shape_cost": (_I, [_I, _I, _I, _I, _I, _I, _I, _I, _I, _I, _I, _I, POINTER(c_int), POINTER(c_int),
                                     POINTER(c_float)]),
    "socket_group_shape": (_I, [_I, _I, POINTER(c_int), POINTER(c_int)]),
    "socket_score_prefers_grouped": (_I, [_I, _I, _I, _I, _I, _I, _I, _I]),
    "socket_score_range_parts_grouped": (_I, [_I, _I, _I, _I, _I, _I, _I, _I]),
    "socket_score_persistent_serves": (_I, [_I, _I, _I, _I, _I, _I, _I, _I]),
    "socket_group_q_probs": (_I, [_P, _I, _P, _I, _I, _I, _I, _I, _P]),
    "socket_score_packed_grouped": (_I, [_P, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _L, _L, _I, _P]),
    "socket_soft_hash_grouped": (_I, [_P, _I, _L, _L, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, c_float, c_float, _P]),
    "socket_soft_hash": (_I, [_P, _I, _L, _L, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, c_float, c_float, _P]),
    "socket_select_workspace_bytes": (_Z, [_I, _I, _I, _I]),
    "socket_select_workspace_zero_bytes": (_Z, [_I, _I, _I, _I]),
    "socket_select_list": (_I, [_P, _L, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _P, _L, _I, _P, _P, _Z, _P]),
    "socket_decode_prologue": (_I, [_P, _I, _L, _P, _I, _L, _P, _I, _P, _P, _P, _L, _L, _L, _P, _P, _P, _P, _P, _P, _P,
                                    _I, _I, _I, _I, _I, _I, _I, _I, _I, _L, c_float, c_float, _P]),
    "socket_block_sparse_attention": (_I, [_P, _P, _P, _I] + [_L] * 9 + [_P, _P, _P] + [_L] * 3 + [_I] * 8 + [_P]),
}

_lib = None
_core = None


class SocketHipError(RuntimeError):
    """A libsocket_hip entry point returned a non-zero status."""

    def __init__(self, fn: str, status: int, text: str):
        super().__init__(f"{fn} failed with status {status}: {text}")
        self.status = status


def _load(path: str, signatures: dict, how: str) -> ctypes.CDLL:
    if not os.path.exists(path):
        raise RuntimeError(f"{path} is missing: build it with `{how}` (hipcc, gfx950). There is no fallback path.")
    handle = ctypes.CDLL(path)
    for name, (res, args) in signatures.items():
        fn = getattr(handle, name)
        fn.restype = res
        fn.argtypes = args
    if handle.socket_abi_version() != 5:
        raise RuntimeError(f"{os.path.basename(path)} ABI version mismatch; rebuild it")
    return handle


def lib() -> ctypes.CDLL:
    """The loaded library with argument types set; raises if it is not built."""
    global _lib
    if _lib is None:
        _lib = _load(LIB_PATH, SIGNATURES, "python -m socket_amd.build")
    return _lib


def core() -> ctypes.CDLL:
    """libsocket_core.so alone, for the model families that need nothing else."""
    global _core
    if _core is None:
        _core = _load(CORE_PATH, CORE_SIGNATURES, "python -m socket_amd.build --core")
    return _core


def check(fn: str, status: int) -> None:
    if status != SOCKET_OK:
        text = core().socket_status_string(status).decode()
        raise SocketHipError(fn, status, text)


def dtype_enum(dt: torch.dtype) -> int:
    try:
        return _DTYPE_ENUM[dt]
    except KeyError:
        raise RuntimeError(f"unsupported dtype {dt}: expected float32, bfloat16 or float16") from None


def ptr(t) -> c_void_p:
    return c_void_p(0 if t is None else t.data_ptr())


def stream_ptr(device=None) -> c_void_p:
    """The HIP stream torch is currently issuing work on, as the reference's
    kernels (Triton and load_inline launches) do."""
    return c_void_p(torch.cuda.current_stream(device).cuda_stream)


def require_device(*tensors) -> None:
    for t in tensors:
        if t is not None and not t.is_cuda:
            raise AssertionError("expected a tensor on the HIP device")
