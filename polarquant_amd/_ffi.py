"""ctypes binding of libpolarquant_hip.so (the C ABI declared in include/polarquant.h).

The library is loaded from the package directory; it is never built implicitly
on import of this module when a built library exists.  If it is missing the
loader raises: there is no CPU fallback for any op of this package.
"""
from __future__ import annotations

import ctypes
import os
from ctypes import c_char_p, c_float, c_int, c_int64, c_size_t, c_uint, c_void_p

HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(HERE, "libpolarquant_hip.so")

PQ_F16, PQ_BF16, PQ_F32 = 0, 1, 2          # float32: not in the polar-key library
PQ_EPI_PLAIN, PQ_EPI_RELU_SQ, PQ_EPI_SIGMOID_GATE, PQ_EPI_F32 = 0, 1, 2, 3
PQ_WRAP_FP32 = 1
PQ_ANGLE_UNIFORM = 2
PQ_CODES_PACKED6 = 4
PQ_DEVICE_ATAN2 = 8
PQ_BALANCED_SLICES = 16
PQ_SINGLE_WAVEFRONT = 32
PQ_TEST_SILENT_SCORER = 0x40000000      # honoured by the test build of the library only; the one loaded here refuses it
PQ_STATUS_HANDOVER_TIMEOUT = 1
PQ_EAGER_GPU = PQ_WRAP_FP32 | PQ_DEVICE_ATAN2

STATUS_NAMES = {
    0: "PQ_OK", -1: "PQ_ERR_NULL_POINTER", -2: "PQ_ERR_BAD_SHAPE", -3: "PQ_ERR_BAD_BITS", -4: "PQ_ERR_BAD_DTYPE",
    -5: "PQ_ERR_MISALIGNED", -6: "PQ_ERR_BAD_STRIDE", -7: "PQ_ERR_WORKSPACE", -8: "PQ_ERR_LAUNCH",
    -9: "PQ_ERR_NO_DEVICE",
}

# name -> (restype, argtypes); every symbol of include/polarquant.h
SIGNATURES = {
    "pq_version": (c_int, []),
    "pq_status_string": (c_char_p, [c_int]),
    "pq_decode_scores": (c_int, [c_void_p] * 7 + [c_int] * 7 + [c_uint, c_void_p]),
    "pq_validate_decode_scores": (c_int, [c_void_p] * 7 + [c_int] * 7 + [c_uint]),
    "pq_quantize_groups": (c_int, [c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_uint]
                           + [c_void_p] * 5 + [c_int, c_int, c_void_p]),
    "pq_validate_quantize_groups": (c_int, [c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_uint]
                                    + [c_void_p] * 5 + [c_int, c_int]),
    "pq_selftest_quantizer_math": (c_int, [c_int, c_void_p, c_void_p]),
    "pq_decode_attn": (c_int, [c_void_p] * 6 + [c_int, c_int, c_void_p, c_void_p, c_int, c_int, c_void_p,
                                                c_void_p, c_int64, c_void_p, c_int64, c_float]
                       + [c_int] * 8 + [c_void_p, c_size_t, c_void_p, c_uint, c_void_p, c_void_p]),
    "pq_decode_attn_static": (c_int, [c_void_p] * 6 + [c_int, c_int, c_void_p, c_void_p, c_int, c_int, c_void_p,
                                                       c_void_p, c_int64, c_void_p, c_int64, c_float]
                              + [c_int] * 8 + [c_void_p, c_uint, c_void_p, c_void_p]),
    "pq_validate_decode_attn": (c_int, [c_void_p] * 6 + [c_int, c_int, c_void_p, c_void_p, c_int, c_int, c_void_p,
                                                         c_void_p, c_int64, c_void_p, c_int64, c_float]
                                + [c_int] * 8 + [c_void_p, c_size_t, c_void_p, c_uint]),
    "pq_decode_attn_partials": (c_int, [c_void_p] * 6 + [c_int, c_int, c_void_p, c_void_p, c_int, c_int, c_void_p,
                                                         c_void_p, c_int64, c_void_p, c_int64, c_float]
                                + [c_int] * 8 + [c_void_p, c_size_t, c_uint, c_void_p, c_void_p]),
    "pq_decode_attn_merge": (c_int, [c_void_p, c_size_t, c_int, c_int, c_int, c_int, c_void_p, c_void_p]),
    "pq_quantize_values": (c_int, [c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p,
                                   c_int64, c_int64, c_void_p]),
    "pq_validate_quantize_values": (c_int, [c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p,
                                            c_int64, c_int64]),
    "pq_decode_attn_v4": (c_int, [c_void_p] * 6 + [c_int, c_int, c_void_p, c_void_p, c_int, c_int, c_void_p,
                                                   c_void_p, c_void_p, c_void_p, c_void_p, c_int64,
                                                   c_void_p, c_int64, c_float]
                          + [c_int] * 8 + [c_void_p, c_size_t, c_void_p, c_uint, c_void_p, c_void_p]),
    "pq_validate_decode_attn_v4": (c_int, [c_void_p] * 6 + [c_int, c_int, c_void_p, c_void_p, c_int, c_int, c_void_p,
                                                            c_void_p, c_void_p, c_void_p, c_void_p, c_int64,
                                                            c_void_p, c_int64, c_float]
                                   + [c_int] * 8 + [c_void_p, c_size_t, c_void_p, c_uint]),
    "pq_rope_append": (c_int, [c_void_p] * 5 + [c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_int64,
                                               c_void_p, c_int, c_int, c_int, c_int, c_int64, c_int64, c_void_p]),
    "pq_rmsnorm": (c_int, [c_void_p] * 5 + [c_int, c_int, c_float, c_int, c_void_p]),
    "pq_silu_mul": (c_int, [c_void_p] * 3 + [c_int, c_int, c_int64, c_int, c_void_p]),
    "pq_linear_small_m": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int, c_int, c_int, c_void_p]),
    "pq_validate_linear_small_m": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int, c_int, c_int]),
    "pq_rope_qk": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_void_p, c_void_p,
                           c_int, c_int, c_int, c_int, c_int, c_void_p]),
    "pq_qkv_rope_append": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int, c_int, c_int, c_void_p, c_void_p, c_int64,
                                   c_void_p, c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_void_p, c_int, c_int, c_void_p]),
    "pq_validate_qkv_rope_append": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int, c_int, c_int, c_void_p, c_void_p, c_int64,
                                            c_void_p, c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_void_p, c_int, c_int]),
    "pq_convert_codes6": (c_int, [c_void_p, c_void_p, c_size_t, c_int, c_void_p]),
    "pq_decode_attn_plan": (c_int, [c_int] * 4),
    "pq_decode_attn_v4_plan": (c_int, [c_int] * 5),
    "pq_decode_attn_workspace_bytes": (c_size_t, [c_int] * 3),
}


# the bench-only library (include/polarquant_bench.h): measurement aids, loaded by bench.py and its tests
BENCH_LIB_PATH = os.path.join(HERE, "libpolarquant_bench.so")
BENCH_SIGNATURES = {
    "pq_stream_read": (c_size_t, [c_void_p, c_size_t, c_int, c_void_p, c_void_p]),
    "pq_attn_load_replica": (c_size_t, [c_void_p, c_void_p, c_int, c_int64, c_int64, c_int64, c_int, c_void_p, c_void_p]),
}


# the steps between mixers and matrix products (include/polarquant_steps.h) and the mixers' kernels, by family
# (include/polarquant_latent.h): libraries of their own, so that a decoder builds only what it runs
STEPS_LIB_PATH = os.path.join(HERE, "libpolarquant_steps.so")
STEPS_SIGNATURES = {
    "pq_norm_conv": (c_int, [c_void_p] * 11 + [c_int] * 6 + [c_float] + [c_int] + [c_void_p]),
    "pq_validate_norm_conv": (c_int, [c_void_p] * 11 + [c_int] * 7),
    "pq_relu_sq": (c_int, [c_void_p] * 2 + [c_size_t] + [c_int] + [c_void_p]),
    "pq_gelu_mul": (c_int, [c_void_p] * 2 + [c_int64, c_void_p, c_int64, c_int64, c_int, c_int, c_void_p]),
    "pq_stream_add": (c_int, [c_void_p] * 5 + [c_int64, c_int, c_int, c_void_p]),
    "pq_embed_rows": (c_int, [c_void_p] * 2 + [c_float, c_void_p, c_int64, c_int, c_int64, c_int, c_void_p]),
    "pq_softcap": (c_int, [c_void_p, c_size_t, c_float, c_float, c_void_p]),
    "pq_head_linear": (c_int, [c_void_p] + [c_int64] * 2 + [c_void_p] * 2 + [c_int64] + [c_void_p] + [c_int64] * 2 + [c_int] * 6 + [c_void_p]),
    "pq_validate_head_linear": (c_int, [c_void_p] + [c_int64] * 2 + [c_void_p] * 2 + [c_int64] + [c_void_p] + [c_int64] * 2 + [c_int] * 6),
}

LATENT_LIB_PATH = os.path.join(HERE, "libpolarquant_latent.so")
LATENT_SIGNATURES = {
    "pq_latent_norm": (c_int, [c_void_p] + [c_int64] + [c_void_p] * 4 + [c_int64] + [c_void_p] + [c_int] * 5 + [c_float] + [c_int] + [c_void_p]),
    "pq_validate_latent_norm": (c_int, [c_void_p] + [c_int64] + [c_void_p] * 4 + [c_int64] + [c_void_p] + [c_int] * 6),
    "pq_latent_decode_plan": (c_int, [c_int] * 3 + [c_int64] + [c_int]),
    "pq_latent_decode_workspace_bytes": (c_size_t, [c_int] * 5),
    "pq_latent_decode": (c_int, [c_void_p] * 2 + [c_int64] + [c_void_p] * 3 + [c_int] + [c_void_p] + [c_int] * 4 + [c_float] + [c_int] + [c_void_p] + [c_size_t] + [c_int] + [c_void_p]),
    "pq_validate_latent_decode": (c_int, [c_void_p] * 2 + [c_int64] + [c_void_p] * 3 + [c_int] + [c_void_p] + [c_int] * 5 + [c_void_p] + [c_size_t] + [c_int]),
    "pq_latent_prefill_takes": (c_int, [c_int] * 3),
    "pq_latent_prefill": (c_int, [c_void_p] * 3 + [c_int64] + [c_void_p] * 2 + [c_int64] + [c_void_p] * 2 + [c_int] * 6 + [c_float] + [c_int] + [c_void_p]),
    "pq_validate_latent_prefill": (c_int, [c_void_p] * 3 + [c_int64] + [c_void_p] * 2 + [c_int64] + [c_void_p] * 2 + [c_int] * 7),
}


# windowed attention and recurrent mixers (include/polarquant_recurrent.h)
RECURRENT_LIB_PATH = os.path.join(HERE, "libpolarquant_recurrent.so")
RECURRENT_SIGNATURES = {
    "pq_qk_norm": (c_int, [c_void_p] * 3 + [c_int64] + [c_void_p] * 7 + [c_int] * 8 + [c_float, c_int, c_void_p]),
    "pq_ring_append": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p] + [c_int] * 8 + [c_void_p]),
    "pq_window_plan": (c_int, [c_int] * 6),
    "pq_window_workspace_bytes": (c_size_t, [c_int] * 5),
    "pq_validate_window_attn": (c_int, [c_void_p] * 4 + [c_int64, c_void_p, c_int64] + [c_void_p] * 3 + [c_int, c_void_p, c_int64]
                                + [c_int] * 9 + [c_void_p, c_size_t, c_int]),
    "pq_window_attn": (c_int, [c_void_p] * 4 + [c_int64, c_void_p, c_int64] + [c_void_p] * 3 + [c_int, c_void_p, c_int64] + [c_int] * 8
                       + [c_float, c_float, c_int, c_void_p, c_size_t, c_int, c_void_p]),
    "pq_validate_delta_prep": (c_int, [c_int] * 7 + [c_void_p, c_void_p, c_int64, c_int64, c_int]),
    "pq_delta_prep": (c_int, [c_void_p] * 4 + [c_int64, c_void_p, c_int64] + [c_void_p] * 16 + [c_int] * 9 + [c_void_p]),
    "pq_scan_workspace_bytes": (c_size_t, [c_int] * 6),
    "pq_delta_scan": (c_int, [c_void_p] * 11 + [c_int] * 7 + [c_void_p, c_size_t, c_int, c_void_p]),
    "pq_memory_gates": (c_int, [c_void_p, c_void_p, c_int64] + [c_void_p] * 4 + [c_int64, c_int, c_float, c_int, c_void_p]),
    "pq_memory_scan": (c_int, [c_void_p] * 3 + [c_int64] + [c_void_p] * 6 + [c_float, c_void_p, c_void_p] + [c_int] * 6
                       + [c_void_p, c_size_t, c_int, c_void_p]),
    "pq_head_norm_gate": (c_int, [c_void_p] * 3 + [c_int, c_void_p, c_int64, c_void_p, c_int64, c_int64, c_int, c_int, c_float, c_float, c_int,
                                  c_void_p]),
}


class PolarQuantError(RuntimeError):
    def __init__(self, status: int, where: str):
        self.status = status
        msg = STATUS_NAMES.get(status, str(status))
        try:
            msg += ": " + lib().pq_status_string(status).decode()
        except Exception:                       # (the polar-key library need not be built)
            pass
        super().__init__("%s failed with %s" % (where, msg))


_LOADED = {}


def _load(path: str, signatures) -> ctypes.CDLL:
    """The library at `path` with its symbols' types set, loaded once.  Raises if it has not been built."""
    handle = _LOADED.get(path)
    if handle is None:
        if not os.path.exists(path):
            raise RuntimeError("polarquant_amd: %s is missing; build it with `python -m polarquant_amd.build` "
                               "(there is no CPU fallback)" % path)
        handle = ctypes.CDLL(path)
        for name, (res, args) in signatures.items():
            fn = getattr(handle, name)
            fn.restype = res
            fn.argtypes = args
        _LOADED[path] = handle
    return handle


def lib() -> ctypes.CDLL:
    """The polar-key library."""
    return _load(LIB_PATH, SIGNATURES)


def steps_lib() -> ctypes.CDLL:
    """The layer steps' library."""
    return _load(STEPS_LIB_PATH, STEPS_SIGNATURES)


def latent_lib() -> ctypes.CDLL:
    """The latent-attention library."""
    return _load(LATENT_LIB_PATH, LATENT_SIGNATURES)


def recurrent_lib() -> ctypes.CDLL:
    """The library of windowed attention and recurrent mixers."""
    return _load(RECURRENT_LIB_PATH, RECURRENT_SIGNATURES)


def bench_lib() -> ctypes.CDLL:
    """The measurement-aid library."""
    return _load(BENCH_LIB_PATH, BENCH_SIGNATURES)


def check(status: int, where: str) -> None:
    if status != 0:
        raise PolarQuantError(status, where)
