"""ctypes binding of ``libajq.so`` (declared in ``include/ajq.h``).

The library is loaded lazily and is never built from here: a missing library is
an error the caller sees (``python -m ajllm_amd.build`` makes it).  There is no
CPU or PyTorch fallback behind any of these calls.
"""

from __future__ import annotations

import ctypes
from ctypes import c_char_p, c_float, c_int, c_int64, c_size_t, c_void_p
from pathlib import Path

LIBRARY_PATH = Path(__file__).resolve().parent / "libajq.so"

AJQ_OUT_BF16 = 0
AJQ_OUT_F32 = 1
AJQ_KV_F32 = 0
AJQ_KV_BF16 = 1

# status -> exception class; argument errors are ValueError (the reference CLI turns
# ValueError into a clean exit, src/ajllm/cli.py:57-60), runtime errors RuntimeError.
_ARGUMENT_ERRORS = {-1, -2, -3, -4, -6}

# name -> (restype, argtypes); one entry per declaration in include/ajq.h
SIGNATURES: dict[str, tuple] = {
    "ajq_version": (c_int, []),
    "ajq_last_error": (c_char_p, []),
    "ajq_status_string": (c_char_p, [c_int]),
    "ajq_gemm_gate_supported": (c_int, [c_int, c_int, c_int, c_int]),
    "ajq_w4a16_gemm_gate": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_void_p, c_size_t,
                                    c_void_p]),
    "ajq_w8a16_gemm_gate": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_void_p]),
    "ajq_quantize_w8": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p, c_void_p]),
    "ajq_quantize_w4_g128": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p, c_void_p, c_void_p]),
    "ajq_repack_w4": (c_int, [c_void_p, c_void_p, c_void_p, c_int, c_int, c_void_p, c_void_p, c_void_p]),
    "ajq_unrepack_w4": (c_int, [c_void_p, c_void_p, c_int, c_int, c_void_p, c_void_p, c_void_p, c_void_p]),
    "ajq_repack_w8": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p]),
    "ajq_unrepack_w8": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p]),
    "ajq_w4a16_gemv": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_int, c_void_p]),
    "ajq_w8a16_gemv": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_int, c_void_p]),
    "ajq_w4a16_gemm_workspace_bytes": (c_size_t, [c_int, c_int]),
    "ajq_w4a16_gemm_workspace_bytes_for": (c_size_t, [c_int, c_int, c_int]),
    "ajq_w4a16_gemm": (
        c_int,
        [c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_int, c_void_p, c_size_t, c_void_p],
    ),
    "ajq_w8a16_gemm": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_int, c_void_p]),
    "ajq_noalloc_scratch_bytes": (c_size_t, []),
    "ajq_w4a16_gemm_noalloc": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_int, c_void_p]),
    "ajq_add_rmsnorm": (c_int, [c_void_p, c_void_p, c_void_p, c_float, c_void_p, c_int, c_int, c_void_p]),
    "ajq_rope_cache": (
        c_int,
        [c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int,
         c_int, c_void_p],
    ),
    "ajq_attn_decode_workspace_bytes": (c_size_t, [c_int, c_int]),
    "ajq_attn_row_chunks": (c_int, [c_int, c_int, c_int]),
    "ajq_rope_prefill": (
        c_int,
        [c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_int,
         c_int, c_void_p],
    ),
    "ajq_attn_prefill": (
        c_int,
        [c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_void_p, c_int, c_void_p],
    ),
    "ajq_greedy_pick": (
        c_int,
        [c_void_p, c_int, c_int, c_int, c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_int, c_void_p, c_void_p,
         c_void_p, c_void_p],
    ),
    "ajq_sample_pick": (
        c_int,
        [c_void_p, c_int, c_int, c_int, c_float, c_float, c_void_p, c_int, c_void_p, c_int, c_void_p, c_void_p, c_void_p,
         c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p],
    ),
    "ajq_gemv_merge_max_splits": (c_int, [c_int, c_int]),
    "ajq_w4a16_gemv_merge": (c_int, [c_void_p, c_int, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_int, c_void_p]),
    "ajq_w8a16_gemv_merge": (c_int, [c_void_p, c_int, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_int, c_void_p]),
    "ajq_attn_step_partial": (
        c_int,
        [c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int,
         c_int, c_void_p, c_void_p, c_size_t, c_void_p],
    ),
    "ajq_gemv_fused_supported": (c_int, [c_int, c_int]),
    "ajq_w4a16_gemv_norm": (
        c_int,
        [c_void_p, c_void_p, c_void_p, c_float, c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_int,
         c_void_p],
    ),
    "ajq_w8a16_gemv_norm": (
        c_int,
        [c_void_p, c_void_p, c_void_p, c_float, c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_int,
         c_void_p],
    ),
    "ajq_gemv_epilogue_supported": (c_int, [c_int, c_int]),
    "ajq_gemv_rowscale_supported": (c_int, [c_int, c_int]),
    "ajq_matmul_workspace_bytes": (c_size_t, []),
    "ajq_matmul_workspace_set": (c_int, [c_void_p, c_size_t]),
    "ajq_w4a16_gemv_residual": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_void_p, c_void_p,
                                        c_void_p, c_void_p, c_void_p]),
    "ajq_w8a16_gemv_residual": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_void_p, c_void_p,
                                        c_void_p, c_void_p, c_void_p]),
    "ajq_w4a16_gemv_gated": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_void_p]),
    "ajq_w8a16_gemv_gated": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_void_p]),
    "ajq_w4a16_gemv_norm_sums": (c_int, [c_void_p, c_void_p, c_int, c_void_p, c_float, c_int, c_int, c_void_p, c_void_p,
                                         c_int, c_void_p, c_int, c_int, c_void_p]),
    "ajq_w8a16_gemv_norm_sums": (c_int, [c_void_p, c_void_p, c_int, c_void_p, c_float, c_int, c_int, c_void_p, c_void_p,
                                         c_int, c_void_p, c_int, c_int, c_void_p]),
    "ajq_w4a16_gemv_merge_residual": (c_int, [c_void_p, c_int, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_void_p,
                                              c_void_p, c_void_p, c_void_p, c_void_p]),
    "ajq_w8a16_gemv_merge_residual": (c_int, [c_void_p, c_int, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_void_p,
                                              c_void_p, c_void_p, c_void_p, c_void_p]),
    "ajq_w4a16_gemv_rowscale": (c_int, [c_void_p, c_void_p, c_int, c_float, c_int, c_int, c_void_p, c_void_p, c_int,
                                        c_void_p, c_int, c_int, c_void_p]),
    "ajq_w8a16_gemv_rowscale": (c_int, [c_void_p, c_void_p, c_int, c_float, c_int, c_int, c_void_p, c_void_p, c_int,
                                        c_void_p, c_int, c_int, c_void_p]),
    "ajq_w4a16_gemv_gate": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_int, c_void_p]),
    "ajq_w8a16_gemv_gate": (c_int, [c_void_p, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p, c_int, c_void_p]),
    "ajq_attn_step_workspace_bytes": (c_size_t, [c_int, c_int]),
    "ajq_attn_step": (
        c_int,
        [c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int,
         c_void_p, c_void_p, c_size_t, c_void_p],
    ),
    "ajq_attn_decode": (
        c_int,
        [c_void_p, c_void_p, c_void_p, c_int, c_void_p, c_int, c_int, c_int, c_int, c_int, c_void_p, c_void_p,
         c_size_t, c_void_p],
    ),
    "ajq_swiglu": (c_int, [c_void_p, c_void_p, c_int, c_int, c_void_p]),
}

# libajq_bench.so (include/ajq_bench.h): the device yardstick for bench.py, not an operator
BENCH_LIBRARY_PATH = Path(__file__).resolve().parent / "libajq_bench.so"


BENCH_SIGNATURES: dict[str, tuple] = {
    "ajqb_last_error": (c_char_p, []),
    "ajqb_mfma_rate": (c_int, [c_int, c_int, c_int, c_void_p, c_void_p, c_void_p, c_void_p]),
}

# libajq_dense.so (include/ajq_dense.h): the operators of the dense model family
DENSE_LIBRARY_PATH = Path(__file__).resolve().parent / "libajq_dense.so"

AJQD_BF16 = 0
AJQD_F32 = 1
AJQD_ACTIVATIONS = {"relu": 0, "silu": 1, "gelu_tanh": 2, "squared_relu": 3}


class LatentShape(ctypes.Structure):
    """``ajqd_latent_shape``"""

    _fields_ = [(n, c_int) for n in ("heads", "dimp", "rot", "rotp", "rank", "rankp")] + [("eps", c_float)]


class WindowedAttentionArgs(ctypes.Structure):
    """``ajqd_windowed_attention_args``"""

    _fields_ = ([(n, c_void_p) for n in ("q", "k1", "k2", "v", "sink", "gates", "column_gates", "pos", "out")]
                + [(n, c_int64) for n in ("k1_batch", "k2_batch", "v_batch", "k1_head", "v_head")]
                + [(n, c_int) for n in ("k1_row", "k2_row", "v_row", "d1", "d2", "dv", "batch", "heads", "share", "seq", "rows",
                                        "prior", "window", "keep", "gate_ld", "out_ld")]
                + [("scale", c_float)])


class DenseInArgs(ctypes.Structure):
    """``ajqd_dense_in_args``"""

    _fields_ = ([(n, c_void_p) for n in ("x", "n1", "n2", "gain1", "gain2", "w1", "w2", "y1", "gated")]
                + [(n, c_int) for n in ("batch", "true_width", "width", "tiles1", "tiles2", "gated_ld", "act", "center", "pairs")]
                + [("eps", c_float)])


class KeyValueSplitArgs(ctypes.Structure):
    """``ajqd_key_value_split_args``"""

    _fields_ = ([(n, c_void_p) for n in ("y", "q_gain", "k_gain", "half_turns", "pos", "q", "rows")]
                + [(n, c_int64) for n in ("rows_batch", "rows_head")]
                + [(n, c_int) for n in ("tokens", "seq", "start", "ldy", "heads", "groups", "dim", "dimp", "rot", "q_ld", "q_at", "prior",
                                        "cap", "kept")]
                + [("eps", c_float)])


class ScanArgs(ctypes.Structure):
    """``ajqd_scan_args``"""

    _fields_ = ([(n, c_void_p) for n in ("x", "dt", "low", "z", "a2", "d", "dt_bias", "state", "pos", "out")]
                + [(n, c_int) for n in ("batch", "seq", "start", "inner", "states", "dt_ld", "low_ld", "b_col", "c_col", "z_ld",
                                        "out_ld")])


class ScanStepArgs(ctypes.Structure):
    """``ajqd_scan_step_args``"""

    _fields_ = ([(n, c_void_p) for n in ("y", "ring", "weight", "bias", "pos", "partial", "w_dt", "dt_bias", "a2", "d", "state", "out")]
                + [(n, c_int) for n in ("batch", "ldy", "inner", "taps", "rows", "splits", "rank", "states", "out_ld")])


_P, _I, _F, _L = c_void_p, c_int, c_float, c_int64
DENSE_SIGNATURES: dict[str, tuple] = {
    "ajqd_last_error": (c_char_p, []),
    "ajqd_embed": (c_int, [_P, _I, _I, _P, _I, _P, _I, _I, _P, _P, _P, _P, _I, _I, _P]),
    "ajqd_add_norms": (c_int, [_P, _P, _I, _P, _P, _P, _P, _F, _I, _P, _P, _I, _I, _I, _I, _P]),
    "ajqd_latent_split": (c_int, [_P, _I, _I, ctypes.POINTER(LatentShape), _P, _P, _P, _I, _I, _I, _I, _P, _I, _I, _P, _I, _P,
                                  _I, _P, _L, _P, _I, _P]),
    "ajqd_ring_copy": (c_int, [_P, _I, _I, _P, _I, _I, _I, _I, _I, _I, _I, _I, _P]),
    "ajqd_gated_activation": (c_int, [_P, _I, _P, _I, _I, _I, _I, _I, _P]),
    "ajqd_matvec": (c_int, [_P, _P, _I, _I, _P, _I, _I, _I, _I, _I, _I, _I, _I, _P]),
    "ajqd_windowed_attention": (c_int, [ctypes.POINTER(WindowedAttentionArgs), _I, _I, _P]),
    "ajqd_windowed_prefill_supported": (c_int, [_I, _I, _I]),
    "ajqd_windowed_prefill": (c_int, [ctypes.POINTER(WindowedAttentionArgs), _P]),
    "ajqd_dense_in": (c_int, [ctypes.POINTER(DenseInArgs), _P]),
    "ajqd_dense_out": (c_int, [_P, _P, _P, _P, _P, _I, _I, _I, _P]),
    "ajqd_latent_absorb": (c_int, [_P, _I, ctypes.POINTER(LatentShape), _P, _P, _P, _P, _I, _P, _P, _P, _I, _I, _P]),
    "ajqd_latent_decode_chunks": (c_int, [_I, _I, _I, _I, _I]),
    "ajqd_latent_decode_workspace": (c_size_t, [_I, _I, _I, _I]),
    "ajqd_latent_decode": (c_int, [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _F, _P]),
    "ajqd_latent_expand": (c_int, [_P, _P, _P, _I, _P, _P, _I, _I, _I, _I, _I, _I, _P]),
    "ajqd_embed_streams": (c_int, [_P, _I, _P, _I, _P, _P, _P, _I, _I, _I, _P]),
    "ajqd_streams_norm": (c_int, [_P, _P, _P, _P, _P, _P, _P, _F, _P, _P, _I, _I, _I, _I, _I, _P]),
    "ajqd_dense_out_streams": (c_int, [_P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _P]),
    "ajqd_activation": (c_int, [_P, _P, _L, _I, _I, _P]),
    "ajqd_key_value_split": (c_int, [ctypes.POINTER(KeyValueSplitArgs), _I, _I, _P]),
    "ajqd_group_merge": (c_int, [_P, _P, _I, _P, _I, _I, _I, _I, _I, _I, _P]),
    "ajqd_conv_silu": (c_int, [_P, _I, _P, _P, _P, _I, _P, _I, _I, _I, _I, _P, _I, _P]),
    "ajqd_scan": (c_int, [ctypes.POINTER(ScanArgs), _I, _P]),
    "ajqd_scan_splits": (c_int, [_I, _I]),
    "ajqd_scan_project": (c_int, [_P, _I, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _P]),
    "ajqd_scan_step": (c_int, [ctypes.POINTER(ScanStepArgs), _P]),
}

_lib: ctypes.CDLL | None = None
_dense_lib: ctypes.CDLL | None = None
_bench_lib: ctypes.CDLL | None = None


def load_bench() -> ctypes.CDLL:
    """The bench-only probe library, bound on first use (built by ``python -m ajllm_amd.build``)."""
    global _bench_lib
    if _bench_lib is not None:
        return _bench_lib
    if not BENCH_LIBRARY_PATH.exists():
        raise RuntimeError(f"{BENCH_LIBRARY_PATH} is missing: build it with `python -m ajllm_amd.build`")
    lib = ctypes.CDLL(str(BENCH_LIBRARY_PATH))
    for name, (restype, argtypes) in BENCH_SIGNATURES.items():
        fn = getattr(lib, name)
        fn.restype = restype
        fn.argtypes = argtypes
    _bench_lib = lib
    return lib


def load() -> ctypes.CDLL:
    """Return the loaded library, binding every signature on first use."""
    global _lib
    if _lib is not None:
        return _lib
    if not LIBRARY_PATH.exists():
        raise RuntimeError(
            f"{LIBRARY_PATH} is missing: build it with `python -m ajllm_amd.build` "
            "(the quantized linear has no fallback path)"
        )
    lib = ctypes.CDLL(str(LIBRARY_PATH))
    for name, (restype, argtypes) in SIGNATURES.items():
        fn = getattr(lib, name)
        fn.restype = restype
        fn.argtypes = argtypes
    _lib = lib
    return lib


def load_dense() -> ctypes.CDLL:
    """The dense model family's operators, bound on first use (built by ``python -m ajllm_amd.build``)."""
    global _dense_lib
    if _dense_lib is not None:
        return _dense_lib
    if not DENSE_LIBRARY_PATH.exists():
        raise RuntimeError(f"{DENSE_LIBRARY_PATH} is missing: build it with `python -m ajllm_amd.build` "
                           "(the dense models have no fallback path)")
    lib = ctypes.CDLL(str(DENSE_LIBRARY_PATH))
    for name, (restype, argtypes) in DENSE_SIGNATURES.items():
        fn = getattr(lib, name)
        fn.restype = restype
        fn.argtypes = argtypes
    _dense_lib = lib
    return lib


def check_dense(status: int, what: str) -> None:
    """``check`` for a status of libajq_dense.so."""
    if status == 0:
        return
    message = f"{what}: {load_dense().ajqd_last_error().decode()}"
    raise ValueError(message) if status in _ARGUMENT_ERRORS else RuntimeError(message)


def check(status: int, what: str) -> None:
    """Raise the exception that matches a negative ajq_status."""
    if status == 0:
        return
    lib = load()
    message = lib.ajq_last_error().decode() or lib.ajq_status_string(status).decode()
    if status in _ARGUMENT_ERRORS:
        raise ValueError(f"{what}: {message}")
    raise RuntimeError(f"{what}: {message}")
