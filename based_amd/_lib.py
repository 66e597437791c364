"""ctypes binding of libbased_hip.so (the C ABI declared in include/based_hip.h).

The library is loaded lazily; there is no fallback path.  If the shared object is missing
the first use raises, so a GPU run can never silently go through something else.
"""
from __future__ import annotations

import ctypes as C
import os
import threading

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(_HERE, "libbased_hip.so")  # the in-tree build of every kernel
# Builds of some of the sources (based_amd.build.build_part) lie beside it; `use_part` selects one
# where the whole library has not been built.
_part_path = None

BASED_BF16 = 0
BASED_F32 = 1
PREFILL_SEGMENT_STATE_BYTES = 43008  # BASED_PREFILL_SEGMENT_STATE_BYTES of include/based_hip.h

_I64 = C.c_int64
_P = C.c_void_p

class StreamExtras(C.Structure):
    """based_stream_extras of include/based_hip.h."""

    _fields_ = ([(n, _P) for n in ("post_weight", "add_vec", "add_rows", "add_index", "mix_mu", "mix_ring", "gate_table", "gate_index")]
                + [(n, _I64) for n in ("add_sr", "add_n", "mix_rows", "mixes", "mix_ring_row_stride", "gate_sr", "gate_n")]
                + [(n, C.c_float) for n in ("post_eps", "softcap")])


# name -> (restype, argtypes); must list every symbol declared in include/based_hip.h
SIGNATURES = {
    "based_hip_version": (C.c_int, []),
    "based_hip_last_error": (C.c_char_p, []),
    "based_linear_attn_step": (
        C.c_int,
        [_P, _P, _P, _P, _P, _P] + [_I64] * 3 + [_I64] * 8 + [C.c_float, C.c_int, _P],
    ),
    "based_linear_attn_step_deferred": (
        C.c_int,
        [_P, _P, _P, _P, _P, _P, _P, _P, _P] + [_I64] * 3 + [_I64] * 8 + [C.c_float, C.c_int, C.c_int, _P],
    ),
    "based_linear_attn_flush_deferred": (C.c_int, [_P, _P, _P, _P] + [_I64] * 3 + [_P]),
    "based_linear_attn_prefill": (
        C.c_int,
        [_P, _P, _P, _P, _P, _P] + [_I64] * 4 + [_I64] * 12 + [C.c_float, C.c_int, _P],
    ),
    "based_linear_attn_prefill_plan": (
        C.c_int,
        [_I64] * 4 + [C.c_int, C.POINTER(_I64), C.POINTER(_I64)],
    ),
    "based_linear_attn_prefill_split": (
        C.c_int,
        [_P, _P, _P, _P, _P, _P] + [_I64] * 4 + [_I64] * 12 + [C.c_float, C.c_int, _I64, _P, _I64, _P],
    ),
    "based_linear_attn_prefill_split_static": (
        C.c_int,
        [_P, _P, _P, _P, _P, _P] + [_I64] * 4 + [_I64] * 12 + [C.c_float, C.c_int, _I64, _P],
    ),
    "based_swa_prefill": (
        C.c_int,
        [_P, _P, _P, _P] + [_I64] * 3 + [_I64] * 12 + [C.c_int, C.c_float]
        + [_P, _P, _I64] + [_P, _P] + [_I64] * 4 + [C.c_int, _P],
    ),
    "based_gated_conv_prefill": (
        C.c_int,
        [_P, _P, _P, _P, _P] + [_I64] * 3 + [C.c_int] + [_I64] * 4 + [C.c_int, C.c_int, _P],
    ),
    "based_gated_conv_step": (
        C.c_int,
        [_P, _P, _P, _P, _P] + [_I64] * 2 + [C.c_int] + [_I64] * 2 + [C.c_int, C.c_int, _P],
    ),
    "based_swa_prefill_anydim": (
        C.c_int,
        [_P, _P, _P, _P] + [_I64] * 4 + [_I64] * 12 + [C.c_int, C.c_float] + [_P, _P] + [_I64] * 4 + [C.c_int, _P],
    ),
    "based_swa_prefill_wide": (
        C.c_int,
        [_P, _P, _P, _P] + [_I64] * 4 + [_I64] * 12 + [C.c_int, C.c_float] + [_P, _P, _I64, _I64, C.c_int]
        + [_P, _P] + [_I64] * 4 + [C.c_int, _P],
    ),
    "based_swa_step_wide": (
        C.c_int,
        [_P] * 6 + [_P, _I64] + [_I64] * 4 + [_I64] * 8 + [_I64] * 3 + [C.c_int, C.c_float]
        + [_P, _P, _I64, _I64, C.c_int] + [C.c_int, _P],
    ),
    "based_greedy_step": (C.c_int, [_P, _I64, _I64, _I64, _P, _I64, _P, _I64, _I64, _P, _P, _I64, C.c_int, _P]),
    "based_swa_step_anydim": (
        C.c_int,
        [_P] * 6 + [_P, _I64] + [_I64] * 4 + [_I64] * 8 + [_I64] * 3 + [C.c_int, C.c_float, C.c_int, _P],
    ),
    "based_short_conv_prefill": (
        C.c_int,
        [_P, _P, _P, _P, _P] + [_I64] * 3 + [C.c_int] + [_I64] * 4 + [C.c_int, C.c_int, _P],
    ),
    "based_short_conv_step": (
        C.c_int,
        [_P, _P, _P, _P, _P] + [_I64] * 2 + [C.c_int] + [_I64] * 2 + [C.c_int, C.c_int, _P],
    ),
    "based_add_rms_norm": (
        C.c_int,
        [_P, _P, _P, _P, _P] + [_I64] * 6 + [C.c_float, C.c_int, C.c_int, _P],
    ),
    "based_swiglu": (C.c_int, [_P, _P] + [_I64] * 4 + [C.c_int, _P]),
    "based_decode_linear": (C.c_int, [_P, _I64, _P, _I64, _P, _I64, _P, _P, _I64, _I64, _I64, _I64, C.c_int,
                                      _P, _I64, _P, _I64, _P, C.c_float, C.c_int, _P, C.c_int, _P, _P, C.c_int, _P]),
    "based_add_norm": (C.c_int, [_P] * 5 + [_I64] * 6 + [C.c_float, C.c_int, C.c_float, C.c_int, _P]),
    "based_stream_conv": (C.c_int, [_P] * 6 + [_I64] * 4 + [C.c_int] + [_I64] * 5 + [C.c_int] * 3 + [_P]),
    "based_window_attn_prefill": (
        C.c_int,
        [_P] * 5 + [_I64] * 19 + [C.c_float, C.c_int, C.c_float, C.c_float, _P, _P, _I64, _I64, C.c_int, C.c_int, _P],
    ),
    "based_window_attn_step": (
        C.c_int,
        [_P] * 6 + [_I64] * 14 + [C.c_float, C.c_int, C.c_float, C.c_float, _P, _P, _I64, _I64, C.c_int, C.c_int, _P],
    ),
    "based_gated_delta_scan": (C.c_int, [_P] * 10 + [_I64] * 11 + [C.c_int, C.c_int, _P]),
    "based_gated_rms_norm": (C.c_int, [_P] * 4 + [_I64] * 8 + [C.c_float, C.c_float, C.c_int, _P]),
    "based_gated_delta_step": (
        C.c_int, [_P] * 12 + [_I64] * 8 + [C.c_int] + [_I64] * 7 + [C.c_float, C.c_float, C.c_int, _P]),
    "based_rglru_prefill": (C.c_int, [_P] * 12 + [_I64] * 10 + [C.c_float, C.c_int, C.c_int, _P]),
    "based_rglru_step": (C.c_int, [_P] * 13 + [_I64] * 4 + [C.c_int] + [_I64] * 4 + [C.c_float, C.c_int, _P]),
    "based_decode_linear_stream": (
        C.c_int,
        [_P, _I64, _P, _I64, _P, _I64, _P, _P] + [_I64] * 4 + [_P, _I64, _P, _I64, C.c_float, C.c_int, _P, C.c_float,
                                                              _P, _P, _I64, C.c_int, _P, _I64, C.c_int, _P],
    ),
    "based_add_norm_addends": (
        C.c_int, [_P] * 5 + [_I64] * 6 + [C.c_float, C.c_int, C.c_float, _P, C.c_float, _P, _P, _P, _I64, _I64, C.c_int, _P]),
    "based_token_mix": (C.c_int, [_P] * 5 + [_I64] * 8 + [C.c_int, _P]),
    "based_channel_decay": (C.c_int, [_P] * 4 + [_I64] * 4 + [C.c_int, _P]),
    "based_gelu_mul": (C.c_int, [_P] * 4 + [_I64] * 5 + [C.c_int, _P]),
    "based_token_side_step": (C.c_int, [_P] * 8 + [_I64] * 6 + [C.c_float, _P]),
    "based_softcap": (C.c_int, [_P, _I64, C.c_float, C.c_int, _P]),
    "based_decay_scan_work": (_I64, [_I64] * 6),
    "based_decay_scan": (C.c_int, [_P] * 9 + [_I64] * 14 + [C.c_int, C.c_int, C.c_int, _P]),
    "based_decay_step": (C.c_int, [_P] * 13 + [_I64] * 13 + [C.c_int, C.c_float, C.c_int, _P]),
    "based_group_norm_gate": (C.c_int, [_P] * 4 + [_I64] * 10 + [C.c_float, C.c_float, C.c_int, C.c_int, _P]),
    "based_window_attn_attend": (
        C.c_int, [_P] * 3 + [_I64] * 15 + [C.c_float, C.c_float, _P, _P, _I64, _I64, C.c_int, C.c_int, _P]),
    "based_latent_write": (C.c_int, [_P] * 3 + [_I64] * 10 + [C.c_float, _P, _P, _I64, C.c_int, C.c_int, _P]),
    "based_latent_step": (
        C.c_int, [_P] * 10 + [_I64] * 16 + [C.c_float, C.c_float, C.c_float, _P, _P, _I64, C.c_int, C.c_int, _P]),
    "based_expert_tiles": (_I64, [_I64] * 3),
    "based_expert_tile_rows": (_I64, [_I64] * 3),
    "based_expert_grouped": (C.c_int, [_P] * 14 + [_I64] * 6 + [_P]),
    "based_expert_rows": (C.c_int, [_P] * 5 + [C.c_float, C.c_int, C.c_float] + [_P] * 7 + [_I64] * 6 + [C.c_int, _P]),
    "based_decode_linear_extras": (
        C.c_int,
        [_P, _I64, _P, _I64, _P, _I64, _P, _P] + [_I64] * 4 + [_P, _I64, _P, _I64, C.c_float, C.c_int, _P, C.c_float, _P, _I64, C.c_int,
                                                              _P, _P],
    ),
    "based_decode_linear_mixes": (C.c_int, [_P, _P, _I64, _P] + [_I64] * 6 + [_P]),
    "based_swa_step": (
        C.c_int,
        [_P, _P, _P, _P, _P, _P, _P, _I64] + [_I64] * 3 + [_I64] * 8 + [_I64] * 3
        + [C.c_int, C.c_float] + [_P, _P, _I64] + [C.c_int, _P],
    ),
}

_lib = None
_lock = threading.Lock()


class BasedHipError(RuntimeError):
    """Raised when the native library is missing or a launch is refused by the runtime."""


def part_path(part: str) -> str:
    """Where the build of one named part of the sources lies."""
    return os.path.join(_HERE, f"libbased_hip_{part}.so")


def use_part(part: str) -> None:
    """Lets a process that needs only the kernels of `part` run from that part's build where the
    whole library does not exist.  Entry points the part does not hold raise when they are called."""
    global _part_path
    _part_path = part_path(part)


def _absent(name):
    def refuse(*args):
        raise BasedHipError(f"{name} is not in {_part_path}: build the whole library with `python -m based_amd.build`")

    return refuse


class _Entries:
    """The typed entry points of a loaded library."""

    def __init__(self, handle, partial: bool):
        for name, (res, args) in SIGNATURES.items():
            if partial and not hasattr(handle, name):
                setattr(self, name, _absent(name))
                continue
            fn = getattr(handle, name)
            fn.restype = res
            fn.argtypes = args
            setattr(self, name, fn)


def lib():
    """Returns the loaded library, loading and typing it on first use."""
    global _lib
    if _lib is None:
        with _lock:
            if _lib is None:
                path = LIB_PATH
                if not os.path.exists(path) and _part_path is not None:
                    path = _part_path
                if not os.path.exists(path):
                    raise BasedHipError(
                        f"{path} not found: build it with `python -m based_amd.build` "
                        "(there is no non-HIP fallback)"
                    )
                _lib = _Entries(C.CDLL(path), partial=path != LIB_PATH)
    return _lib


_SHAPE_CODES = (1, 2, 3)  # BASED_ERR_SHAPE / DTYPE / ALIGN -> ValueError, like the reference's
                          # "implementation not supported" ValueError (linear_attention.py:217-218)


def check(code: int) -> None:
    if code == 0:
        return
    msg = lib().based_hip_last_error().decode("utf-8", "replace")
    if code in _SHAPE_CODES or code == 4:
        raise ValueError(msg)
    raise BasedHipError(msg)
