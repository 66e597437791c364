"""The C-ABI library loads and exports every symbol include/based_hip.h declares, the ctypes
binding covers exactly that set, and argument validation works without a GPU (validation
happens before any HIP call)."""
import ctypes
import os
import re

import pytest

from based_amd import _lib

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def _declared():
    text = open(os.path.join(ROOT, "include", "based_hip.h")).read()
    return set(re.findall(r"BASED_API\s+[\w\s\*]+?\b(based_\w+)\s*\(", text))


def test_header_symbols_are_exported_and_bound():
    declared = _declared()
    assert {"based_linear_attn_step", "based_linear_attn_prefill", "based_swa_prefill", "based_swa_step",
            "based_hip_version", "based_hip_last_error"} <= declared
    assert os.path.exists(_lib.LIB_PATH), "build the library first: python -m based_amd.build"
    handle = ctypes.CDLL(_lib.LIB_PATH)
    for name in declared:
        assert hasattr(handle, name), f"{name} declared in the header but not exported"
    assert set(_lib.SIGNATURES) == declared


def test_header_constants_match_binding():
    text = open(os.path.join(ROOT, "include", "based_hip.h")).read()
    m = re.search(r"#define\s+BASED_PREFILL_SEGMENT_STATE_BYTES\s+(\d+)", text)
    assert m and int(m.group(1)) == _lib.PREFILL_SEGMENT_STATE_BYTES


def test_version_and_error_string():
    lib = _lib.lib()
    assert lib.based_hip_version() >= 1
    assert isinstance(lib.based_hip_last_error(), bytes)


def test_argument_validation_without_gpu():
    lib = _lib.lib()
    # null pointers -> BASED_ERR_ARG (4), nothing launched
    rc = lib.based_linear_attn_step(None, None, None, None, None, None, 1, 1, 64, 0, 0, 0, 0, 0, 0, 0, 0, 1e-12, 0, None)
    assert rc == 4 and b"null" in lib.based_hip_last_error()
    with pytest.raises(ValueError):
        _lib.check(rc)
    buf = (ctypes.c_float * 64)()
    p = ctypes.cast(buf, ctypes.c_void_p)
    # unsupported head dim -> BASED_ERR_SHAPE (1)
    rc = lib.based_linear_attn_step(p, p, p, p, p, p, 1, 1, 40, 0, 0, 0, 0, 0, 0, 0, 0, 1e-12, 0, None)
    assert rc == 1
    # window too wide -> BASED_ERR_SHAPE
    rc = lib.based_swa_prefill(p, p, p, p, 1, 1, 8, 0, 64, 64, 0, 64, 64, 0, 64, 64, 0, 64, 64, 129, 0.125, None, None, 0, None, None, 0, 0, 0, 0, 0, None)
    assert rc == 1
    # fp32 is not a sliding-window element type -> BASED_ERR_DTYPE (2)
    rc = lib.based_swa_prefill(p, p, p, p, 1, 1, 8, 0, 64, 64, 0, 64, 64, 0, 64, 64, 0, 64, 64, 64, 0.125, None, None, 0, None, None, 0, 0, 0, 0, 1, None)
    assert rc == 2
    # misaligned stride -> BASED_ERR_ALIGN (3)
    rc = lib.based_linear_attn_prefill(p, p, p, p, None, None, 1, 1, 8, 64, 0, 0, 20, 0, 0, 16, 0, 0, 64, 0, 0, 64, 1e-12, 0, None)
    assert rc == 3
    # one state pointer without the other -> BASED_ERR_ARG
    rc = lib.based_linear_attn_prefill(p, p, p, p, p, None, 1, 1, 8, 64, 0, 0, 16, 0, 0, 16, 0, 0, 64, 0, 0, 64, 1e-12, 0, None)
    assert rc == 4
    # empty batch is a no-op success
    rc = lib.based_swa_prefill(p, p, p, p, 0, 1, 8, 0, 64, 64, 0, 64, 64, 0, 64, 64, 0, 64, 64, 64, 0.125, None, None, 0, None, None, 0, 0, 0, 0, 0, None)
    assert rc == 0
    # one rotary table without the other -> BASED_ERR_ARG
    rc = lib.based_swa_prefill(p, p, p, p, 1, 1, 8, 0, 64, 64, 0, 64, 64, 0, 64, 64, 0, 64, 64, 64, 0.125, p, None, 8, None, None, 0, 0, 0, 0, 0, None)
    assert rc == 4
    # gated convolution: kernel size outside 2..4 -> BASED_ERR_SHAPE
    rc = lib.based_gated_conv_prefill(p, p, None, p, None, 1, 4, 8, 5, 64, 16, 32, 8, 0, 0, None)
    assert rc == 1
    # allocation-free segmented prefill: more scratch than the static array holds -> BASED_ERR_SHAPE,
    # refused before any HIP call
    rc = lib.based_linear_attn_prefill_split_static(p, p, p, p, None, None, 256, 16, 4096, 64, 0, 0, 16, 0, 0, 16,
                                                    0, 0, 64, 0, 0, 64, 1e-12, 0, 4, None)
    assert rc == 1 and b"scratch" in lib.based_hip_last_error()


def test_parts_hold_what_they_are_for():
    """The partial build for streamed models names existing sources, and these define every entry point
    the streamed operations call."""
    from based_amd import build

    text = ""
    for name in build.PARTS["streaming"]:
        text += open(os.path.join(build.CSRC, f"{name}.hip")).read()
    for entry in ("based_add_norm", "based_stream_conv", "based_window_attn_prefill", "based_window_attn_step",
                  "based_gated_delta_scan", "based_gated_rms_norm", "based_gated_delta_step", "based_rglru_prefill",
                  "based_rglru_step", "based_decode_linear_stream", "based_decode_linear", "based_swiglu", "based_greedy_step",
                  "based_hip_last_error"):
        assert re.search(rf"BASED_API [\w\*]+\s*\**{entry}\(|BASED_API const char\* {entry}\(", text), entry


def test_header_matches_argument_lists():
    """Every ctypes argument list has the number and kinds of arguments the header declares."""
    text = re.sub(r"/\*.*?\*/", "", open(os.path.join(ROOT, "include", "based_hip.h")).read(), flags=re.S)
    names = {"c_void_p": "p", "c_char_p": "p", "c_long": "l", "c_longlong": "l", "c_float": "f", "c_int": "i"}
    for m in re.finditer(r"BASED_API\s+[\w\s\*]+?\b(based_\w+)\s*\(([^;]*?)\);", text, re.S):
        args = [x for x in m.group(2).split(",") if x.strip() != "void"]
        kinds = ["p" if "*" in x else "l" if "int64" in x else "f" if "float" in x else "i" for x in args]
        assert kinds == [names.get(t.__name__, "p") for t in _lib.SIGNATURES[m.group(1)][1]], m.group(1)


def test_streamed_argument_validation_without_gpu():
    lib = _lib.lib()
    buf = (ctypes.c_float * 64)()
    p = ctypes.cast(buf, ctypes.c_void_p)
    assert lib.based_add_norm(None, None, None, None, None, 1, 8, 8, 8, 8, 8, 1e-5, 1, 1.0, 0, None) == 4
    # nine taps -> BASED_ERR_SHAPE; in place -> BASED_ERR_ARG
    q = ctypes.c_void_p(p.value + 64)
    assert lib.based_stream_conv(p, p, None, q, None, None, 0, 1, 1, 8, 9, 8, 8, 8, 8, 0, 0, 0, 0, None) == 1
    assert lib.based_stream_conv(p, p, None, p, None, None, 0, 1, 1, 8, 4, 8, 8, 8, 8, 0, 0, 0, 0, None) == 4
    # three query heads over two key/value heads; a portion that runs past the cache
    tail = (0.1, 0, 0.0, 1.0, None, None, 0, 0, 0, 0, None)
    assert lib.based_window_attn_prefill(p, p, p, p, p, 0, 1, 2, 3, 2, 8, 8, 4, *([8] * 10), 4, *tail) == 1
    assert lib.based_window_attn_prefill(p, p, p, p, p, 3, 1, 2, 2, 2, 8, 8, 4, *([8] * 10), 4, *tail) == 1
    # query/key size above 256
    assert lib.based_gated_delta_scan(*([p] * 10), 1, 1, 1, 1, 264, 8, 8, 8, 8, 8, 8, 1, 0, None) == 1
    # channels that do not divide into blocks
    assert lib.based_rglru_prefill(*([p] * 12), 1, 1, 10, 3, *([8] * 6), 8.0, 1, 0, None) == 1
    assert b"blocks" in lib.based_hip_last_error()
