"""Tensor-level wrappers over the C ABI: validate, take pointers/strides, enqueue on torch's
current stream.  PyTorch is used for device memory and streams only."""
from __future__ import annotations

import ctypes
import math
from typing import NamedTuple, Optional, Tuple

import torch

from . import _lib

FEATURE_DIM = 16
EXPANDED_DIM = 273


def _dtype_code(t: torch.Tensor) -> int:
    if t.dtype == torch.bfloat16:
        return _lib.BASED_BF16
    if t.dtype == torch.float32:
        return _lib.BASED_F32
    raise ValueError(f"unsupported dtype {t.dtype} (bfloat16 or float32)")


# torch's current stream on a device as a raw hipStream_t.  The private accessor skips building a
# Stream object (several microseconds per call, which a single-token step notices); where a torch
# build lacks it the public route is taken.
_raw_stream = getattr(torch._C, "_cuda_getCurrentRawStream", None)


def _stream_ptr(t: torch.Tensor) -> int:
    if _raw_stream is not None:
        return _raw_stream(t.device.index)
    return torch.cuda.current_stream(t.device).cuda_stream


class _on_device:
    """Enters `torch.cuda.device(dev)` only when dev is not already current (entering the context
    costs microseconds, which matters for single-token steps)."""

    __slots__ = ("ctx",)

    def __init__(self, dev: torch.device):
        self.ctx = None if torch.cuda.current_device() == dev.index else torch.cuda.device(dev)

    def __enter__(self):
        if self.ctx is not None:
            self.ctx.__enter__()

    def __exit__(self, *exc):
        if self.ctx is not None:
            self.ctx.__exit__(*exc)
        return False


# Argument checks of the single-token entry points are done once per distinct combination of
# shapes, strides, dtypes and device (a decode loop presents the same combination every step).
_CHECKED: dict = {}


def _require_cuda(*ts: torch.Tensor) -> None:
    dev = ts[0].device
    for t in ts:
        if not t.is_cuda:
            raise ValueError("based_amd kernels need tensors on a HIP device (no CPU path)")
        if t.device != dev:
            raise ValueError("all tensors must live on the same device")


def linear_attn_step(q, k, v, kv_state, k_state, eps: float = 1e-12, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """One decode step.  q, k: (B, H, 1, 16) raw; v: (B, H, 1, dv); kv_state (B,H,1,dv,273)
    and k_state (B,H,1,1,273) fp32 contiguous, updated in place.  Returns y (B, H, 1, dv)
    (written into `out` when given)."""
    key = ("lin_step", q.shape, q.stride(), k.shape, k.stride(), v.shape, v.stride(), kv_state.shape, kv_state.stride(),
           k_state.shape, k_state.stride(), q.dtype, k.dtype, v.dtype, kv_state.dtype, k_state.dtype, q.device,
           k.device, v.device, kv_state.device, k_state.device)
    if key not in _CHECKED:
        _require_cuda(q, k, v, kv_state, k_state)
        B, H, l, d = q.shape
        assert l == 1, f"q.shape is {tuple(q.shape)} but should be ({B}, {H}, 1, {d})"
        dv = v.shape[-1]
        if d != FEATURE_DIM or k.shape != q.shape or v.shape[:3] != q.shape[:3]:
            raise ValueError(f"bad shapes q{tuple(q.shape)} k{tuple(k.shape)} v{tuple(v.shape)}")
        if kv_state.dtype != torch.float32 or k_state.dtype != torch.float32:
            raise ValueError("decode states must be float32")
        if tuple(kv_state.shape) != (B, H, 1, dv, EXPANDED_DIM) or tuple(k_state.shape) != (B, H, 1, 1, EXPANDED_DIM):
            raise ValueError(f"bad state shapes {tuple(kv_state.shape)} {tuple(k_state.shape)}")
        if not (kv_state.is_contiguous() and k_state.is_contiguous()):
            raise ValueError("decode states must be contiguous")
        if not (q.dtype == k.dtype == v.dtype):
            raise ValueError("q, k, v must share a dtype")
        for t in (q, k, v):
            if t.stride(-1) != 1:
                raise ValueError("innermost dimension must be contiguous")
        _dtype_code(q)
        _CHECKED[key] = True
    B, H, _, _ = q.shape
    dv = v.shape[-1]
    if out is None:
        y = torch.empty(B, H, 1, dv, dtype=q.dtype, device=q.device)
    else:
        y = out
        if tuple(y.shape) != (B, H, 1, dv) or y.dtype != q.dtype or y.device != q.device or y.stride(-1) != 1:
            raise ValueError(f"out must be a ({B}, {H}, 1, {dv}) {q.dtype} tensor on {q.device}")
    with _on_device(q.device):
        _lib.check(_lib.lib().based_linear_attn_step(
            q.data_ptr(), k.data_ptr(), v.data_ptr(), kv_state.data_ptr(), k_state.data_ptr(), y.data_ptr(),
            B, H, dv,
            q.stride(0), q.stride(1), k.stride(0), k.stride(1),
            v.stride(0), v.stride(1), y.stride(0), y.stride(1),
            float(eps), _dtype_code(q), _stream_ptr(q)))
    return y


DEFERRED_MAX_STEPS = 8  # BASED_DEFERRED_MAX_STEPS


def deferred_step_buffers(batch: int, heads: int, dv: int, device) -> tuple:
    """The ring of `linear_attn_step_deferred` for (batch, heads) states: keys (B, H, 8, 16) and
    values (B, H, 8, dv) in fp32, and the per-(batch, head) fill count (B, H) int32, all zero."""
    return (torch.zeros(batch, heads, DEFERRED_MAX_STEPS, FEATURE_DIM, dtype=torch.float32, device=device),
            torch.zeros(batch, heads, DEFERRED_MAX_STEPS, dv, dtype=torch.float32, device=device),
            torch.zeros(batch, heads, dtype=torch.int32, device=device))


def _check_deferred(kv_state, pending):
    pend_k, pend_v, pend_n = pending
    B, H, _, dv, _ = kv_state.shape
    _require_cuda(kv_state, pend_k, pend_v, pend_n)
    if (tuple(pend_k.shape) != (B, H, DEFERRED_MAX_STEPS, FEATURE_DIM) or tuple(pend_v.shape) != (B, H, DEFERRED_MAX_STEPS, dv)
            or tuple(pend_n.shape) != (B, H)):
        raise ValueError(f"bad ring shapes {tuple(pend_k.shape)} {tuple(pend_v.shape)} {tuple(pend_n.shape)} for a "
                         f"state {tuple(kv_state.shape)}")
    if pend_k.dtype != torch.float32 or pend_v.dtype != torch.float32 or pend_n.dtype != torch.int32:
        raise ValueError("the ring is float32 keys and values and an int32 count")
    if not (pend_k.is_contiguous() and pend_v.is_contiguous() and pend_n.is_contiguous()):
        raise ValueError("the ring must be contiguous")


def linear_attn_step_deferred(q, k, v, kv_state, k_state, pending, period: int, eps: float = 1e-12,
                              out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """`linear_attn_step` with the write-back of kv_state deferred: the step reads kv_state, updates
    k_state and parks the token's raw k and v in `pending` (from `deferred_step_buffers`); every
    `period`-th step (1..8) applies the parked tokens and its own to kv_state in one pass.  The
    output is the one of `linear_attn_step` up to fp32 summation order; kv_state is current only
    after such a step or after `linear_attn_flush_deferred`.  Leading rows of larger states and
    rings may be passed (views of the first B rows)."""
    key = ("lin_step_deferred", q.shape, q.stride(), k.shape, k.stride(), v.shape, v.stride(), kv_state.shape,
           kv_state.stride(), k_state.shape, k_state.stride(), q.dtype, k.dtype, v.dtype, kv_state.dtype, k_state.dtype,
           q.device, k.device, v.device, kv_state.device, k_state.device,
           tuple((t.shape, t.stride(), t.dtype, t.device) for t in pending), int(period))
    if key not in _CHECKED:
        _require_cuda(q, k, v, kv_state, k_state)
        B, H, l, d = q.shape
        assert l == 1, f"q.shape is {tuple(q.shape)} but should be ({B}, {H}, 1, {d})"
        dv = v.shape[-1]
        if d != FEATURE_DIM or k.shape != q.shape or v.shape[:3] != q.shape[:3]:
            raise ValueError(f"bad shapes q{tuple(q.shape)} k{tuple(k.shape)} v{tuple(v.shape)}")
        if kv_state.dtype != torch.float32 or k_state.dtype != torch.float32:
            raise ValueError("decode states must be float32")
        if tuple(kv_state.shape) != (B, H, 1, dv, EXPANDED_DIM) or tuple(k_state.shape) != (B, H, 1, 1, EXPANDED_DIM):
            raise ValueError(f"bad state shapes {tuple(kv_state.shape)} {tuple(k_state.shape)}")
        if not (kv_state.is_contiguous() and k_state.is_contiguous()):
            raise ValueError("decode states must be contiguous")
        if not (q.dtype == k.dtype == v.dtype):
            raise ValueError("q, k, v must share a dtype")
        for t in (q, k, v):
            if t.stride(-1) != 1:
                raise ValueError("innermost dimension must be contiguous")
        if not 1 <= int(period) <= DEFERRED_MAX_STEPS:
            raise ValueError(f"period must be in [1, {DEFERRED_MAX_STEPS}], got {period}")
        _check_deferred(kv_state, pending)
        _dtype_code(q)
        _CHECKED[key] = True
    B, H, _, _ = q.shape
    dv = v.shape[-1]
    if out is None:
        y = torch.empty(B, H, 1, dv, dtype=q.dtype, device=q.device)
    else:
        y = out
        if tuple(y.shape) != (B, H, 1, dv) or y.dtype != q.dtype or y.device != q.device or y.stride(-1) != 1:
            raise ValueError(f"out must be a ({B}, {H}, 1, {dv}) {q.dtype} tensor on {q.device}")
    pend_k, pend_v, pend_n = pending
    with _on_device(q.device):
        _lib.check(_lib.lib().based_linear_attn_step_deferred(
            q.data_ptr(), k.data_ptr(), v.data_ptr(), kv_state.data_ptr(), k_state.data_ptr(), pend_k.data_ptr(),
            pend_v.data_ptr(), pend_n.data_ptr(), y.data_ptr(), B, H, dv,
            q.stride(0), q.stride(1), k.stride(0), k.stride(1), v.stride(0), v.stride(1), y.stride(0), y.stride(1),
            float(eps), int(period), _dtype_code(q), _stream_ptr(q)))
    return y


def linear_attn_flush_deferred(kv_state, pending) -> None:
    """Applies the tokens parked by `linear_attn_step_deferred` to kv_state (B,H,1,dv,273) and
    empties the ring."""
    if kv_state.dtype != torch.float32 or kv_state.dim() != 5 or not kv_state.is_contiguous():
        raise ValueError("kv_state must be a contiguous float32 (B, H, 1, dv, 273) tensor")
    _check_deferred(kv_state, pending)
    B, H, _, dv, _ = kv_state.shape
    pend_k, pend_v, pend_n = pending
    with _on_device(kv_state.device):
        _lib.check(_lib.lib().based_linear_attn_flush_deferred(kv_state.data_ptr(), pend_k.data_ptr(), pend_v.data_ptr(),
                                                               pend_n.data_ptr(), B, H, dv, _stream_ptr(kv_state)))


def _rope_tables(rope, device, need_rows, head_dim):
    """rope = (cos, sin) or (cos, sin, interleaved): fp32 (n_pos, rotary_dim / 2) contiguous device
    tables -> (cos_ptr, sin_ptr, n_pos, rotary_dim, interleaved), or Nones / zeros without rotary."""
    if rope is None:
        return None, None, 0, 0, False
    cos, sin = rope[0], rope[1]
    interleaved = bool(rope[2]) if len(rope) > 2 else False
    for t in (cos, sin):
        if not t.is_cuda or t.device != device or t.dtype != torch.float32 or t.dim() != 2 or not t.is_contiguous():
            raise ValueError("rotary tables must be contiguous fp32 (n_pos, rotary_dim / 2) tensors on the device of q")
    rotary_dim = 2 * cos.shape[1]
    if cos.shape != sin.shape or cos.shape[0] < need_rows:
        raise ValueError(f"rotary tables hold {cos.shape[0]} positions, need {need_rows}")
    if rotary_dim % 16 != 0 or not 0 < rotary_dim <= head_dim:
        raise ValueError(f"rotary_dim {rotary_dim} must be a multiple of 16 and at most the head dim {head_dim}")
    return cos.data_ptr(), sin.data_ptr(), cos.shape[0], rotary_dim, interleaved


def _swa_fast64(D: int, rotary_dim: int, interleaved: bool, impl) -> bool:
    """Head dim 64 without rotary, or rotated over the whole head in half-split pairs, runs the
    kernels built for exactly that (two heads per workgroup, 128-byte rows)."""
    return impl is None and D == 64 and (rotary_dim == 0 or (rotary_dim == 64 and not interleaved))


def swa_prefill(q, k, v, w_left: int = 64, scale: Optional[float] = None, rope=None, kv_cache=None,
                out: Optional[torch.Tensor] = None, impl: Optional[str] = None) -> torch.Tensor:
    """Sliding-window causal attention.  q, k, v: (B, L, H, D) bf16 (any strides with the
    last dim contiguous, e.g. slices of a packed qkv), D a multiple of 8 up to 128.  Query i sees
    keys [i - w_left, i], 0 <= w_left <= 128.
    rope: None, or (cos, sin[, interleaved]) with fp32 (n_pos >= L, rotary_dim / 2) tables: the
    first rotary_dim channels of q and k are rotated in the kernel at positions 0..L-1, in
    half-split pairs (c, c + rotary_dim / 2) or, interleaved, pairs (2i, 2i + 1).
    kv_cache: None or a (B, max_seqlen >= L, 2, H, D) bf16 cache whose rows 0..L-1 receive the
    (rotated) k and v.  out: None or a (B, L, H, D) tensor (last dim contiguous) to write into.
    impl: None (MFMA kernels), "wide" (the general MFMA kernel also where the 64-channel one would
    do) or "plain" (the one-wavefront-per-query kernel, no rotary: a second statement for tests)."""
    _require_cuda(q, k, v)
    B, L, H, D = q.shape
    if k.shape != q.shape or v.shape != q.shape:
        raise ValueError(f"bad shapes q{tuple(q.shape)} k{tuple(k.shape)} v{tuple(v.shape)}")
    for t in (q, k, v):
        if t.stride(-1) != 1:
            raise ValueError("innermost dimension must be contiguous")
    scale = 1.0 / math.sqrt(D) if scale is None else float(scale)
    cos_ptr, sin_ptr, n_pos, rotary_dim, interleaved = _rope_tables(rope, q.device, L, D)
    if impl == "plain" and rope is not None:
        raise ValueError("the plain kernel has no in-kernel rotary")
    kc_ptr = vc_ptr = None
    c_strides, max_seqlen = (0, 0, 0), 0
    if kv_cache is not None:
        _require_cuda(q, kv_cache)
        if (kv_cache.dim() != 5 or kv_cache.shape[0] != B or kv_cache.shape[2] != 2
                or tuple(kv_cache.shape[3:]) != (H, D) or kv_cache.dtype != q.dtype or kv_cache.stride(-1) != 1):
            raise ValueError(f"bad cache {tuple(kv_cache.shape)} {kv_cache.dtype}")
        kc, vc = kv_cache[:, :, 0], kv_cache[:, :, 1]
        kc_ptr, vc_ptr = kc.data_ptr(), vc.data_ptr()
        c_strides, max_seqlen = (kc.stride(0), kc.stride(1), kc.stride(2)), kv_cache.shape[1]
    if out is None:
        o = torch.empty(B, L, H, D, dtype=q.dtype, device=q.device)
    else:
        o = out
        if tuple(o.shape) != (B, L, H, D) or o.dtype != q.dtype or o.device != q.device or o.stride(-1) != 1:
            raise ValueError(f"out must be a ({B}, {L}, {H}, {D}) {q.dtype} tensor on {q.device}")
    strides = (q.stride(0), q.stride(1), q.stride(2), k.stride(0), k.stride(1), k.stride(2),
               v.stride(0), v.stride(1), v.stride(2), o.stride(0), o.stride(1), o.stride(2))
    with _on_device(q.device):
        if _swa_fast64(D, rotary_dim, interleaved, impl):
            _lib.check(_lib.lib().based_swa_prefill(
                q.data_ptr(), k.data_ptr(), v.data_ptr(), o.data_ptr(), B, H, L, *strides,
                int(w_left), scale, cos_ptr, sin_ptr, n_pos, kc_ptr, vc_ptr, *c_strides, max_seqlen,
                _dtype_code(q), _stream_ptr(q)))
        elif impl == "plain":
            _lib.check(_lib.lib().based_swa_prefill_anydim(
                q.data_ptr(), k.data_ptr(), v.data_ptr(), o.data_ptr(), B, H, L, D, *strides,
                int(w_left), scale, kc_ptr, vc_ptr, *c_strides, max_seqlen, _dtype_code(q), _stream_ptr(q)))
        else:
            _lib.check(_lib.lib().based_swa_prefill_wide(
                q.data_ptr(), k.data_ptr(), v.data_ptr(), o.data_ptr(), B, H, L, D, *strides,
                int(w_left), scale, cos_ptr, sin_ptr, n_pos, rotary_dim, int(interleaved), kc_ptr, vc_ptr, *c_strides,
                max_seqlen, _dtype_code(q), _stream_ptr(q)))
    return o


def swa_step(q, k_new, v_new, kv_cache, pos, w_left: int = 64, scale: Optional[float] = None, rope=None,
             out: Optional[torch.Tensor] = None, impl: Optional[str] = None) -> torch.Tensor:
    """Decode step.  q, k_new, v_new: (B, 1, H, D) bf16; kv_cache (B, max_seqlen, 2, H, D)
    bf16, row `pos` is written in place, then rows [pos - w_left, pos] are attended.  D a multiple
    of 8 up to 128.
    pos: int (same for the whole batch) or an int32 device tensor of B positions.
    rope: None or (cos, sin[, interleaved]) tables as for swa_prefill: q and k_new are rotated at `pos` first.
    out: None or a (B, 1, H, D) tensor (last dim contiguous) to write into.  impl: as for swa_prefill."""
    key = ("swa_step", q.shape, q.stride(), k_new.shape, k_new.stride(), v_new.shape, v_new.stride(), kv_cache.shape,
           kv_cache.stride(), q.dtype, k_new.dtype, v_new.dtype, kv_cache.dtype, q.device, k_new.device, v_new.device,
           kv_cache.device)
    if key not in _CHECKED:
        _require_cuda(q, k_new, v_new, kv_cache)
        B, one, H, D = q.shape
        if one != 1 or k_new.shape != q.shape or v_new.shape != q.shape:
            raise ValueError(f"bad shapes q{tuple(q.shape)} k{tuple(k_new.shape)} v{tuple(v_new.shape)}")
        if kv_cache.dim() != 5 or kv_cache.shape[0] < B or kv_cache.shape[2] != 2 or tuple(kv_cache.shape[3:]) != (H, D):
            raise ValueError(f"bad cache shape {tuple(kv_cache.shape)}")
        if kv_cache.dtype != q.dtype or kv_cache.stride(-1) != 1:
            raise ValueError("cache must share q's dtype and have a contiguous last dim")
        for t in (q, k_new, v_new):
            if t.stride(-1) != 1:
                raise ValueError("innermost dimension must be contiguous")
        _dtype_code(q)
        _CHECKED[key] = True
    B, _, H, D = q.shape
    scale = 1.0 / math.sqrt(D) if scale is None else float(scale)
    if impl == "plain" and rope is not None:
        raise ValueError("the plain kernel has no in-kernel rotary")
    if isinstance(pos, torch.Tensor):
        if pos.dtype != torch.int32 or not pos.is_cuda or pos.numel() < B or not pos.is_contiguous():
            raise ValueError("cache_seqlens must be a contiguous int32 device tensor with B entries")
        seq_ptr, pos_host = pos.data_ptr(), 0
        cos_ptr, sin_ptr, n_pos, rotary_dim, interleaved = _rope_tables(rope, q.device, 1, D)
    else:
        seq_ptr, pos_host = None, int(pos)
        cos_ptr, sin_ptr, n_pos, rotary_dim, interleaved = _rope_tables(rope, q.device, pos_host + 1, D)
    if out is None:
        o = torch.empty(B, 1, H, D, dtype=q.dtype, device=q.device)
    else:
        o = out
        if tuple(o.shape) != (B, 1, H, D) or o.dtype != q.dtype or o.device != q.device or o.stride(-1) != 1:
            raise ValueError(f"out must be a ({B}, 1, {H}, {D}) {q.dtype} tensor on {q.device}")
    c_sb, c_st, _, c_sh, _ = kv_cache.stride()
    kc_ptr = kv_cache.data_ptr()
    vc_ptr = kc_ptr + kv_cache.stride(2) * kv_cache.element_size()
    strides = (q.stride(0), q.stride(2), k_new.stride(0), k_new.stride(2),
               v_new.stride(0), v_new.stride(2), o.stride(0), o.stride(2), c_sb, c_st, c_sh)
    with _on_device(q.device):
        if _swa_fast64(D, rotary_dim, interleaved, impl):
            _lib.check(_lib.lib().based_swa_step(
                q.data_ptr(), k_new.data_ptr(), v_new.data_ptr(), kc_ptr, vc_ptr, o.data_ptr(),
                seq_ptr, pos_host, B, H, kv_cache.shape[1], *strides,
                int(w_left), scale, cos_ptr, sin_ptr, n_pos, _dtype_code(q), _stream_ptr(q)))
        elif impl == "plain":
            _lib.check(_lib.lib().based_swa_step_anydim(
                q.data_ptr(), k_new.data_ptr(), v_new.data_ptr(), kc_ptr, vc_ptr, o.data_ptr(),
                seq_ptr, pos_host, B, H, D, kv_cache.shape[1], *strides, int(w_left), scale, _dtype_code(q),
                _stream_ptr(q)))
        else:
            _lib.check(_lib.lib().based_swa_step_wide(
                q.data_ptr(), k_new.data_ptr(), v_new.data_ptr(), kc_ptr, vc_ptr, o.data_ptr(),
                seq_ptr, pos_host, B, H, D, kv_cache.shape[1], *strides, int(w_left), scale,
                cos_ptr, sin_ptr, n_pos, rotary_dim, int(interleaved), _dtype_code(q), _stream_ptr(q)))
    return o


def linear_attn_prefill(q, k, v, eps: float = 1e-12, return_state: bool = False, split=None
                        ) -> Tuple[torch.Tensor, Optional[torch.Tensor], Optional[torch.Tensor]]:
    """Causal Taylor linear attention.  q, k: (B, H, L, 16) raw; v: (B, H, L, dv); any strides
    with the last dim contiguous (e.g. `(B, L, H, d).transpose(1, 2)` views).

    Returns (y, kv_state, k_state): y (B, H, L, dv) in q's dtype, stored so that
    `y.transpose(1, 2).reshape(B, L, H*dv)` is a free view; states are fp32
    (B, H, 1, dv, 273) / (B, H, 1, 1, 273), or None unless return_state.

    split: None = let the library decide whether to scan each sequence in concurrent segments
    (small batches); False = never; an int > 1 = that many segments."""
    _require_cuda(q, k, v)
    B, H, L, d = q.shape
    dv = v.shape[-1]
    if d != FEATURE_DIM or k.shape != q.shape or tuple(v.shape[:3]) != (B, H, L):
        raise ValueError(f"bad shapes q{tuple(q.shape)} k{tuple(k.shape)} v{tuple(v.shape)} (feature dim 16)")
    if not (q.dtype == k.dtype == v.dtype):
        raise ValueError("q, k, v must share a dtype")
    for t in (q, k, v):
        if t.stride(-1) != 1:
            raise ValueError("innermost dimension must be contiguous")
    y = torch.empty(B, L, H, dv, dtype=q.dtype, device=q.device).transpose(1, 2)
    kv_state = k_state = None
    if return_state:
        kv_state = torch.empty(B, H, 1, dv, EXPANDED_DIM, dtype=torch.float32, device=q.device)
        k_state = torch.empty(B, H, 1, 1, EXPANDED_DIM, dtype=torch.float32, device=q.device)
    lib = _lib.lib()
    n_seg, ws_bytes = ctypes.c_int64(1), ctypes.c_int64(0)
    if split is not False:
        _lib.check(lib.based_linear_attn_prefill_plan(B, H, L, dv, _dtype_code(q), ctypes.byref(n_seg),
                                                      ctypes.byref(ws_bytes)))
    if isinstance(split, int) and not isinstance(split, bool) and split > 1:
        n_seg = ctypes.c_int64(split)  # explicit segment count (tests)
        ws_bytes = ctypes.c_int64(B * H * ((dv + 63) // 64) * split * _lib.PREFILL_SEGMENT_STATE_BYTES)
    args = (q.data_ptr(), k.data_ptr(), v.data_ptr(), y.data_ptr(),
            kv_state.data_ptr() if return_state else None, k_state.data_ptr() if return_state else None,
            B, H, L, dv,
            q.stride(0), q.stride(1), q.stride(2), k.stride(0), k.stride(1), k.stride(2),
            v.stride(0), v.stride(1), v.stride(2), y.stride(0), y.stride(1), y.stride(2),
            float(eps), _dtype_code(q))
    with _on_device(q.device):
        if n_seg.value > 1:
            # scratch for the per-segment states; torch's caching allocator makes this cheap
            ws = torch.empty(ws_bytes.value, dtype=torch.uint8, device=q.device)
            _lib.check(lib.based_linear_attn_prefill_split(*args, n_seg.value, ws.data_ptr(), ws_bytes.value,
                                                           _stream_ptr(q)))
        else:
            _lib.check(lib.based_linear_attn_prefill(*args, _stream_ptr(q)))
    return y, kv_state, k_state


def gated_conv_prefill(u, weight, bias=None, state=None, gated: bool = True) -> torch.Tensor:
    """y = silu(causal depthwise conv(u[..., :D]) + bias) * u[..., D:].  u: (B, L, 2D) with a
    contiguous last dimension; weight: the (D, 1, K) nn.Conv1d weight; bias (D) or None; state
    None or (B, D, K) contiguous, overwritten with the last K inputs.  Returns y (B, L, D).
    gated=False: the convolution alone, y = conv(u) + bias with u (B, L, D)."""
    _require_cuda(u, weight)
    if u.dim() != 3 or (gated and u.shape[-1] % 2 != 0):
        raise ValueError(f"u must be (B, L, 2D), got {tuple(u.shape)}")
    B, L, D2 = u.shape
    D = D2 // 2 if gated else D2
    if weight.dim() != 3 or weight.shape[0] != D or weight.shape[1] != 1:
        raise ValueError(f"weight must be ({D}, 1, K), got {tuple(weight.shape)}")
    K = weight.shape[2]
    if weight.dtype != u.dtype or (bias is not None and bias.dtype != u.dtype):
        raise ValueError("weight and bias must have the dtype of u")
    if u.stride(-1) != 1:
        raise ValueError("innermost dimension must be contiguous")
    weight = weight.contiguous()
    if bias is not None:
        _require_cuda(u, bias)
        bias = bias.contiguous()
        if tuple(bias.shape) != (D,):
            raise ValueError(f"bias must be ({D},), got {tuple(bias.shape)}")
    state_code = _lib.BASED_BF16
    if state is not None:
        _require_cuda(u, state)
        if tuple(state.shape) != (B, D, K) or not state.is_contiguous():
            raise ValueError(f"state must be a contiguous ({B}, {D}, {K}) tensor, got {tuple(state.shape)}")
        state_code = _dtype_code(state)
    y = torch.empty(B, L, D, dtype=u.dtype, device=u.device)
    fn = _lib.lib().based_gated_conv_prefill if gated else _lib.lib().based_short_conv_prefill
    with _on_device(u.device):
        _lib.check(fn(
            u.data_ptr(), weight.data_ptr(), bias.data_ptr() if bias is not None else None, y.data_ptr(),
            state.data_ptr() if state is not None else None, B, L, D, K,
            u.stride(0), u.stride(1), y.stride(0), y.stride(1), _dtype_code(u), state_code, _stream_ptr(u)))
    return y


def gated_conv_step(u, state, weight, bias=None, gated: bool = True) -> torch.Tensor:
    """Single-token gated short convolution.  u: (B, 1, 2D) or (B, 2D); state (B, D, K)
    contiguous, rolled and updated in place.  Returns y with u's leading shape and D channels.
    gated=False: the convolution alone on u (B, 1, D) or (B, D)."""
    _require_cuda(u, state, weight)
    squeeze = u.dim() == 3
    if squeeze:
        if u.shape[1] != 1:
            raise ValueError(f"step takes one token, got {tuple(u.shape)}")
        u2d = u[:, 0]
    else:
        u2d = u
    B, D2 = u2d.shape
    D = D2 // 2 if gated else D2
    K = weight.shape[-1]
    if tuple(weight.shape) != (D, 1, K) or tuple(state.shape) != (B, D, K) or not state.is_contiguous():
        raise ValueError(f"bad shapes u{tuple(u.shape)} weight{tuple(weight.shape)} state{tuple(state.shape)}")
    if weight.dtype != u.dtype or (bias is not None and bias.dtype != u.dtype):
        raise ValueError("weight and bias must have the dtype of u")
    if u2d.stride(-1) != 1:
        raise ValueError("innermost dimension must be contiguous")
    weight = weight.contiguous()
    if bias is not None:
        _require_cuda(u, bias)
        bias = bias.contiguous()
    y = torch.empty(B, D, dtype=u.dtype, device=u.device)
    fn = _lib.lib().based_gated_conv_step if gated else _lib.lib().based_short_conv_step
    with _on_device(u.device):
        _lib.check(fn(
            u2d.data_ptr(), state.data_ptr(), weight.data_ptr(), bias.data_ptr() if bias is not None else None,
            y.data_ptr(), B, D, K, u2d.stride(0), y.stride(0), _dtype_code(u), _dtype_code(state), _stream_ptr(u)))
    return y.unsqueeze(1) if squeeze else y


ADD_RMS_NORM_MAX_DIM = 4096  # widest row based_add_rms_norm takes


def add_rms_norm(x, residual, weight, eps: float = 1e-5, residual_in_fp32: bool = True, want_residual: bool = True):
    """Prenorm block glue in one launch: r = x + residual (r = x when residual is None),
    y = rms_norm(r cast to x.dtype) * weight, and r itself (fp32 when residual_in_fp32, else
    x.dtype).  x: (..., D) with contiguous rows; returns (y, r) with r None if not wanted."""
    D = x.shape[-1]
    key = ("add_rms_norm", x.shape, x.stride(), x.dtype, x.device, weight.shape, weight.dtype, weight.device,
           None if residual is None else (residual.shape, residual.stride(), residual.dtype, residual.device))
    if key not in _CHECKED:
        _require_cuda(x, weight)
        if weight.shape != (D,) or weight.dtype != x.dtype or not weight.is_contiguous():
            raise ValueError(f"weight must be a contiguous ({D},) of {x.dtype}, got {tuple(weight.shape)} {weight.dtype}")
        if residual is not None:
            _require_cuda(x, residual)
            if residual.shape != x.shape:
                raise ValueError(f"residual {tuple(residual.shape)} does not match x {tuple(x.shape)}")
            if x.dtype == torch.float32 and residual.dtype != torch.float32:
                raise ValueError("fp32 activations need an fp32 residual stream")
            if residual.dtype not in (torch.float32, torch.bfloat16):
                raise ValueError(f"unsupported residual dtype {residual.dtype}")
        _dtype_code(x)
        _CHECKED[key] = True
    x2 = x if x.dim() == 2 else x.reshape(-1, D)
    if x2.stride(-1) != 1:
        x2 = x2.contiguous()
    rows = x2.shape[0]
    res_dtype = torch.float32 if residual_in_fp32 else x.dtype
    r2 = None
    if residual is not None:
        # a residual stream of another dtype (first block with residual_in_fp32=False, ...) keeps its own
        res_dtype = residual.dtype
        r2 = residual if residual.dim() == 2 else residual.reshape(-1, D)
        if r2.stride(-1) != 1:
            r2 = r2.contiguous()
    if x.dtype == torch.float32 and res_dtype != torch.float32:
        raise ValueError("fp32 activations need an fp32 residual stream")
    y = torch.empty(rows, D, dtype=x.dtype, device=x.device)
    out = torch.empty(rows, D, dtype=res_dtype, device=x.device) if want_residual else None
    res_code = _lib.BASED_F32 if res_dtype == torch.float32 else _lib.BASED_BF16
    with _on_device(x.device):
        _lib.check(_lib.lib().based_add_rms_norm(
            x2.data_ptr(), r2.data_ptr() if r2 is not None else None, weight.data_ptr(), y.data_ptr(),
            out.data_ptr() if out is not None else None, rows, D, x2.stride(0),
            r2.stride(0) if r2 is not None else 0, D, D if out is not None else 0,
            float(eps), _dtype_code(x), res_code, _stream_ptr(x)))
    return y.view(x.shape), (out.view(x.shape) if out is not None else None)


def swiglu(u) -> torch.Tensor:
    """u (..., 2F) -> u[..., :F] * silu(u[..., F:]), one pass."""
    _require_cuda(u)
    F2 = u.shape[-1]
    if F2 % 2 != 0:
        raise ValueError(f"last dimension must be even, got {F2}")
    F = F2 // 2
    u2 = u.reshape(-1, F2)
    if u2.stride(-1) != 1:
        u2 = u2.contiguous()
    out = torch.empty(u2.shape[0], F, dtype=u.dtype, device=u.device)
    with _on_device(u.device):
        _lib.check(_lib.lib().based_swiglu(u2.data_ptr(), out.data_ptr(), u2.shape[0], F, u2.stride(0), out.stride(0),
                                           _dtype_code(u), _stream_ptr(u)))
    return out.view(*u.shape[:-1], F)


def greedy_step(logits, next_ids, lengths, sequences=None, position_ids=None, vocab_size=None) -> None:
    """Greedy sampling of one decoding step plus the loop's bookkeeping, in one launch (recordable
    in the decode graph): per row b, tok = argmax(logits[b, :vocab_size]) (first index of the
    maximum, NaN largest, as torch.argmax), written to next_ids[b] and to
    sequences[b, lengths[b] + 1]; lengths[b] and position_ids[b] advance by one.

    logits (B, V) bf16 / fp32 with contiguous rows; next_ids (B,) or (B, 1) int64; lengths (B,)
    int32; sequences (B, max_length) int64 or None; position_ids (B,) or (B, 1) int64 or None."""
    _require_cuda(logits, next_ids, lengths)
    if logits.ndim != 2 or logits.stride(-1) != 1:
        raise ValueError("logits must be (B, V) with contiguous rows")
    B, V = logits.shape
    V = V if vocab_size is None else int(vocab_size)
    if not 0 < V <= logits.shape[1]:
        raise ValueError(f"vocab_size {V} outside (0, {logits.shape[1]}]")
    if next_ids.dtype != torch.int64 or next_ids.numel() != B or lengths.dtype != torch.int32 or lengths.numel() != B \
            or not lengths.is_contiguous():
        raise ValueError("next_ids must hold B int64 values, lengths B contiguous int32 values")
    for t, name in ((sequences, "sequences"), (position_ids, "position_ids")):
        if t is not None and (t.dtype != torch.int64 or t.shape[0] != B or not t.is_cuda):
            raise ValueError(f"{name} must be an int64 device tensor with B rows")
    if sequences is not None and (sequences.ndim != 2 or sequences.stride(1) != 1):
        raise ValueError("sequences must be (B, max_length) with contiguous rows")
    if position_ids is not None and position_ids.numel() != B:
        raise ValueError("position_ids must hold B values")
    with _on_device(logits.device):
        _lib.check(_lib.lib().based_greedy_step(
            logits.data_ptr(), B, V, logits.stride(0), next_ids.data_ptr(), next_ids.stride(0),
            sequences.data_ptr() if sequences is not None else None,
            sequences.stride(0) if sequences is not None else 0,
            sequences.shape[1] if sequences is not None else 0, lengths.data_ptr(),
            position_ids.data_ptr() if position_ids is not None else None,
            position_ids.stride(0) if position_ids is not None else 0, _dtype_code(logits), _stream_ptr(logits)))


DECODE_LINEAR_MAX_ROWS = 32  # BASED_DECODE_LINEAR_MAX_ROWS of include/based_hip.h
PROLOGUE_NONE, PROLOGUE_ADD_RMS_NORM, PROLOGUE_SWIGLU, PROLOGUE_STREAM = 0, 1, 2, 3
EPILOGUE_NONE, EPILOGUE_SWIGLU, EPILOGUE_GATED_CONV_STEP = 0, 1, 2


def decode_linear_weight_ok(weight: torch.Tensor) -> bool:
    """Whether `decode_linear` takes projections through this weight: bf16 (N, K) on the GPU with
    contiguous rows, K a multiple of 8 up to 4096."""
    return (weight.is_cuda and weight.dtype == torch.bfloat16 and weight.dim() == 2 and weight.stride(1) == 1
            and weight.stride(0) % 8 == 0 and weight.shape[1] % 8 == 0 and weight.shape[1] <= 4096)


def decode_linear(x, weight, bias=None, *, prologue: int = PROLOGUE_NONE, residual_in=None, residual_out=None,
                  norm_weight=None, eps: float = 1e-5, row_index=None, epilogue: int = EPILOGUE_NONE,
                  conv_state=None, conv_weight=None, conv_bias=None, out: Optional[torch.Tensor] = None,
                  mult: float = 1.0, norm_kind: int = 0, input_conv=None, addends=None, mix=None, gate=None,
                  softcap: float = 0.0) -> torch.Tensor:
    """y = epi(pro(x) @ weight.T (+ bias)) for the few rows of a single-token step, one launch.

    x: (M, K) bf16 rows (M <= 32; any leading shape is flattened), or for PROLOGUE_SWIGLU (M, 2K):
    value | gate.  weight: (N, K) bf16; bias None or (N).  PROLOGUE_ADD_RMS_NORM first forms
    r = x + residual_in (fp32, residual_in may be None), writes r to residual_out (fp32, may be
    None, never residual_in itself) and projects rms_norm(r) * norm_weight.  row_index: None, or an
    int64 device vector of M row numbers into x (the embedding table).
    EPILOGUE_SWIGLU: weight is (2F, K), y[:, f] = p[:, f] * silu(p[:, F + f]).
    EPILOGUE_GATED_CONV_STEP: weight is (2F, K); the gated short-convolution step on p with
    conv_state (M, F, k) rolled in place, conv_weight the (F, 1, k) or (F, k) Conv1d weight,
    conv_bias None or (F).  Returns y (M, N) or (M, F), written into `out` when given.

    PROLOGUE_STREAM: r = residual_in + mult * x in fp32 (written to residual_out), then the norm
    `norm_kind` of that sum times norm_weight, rounded to bf16, and with input_conv =
    (weight (taps, K), ring (M, taps, K), pos) that row plus its causal convolution; epilogues NONE and
    SWIGLU.  Instead of input_conv: `addends` (`Addends`) in the sum, NORM_NONE; mix = (mu (S, K), ring (M, 2, K), pos, rows):
    weight rows i * rows .. read the i-th mix of the row with the one of the token before (`token_mix`), the last mix
    all rows that are left; gate = (table (n, N), index (M)): gelu_tanh(y) * table[index]; softcap > 0: softcap * tanh(y / softcap)."""
    if prologue == PROLOGUE_STREAM:
        if conv_state is not None or conv_weight is not None or conv_bias is not None:
            raise ValueError("the streamed-input prologue has no convolution epilogue")
        if addends is not None or mix is not None or gate is not None or softcap or norm_kind == NORM_NONE:
            if input_conv is not None:
                raise ValueError("an input convolution takes no addends, mixes, gate or cap")
            return _decode_linear_extras(x, weight, bias, epilogue, residual_in, residual_out, norm_weight, eps, row_index, mult,
                                         norm_kind, addends or Addends(), mix, gate, softcap, out)
        return _decode_linear_stream(x, weight, bias, epilogue, residual_in, residual_out, norm_weight, eps, row_index, mult,
                                     norm_kind, input_conv, out)
    if addends is not None or mix is not None or gate is not None or softcap:
        raise ValueError("addends, mixes, gate and cap belong to PROLOGUE_STREAM")
    N, K = weight.shape
    x2 = x if x.dim() == 2 else x.reshape(-1, x.shape[-1])
    M = x2.shape[0] if row_index is None else row_index.numel()
    n_out = N if epilogue == EPILOGUE_NONE else N // 2
    key = ("decode_linear", x2.shape, x2.stride(), x2.dtype, x2.device, weight.shape, weight.stride(), weight.dtype,
           weight.device, prologue, epilogue,
           None if bias is None else (bias.shape, bias.dtype, bias.device, bias.stride()),
           None if residual_in is None else (residual_in.shape, residual_in.stride(), residual_in.dtype, residual_in.device),
           None if residual_out is None else (residual_out.shape, residual_out.stride(), residual_out.dtype, residual_out.device),
           None if norm_weight is None else (norm_weight.shape, norm_weight.dtype, norm_weight.device, norm_weight.stride()),
           None if row_index is None else (row_index.shape, row_index.dtype, row_index.device, row_index.stride()),
           None if conv_state is None else (conv_state.shape, conv_state.stride(), conv_state.dtype, conv_state.device),
           None if conv_weight is None else (conv_weight.shape, conv_weight.stride(), conv_weight.dtype, conv_weight.device),
           None if conv_bias is None else (conv_bias.shape, conv_bias.stride(), conv_bias.dtype, conv_bias.device))
    if key not in _CHECKED:
        _require_cuda(x2, weight)
        if x2.dtype != torch.bfloat16 or weight.dtype != torch.bfloat16:
            raise ValueError("decode_linear takes bfloat16 activations and weights")
        if weight.dim() != 2 or weight.stride(1) != 1 or x2.stride(1) != 1:
            raise ValueError("weight must be (N, K) and rows of x and weight contiguous")
        if x2.shape[1] != (2 * K if prologue == PROLOGUE_SWIGLU else K):
            raise ValueError(f"x {tuple(x.shape)} does not match weight {tuple(weight.shape)} (prologue {prologue})")
        if M > DECODE_LINEAR_MAX_ROWS:
            raise ValueError(f"decode_linear takes at most {DECODE_LINEAR_MAX_ROWS} rows, got {M}")
        if bias is not None:
            _require_cuda(x2, bias)
            if tuple(bias.shape) != (N,) or bias.dtype != torch.bfloat16 or not bias.is_contiguous():
                raise ValueError(f"bias must be a contiguous bfloat16 ({N},)")
        if prologue == PROLOGUE_ADD_RMS_NORM:
            if norm_weight is None:
                raise ValueError("the norm prologue needs norm_weight")
            _require_cuda(x2, norm_weight)
            if tuple(norm_weight.shape) != (K,) or norm_weight.dtype != torch.bfloat16 or not norm_weight.is_contiguous():
                raise ValueError(f"norm_weight must be a contiguous bfloat16 ({K},)")
            for r in (residual_in, residual_out):
                if r is not None:
                    _require_cuda(x2, r)
                    if r.dtype != torch.float32 or r.dim() != 2 or tuple(r.shape) != (M, K) or r.stride(1) != 1:
                        raise ValueError(f"residuals must be float32 ({M}, {K}) with contiguous rows")
        elif residual_in is not None or residual_out is not None or norm_weight is not None:
            raise ValueError("residual and norm arguments belong to PROLOGUE_ADD_RMS_NORM")
        if row_index is not None:
            _require_cuda(x2, row_index)
            if row_index.dtype != torch.int64 or row_index.dim() != 1 or not row_index.is_contiguous():
                raise ValueError("row_index must be a contiguous int64 device vector")
        if epilogue != EPILOGUE_NONE and N % 2 != 0:
            raise ValueError("a paired epilogue needs an even number of weight rows")
        if epilogue == EPILOGUE_GATED_CONV_STEP:
            if conv_state is None or conv_weight is None:
                raise ValueError("the convolution epilogue needs conv_state and conv_weight")
            _require_cuda(x2, conv_state, conv_weight)
            k = conv_weight.shape[-1]
            if (conv_weight.numel() != n_out * k or conv_weight.shape[0] != n_out or not conv_weight.is_contiguous()
                    or conv_weight.dtype != torch.bfloat16):
                raise ValueError(f"conv_weight must be a contiguous bfloat16 ({n_out}, 1, k), got {tuple(conv_weight.shape)}")
            if tuple(conv_state.shape) != (M, n_out, k) or not conv_state.is_contiguous():
                raise ValueError(f"conv_state must be a contiguous ({M}, {n_out}, {k}) tensor, got {tuple(conv_state.shape)}")
            _dtype_code(conv_state)
            if conv_bias is not None:
                _require_cuda(x2, conv_bias)
                if tuple(conv_bias.shape) != (n_out,) or conv_bias.dtype != torch.bfloat16 or not conv_bias.is_contiguous():
                    raise ValueError(f"conv_bias must be a contiguous bfloat16 ({n_out},)")
        elif conv_state is not None or conv_weight is not None or conv_bias is not None:
            raise ValueError("convolution arguments belong to EPILOGUE_GATED_CONV_STEP")
        _CHECKED[key] = True
    if out is None:
        y = torch.empty(M, n_out, dtype=torch.bfloat16, device=x2.device)
    else:
        y = out
        if tuple(y.shape) != (M, n_out) or y.dtype != torch.bfloat16 or y.device != x2.device or y.stride(1) != 1:
            raise ValueError(f"out must be a ({M}, {n_out}) bfloat16 tensor on {x2.device} with contiguous rows")
    conv = epilogue == EPILOGUE_GATED_CONV_STEP
    with _on_device(x2.device):
        _lib.check(_lib.lib().based_decode_linear(
            x2.data_ptr(), x2.stride(0), None if row_index is None else row_index.data_ptr(),
            x2.shape[0] if row_index is not None else 0,
            weight.data_ptr(), weight.stride(0), None if bias is None else bias.data_ptr(),
            y.data_ptr(), y.stride(0), M, N, K, prologue,
            None if residual_in is None else residual_in.data_ptr(), 0 if residual_in is None else residual_in.stride(0),
            None if residual_out is None else residual_out.data_ptr(), 0 if residual_out is None else residual_out.stride(0),
            None if norm_weight is None else norm_weight.data_ptr(), float(eps), epilogue,
            conv_state.data_ptr() if conv else None, _dtype_code(conv_state) if conv else 0,
            conv_weight.data_ptr() if conv else None,
            conv_bias.data_ptr() if conv and conv_bias is not None else None,
            conv_weight.shape[-1] if conv else 0, _stream_ptr(x2)))
    return y


# --------------------------------------------------------------------------------------------------
# Streaming layers: portions of any length on caches, rings of past inputs and fp32 states
# --------------------------------------------------------------------------------------------------
NORM_RMS, NORM_LAYER, NORM_NONE = 0, 1, 2
ACT_NONE, ACT_SILU, ACT_SIGMOID = 0, 1, 2
STREAM_MAX_TAPS = 8  # BASED_STREAM_MAX_TAPS
DELTA_BLOCK, DELTA_PREP_FLOATS = 16, 592  # tokens per block of based_gated_delta_scan, BASED_DELTA_PREP_FLOATS
RGLRU_SEGMENT = 64   # tokens per segment of based_rglru_prefill


def _ptr(t):
    return None if t is None else t.data_ptr()


def _check_rows(*ts) -> None:
    _require_cuda(*ts)
    for t in ts:
        if t.stride(-1) != 1:
            raise ValueError("innermost dimension must be contiguous")


def _check_same_dtype(x, *ts) -> None:
    for t in ts:
        if t is not None and t.dtype != x.dtype:
            raise ValueError(f"expected {x.dtype}, got {t.dtype}")


def _pos_args(pos, rows: int):
    """pos: an int for every row, or a contiguous int32 device vector of at least `rows` positions."""
    if isinstance(pos, torch.Tensor):
        if pos.dtype != torch.int32 or not pos.is_cuda or pos.dim() != 1 or pos.numel() < rows or not pos.is_contiguous():
            raise ValueError(f"positions must be a contiguous int32 device vector with {rows} entries")
        return pos.data_ptr(), 0
    return None, int(pos)


def _check_ring(ring, rows: int, taps: int, channels: int, like) -> None:
    if (ring.dim() != 3 or tuple(ring.shape) != (rows, taps, channels) or ring.stride(2) != 1 or ring.stride(1) != channels
            or ring.dtype != like.dtype or ring.device != like.device):
        raise ValueError(f"ring must be ({rows}, {taps}, {channels}) {like.dtype} with contiguous slots, got {tuple(ring.shape)} {ring.dtype}")


class Addends(NamedTuple):
    """What a residual sum receives besides mult * x: x may first be divided by its own RMS and weighted (post_weight,
    post_eps); a vector (D) for every row; a row of table (n, D) per row, index (rows) int64."""

    post_weight: Optional[torch.Tensor] = None
    post_eps: float = 0.0
    vec: Optional[torch.Tensor] = None
    table: Optional[torch.Tensor] = None
    index: Optional[torch.Tensor] = None


def _addend_args(addends: Addends, x, rows: int, D: int):
    """(post_weight, post_eps, vec, table, index, table stride, table rows), checked."""
    for t in (addends.post_weight, addends.vec):
        if t is not None and (tuple(t.shape) != (D,) or not t.is_contiguous() or t.dtype != x.dtype or t.device != x.device):
            raise ValueError(f"an added vector must be a contiguous ({D},) {x.dtype} on the device of x")
    table, index = addends.table, addends.index
    if table is not None:
        if table.dim() != 2 or table.shape[1] != D or table.stride(1) != 1 or table.dtype != x.dtype or table.device != x.device:
            raise ValueError(f"the table of added rows must be (n, {D}) {x.dtype} on the device of x")
        if index is None or index.dtype != torch.int64 or index.numel() != rows or not index.is_contiguous() or index.device != x.device:
            raise ValueError(f"the index of added rows must be {rows} contiguous int64 on the device of x")
    return (_ptr(addends.post_weight), float(addends.post_eps), _ptr(addends.vec), _ptr(table), _ptr(index) if table is not None else None,
            0 if table is None else table.stride(0), 0 if table is None else table.shape[0])


def add_norm(x, residual, weight, eps: float, kind: int = NORM_LAYER, mult: float = 1.0, want_residual: bool = True,
             residual_out=None, addends: Optional[Addends] = None):
    """r = residual + mult * x in fp32 (r = x without a residual), and what `addends` brings; y = norm(r) * weight in x's
    dtype (NORM_NONE: r rounded, no weight).  x: (..., D); residual fp32 of the same shape or None.
    Returns (y, r), r None if not wanted (written into residual_out, fp32 with contiguous rows and not `residual`, when given)."""
    D = x.shape[-1]
    _require_cuda(x)
    if kind != NORM_NONE:
        _require_cuda(x, weight)
        _check_same_dtype(x, weight)
        if tuple(weight.shape) != (D,) or not weight.is_contiguous():
            raise ValueError(f"weight must be a contiguous ({D},), got {tuple(weight.shape)}")
    x2 = x.reshape(-1, D)
    if x2.stride(1) != 1:
        x2 = x2.contiguous()
    r2 = None
    if residual is not None:
        _require_cuda(x, residual)
        if residual.shape != x.shape or residual.dtype != torch.float32:
            raise ValueError(f"residual must be float32 {tuple(x.shape)}, got {residual.dtype} {tuple(residual.shape)}")
        r2 = residual.reshape(-1, D)
        if r2.stride(1) != 1:
            r2 = r2.contiguous()
    rows = x2.shape[0]
    y = torch.empty(rows, D, dtype=x.dtype, device=x.device)
    if residual_out is not None:
        out = residual_out.view(rows, D)
        if out.dtype != torch.float32 or out.stride(1) != 1 or out.device != x.device:
            raise ValueError("residual_out must be float32 with contiguous rows on the device of x")
    else:
        out = torch.empty(rows, D, dtype=torch.float32, device=x.device) if want_residual else None
    args = (x2.data_ptr(), _ptr(r2), None if kind == NORM_NONE else weight.data_ptr(), y.data_ptr(), _ptr(out), rows, D, x2.stride(0),
            0 if r2 is None else r2.stride(0), D, D if out is None else out.stride(0), float(eps), int(kind), float(mult))
    with _on_device(x.device):
        if addends is None and kind != NORM_NONE:
            _lib.check(_lib.lib().based_add_norm(*args, _dtype_code(x), _stream_ptr(x)))
        else:
            _lib.check(_lib.lib().based_add_norm_addends(*args, *_addend_args(addends or Addends(), x, rows, D), _dtype_code(x),
                                                         _stream_ptr(x)))
    return y.view(x.shape), None if out is None else out.view(x.shape)


def stream_conv(x, weight, bias=None, ring=None, pos=0, activation: int = ACT_NONE, add_input: bool = False) -> torch.Tensor:
    """y_t = [x_t +] act(bias + sum_j weight[j] * x_{t - taps + 1 + j}) on each channel of x (B, L, D), the
    portion of a sequence that starts at `pos`.  weight (taps, D); ring (B, taps, D) or None (nothing
    before the portion): read for the inputs before it, left with its last ones."""
    B, L, D = x.shape
    taps = weight.shape[0]
    _check_rows(x, weight)
    _check_same_dtype(x, weight, bias)
    if tuple(weight.shape) != (taps, D) or not weight.is_contiguous() or not 1 <= taps <= STREAM_MAX_TAPS:
        raise ValueError(f"weight must be a contiguous (taps, {D}) with 1 to {STREAM_MAX_TAPS} taps, got {tuple(weight.shape)}")
    if bias is not None and (tuple(bias.shape) != (D,) or not bias.is_contiguous() or not bias.is_cuda):
        raise ValueError(f"bias must be a contiguous ({D},) on the device")
    if ring is not None:
        _check_ring(ring, B, taps, D, x)
    pos_ptr, pos_host = _pos_args(pos, B)
    y = torch.empty(B, L, D, dtype=x.dtype, device=x.device)
    with _on_device(x.device):
        _lib.check(_lib.lib().based_stream_conv(
            x.data_ptr(), weight.data_ptr(), _ptr(bias), y.data_ptr(), _ptr(ring), pos_ptr, pos_host, B, L, D, taps, x.stride(0),
            x.stride(1), y.stride(0), y.stride(1), 0 if ring is None else ring.stride(0), int(activation), int(add_input),
            _dtype_code(x), _stream_ptr(x)))
    return y


def _window_shapes(q, k, v, kv_cache, heads: int, kv_heads: int, out):
    """q (..., H * d), k (..., G * d), v (..., G * dv), cache (B, S, G, d + dv): the sizes, checked."""
    _check_rows(q, k, v, kv_cache, out)
    _check_same_dtype(q, k, v, kv_cache, out)
    d, dv = q.shape[-1] // heads, v.shape[-1] // kv_heads
    if q.shape[-1] != heads * d or k.shape[-1] != kv_heads * d or v.shape[-1] != kv_heads * dv or out.shape[-1] != heads * dv:
        raise ValueError(f"bad head sizes q{tuple(q.shape)} k{tuple(k.shape)} v{tuple(v.shape)} out{tuple(out.shape)}")
    if not (q.shape[:-1] == k.shape[:-1] == v.shape[:-1] == out.shape[:-1]):
        raise ValueError("q, k, v and out must agree in batch and length")
    if (kv_cache.dim() != 4 or kv_cache.shape[0] != q.shape[0] or tuple(kv_cache.shape[2:]) != (kv_heads, d + dv)
            or kv_cache.stride(2) != d + dv):
        raise ValueError(f"cache must be ({q.shape[0]}, S, {kv_heads}, {d + dv}), got {tuple(kv_cache.shape)}")
    return d, dv


def _stream_rope(rope, device):
    """(cos, sin, interleaved) tables or None -> (cos_ptr, sin_ptr, n_pos, rotary_dim, half_split)."""
    if rope is None:
        return None, None, 0, 0, 0
    cos, sin, interleaved = rope
    for t in (cos, sin):
        if t.device != device or t.dtype != torch.float32 or t.dim() != 2 or not t.is_contiguous() or t.shape != cos.shape:
            raise ValueError("rotary tables must be contiguous fp32 (n_pos, rotary_dim / 2) tensors on the device of q")
    return cos.data_ptr(), sin.data_ptr(), cos.shape[0], 2 * cos.shape[1], int(not interleaved)


def window_attn_prefill(q, k, v, kv_cache, heads: int, kv_heads: int, window: int, scale: float, start: int = 0, rope=None,
                        value_norm_eps: Optional[float] = None, out_scale: float = 1.0, *, out):
    """Causal attention of a portion at positions start .. start + L - 1 over the last `window` keys (itself
    included).  q (B, L, H * d), k (B, L, G * d), v (B, L, G * dv); kv_cache (B, S, G, d + dv) receives the
    portion's rotated keys and (normalised, when value_norm_eps is given) values and is attended.
    Written, times out_scale, into out (B, L, H * dv)."""
    d, dv = _window_shapes(q, k, v, kv_cache, heads, kv_heads, out)
    cos_ptr, sin_ptr, n_pos, rot, half = _stream_rope(rope, q.device)
    B, L = q.shape[:2]
    with _on_device(q.device):
        _lib.check(_lib.lib().based_window_attn_prefill(
            q.data_ptr(), k.data_ptr(), v.data_ptr(), kv_cache.data_ptr(), out.data_ptr(), int(start), B, L, heads, kv_heads, d, dv,
            kv_cache.shape[1], q.stride(0), q.stride(1), k.stride(0), k.stride(1), v.stride(0), v.stride(1), out.stride(0),
            out.stride(1), kv_cache.stride(0), kv_cache.stride(1), int(window), float(scale), int(value_norm_eps is not None),
            float(value_norm_eps or 0.0), float(out_scale), cos_ptr, sin_ptr, n_pos, rot, half, _dtype_code(q), _stream_ptr(q)))
    return out


def window_attn_step(q, k, v, kv_cache, heads: int, kv_heads: int, window: int, scale: float, pos, rope=None,
                     value_norm_eps: Optional[float] = None, out_scale: float = 1.0, *, out):
    """One token per sequence: q (B, H * d), k (B, G * d), v (B, G * dv), out (B, H * dv); `pos` an int or an
    int32 device vector.  Otherwise as window_attn_prefill."""
    d, dv = _window_shapes(q, k, v, kv_cache, heads, kv_heads, out)
    cos_ptr, sin_ptr, n_pos, rot, half = _stream_rope(rope, q.device)
    B = q.shape[0]
    pos_ptr, pos_host = _pos_args(pos, B)
    with _on_device(q.device):
        _lib.check(_lib.lib().based_window_attn_step(
            q.data_ptr(), k.data_ptr(), v.data_ptr(), kv_cache.data_ptr(), out.data_ptr(), pos_ptr, pos_host, B, heads, kv_heads, d,
            dv, kv_cache.shape[1], q.stride(0), k.stride(0), v.stride(0), out.stride(0), kv_cache.stride(0), kv_cache.stride(1),
            int(window), float(scale), int(value_norm_eps is not None), float(value_norm_eps or 0.0), float(out_scale), cos_ptr,
            sin_ptr, n_pos, rot, half, _dtype_code(q), _stream_ptr(q)))
    return out


def _check_delta(state, rows: int, heads: int, d: int, dv: int) -> None:
    if (state.dim() != 4 or tuple(state.shape[:3]) != (rows, heads, d) or state.shape[3] < dv or state.shape[3] % 4 != 0
            or state.dtype != torch.float32 or not state.is_contiguous() or not state.is_cuda):
        raise ValueError(f"state must be a contiguous float32 ({rows}, {heads}, {d}, {dv} rounded up to 4), got {tuple(state.shape)}")


def gated_delta_scan(q, k, v, a_gate, b_gate, a_log, dt_bias, state, heads: int, kv_heads: int, fresh: bool) -> torch.Tensor:
    """The gated delta recurrence over a portion.  q, k (B, L, G * d) and v (B, L, H * dv) share their strides
    (slices of one tensor); a_gate, b_gate (B, L, H); state (B, H, d, dv rounded up to 4) fp32, updated in
    place, taken as zero when `fresh`.  Returns o (B, L, H, dv) fp32."""
    _check_rows(q, k, v, a_gate, b_gate)
    _check_same_dtype(q, k, v, a_gate, b_gate, a_log, dt_bias)
    B, L = q.shape[:2]
    d, dv = q.shape[-1] // kv_heads, v.shape[-1] // heads
    if q.shape != k.shape or tuple(v.shape[:2]) != (B, L) or q.shape[-1] != kv_heads * d or v.shape[-1] != heads * dv:
        raise ValueError(f"bad shapes q{tuple(q.shape)} k{tuple(k.shape)} v{tuple(v.shape)}")
    if not (q.stride() == k.stride() == v.stride()) or a_gate.stride() != b_gate.stride():
        raise ValueError("q, k and v must share their strides, and the two gates theirs")
    if tuple(a_gate.shape) != (B, L, heads) or b_gate.shape != a_gate.shape:
        raise ValueError(f"gates must be ({B}, {L}, {heads})")
    _check_delta(state, B, heads, d, dv)
    o = torch.empty(B, L, heads, dv, dtype=torch.float32, device=q.device)
    work = torch.empty(B, heads, 2 * ((L + 2 * DELTA_BLOCK - 1) // (2 * DELTA_BLOCK)), DELTA_PREP_FLOATS, dtype=torch.float32, device=q.device)
    with _on_device(q.device):
        _lib.check(_lib.lib().based_gated_delta_scan(
            q.data_ptr(), k.data_ptr(), v.data_ptr(), a_gate.data_ptr(), b_gate.data_ptr(), a_log.data_ptr(), dt_bias.data_ptr(),
            state.data_ptr(), work.data_ptr(), o.data_ptr(), B, L, heads, kv_heads, d, dv, state.shape[3], q.stride(0), q.stride(1),
            a_gate.stride(0), a_gate.stride(1), int(fresh), _dtype_code(q), _stream_ptr(q)))
    return o


def gated_rms_norm(o, weight, gate, eps: float, scale: float = 1.0, *, out) -> torch.Tensor:
    """out = o / sqrt(mean(o^2) + eps) * weight * silu(gate) * scale per head; o (B, L, H, dv) fp32, gate and
    out (B, L, H * dv)."""
    B, L, H, dv = o.shape
    _check_rows(gate, out)
    _check_same_dtype(gate, out, weight)
    if o.dtype != torch.float32 or not o.is_contiguous() or tuple(gate.shape) != (B, L, H * dv) or out.shape != gate.shape \
            or tuple(weight.shape) != (dv,):
        raise ValueError(f"bad shapes o{tuple(o.shape)} gate{tuple(gate.shape)} out{tuple(out.shape)} weight{tuple(weight.shape)}")
    with _on_device(o.device):
        _lib.check(_lib.lib().based_gated_rms_norm(o.data_ptr(), weight.data_ptr(), gate.data_ptr(), out.data_ptr(), B, L, H, dv,
                                                   gate.stride(0), gate.stride(1), out.stride(0), out.stride(1), float(eps),
                                                   float(scale), _dtype_code(gate), _stream_ptr(gate)))
    return out


def gated_delta_step(x, conv_weight, ring, a_gate, b_gate, gate, a_log, dt_bias, norm_weight, state, heads: int, kv_heads: int,
                     d: int, dv: int, k_off: int, v_off: int, pos, eps: float, scale: float = 1.0, *, out) -> torch.Tensor:
    """One token of the delta-rule block between its projections: x (B, C) is what the short convolution
    reads (queries at channel 0, keys at k_off, values at v_off), conv_weight (taps, C), ring (B, taps, C);
    a_gate, b_gate (B, H), gate and out (B, H * dv)."""
    _check_rows(x, a_gate, b_gate, gate, out)
    _check_same_dtype(x, conv_weight, a_gate, b_gate, gate, a_log, dt_bias, norm_weight, out)
    B, C = x.shape
    taps = conv_weight.shape[0]
    if tuple(conv_weight.shape) != (taps, C) or not conv_weight.is_contiguous():
        raise ValueError(f"conv_weight must be a contiguous (taps, {C}), got {tuple(conv_weight.shape)}")
    if tuple(a_gate.shape) != (B, heads) or b_gate.shape != a_gate.shape or a_gate.stride() != b_gate.stride() \
            or tuple(gate.shape) != (B, heads * dv) or out.shape != gate.shape:
        raise ValueError("bad gate or output shapes")
    _check_ring(ring, B, taps, C, x)
    _check_delta(state, B, heads, d, dv)
    pos_ptr, pos_host = _pos_args(pos, B)
    with _on_device(x.device):
        _lib.check(_lib.lib().based_gated_delta_step(
            x.data_ptr(), conv_weight.data_ptr(), ring.data_ptr(), a_gate.data_ptr(), b_gate.data_ptr(), gate.data_ptr(),
            a_log.data_ptr(), dt_bias.data_ptr(), norm_weight.data_ptr(), state.data_ptr(), out.data_ptr(), pos_ptr, pos_host, B,
            heads, kv_heads, d, dv, state.shape[3], C, taps, k_off, v_off, x.stride(0), a_gate.stride(0), gate.stride(0),
            out.stride(0), ring.stride(0), float(eps), float(scale), _dtype_code(x), _stream_ptr(x)))
    return out


def _check_lru(x, y, ra, rb, ri, ib, lam, state, out, rows: int):
    _check_rows(x, y, out)
    _check_same_dtype(x, y, ra, rb, ri, ib, lam, out)
    W = x.shape[-1]
    blocks, n = ra.shape[:2]
    if blocks * n != W or tuple(ra.shape) != (blocks, n, n) or ri.shape != ra.shape or y.shape != x.shape or out.shape != x.shape:
        raise ValueError(f"bad shapes x{tuple(x.shape)} y{tuple(y.shape)} ra{tuple(ra.shape)} ri{tuple(ri.shape)}")
    for t in (ra, ri, rb, ib, lam):
        if not t.is_contiguous() or (t.dim() < 3 and t.numel() != W):
            raise ValueError("gate parameters must be contiguous, one value per channel")
    if tuple(state.shape) != (rows, W) or state.dtype != torch.float32 or not state.is_contiguous():
        raise ValueError(f"state must be a contiguous float32 ({rows}, {W}), got {tuple(state.shape)}")
    return W, blocks


def rglru_prefill(u, y, ra, rb, ri, ib, lam, state, decay_scale: float, fresh: bool, *, out) -> torch.Tensor:
    """The gated linear recurrence over a portion: u (B, L, W) convolved, y (B, L, W) before its gelu; ra, ri
    (blocks, n, n) as [out, in], rb, ib, lam (W) values; state (B, W) fp32, updated in place, taken as
    zero when `fresh`.  out (B, L, W) = S * gelu_tanh(y)."""
    B, L, _ = u.shape
    W, blocks = _check_lru(u, y, ra, rb, ri, ib, lam, state, out, B)
    segs = (L + RGLRU_SEGMENT - 1) // RGLRU_SEGMENT
    work = torch.empty(2, B, L, W, dtype=torch.float32, device=u.device)
    agg = torch.empty(B, segs + 1, 2, W, dtype=torch.float32, device=u.device)
    with _on_device(u.device):
        _lib.check(_lib.lib().based_rglru_prefill(
            u.data_ptr(), y.data_ptr(), ra.data_ptr(), rb.data_ptr(), ri.data_ptr(), ib.data_ptr(), lam.data_ptr(),
            work[0].data_ptr(), work[1].data_ptr(), agg.data_ptr(), state.data_ptr(), out.data_ptr(), B, L, W, blocks, u.stride(0),
            u.stride(1), y.stride(0), y.stride(1), out.stride(0), out.stride(1), float(decay_scale), int(fresh), _dtype_code(u),
            _stream_ptr(u)))
    return out


def rglru_step(x, y, conv_weight, conv_bias, ring, ra, rb, ri, ib, lam, state, decay_scale: float, pos, *, out) -> torch.Tensor:
    """One token of it with the short convolution in front: x, y, out (B, W); conv_weight (taps, W), conv_bias
    (W) or None, ring (B, taps, W)."""
    B = x.shape[0]
    W, blocks = _check_lru(x, y, ra, rb, ri, ib, lam, state, out, B)
    taps = conv_weight.shape[0]
    _check_same_dtype(x, conv_weight, conv_bias)
    if tuple(conv_weight.shape) != (taps, W) or not conv_weight.is_contiguous():
        raise ValueError(f"conv_weight must be a contiguous (taps, {W}), got {tuple(conv_weight.shape)}")
    _check_ring(ring, B, taps, W, x)
    pos_ptr, pos_host = _pos_args(pos, B)
    with _on_device(x.device):
        _lib.check(_lib.lib().based_rglru_step(
            x.data_ptr(), y.data_ptr(), conv_weight.data_ptr(), _ptr(conv_bias), ring.data_ptr(), ra.data_ptr(), rb.data_ptr(),
            ri.data_ptr(), ib.data_ptr(), lam.data_ptr(), state.data_ptr(), out.data_ptr(), pos_ptr, pos_host, B, W, blocks, taps,
            x.stride(0), y.stride(0), out.stride(0), ring.stride(0), float(decay_scale), _dtype_code(x), _stream_ptr(x)))
    return out


def token_mix(x, mu, ring=None, pos=0) -> torch.Tensor:
    """(S, B, L, D): x_t + (x_{t-1} - x_t) * mu_s of a portion x (B, L, D) that starts at `pos`; mu (S, D); ring (B, 2, D) or
    None (nothing before the portion): read for the input before it, left with its last one."""
    B, L, D = x.shape
    _check_rows(x, mu)
    _check_same_dtype(x, mu)
    if mu.dim() != 2 or mu.shape[1] != D or not mu.is_contiguous():
        raise ValueError(f"mu must be a contiguous (mixes, {D}), got {tuple(mu.shape)}")
    if ring is not None:
        _check_ring(ring, B, 2, D, x)
    pos_ptr, pos_host = _pos_args(pos, B)
    y = torch.empty(mu.shape[0], B, L, D, dtype=x.dtype, device=x.device)
    with _on_device(x.device):
        _lib.check(_lib.lib().based_token_mix(x.data_ptr(), mu.data_ptr(), y.data_ptr(), _ptr(ring), pos_ptr, pos_host, B, L, D, mu.shape[0],
                                              x.stride(0), x.stride(1), 0 if ring is None else ring.stride(0), _dtype_code(x),
                                              _stream_ptr(x)))
    return y


def channel_decay(hidden, w2, w0) -> torch.Tensor:
    """log2 of exp(-exp(w2 tanh(hidden) + w0)): hidden (B, L, R) -> (B, L, C) fp32; w2 (C, R), w0 (C)."""
    B, L, R = hidden.shape
    _check_rows(hidden, w2)
    _check_same_dtype(hidden, w2, w0)
    C = w2.shape[0]
    h2 = hidden.reshape(-1, R)
    if tuple(w2.shape) != (C, R) or not w2.is_contiguous() or tuple(w0.shape) != (C,) or not w0.is_contiguous() or not w0.is_cuda:
        raise ValueError(f"w2 {tuple(w2.shape)} and w0 {tuple(w0.shape)} must be contiguous (channels, {R}) and (channels,)")
    y = torch.empty(B, L, C, dtype=torch.float32, device=hidden.device)
    with _on_device(hidden.device):
        _lib.check(_lib.lib().based_channel_decay(h2.data_ptr(), w2.data_ptr(), w0.data_ptr(), y.data_ptr(), B * L, h2.stride(0), C, R,
                                                  _dtype_code(hidden), _stream_ptr(hidden)))
    return y


def gelu_mul(g, table, index) -> torch.Tensor:
    """gelu_tanh(g) * table[index]: g (rows, n), table (entries, n) with rows at any stride, index (rows) int64."""
    rows, n = g.shape
    _check_rows(g, table)
    _check_same_dtype(g, table)
    if table.dim() != 2 or table.shape[1] != n or index.dtype != torch.int64 or index.numel() != rows or not index.is_contiguous() \
            or not index.is_cuda:
        raise ValueError(f"bad shapes g{tuple(g.shape)} table{tuple(table.shape)} index{tuple(index.shape)}")
    y = torch.empty(rows, n, dtype=g.dtype, device=g.device)
    with _on_device(g.device):
        _lib.check(_lib.lib().based_gelu_mul(g.data_ptr(), table.data_ptr(), index.data_ptr(), y.data_ptr(), rows, n, g.stride(0),
                                             table.stride(0), table.shape[0], _dtype_code(g), _stream_ptr(g)))
    return y


SIDE_STEP_MAX_DIM, SIDE_STEP_MAX_INNER = 4096, 512


def token_side_step_ok(gate_w, proj_w) -> bool:
    """Whether `token_side_step` takes these weights: bf16 (n, D) and (D, n) with whole 16-byte pieces."""
    n, D = gate_w.shape
    return (gate_w.is_cuda and gate_w.dtype == torch.bfloat16 and proj_w.dtype == torch.bfloat16 and gate_w.is_contiguous()
            and proj_w.is_contiguous() and n % 8 == 0 and D % 8 == 0 and D <= SIDE_STEP_MAX_DIM and n <= SIDE_STEP_MAX_INNER)


def token_side_step(x, residual, residual_out, gate_w, proj_w, table, index, mult: float = 1.0) -> torch.Tensor:
    """r = residual + mult * x in fp32 (x without a residual), written to residual_out, and proj_w (gelu_tanh(gate_w r) * table[index]), for
    single tokens in one launch: x (M, D) bf16, gate_w (n, D), proj_w (D, n), table (entries, n) with rows at any stride, index (M)."""
    M, D = x.shape
    n = gate_w.shape[0]
    _require_cuda(x, residual_out, gate_w, proj_w, table, index)
    _check_same_dtype(x, gate_w, proj_w, table)
    if x.dtype != torch.bfloat16 or x.stride(1) != 1 or tuple(gate_w.shape) != (n, D) or tuple(proj_w.shape) != (D, n) \
            or not gate_w.is_contiguous() or not proj_w.is_contiguous():
        raise ValueError(f"bad shapes x{tuple(x.shape)} gate_w{tuple(gate_w.shape)} proj_w{tuple(proj_w.shape)}")
    if table.dim() != 2 or table.shape[1] != n or table.stride(1) != 1 or index.dtype != torch.int64 or index.numel() != M \
            or not index.is_contiguous():
        raise ValueError(f"bad table {tuple(table.shape)} or index {tuple(index.shape)}")
    for r in (residual, residual_out):
        if r is not None and (r.dtype != torch.float32 or tuple(r.shape) != (M, D) or not r.is_contiguous()):
            raise ValueError(f"residuals must be contiguous float32 ({M}, {D})")
    y = torch.empty(M, D, dtype=x.dtype, device=x.device)
    with _on_device(x.device):
        _lib.check(_lib.lib().based_token_side_step(x.data_ptr(), _ptr(residual), residual_out.data_ptr(), gate_w.data_ptr(), proj_w.data_ptr(),
                                                    table.data_ptr(), index.data_ptr(), y.data_ptr(), M, D, n, x.stride(0), table.stride(0),
                                                    table.shape[0], float(mult), _stream_ptr(x)))
    return y


def softcap_(x, cap: float) -> torch.Tensor:
    """x <- cap * tanh(x / cap), in place."""
    _require_cuda(x)
    if not x.is_contiguous():
        raise ValueError("x must be contiguous")
    with _on_device(x.device):
        _lib.check(_lib.lib().based_softcap(x.data_ptr(), x.numel(), float(cap), _dtype_code(x), _stream_ptr(x)))
    return x


def _check_decay_state(state, rows: int, heads: int, d: int, dv: int) -> None:
    if (state.dim() != 4 or tuple(state.shape[:3]) != (rows, heads, dv) or state.shape[3] < d or state.shape[3] % 4 != 0
            or state.dtype != torch.float32 or not state.is_contiguous() or not state.is_cuda):
        raise ValueError(f"state must be a contiguous float32 ({rows}, {heads}, {dv}, {d} rounded up to 4), got {tuple(state.shape)}")


def head_decays(decay, device) -> torch.Tensor:
    """(2, H) fp32 for the head form of decay_scan and decay_step: base-2 logarithms of the decays as fp32 holds them, and the decays.
    A decay of zero is one whose powers are zero (0 * -inf would not be a number)."""
    value = torch.tensor(list(decay), dtype=torch.float32)
    log2 = torch.where(value > 0, value.double().log2(), torch.full_like(value, -1e4).double()).float()
    return torch.stack([log2, value]).to(device)


def _check_head_decay(head_decay, heads: int, device) -> None:
    if head_decay.dtype != torch.float32 or tuple(head_decay.shape) != (2, heads) or head_decay.device != device \
            or not head_decay.is_contiguous():
        raise ValueError(f"head_decay must be a contiguous float32 (2, {heads}) on the device of q (head_decays)")


def decay_scan(q, k, v, state, heads: int, *, channel_log2=None, bonus=None, head_decay=None, activation: int = ACT_NONE,
               fresh: bool) -> torch.Tensor:
    """Linear attention with decaying states over a portion: q, k (B, L, H * d), v (B, L, H * dv) -> o (B, L, H * dv); state (B, H, dv,
    d rounded up to 4) fp32, updated in place, taken as zero when `fresh`.  channel_log2 (B, L, H * d) fp32 with bonus (H, d):
    o_t = (S + diag(u) k v^T)^T q, S <- diag(w) S + k v^T; head_decay (2, H) of `head_decays`: S <- w S + k v^T, o = S^T q."""
    _check_rows(q, k, v)
    _check_same_dtype(q, k, v, bonus)
    B, L = q.shape[:2]
    d, dv = q.shape[-1] // heads, v.shape[-1] // heads
    if q.shape != k.shape or tuple(q.shape) != (B, L, heads * d) or tuple(v.shape) != (B, L, heads * dv):
        raise ValueError(f"bad shapes q{tuple(q.shape)} k{tuple(k.shape)} v{tuple(v.shape)}")
    _check_decay_state(state, B, heads, d, dv)
    if channel_log2 is not None:
        if tuple(channel_log2.shape) != (B, L, heads * d) or channel_log2.dtype != torch.float32 or not channel_log2.is_contiguous() \
                or bonus is None or tuple(bonus.shape) != (heads, d) or not bonus.is_contiguous():
            raise ValueError(f"channel decays must be contiguous float32 ({B}, {L}, {heads * d}) with a bonus ({heads}, {d})")
        _require_cuda(q, channel_log2, bonus)
    else:
        _check_head_decay(head_decay, heads, q.device)
    lib = _lib.lib()
    work = None
    if q.dtype == torch.bfloat16:
        n = lib.based_decay_scan_work(B, L, heads, d, dv, state.shape[3])
        work = torch.empty(n, dtype=torch.float32, device=q.device) if n else None
    o = torch.empty(B, L, heads * dv, dtype=q.dtype, device=q.device)
    with _on_device(q.device):
        _lib.check(lib.based_decay_scan(
            q.data_ptr(), k.data_ptr(), v.data_ptr(), _ptr(channel_log2), _ptr(head_decay), _ptr(bonus), state.data_ptr(), _ptr(work),
            o.data_ptr(), B, L, heads, d, dv, state.shape[3], q.stride(0), q.stride(1), k.stride(0), k.stride(1), v.stride(0), v.stride(1),
            o.stride(0), o.stride(1), int(activation), int(fresh), _dtype_code(q), _stream_ptr(q)))
    return o


def decay_step(q, k, v, state, heads: int, pos, *, head_decay=None, bonus=None, hidden=None, w2=None, w0=None, gate=None, norm_weight=None,
               eps: float = 0.0, activation: int = ACT_NONE, out) -> torch.Tensor:
    """One token of it: q, k (B, H * d), v, out (B, H * dv).  With head_decay the head form; with `hidden` (B, R), w2 (H * d, R), w0 (H * d),
    bonus (H, d) the channel form, its output divided by its RMS per head, times norm_weight (H * dv) and silu(gate) (B, H * dv)."""
    _check_rows(q, k, v, out)
    _check_same_dtype(q, k, v, out, bonus, hidden, w2, w0, gate, norm_weight)
    B = q.shape[0]
    d, dv = q.shape[-1] // heads, v.shape[-1] // heads
    if q.shape != k.shape or tuple(q.shape) != (B, heads * d) or tuple(v.shape) != (B, heads * dv) or out.shape != v.shape:
        raise ValueError(f"bad shapes q{tuple(q.shape)} k{tuple(k.shape)} v{tuple(v.shape)} out{tuple(out.shape)}")
    _check_decay_state(state, B, heads, d, dv)
    R = 0
    if hidden is not None:
        _check_rows(hidden, gate)
        R = hidden.shape[-1]
        if (tuple(hidden.shape) != (B, R) or tuple(w2.shape) != (heads * d, R) or w0.numel() != heads * d or bonus.numel() != heads * d
                or tuple(gate.shape) != (B, heads * dv) or norm_weight.numel() != heads * dv):
            raise ValueError("bad shapes of the decay's or the output's parameters")
        for t in (w2, w0, bonus, norm_weight):
            if not t.is_contiguous() or not t.is_cuda:
                raise ValueError("parameters must be contiguous device tensors")
    else:
        _check_head_decay(head_decay, heads, q.device)
    pos_ptr, pos_host = _pos_args(pos, B)
    with _on_device(q.device):
        _lib.check(_lib.lib().based_decay_step(
            q.data_ptr(), k.data_ptr(), v.data_ptr(), _ptr(head_decay), _ptr(bonus), _ptr(hidden), _ptr(w2), _ptr(w0), _ptr(gate),
            _ptr(norm_weight), state.data_ptr(), out.data_ptr(), pos_ptr, pos_host, B, heads, d, dv, state.shape[3], R, q.stride(0),
            k.stride(0), v.stride(0), 0 if hidden is None else hidden.stride(0), 0 if gate is None else gate.stride(0), out.stride(0),
            int(activation), float(eps), _dtype_code(q), _stream_ptr(q)))
    return out


def group_norm_gate(o, weight, gate, groups: int, eps: float, activation: int, scale: float = 1.0, *, out) -> torch.Tensor:
    """out = o / sqrt(mean(o^2) + eps) * weight * act(gate) * scale over each of `groups` parts of a row; o, gate, out (B, L, groups * n),
    weight (groups * n); ACT_SILU or ACT_SIGMOID."""
    B, L, W = o.shape
    _check_rows(o, gate, out)
    _check_same_dtype(o, gate, out, weight)
    if gate.shape != o.shape or out.shape != o.shape or weight.numel() != W or W % groups != 0 or not weight.is_contiguous():
        raise ValueError(f"bad shapes o{tuple(o.shape)} gate{tuple(gate.shape)} out{tuple(out.shape)} weight{tuple(weight.shape)}")
    with _on_device(o.device):
        _lib.check(_lib.lib().based_group_norm_gate(o.data_ptr(), weight.data_ptr(), gate.data_ptr(), out.data_ptr(), B, L, groups, W // groups,
                                                    o.stride(0), o.stride(1), gate.stride(0), gate.stride(1), out.stride(0), out.stride(1),
                                                    float(eps), float(scale), int(activation), _dtype_code(o), _stream_ptr(o)))
    return out


def window_attn_attend(q, kv, heads: int, kv_heads: int, dim: int, window: int, scale: float, start: int = 0, rope=None,
                       out_scale: float = 1.0, *, out):
    """window_attn_prefill on rows that kv (B, S, G, d + dv) already holds: only q (B, L, H * d) is rotated."""
    _check_rows(q, kv, out)
    _check_same_dtype(q, kv, out)
    B, L = q.shape[:2]
    dv = out.shape[-1] // heads
    if (tuple(q.shape) != (B, L, heads * dim) or tuple(out.shape) != (B, L, heads * dv) or kv.dim() != 4 or kv.shape[0] != B
            or tuple(kv.shape[2:]) != (kv_heads, dim + dv) or kv.stride(2) != dim + dv):
        raise ValueError(f"bad shapes q{tuple(q.shape)} kv{tuple(kv.shape)} out{tuple(out.shape)}")
    cos_ptr, sin_ptr, n_pos, rot, half = _stream_rope(rope, q.device)
    with _on_device(q.device):
        _lib.check(_lib.lib().based_window_attn_attend(
            q.data_ptr(), kv.data_ptr(), out.data_ptr(), int(start), B, L, heads, kv_heads, dim, dv, kv.shape[1], q.stride(0), q.stride(1),
            out.stride(0), out.stride(1), kv.stride(0), kv.stride(1), int(window), float(scale), float(out_scale), cos_ptr, sin_ptr, n_pos,
            rot, half, _dtype_code(q), _stream_ptr(q)))
    return out


def _latent_rows(x, norm_weight, cache, rope):
    """Latent and rotated sizes of x (..., R + rot) and cache (B, S, R + rot), checked."""
    _check_rows(x, cache)
    _check_same_dtype(x, cache, norm_weight)
    R, W = norm_weight.numel(), x.shape[-1]
    cos_ptr, sin_ptr, n_pos, rot, half = _stream_rope(rope, x.device)
    if R + rot != W or cache.dim() != 3 or cache.shape[0] != x.shape[0] or cache.shape[2] != W or not norm_weight.is_contiguous():
        raise ValueError(f"bad shapes x{tuple(x.shape)} cache{tuple(cache.shape)} norm{tuple(norm_weight.shape)}, rotary size {rot}")
    return R, rot, cos_ptr, sin_ptr, n_pos, half


def latent_write(x, norm_weight, cache, start: int, eps: float, rope) -> None:
    """Rows start .. start + L - 1 of a latent cache (B, S, R + rot) from x (B, L, R + rot): the first R channels divided by their RMS
    and weighted, the others rotated."""
    R, rot, cos_ptr, sin_ptr, n_pos, half = _latent_rows(x, norm_weight, cache, rope)
    B, L = x.shape[:2]
    with _on_device(x.device):
        _lib.check(_lib.lib().based_latent_write(x.data_ptr(), norm_weight.data_ptr(), cache.data_ptr(), int(start), B, L, cache.shape[1], R, rot,
                                                 x.stride(0), x.stride(1), cache.stride(0), cache.stride(1), float(eps), cos_ptr, sin_ptr,
                                                 n_pos, half, _dtype_code(x), _stream_ptr(x)))


LATENT_STEP_TARGET = 256  # workgroups that the keys of a step are dealt to, where there are enough
LATENT_STEP_MAX_SPLITS = 64


def latent_step(q, x, norm_weight, weight, cache, heads: int, dim: int, window: int, scale: float, pos, eps: float, rope,
                out_scale: float = 1.0, *, out) -> torch.Tensor:
    """One token per sequence on a latent cache: q (B, H * (rot + d)) with a head's rotated channels first, x (B, R + rot) the token's own
    row before norm and rotation, weight (H * (rot + d + dv), >= R): of each head rot rows that are not read, uk, uv.
    Written, times out_scale, into out (B, H * dv)."""
    R, rot, cos_ptr, sin_ptr, n_pos, half = _latent_rows(x, norm_weight, cache, rope)
    _check_rows(q, weight, out)
    _check_same_dtype(x, q, weight, out)
    B, S = x.shape[0], cache.shape[1]
    dv = out.shape[-1] // heads
    if tuple(q.shape) != (B, heads * (rot + dim)) or tuple(out.shape) != (B, heads * dv) or weight.shape[0] != heads * (rot + dim + dv) \
            or weight.shape[1] < R:
        raise ValueError(f"bad shapes q{tuple(q.shape)} weight{tuple(weight.shape)} out{tuple(out.shape)}")
    groups = B * ((heads + 15) // 16)
    splits = max(1, min(LATENT_STEP_TARGET // groups, (min(window, S) + 63) // 64, LATENT_STEP_MAX_SPLITS))
    f32 = dict(dtype=torch.float32, device=x.device)
    work_q = torch.empty(B, heads, R + rot, **f32)
    part, part_ml = torch.empty(B, splits, heads, R, **f32), torch.empty(B, splits, heads, 2, **f32)
    pos_ptr, pos_host = _pos_args(pos, B)
    with _on_device(x.device):
        _lib.check(_lib.lib().based_latent_step(
            q.data_ptr(), x.data_ptr(), norm_weight.data_ptr(), weight.data_ptr(), cache.data_ptr(), work_q.data_ptr(), part.data_ptr(),
            part_ml.data_ptr(), out.data_ptr(), pos_ptr, pos_host, B, heads, dim, dv, S, R, rot, splits, q.stride(0), x.stride(0),
            weight.stride(0), cache.stride(0), cache.stride(1), out.stride(0), int(window), float(scale), float(eps), float(out_scale),
            cos_ptr, sin_ptr, n_pos, half, _dtype_code(x), _stream_ptr(x)))
    return out


# Choices up to which experts are evaluated one choice at a time: beyond, rows of one expert share its matrices.
EXPERT_ROWS_MAX = 16
EXPERT_NORM_MAX_DIM = 4096


def experts(h, router, w1, w2, top: int, norm=None) -> torch.Tensor:
    """y = sum over the `top` experts of a token with the largest sigmoid(router h) of w2_e (silu(gate) * up), [up; gate] = score * w1_e h.
    h (..., D), router (E, D), w1 (E, 2 F, D) up rows first, w2 (E, D, F).  norm = (residual fp32 or None, residual_out fp32 or None, weight,
    eps, kind, mult): h is the input of `add_norm` with these and the layer reads its norm."""
    D = h.shape[-1]
    E, F = w2.shape[0], w2.shape[2]
    h2 = h.reshape(-1, D)
    _check_rows(h2, router, w1, w2)
    _check_same_dtype(h2, router, w1, w2)
    if tuple(router.shape) != (E, D) or tuple(w1.shape) != (E, 2 * F, D) or tuple(w2.shape) != (E, D, F):
        raise ValueError(f"bad shapes router{tuple(router.shape)} w1{tuple(w1.shape)} w2{tuple(w2.shape)}")
    if not (router.is_contiguous() and w1.is_contiguous() and w2.is_contiguous()):
        raise ValueError("expert weights must be contiguous")
    if not 1 <= top <= E:
        raise ValueError(f"{top} of {E} experts")
    n, dev = h2.shape[0], h2.device
    lib = _lib.lib()
    grouped = h2.dtype == torch.bfloat16 and n * top > EXPERT_ROWS_MAX and D % 8 == 0 and F % 8 == 0 and h2.stride(0) % 8 == 0
    i32 = dict(dtype=torch.int32, device=dev)
    norm_args = (None, None, None, None, 1.0, NORM_RMS, 0.0)
    if norm is not None:
        residual, residual_out, weight, eps, kind, mult = norm
        if grouped or h2.dtype != torch.bfloat16 or D % 8 != 0 or D > EXPERT_NORM_MAX_DIM or n * top > EXPERT_ROWS_MAX:
            h2, _ = add_norm(h2, residual, weight, eps, kind, mult, residual_out is not None, residual_out)
        else:
            for r in (residual, residual_out):
                if r is not None and (r.dtype != torch.float32 or tuple(r.shape) != (n, D) or not r.is_contiguous() or not r.is_cuda):
                    raise ValueError(f"residuals must be contiguous float32 ({n}, {D}) device tensors")
            _check_same_dtype(h2, weight)
            if tuple(weight.shape) != (D,) or not weight.is_contiguous() or not weight.is_cuda:
                raise ValueError(f"the norm's weight must be a contiguous ({D},) on the device")
            normed = torch.empty_like(h2)
            norm_args = (_ptr(residual), _ptr(residual_out), weight.data_ptr(), normed.data_ptr(), float(mult), int(kind), float(eps))
    ids, scores = torch.empty(n, top, **i32), torch.empty(n, top, dtype=torch.float32, device=dev)
    y = torch.empty(n, D, dtype=h2.dtype, device=dev)
    with _on_device(dev):
        if grouped:
            tiles, rows = lib.based_expert_tiles(n, E, top), lib.based_expert_tile_rows(n, E, top)
            rank = torch.empty(n, top, **i32)
            counts = (torch.empty if n <= 16 else torch.zeros)(E, **i32)  # (so few tokens are counted by one workgroup)
            plan = torch.empty(E + 1 + tiles + tiles * rows, **i32)
            act = torch.empty(tiles * rows, F, dtype=h2.dtype, device=dev)
            part = torch.empty(n * top, D, dtype=h2.dtype, device=dev) if top > 1 else None
            _lib.check(lib.based_expert_grouped(
                h2.data_ptr(), router.data_ptr(), w1.data_ptr(), w2.data_ptr(), ids.data_ptr(), scores.data_ptr(), rank.data_ptr(),
                counts.data_ptr(), plan.data_ptr(), plan[E + 1:].data_ptr(), plan[E + 1 + tiles:].data_ptr(), act.data_ptr(), _ptr(part),
                y.data_ptr(), n, D, F, E, top, h2.stride(0), _stream_ptr(h2)))
        else:
            act = torch.empty(n * top, F, dtype=h2.dtype, device=dev)
            _lib.check(lib.based_expert_rows(h2.data_ptr(), *norm_args, router.data_ptr(), w1.data_ptr(), w2.data_ptr(), ids.data_ptr(),
                                             scores.data_ptr(), act.data_ptr(), y.data_ptr(), n, D, F, E, top, h2.stride(0), _dtype_code(h2),
                                             _stream_ptr(h2)))
    return y.view(h.shape)


# Rows up to which the streamed-input prologue is evaluated inside the projection.  Every workgroup of it
# repeats the prologue for every row; beyond one register tile of rows that costs more than launches of its own.
STREAM_PROLOGUE_MAX_ROWS = 8


def _decode_linear_stream(x, weight, bias, epilogue, residual_in, residual_out, norm_weight, eps, row_index, mult, norm_kind,
                          input_conv, out):
    """`decode_linear` behind PROLOGUE_STREAM."""
    N, K = weight.shape
    x2 = x if x.dim() == 2 else x.reshape(-1, x.shape[-1])
    M = x2.shape[0] if row_index is None else row_index.numel()
    n_out = N if epilogue == EPILOGUE_NONE else N // 2
    _require_cuda(x2, weight, norm_weight)
    if x2.dtype != torch.bfloat16 or weight.dtype != torch.bfloat16 or norm_weight.dtype != torch.bfloat16 or x2.shape[1] != K \
            or weight.stride(1) != 1 or x2.stride(1) != 1 or tuple(norm_weight.shape) != (K,) or not norm_weight.is_contiguous():
        raise ValueError("x, weight and norm_weight must be bfloat16 rows of the contraction length")
    if bias is not None and (tuple(bias.shape) != (N,) or bias.dtype != torch.bfloat16 or not bias.is_contiguous()):
        raise ValueError(f"bias must be a contiguous bfloat16 ({N},)")
    for r in (residual_in, residual_out):
        if r is not None and (r.dtype != torch.float32 or tuple(r.shape) != (M, K) or r.stride(1) != 1 or not r.is_cuda):
            raise ValueError(f"residuals must be float32 ({M}, {K}) device tensors with contiguous rows")
    if row_index is not None and (row_index.dtype != torch.int64 or row_index.dim() != 1 or not row_index.is_contiguous()
                                  or not row_index.is_cuda):
        raise ValueError("row_index must be a contiguous int64 device vector")
    conv_w = ring = pos_ptr = None
    taps = pos_host = ring_stride = 0
    if input_conv is not None:
        conv_w, ring, pos = input_conv
        taps = conv_w.shape[0]
        if tuple(conv_w.shape) != (taps, K) or not conv_w.is_contiguous() or conv_w.dtype != torch.bfloat16 or not conv_w.is_cuda:
            raise ValueError(f"the input convolution's weight must be a contiguous bfloat16 (taps, {K})")
        _check_ring(ring, M, taps, K, x2)
        ring_stride = ring.stride(0)
        pos_ptr, pos_host = _pos_args(pos, M)
    if M > STREAM_PROLOGUE_MAX_ROWS:
        rows = x2 if row_index is None else x2.index_select(0, row_index)
        h, _ = add_norm(rows, residual_in, norm_weight, eps, norm_kind, mult, residual_out is not None, residual_out)
        if input_conv is not None:
            h = stream_conv(h.unsqueeze(1), conv_w, None, ring, input_conv[2], add_input=True).squeeze(1)
        return decode_linear(h, weight, bias, epilogue=epilogue, out=out)
    y = torch.empty(M, n_out, dtype=torch.bfloat16, device=x2.device) if out is None else out
    if tuple(y.shape) != (M, n_out) or y.dtype != torch.bfloat16 or y.stride(1) != 1:
        raise ValueError(f"out must be a ({M}, {n_out}) bfloat16 tensor with contiguous rows")
    with _on_device(x2.device):
        _lib.check(_lib.lib().based_decode_linear_stream(
            x2.data_ptr(), x2.stride(0), _ptr(row_index), 0 if row_index is None else x2.shape[0], weight.data_ptr(), weight.stride(0),
            _ptr(bias), y.data_ptr(), y.stride(0), M, N, K, _ptr(residual_in), 0 if residual_in is None else residual_in.stride(0),
            _ptr(residual_out), 0 if residual_out is None else residual_out.stride(0), float(mult), int(norm_kind),
            norm_weight.data_ptr(), float(eps), _ptr(conv_w), _ptr(ring), ring_stride, taps, pos_ptr, pos_host, epilogue,
            _stream_ptr(x2)))
    return y


def decode_linear_mixes(x, weight, mix_rows: int) -> torch.Tensor:
    """(M, N): weight rows i * mix_rows .. times row m of x[i], x (mixes, M, K) bf16; the last mix all rows that are left."""
    S, M, K = x.shape
    N = weight.shape[0]
    _require_cuda(x, weight)
    if x.dtype != torch.bfloat16 or weight.dtype != torch.bfloat16 or weight.shape[1] != K or weight.stride(1) != 1 or not x.is_contiguous():
        raise ValueError("x and weight must be bfloat16 rows of the contraction length, x contiguous")
    y = torch.empty(M, N, dtype=torch.bfloat16, device=x.device)
    with _on_device(x.device):
        _lib.check(_lib.lib().based_decode_linear_mixes(x.data_ptr(), weight.data_ptr(), weight.stride(0), y.data_ptr(), N, M, N, K, S,
                                                        int(mix_rows), _stream_ptr(x)))
    return y


def _decode_linear_extras(x, weight, bias, epilogue, residual_in, residual_out, norm_weight, eps, row_index, mult, norm_kind, addends, mix,
                          gate, softcap, out):
    """`decode_linear` behind PROLOGUE_STREAM with what else may surround it."""
    N, K = weight.shape
    x2 = x if x.dim() == 2 else x.reshape(-1, x.shape[-1])
    M = x2.shape[0] if row_index is None else row_index.numel()
    n_out = N if epilogue == EPILOGUE_NONE else N // 2
    _require_cuda(x2, weight)
    if x2.dtype != torch.bfloat16 or weight.dtype != torch.bfloat16 or x2.shape[1] != K or weight.stride(1) != 1 or x2.stride(1) != 1:
        raise ValueError("x and weight must be bfloat16 rows of the contraction length")
    if norm_kind != NORM_NONE and (norm_weight is None or norm_weight.dtype != torch.bfloat16 or tuple(norm_weight.shape) != (K,)
                                   or not norm_weight.is_contiguous() or not norm_weight.is_cuda):
        raise ValueError(f"norm_weight must be a contiguous bfloat16 ({K},) on the device")
    if bias is not None and (tuple(bias.shape) != (N,) or bias.dtype != torch.bfloat16 or not bias.is_contiguous()):
        raise ValueError(f"bias must be a contiguous bfloat16 ({N},)")
    for r in (residual_in, residual_out):
        if r is not None and (r.dtype != torch.float32 or tuple(r.shape) != (M, K) or r.stride(1) != 1 or not r.is_cuda):
            raise ValueError(f"residuals must be float32 ({M}, {K}) device tensors with contiguous rows")
    if row_index is not None and (row_index.dtype != torch.int64 or row_index.dim() != 1 or not row_index.is_contiguous()
                                  or not row_index.is_cuda):
        raise ValueError("row_index must be a contiguous int64 device vector")
    pos_ptr, pos_host = None, 0
    if mix is not None:
        mu, ring, pos, mix_rows = mix
        _check_ring(ring, M, 2, K, x2)
        if mu.dim() != 2 or mu.shape[1] != K or not mu.is_contiguous() or mu.dtype != torch.bfloat16 or not mu.is_cuda:
            raise ValueError(f"mu must be a contiguous bfloat16 (mixes, {K})")
        pos_ptr, pos_host = _pos_args(pos, M)
    if gate is not None:
        table, index = gate
        if (epilogue != EPILOGUE_NONE or table.dim() != 2 or table.shape[1] != N or table.stride(1) != 1 or table.dtype != torch.bfloat16
                or not table.is_cuda or index.dtype != torch.int64 or index.numel() != M or not index.is_contiguous() or not index.is_cuda):
            raise ValueError(f"the gate must be a bfloat16 (entries, {N}) table with {M} contiguous int64 entries")
    extra = _addend_args(addends, x2, M, K)
    if M > STREAM_PROLOGUE_MAX_ROWS:
        rows = x2 if row_index is None else x2.index_select(0, row_index)
        h, _ = add_norm(rows, residual_in, norm_weight, eps, norm_kind, mult, residual_out is not None, residual_out, addends)
        if mix is not None:
            if bias is not None or out is not None or epilogue != EPILOGUE_NONE:
                raise ValueError("mixes take no bias, epilogue or given output")
            return decode_linear_mixes(token_mix(h.unsqueeze(1), mu, ring, pos).squeeze(2), weight, mix_rows)
        y = decode_linear(h, weight, bias, epilogue=epilogue, out=out)
        if gate is not None:
            y = gelu_mul(y, table, index)
        return softcap_(y, softcap) if softcap else y
    y = torch.empty(M, n_out, dtype=torch.bfloat16, device=x2.device) if out is None else out
    if tuple(y.shape) != (M, n_out) or y.dtype != torch.bfloat16 or y.stride(1) != 1:
        raise ValueError(f"out must be a ({M}, {n_out}) bfloat16 tensor with contiguous rows")
    post_weight, post_eps, vec, add_rows, add_index, add_sr, add_n = extra
    ex = _lib.StreamExtras(post_weight=post_weight, post_eps=post_eps, add_vec=vec, add_rows=add_rows, add_index=add_index, add_sr=add_sr,
                           add_n=add_n, softcap=float(softcap))
    if mix is not None:
        ex.mix_mu, ex.mix_ring, ex.mix_ring_row_stride = mu.data_ptr(), ring.data_ptr(), ring.stride(0)
        ex.mixes, ex.mix_rows = mu.shape[0], int(mix_rows)
    if gate is not None:
        ex.gate_table, ex.gate_index, ex.gate_sr, ex.gate_n = table.data_ptr(), index.data_ptr(), table.stride(0), table.shape[0]
    with _on_device(x2.device):
        _lib.check(_lib.lib().based_decode_linear_extras(
            x2.data_ptr(), x2.stride(0), _ptr(row_index), 0 if row_index is None else x2.shape[0], weight.data_ptr(), weight.stride(0),
            _ptr(bias), y.data_ptr(), y.stride(0), M, N, K, _ptr(residual_in), 0 if residual_in is None else residual_in.stride(0),
            _ptr(residual_out), 0 if residual_out is None else residual_out.stride(0), float(mult), int(norm_kind),
            None if norm_kind == NORM_NONE else norm_weight.data_ptr(), float(eps), pos_ptr, pos_host, epilogue, ctypes.byref(ex),
            _stream_ptr(x2)))
    return y
