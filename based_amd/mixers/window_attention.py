"""Sliding-window softmax attention with grouped heads as the part of a mixer between its projections
(see SideBySide): window of any size, key and value sizes of their own, rotary positions on leading
channels in either pair layout, an explicit score scale, an optional value norm."""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from .. import ops
from .slide_attention import RotaryEmbedding
from .streaming import cached, portion_start


class _ExactRotary(RotaryEmbedding):
    """Tables from angles formed in 64 bits, so that far positions lose nothing to p * f in fp32."""

    def _cos_sin(self, positions):
        freq = self.base ** (-torch.arange(0, self.dim, 2, dtype=torch.float64) / self.dim)
        angles = torch.outer(positions.cpu().double(), freq)
        return angles.cos().float().to(positions.device), angles.sin().float().to(positions.device)


class WindowAttention(nn.Module):
    """Core with segments q (heads * dim), k (kv_heads * dim), v (kv_heads * vdim) and heads * vdim outputs.
    Position i attends j with 0 <= i - j < window."""

    def __init__(self, heads: int, dim: int, window: int, kv_heads: Optional[int] = None, vdim: Optional[int] = None,
                 scale: Optional[float] = None, rotary_dim: int = 0, rotary_base: float = 10000.0, rotary_interleaved: bool = True,
                 value_norm_eps: Optional[float] = None, layer_idx=None, name: str = "attn", device=None, dtype=None):
        super().__init__()
        kv_heads = heads if kv_heads is None else kv_heads
        vdim = dim if vdim is None else vdim
        if heads % kv_heads != 0:
            raise ValueError(f"{heads} query heads do not divide into {kv_heads} key/value heads")
        if rotary_dim % 2 != 0 or rotary_dim > dim:
            raise ValueError(f"rotary_dim {rotary_dim} must be even and at most the head size {dim}")
        if window < 1:
            raise ValueError(f"window {window}")
        self.heads, self.kv_heads, self.dim, self.vdim, self.window = heads, kv_heads, dim, vdim, window
        self.scale = dim ** -0.5 if scale is None else float(scale)
        self.value_norm_eps = value_norm_eps
        self.layer_idx, self.name = layer_idx, name
        self.rotary = _ExactRotary(rotary_dim, base=rotary_base, interleaved=rotary_interleaved) if rotary_dim > 0 else None
        self.register_buffer("_like", torch.empty(0, device=device, dtype=dtype), persistent=False)  # device and dtype of the cache

    segments = property(lambda self: (("q", self.heads * self.dim), ("k", self.kv_heads * self.dim), ("v", self.kv_heads * self.vdim)))
    out_features = property(lambda self: self.heads * self.vdim)

    def allocate_cache(self, batch_size: int, max_seqlen: int, dtype=None):
        return torch.empty(batch_size, max_seqlen, self.kv_heads, self.dim + self.vdim, device=self._like.device, dtype=self._like.dtype)

    def allocations(self):
        return {self.name: self.allocate_cache}

    def forward(self, part, out, out_scale: float = 1.0, inference_params=None):
        """part(name) -> that segment of the projection, (B, L, features); writes out (B, L, out_features)."""
        q, k, v = part("q"), part("k"), part("v")
        B, L = q.shape[:2]
        start, step = portion_start(inference_params, B, L)
        if inference_params is None:
            kv, n_pos = self.allocate_cache(B, L), L
        else:
            kv = cached(inference_params, self.layer_idx, self.name, self.allocate_cache, B)
            n_pos = kv.shape[1]
        rope = None if self.rotary is None else self.rotary.tables(n_pos, q.device)
        args = (kv, self.heads, self.kv_heads, self.window, self.scale)
        kw = dict(rope=rope, value_norm_eps=self.value_norm_eps, out_scale=out_scale)
        if step:
            ops.window_attn_step(q[:, 0], k[:, 0], v[:, 0], *args, start, out=out[:, 0], **kw)
        else:
            ops.window_attn_prefill(q, k, v, *args, start, out=out, **kw)
