"""Sliding-window softmax attention over a cache of latents as the part of a mixer between its projections
(see SideBySide).  A token is cached as one normalised latent and one rotated key part that all heads
share.  Prompts expand the rows they see to keys and values with one matrix product; single tokens
attend in the latent space."""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from .. import ops
from .streaming import cached, portion_start
from .window_attention import _ExactRotary

NO_WINDOW = 1 << 30


class LatentAttention(nn.Module):
    """Core with segments q (heads * (rot_dim + dim), a head's rotated channels first), kv (kv_rank + rot_dim: the latent, the shared key
    part) and heads * vdim outputs.  Position i attends j with 0 <= i - j < window (None: every j <= i).

    `expand` maps a cache row to every head's key [rotated part | uk c] and value uv c, laid out like the rows of a key/value
    cache: the rows of a head are rot_dim rows of an identity on the shared part, dim rows of uk, vdim rows of uv."""

    def __init__(self, heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, window: Optional[int] = None,
                 scale: Optional[float] = None, rotary_base: float = 10000.0, rotary_interleaved: bool = False, norm_eps: float = 1e-5,
                 layer_idx=None, name: str = "latent", device=None, dtype=None):
        super().__init__()
        fk = {"device": device, "dtype": dtype}
        if rot_dim % 2 != 0 or rot_dim < 0:
            raise ValueError(f"rot_dim {rot_dim} must be even")
        if window is not None and window < 1:
            raise ValueError(f"window {window}")
        self.heads, self.dim, self.rot_dim, self.vdim, self.kv_rank = heads, dim, rot_dim, vdim, kv_rank
        self.window = NO_WINDOW if window is None else window
        self.scale = (dim + rot_dim) ** -0.5 if scale is None else float(scale)
        self.norm_eps, self.layer_idx, self.name = norm_eps, layer_idx, name
        self.rotary = _ExactRotary(rot_dim, base=rotary_base, interleaved=rotary_interleaved) if rot_dim > 0 else None
        self.norm_weight = nn.Parameter(torch.ones(kv_rank, **fk))
        self.expand = nn.Parameter(self.expansion(torch.empty(heads * dim, kv_rank, **fk).normal_(std=kv_rank ** -0.5),
                                                  torch.empty(heads * vdim, kv_rank, **fk).normal_(std=kv_rank ** -0.5), heads, rot_dim))

    @staticmethod
    def expansion(uk, uv, heads: int, rot_dim: int):
        """`expand` from uk (heads * dim, kv_rank) and uv (heads * vdim, kv_rank)."""
        rank = uk.shape[1]
        uk, uv = uk.view(heads, -1, rank), uv.view(heads, -1, rank)
        rows = uk.new_zeros(heads, rot_dim + uk.shape[1] + uv.shape[1], rank + rot_dim)
        rows[:, :rot_dim, rank:] = torch.eye(rot_dim, dtype=uk.dtype, device=uk.device)
        rows[:, rot_dim:rot_dim + uk.shape[1], :rank] = uk
        rows[:, rot_dim + uk.shape[1]:, :rank] = uv
        return rows.view(-1, rank + rot_dim)

    segments = property(lambda self: (("q", self.heads * (self.rot_dim + self.dim)), ("kv", self.kv_rank + self.rot_dim)))
    out_features = property(lambda self: self.heads * self.vdim)

    def allocate_cache(self, batch_size: int, max_seqlen: int, dtype=None):
        return torch.empty(batch_size, max_seqlen, self.kv_rank + self.rot_dim, device=self.norm_weight.device, dtype=self.norm_weight.dtype)

    def allocations(self):
        return {self.name: self.allocate_cache}

    def forward(self, part, out, out_scale: float = 1.0, inference_params=None):
        """part(name) -> that segment of the projection, (B, L, features); writes out (B, L, out_features)."""
        q, x = part("q"), part("kv")
        B, L = q.shape[:2]
        start, step = portion_start(inference_params, B, L)
        if inference_params is None:
            cache, n_pos = self.allocate_cache(B, L), L
        else:
            cache = cached(inference_params, self.layer_idx, self.name, self.allocate_cache, B)
            n_pos = cache.shape[1]
        rope = None if self.rotary is None else self.rotary.tables(n_pos, q.device)
        if step:
            ops.latent_step(q[:, 0], x[:, 0], self.norm_weight, self.expand, cache, self.heads, self.dim, self.window, self.scale, start,
                            self.norm_eps, rope, out_scale, out=out[:, 0])
            return
        ops.latent_write(x, self.norm_weight, cache, start, self.norm_eps, rope)
        # keys and values of every row that the portion sees; positions count from the first of them
        lo = max(0, start - self.window + 1)
        kv = F.linear(cache[:, lo:start + L], self.expand).view(B, start + L - lo, self.heads, -1)
        if rope is not None:
            rope = (rope[0][lo:], rope[1][lo:], rope[2])
        ops.window_attn_attend(q, kv, self.heads, self.heads, self.rot_dim + self.dim, self.window, self.scale, start - lo, rope, out_scale,
                               out=out)
