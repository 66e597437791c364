"""Gated delta rule as the part of a mixer between its projections (see SideBySide): short convolutions
with silu on q, k and v, unit-norm q and k, one decay and one step size per head, a matrix state per
head in fp32, and an RMS norm and a silu gate on the way out."""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn as nn

from .. import ops
from .streaming import StreamConv, cached, portion_start, round_up


class GatedDeltaRule(nn.Module):
    """Core with segments q, k (kv_heads * dim), v, g (heads * vdim), b, a (heads) and heads * vdim outputs;
    head h uses query/key head h // (heads / kv_heads)."""

    def __init__(self, heads: int, dim: int, vdim: int, conv_taps: int, kv_heads: Optional[int] = None, norm_eps: float = 1e-5,
                 layer_idx=None, name: str = "delta", device=None, dtype=None):
        super().__init__()
        fk = {"device": device, "dtype": dtype}
        kv_heads = heads if kv_heads is None else kv_heads
        if heads % kv_heads != 0:
            raise ValueError(f"{heads} heads do not divide into {kv_heads} query/key heads")
        self.heads, self.kv_heads, self.dim, self.vdim, self.norm_eps = heads, kv_heads, dim, vdim, norm_eps
        self.layer_idx, self.name = layer_idx, name
        # channels of the convolution: the q, k and v segments as they lie in the projection
        self.k_off = round_up(kv_heads * dim)
        self.v_off = 2 * self.k_off
        self.conv = StreamConv(self.v_off + round_up(heads * vdim), conv_taps, activation=ops.ACT_SILU, layer_idx=layer_idx,
                               name=f"{name}.conv", **fk)
        self.A_log = nn.Parameter(torch.zeros(heads, **fk))
        self.dt_bias = nn.Parameter(torch.full((heads,), -2.0, **fk))
        self.norm_weight = nn.Parameter(torch.ones(vdim, **fk))

    segments = property(lambda self: (("q", self.kv_heads * self.dim), ("k", self.kv_heads * self.dim), ("v", self.heads * self.vdim),
                                      ("g", self.heads * self.vdim), ("b", self.heads), ("a", self.heads)))
    out_features = property(lambda self: self.heads * self.vdim)

    def allocate_state(self, batch_size: int, max_seqlen: int = 0, dtype=None):
        return torch.zeros(batch_size, self.heads, self.dim, round_up(self.vdim, 4), device=self.A_log.device, dtype=torch.float32)

    def allocations(self):
        return {self.name: self.allocate_state, self.conv.name: self.conv.allocate_ring}

    def forward(self, part, out, out_scale: float = 1.0, inference_params=None):
        x = part("q", self.conv.channels)  # q, k and v with what lies between them
        a, b, g = part("a"), part("b"), part("g")
        B, L = x.shape[:2]
        start, step = portion_start(inference_params, B, L)
        if inference_params is None:
            state = self.allocate_state(B)
        else:
            state = cached(inference_params, self.layer_idx, self.name, self.allocate_state, B)
        if step:
            ops.gated_delta_step(x[:, 0], self.conv.weight, self.conv.ring(inference_params, B), a[:, 0], b[:, 0], g[:, 0], self.A_log,
                                 self.dt_bias, self.norm_weight, state, self.heads, self.kv_heads, self.dim, self.vdim, self.k_off,
                                 self.v_off, start, self.norm_eps, out_scale, out=out[:, 0])
            return
        c = self.conv(x, inference_params)
        nk, nv = self.kv_heads * self.dim, self.heads * self.vdim
        o = ops.gated_delta_scan(c[..., :nk], c[..., self.k_off:self.k_off + nk], c[..., self.v_off:self.v_off + nv], a, b, self.A_log,
                                 self.dt_bias, state, self.heads, self.kv_heads, fresh=not isinstance(start, torch.Tensor) and start == 0)
        ops.gated_rms_norm(o, self.norm_weight, g, self.norm_eps, out_scale, out=out)
