"""Linear attention with a constant decay per head as the part of a mixer between its projections (see
SideBySide): silu on q, k and v, a matrix state per head in fp32, one RMS norm over all heads and a
sigmoid gate on the way out."""
from __future__ import annotations

import torch
import torch.nn as nn

from .. import ops
from .streaming import cached, portion_start, round_up


class DecayAttention(nn.Module):
    """Core with segments q, k (heads * dim), v, g (heads * vdim) and heads * vdim outputs: S <- decay_h S + k v^T, o = S^T q."""

    def __init__(self, heads: int, dim: int, vdim: int, decay, norm_eps: float = 1e-5, layer_idx=None, name: str = "decay", device=None,
                 dtype=None):
        super().__init__()
        if len(decay) != heads or min(decay) < 0 or max(decay) > 1:
            raise ValueError(f"{heads} decays between 0 and 1, one per head: got {decay}")
        self.heads, self.dim, self.vdim, self.norm_eps = heads, dim, vdim, norm_eps
        self.layer_idx, self.name = layer_idx, name
        self.decay = tuple(float(w) for w in decay)
        self.norm_weight = nn.Parameter(torch.ones(heads * vdim, device=device, dtype=dtype))

    segments = property(lambda self: (("q", self.heads * self.dim), ("k", self.heads * self.dim), ("v", self.heads * self.vdim),
                                      ("g", self.heads * self.vdim)))
    out_features = property(lambda self: self.heads * self.vdim)

    def _head_decay(self, device):
        """The decays on the device, in fp32 whatever the model's dtype; kept (a recorded graph holds their address)."""
        made = self.__dict__.setdefault("_device_decay", {})
        if device not in made:
            made[device] = ops.head_decays(self.decay, device)
        return made[device]

    def allocate_state(self, batch_size: int, max_seqlen: int = 0, dtype=None):
        return torch.zeros(batch_size, self.heads, self.vdim, round_up(self.dim, 4), device=self.norm_weight.device, dtype=torch.float32)

    def allocations(self):
        return {self.name: self.allocate_state}

    def forward(self, part, out, out_scale: float = 1.0, inference_params=None):
        q, k, v, g = part("q"), part("k"), part("v"), part("g")
        B, L = q.shape[:2]
        start, step = portion_start(inference_params, B, L)
        if inference_params is None:
            state = self.allocate_state(B)
        else:
            state = cached(inference_params, self.layer_idx, self.name, self.allocate_state, B)
        decay = self._head_decay(q.device)
        if step:
            o = torch.empty(B, 1, self.out_features, dtype=q.dtype, device=q.device)
            ops.decay_step(q[:, 0], k[:, 0], v[:, 0], state, self.heads, start, head_decay=decay, activation=ops.ACT_SILU, out=o[:, 0])
        else:
            o = ops.decay_scan(q, k, v, state, self.heads, head_decay=decay, activation=ops.ACT_SILU, fresh=start == 0)
        ops.group_norm_gate(o, self.norm_weight, g, 1, self.norm_eps, ops.ACT_SIGMOID, out_scale, out=out)
