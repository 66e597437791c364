"""Recurrent block with a real-gated linear recurrent unit: out_proj(S * gelu_tanh(W_y h + b)), where S is
the gated linear recurrence over the convolved second branch conv(W_x h + b), with block-diagonal
gates and a vector state per sequence in fp32."""
from __future__ import annotations

import torch
import torch.nn as nn

from .. import ops
from .streaming import StreamConv, cached, portion_start, project, round_up


class RGLRU(nn.Module):
    def __init__(self, d_model: int, width: int, blocks: int, conv_taps: int, decay_scale: float = 8.0, bias: bool = True,
                 layer_idx=None, device=None, dtype=None):
        super().__init__()
        fk = {"device": device, "dtype": dtype}
        if width % blocks != 0:
            raise ValueError(f"{width} channels do not divide into {blocks} blocks")
        self.width, self.blocks, self.decay_scale, self.layer_idx = width, blocks, decay_scale, layer_idx
        self.x_off = round_up(width)  # rows of in_proj: y, then x
        n = width // blocks
        self.in_proj = nn.Linear(d_model, 2 * self.x_off, bias=bias, **fk)
        self.conv = StreamConv(width, conv_taps, bias=bias, layer_idx=layer_idx, name="conv", **fk)
        self.gate_r = nn.Parameter(torch.empty(blocks, n, n, **fk))   # [out, in]
        self.gate_i = nn.Parameter(torch.empty(blocks, n, n, **fk))
        nn.init.normal_(self.gate_r, std=n ** -0.5)
        nn.init.normal_(self.gate_i, std=n ** -0.5)
        self.bias_r = nn.Parameter(torch.zeros(width, **fk))
        self.bias_i = nn.Parameter(torch.zeros(width, **fk))
        self.lam = nn.Parameter(torch.full((width,), -3.0, **fk))
        self.out_proj = nn.Linear(self.x_off, d_model, bias=False, **fk)

    def allocate_state(self, batch_size: int, max_seqlen: int = 0, dtype=None):
        return torch.zeros(batch_size, self.width, device=self.lam.device, dtype=torch.float32)

    def allocate_inference_cache(self, batch_size: int, max_seqlen: int, dtype=None, **kwargs):
        return {"state": self.allocate_state(batch_size), "conv": self.conv.allocate_ring(batch_size)}

    def _mix(self, proj, inference_params):
        B, L = proj.shape[:2]
        y, x = proj[..., :self.width], proj[..., self.x_off:self.x_off + self.width]
        start, step = portion_start(inference_params, B, L)
        if inference_params is None:
            state = self.allocate_state(B)
        else:
            state = cached(inference_params, self.layer_idx, "state", self.allocate_state, B)
        out = (torch.empty if self.x_off == self.width else torch.zeros)(B, L, self.x_off, dtype=proj.dtype, device=proj.device)
        gates = (self.gate_r, self.bias_r, self.gate_i, self.bias_i, self.lam)
        if step:
            ops.rglru_step(x[:, 0], y[:, 0], self.conv.weight, self.conv.bias, self.conv.ring(inference_params, B), *gates, state,
                           self.decay_scale, start, out=out[:, 0, :self.width])
        else:
            u = self.conv(x, inference_params)
            ops.rglru_prefill(u, y, *gates, state, self.decay_scale, fresh=not isinstance(start, torch.Tensor) and start == 0,
                              out=out[..., :self.width])
        return out

    def supports_decode_step(self) -> bool:
        return ops.decode_linear_weight_ok(self.in_proj.weight) and ops.decode_linear_weight_ok(self.out_proj.weight)

    def decode_step(self, x, inference_params, **prologue):
        """One token per sequence with the projections as `ops.decode_linear` launches."""
        proj = ops.decode_linear(x, self.in_proj.weight, self.in_proj.bias, **prologue)
        return ops.decode_linear(self._mix(proj.unsqueeze(1), inference_params)[:, 0], self.out_proj.weight)

    def forward(self, x, inference_params=None, **kwargs):
        """x (batch, seqlen, d_model) -> (batch, seqlen, d_model)."""
        return project(self._mix(project(x, self.in_proj), inference_params), self.out_proj)
