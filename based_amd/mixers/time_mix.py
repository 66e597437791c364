"""Time mixing with a decay per key channel: every projection reads its own mix of a token's input and the
input of the token before; a matrix state per head in fp32 with data-dependent decays from a low-rank
map, a bonus for the current token, an RMS norm per head and a silu gate on the way out."""
from __future__ import annotations

import torch
import torch.nn as nn
import torch.nn.functional as F

from .. import ops
from .streaming import cached, portion_start, project, round_up


class TimeMix(nn.Module):
    """o_t = (S + diag(u) k_t v_t^T)^T r_t, then S <- diag(w_t) S + k_t v_t^T, w = exp(-exp(w2 tanh(w1 x_w) + w0)).

    in_proj holds the rows of r, k, v, g (heads * dim each, on multiples of `SEGMENT` rows) and w1; mu one row per mix in that order."""

    MIXES = ("r", "k", "v", "g", "w")
    SEGMENT = 32

    def __init__(self, d_model: int, heads: int, dim: int, rank: int, norm_eps: float = 1e-5, layer_idx=None, device=None, dtype=None):
        super().__init__()
        fk = {"device": device, "dtype": dtype}
        self.heads, self.dim, self.rank, self.norm_eps, self.layer_idx = heads, dim, rank, norm_eps, layer_idx
        self.width = heads * dim
        self.segment = round_up(self.width, self.SEGMENT)
        self.mu = nn.Parameter(torch.full((len(self.MIXES), d_model), 0.5, **fk))
        self.in_proj = nn.Linear(d_model, 4 * self.segment + round_up(rank), bias=False, **fk)
        self.w2 = nn.Parameter(torch.empty(self.width, rank, **fk).normal_(std=0.1))
        self.w0 = nn.Parameter(torch.full((self.width,), -3.0, **fk))
        self.bonus = nn.Parameter(torch.zeros(heads, dim, **fk))
        self.norm_weight = nn.Parameter(torch.ones(self.width, **fk))
        self.out_proj = nn.Linear(round_up(self.width), d_model, bias=False, **fk)

    def allocate_state(self, batch_size: int, max_seqlen: int = 0, dtype=None):
        return torch.zeros(batch_size, self.heads, self.dim, round_up(self.dim, 4), device=self.mu.device, dtype=torch.float32)

    def allocate_ring(self, batch_size: int, max_seqlen: int = 0, dtype=None):
        return torch.zeros(batch_size, 2, self.mu.shape[1], device=self.mu.device, dtype=self.mu.dtype)

    def allocate_inference_cache(self, batch_size: int, max_seqlen: int, dtype=None, **kwargs):
        return {"state": self.allocate_state(batch_size), "before": self.allocate_ring(batch_size)}

    def _rows(self, i: int) -> slice:
        """Rows of in_proj that read mix i."""
        return slice(i * self.segment, i * self.segment + (self.width if i < 4 else self.rank))

    def _cached(self, inference_params, batch: int):
        if inference_params is None:
            return self.allocate_state(batch), None
        return (cached(inference_params, self.layer_idx, "state", self.allocate_state, batch),
                cached(inference_params, self.layer_idx, "before", self.allocate_ring, batch))

    def _context(self, rows, like):
        make = torch.empty if self.out_proj.in_features == self.width else torch.zeros
        return make(*rows, self.out_proj.in_features, dtype=like.dtype, device=like.device)

    def _step(self, r, k, v, g, hidden, state, pos):
        """One token behind the projections, every argument (B, features)."""
        out = self._context(r.shape[:1], r)
        ops.decay_step(r, k, v, state, self.heads, pos, bonus=self.bonus, hidden=hidden, w2=self.w2, w0=self.w0, gate=g,
                       norm_weight=self.norm_weight, eps=self.norm_eps, out=out[:, :self.width])
        return out

    def supports_decode_step(self) -> bool:
        return ops.decode_linear_weight_ok(self.in_proj.weight) and ops.decode_linear_weight_ok(self.out_proj.weight)

    def decode_step(self, x, inference_params, **prologue):
        """One token per sequence: norm and mixes inside the input projections (`ops.decode_linear`)."""
        rows = x.shape[0] if prologue.get("row_index") is None else prologue["row_index"].numel()
        pos, _ = portion_start(inference_params, rows, 1)
        state, ring = self._cached(inference_params, rows)
        proj = ops.decode_linear(x, self.in_proj.weight, mix=(self.mu, ring, pos, self.segment), **prologue)
        return ops.decode_linear(self._step(*(proj[:, self._rows(i)] for i in range(len(self.MIXES))), state, pos), self.out_proj.weight)

    def forward(self, x, inference_params=None, **kwargs):
        """x (batch, seqlen, d_model) -> (batch, seqlen, d_model)."""
        B, L = x.shape[:2]
        start, step = portion_start(inference_params, B, L)
        state, ring = self._cached(inference_params, B)
        mixed = ops.token_mix(x, self.mu, ring, start)
        r, k, v, g, hidden = (F.linear(mixed[i], self.in_proj.weight[self._rows(i)]) for i in range(len(self.MIXES)))
        if step:
            return project(self._step(r[:, 0], k[:, 0], v[:, 0], g[:, 0], hidden[:, 0], state, start), self.out_proj).unsqueeze(1)
        decay = ops.channel_decay(hidden, self.w2, self.w0)
        o = ops.decay_scan(r, k, v, state, self.heads, channel_log2=decay, bonus=self.bonus, fresh=start == 0)
        out = self._context((B, L), x)
        ops.group_norm_gate(o, self.norm_weight, g, self.heads, self.norm_eps, ops.ACT_SILU, out=out[..., :self.width])
        return project(out, self.out_proj)
