"""Mixer cores that read the same input, side by side: one stacked input projection, the cores, and one
output projection over the concatenated outputs, each multiplied by its scale before it is rounded:
sum_i scale_i W_i core_i(x).  With one core it is an ordinary mixer.

A core has `segments` (name, rows of the input projection), `out_features`, `allocations()` (name ->
allocator of its caches) and forward(part, out, out_scale, inference_params)."""
from __future__ import annotations

import torch
import torch.nn as nn

from .. import ops
from .streaming import project, round_up


class SideBySide(nn.Module):
    def __init__(self, d_model: int, cores, scales=None, layer_idx=None, device=None, dtype=None):
        """cores: modules, or functions of (layer_idx, name, device, dtype) that return one."""
        super().__init__()
        fk = {"device": device, "dtype": dtype}
        self.layer_idx = layer_idx
        self.cores = nn.ModuleList(c if isinstance(c, nn.Module) else c(layer_idx=layer_idx, name=f"core{i}", **fk)
                                   for i, c in enumerate(cores))
        self.scales = [1.0] * len(self.cores) if scales is None else [float(s) for s in scales]
        # every segment starts on a multiple of 8 rows: 16-byte pieces in its slice of the projection
        self.in_rows = []   # per core: name -> (first row, rows)
        row = 0
        for core in self.cores:
            rows = {}
            for name, n in core.segments:
                rows[name] = (row, n)
                row += round_up(n)
            self.in_rows.append(rows)
        self.out_cols = []  # per core: (first column of out_proj, columns)
        col = 0
        for core in self.cores:
            self.out_cols.append((col, core.out_features))
            col += round_up(core.out_features)
        self._gaps = any(core.out_features % 8 for core in self.cores)
        self.in_proj = nn.Linear(d_model, row, bias=False, **fk)
        self.out_proj = nn.Linear(col, d_model, bias=False, **fk)

    def allocate_inference_cache(self, batch_size: int, max_seqlen: int, dtype=None, **kwargs):
        return {name: make(batch_size, max_seqlen) for core in self.cores for name, make in core.allocations().items()}

    def _mix(self, proj, inference_params):
        """proj (B, L, rows of in_proj) -> (B, L, columns of out_proj)."""
        B, L = proj.shape[:2]
        # columns between the cores' outputs meet zero weights and only have to be finite
        ctx = (torch.zeros if self._gaps else torch.empty)(B, L, self.out_proj.in_features, dtype=proj.dtype, device=proj.device)
        for core, rows, (col, n), scale in zip(self.cores, self.in_rows, self.out_cols, self.scales):
            def part(name, width=None, rows=rows):
                first, width_ = rows[name]
                return proj[..., first:first + (width_ if width is None else width)]

            core(part, ctx[..., col:col + n], scale, inference_params)
        return ctx

    def supports_decode_step(self) -> bool:
        return ops.decode_linear_weight_ok(self.in_proj.weight) and ops.decode_linear_weight_ok(self.out_proj.weight)

    def decode_step(self, x, inference_params, **prologue):
        """One token per sequence with the projections as `ops.decode_linear` launches."""
        proj = ops.decode_linear(x, self.in_proj.weight, **prologue)
        ctx = self._mix(proj.unsqueeze(1), inference_params)
        return ops.decode_linear(ctx[:, 0], self.out_proj.weight)

    def forward(self, x, inference_params=None, **kwargs):
        """x (batch, seqlen, d_model) -> (batch, seqlen, d_model)."""
        return project(self._mix(project(x, self.in_proj), inference_params), self.out_proj)
