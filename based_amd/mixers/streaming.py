"""What the streamed layers share: the per-layer store of caches inside InferenceParams, the place of a
portion in its sequence, rounded-up segments of stacked projections, and the causal convolution on a
ring of past inputs.

A streamed layer takes portions of any length: `InferenceParams.seqlen_offset` tokens lie before the
portion, a single token behind a prompt runs the step kernels, and with `lengths_per_sample` set its
position comes from the device (a recorded decode graph).  Nothing is cleared between sequences: a
portion at offset 0 starts every recurrence at zero and reads no ring."""
from __future__ import annotations

import torch
import torch.nn as nn
import torch.nn.functional as F

from .. import ops


def round_up(n: int, to: int = 8) -> int:
    return (n + to - 1) // to * to


def project(x, linear: nn.Linear):
    return F.linear(x, linear.weight, linear.bias)


def portion_start(inference_params, batch: int, seqlen: int):
    """(start, step): where the portion begins (an int, or the device positions of a decoding step) and
    whether it is one token behind others, which the step kernels take."""
    if inference_params is None or inference_params.seqlen_offset == 0:
        return 0, False
    offset = inference_params.seqlen_offset
    if seqlen != 1:
        return offset, False
    lengths = inference_params.lengths_per_sample
    if lengths is not None:
        b0 = inference_params.batch_size_offset
        return lengths[b0:b0 + batch], True
    return offset, True


def cached(inference_params, layer_idx, name: str, allocate, batch: int):
    """The rows of this batch of the tensor `name` of a layer, created for the largest batch when it is not there."""
    store = inference_params.key_value_memory_dict.setdefault(inference_params.layer_key(layer_idx), {})
    if name not in store:
        store[name] = allocate(inference_params.max_batch_size, inference_params.max_seqlen)
    b0 = inference_params.batch_size_offset
    return store[name][b0:b0 + batch]


class StreamConv(nn.Module):
    """y_t = [x_t +] act(bias + sum_j weight[j] x_{t - taps + 1 + j}) per channel; weight (taps, channels)."""

    def __init__(self, channels: int, taps: int, bias: bool = False, activation: int = ops.ACT_NONE, add_input: bool = False,
                 layer_idx=None, name: str = "conv", device=None, dtype=None):
        super().__init__()
        if not 1 <= taps <= ops.STREAM_MAX_TAPS:
            raise NotImplementedError(f"{taps} taps: the convolution kernels take 1 to {ops.STREAM_MAX_TAPS}")
        self.channels, self.taps, self.activation, self.add_input = channels, taps, activation, add_input
        self.layer_idx, self.name = layer_idx, name
        self.weight = nn.Parameter(torch.empty(taps, channels, device=device, dtype=dtype))
        self.bias = nn.Parameter(torch.zeros(channels, device=device, dtype=dtype)) if bias else None
        nn.init.normal_(self.weight, std=taps ** -0.5)

    def allocate_ring(self, batch_size: int, max_seqlen: int = 0, dtype=None):
        return torch.zeros(batch_size, self.taps, self.channels, device=self.weight.device, dtype=self.weight.dtype)

    def ring(self, inference_params, batch: int):
        if inference_params is None:
            return None
        return cached(inference_params, self.layer_idx, self.name, self.allocate_ring, batch)

    def forward(self, x, inference_params=None):
        start, _ = portion_start(inference_params, x.shape[0], x.shape[1])
        return ops.stream_conv(x, self.weight, self.bias, self.ring(inference_params, x.shape[0]), start, self.activation,
                               self.add_input)
