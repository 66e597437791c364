"""Minimal Based language-model stack around the HIP mixers (plain PyTorch glue).

Just enough of based/models/gpt.py (create_mixer_cls :64-96, create_block :347-394, _init_weights
:463-485, GPTModel :510-736, GPTLMHeadModel :739-827), block.py (:114-163), mlp.py (GatedMlp
:99-157) and the RMSNorm closed form (based/ops/triton/layer_norm.py:117-118) to run the
27-layer Based-360m shape end to end: embeddings -> [prenorm Block(mixer, SwiGLU MLP)] x N ->
final norm -> tied LM head, with the generation cache threaded through.  The GEMMs and the
embedding lookup are ordinary torch (hipBLASLt); mixers, add + RMSNorm and the SwiGLU gate are
the HIP kernels, and there is no host-tensor path.
"""
from __future__ import annotations

import math
from collections import namedtuple
from functools import partial
from types import SimpleNamespace
from typing import NamedTuple, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from . import ops

from .generation import GenerationMixin
from .mixers.convolution import BaseConv, ShortConvolution
from .mixers.decay_attention import DecayAttention
from .mixers.gated_delta import GatedDeltaRule
from .mixers.latent_attention import LatentAttention
from .mixers.linear_attention import LinearAttention, TaylorExp
from .mixers.rglru import RGLRU
from .mixers.side_by_side import SideBySide
from .mixers.slide_attention import SlidingAttention
from .mixers.streaming import StreamConv, portion_start, round_up
from .mixers.time_mix import TimeMix
from .mixers.window_attention import WindowAttention

# `_target_` strings accepted in mixer config dicts: the reference's own paths and this package's.
_TARGETS = {
    "based.models.mixers.linear_attention.LinearAttention": LinearAttention,
    "based.models.mixers.linear_attention.TaylorExp": TaylorExp,
    "based.models.mixers.slide_attention.SlidingAttention": SlidingAttention,
    "based.models.mixers.convolution.BaseConv": BaseConv,
    "based.models.mixers.convolution.ShortConvolution": ShortConvolution,
    "based_amd.mixers.linear_attention.LinearAttention": LinearAttention,
    "based_amd.mixers.linear_attention.TaylorExp": TaylorExp,
    "based_amd.mixers.slide_attention.SlidingAttention": SlidingAttention,
    "based_amd.mixers.convolution.BaseConv": BaseConv,
    "based_amd.mixers.convolution.ShortConvolution": ShortConvolution,
    "based_amd.mixers.decay_attention.DecayAttention": DecayAttention,
    "based_amd.mixers.gated_delta.GatedDeltaRule": GatedDeltaRule,
    "based_amd.mixers.latent_attention.LatentAttention": LatentAttention,
    "based_amd.mixers.rglru.RGLRU": RGLRU,
    "based_amd.mixers.side_by_side.SideBySide": SideBySide,
    "based_amd.mixers.time_mix.TimeMix": TimeMix,
    "based_amd.mixers.window_attention.WindowAttention": WindowAttention,
}


def _instantiate(spec: dict, *args, **extra):
    """Tiny stand-in for hydra.utils.instantiate: nested dicts with `_target_` become objects; in a list
    they become constructors, which the mixer that holds the list completes (layer_idx, device, ...)."""
    spec = dict(spec)
    cls = _TARGETS[spec.pop("_target_")]

    def value(v):
        if isinstance(v, dict) and "_target_" in v:
            return _instantiate(v)
        if isinstance(v, (list, tuple)) and any(isinstance(x, dict) and "_target_" in x for x in v):
            return [partial(_TARGETS[x["_target_"]], **{k: y for k, y in x.items() if k != "_target_"}) for x in v]
        return v

    kwargs = {k: value(v) for k, v in spec.items()}
    kwargs.update(extra)
    return cls(*args, **kwargs)


class StackConfig(SimpleNamespace):
    """Attribute bag with the GPT2Config fields the stack reads (gpt.py:58-61 lets the config
    carry arbitrary attributes; so does this)."""

    def __init__(self, **kw):
        defaults = dict(
            n_embd=1024, n_layer=27, n_head=16, n_inner=None, vocab_size=50277, pad_vocab_size_multiple=8,
            layer_norm_epsilon=1e-5, rms_norm=True, residual_in_fp32=True, initializer_range=0.02,
            tie_word_embeddings=True, activation_function="swiglu", mlp_fc1_bias=False, mlp_fc2_bias=False,
            mlp_type="base", ff_mult=2,
            qkv_proj_bias=False, out_proj_bias=False, rotary_emb_fraction=0.0, rotary_emb_base=10000.0,
            rotary_emb_interleaved=False, scale_attn_weights=True, max_position_embeddings=0,
            mixer=None, alt_mixer=None, alt_mixer_layers=None, alt_mixer_2=None, alt_mixer_2_layers=None,
            # Streamed designs.  layer_specs: one {"mixer": spec, "mlp": spec} per layer instead of the mixer /
            # alt_mixer routing, the feed-forward None, {"hidden": n} or {"hidden": n, "experts": e, "top": k};
            # stream_norm: "layer" or "rms" without a bias on the fp32 residual sum; residual_mult: factor of
            # every sublayer's output; input_conv_taps: causal convolution added to what a mixer reads (0: none).
            # loop: {"start": i, "stop": j, "times": n}: layers i .. j - 1 run n times in a row with the same
            # weights and caches of their own, a learned vector per pass (and, from the second on, the embedding)
            # added before each; token_side_dim: size of the token input that every layer adds behind its
            # feed-forward (0: none); logit_softcap: c tanh(logits / c).
            layer_specs=None, stream_norm=None, residual_mult=1.0, input_conv_taps=0, loop=None, token_side_dim=0,
            logit_softcap=None,
        )
        defaults.update(kw)
        super().__init__(**defaults)

    # What the reference assumes for a key that a config dictionary does not carry: transformers'
    # GPT2Config constructor defaults plus the getattr defaults of based/models/gpt.py:100-113,
    # 206-208, 254, 262, 352, 359, 529, 745.  They differ from the defaults above (which describe
    # the released Based configurations): a config.json written by the reference's training code
    # that omits a key must mean here what it means there.
    REFERENCE_DEFAULTS = dict(
        n_embd=768, n_layer=12, n_head=12, n_inner=None, vocab_size=50257, pad_vocab_size_multiple=1,
        layer_norm_epsilon=1e-5, rms_norm=False, residual_in_fp32=False, initializer_range=0.02,
        tie_word_embeddings=True, activation_function="gelu_new", mlp_fc1_bias=True, mlp_fc2_bias=True,
        mlp_type="base", ff_mult=2, qkv_proj_bias=True, out_proj_bias=True, rotary_emb_fraction=0.0,
        rotary_emb_base=10000.0, rotary_emb_interleaved=False, scale_attn_weights=True,
        max_position_embeddings=0, n_positions=1024,
    )

    @classmethod
    def from_reference_dict(cls, d: dict) -> "StackConfig":
        """Config from a dictionary in the reference's format (the content of a checkpoint's
        config.json, or the keyword arguments its tests pass to GPT2MixerConfig), missing keys
        filled with the reference's defaults.  GPT2Config's `n_positions` feeds
        `max_position_embeddings` (its attribute map), as the reference's model reads it."""
        cfg = dict(cls.REFERENCE_DEFAULTS)
        cfg.update(d)
        if "max_position_embeddings" not in d:
            cfg["max_position_embeddings"] = cfg["n_positions"]
        return cls(**cfg)

    @property
    def hidden_size(self):
        return self.n_embd

    @property
    def num_hidden_layers(self):
        return self.n_layer

    @property
    def num_attention_heads(self):
        return self.n_head


def based_360m_config(**overrides) -> StackConfig:
    """The 360M-scale benchmark stack: the layer plan of the released Based-360m (BaseConv everywhere
    except Taylor linear attention at layers {1,6,11,16,21} and sliding-window attention at
    {2,7,12,17,22}; train/configs/experiment/reference/based-360m.yaml:53-65) with window_size 128,
    i.e. 64 keys to the left, and no rotary.  The released checkpoint itself uses window_size 256
    and rotary over the whole head: `based_360m_released_config`."""
    cfg = dict(
        n_embd=1024, n_layer=27, n_head=16, n_inner=2048, vocab_size=50277,
        mixer={"_target_": "based.models.mixers.convolution.BaseConv", "l_max": 2048, "use_bias": True,
               "expand_proj": 4, "kernel_size": 3},
        alt_mixer={"_target_": "based.models.mixers.linear_attention.LinearAttention", "l_max": 2048,
                   "feature_map": {"_target_": "based.models.mixers.linear_attention.TaylorExp", "input_dim": 16},
                   "feature_dim": 16, "num_heads": 16},
        alt_mixer_layers=[1, 6, 11, 16, 21],
        alt_mixer_2={"_target_": "based.models.mixers.slide_attention.SlidingAttention", "window_size": 128,
                     "num_heads": 16, "causal": True},
        alt_mixer_2_layers=[2, 7, 12, 17, 22],
    )
    cfg.update(overrides)
    return StackConfig(**cfg)


def based_360m_released_config(**overrides) -> StackConfig:
    """The model section of train/configs/experiment/reference/based-360m.yaml:49-115 as written:
    window_size 256 (128 keys to the left), rotary_emb_fraction 1, parallel_implementation
    "fla_parallel" on the linear-attention layers, everything else as `based_360m_config`."""
    cfg = vars(based_360m_config())
    cfg = {k: (dict(v) if isinstance(v, dict) else v) for k, v in cfg.items()}
    cfg["alt_mixer"]["parallel_implementation"] = "fla_parallel"
    cfg["alt_mixer_2"]["window_size"] = 256
    cfg.update(rotary_emb_fraction=1, n_positions=2048, max_position_embeddings=0)
    cfg.update(overrides)
    return StackConfig(**cfg)


def create_mixer_cls(config, layer_idx=None, device=None, dtype=None):
    """Layer -> mixer routing of gpt.py:64-96."""
    if config.layer_specs is not None:
        return partial(_instantiate, config.layer_specs[layer_idx]["mixer"], device=device, dtype=dtype, layer_idx=layer_idx)
    value = config.mixer
    if config.alt_mixer_2_layers is not None and layer_idx in config.alt_mixer_2_layers:
        value = config.alt_mixer_2
    elif config.alt_mixer_layers is not None and layer_idx in config.alt_mixer_layers:
        value = config.alt_mixer
    if value is None:
        raise NotImplementedError("plain multi-head attention layers are outside this build")
    value = dict(value)
    if "slide" in value["_target_"]:
        head_dim = config.hidden_size // config.num_attention_heads
        value.update({
            "num_heads": config.num_attention_heads,
            "qkv_proj_bias": config.qkv_proj_bias,
            "out_proj_bias": config.out_proj_bias,
            "softmax_scale": head_dim ** (-0.5) if config.scale_attn_weights else 1.0,
            "causal": True,
            "rotary_emb_dim": int(config.rotary_emb_fraction * head_dim),
            "rotary_emb_base": config.rotary_emb_base,
            "rotary_emb_interleaved": config.rotary_emb_interleaved,
        })
    return partial(_instantiate, value, device=device, dtype=dtype, layer_idx=layer_idx)


def _norm_kernel_takes(x, residual, weight) -> bool:
    """Whether `ops.add_rms_norm` accepts these device tensors: rows of a multiple of 8 up to 4096
    elements, bf16 or fp32 activations with a weight of the same dtype, a residual
    stream in bf16 or fp32 (fp32 for fp32 activations)."""
    D = x.shape[-1]
    if not (x.is_cuda and weight.is_cuda):
        raise ValueError("based_amd runs on HIP device tensors only (no CPU path)")
    if not (x.dtype in (torch.bfloat16, torch.float32) and weight.dtype == x.dtype
            and D % 8 == 0 and D <= ops.ADD_RMS_NORM_MAX_DIM and weight.is_contiguous()):
        return False
    if residual is None:
        return True
    return (residual.shape == x.shape and residual.dtype in (torch.bfloat16, torch.float32)
            and not (x.dtype == torch.float32 and residual.dtype != torch.float32))


class RMSNorm(nn.Module):
    """x * rsqrt(mean(x^2) + eps) * weight (based/ops/triton/layer_norm.py:117-118), no bias."""

    def __init__(self, hidden_size, eps=1e-5, device=None, dtype=None):
        super().__init__()
        self.eps = eps
        self.weight = nn.Parameter(torch.ones(hidden_size, device=device, dtype=dtype))

    def forward(self, x):
        if _norm_kernel_takes(x, None, self.weight):
            return ops.add_rms_norm(x, None, self.weight, self.eps, want_residual=False)[0]
        # shapes, dtypes or devices the kernel is not built for: the closed form as the reference states it
        rstd = 1 / torch.sqrt(x.square().mean(dim=-1, keepdim=True) + self.eps)
        return (x * rstd * self.weight).to(x.dtype)


class StreamNorm(nn.Module):
    """Layer norm without a bias ("layer") or RMS norm ("rms") of the fp32 residual sum
    residual + mult * x, in one launch with that sum (`ops.add_norm`)."""

    KINDS = {"layer": ops.NORM_LAYER, "rms": ops.NORM_RMS}

    def __init__(self, hidden_size, eps=1e-5, kind="layer", mult=1.0, device=None, dtype=None):
        super().__init__()
        self.eps, self.kind, self.mult = eps, self.KINDS[kind], mult
        self.weight = nn.Parameter(torch.ones(hidden_size, device=device, dtype=dtype))

    def forward(self, x):
        return ops.add_norm(x, None, self.weight, self.eps, self.kind, want_residual=False)[0]


def norm_prologue(norm, residual_in, residual_out=None):
    """Arguments of `ops.decode_linear` that put residual add + `norm` in front of a projection."""
    common = dict(residual_in=residual_in, residual_out=residual_out, norm_weight=norm.weight, eps=norm.eps)
    if isinstance(norm, StreamNorm):
        return dict(prologue=ops.PROLOGUE_STREAM, mult=norm.mult, norm_kind=norm.kind, **common)
    return dict(prologue=ops.PROLOGUE_ADD_RMS_NORM, **common)


def norm_fuses(norm) -> bool:
    return isinstance(norm, (RMSNorm, StreamNorm)) and norm.weight.dtype == torch.bfloat16


def add_norm(norm, hidden_states, residual, residual_in_fp32: bool, want_residual: bool = True, addends=None):
    """residual + hidden, the norm of the sum, and the sum itself for the next block
    (block.py:134-139; gpt.py:676-694 for the closing norm).  RMSNorm on tensors the kernel takes
    is one launch; nn.LayerNorm (`rms_norm: False`, the reference's default) and everything the
    kernel refuses run the reference's own torch statement.  addends (`ops.Addends`): what else the sum of a
    StreamNorm receives."""
    if isinstance(norm, StreamNorm):
        return ops.add_norm(hidden_states, residual, norm.weight, norm.eps, norm.kind, norm.mult, want_residual, addends=addends)
    if addends is not None:
        raise NotImplementedError("only a StreamNorm takes addends")
    if isinstance(norm, RMSNorm) and _norm_kernel_takes(hidden_states, residual, norm.weight):
        if residual is None:
            return ops.add_rms_norm(hidden_states, None, norm.weight, norm.eps, residual_in_fp32, want_residual)
        return ops.add_rms_norm(hidden_states, residual, norm.weight, norm.eps,
                                residual.dtype == torch.float32, want_residual)
    residual = (hidden_states + residual) if residual is not None else hidden_states
    hidden_states = norm(residual.to(dtype=norm.weight.dtype))
    if not want_residual:
        return hidden_states, None
    if residual_in_fp32:
        residual = residual.to(torch.float32)
    return hidden_states, residual


_GATE_ACTIVATIONS = {"glu": torch.sigmoid, "swiglu": F.silu, "geglu": F.gelu}


class GatedMlp(nn.Module):
    """Gated MLP of based/models/mlp.py:99-157.  Layout 'base': fc2(y * act(gate)) with
    y, gate = fc1(x).chunk(2).  Layout 'alt' (the NeoX-style MLP of the reference's test
    configuration): fc2(act(fc1(x)) * fc3(x)) with a hidden size derived from ff_mult.
    activation: "swiglu" (silu; the released models), "geglu" (gelu) or "glu" (sigmoid),
    chosen as in gpt.py:238-243.  The released combination (base + swiglu) gates in one HIP
    kernel; the others are two element-wise torch operations."""

    def __init__(self, in_features, hidden_features=None, activation="swiglu", bias1=False, bias2=False,
                 multiple_of=256, mlp_type="base", ff_mult=2, device=None, dtype=None):
        super().__init__()
        if activation not in _GATE_ACTIVATIONS:
            raise NotImplementedError(f"activation_function {activation!r}: only gated MLPs (glu / swiglu / geglu)")
        fk = {"device": device, "dtype": dtype}
        self.activation = activation
        self.mlp_type = mlp_type
        if mlp_type == "base":
            hidden_features = hidden_features if hidden_features is not None else int(8 * in_features / 3)
            hidden_features = (hidden_features + multiple_of - 1) // multiple_of * multiple_of
            self.fc1 = nn.Linear(in_features, 2 * hidden_features, bias=bias1, **fk)
        else:
            hidden_features = int(2 * in_features * ff_mult / 3)
            hidden_features = (hidden_features + multiple_of - 1) // multiple_of * multiple_of
            self.fc1 = nn.Linear(in_features, hidden_features, bias=bias1, **fk)
            self.fc3 = nn.Linear(in_features, hidden_features, bias=bias1, **fk)
        self.fc2 = nn.Linear(hidden_features, in_features, bias=bias2, **fk)

    def forward(self, x):
        if self.mlp_type != "base":
            return self.fc2(_GATE_ACTIVATIONS[self.activation](self.fc1(x)) * self.fc3(x))
        if self.activation == "swiglu":
            return self.fc2(ops.swiglu(self.fc1(x)))
        y, gate = self.fc1(x).chunk(2, dim=-1)
        return self.fc2(y * _GATE_ACTIVATIONS[self.activation](gate))


class ExpertMlp(nn.Module):
    """Mixture of gated feed-forwards with sigmoid routing (`ops.experts`): of `experts` of them a token takes the `top` with the largest
    scores, each of which multiplies its expert's input."""

    def __init__(self, in_features, hidden_features, experts, top, device=None, dtype=None):
        super().__init__()
        fk = {"device": device, "dtype": dtype}
        if not 1 <= top <= experts:
            raise ValueError(f"{top} of {experts} experts")
        # hidden sizes are rounded up to 16-byte pieces; the extra ones carry zero weights
        hidden = round_up(hidden_features)
        self.top = top
        self.router = nn.Parameter(torch.empty(experts, in_features, **fk).normal_(std=in_features ** -0.5))
        self.w1 = nn.Parameter(torch.empty(experts, 2 * hidden, in_features, **fk).normal_(std=0.02))
        self.w2 = nn.Parameter(torch.empty(experts, in_features, hidden, **fk).normal_(std=0.02))

    def forward(self, x, norm=None):
        return ops.experts(x, self.router, self.w1, self.w2, self.top, norm)


class TokenSide(nn.Module):
    """A layer's own token input, added to the residual stream x behind the feed-forward:
    norm(proj(gelu_tanh(gate x) * e)), e the layer's columns of a table by token.  The norm is taken where the next
    layer's sum is formed (`out_addends`)."""

    def __init__(self, d_model, dim, layer_idx, eps, device=None, dtype=None):
        super().__init__()
        fk = {"device": device, "dtype": dtype}
        self.dim, self.first = dim, layer_idx * dim
        self.gate = nn.Linear(d_model, dim, bias=False, **fk)
        self.proj = nn.Linear(dim, d_model, bias=False, **fk)
        self.norm = StreamNorm(d_model, eps=eps, kind="rms", **fk)

    def table(self, side_table):
        return side_table[:, self.first:self.first + self.dim]

    def out_addends(self):
        return ops.Addends(post_weight=self.norm.weight, post_eps=self.norm.eps)

    def forward(self, hidden_states, residual, mult, ids, side_table):
        """(what proj gives, the residual stream with hidden_states in it)."""
        x, residual = ops.add_norm(hidden_states, residual, None, 0.0, ops.NORM_NONE, mult)
        g = self.gate(x)
        g = ops.gelu_mul(g.reshape(-1, self.dim), self.table(side_table), ids.reshape(-1)).view(g.shape)
        return self.proj(g), residual


class Block(nn.Module):
    """Prenorm block: add -> norm1 -> mixer -> add -> norm2 -> mlp, returning (hidden, residual)
    (block.py:134-163, dropout-free).  mlp_cls None: the mixer alone.  input_conv_cls: a causal
    convolution between norm1 and the mixer whose output is added to its input.  side_cls: a token input
    behind the feed-forward; what the next sum then does with `hidden` says `out_addends`."""

    def __init__(self, dim, mixer_cls, mlp_cls, norm_cls, residual_in_fp32=True, layer_idx=None, input_conv_cls=None, side_cls=None):
        super().__init__()
        self.residual_in_fp32 = residual_in_fp32
        self.layer_idx = layer_idx
        self.mixer = mixer_cls(dim)
        self.norm1 = norm_cls(dim)
        self.input_conv = None if input_conv_cls is None else input_conv_cls(dim, layer_idx=layer_idx)
        self.mlp = None if mlp_cls is None else mlp_cls(dim)
        self.norm2 = None if mlp_cls is None else norm_cls(dim)
        self.side = None if side_cls is None else side_cls(dim, layer_idx=layer_idx)

    def out_addends(self):
        """How the sum behind this block takes its hidden states (None: as they are)."""
        return None if self.side is None else self.side.out_addends()

    def allocate_inference_cache(self, batch_size, max_seqlen, dtype=None, **kwargs):
        cache = self.mixer.allocate_inference_cache(batch_size, max_seqlen, dtype=dtype, **kwargs)
        if self.input_conv is not None:
            cache[self.input_conv.name] = self.input_conv.allocate_ring(batch_size)
        return cache

    def _add_norm(self, norm, hidden_states, residual, addends=None):
        """residual + hidden, the norm of the sum, and the sum kept for the next block
        (block.py:134-139)."""
        return add_norm(norm, hidden_states, residual, self.residual_in_fp32, addends=addends)

    def supports_decode_step(self) -> bool:
        mlp = self.mlp
        side = self.side
        if side is not None and not ops.token_side_step_ok(side.gate.weight, side.proj.weight):
            return False
        return (getattr(self.mixer, "supports_decode_step", lambda: False)()
                and (mlp is None or (isinstance(mlp, ExpertMlp) and isinstance(self.norm2, StreamNorm) and norm_fuses(self.norm2)) or (
                                     isinstance(mlp, GatedMlp) and mlp.mlp_type == "base" and mlp.activation == "swiglu"
                                     and ops.decode_linear_weight_ok(mlp.fc1.weight)
                                     and ops.decode_linear_weight_ok(mlp.fc2.weight) and norm_fuses(self.norm2)))
                and norm_fuses(self.norm1) and self.residual_in_fp32)

    def decode_step(self, hidden_states, residual, spare, inference_params, row_index=None, addends=None, ids=None, side_table=None):
        """The block for one token per sequence in four to seven launches: both norms run inside the
        projection that consumes them (`ops.decode_linear`), the SwiGLU gate in the tail of fc1.
        hidden_states (b, dim) bf16 (or the embedding table with `row_index`), residual fp32
        (b, dim) or None; `spare` is a second fp32 (b, dim) buffer: the two take turns as the
        input and the output of the residual stream.  addends: what else the first sum receives; ids and side_table:
        tokens and table of the token input.  Returns (hidden, residual, spare)."""
        if residual is None:
            residual, (mid, last) = None, spare
        else:
            mid, last = spare, residual
        norm = norm_prologue(self.norm1, residual, mid)
        if row_index is not None:
            norm["row_index"] = row_index
        if addends is not None:
            norm["addends"] = addends
        if self.input_conv is not None:
            rows = mid.shape[0]
            pos, _ = portion_start(inference_params, rows, 1)
            norm["input_conv"] = (self.input_conv.weight, self.input_conv.ring(inference_params, rows), pos)
        hidden_states = self.mixer.decode_step(hidden_states, inference_params, **norm)
        if isinstance(self.mlp, ExpertMlp):
            n = self.norm2
            hidden_states = self.mlp(hidden_states, norm=(mid, last, n.weight, n.eps, n.kind, n.mult))
            mid, last = last, mid
        elif self.mlp is not None:
            norm = norm_prologue(self.norm2, mid, last)
            fc1, fc2 = self.mlp.fc1, self.mlp.fc2
            if fc1.weight.shape[1] <= 2048:
                # the gate in the tail of fc1
                gated = ops.decode_linear(hidden_states, fc1.weight, fc1.bias, epilogue=ops.EPILOGUE_SWIGLU, **norm)
                hidden_states = ops.decode_linear(gated, fc2.weight, fc2.bias)
            else:
                # wider models: the gate in front of fc2
                gate_in = ops.decode_linear(hidden_states, fc1.weight, fc1.bias, **norm)
                hidden_states = ops.decode_linear(gate_in, fc2.weight, fc2.bias, prologue=ops.PROLOGUE_SWIGLU)
            mid, last = last, mid
        if self.side is not None:
            side = self.side
            hidden_states = ops.token_side_step(hidden_states, mid, last, side.gate.weight, side.proj.weight, side.table(side_table), ids,
                                                self.norm1.mult)
            mid, last = last, mid
        return hidden_states, mid, last

    def forward(self, hidden_states, residual=None, mixer_kwargs=None, position_ids=None, decay=None, addends=None, ids=None,
                side_table=None):
        hidden_states, residual = self._add_norm(self.norm1, hidden_states, residual, addends)
        mixer_kwargs = mixer_kwargs or {}
        if self.input_conv is not None:
            hidden_states = self.input_conv(hidden_states, mixer_kwargs.get("inference_params"))
        if position_ids is not None or decay is not None:
            hidden_states = self.mixer(hidden_states, position_ids=position_ids, decay=decay, **mixer_kwargs)
        else:
            hidden_states = self.mixer(hidden_states, **mixer_kwargs)
        if self.mlp is not None:
            hidden_states, residual = self._add_norm(self.norm2, hidden_states, residual)
            hidden_states = self.mlp(hidden_states)
        if self.side is not None:
            hidden_states, residual = self.side(hidden_states, residual, self.norm1.mult, ids, side_table)
        return hidden_states, residual


def _init_weights(module, n_layer, initializer_range=0.02):
    if isinstance(module, nn.Linear):
        nn.init.normal_(module.weight, std=initializer_range)
        if module.bias is not None:
            nn.init.zeros_(module.bias)
    elif isinstance(module, nn.Embedding):
        nn.init.normal_(module.weight, std=initializer_range)
    for name, p in module.named_parameters():
        if name in ["out_proj.weight", "fc2.weight"]:
            nn.init.normal_(p, mean=0.0, std=initializer_range / math.sqrt(2 * n_layer))


class LayerRun(NamedTuple):
    """One run of a layer: which, in which pass of the loop, and whether the pass starts with it."""

    layer: int
    layer_pass: int
    starts_pass: bool


def layer_runs(n_layer: int, loop: Optional[dict]):
    """The layers in the order they run; those of the loop once per pass."""
    start, stop, times = (loop["start"], loop["stop"], loop["times"]) if loop else (0, 0, 1)
    if not (0 <= start <= stop <= n_layer and times >= 1) or (loop and start == stop):
        raise ValueError(f"loop {loop} over {n_layer} layers")
    body = [LayerRun(i, t, i == start) for t in range(times) for i in range(start, stop)]
    return [LayerRun(i, 0, False) for i in range(start)] + body + [LayerRun(i, 0, False) for i in range(stop, n_layer)]


class GPTModel(nn.Module):
    def __init__(self, config: StackConfig, device=None, dtype=None):
        super().__init__()
        fk = {"device": device, "dtype": dtype}
        self.config = config
        self.residual_in_fp32 = config.residual_in_fp32
        vocab = math.ceil(config.vocab_size / config.pad_vocab_size_multiple) * config.pad_vocab_size_multiple
        self.embeddings = nn.Module()
        self.embeddings.word_embeddings = nn.Embedding(vocab, config.hidden_size, **fk)
        if config.max_position_embeddings > 0:
            self.embeddings.position_embeddings = nn.Embedding(config.max_position_embeddings, config.hidden_size, **fk)
        # rms_norm absent from a reference config means nn.LayerNorm (gpt.py:352,537)
        if config.stream_norm is not None:
            norm_cls = partial(StreamNorm, eps=config.layer_norm_epsilon, kind=config.stream_norm, mult=config.residual_mult, **fk)
        else:
            if config.residual_mult != 1.0:
                raise NotImplementedError("residual_mult needs stream_norm")
            norm_cls = partial(RMSNorm if config.rms_norm else nn.LayerNorm, eps=config.layer_norm_epsilon, **fk)
        input_conv_cls = None
        if config.input_conv_taps > 0:
            input_conv_cls = partial(StreamConv, taps=config.input_conv_taps, add_input=True, name="input_conv", **fk)
        mlp_cls = partial(GatedMlp, hidden_features=config.n_inner, activation=config.activation_function,
                          bias1=config.mlp_fc1_bias, bias2=config.mlp_fc2_bias, mlp_type=config.mlp_type,
                          ff_mult=config.ff_mult, **fk)

        def layer_mlp(i):
            if config.layer_specs is None:
                return mlp_cls
            spec = config.layer_specs[i]["mlp"]
            # hidden sizes are rounded up to the 16-byte pieces of the gate kernel; the extra ones carry zero weights
            if spec is not None and "experts" in spec:
                return partial(ExpertMlp, hidden_features=spec["hidden"], experts=spec["experts"], top=spec["top"], **fk)
            return None if spec is None else partial(mlp_cls, hidden_features=spec["hidden"], multiple_of=8)

        self.runs = layer_runs(config.num_hidden_layers, config.loop)
        side_cls = None
        if config.token_side_dim > 0:
            side_cls = partial(TokenSide, dim=config.token_side_dim, eps=config.layer_norm_epsilon, **fk)
            self.embeddings.side_embeddings = nn.Embedding(vocab, config.num_hidden_layers * config.token_side_dim, **fk)
        if (config.loop or side_cls) and config.stream_norm is None:
            raise NotImplementedError("loop and token_side_dim need stream_norm")
        self.loop_step = nn.Parameter(torch.zeros(config.loop["times"], config.hidden_size, **fk)) if config.loop else None
        self.layers = nn.ModuleList([
            Block(config.hidden_size, create_mixer_cls(config, layer_idx=i, **fk), layer_mlp(i), norm_cls,
                  residual_in_fp32=config.residual_in_fp32, layer_idx=i, input_conv_cls=input_conv_cls, side_cls=side_cls)
            for i in range(config.num_hidden_layers)
        ])
        self.ln_f = norm_cls(config.hidden_size)
        self.apply(partial(_init_weights, n_layer=config.num_hidden_layers,
                           initializer_range=config.initializer_range))

    def allocate_inference_cache(self, batch_size, max_seqlen, dtype=None, **kwargs):
        return {i if t == 0 else (i, t): self.layers[i].allocate_inference_cache(batch_size, max_seqlen, dtype=dtype, **kwargs)
                for i, t, _ in self.runs}

    def _side_table(self):
        return self.embeddings.side_embeddings.weight if self.config.token_side_dim > 0 else None

    def _run_addends(self, run: LayerRun, addends, ids):
        """What the first sum of a run receives: `addends` from the block before, and what starts a pass of the loop."""
        if self.loop_step is None or not run.starts_pass:
            return addends
        addends = (addends or ops.Addends())._replace(vec=self.loop_step[run.layer_pass])
        if run.layer_pass > 0:
            addends = addends._replace(table=self.embeddings.word_embeddings.weight, index=ids)
        return addends

    # Single-token steps of a bf16 model run through `decode_layers`: every projection is an
    # `ops.decode_linear` launch with the element-wise work in front of it folded in.  Set to False
    # to send them through the general path (torch GEMMs + stand-alone norm and gate kernels).
    fused_decode = True

    def decode_layers_ok(self, input_ids, inference_params) -> bool:
        if not (self.fused_decode and inference_params is not None and inference_params.seqlen_offset > 0
                and input_ids.shape[1] == 1 and input_ids.shape[0] <= ops.DECODE_LINEAR_MAX_ROWS
                and input_ids.is_cuda and not torch.is_grad_enabled()
                and self.config.max_position_embeddings == 0):
            return False
        # the answer depends on dtypes and devices of the parameters only: worked out once per
        # (dtype, device) of the embedding table
        table = self.embeddings.word_embeddings.weight
        cached = self.__dict__.get("_decode_layers_supported")
        if cached is None or cached[0] != (table.dtype, table.device):
            ok = (ops.decode_linear_weight_ok(table) and norm_fuses(self.ln_f)
                  and all(layer.supports_decode_step() for layer in self.layers))
            cached = ((table.dtype, table.device), ok)
            self.__dict__["_decode_layers_supported"] = cached
        return cached[1]

    def decode_layers(self, input_ids, inference_params):
        """All blocks for one token per sequence.  Returns (hidden (b, dim) bf16, residual (b, dim)
        fp32): the inputs of the closing add + norm, which the caller folds into what follows."""
        b = input_ids.shape[0]
        table = self.embeddings.word_embeddings.weight
        key = (b, table.device)
        buffers = self.__dict__.setdefault("_decode_residuals", {}).get(key)
        if buffers is None:
            buffers = tuple(torch.empty(b, table.shape[1], dtype=torch.float32, device=table.device) for _ in range(2))
            self._decode_residuals[key] = buffers
        ids = input_ids.reshape(-1).contiguous()  # a column of a wider id tensor is a strided view
        hidden_states, residual, spare, addends = table, None, buffers, None
        more = {"ids": ids, "side_table": self._side_table()} if self.config.token_side_dim > 0 else {}
        for n, run in enumerate(self.runs):
            layer = self.layers[run.layer]
            inference_params.layer_pass = run.layer_pass
            hidden_states, residual, spare = layer.decode_step(hidden_states, residual, spare, inference_params,
                                                               row_index=ids if n == 0 else None,
                                                               addends=self._run_addends(run, addends, ids), **more)
            addends = layer.out_addends()
        inference_params.layer_pass = 0
        return hidden_states, residual

    def closing_addends(self):
        """What the closing sum receives besides the last block's output."""
        return self.layers[self.runs[-1].layer].out_addends()

    def forward(self, input_ids, position_ids=None, inference_params=None, stream=None):
        if self.decode_layers_ok(input_ids, inference_params):
            hidden_states, residual = self.decode_layers(input_ids, inference_params)
            return add_norm(self.ln_f, hidden_states, residual, True, want_residual=False,
                            addends=self.closing_addends())[0].unsqueeze(1)
        hidden_states = self.embeddings.word_embeddings(input_ids)
        if self.config.max_position_embeddings > 0:
            if position_ids is None:
                position_ids = torch.arange(input_ids.shape[1], dtype=torch.long, device=input_ids.device)
            hidden_states = hidden_states + self.embeddings.position_embeddings(position_ids)
        residual = None
        mixer_kwargs = {}
        if inference_params is not None:
            mixer_kwargs["inference_params"] = inference_params
            mixer_kwargs["stream"] = stream
        addends, more = None, {}
        ids = None
        if self.loop_step is not None or self.config.token_side_dim > 0:
            ids = input_ids.reshape(-1).contiguous()
            more = {"ids": ids, "side_table": self._side_table()}
        for run in self.runs:
            layer = self.layers[run.layer]
            if inference_params is not None:
                inference_params.layer_pass = run.layer_pass
            addends = self._run_addends(run, addends, ids)
            if addends is not None:
                more["addends"] = addends
            hidden_states, residual = layer(hidden_states, residual=residual, position_ids=position_ids,
                                            mixer_kwargs=mixer_kwargs, **more)
            more.pop("addends", None)
            addends = layer.out_addends()
        if inference_params is not None:
            inference_params.layer_pass = 0
        return add_norm(self.ln_f, hidden_states, residual, self.residual_in_fp32, want_residual=False, addends=addends)[0]


class GPTLMHeadModel(nn.Module, GenerationMixin):
    def __init__(self, config: StackConfig, device=None, dtype=None):
        super().__init__()
        self.config = config
        self.transformer = GPTModel(config, device=device, dtype=dtype)
        vocab = self.transformer.embeddings.word_embeddings.num_embeddings
        self.lm_head = nn.Linear(config.n_embd, vocab, bias=False, device=device, dtype=dtype)
        self.apply(partial(_init_weights, n_layer=config.num_hidden_layers,
                           initializer_range=config.initializer_range))
        if config.tie_word_embeddings:
            self.lm_head.weight = self.transformer.embeddings.word_embeddings.weight

    def allocate_inference_cache(self, batch_size, max_seqlen, dtype=None, **kwargs):
        return self.transformer.allocate_inference_cache(batch_size, max_seqlen, dtype=dtype, **kwargs)

    @classmethod
    def from_pretrained_local(cls, directory, device=None, dtype=None, strict=True):
        """Builds the model from a LOCAL directory laid out like the released checkpoints:
        `config.json` (the GPT2Config dictionary) and `pytorch_model.bin` or `model.safetensors`.
        Counterpart of from_pretrained_hf (gpt.py:446-459) without the hub: same key clean-up
        (leading "model." stripped, training-metric entries dropped).  The weights file is read
        with a loader that executes nothing from it.  A config.json that names an `architecture` of
        `based_amd.architectures` has its own keys and tensor names, which that module translates."""
        import json
        import os
        import re

        from . import architectures

        with open(os.path.join(directory, "config.json")) as f:
            raw = json.load(f)
        design = architectures.find(raw)
        st_path = os.path.join(directory, "model.safetensors")
        if os.path.exists(st_path):
            from safetensors.torch import load_file

            state = load_file(st_path, device="cpu")
        else:
            state = torch.load(os.path.join(directory, "pytorch_model.bin"), map_location="cpu", weights_only=True)
        if design:
            config = StackConfig(**design.stack_config(raw, {name: tuple(t.shape) for name, t in state.items()}))
        else:
            config = StackConfig.from_reference_dict(raw)
        model = cls(config, device=device, dtype=dtype)
        if design:
            model.load_state_dict(design.convert_state(raw, state), strict=strict)
            return model
        state = {re.sub(r"^model\.", "", k): v for k, v in state.items() if "metrics" not in k}
        if config.tie_word_embeddings and "lm_head.weight" not in state:
            state["lm_head.weight"] = state["transformer.embeddings.word_embeddings.weight"]
        model.load_state_dict(state, strict=strict)
        return model

    def load_state_dict(self, state_dict, strict=True, **kwargs):
        """Also accepts checkpoints written with the older order of the layers in a block (norm
        after the mixer / MLP, a leading `transformer.ln_0`): their norm parameters are moved to
        the current prenorm slots exactly as the reference does (gpt.py:829-853); norms without
        a bias (RMSNorm) simply have no bias entries to move."""
        if "transformer.ln_0.weight" in state_dict:
            state_dict = dict(state_dict)
            n_layers = len(self.transformer.layers)

            def move(src, dst):
                for suffix in ("weight", "bias"):
                    if f"{src}.{suffix}" in state_dict:
                        state_dict[f"{dst}.{suffix}"] = state_dict.pop(f"{src}.{suffix}")

            move(f"transformer.layers.{n_layers - 1}.norm2", "transformer.ln_f")
            for l in reversed(range(n_layers)):
                move(f"transformer.layers.{l}.norm1", f"transformer.layers.{l}.norm2")
                if l > 0:
                    move(f"transformer.layers.{l - 1}.norm2", f"transformer.layers.{l}.norm1")
            move("transformer.ln_0", "transformer.layers.0.norm1")
        return super().load_state_dict(state_dict, strict=strict, **kwargs)

    def forward(self, input_ids, position_ids=None, inference_params=None, num_last_tokens=0, stream=None,
                logits_at=None, **kwargs):
        """logits_at: None, or the places within the portion whose logits are wanted."""
        assert input_ids.ndim == 2, f"Expected `input_ids` to have shape [b, slen], but got shape {input_ids.shape}"
        CausalLMOutput = namedtuple("CausalLMOutput", ["logits"])
        if (self.transformer.decode_layers_ok(input_ids, inference_params)
                and ops.decode_linear_weight_ok(self.lm_head.weight)):
            # closing add + norm inside the LM head's projection
            hidden_states, residual = self.transformer.decode_layers(input_ids, inference_params)
            ln_f = self.transformer.ln_f
            norm = norm_prologue(ln_f, residual)
            if isinstance(ln_f, StreamNorm):
                norm.update(addends=self.transformer.closing_addends(), softcap=self.config.logit_softcap or 0.0)
                return CausalLMOutput(logits=ops.decode_linear(hidden_states, self.lm_head.weight, self.lm_head.bias, **norm).unsqueeze(1))
            logits = ops.decode_linear(hidden_states, self.lm_head.weight, self.lm_head.bias, **norm)
            return CausalLMOutput(logits=self._capped(logits).unsqueeze(1))
        hidden_states = self.transformer(input_ids, position_ids=position_ids, inference_params=inference_params,
                                         stream=stream)
        if num_last_tokens > 0:
            hidden_states = hidden_states[:, -num_last_tokens:]
        if logits_at is not None:
            hidden_states = hidden_states[:, logits_at]
        return CausalLMOutput(logits=self._capped(self.lm_head(hidden_states)))

    def _capped(self, logits):
        return logits if self.config.logit_softcap is None else ops.softcap_(logits, self.config.logit_softcap)
