"""Peponex: a decoder-only stack of three kinds of layers on an fp32 residual stream.

    x <- x + mixer(rms_norm(x));   x <- x + feed_forward(rms_norm(x))                (layers with one)
    x <- x + rms_norm(proj(gelu(gate x) * e_i(token)))                               (a token input of every layer)

"wkv" layers mix tokens and run a recurrence with a decay per channel, "lightning" layers linear attention with
constant decays, "latent_attention" layers sliding-window attention over a latent cache.  A feed-forward
is a gated MLP or a mixture of experts.  Some layers run several times in a row with the same weights; before each
pass a vector of its own is added and, from the second on, the embedding once more.  Logits are capped."""
from __future__ import annotations

import torch

from ..mixers.latent_attention import LatentAttention
from ..mixers.streaming import round_up
from ..mixers.time_mix import TimeMix
from .sozilix import _beside, _stack


def _mixer_spec(layer: dict, eps: float, rank: int) -> dict:
    m = layer["mixer"]
    if layer["type"] == "wkv":
        return {"_target_": "based_amd.mixers.time_mix.TimeMix", "heads": m["heads"], "dim": m["dim"], "rank": rank, "norm_eps": eps}
    if layer["type"] == "lightning":
        core = {"_target_": "based_amd.mixers.decay_attention.DecayAttention", "heads": m["heads"], "dim": m["dim"], "vdim": m["vdim"],
                "decay": tuple(m["decay"]), "norm_eps": eps}
    elif layer["type"] == "latent_attention":
        core = {"_target_": "based_amd.mixers.latent_attention.LatentAttention", "heads": m["heads"], "dim": m["dim"], "rot_dim": m["rot_dim"],
                "vdim": m["vdim"], "kv_rank": m["kv_rank"], "window": m["mask"]["size"], "scale": m["scale"],
                "rotary_base": m["rot"]["base"], "rotary_interleaved": False, "norm_eps": eps}
    else:
        raise NotImplementedError(f"layer type {layer['type']!r}")
    return {"_target_": "based_amd.mixers.side_by_side.SideBySide", "cores": [core]}


def _mlp_spec(layer: dict):
    mlp = layer["mlp"]
    if mlp is None:
        return None
    if mlp["kind"] == "dense":
        return {"hidden": mlp["ff"]}
    if mlp["kind"] == "moe":
        return {"hidden": mlp["expert"]["ff"], "experts": mlp["router"]["experts"], "top": mlp["router"]["top"]}
    raise NotImplementedError(f"feed-forward kind {mlp['kind']!r}")


def stack_config(raw: dict, shapes: dict) -> dict:
    """Keywords of StackConfig for a Peponex config.json; `shapes`: tensor name -> shape, for the sizes only they tell."""
    eps = raw["norm"]["eps"]
    rank = lambda i: shapes[f"l{i}.mix.w1"][0] if raw["layers"][i]["type"] == "wkv" else 0
    side = raw.get("token_side")
    return dict(
        n_embd=raw["width"], n_layer=len(raw["layers"]), vocab_size=raw["vocab"], pad_vocab_size_multiple=1, layer_norm_epsilon=eps,
        stream_norm="rms", residual_in_fp32=True, tie_word_embeddings=False, max_position_embeddings=0,
        layer_specs=[{"mixer": _mixer_spec(layer, eps, rank(i)), "mlp": _mlp_spec(layer)} for i, layer in enumerate(raw["layers"])],
        loop=raw.get("loop"), token_side_dim=side["dim"] if side else 0, logit_softcap=raw.get("logit_softcap"),
    )


def _rotated_first(q, heads: int, dim: int, rot_dim: int):
    """Rows of the query projection with a head's rotated channels in front of the others."""
    q = q.view(heads, dim + rot_dim, -1)
    return torch.cat([q[:, dim:], q[:, :dim]], dim=1).reshape(heads * (dim + rot_dim), -1)


def _pad(x, dim: int, to: int = 8):
    """Zeros behind dimension `dim` up to a multiple of `to`."""
    gap = round_up(x.shape[dim], to) - x.shape[dim]
    if not gap:
        return x
    shape = list(x.shape)
    shape[dim] = gap
    return torch.cat([x, x.new_zeros(shape)], dim=dim)


def convert_state(raw: dict, w: dict) -> dict:
    """The stack's state dict from the design's tensors: projections of the same input stacked, experts in one tensor."""
    out = {
        "transformer.embeddings.word_embeddings.weight": w["embed"],
        "transformer.ln_f.weight": w["final.norm"],
        "lm_head.weight": w["head"],
    }
    if raw.get("loop"):
        out["transformer.loop_step"] = w["loop.step"]
    if raw.get("token_side"):
        out["transformer.embeddings.side_embeddings.weight"] = w["side.embed"]
    for i, layer in enumerate(raw["layers"]):
        src, dst, m = f"l{i}", f"transformer.layers.{i}", layer["mixer"]
        mix = f"{dst}.mixer"
        t = lambda name: w[f"{src}.mix.{name}"]
        out[f"{dst}.norm1.weight"] = w[f"{src}.norm1"]
        if layer["type"] == "wkv":
            out[f"{mix}.mu"] = torch.stack([t(f"mu.{n}") for n in TimeMix.MIXES])
            out[f"{mix}.in_proj.weight"] = torch.cat([_stack([t("r"), t("k"), t("v"), t("g")], TimeMix.SEGMENT), _stack([t("w1")])])
            out[f"{mix}.w2"], out[f"{mix}.w0"], out[f"{mix}.bonus"] = t("w2"), t("w0"), t("u")
            out[f"{mix}.norm_weight"] = t("norm")
        elif layer["type"] == "lightning":
            out[f"{mix}.in_proj.weight"] = _stack([t("q"), t("k"), t("v"), t("g")])
            out[f"{mix}.cores.0.norm_weight"] = t("norm")
        else:
            out[f"{mix}.in_proj.weight"] = _stack([_rotated_first(t("q"), m["heads"], m["dim"], m["rot_dim"]), t("dkv")])
            out[f"{mix}.cores.0.norm_weight"] = t("dkv.norm")
            out[f"{mix}.cores.0.expand"] = LatentAttention.expansion(t("uk"), t("uv"), m["heads"], m["rot_dim"])
        out[f"{mix}.out_proj.weight"] = _beside([t("o")])
        mlp = layer["mlp"]
        if mlp is not None:
            out[f"{dst}.norm2.weight"] = w[f"{src}.norm2"]
            if mlp["kind"] == "dense":
                # the gate kernels take (value, gate): value * silu(gate)
                out[f"{dst}.mlp.fc1.weight"] = _stack([w[f"{src}.mlp.up"], w[f"{src}.mlp.gate"]])
                out[f"{dst}.mlp.fc2.weight"] = _beside([w[f"{src}.mlp.down"]])
            else:
                of = lambda name: torch.stack([w[f"{src}.mlp.e{e}.{name}"] for e in range(mlp["router"]["experts"])])
                out[f"{dst}.mlp.router"] = w[f"{src}.mlp.router"]
                out[f"{dst}.mlp.w1"] = torch.cat([_pad(of("up"), 1), _pad(of("gate"), 1)], dim=1)
                out[f"{dst}.mlp.w2"] = _pad(of("down"), 2)
        if raw.get("token_side"):
            out[f"{dst}.side.gate.weight"], out[f"{dst}.side.proj.weight"] = w[f"{src}.side.gate"], w[f"{src}.side.proj"]
            out[f"{dst}.side.norm.weight"] = w[f"{src}.side.norm"]
    return out
