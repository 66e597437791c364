"""Plain CPU statement of the Sozilix design: one function per mechanism, token by token where the
definition is a recurrence, no caches, no shared code with the package.

TEST INFRASTRUCTURE ONLY: the shipped package never imports this file.  Everything is evaluated in
the dtype of the tensors that are passed in (the tests pass float64).  A whole model is
`forward(cfg, w, tokens)` with `cfg` the config.json dictionary and `w` a dict name -> tensor.

Pinned by tests/test_sozilix_oracle.py: torch's library routines (layer_norm, conv1d, SDPA, gelu),
closed forms, complex-number rotations and an explicit unrolled product for the recurrences.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, weight, eps):
    centred = x - x.mean(-1, keepdim=True)
    return centred / torch.sqrt((centred * centred).mean(-1, keepdim=True) + eps) * weight


def silu(z):
    return z / (1 + torch.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + z.clamp_min(0)


def causal_conv(x, w, bias=None):
    """x (T, C), w (C, taps): y_t = sum_j w[:, j] x_{t - taps + 1 + j}, zeros before the start."""
    T, taps = x.shape[0], w.shape[1]
    y = torch.zeros_like(x)
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                y[t] = y[t] + w[:, j] * x[s]
    return y if bias is None else y + bias


def input_conv(h, w):
    return h + causal_conv(h, w)


def rotate(x, base, dims):
    """x (T, heads, dim): pairs (2i, 2i+1) of the first `dims` channels turned by p * base^(-2i/dims)."""
    y = x.clone()
    for i in range(dims // 2):
        ang = torch.arange(x.shape[0], dtype=torch.float64) * base ** (-2.0 * i / dims)
        c, s = ang.cos().to(x.dtype)[:, None], ang.sin().to(x.dtype)[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        y[:, :, 2 * i] = u * c - v * s
        y[:, :, 2 * i + 1] = v * c + u * s
    return y


def window_softmax(q, k, v, scale, window):
    """q (T, H, d), k (T, G, d), v (T, G, dv): position i attends j with 0 <= i - j < window."""
    T, H, _ = q.shape
    group = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    idx = torch.arange(T)
    dist = idx[:, None] - idx[None, :]
    seen = (dist >= 0) & (dist < window)
    for h in range(H):
        g = h // group
        s = (q[:, h] @ k[:, g].T) * scale
        s = s.masked_fill(~seen, float("-inf"))
        out[:, h] = torch.softmax(s, dim=-1) @ v[:, g]
    return out


def windowed_attention(h, w, pre, spec, eps):
    """The left half: grouped heads, partial rotation, values divided by their RMS."""
    T = h.shape[0]
    H, G, d, dv = spec["heads"], spec["kv_heads"], spec["dim"], spec["vdim"]
    q = rotate((h @ w[pre + ".q"].T).view(T, H, d), spec["rot"]["base"], spec["rot"]["dims"])
    k = rotate((h @ w[pre + ".k"].T).view(T, G, d), spec["rot"]["base"], spec["rot"]["dims"])
    v = rms((h @ w[pre + ".v"].T).view(T, G, dv), eps)
    o = window_softmax(q, k, v, spec["scale"], spec["mask"]["size"])
    return o.reshape(T, H * dv) @ w[pre + ".o"].T


def delta_rule(q, k, v, g, beta):
    """q, k (T, H, d), v (T, H, dv), g, beta (T, H): the gated delta recurrence, one token at a time."""
    T, H, d = q.shape
    o = torch.zeros_like(v)
    for h in range(H):
        S = torch.zeros(d, v.shape[2], dtype=v.dtype)
        for t in range(T):
            S = g[t, h] * S
            u = beta[t, h] * (v[t, h] - S.T @ k[t, h])
            S = S + torch.outer(k[t, h], u)
            o[t, h] = S.T @ q[t, h]
    return o


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def gated_delta(h, w, pre, spec, eps):
    """The right half: gated delta rule with short convolutions, output norm and gate."""
    T = h.shape[0]
    H, G, d, dv = spec["heads"], spec["kv_heads"], spec["dim"], spec["vdim"]
    q, k, v = (silu(causal_conv(h @ w[f"{pre}.{n}"].T, w[f"{pre}.{n}.conv"])) for n in "qkv")
    share = H // G
    q = (unit(q.view(T, G, d)) * d ** -0.5).repeat_interleave(share, dim=1)
    k = unit(k.view(T, G, d)).repeat_interleave(share, dim=1)
    beta = torch.sigmoid(h @ w[pre + ".b"].T)
    g = torch.exp(-torch.exp(w[pre + ".A_log"]) * softplus(h @ w[pre + ".a"].T + w[pre + ".dt_bias"]))
    o = delta_rule(q, k, v.view(T, H, dv), g, beta)
    o = rms(o, eps) * w[pre + ".norm"] * silu(h @ w[pre + ".g"].T).view(T, H, dv)
    return o.reshape(T, H * dv) @ w[pre + ".o"].T


def parallel_mixer(h, w, pre, spec, eps):
    return (spec["left_scale"] * windowed_attention(h, w, pre + ".left", spec["left"], eps)
            + spec["right_scale"] * gated_delta(h, w, pre + ".right", spec["right"], eps))


def gated_linear_unit(u, ra, ra_b, ri, ri_b, lam):
    """u (T, width); ra, ri (blocks, n, n) as [out, in]: the real-gated linear recurrence, (T, width)."""
    T, width = u.shape
    blocks, n = ra.shape[0], ra.shape[1]
    r, i = torch.zeros_like(u), torch.zeros_like(u)
    for b in range(blocks):
        part = slice(b * n, (b + 1) * n)
        r[:, part] = torch.sigmoid(u[:, part] @ ra[b].T + ra_b[b])
        i[:, part] = torch.sigmoid(u[:, part] @ ri[b].T + ri_b[b])
    log_a = -8 * r * softplus(lam)
    S = torch.zeros(width, dtype=u.dtype)
    out = torch.zeros_like(u)
    for t in range(T):
        S = torch.exp(log_a[t]) * S + torch.sqrt(-torch.expm1(2 * log_a[t])) * i[t] * u[t]
        out[t] = S
    return out


def rglru_mixer(h, w, pre, spec, eps):
    y = gelu_tanh(h @ w[pre + ".y"].T + w[pre + ".y.b"])
    u = causal_conv(h @ w[pre + ".x"].T + w[pre + ".x.b"], w[pre + ".conv"], w[pre + ".conv.b"])
    S = gated_linear_unit(u, w[pre + ".ra"], w[pre + ".ra.b"], w[pre + ".ri"], w[pre + ".ri.b"], w[pre + ".lam"])
    return (S * y) @ w[pre + ".o"].T


def dense_mlp(h, w, pre):
    return (silu(h @ w[pre + ".gate"].T) * (h @ w[pre + ".up"].T)) @ w[pre + ".down"].T


MIXERS = {"parallel": parallel_mixer, "rglru": rglru_mixer}


def forward(cfg, w, tokens, layers_out=None):
    """Logits (T, vocab) of one sequence; `layers_out`, a list, receives the residual stream after every layer."""
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x = w["embed"][tokens]
    for i, layer in enumerate(cfg["layers"]):
        h = input_conv(layer_norm(x, w[f"l{i}.norm1"], eps), w[f"l{i}.canon1"])
        x = x + m * MIXERS[layer["type"]](h, w, f"l{i}.mix", layer["mixer"], eps)
        if layer["mlp"] is not None:
            x = x + m * dense_mlp(layer_norm(x, w[f"l{i}.norm2"], eps), w, f"l{i}.mlp")
        if layers_out is not None:
            layers_out.append(x)
    return layer_norm(x, w["final.norm"], eps) @ w["head"].T
