"""Plain CPU statement of the Peponex design: one function per mechanism, token by token where the
definition is a recurrence, no caches, no shared code with the package.

TEST INFRASTRUCTURE ONLY: the shipped package never imports this file.  Everything is evaluated in
the dtype of the tensors that are passed in (the tests pass float64).  A whole model is
`forward(cfg, w, tokens)` with `cfg` the config.json dictionary and `w` a dict name -> tensor.

Pinned by tests/test_peponex_oracle.py: torch's library routines (SDPA, gelu, rms_norm, topk), complex
rotations, and explicit sums over all earlier tokens for the recurrences.
"""
from __future__ import annotations

import torch

from .sozilix_oracle import dense_mlp, gelu_tanh, rms, silu


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def token_mix(h, mu):
    """h (T, D): h + (h of the token before - h) * mu, zeros before the first."""
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * mu


def channel_decay(x, w1, w2, w0):
    """exp(-exp(w2 tanh(w1 x) + w0)), (T, channels)."""
    return torch.exp(-torch.exp(torch.tanh(x @ w1.T) @ w2.T + w0))


def bonus_recurrence(r, k, v, w, u):
    """r, k, w (T, H, d), v (T, H, dv), u (H, d): o_t = (S + diag(u) k_t v_t^T)^T r_t, then S <- diag(w_t) S + k_t v_t^T."""
    T, H, _ = r.shape
    o = torch.zeros_like(v)
    for h in range(H):
        S = torch.zeros(r.shape[2], v.shape[2], dtype=v.dtype)
        for t in range(T):
            now = torch.outer(k[t, h], v[t, h])
            o[t, h] = (S + u[h][:, None] * now).T @ r[t, h]
            S = w[t, h][:, None] * S + now
    return o


def decay_recurrence(q, k, v, decay):
    """q, k (T, H, d), v (T, H, dv), decay (H): S <- decay S + k_t v_t^T, o_t = S^T q_t."""
    T, H, _ = q.shape
    o = torch.zeros_like(v)
    for h in range(H):
        S = torch.zeros(q.shape[2], v.shape[2], dtype=v.dtype)
        for t in range(T):
            S = decay[h] * S + torch.outer(k[t, h], v[t, h])
            o[t, h] = S.T @ q[t, h]
    return o


def wkv_mixer(h, w, pre, spec, eps):
    T, H, d = h.shape[0], spec["heads"], spec["dim"]
    mixed = {n: token_mix(h, w[f"{pre}.mu.{n}"]) for n in "rkvgw"}
    r, k, v = ((mixed[n] @ w[f"{pre}.{n}"].T).view(T, H, d) for n in "rkv")
    gate = silu(mixed["g"] @ w[f"{pre}.g"].T)
    decay = channel_decay(mixed["w"], w[f"{pre}.w1"], w[f"{pre}.w2"], w[f"{pre}.w0"]).view(T, H, d)
    o = rms(bonus_recurrence(r, k, v, decay, w[f"{pre}.u"]), eps).reshape(T, H * d)
    return (o * w[f"{pre}.norm"] * gate) @ w[f"{pre}.o"].T


def lightning_mixer(h, w, pre, spec, eps):
    T, H = h.shape[0], spec["heads"]
    q, k = (silu(h @ w[f"{pre}.{n}"].T).view(T, H, spec["dim"]) for n in "qk")
    v = silu(h @ w[f"{pre}.v"].T).view(T, H, spec["vdim"])
    o = decay_recurrence(q, k, v, torch.tensor(spec["decay"], dtype=h.dtype)).reshape(T, -1)
    return (rms(o, eps) * w[f"{pre}.norm"] * sigmoid(h @ w[f"{pre}.g"].T)) @ w[f"{pre}.o"].T


def rotate_halves(x, base, dims):
    """x (T, ..., dim): channels i and i + dims/2 of the first `dims` turned by p * base^(-2i/dims)."""
    y = x.clone()
    p = torch.arange(x.shape[0], dtype=torch.float64).view(-1, *[1] * (x.dim() - 2))
    for i in range(dims // 2):
        j = i + dims // 2
        ang = p * float(base) ** (-2.0 * i / dims)
        c, s = ang.cos().to(x.dtype), ang.sin().to(x.dtype)
        y[..., i] = x[..., i] * c - x[..., j] * s
        y[..., j] = x[..., j] * c + x[..., i] * s
    return y


def window_weights(scores, window):
    """scores (T, T): softmax of row i over j with 0 <= i - j < window."""
    idx = torch.arange(scores.shape[0])
    dist = idx[:, None] - idx[None, :]
    return torch.softmax(scores.masked_fill((dist < 0) | (dist >= window), float("-inf")), dim=-1)


def latent_mixer(h, w, pre, spec, eps):
    T, H, d, r, dv, R = h.shape[0], spec["heads"], spec["dim"], spec["rot_dim"], spec["vdim"], spec["kv_rank"]
    q = (h @ w[f"{pre}.q"].T).view(T, H, d + r)
    down = h @ w[f"{pre}.dkv"].T
    c = rms(down[:, :R], eps) * w[f"{pre}.dkv.norm"]
    q_rot, k_rot = rotate_halves(q[..., d:], spec["rot"]["base"], r), rotate_halves(down[:, R:], spec["rot"]["base"], r)
    k = (c @ w[f"{pre}.uk"].T).view(T, H, d)
    v = (c @ w[f"{pre}.uv"].T).view(T, H, dv)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for i in range(H):
        scores = (q[:, i, :d] @ k[:, i].T + q_rot[:, i] @ k_rot.T) * spec["scale"]
        out[:, i] = window_weights(scores, spec["mask"]["size"]) @ v[:, i]
    return out.reshape(T, H * dv) @ w[f"{pre}.o"].T


def route(h, router, top):
    """The `top` largest sigmoid scores of every token: (indices, scores), (T, top)."""
    s = sigmoid(h @ router.T)
    values, ids = s.sort(dim=-1, descending=True, stable=True)
    return ids[:, :top], values[:, :top]


def expert_mlp(h, w, pre, spec):
    """Sum over a token's experts of expert(score * h)."""
    ids, scores = route(h, w[f"{pre}.router"], spec["router"]["top"])
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(ids[t].tolist(), scores[t]):
            y[t] += dense_mlp((s * h[t])[None], w, f"{pre}.e{e}")[0]
    return y


def token_side(x, w, pre, e, eps):
    """What the per-layer token input e (T, dim) adds to x."""
    y = (gelu_tanh(x @ w[f"{pre}.gate"].T) * e) @ w[f"{pre}.proj"].T
    return rms(y, eps) * w[f"{pre}.norm"]


MIXERS = {"wkv": wkv_mixer, "lightning": lightning_mixer, "latent_attention": latent_mixer}


def layer_runs(cfg):
    """(layer, pass) in the order they run; pass is None outside the loop."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if loop is None:
        return [(i, None) for i in range(n)]
    body = [(i, t) for t in range(loop["times"]) for i in range(loop["start"], loop["stop"])]
    return [(i, None) for i in range(loop["start"])] + body + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg, w, tokens, layers_out=None):
    """Logits (T, vocab) of one sequence; `layers_out`, a list, receives the residual stream after every layer run."""
    eps = cfg["norm"]["eps"]
    x = first = w["embed"][tokens]
    dim = cfg["token_side"]["dim"] if cfg.get("token_side") else 0
    for i, t in layer_runs(cfg):
        if t is not None and i == cfg["loop"]["start"]:
            if t > 0:
                x = x + first
            x = x + w["loop.step"][t]
        layer = cfg["layers"][i]
        x = x + MIXERS[layer["type"]](rms(x, eps) * w[f"l{i}.norm1"], w, f"l{i}.mix", layer["mixer"], eps)
        mlp = layer["mlp"]
        if mlp is not None:
            h = rms(x, eps) * w[f"l{i}.norm2"]
            x = x + (dense_mlp(h, w, f"l{i}.mlp") if mlp["kind"] == "dense" else expert_mlp(h, w, f"l{i}.mlp", mlp))
        if dim:
            x = x + token_side(x, w, f"l{i}.side", w["side.embed"][tokens][:, i * dim:(i + 1) * dim], eps)
        if layers_out is not None:
            layers_out.append(x)
    logits = (rms(x, eps) * w["final.norm"]) @ w["head"].T
    cap = cfg.get("logit_softcap")
    return logits if cap is None else cap * torch.tanh(logits / cap)
