"""The plain statement of the Sozilix mechanisms (oracle/sozilix_oracle.py) against library routines, closed
forms and unrolled products, and the translation of its config and tensors into the stack (CPU)."""
import json

import pytest
import torch
import torch.nn.functional as F

import sozilix_cases as cases
from oracle import sozilix_oracle as O

g = torch.Generator().manual_seed(3)
rnd = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
close = lambda a, b, tol=1e-10: torch.testing.assert_close(a, b, rtol=tol, atol=tol)


def test_norms_and_activations():
    x, w = rnd(5, 24), rnd(24)
    close(O.layer_norm(x, w, 1e-3), F.layer_norm(x, (24,), w, None, 1e-3))
    close(O.rms(x, 0.1), F.rms_norm(x, (24,), None, 0.1))
    close(O.silu(x), F.silu(x))
    close(O.gelu_tanh(x), F.gelu(x, approximate="tanh"))
    close(O.softplus(40 * x), torch.logaddexp(40 * x, torch.zeros_like(x)))
    close(O.unit(x), x / (x.pow(2).sum(-1, keepdim=True) + 1e-6).sqrt())


@pytest.mark.parametrize("taps", [1, 2, 5])
def test_causal_conv_is_conv1d(taps):
    x, w, b = rnd(9, 6), rnd(6, taps), rnd(6)
    ref = F.conv1d(F.pad(x.T[None], (taps - 1, 0)), w[:, None], b, groups=6)[0].T
    close(O.causal_conv(x, w, b), ref)
    close(O.input_conv(x, w), x + ref - b)


def test_rotation_is_a_complex_product():
    x = rnd(7, 3, 10)
    y = O.rotate(x, 50.0, 6)
    z = torch.view_as_complex(x[..., :6].reshape(7, 3, 3, 2).contiguous())
    ang = torch.arange(7.0, dtype=torch.float64)[:, None] * 50.0 ** (-torch.arange(0, 6, 2, dtype=torch.float64) / 6)
    ref = torch.view_as_real(z * torch.polar(torch.ones_like(ang), ang)[:, None]).reshape(7, 3, 6)
    close(y[..., :6], ref)
    assert torch.equal(y[..., 6:], x[..., 6:]) and torch.equal(y[0], x[0])


@pytest.mark.parametrize("window", [1, 4, 100])
def test_window_softmax_is_sdpa_with_a_band(window):
    q, k, v = rnd(11, 6, 8), rnd(11, 2, 8), rnd(11, 2, 5)
    i = torch.arange(11)
    band = (i[:, None] >= i[None]) & (i[:, None] - i[None] < window)
    ref = F.scaled_dot_product_attention(q.transpose(0, 1), k.transpose(0, 1).repeat_interleave(3, 0),
                                         v.transpose(0, 1).repeat_interleave(3, 0), attn_mask=band, scale=0.3).transpose(0, 1)
    close(O.window_softmax(q, k, v, 0.3, window), ref)
    if window == 1:
        close(O.window_softmax(q, k, v, 0.3, 1), v.repeat_interleave(3, 1))


def test_delta_rule_is_its_unrolled_product():
    """S_t = g_t (I - beta_t k_t k_t^T) S_{t-1} + beta_t k_t v_t^T, multiplied out."""
    T, H, d, dv = 6, 2, 4, 3
    q, k, v = rnd(T, H, d), rnd(T, H, d), rnd(T, H, dv)
    dec, beta = torch.rand(T, H, generator=g, dtype=torch.float64), torch.rand(T, H, generator=g, dtype=torch.float64)
    o = O.delta_rule(q, k, v, dec, beta)
    for h in range(H):
        for t in range(T):
            S = torch.zeros(d, dv, dtype=torch.float64)
            for s in range(t + 1):
                M = torch.eye(d, dtype=torch.float64)
                for r in range(s + 1, t + 1):
                    M = dec[r, h] * (torch.eye(d, dtype=torch.float64) - beta[r, h] * torch.outer(k[r, h], k[r, h])) @ M
                S = S + M @ (beta[s, h] * torch.outer(k[s, h], v[s, h]))
            close(o[t, h], S.T @ q[t, h])


def test_linear_unit_is_its_weighted_sum():
    T, blocks, n = 7, 2, 3
    u, lam = rnd(T, 6), rnd(6)
    ra, ri, rb, ib = rnd(blocks, n, n), rnd(blocks, n, n), rnd(blocks, n), rnd(blocks, n)
    full = lambda m: torch.block_diag(*m)
    r, i = torch.sigmoid(u @ full(ra).T + rb.reshape(-1)), torch.sigmoid(u @ full(ri).T + ib.reshape(-1))
    a = torch.exp(-8 * r * F.softplus(lam))
    x = (1 - a * a).sqrt() * i * u
    ref = torch.stack([sum(torch.prod(a[s + 1:t + 1], 0) * x[s] for s in range(t + 1)) for t in range(T)])
    close(O.gated_linear_unit(u, ra, rb, ri, ib, lam), ref, 1e-9)


@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_model_is_causal_and_config_translates(name):
    cfg = json.loads(json.dumps(cases.CONFIGS[name]))
    w = cases.weights(cfg)
    toks = cases.tokens(cfg, 12)
    layers = []
    y = O.forward(cfg, w, torch.tensor(toks), layers)
    assert y.shape == (12, cfg["vocab"]) and len(layers) == len(cfg["layers"]) and torch.isfinite(y).all()
    close(O.forward(cfg, w, torch.tensor(toks[:7])), y[:7])
    model = cases.build(cfg, w, "cpu", torch.float32)   # every parameter is filled (strict load)
    assert len(model.transformer.layers) == len(cfg["layers"])
    assert [b.mlp is not None for b in model.transformer.layers] == [l["mlp"] is not None for l in cfg["layers"]]
    assert model.lm_head.weight is not model.transformer.embeddings.word_embeddings.weight


def test_unknown_names_are_refused():
    from based_amd import architectures

    cfg = json.loads(json.dumps(cases.CONFIGS["ones"]))
    with pytest.raises(NotImplementedError):
        architectures.find({**cfg, "architecture": "Other"})
    cfg["layers"][1]["type"] = "other"
    with pytest.raises(NotImplementedError):
        architectures.find(cfg).stack_config(cfg)
    assert architectures.find({"n_embd": 8}) is None


def test_replay_hands_caches_back():
    from based_amd.replay import Replay

    class Fake(torch.nn.Module):
        def __init__(self):
            super().__init__()
            self.p = torch.nn.Parameter(torch.zeros(1))

        def forward(self, ids, inference_params=None, logits_at=None):
            from types import SimpleNamespace
            at = inference_params.seqlen_offset + torch.arange(ids.shape[1])
            return SimpleNamespace(logits=at[None, :, None].float().expand(1, -1, 4)[:, logits_at])

    r = Replay(Fake(), 8)
    assert r.feed("a", [1, 2, 3], [2, 0])[:, 0].tolist() == [2, 0]
    assert r.feed("a", [4], [0])[:, 0].tolist() == [3] and r.feed("a", [4], []).shape == (0, 4)
    first = r.live["a"]
    r.end("a")
    assert r.feed("b", [1, 2], [1])[:, 0].tolist() == [1] and r.live["b"] is first
    with pytest.raises(ValueError):
        r.feed("b", [0] * 7, [])
