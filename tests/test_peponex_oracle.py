"""The plain statement of the Peponex mechanisms (oracle/peponex_oracle.py) against library routines, closed
forms and explicit sums over all earlier tokens, and the parts of the product that need no GPU."""
import math

import pytest
import torch
import torch.nn.functional as F

import peponex_cases as cases
from oracle import peponex_oracle as O

F64 = torch.float64


def rnd(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F64)


def test_token_mix():
    h, mu = rnd(7, 5), rnd(5, seed=1)
    y = O.token_mix(h, mu)
    assert torch.allclose(y[0], h[0] * (1 - mu))
    assert torch.allclose(y[1:], torch.lerp(h[1:], h[:-1], mu))


def test_channel_decay():
    x, w1, w2, w0 = rnd(6, 5), rnd(3, 5, seed=1), rnd(4, 3, seed=2), rnd(4, seed=3)
    z = F.linear(torch.tanh(F.linear(x, w1)), w2, w0)
    assert torch.allclose(O.channel_decay(x, w1, w2, w0).log(), -z.exp())


def test_bonus_recurrence_is_the_sum_over_earlier_tokens():
    T, H, d, dv = 9, 2, 3, 4
    r, k, v, u = rnd(T, H, d), rnd(T, H, d, seed=1), rnd(T, H, dv, seed=2), rnd(H, d, seed=3)
    w = torch.sigmoid(rnd(T, H, d, seed=4))
    o = O.bonus_recurrence(r, k, v, w, u)
    for t in range(T):
        for h in range(H):
            want = (r[t, h] * u[h] * k[t, h]).sum() * v[t, h]
            for s in range(t):
                want = want + (r[t, h] * w[s + 1:t, h].prod(0) * k[s, h]).sum() * v[s, h]
            assert torch.allclose(o[t, h], want)


def test_decay_recurrence_is_the_sum_over_tokens():
    T, H = 9, 3
    q, k, v, decay = rnd(T, H, 4), rnd(T, H, 4, seed=1), rnd(T, H, 2, seed=2), torch.tensor([0.3, 1.0, 0.0], dtype=F64)
    o = O.decay_recurrence(q, k, v, decay)
    gap = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    for h in range(H):
        weight = torch.where(gap >= 0, decay[h] ** gap.clamp_min(0), torch.zeros((), dtype=F64))
        assert torch.allclose(o[:, h], (q[:, h] @ k[:, h].T * weight) @ v[:, h])


def test_rotation_is_complex_multiplication():
    x = rnd(11, 3, 10)
    y = O.rotate_halves(x, 50.0, 6)
    z = torch.complex(x[..., :3], x[..., 3:6])
    ang = torch.arange(11, dtype=F64)[:, None] * 50.0 ** (-torch.arange(0, 6, 2, dtype=F64) / 6)
    z = z * torch.polar(torch.ones_like(ang), ang)[:, None]
    assert torch.allclose(y[..., :6], torch.cat([z.real, z.imag], -1)) and torch.equal(y[..., 6:], x[..., 6:])


@pytest.mark.parametrize("window", [1, 4, 100])
def test_window_weights(window):
    s, v = rnd(12, 12), rnd(12, 5, seed=1)
    idx = torch.arange(12)
    mask = (idx[:, None] >= idx[None, :]) & (idx[:, None] - idx[None, :] < window)
    want = F.scaled_dot_product_attention(s[None], torch.eye(12, dtype=F64)[None], v[None], attn_mask=mask, scale=1.0)[0]
    assert torch.allclose(O.window_weights(s, window) @ v, want)


def test_latent_mixer_attends_expanded_keys():
    """Against a library attention over explicit keys [unrotated | rotated] and values."""
    cfg = cases.CONFIGS["mixed"]
    w, m, eps, T = cases.weights("mixed"), cfg["layers"][1]["mixer"], 1e-5, 40
    h = rnd(T, cfg["width"])
    H, d, r, R, dv = m["heads"], m["dim"], m["rot_dim"], m["kv_rank"], m["vdim"]
    pre = "l1.mix"
    q = F.linear(h, w[pre + ".q"]).view(T, H, d + r)
    down = F.linear(h, w[pre + ".dkv"])
    c = F.rms_norm(down[:, :R], (R,), w[pre + ".dkv.norm"], eps)
    turn = lambda x: O.rotate_halves(x, m["rot"]["base"], r)
    q = torch.cat([q[..., :d], turn(q[..., d:])], -1)
    k = torch.cat([F.linear(c, w[pre + ".uk"]).view(T, H, d), turn(down[:, R:])[:, None].expand(T, H, r)], -1)
    v = F.linear(c, w[pre + ".uv"]).view(T, H, dv)
    idx = torch.arange(T)
    mask = (idx[:, None] >= idx[None, :]) & (idx[:, None] - idx[None, :] < m["mask"]["size"])
    o = F.scaled_dot_product_attention(q.transpose(0, 1), k.transpose(0, 1), v.transpose(0, 1), attn_mask=mask, scale=m["scale"])
    assert torch.allclose(O.latent_mixer(h, w, pre, m, eps), F.linear(o.transpose(0, 1).reshape(T, -1), w[pre + ".o"]))


def test_experts():
    cfg, w = cases.CONFIGS["mixed"], cases.weights("mixed")
    spec, pre = cfg["layers"][1]["mlp"], "l1.mlp"
    h = rnd(20, cfg["width"]) * 4
    s = torch.sigmoid(F.linear(h, w[pre + ".router"]))
    top = s.topk(spec["router"]["top"], dim=-1)
    ids, scores = O.route(h, w[pre + ".router"], spec["router"]["top"])
    assert torch.equal(ids, top.indices) and torch.allclose(scores, top.values)
    y = torch.zeros_like(h)
    for e in range(spec["router"]["experts"]):
        x = h * s[:, e:e + 1]
        out = F.linear(F.silu(F.linear(x, w[f"{pre}.e{e}.gate"])) * F.linear(x, w[f"{pre}.e{e}.up"]), w[f"{pre}.e{e}.down"])
        y = y + out * (top.indices == e).any(-1, keepdim=True)
    assert torch.allclose(O.expert_mlp(h, w, pre, spec), y)


def test_token_side():
    x, e = rnd(5, 6), rnd(5, 3, seed=1)
    w = {"s.gate": rnd(3, 6, seed=2), "s.proj": rnd(6, 3, seed=3), "s.norm": rnd(6, seed=4)}
    y = F.linear(F.gelu(F.linear(x, w["s.gate"]), approximate="tanh") * e, w["s.proj"])
    assert torch.allclose(O.token_side(x, w, "s", e, 1e-5), F.rms_norm(y, (6,), w["s.norm"], 1e-5))


def test_layer_runs():
    cfg = {"layers": [0] * 5, "loop": {"start": 1, "stop": 3, "times": 2}}
    assert O.layer_runs(cfg) == [(0, None), (1, 0), (2, 0), (1, 1), (2, 1), (3, None), (4, None)]
    assert O.layer_runs({"layers": [0] * 2}) == [(0, None), (1, None)]


@pytest.mark.parametrize("name", ["mixed", "ones", "odd", "wide"])
def test_model_is_causal_and_every_part_reaches_the_logits(name):
    cfg, w = cases.CONFIGS[name], cases.weights(name)
    toks = torch.tensor(cases.tokens(cfg, 12))
    layers = []
    y = O.forward(cfg, w, toks, layers)
    assert len(layers) == len(O.layer_runs(cfg)) and torch.isfinite(y).all()
    assert torch.allclose(O.forward(cfg, w, toks[:7]), y[:7])
    for key in w:
        if ".mlp.e" in key or key == "head" or key.endswith("w0"):
            continue
        other = dict(w)
        other[key] = w[key] + 0.5 * torch.randn(w[key].shape, generator=torch.Generator().manual_seed(9), dtype=F64)
        if key == "embed" or not torch.allclose(O.forward(cfg, other, toks), y, rtol=1e-6, atol=1e-6):
            continue
        # one expert of one is always chosen and a mix of nothing before changes nothing: nothing else may be silent
        assert key.endswith("router") or (name == "ones" and (".q" in key or "uk" in key)), key


# ---- product code that runs without a GPU ----
def test_layer_runs_of_the_stack():
    from based_amd.stack import layer_runs

    assert layer_runs(5, {"start": 1, "stop": 3, "times": 2}) == [
        (0, 0, False), (1, 0, True), (2, 0, False), (1, 1, True), (2, 1, False), (3, 0, False), (4, 0, False)]
    assert layer_runs(2, None) == [(0, 0, False), (1, 0, False)]
    for bad in ({"start": 2, "stop": 2, "times": 1}, {"start": 0, "stop": 3, "times": 1}, {"start": 0, "stop": 1, "times": 0}):
        with pytest.raises(ValueError):
            layer_runs(2, bad)


def test_passes_have_caches_of_their_own():
    from based_amd.generation import InferenceParams
    from based_amd.mixers.streaming import cached

    params = InferenceParams(max_seqlen=4, max_batch_size=2)
    make = lambda b, s: torch.zeros(b, s)
    first = cached(params, 3, "x", make, 2)
    params.layer_pass = 1
    second = cached(params, 3, "x", make, 2)
    assert first.data_ptr() != second.data_ptr() and set(params.key_value_memory_dict) == {3, (3, 1)}
    params.layer_pass = 0
    assert cached(params, 3, "x", make, 2).data_ptr() == first.data_ptr()


def test_converted_weights_and_models_on_the_cpu():
    """Every tensor of the stack is filled from the design's, and allocated caches cover every run."""
    from based_amd import architectures

    assert "Peponex" in architectures.DESIGNS
    for name in cases.CONFIGS:
        cfg, w = cases.CONFIGS[name], cases.weights(name)
        model = cases.build(cfg, w, "cpu", torch.float32)  # strict loading
        caches = model.allocate_inference_cache(2, 8)
        assert len(caches) == len(O.layer_runs(cfg))
    with pytest.raises(NotImplementedError):
        architectures.peponex.stack_config({**cases.CONFIGS["ones"], "layers": [{"type": "x", "mixer": {}, "mlp": None}]}, {})


def test_rotated_channels_come_first():
    from based_amd.architectures.peponex import _rotated_first

    q = torch.arange(2 * 5.0)[:, None]
    assert _rotated_first(q, 2, 3, 2)[:, 0].tolist() == [3, 4, 0, 1, 2, 8, 9, 5, 6, 7]


def test_latent_expansion():
    from based_amd.mixers.latent_attention import LatentAttention

    H, d, dv, R, r = 2, 3, 4, 5, 2
    uk, uv = rnd(H * d, R), rnd(H * dv, R, seed=1)
    row = rnd(R + r, seed=2)
    out = (LatentAttention.expansion(uk, uv, H, r) @ row).view(H, r + d + dv)
    for h in range(H):
        assert torch.equal(out[h, :r], row[R:])
        assert torch.allclose(out[h, r:r + d], uk.view(H, d, R)[h] @ row[:R]) and torch.allclose(out[h, r + d:], uv.view(H, dv, R)[h] @ row[:R])


def test_head_decays():
    from based_amd import ops

    t = ops.head_decays((0.5, 1.0, 0.0, 0.999), "cpu")
    assert t.dtype == torch.float32 and t[1].tolist() == [0.5, 1.0, 0.0, torch.tensor(0.999).item()]
    assert t[0, 0] == -1 and t[0, 1] == 0 and 2.0 ** t[0, 2].item() == 0 and math.isfinite(t[0, 2].item())
