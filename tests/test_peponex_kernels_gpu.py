"""The operations behind time mixing, decaying linear attention, latent attention, experts and token inputs against
their plain statement (oracle/peponex_oracle.py): float32 against float64 on the same numbers, bfloat16
against float64 on the rounded inputs."""
import math

import pytest
import torch

from oracle import peponex_oracle as O

pytestmark = pytest.mark.gpu
F32, BF16 = torch.float32, torch.bfloat16
TOL = {F32: 3e-6, BF16: 6e-3}
DTYPES = [F32, BF16]


def rnd(*shape, seed=0, dtype=F32, scale=1.0, mean=0.0):
    return (torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale + mean).to(dtype)


def close(got, want, tol):
    got, want = got.double().cpu(), want.double()
    err = float((got - want).norm() / want.norm().clamp_min(1e-30))
    assert err < tol, err


# ---- norms with addends, element-wise operations ----
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [8, 84, 520, 2048, 4104])
def test_add_norm_with_addends(dev, D, dtype):
    from based_amd import ops

    rows = 11
    x, w, post, vec, table = (rnd(*s, seed=i, dtype=dtype) for i, s in enumerate([(rows, D), (D,), (D,), (D,), (7, D)]))
    res = rnd(rows, D, seed=9)
    idx = torch.randint(7, (rows,), generator=torch.Generator().manual_seed(1))
    d = lambda t: t.to(dev)
    for kind in (ops.NORM_RMS, ops.NORM_NONE):
        for r in (None, res):
            full = ops.Addends(d(post), 1e-3, d(vec), d(table), d(idx))
            y, out = ops.add_norm(d(x), None if r is None else d(r), d(w), 1e-5, kind, 0.7, addends=full)
            want = O.rms(x.double(), 1e-3) * post.double()
            want = (want if r is None else r.double() + 0.7 * want) + vec.double() + table.double()[idx]
            close(out, want, 1e-6)
            close(y, want if kind == ops.NORM_NONE else O.rms(want, 1e-5) * w.double(), TOL[dtype])
    y, out = ops.add_norm(d(x), d(res), d(w), 1e-5, ops.NORM_RMS, 1.0, addends=ops.Addends(vec=d(vec)))
    close(out, res.double() + x.double() + vec.double(), 1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [8, 20, 264])
def test_token_mix_in_portions(dev, D, dtype):
    from based_amd import ops

    B, T, S = 2, 23, 3
    x, mu = rnd(B, T, D, dtype=dtype), rnd(S, D, seed=1, dtype=dtype)
    want = torch.stack([torch.stack([O.token_mix(x[b].double(), mu[s].double()) for b in range(B)]) for s in range(S)])
    close(ops.token_mix(x.to(dev), mu.to(dev)), want, TOL[dtype])
    for cuts in ([23], [1] * 23, [2, 3, 1, 8, 9]):
        ring = torch.full((B, 2, D), float("nan"), dtype=dtype, device=dev)
        at, got = 0, []
        for n in cuts:
            got.append(ops.token_mix(x[:, at:at + n].to(dev), mu.to(dev), ring, at))
            at += n
        close(torch.cat(got, 2), want, TOL[dtype])
    # rows at positions of their own
    pos = torch.tensor([0, 5], dtype=torch.int32, device=dev)
    ring = torch.full((B, 2, D), float("nan"), dtype=dtype, device=dev)
    ring[1, 4 % 2] = x[1, 4].to(dev)
    y = ops.token_mix(torch.stack([x[0, :1], x[1, 5:6]]).to(dev), mu.to(dev), ring, pos)
    close(y[:, 0, 0], want[:, 0, 0], TOL[dtype])
    close(y[:, 1, 0], want[:, 1, 5], TOL[dtype])
    assert torch.equal(ring[1, 1].cpu(), x[1, 5])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rank,C", [(1, 16), (7, 60), (24, 200), (64, 96), (256, 64), (300, 40)])
def test_channel_decay(dev, rank, C, dtype):
    from based_amd import ops

    h, w2, w0 = rnd(2, 37, rank, dtype=dtype, scale=2), rnd(C, rank, seed=1, dtype=dtype, scale=rank ** -0.5), rnd(C, seed=2, dtype=dtype, scale=2)
    got = ops.channel_decay(h.to(dev), w2.to(dev), w0.to(dev)).double().cpu()
    want = -torch.exp(torch.tanh(h.double()) @ w2.double().T + w0.double()) / math.log(2)
    # 32-bit whatever the element type (pairs of bf16 in the product: 16 bits)
    assert float(((got - want) / want).abs().max()) < (2e-5 if dtype == F32 else 2e-4)


@pytest.mark.parametrize("dtype", DTYPES)
def test_gelu_mul_and_softcap(dev, dtype):
    from based_amd import ops

    g, table = rnd(9, 12, dtype=dtype, scale=3), rnd(5, 40, seed=1, dtype=dtype)
    idx = torch.tensor([0, 4, 4, 1, 2, 3, 0, 1, 2])
    part = table.to(dev)[:, 24:36]
    close(ops.gelu_mul(g.to(dev), part, idx.to(dev)), O.gelu_tanh(g.double()) * table[:, 24:36].double()[idx], TOL[dtype])
    x = rnd(3, 1, 37, dtype=dtype, scale=40)
    close(ops.softcap_(x.to(dev).clone(), 30.0), 30 * torch.tanh(x.double() / 30), TOL[dtype])
    small = rnd(64, dtype=dtype, scale=1e-3)
    close(ops.softcap_(small.to(dev).clone(), 2.0), 2 * torch.tanh(small.double() / 2), TOL[dtype])
    assert ops.softcap_(torch.empty(0, 8, device=dev, dtype=dtype), 2.0).numel() == 0


# ---- recurrences ----
def channel_case(B, T, H, d, dv, dtype, seed=0, strong=False):
    r, k = rnd(B, T, H, d, seed=seed, dtype=dtype), rnd(B, T, H, d, seed=seed + 1, dtype=dtype)
    v, u = rnd(B, T, H, dv, seed=seed + 2, dtype=dtype), rnd(H, d, seed=seed + 3, dtype=dtype)
    # from decays that keep hundreds of tokens to ones that keep nothing
    z = rnd(B, T, H, d, seed=seed + 4, scale=1.0 if strong else 0.5) + torch.linspace(-7, 5 if strong else 0, d)
    lw = -torch.exp(z) / math.log(2)
    return r, k, v, u, lw


def want_channel(case, state=None):
    r, k, v, u, lw = (t.double() for t in case)
    B, T, H, d = r.shape
    out = []
    for b in range(B):
        if state is None:
            out.append(O.bonus_recurrence(r[b], k[b], v[b], 2.0 ** lw[b], u))
    return torch.stack(out).reshape(B, T, -1)


def run_channel(dev, case, cuts, state=None):
    from based_amd import ops

    r, k, v, u, lw = (t.to(dev) for t in case)
    B, T, H, d = r.shape
    dv = v.shape[-1]
    if state is None:
        state = torch.full((B, H, dv, (d + 3) // 4 * 4), float("nan"), device=dev)
    at, out = 0, []
    for n in cuts:
        s = slice(at, at + n)
        out.append(ops.decay_scan(r[:, s].flatten(2), k[:, s].flatten(2), v[:, s].flatten(2), state, H, channel_log2=lw[:, s].flatten(2).contiguous(),
                                  bonus=u, fresh=at == 0))
        at += n
    return torch.cat(out, 1)


SHAPES = [(1, 150, 2, 64, 64), (2, 70, 3, 20, 20), (1, 200, 1, 48, 80), (1, 130, 2, 32, 16), (1, 90, 1, 96, 40), (1, 140, 1, 128, 128),
          (1, 33, 2, 7, 9), (1, 40, 1, 200, 24), (1, 17, 1, 4, 4)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", SHAPES)
def test_channel_decay_scan(dev, shape, dtype):
    T = shape[1]
    for strong in (False, True):
        case = channel_case(*shape, dtype, strong=strong)
        want = want_channel(case)
        for cuts in ([T], [2, T - 2], [3, 10, 2, T - 15], [T - 1, 1]):
            close(run_channel(dev, case, cuts), want, TOL[dtype])


@pytest.mark.parametrize("dtype", DTYPES)
def test_channel_decay_scan_in_segments(dev, dtype):
    """Long enough to be cut into segments (bf16), with what an earlier portion left."""
    case = channel_case(1, 1100, 2, 32, 40, dtype)
    want = want_channel(case)
    for cuts in ([1100], [37, 1063], [700, 400]):
        got = run_channel(dev, case, cuts)
        close(got, want, TOL[dtype])
        close(got[:, -20:], want[:, -20:], 2 * TOL[dtype])


def test_channel_scan_keeps_far_tokens(dev):
    """One key and value far back that a later query asks for, among hundreds of others: a slowly decaying channel of its own."""
    T, H, d, dv = 700, 1, 64, 64
    r, k, v, u, lw = channel_case(1, T, H, d, dv, BF16)
    lw[..., 5] = -1e-4
    k[..., 5] = 0
    r[..., 5] = 0
    k[0, 3, 0, 5], r[0, 690, 0, 5] = 20, 20
    want = want_channel((r, k, v, u, lw))
    got = run_channel(dev, (r, k, v, u, lw), [T])
    close(got[:, 690], want[:, 690], TOL[BF16])
    far = v[0, 3, 0].double() * 400 * 2.0 ** float(lw[0, 4:690, 0, 5].double().sum())
    assert float((got[0, 690].double().cpu() - far).norm() / far.norm()) < 0.3  # the far token is what the query finds


HEAD_SHAPES = [(1, 150, 2, 64, 64, [0.9, 0.999]), (2, 70, 3, 20, 36, [0.0, 1.0, 0.5]), (1, 200, 1, 48, 80, [0.7]), (1, 140, 2, 128, 136, [0.99, 0.2]),
               (1, 33, 2, 7, 9, [0.3, 1.0]), (1, 1100, 2, 32, 40, [0.9995, 0.6]), (1, 17, 1, 160, 12, [0.95])]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", HEAD_SHAPES)
def test_head_decay_scan_and_steps(dev, shape, dtype):
    from based_amd import ops

    B, T, H, d, dv, decay = shape
    q, k = rnd(B, T, H * d, dtype=dtype), rnd(B, T, H * d, seed=1, dtype=dtype)
    v = rnd(B, T, H * dv, seed=2, dtype=dtype)
    # what the kernels read behind silu, as the element type keeps it
    a = lambda x: O.silu(x.double()).to(dtype).double()
    want = torch.stack([O.decay_recurrence(a(q[b]).view(T, H, d), a(k[b]).view(T, H, d), a(v[b]).view(T, H, dv),
                                           torch.tensor(decay, dtype=torch.float32).double()) for b in range(B)]).reshape(B, T, -1)
    hd = ops.head_decays(decay, dev)
    D = lambda t: t.to(dev)
    for cuts in ([T], [2, T - 7, 1, 1, 1, 1, 1], [T // 2, T - T // 2]):
        state = torch.full((B, H, dv, (d + 3) // 4 * 4), float("nan"), device=dev)
        at, got = 0, []
        for n in cuts:
            s = slice(at, at + n)
            if n == 1 and at > 0:
                o = torch.empty(B, H * dv, dtype=dtype, device=dev)
                ops.decay_step(D(q[:, at]), D(k[:, at]), D(v[:, at]), state, H, at, head_decay=hd, activation=ops.ACT_SILU, out=o)
                got.append(o[:, None])
            else:
                got.append(ops.decay_scan(D(q[:, s]), D(k[:, s]), D(v[:, s]), state, H, head_decay=hd, activation=ops.ACT_SILU, fresh=at == 0))
            at += n
        close(torch.cat(got, 1), want, 2 * TOL[dtype] if T > 1000 else TOL[dtype])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,rank", [(2, 64, 24), (3, 20, 7), (1, 128, 64), (2, 7, 1), (1, 256, 16), (5, 32, 200)])
def test_channel_decay_steps(dev, H, d, rank, dtype):
    """Steps from the first token on (into a state that holds anything), rows at positions of their own."""
    from based_amd import ops

    B, T, eps = 2, 12, 1e-5
    r, k, v, g = (rnd(B, T, H * d, seed=i, dtype=dtype) for i in range(4))
    hid = rnd(B, T, rank, seed=5, dtype=dtype)
    w2, w0, u = rnd(H * d, rank, seed=6, dtype=dtype, scale=rank ** -0.5), rnd(H * d, seed=7, dtype=dtype, scale=2, mean=-1), rnd(H, d, seed=8, dtype=dtype)
    nw = rnd(H * d, seed=9, dtype=dtype)
    w = torch.exp(-torch.exp(torch.tanh(hid.double()) @ w2.double().T + w0.double()))
    want = []
    for b in range(B):
        o = O.bonus_recurrence(r[b].double().view(T, H, d), k[b].double().view(T, H, d), v[b].double().view(T, H, d), w[b].view(T, H, d), u.double())
        want.append(O.rms(o, eps).reshape(T, -1) * nw.double() * O.silu(g[b].double()))
    want = torch.stack(want)
    D = lambda t: t.to(dev)
    state = torch.full((B, H, d, (d + 3) // 4 * 4), float("nan"), device=dev)
    for t in range(T):
        o = torch.empty(B, H * d, dtype=dtype, device=dev)
        # row 1 lags two tokens behind: its position comes from the device; before its start it is not run
        at = [t, max(t - 2, -1)]
        pos = torch.tensor(at, dtype=torch.int32, device=dev)
        pick = lambda x: D(torch.stack([x[0, at[0]], x[1, max(at[1], 0)]]))
        ops.decay_step(pick(r), pick(k), pick(v), state, H, pos, bonus=D(u), hidden=pick(hid), w2=D(w2), w0=D(w0), gate=pick(g), norm_weight=D(nw),
                       eps=eps, out=o)
        close(o[0], want[0, t], 3 * TOL[dtype])
        if at[1] >= 0:
            close(o[1], want[1, at[1]], 3 * TOL[dtype])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("G,n", [(1, 8), (1, 300), (3, 20), (4, 64), (2, 128), (1, 3000), (16, 64)])
def test_group_norm_gate(dev, G, n, dtype):
    from based_amd import ops

    o, g, w = rnd(2, 5, G * n, dtype=dtype), rnd(2, 5, G * n, seed=1, dtype=dtype), rnd(G * n, seed=2, dtype=dtype)
    for act, f in ((ops.ACT_SILU, O.silu), (ops.ACT_SIGMOID, O.sigmoid)):
        out = torch.empty(2, 5, G * n, dtype=dtype, device=dev)
        ops.group_norm_gate(o.to(dev), w.to(dev), g.to(dev), G, 1e-3, act, 0.6, out=out)
        want = O.rms(o.double().view(2, 5, G, n), 1e-3).reshape(2, 5, -1) * w.double() * f(g.double()) * 0.6
        close(out, want, TOL[dtype])


# ---- latent attention ----
def latent_core(dev, dtype, H, d, r, dv, R, window, seed=0, interleaved=False):
    from based_amd.mixers.latent_attention import LatentAttention

    core = LatentAttention(H, d, r, dv, R, window, scale=0.8 * (d + r) ** -0.5, rotary_base=500.0, rotary_interleaved=interleaved, layer_idx=0,
                           device=dev, dtype=dtype)
    uk, uv, nw = rnd(H * d, R, seed=seed, scale=R ** -0.5).bfloat16(), rnd(H * dv, R, seed=seed + 1, scale=R ** -0.5).bfloat16(), rnd(R, seed=seed + 2, scale=0.2, mean=1.0).bfloat16()
    with torch.no_grad():
        core.norm_weight.copy_(nw)
        core.expand.copy_(LatentAttention.expansion(uk, uv, H, r))
    return core.eval(), uk.double(), uv.double(), nw.double()


def latent_want(core, uk, uv, nw, q, x):
    """q (T, H, r + d) with the rotated channels first, x (T, R + r), float64."""
    T, H, r, R = q.shape[0], core.heads, core.rot_dim, core.kv_rank
    turn = lambda y: O.rotate_halves(y, 500.0, r)
    c = O.rms(x[:, :R], core.norm_eps) * nw
    k = (c @ uk.T).view(T, H, core.dim)
    v = (c @ uv.T).view(T, H, core.vdim)
    kr = turn(x[:, R:])
    qr = turn(q[..., :r])
    out = []
    for h in range(H):
        s = (q[:, h, r:] @ k[:, h].T + qr[:, h] @ kr.T) * core.scale
        out.append(O.window_weights(s, core.window) @ v[:, h])
    return torch.stack(out, 1).reshape(T, -1)


def run_latent(core, dev, dtype, q, x, cuts, params=None):
    from based_amd.generation import InferenceParams

    T = x.shape[1]
    params = params or InferenceParams(max_seqlen=T, max_batch_size=x.shape[0])
    B, at, out = x.shape[0], 0, []
    for n in cuts:
        parts = {"q": q[:, at:at + n].flatten(2).to(dev, dtype), "kv": x[:, at:at + n].to(dev, dtype)}
        o = torch.empty(B, n, core.out_features, dtype=dtype, device=dev)
        with torch.inference_mode():
            core(lambda name: parts[name], o, inference_params=params)
        params.seqlen_offset += n
        out.append(o)
        at += n
    return torch.cat(out, 1)


LATENT = [(2, 40, 16, 24, 96, 33), (5, 16, 32, 64, 64, 64), (18, 64, 64, 96, 256, 100), (16, 128, 64, 128, 512, 70), (3, 14, 6, 10, 36, 9), (1, 8, 2, 8, 8, 1)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,r,dv,R,window", LATENT)
def test_latent_attention(dev, H, d, r, dv, R, window, dtype):
    core, uk, uv, nw = latent_core(dev, dtype, H, d, r, dv, R, window)
    T = 150
    q, x = rnd(1, T, H, r + d, seed=4).bfloat16(), rnd(1, T, R + r, seed=5).bfloat16()
    want = latent_want(core, uk, uv, nw, q[0].double(), x[0].double())
    for cuts in ([T], [100] + [1] * 50, [2] * 75, [65, 63, 22], [1] * 10 + [140]):
        close(run_latent(core, dev, dtype, q, x, cuts)[0], want, 2 * TOL[dtype])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [1, 9, 64, 65, 128, 200])
def test_latent_window_edges(dev, window, dtype):
    """A key that one query matches far better than any other, just inside and just outside the window, in prompts and steps."""
    H, d, r, dv, R, T = 2, 72, 16, 16, 104, 330
    core, uk, uv, nw = latent_core(dev, dtype, H, d, r, dv, R, window)
    for edge, seen in ((window - 1, True), (window, False)):
        for i in (T - 1, 257, 200):
            j = i - edge
            if j < 0:
                continue
            q, x = rnd(1, T, H, r + d, seed=4, scale=0.3).bfloat16(), rnd(1, T, R + r, seed=5).bfloat16()
            # queries point at what key j is, so that its score stands out
            c = O.rms(x[0, j, :R].double(), core.norm_eps) * nw
            key = (uk @ c).view(H, d)
            q[0, i, :, r:] = (key * 60 / key.square().sum(-1, keepdim=True) / core.scale).bfloat16()
            want = latent_want(core, uk, uv, nw, q[0].double(), x[0].double())
            value = uv @ c
            assert (float((want[i] - value).norm() / value.norm()) < 0.05) == seen  # the test shows what it is for
            for cuts in ([T], [i] + [1] * (T - i), [i - 1, 2] + ([T - i - 1] if i < T - 1 else [])):
                close(run_latent(core, dev, dtype, q, x, cuts)[0, i], want[i], 6 * TOL[dtype])


@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_steps_of_rows_at_their_own_positions(dev, dtype):
    """Device positions, one far beyond the other, so that the keys of one row fill many splits and of another none."""
    from based_amd.generation import InferenceParams

    H, d, r, dv, R, window, T = 4, 24, 8, 32, 64, 700, 900
    core, uk, uv, nw = latent_core(dev, dtype, H, d, r, dv, R, window)
    q, x = rnd(3, T, H, r + d, seed=4).bfloat16(), rnd(3, T, R + r, seed=5).bfloat16()
    at = [880, 3, 70]
    params = InferenceParams(max_seqlen=T, max_batch_size=3)
    for b in range(3):
        params.seqlen_offset, params.batch_size_offset = 0, b
        run_latent(core, dev, dtype, q[b:b + 1, :at[b]], x[b:b + 1, :at[b]], [at[b]], params)
    params.batch_size_offset, params.seqlen_offset = 0, max(at)
    params.lengths_per_sample = torch.tensor(at, dtype=torch.int32, device=dev)
    for step in range(3):
        pick = lambda y: torch.stack([y[b, at[b] + step] for b in range(3)])[:, None]
        o = run_latent(core, dev, dtype, pick(q), pick(x), [1], params)
        params.lengths_per_sample += 1
        for b in range(3):
            n = at[b] + step + 1
            want = latent_want(core, uk, uv, nw, q[b, :n].double(), x[b, :n].double())[-1]
            close(o[b, 0], want, 2 * TOL[dtype])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,r,dv,R,window", [(4, 24, 8, 32, 64, 30), (3, 136, 16, 96, 264, 50), (17, 64, 32, 64, 512, 90), (2, 14, 6, 10, 40, 7)])
def test_latent_steps_of_many_rows(dev, H, d, r, dv, R, window, dtype):
    """More rows than one tile of 16, at positions from the first one on; a row that is at no position has no say in the others."""
    from based_amd.generation import InferenceParams

    B, T = 19, 120
    core, uk, uv, nw = latent_core(dev, dtype, H, d, r, dv, R, window)
    q, x = rnd(B, T, H, r + d, seed=4).bfloat16(), rnd(B, T, R + r, seed=5).bfloat16()
    at = [(37 * b) % (T - 2) for b in range(B)]
    params = InferenceParams(max_seqlen=T, max_batch_size=B)
    for b in range(B):
        params.seqlen_offset, params.batch_size_offset = 0, b
        if at[b]:
            run_latent(core, dev, dtype, q[b:b + 1, :at[b]], x[b:b + 1, :at[b]], [at[b]], params)
    params.batch_size_offset, params.seqlen_offset = 0, max(at)
    idle = 5
    for step in range(2):
        places = [a + step for a in at]
        params.lengths_per_sample = torch.tensor([-1 if b == idle else p for b, p in enumerate(places)], dtype=torch.int32, device=dev)
        pick = lambda y: torch.stack([y[b, places[b]] for b in range(B)])[:, None]
        o = run_latent(core, dev, dtype, pick(q), pick(x), [1], params)
        for b in range(B):
            if b != idle:
                n = places[b] + 1
                close(o[b, 0], latent_want(core, uk, uv, nw, q[b, :n].double(), x[b, :n].double())[-1], 2 * TOL[dtype])


# ---- experts ----
def expert_case(n, D, F, E, top, dtype, seed=0):
    h, router = rnd(n, D, seed=seed, dtype=dtype), rnd(E, D, seed=seed + 1, dtype=dtype, scale=2 * D ** -0.5)
    w1, w2 = rnd(E, 2 * F, D, seed=seed + 2, dtype=dtype, scale=D ** -0.5), rnd(E, D, F, seed=seed + 3, dtype=dtype, scale=F ** -0.5)
    w = {"m.router": router.double()}
    for e in range(E):
        w[f"m.e{e}.up"], w[f"m.e{e}.gate"], w[f"m.e{e}.down"] = w1[e, :F].double(), w1[e, F:].double(), w2[e].double()
    return h, router, w1, w2, w


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,D,F,E,top", [(1, 64, 16, 4, 1), (9, 192, 40, 5, 2), (3, 84, 22, 3, 3), (200, 128, 64, 8, 1), (333, 192, 72, 6, 2),
                                         (700, 64, 200, 3, 2), (150, 256, 136, 130, 3), (260, 84, 30, 4, 2), (5, 64, 8, 1, 1), (1100, 136, 64, 4, 4), (16, 128, 64, 8, 2), (24, 128, 40, 20, 2),
                                         (32, 1024, 64, 40, 4), (31, 64, 64, 3, 1), (5000, 64, 72, 6, 2), (4100, 128, 264, 100, 2)])
def test_experts(dev, n, D, F, E, top, dtype):
    from based_amd import ops

    h, router, w1, w2, w = expert_case(n, D, F, E, top, dtype)
    spec = {"router": {"top": top}}
    want = O.expert_mlp(h.double(), w, "m", spec)
    got = ops.experts(h.to(dev), router.to(dev), w1.to(dev), w2.to(dev), top).double().cpu()
    # rows whose choice is a close call are left out
    s = O.sigmoid(h.double() @ router.double().T).sort(-1, descending=True).values
    clear = torch.ones(n, dtype=torch.bool) if top == E else s[:, top - 1] - s[:, top] > 1e-5
    assert clear.sum() >= 0.98 * n
    close(got[clear], want[clear], 2 * TOL[dtype])


def test_expert_products_do_not_depend_on_the_batch(dev):
    """Grouped tiles against one choice at a time, with experts that nobody chooses and one that everybody does."""
    from based_amd import ops

    h, router, w1, w2, _ = expert_case(300, 128, 64, 7, 2, BF16)
    router = router * 0.05
    router[3] = 0
    h[:, 0] = 4.0
    router[3, 0], router[5, 0] = 2.0, -2.0
    args = [t.to(dev) for t in (router, w1, w2)]
    whole = ops.experts(h.to(dev), *args, 2)
    alone = torch.cat([ops.experts(h[i:i + 20].to(dev), *args, 2) for i in range(0, 300, 20)])
    assert float((whole.double() - alone.double()).norm() / alone.double().norm()) < 4e-3


@pytest.mark.parametrize("n,D,top", [(1, 64, 1), (4, 1024, 2), (3, 4096, 3), (9, 192, 2)])
def test_experts_behind_their_norm(dev, n, D, top):
    from based_amd import ops

    x, router, w1, w2, w = expert_case(n, D, 40, 5, top, BF16)
    router = router * 3  # (clear choices)
    w["m.router"] = router.double()
    res, nw = rnd(n, D, seed=7), rnd(D, seed=8, dtype=BF16, scale=0.2, mean=1.0)
    d = lambda t: t.to(dev)
    for kind in (ops.NORM_RMS, ops.NORM_LAYER):
        for r in (res, None):
            out = torch.empty(n, D, device=dev)
            y = ops.experts(d(x), d(router), d(w1), d(w2), top, norm=(None if r is None else d(r), out, d(nw), 1e-5, kind, 0.5))
            total = x.double() if r is None else r.double() + 0.5 * x.double()
            close(out, total, 1e-6)
            h = (total if kind == ops.NORM_RMS else total - total.mean(-1, keepdim=True))
            h = (O.rms(h, 1e-5) * nw.double()).bfloat16().double()
            close(y, O.expert_mlp(h, w, "m", {"router": {"top": top}}), 3 * TOL[BF16])


# ---- projections of single tokens ----
@pytest.mark.parametrize("M", [1, 3, 8, 9, 32])
@pytest.mark.parametrize("K,rows,rank", [(64, 32, 8), (192, 64, 24), (1024, 96, 40), (2048, 32, 16), (4096, 64, 64)])
def test_projection_of_token_mixes(dev, M, K, rows, rank):
    from based_amd import ops

    S, N = 5, 4 * rows + rank
    x, w = rnd(M, K, dtype=BF16), rnd(N, K, seed=1, dtype=BF16, scale=K ** -0.5)
    mu, nw, post, vec = rnd(S, K, seed=2, dtype=BF16), rnd(K, seed=3, dtype=BF16), rnd(K, seed=4, dtype=BF16), rnd(K, seed=5, dtype=BF16)
    res, table, before = rnd(M, K, seed=6), rnd(6, K, seed=7, dtype=BF16), rnd(M, K, seed=8, dtype=BF16)
    idx = torch.arange(M) % 6
    pos = torch.arange(M, dtype=torch.int32)  # row 0 has nothing before it
    ring = torch.full((M, 2, K), float("nan"), dtype=BF16)
    for m in range(1, M):
        ring[m, (m - 1) % 2] = before[m]
    d = lambda t: t.to(dev)
    ring_d, out = d(ring), torch.empty(M, K, device=dev)
    y = ops.decode_linear(d(x), d(w), prologue=ops.PROLOGUE_STREAM, residual_in=d(res), residual_out=out, norm_weight=d(nw), eps=1e-5, mult=0.5,
                          norm_kind=ops.NORM_RMS, addends=ops.Addends(d(post), 1e-4, d(vec), d(table), d(idx)), mix=(d(mu), ring_d, d(pos), rows))
    total = res.double() + 0.5 * O.rms(x.double(), 1e-4) * post.double() + vec.double() + table.double()[idx]
    close(out, total, 1e-6)
    h = O.rms(total, 1e-5) * nw.double()
    close(torch.stack([ring_d[m, m % 2] for m in range(M)]), h, TOL[BF16])
    h = h.bfloat16().double()
    prev = before.double().clone()
    prev[0] = 0
    want = torch.cat([(h + (prev - h) * mu[min(i // rows, 4)].double()) @ w[i:i + 1].double().T for i in range(N)], 1)
    close(y, want, 2 * TOL[BF16])


@pytest.mark.parametrize("M", [1, 4, 12])
@pytest.mark.parametrize("N,K", [(24, 192), (8, 1024), (520, 64)])
def test_projection_with_gate_table_and_cap(dev, M, N, K):
    from based_amd import ops

    x, w, res = rnd(M, K, dtype=BF16), rnd(N, K, seed=1, dtype=BF16, scale=K ** -0.5), rnd(M, K, seed=2)
    table, idx = rnd(5, 3 * N, seed=3, dtype=BF16), torch.arange(M) % 5
    d = lambda t: t.to(dev)
    out = torch.empty(M, K, device=dev)
    y = ops.decode_linear(d(x), d(w), prologue=ops.PROLOGUE_STREAM, norm_kind=ops.NORM_NONE, residual_in=d(res), residual_out=out,
                          gate=(d(table)[:, N:2 * N], d(idx)))
    r = res.double() + x.double()
    close(out, r, 1e-6)
    close(y, O.gelu_tanh(r.bfloat16().double() @ w.double().T) * table[:, N:2 * N].double()[idx], 2 * TOL[BF16])
    nw = rnd(K, seed=4, dtype=BF16)
    y = ops.decode_linear(d(x), d(w), prologue=ops.PROLOGUE_STREAM, norm_kind=ops.NORM_RMS, norm_weight=d(nw), eps=1e-5, residual_in=d(res), softcap=1.5)
    close(y, 1.5 * torch.tanh((O.rms(r, 1e-5) * nw.double()).bfloat16().double() @ w.double().T / 1.5), 2 * TOL[BF16])


@pytest.mark.parametrize("M", [1, 5, 32, 300])
@pytest.mark.parametrize("n,D", [(8, 64), (24, 192), (64, 1024), (136, 1544), (16, 4096), (512, 512), (32, 264), (128, 1000)])
def test_token_input_of_single_tokens(dev, M, n, D):
    from based_amd import ops

    x, gw, pw, res = rnd(M, D, dtype=BF16), rnd(n, D, seed=1, dtype=BF16, scale=D ** -0.5), rnd(D, n, seed=2, dtype=BF16, scale=n ** -0.5), rnd(M, D, seed=3)
    table, idx = rnd(7, 3 * n, seed=4, dtype=BF16), torch.arange(M) % 7
    d = lambda t: t.to(dev)
    assert ops.token_side_step_ok(d(gw), d(pw))
    for r in (res, None):
        out = torch.empty(M, D, device=dev)
        y = ops.token_side_step(d(x), None if r is None else d(r), out, d(gw), d(pw), d(table)[:, n:2 * n], d(idx), 0.5)
        total = x.double() if r is None else r.double() + 0.5 * x.double()
        close(out, total, 1e-6)
        g = O.gelu_tanh(total.bfloat16().double() @ gw.double().T) * table[:, n:2 * n].double()[idx]
        close(y, g @ pw.double().T, 2 * TOL[BF16])


def test_refusals(dev):
    from based_amd import ops

    z = lambda *s, **k: torch.zeros(*s, device=dev, **{"dtype": BF16, **k})
    with pytest.raises(ValueError, match="state"):
        ops.decay_scan(z(1, 4, 16), z(1, 4, 16), z(1, 4, 16), z(1, 2, 8, 4, dtype=F32), 2, head_decay=ops.head_decays([0.5, 0.5], dev), fresh=True)
    with pytest.raises(ValueError, match="key size"):
        ops.decay_scan(z(1, 4, 300), z(1, 4, 300), z(1, 4, 8), z(1, 1, 8, 300, dtype=F32), 1, head_decay=ops.head_decays([0.5], dev), fresh=True)
    with pytest.raises(ValueError, match="experts"):
        ops.experts(z(2, 8), z(3, 8), z(3, 16, 8), z(3, 8, 8), 4)
    with pytest.raises(ValueError, match="mixes"):
        ops.decode_linear(z(2, 64), z(100, 64), prologue=ops.PROLOGUE_STREAM, norm_weight=z(64), mix=(z(5, 64), z(2, 2, 64), 0, 20))
