"""Each streamed operation against its plain statement (oracle/sozilix_oracle.py), in float32 against
float64 and in bfloat16: sizes with and without whole 16-byte pieces, portions, window edges that one
outstanding score makes visible, decays that vanish, positions from the device."""
import pytest
import torch

from conftest import rel_l2
from oracle import sozilix_oracle as O

pytestmark = pytest.mark.gpu
F32, BF16 = torch.float32, torch.bfloat16
TOL = {F32: 2e-6, BF16: 6e-3}


def rnd(seed, *shape, dtype=F32):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)).to(dtype)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("D", [8, 100, 256, 1000, 1536, 4096, 4104])
@pytest.mark.parametrize("kind", [0, 1])
def test_add_norm(dev, dtype, D, kind):
    from based_amd import ops

    x, res, w = 3 + rnd(1, 5, D, dtype=dtype), rnd(2, 5, D), rnd(3, D, dtype=dtype)
    for r in (None, res):
        y, out = ops.add_norm(x.to(dev), None if r is None else r.to(dev), w.to(dev), 1e-3, kind, 0.7)
        s = x.double() if r is None else r.double() + 0.7 * x.double()
        ref = O.layer_norm(s, w.double(), 1e-3) if kind == ops.NORM_LAYER else O.rms(s, 1e-3) * w.double()
        assert out.dtype == F32 and rel_l2(out, s) < 2e-7
        assert rel_l2(y, ref) < TOL[dtype]
    assert ops.add_norm(x.to(dev), None, w.to(dev), 1e-3, want_residual=False)[1] is None


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("taps,D", [(1, 16), (2, 40), (3, 37), (4, 264), (8, 24)])
def test_stream_conv_portions_and_rings(dev, dtype, taps, D):
    from based_amd import ops

    L, B = 41, 2
    x, w, b = rnd(4, B, L, D, dtype=dtype), rnd(5, taps, D, dtype=dtype), rnd(6, D, dtype=dtype)
    ref = torch.stack([O.causal_conv(x[i].double(), w.double().T, b.double()) for i in range(B)])
    xd, wd, bd = x.to(dev), w.to(dev), b.to(dev)
    assert rel_l2(ops.stream_conv(xd, wd, bd), ref) < TOL[dtype]
    y = ops.stream_conv(xd, wd, None, activation=ops.ACT_SILU, add_input=True)
    assert rel_l2(y, O.silu(ref - b.double()) + x.double()) < TOL[dtype]
    for cuts in ([1], [2], [3, 1, 9], [17, 2]):
        # the ring starts as garbage: nothing before position 0 may be read
        ring = torch.full((B, taps, D), float("nan"), dtype=dtype, device=dev)
        out, at, i = [], 0, 0
        while at < L:
            n = min(cuts[i % len(cuts)], L - at)
            pos = at if i % 2 else torch.full((B,), at, dtype=torch.int32, device=dev)
            out.append(ops.stream_conv(xd[:, at:at + n], wd, bd, ring, pos))
            at, i = at + n, i + 1
        assert rel_l2(torch.cat(out, 1), ref) < TOL[dtype], cuts


def window_case(seed, B, L, H, G, d, dv, dtype):
    """Queries and keys whose scores single out keys: keys are scaled by factors that differ strongly, so
    that the largest visible one takes most of the weight and a key too many or too few shows."""
    g = torch.Generator().manual_seed(seed)
    axis = torch.randn(d, generator=g)
    q = axis + 0.2 * torch.randn(B, L, H, d, generator=g)
    k = axis * (4 * torch.rand(B, L, G, 1, generator=g) - 1) + 0.2 * torch.randn(B, L, G, d, generator=g)
    v = torch.randn(B, L, G, dv, generator=g)
    return q.to(dtype), k.to(dtype), v.to(dtype)


def window_ref(q, k, v, scale, window, rot, base, eps):
    out = []
    for b in range(q.shape[0]):
        qq, kk, vv = q[b].double(), k[b].double(), v[b].double()
        if rot:
            qq, kk = O.rotate(qq, base, rot), O.rotate(kk, base, rot)
        if eps is not None:
            vv = O.rms(vv, eps)
        out.append(O.window_softmax(qq, kk, vv, scale, window))
    return torch.stack(out)


WINDOW_SHAPES = [(4, 2, 64, 64), (3, 1, 32, 128), (8, 8, 16, 40), (6, 2, 128, 32), (5, 5, 96, 256), (9, 1, 256, 64), (4, 2, 20, 12)]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("H,G,d,dv", WINDOW_SHAPES)
@pytest.mark.parametrize("window", [1, 17, 64, 65, 1000])
def test_window_attention(dev, dtype, H, G, d, dv, window):
    from based_amd import ops
    from based_amd.mixers.window_attention import _ExactRotary

    B, L, scale = 2, 150, 6.0 / d
    rot = 8 if d >= 16 else 0
    q, k, v = window_case(H * 1000 + window, B, L, H, G, d, dv, dtype)
    ref = window_ref(q, k, v, scale, window, rot, 100.0, 1e-3).reshape(B, L, H * dv)
    tables = _ExactRotary(rot, base=100.0, interleaved=True).tables(L, dev)
    qd, kd, vd = (t.to(dev).flatten(2) for t in (q, k, v))
    tol = 1e-5 if dtype == F32 else 2e-2
    for cuts in ([L], [70, 2, 3, 50], [1], [149, 1]):
        cache = torch.full((B, L, G, d + dv), float("nan"), dtype=dtype, device=dev)
        out = torch.empty(B, L, H * dv, dtype=dtype, device=dev)
        at, i = 0, 0
        while at < L:
            n = min(cuts[min(i, len(cuts) - 1)], L - at)
            s = slice(at, at + n)
            kw = dict(rope=tables, value_norm_eps=1e-3, out_scale=0.5)
            if n == 1 and at > 0:
                pos = at if i % 2 else torch.full((B,), at, dtype=torch.int32, device=dev)
                ops.window_attn_step(qd[:, at], kd[:, at], vd[:, at], cache, H, G, window, scale, pos, out=out[:, at], **kw)
            else:
                ops.window_attn_prefill(qd[:, s], kd[:, s], vd[:, s], cache, H, G, window, scale, at, out=out[:, s], **kw)
            at, i = at + n, i + 1
        # per position: a key too many or too few is an error of the order of one there
        err = (out.double().cpu() - 0.5 * ref).norm(dim=-1) / (0.5 * ref).norm(dim=-1)
        assert float(err.max()) < tol, (cuts, int(err.argmax() % L))


def test_window_attention_half_split_rotation_and_long_window(dev):
    """Half-split pairs, no value norm, and a window of several rounds of the step kernel."""
    from based_amd import ops
    from based_amd.mixers.window_attention import _ExactRotary

    B, L, H, G, d, dv, window = 1, 700, 2, 1, 64, 64, 600
    q, k, v = window_case(5, B, L, H, G, d, dv, BF16)
    tables = _ExactRotary(32, base=1000.0, interleaved=False).tables(L, dev)
    perm = torch.tensor([c // 2 + (c % 2) * 16 for c in range(32)] + list(range(32, 64)))  # interleaved place of a half-split channel
    ref = window_ref(q[..., perm], k[..., perm], v, 0.1, window, 32, 1000.0, None).reshape(B, L, -1)
    qd, kd, vd = (t.to(dev).flatten(2) for t in (q, k, v))
    cache = torch.full((B, L, G, d + dv), float("nan"), dtype=BF16, device=dev)
    out = torch.empty(B, L, H * dv, dtype=BF16, device=dev)
    ops.window_attn_prefill(qd[:, :690], kd[:, :690], vd[:, :690], cache, H, G, window, 0.1, 0, rope=tables, out=out[:, :690])
    for t in range(690, L):
        ops.window_attn_step(qd[:, t], kd[:, t], vd[:, t], cache, H, G, window, 0.1, t, rope=tables, out=out[:, t])
    err = (out.double().cpu() - ref).norm(dim=-1) / ref.norm(dim=-1)
    assert float(err.max()) < 2e-2


def delta_ref(x, w, a, b, a_log, dt_bias, H, G, d, dv):
    """Convolution, silu, unit norms, gates and recurrence of one sequence; x (T, C) = q | k | v."""
    c = O.silu(O.causal_conv(x.double(), w.double().T))
    T, nk = x.shape[0], G * d
    q = (O.unit(c[:, :nk].view(T, G, d)) * d ** -0.5).repeat_interleave(H // G, 1)
    k = O.unit(c[:, nk:2 * nk].view(T, G, d)).repeat_interleave(H // G, 1)
    g = torch.exp(-torch.exp(a_log.double()) * O.softplus(a.double() + dt_bias.double()))
    return O.delta_rule(q, k, c[:, 2 * nk:].view(T, H, dv), g, torch.sigmoid(b.double()))


DELTA_SHAPES = [(4, 2, 32, 64), (2, 2, 64, 128), (6, 1, 128, 128), (3, 3, 96, 40), (2, 1, 256, 256), (3, 1, 24, 72), (1, 1, 16, 8)]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("H,G,d,dv", DELTA_SHAPES)
@pytest.mark.parametrize("strong_decay", [False, True])
def test_gated_delta(dev, dtype, H, G, d, dv, strong_decay):
    """The scan in portions and the fused step.  Strong decays drive the running product of decays far
    below its rescaling threshold, and to zero."""
    from based_amd import ops

    B, L, taps = 2, 60, 4
    C = 2 * G * d + H * dv
    x, w = rnd(11, B, L, C, dtype=dtype), 0.6 * rnd(12, taps, C)
    w = w.to(dtype)
    a, b = rnd(13, B, L, H, dtype=dtype), rnd(14, B, L, H, dtype=dtype)
    a_log = (rnd(15, H) + (3.0 if strong_decay else -2.0)).to(dtype)
    dt_bias = rnd(16, H, dtype=dtype)
    if strong_decay:
        a = (4 * a.float()).to(dtype)
    gate, nw = rnd(17, B, L, H * dv, dtype=dtype), rnd(18, dv, dtype=dtype)
    raw = torch.stack([delta_ref(x[i], w, a[i], b[i], a_log, dt_bias, H, G, d, dv) for i in range(B)])
    ref = (O.rms(raw, 1e-3) * nw.double() * O.silu(gate.double()).view(B, L, H, dv) * 0.7).reshape(B, L, H * dv)
    xd, wd, ad, bd, gd = (t.to(dev) for t in (x, w, a, b, gate))
    al, db, nwd = a_log.to(dev), dt_bias.to(dev), nw.to(dev)
    nk = G * d
    for cuts in ([L], [16, 2, 15, 3], [1], [33, 1]):
        state = torch.full((B, H, d, (dv + 3) // 4 * 4), float("nan"), device=dev)
        ring = torch.full((B, taps, C), float("nan"), dtype=dtype, device=dev)
        out = torch.empty(B, L, H * dv, dtype=dtype, device=dev)
        at, i = 0, 0
        while at < L:
            n = min(cuts[min(i, len(cuts) - 1)], L - at)
            s = slice(at, at + n)
            if n == 1:
                pos = at if i % 2 else torch.full((B,), at, dtype=torch.int32, device=dev)
                ops.gated_delta_step(xd[:, at], wd, ring, ad[:, at], bd[:, at], gd[:, at], al, db, nwd, state, H, G, d, dv, nk, 2 * nk,
                                     pos, 1e-3, 0.7, out=out[:, at])
            else:
                c = ops.stream_conv(xd[:, s], wd, None, ring, at, activation=ops.ACT_SILU)
                o = ops.gated_delta_scan(c[..., :nk], c[..., nk:2 * nk], c[..., 2 * nk:], ad[:, s], bd[:, s], al, db, state, H, G,
                                         fresh=at == 0)
                ops.gated_rms_norm(o, nwd, gd[:, s], 1e-3, 0.7, out=out[:, s])
            at, i = at + n, i + 1
        err = rel_l2(out, ref)
        assert err < (3e-5 if dtype == F32 else 2e-2), (cuts, err)


@pytest.mark.parametrize("B,H,dv", [(3, 16, 48), (16, 24, 128), (24, 16, 200)])
def test_gated_delta_scan_column_splits(dev, B, H, dv):
    """Enough (sequence, head) pairs for the forms with two and four columns per lane."""
    from based_amd import ops

    d, L = 64, 37
    q, k, v = (rnd(s, B, L, H * n) for s, n in ((21, d), (22, d), (23, dv)))
    qkv = torch.cat([q, k, v], -1)
    a, b, al, db = rnd(24, B, L, H), rnd(25, B, L, H), rnd(26, H) - 1, rnd(27, H)
    c = qkv.to(dev)
    state = torch.full((B, H, d, (dv + 3) // 4 * 4), float("nan"), device=dev)
    n = H * d
    o = ops.gated_delta_scan(c[..., :n], c[..., n:2 * n], c[..., 2 * n:], a.to(dev), b.to(dev), al.to(dev), db.to(dev), state, H, H, True)
    for i in (0, B - 1):
        g = torch.exp(-torch.exp(al.double()) * O.softplus(a[i].double() + db.double()))
        ref = O.delta_rule(O.unit(q[i].double().view(L, H, d)) * d ** -0.5, O.unit(k[i].double().view(L, H, d)),
                           v[i].double().view(L, H, dv), g, torch.sigmoid(b[i].double()))
        assert rel_l2(o[i], ref) < 3e-6


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("W,blocks", [(64, 1), (160, 2), (96, 3), (256, 1), (54, 2), (8, 8), (520, 2)])
@pytest.mark.parametrize("B", [1, 11])
def test_rglru(dev, dtype, W, blocks, B):
    from based_amd import ops

    L, taps, n = 150, 3, W // blocks
    x, y = rnd(31, B, L, W, dtype=dtype), rnd(32, B, L, W, dtype=dtype)
    w, cb = rnd(33, taps, W, dtype=dtype), rnd(34, W, dtype=dtype)
    ra, ri = (rnd(s, blocks, n, n) * n ** -0.5 for s in (35, 36))
    ra, ri = ra.to(dtype), ri.to(dtype)
    rb, ib = rnd(37, W, dtype=dtype), rnd(38, W, dtype=dtype)
    lam = (2 * rnd(39, W) - 3).to(dtype)   # decays from close to 1 to small
    rows = (0, B - 1)
    ref = []
    for i in rows:
        u = O.causal_conv(x[i].double(), w.double().T, cb.double())
        if dtype == BF16:
            u = u.to(BF16).double()  # the convolution's output is kept in the element type
        S = O.gated_linear_unit(u, ra.double(), rb.double().view(blocks, n), ri.double(), ib.double().view(blocks, n), lam.double())
        ref.append(S * O.gelu_tanh(y[i].double()))
    ref = torch.stack(ref)
    xd, yd, wd, cbd = (t.to(dev) for t in (x, y, w, cb))
    gates = [t.to(dev) for t in (ra, rb, ri, ib, lam)]
    for cuts in ([L], [64, 2, 65, 3], [1], [129, 1]):
        state = torch.full((B, W), float("nan"), device=dev)
        ring = torch.full((B, taps, W), float("nan"), dtype=dtype, device=dev)
        out = torch.empty(B, L, W, dtype=dtype, device=dev)
        at, i = 0, 0
        while at < L:
            m = min(cuts[min(i, len(cuts) - 1)], L - at)
            s = slice(at, at + m)
            if m == 1:
                pos = at if i % 2 else torch.full((B,), at, dtype=torch.int32, device=dev)
                ops.rglru_step(xd[:, at], yd[:, at], wd, cbd, ring, *gates, state, 8.0, pos, out=out[:, at])
            else:
                u = ops.stream_conv(xd[:, s], wd, cbd, ring, at)
                ops.rglru_prefill(u, yd[:, s], *gates, state, 8.0, fresh=at == 0, out=out[:, s])
            at, i = at + m, i + 1
        err = rel_l2(out[list(rows)], ref)
        assert err < (1e-5 if dtype == F32 else 8e-3), (cuts, err)


@pytest.mark.parametrize("M,N,K", [(1, 100, 64), (3, 264, 256), (8, 48, 1032), (13, 64, 2048), (32, 40, 520), (2, 72, 4096)])
@pytest.mark.parametrize("kind", [0, 1])
@pytest.mark.parametrize("taps", [0, 1, 4, 8])
def test_decode_linear_stream(dev, M, N, K, kind, taps):
    """Three consecutive steps (the ring feeds the convolution), with a gather in front and the gate behind."""
    from based_amd import ops

    x, res, nw = rnd(41, 3, M, K, dtype=BF16), rnd(42, 3, M, K), (1 + 0.1 * rnd(43, K)).to(BF16)
    w, bias = (rnd(44, N, K) * K ** -0.5).to(BF16), rnd(45, N, dtype=BF16)
    cw = (0.3 * rnd(46, max(taps, 1), K)).to(BF16)
    ring = torch.full((M, max(taps, 1), K), float("nan"), dtype=BF16, device=dev)
    norm = (lambda s: O.layer_norm(s, nw.double(), 1e-3)) if kind == ops.NORM_LAYER else (lambda s: O.rms(s, 1e-3) * nw.double())
    past = []
    for t in range(3):
        pos = torch.full((M,), t, dtype=torch.int32, device=dev) if t % 2 else t
        rout = torch.empty(M, K, device=dev)
        kw = dict(prologue=ops.PROLOGUE_STREAM, residual_in=res[t].to(dev), norm_weight=nw.to(dev), eps=1e-3, mult=0.7, norm_kind=kind)
        if taps:
            kw["input_conv"] = (cw.to(dev), ring, pos)
        y = ops.decode_linear(x[t].to(dev), w.to(dev), bias.to(dev), residual_out=rout, **kw)
        s = res[t].double() + 0.7 * x[t].double()
        past.append(norm(s).to(BF16).double())
        h = past[-1]
        if taps:
            h = h + sum(cw[taps - 1 - j].double() * past[t - j] for j in range(min(taps, t + 1)))
        assert rel_l2(rout, s) < 2e-7
        assert rel_l2(y, h @ w.double().T + bias.double()) < 8e-3
    # gather + gate, no residual: the factor does not apply
    table = rnd(47, 50, K, dtype=BF16)
    idx = torch.randint(50, (M,), generator=torch.Generator().manual_seed(1))
    kw = dict(prologue=ops.PROLOGUE_STREAM, norm_weight=nw.to(dev), eps=1e-3, mult=0.7, norm_kind=kind, row_index=idx.to(dev))
    h = norm(table[idx].double()) @ w.double().T
    if K <= 2048:
        y = ops.decode_linear(table.to(dev), w.to(dev), epilogue=ops.EPILOGUE_SWIGLU, **kw)
        h = h[:, :N // 2] * O.silu(h[:, N // 2:])
    else:
        y = ops.decode_linear(table.to(dev), w.to(dev), **kw)
    assert rel_l2(y, h) < 1.5e-2


def test_bad_arguments_are_refused(dev):
    from based_amd import ops

    x = torch.zeros(1, 4, 16, dtype=BF16, device=dev)
    with pytest.raises(ValueError):
        ops.stream_conv(x, torch.zeros(9, 16, dtype=BF16, device=dev))
    with pytest.raises(ValueError):
        ops.stream_conv(x, torch.zeros(3, 16, dtype=BF16, device=dev), ring=torch.zeros(1, 2, 16, dtype=BF16, device=dev))
    cache = torch.zeros(1, 4, 1, 32, dtype=BF16, device=dev)
    with pytest.raises(ValueError):  # the portion runs past the cache
        ops.window_attn_prefill(x, x, x, cache, 1, 1, 4, 1.0, 1, out=torch.empty_like(x))
    with pytest.raises(ValueError):
        ops.window_attn_step(x[:, 0], x[:, 0], x[:, 0], cache, 1, 1, 4, 1.0, 4, out=torch.empty_like(x[:, 0]))
    with pytest.raises(ValueError):
        ops.window_attn_prefill(x.cpu(), x, x, cache, 1, 1, 4, 1.0, 0, out=torch.empty_like(x))
