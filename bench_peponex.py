"""`bench.py --only peponex`: the operations of the Peponex layers beside the closest operations of the
framework's other models at equal size, and a 27-run model beside theirs (random weights, bf16).

Timing and pricing as in bench_sozilix.py.  A product whose operands the design keeps in 32 bits (recurrences)
is priced at the fp32 matrix peak, others at the bf16 peak; `frac` is the longer bound over the time."""
from __future__ import annotations

import bench_sozilix
from bench_sozilix import _entry, _graph_ms


def bench_kernels(torch, ops, B=8, L=4096, D=1024):
    import torch.nn.functional as F

    dev = torch.device("cuda:0")
    bf = torch.bfloat16
    rnd = lambda *s: torch.randn(*s, device=dev, dtype=bf)
    out = {}
    N = B * L

    def time(fn, n=2):
        return _graph_ms(torch, fn, n)

    def pair(name, ours, like_name, like):
        out[name] = {**ours, "like": {"op": like_name, **like}, "distance_ratio": round(like["frac"] / ours["frac"], 2)}

    # ---- element-wise work of prompts ----
    xs, rs, w = [rnd(N, D) for _ in range(2)], [torch.randn(N, D, device=dev) for _ in range(2)], rnd(D)
    norm = _entry(time(lambda i: ops.add_rms_norm(xs[i], rs[i], w, 1e-5)), N * D * 12)
    table, idx = rnd(1000, D), torch.randint(1000, (N,), device=dev)
    add = ops.Addends(post_weight=w, post_eps=1e-5, vec=w, table=table, index=idx)
    pair("add_norm with addends B*L=%d D=%d" % (N, D),
         _entry(time(lambda i: ops.add_norm(xs[i], rs[i], w, 1e-5, ops.NORM_RMS, addends=add)), N * D * 12), "add_rms_norm", norm)
    del rs
    xs3, mu = [x.view(B, L, D) for x in xs], rnd(5, D)
    cw, ring = rnd(4, D), torch.zeros(B, 4, D, device=dev, dtype=bf)
    conv = _entry(time(lambda i: ops.stream_conv(xs3[i], cw, None, ring, 0, add_input=True)), N * D * 4)
    pair("token_mix 5 mixes", _entry(time(lambda i: ops.token_mix(xs3[i], mu)), N * D * 12), "stream_conv taps=4", conv)
    hid, w2, w0 = [rnd(B, L, 64) for _ in range(2)], rnd(D, 64), rnd(D)
    pair("channel_decay rank=64 C=%d" % D, _entry(time(lambda i: ops.channel_decay(hid[i], w2, w0)), N * (128 + 4 * D)), "add_rms_norm", norm)
    y = torch.empty(B, L, D, device=dev, dtype=bf)
    for G in (16, 1):
        pair("group_norm_gate groups=%d" % G,
             _entry(time(lambda i: ops.group_norm_gate(xs3[i], w, xs3[1 - i], G, 1e-5, ops.ACT_SIGMOID, out=y)), N * D * 6), "add_rms_norm", norm)
    del y, hid

    # ---- recurrences over prompts ----
    for H, d in ((16, 64), (8, 128)):
        q, k, v = ([rnd(B, L, H * d) for _ in range(2)] for _ in range(3))
        lw, u = [-torch.exp(torch.randn(B, L, H * d, device=dev) - 4) for _ in range(2)], rnd(H, d)
        st, hd = torch.zeros(B, H, d, d, device=dev), ops.head_decays([0.99] * H, dev)
        c, ab = [rnd(B, L, 3 * H * d) for _ in range(2)], rnd(B, L, 2 * H)
        al, db, nk = rnd(H), rnd(H), H * d
        delta = _entry(time(lambda i: ops.gated_delta_scan(c[i][..., :nk], c[i][..., nk:2 * nk], c[i][..., 2 * nk:], ab[..., :H], ab[..., H:], al,
                                                           db, st, H, H, True)), N * H * (3 * d * 2 + d * 4), fp32_flop=N * H * 6 * d * d)
        pair("decay_scan per channel H=%d d=%d" % (H, d),
             _entry(time(lambda i: ops.decay_scan(q[i], k[i], v[i], st, H, channel_log2=lw[i], bonus=u, fresh=True)),
                    N * H * d * 12, fp32_flop=N * H * 4 * d * d), "gated_delta_scan", delta)
        pair("decay_scan per head H=%d d=%d" % (H, d),
             _entry(time(lambda i: ops.decay_scan(q[i], k[i], v[i], st, H, head_decay=hd, activation=ops.ACT_SILU, fresh=True)),
                    N * H * d * 8, fp32_flop=N * H * 4 * d * d), "gated_delta_scan", delta)
        del q, k, v, lw, c

    # ---- latent attention over prompts, against window attention with as many heads of its own ----
    H, d, r, dv, R = 16, 64, 32, 64, 256
    turn = lambda n: torch.outer(torch.arange(L, device=dev).float(), 10000.0 ** (-torch.arange(0, n, 2, device=dev).float() / n))
    rope = (turn(r).cos().contiguous(), turn(r).sin().contiguous(), False)
    lat, cache, nw = [rnd(B, L, R + r) for _ in range(2)], torch.empty(B, L, R + r, device=dev, dtype=bf), rnd(R)
    pair("latent_write R=%d rot=%d" % (R, r), _entry(time(lambda i: ops.latent_write(lat[i], nw, cache, 0, 1e-5, rope)), N * (R + r) * 4),
         "add_rms_norm", norm)
    ew = rnd(H * (r + d + dv), R + r)
    kv = [F.linear(cache, ew).view(B, L, H, -1) for _ in range(2)]
    q, o = [rnd(B, L, H * (r + d)) for _ in range(2)], torch.empty(B, L, H * dv, device=dev, dtype=bf)
    q64, kv64, o64 = [rnd(B, L, H * 64) for _ in range(2)], [torch.empty(B, L, H, 128, device=dev, dtype=bf) for _ in range(2)], torch.empty_like(o)
    rope64 = (turn(32).cos().contiguous(), turn(32).sin().contiguous(), True)
    for W in (129, 1024):
        like = _entry(time(lambda i: ops.window_attn_prefill(q64[i], q64[i], q64[i], kv64[i], H, H, W, 0.125, 0, rope=rope64, out=o64)),
                      N * H * 2 * (4 * 64 + 2 * 128), bf16_flop=N * H * W * 4 * 64)
        pair("window_attn_attend on expanded latents window=%d" % W,
             _entry(time(lambda i: ops.window_attn_attend(q[i], kv[i], H, H, r + d, W, 0.1, 0, rope, out=o)),
                    N * H * 2 * (2 * (r + d) + 2 * dv), bf16_flop=N * H * W * 2 * (r + d + dv)), "window_attn_prefill H=16 d=64", like)
    del kv, q, q64, kv64, lat

    # ---- experts over prompts, against the dense feed-forward of the same products ----
    h, fc1, fc2 = rnd(N, D), rnd(4096, D) * 0.03, rnd(D, 2048) * 0.03
    for n in (N, 2048):
        dense = _entry(time(lambda i: F.linear(ops.swiglu(F.linear(h[:n], fc1)), fc2)), n * D * 4 + 3 * 2048 * D * 2, bf16_flop=n * 6 * 2048 * D)
        for E, top, ff in ((8, 1, 2048), (8, 2, 1024), (64, 4, 512)):
            router, w1, w2 = rnd(E, D), rnd(E, 2 * ff, D) * 0.03, rnd(E, D, ff) * 0.03
            pair("experts %d of %d ff=%d n=%d" % (top, E, ff, n),
                 _entry(time(lambda i: ops.experts(h[:n], router, w1, w2, top)), n * D * 4 + E * 3 * ff * D * 2, bf16_flop=n * top * 6 * ff * D),
                 "fc1 + swiglu + fc2 ff=2048", dense)
    del h

    # ---- single tokens ----
    for M in (4, 128):
        pos = torch.full((M,), 2000, dtype=torch.int32, device=dev)
        for H2, d2 in ((16, 64), (8, 128)):
            n = 8
            st = [torch.zeros(M, H2, d2, d2, device=dev) for _ in range(n)]
            a, hid, w2, w0, u = rnd(4, M, H2 * d2), rnd(M, 64), rnd(H2 * d2, 64), rnd(H2 * d2), rnd(H2, d2)
            nw2, o1, hd = rnd(H2 * d2), torch.empty(M, H2 * d2, device=dev, dtype=bf), ops.head_decays([0.99] * H2, dev)
            C = 3 * H2 * d2
            x, cw, ring, ab, al, wn = rnd(M, C), rnd(4, C), torch.zeros(M, 4, C, device=dev, dtype=bf), rnd(M, 2 * H2), rnd(H2), rnd(d2)
            delta = _entry(time(lambda i: ops.gated_delta_step(x, cw, ring, ab[:, :H2], ab[:, H2:], a[0], al, al, wn, st[i], H2, H2, d2, d2, H2 * d2,
                                                               2 * H2 * d2, pos, 1e-5, out=o1), n), M * (H2 * d2 * d2 * 8 + C * 10 + H2 * d2 * 4))
            pair("decay_step per channel B=%d H=%d d=%d" % (M, H2, d2),
                 _entry(time(lambda i: ops.decay_step(a[0], a[1], a[2], st[i], H2, pos, bonus=u, hidden=hid, w2=w2, w0=w0, gate=a[3],
                                                      norm_weight=nw2, eps=1e-5, out=o1), n), M * (H2 * d2 * d2 * 8 + H2 * d2 * 10)),
                 "gated_delta_step", delta)
            pair("decay_step per head B=%d H=%d d=%d" % (M, H2, d2),
                 _entry(time(lambda i: ops.decay_step(a[0], a[1], a[2], st[i], H2, pos, head_decay=hd, activation=ops.ACT_SILU, out=o1), n),
                        M * (H2 * d2 * d2 * 8 + H2 * d2 * 8)), "gated_delta_step", delta)
            del st
        for W in (129, 1024):
            S = 2048
            cc, kvg = [rnd(M, S, R + r) for _ in range(2)], [rnd(M, S, 4, 128) for _ in range(2)]
            q1, x1, o1 = rnd(M, H * (r + d)), rnd(M, R + r), torch.empty(M, H * dv, device=dev, dtype=bf)
            kv1 = rnd(M, 256)
            like = _entry(time(lambda i: ops.window_attn_step(q1[:, :1024], kv1, kv1, kvg[i], H, 4, W, 0.125, pos, rope=rope64, out=o1)),
                          M * 2 * (W * 4 * 128 + 2 * H * 64))
            pair("latent_step B=%d H=%d R=%d window=%d" % (M, H, R, W),
                 _entry(time(lambda i: ops.latent_step(q1, x1, nw, ew, cc[i], H, d, W, 0.1, pos, 1e-5, rope, out=o1)),
                        M * 2 * (W * (R + r) + H * (r + d + dv)) + H * (d + dv) * R * 2), "window_attn_step H=16 G=4 d=64", like)
            del cc, kvg
    M, n = 4, 24
    pos = torch.full((M,), 1000, dtype=torch.int32, device=dev)
    x, res, ro, nw = rnd(M, D), torch.randn(M, D, device=dev), torch.empty(M, D, device=dev), rnd(D)
    ws = [rnd(4096 + 64, D) for _ in range(n)]
    rows = dict(residual_in=res, residual_out=ro, norm_weight=nw)
    like = _entry(time(lambda i: ops.decode_linear(x, ws[i], prologue=ops.PROLOGUE_ADD_RMS_NORM, **rows), n), ws[0].numel() * 2)
    tok = torch.arange(M, device=dev)
    add = ops.Addends(post_weight=nw, post_eps=1e-5, vec=nw, table=table, index=tok)
    ring = torch.zeros(M, 2, D, device=dev, dtype=bf)
    more = dict(prologue=ops.PROLOGUE_STREAM, norm_kind=ops.NORM_RMS, **rows)
    for name, kw in (("addends", dict(addends=add)), ("addends + 5 token mixes", dict(addends=add, mix=(mu, ring, pos, 1024))),
                     ("addends + cap", dict(addends=add, softcap=30.0))):
        pair("decode_linear 4160x1024 M=4, norm + %s" % name, _entry(time(lambda i: ops.decode_linear(x, ws[i], **more, **kw), n), ws[0].numel() * 2),
             "decode_linear (RMS norm)", like)
    sg, sp, st = [rnd(64, D) for _ in range(n)], [rnd(D, 64) for _ in range(n)], rnd(1000, 64)
    for M in (4, 32):
        x, res, ro, tok = rnd(M, D), torch.randn(M, D, device=dev), torch.empty(M, D, device=dev), torch.arange(M, device=dev)

        def small(i):
            ops.decode_linear(ops.decode_linear(x, sg[i], prologue=ops.PROLOGUE_ADD_RMS_NORM, residual_in=res, residual_out=ro, norm_weight=nw),
                              sp[i])

        pair("token_side_step 64 of 1024 M=%d" % M, _entry(time(lambda i: ops.token_side_step(x, res, ro, sg[i], sp[i], st, tok), n), 4 * 64 * D),
             "decode_linear 64x1024 (RMS norm), 1024x64", _entry(time(small, n), 4 * 64 * D))
    for M in (4, 32):
        x, res, ro = rnd(M, D), torch.randn(M, D, device=dev), torch.empty(M, D, device=dev)
        f1, f2 = [rnd(4096, D) for _ in range(12)], [rnd(D, 2048) for _ in range(12)]

        def dense(i):
            ops.decode_linear(ops.decode_linear(x, f1[i], prologue=ops.PROLOGUE_ADD_RMS_NORM, residual_in=res, residual_out=ro, norm_weight=nw,
                                                epilogue=ops.EPILOGUE_SWIGLU), f2[i])

        like = _entry(time(dense, 12), 3 * 2048 * D * 2)
        del f1, f2
        for E, top, ff in ((8, 1, 2048), (8, 2, 1024), (64, 4, 512)):
            router = rnd(E, D)
            ww = [(rnd(E, 2 * ff, D) * 0.03, rnd(E, D, ff) * 0.03) for _ in range(4)]
            s = (ops.add_norm(x, res, nw, 1e-5, ops.NORM_RMS)[0].float() @ router.float().T).topk(top).indices
            used = int(s.unique().numel())  # experts whose matrices this batch reads
            pair("experts behind their norm, %d of %d ff=%d M=%d (%d read)" % (top, E, ff, M, used),
                 _entry(time(lambda i: ops.experts(x, router, *ww[i], top, norm=(res, ro, nw, 1e-5, ops.NORM_RMS, 1.0)), 4), used * 3 * ff * D * 2),
                 "decode_linear norm + fc1 + gate, fc2 (ff=2048)", like)
            del ww
    return out


def peponex_config(D=1024, vocab=50280, ff=2048):
    """A model of the Based-360m's width, runs of layers and products per token: nine times a time-mixing, a decaying and a latent
    layer, three of the layers run twice, every third feed-forward a mixture of two of eight experts of half the size."""
    dense, moe = {"kind": "dense", "ff": ff}, {"kind": "moe", "expert": {"ff": ff // 2}, "router": {"experts": 8, "top": 2}}
    kinds = [
        {"type": "wkv", "mixer": {"heads": 16, "dim": 64}},
        {"type": "lightning", "mixer": {"heads": 16, "dim": 64, "vdim": 64, "decay": [1 - 2.0 ** (-2 - 8 * h / 15) for h in range(16)]}},
        {"type": "latent_attention", "mixer": {"heads": 16, "dim": 64, "rot_dim": 32, "vdim": 64, "kv_rank": 256, "mask": {"size": 512},
                                               "rot": {"base": 10000.0, "dims": 32}, "scale": 96 ** -0.5}}]
    return {"architecture": "Peponex", "width": D, "vocab": vocab, "norm": {"eps": 1e-5}, "token_side": {"dim": 64}, "logit_softcap": 30.0,
            "loop": {"start": 3, "stop": 6, "times": 2}, "layers": [{**kinds[i % 3], "mlp": moe if i % 3 == 1 else dense} for i in range(24)]}


def bench(torch):
    from based_amd import architectures, ops
    from based_amd.stack import StackConfig

    with torch.inference_mode():
        kernels = bench_kernels(torch, ops)
    torch.cuda.empty_cache()
    raw = peponex_config()
    shapes = {f"l{i}.mix.w1": (64, raw["width"]) for i in range(len(raw["layers"]))}
    makes = {"peponex": lambda: StackConfig(**architectures.find(raw).stack_config(raw, shapes)), **bench_sozilix.model_configs()}
    return {"kernels": kernels, "models": bench_sozilix.bench_models(torch, makes)}
