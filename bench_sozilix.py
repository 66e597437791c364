"""`bench.py --only sozilix`: the streamed layers beside the closest operations of the Based models at equal
size, and a 27-layer model of each (random weights, bf16).

Every operation is timed inside a recorded graph over several independent input / output sets visited
in turn (more bytes than the 256 MB last-level cache holds, where the sizes allow it).  `frac` prices
its algorithmic bytes against 8 TB/s or its fp32 products against the fp32 matrix peak, whichever bound
is the longer one; the figure of the like operation is its own, priced the same way."""
from __future__ import annotations

import time

HBM_PEAK = 8000.0e9
FP32_PEAK = 157.3e12   # fp32 matrix and (packed) vector peak, published
BF16_PEAK = 2500.0e12


def _graph_ms(torch, fn, n_sets, replays=8):
    """Milliseconds per launch of fn(set), recorded once over all sets."""
    side = torch.cuda.Stream()
    side.wait_stream(torch.cuda.current_stream())
    with torch.cuda.stream(side):
        for i in range(n_sets):
            fn(i)
        side.synchronize()
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(graph, stream=side):
            for i in range(n_sets):
                fn(i)
    torch.cuda.current_stream().wait_stream(side)
    for _ in range(3):
        graph.replay()
    e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    e0.record()
    for _ in range(replays):
        graph.replay()
    e1.record()
    torch.cuda.synchronize()
    return e0.elapsed_time(e1) / (replays * n_sets)


def _entry(ms, nbytes=0, fp32_flop=0, bf16_flop=0, **more):
    limits = {"hbm": nbytes / HBM_PEAK, "fp32": fp32_flop / FP32_PEAK, "bf16 mfma": bf16_flop / BF16_PEAK}
    bound = max(limits, key=limits.get)
    return {"us": round(ms * 1e3, 2), "bound": bound, "roofline_us": round(limits[bound] * 1e6, 2),
            "frac": round(limits[bound] / (ms * 1e-3), 4), **more}


def bench_kernels(torch, ops, B=8, L=4096, D=1024, decode_B=128):
    dev = torch.device("cuda:0")
    bf = torch.bfloat16
    rnd = lambda *s: torch.randn(*s, device=dev, dtype=bf)
    out = {}
    N = B * L

    def pair(name, ours, like_name, like):
        out[name] = {**ours, "like": {"op": like_name, **like}, "distance_ratio": round(like["frac"] / ours["frac"], 2)}

    # norm with the residual sum
    n = 3
    xs, rs, w = [rnd(N, D) for _ in range(n)], [torch.randn(N, D, device=dev) for _ in range(n)], rnd(D)
    ln = _entry(_graph_ms(torch, lambda i: ops.add_norm(xs[i], rs[i], w, 1e-5, ops.NORM_LAYER, 0.7), n), N * D * 12)
    rms = _entry(_graph_ms(torch, lambda i: ops.add_rms_norm(xs[i], rs[i], w, 1e-5), n), N * D * 12)
    pair("add_norm B*L=%d D=%d" % (N, D), ln, "add_rms_norm", rms)
    del rs
    # causal convolution against the gated one (whose projection is twice as wide)
    xs3 = [x.view(B, L, D) for x in xs]
    cw = rnd(4, D)
    ring = torch.zeros(B, 4, D, device=dev, dtype=bf)
    sc = _entry(_graph_ms(torch, lambda i: ops.stream_conv(xs3[i], cw, None, ring, 0, add_input=True), n), N * D * 4)
    us = [rnd(B, L, 2 * D) for _ in range(n)]
    gw, gb = rnd(D, 1, 4), rnd(D)
    gc = _entry(_graph_ms(torch, lambda i: ops.gated_conv_prefill(us[i], gw, gb), n), N * D * 6)
    pair("stream_conv taps=4", sc, "gated_conv_prefill", gc)
    # linear recurrent unit
    blocks = 8
    gates = [rnd(blocks, D // blocks, D // blocks), rnd(D), rnd(blocks, D // blocks, D // blocks), rnd(D), rnd(D) - 3]
    st = torch.zeros(B, D, device=dev)
    ys = [rnd(B, L, D) for _ in range(n)]
    o = torch.empty(B, L, D, device=dev, dtype=bf)
    ms = _graph_ms(torch, lambda i: ops.rglru_prefill(xs3[i], ys[i], *gates, st, 8.0, True, out=o), n)
    # both launches together: u, y, out once, the fp32 decay and input written and read
    pair("rglru_prefill W=%d blocks=%d" % (D, blocks), _entry(ms, N * D * (2 + 8 + 8 + 2 + 2), algorithmic_min_bytes=N * D * 6),
         "gated_conv_prefill", gc)
    del us, ys, o
    # window attention, 129 keys per query (128 to the left), rotary, cache filled
    H, d = 16, 64
    ang = torch.outer(torch.arange(L, device=dev).float(), 10000.0 ** (-torch.arange(0, d, 2, device=dev).float() / d))
    rope = (ang.cos().contiguous(), ang.sin().contiguous())
    qkv = [rnd(B, L, 3, H, d) for _ in range(n)]
    caches = [torch.empty(B, L, 2, H, d, device=dev, dtype=bf) for _ in range(n)]
    outs = [torch.empty(B, L, H, d, device=dev, dtype=bf) for _ in range(n)]
    ms = _graph_ms(torch, lambda i: ops.swa_prefill(qkv[i][:, :, 0], qkv[i][:, :, 1], qkv[i][:, :, 2], w_left=128, rope=rope,
                                                    kv_cache=caches[i], out=outs[i]), n)
    swa = _entry(ms, N * H * d * 2 * 6, bf16_flop=N * H * 129 * 4 * d)
    for G in (16, 4):
        kvs = [torch.empty(B, L, G, 2 * d, device=dev, dtype=bf) for _ in range(n)]
        parts = [x.view(B, L, 3 * H * d) for x in qkv]
        fn = lambda i: ops.window_attn_prefill(parts[i][..., :H * d], parts[i][..., H * d:H * d + G * d],
                                               parts[i][..., 2 * H * d:2 * H * d + G * d], kvs[i], H, G, 129, 0.125, 0,
                                               rope=(*rope, True), value_norm_eps=1e-5, out=outs[i].view(B, L, H * d))
        # q, o and the new k, v rows once; the cache rows written and, being the operand of the second launch, read
        nbytes = N * 2 * (2 * H * d + 2 * G * d + 2 * 2 * G * d)
        pair("window_attn_prefill H=%d G=%d d=%d window=129" % (H, G, d), _entry(_graph_ms(torch, fn, n), nbytes, bf16_flop=N * H * 129 * 4 * d),
             "swa_prefill (rotary, cache)", swa)
    del qkv, caches, outs, parts, kvs
    # delta rule against Taylor linear attention
    ql = [rnd(B, H, L, 16) for _ in range(n)]
    vl = [rnd(B, H, L, 64) for _ in range(n)]
    lin = _entry(_graph_ms(torch, lambda i: ops.linear_attn_prefill(ql[i], ql[i], vl[i], return_state=True), n),
                 N * H * (2 * 16 + 2 * 64) * 2, bf16_flop=N * H * (2 * 2 * 153 * 65 + 64 * (2 * 16 + 2 * 64)))
    del ql, vl
    for H2, d2, dv2 in ((8, 128, 128), (16, 64, 64)):
        c = [rnd(B, L, H2 * (2 * d2 + dv2)) for _ in range(2)]
        ab = rnd(B, L, 2 * H2)
        al, db = rnd(H2), rnd(H2)
        st = torch.zeros(B, H2, d2, dv2, device=dev)
        nk = H2 * d2
        fn = lambda i: ops.gated_delta_scan(c[i][..., :nk], c[i][..., nk:2 * nk], c[i][..., 2 * nk:], ab[..., :H2], ab[..., H2:], al, db, st,
                                            H2, H2, True)
        # S^T k, S^T q and the update: three products of d x dv
        pair("gated_delta_scan H=%d d=%d dv=%d" % (H2, d2, dv2),
             _entry(_graph_ms(torch, fn, 2), N * H2 * ((2 * d2 + dv2) * 2 + dv2 * 4), fp32_flop=N * H2 * 6 * d2 * dv2),
             "linear_attn_prefill H=16 dv=64", lin)
        o = torch.randn(B, L, H2, dv2, device=dev)
        gate, y = rnd(B, L, H2 * dv2), torch.empty(B, L, H2 * dv2, device=dev, dtype=bf)
        wn = rnd(dv2)
        ms = _graph_ms(torch, lambda i: ops.gated_rms_norm(o, wn, gate, 1e-5, out=y), 1)
        pair("gated_rms_norm H=%d dv=%d (one set)" % (H2, dv2), _entry(ms, N * H2 * dv2 * 8), "add_rms_norm", rms)
        del c, o, gate, y
    # ---- single-token steps ----
    M, n = decode_B, 8
    pos = torch.full((M,), 1000, dtype=torch.int32, device=dev)
    q1, k1, v1 = rnd(M, H * d), rnd(M, H * d), rnd(M, H * d)
    kvs = [rnd(M, 1024, 16, 2 * d) for _ in range(2)]
    o1 = torch.empty(M, H * d, device=dev, dtype=bf)
    c5 = [x.view(M, 1024, 2, H, d) for x in kvs]
    fn = lambda i: ops.swa_step(q1.view(M, 1, H, d), k1.view(M, 1, H, d), v1.view(M, 1, H, d), c5[i], pos, w_left=128, rope=rope,
                                out=o1.view(M, 1, H, d))
    swa1 = _entry(_graph_ms(torch, fn, 2), M * H * d * 2 * (2 * 129 + 4))
    fn = lambda i: ops.window_attn_step(q1, k1, v1, kvs[i], H, H, 129, 0.125, pos, rope=(*rope, True), value_norm_eps=1e-5, out=o1)
    pair("window_attn_step B=%d H=16 G=16 window=129" % M, _entry(_graph_ms(torch, fn, 2), M * H * d * 2 * (2 * 129 + 4)), "swa_step", swa1)
    G = 4
    kv4 = [x.view(M, 4096, 4, 2 * d)[:, :1024] for x in kvs]
    fn = lambda i: ops.window_attn_step(q1, k1[:, :G * d], v1[:, :G * d], kv4[i], H, G, 129, 0.125, pos, rope=(*rope, True),
                                        value_norm_eps=1e-5, out=o1)
    pair("window_attn_step B=%d H=16 G=4 window=129" % M,
         _entry(_graph_ms(torch, fn, 2), M * 2 * d * (2 * G * 129 + 2 * H + 2 * G)), "swa_step", swa1)
    # the grouped form again with as many bytes per launch as the ungrouped one
    M4 = 4 * M
    q4, k4, pos4 = rnd(M4, H * d), rnd(M4, G * d), torch.full((M4,), 1000, dtype=torch.int32, device=dev)
    o4 = torch.empty(M4, H * d, device=dev, dtype=bf)
    kvb = [x.view(M4, 1024, 4, 2 * d) for x in kvs]
    fn = lambda i: ops.window_attn_step(q4, k4, k4, kvb[i], H, G, 129, 0.125, pos4, rope=(*rope, True), value_norm_eps=1e-5, out=o4)
    pair("window_attn_step B=%d H=16 G=4 window=129" % M4,
         _entry(_graph_ms(torch, fn, 2), M4 * 2 * d * (2 * G * 129 + 2 * H + 2 * G)), "swa_step", swa1)
    del kvs, c5, kv4, kvb
    kvst = [torch.zeros(M, 16, 1, 64, 273, device=dev) for _ in range(3)]
    kst = torch.ones(M, 16, 1, 1, 273, device=dev)
    q2, v2 = rnd(M, 16, 1, 16), rnd(M, 16, 1, 64)
    lin1 = _entry(_graph_ms(torch, lambda i: ops.linear_attn_step(q2, q2, v2, kvst[i], kst), 3), M * 16 * (2 * 273 * 65 * 4 + 320))
    del kvst
    for H2, d2, dv2 in ((8, 128, 128), (16, 64, 64)):
        C = H2 * (2 * d2 + dv2)
        sts = [torch.zeros(M, H2, d2, dv2, device=dev) for _ in range(n)]
        ring = torch.zeros(M, 4, C, device=dev, dtype=bf)
        x, cw, ab, g, y = rnd(M, C), rnd(4, C), rnd(M, 2 * H2), rnd(M, H2 * dv2), torch.empty(M, H2 * dv2, device=dev, dtype=bf)
        al, db, wn = rnd(H2), rnd(H2), rnd(dv2)
        fn = lambda i: ops.gated_delta_step(x, cw, ring, ab[:, :H2], ab[:, H2:], g, al, db, wn, sts[i], H2, H2, d2, dv2, H2 * d2, 2 * H2 * d2,
                                            pos, 1e-5, out=y)
        pair("gated_delta_step B=%d H=%d d=%d dv=%d" % (M, H2, d2, dv2),
             _entry(_graph_ms(torch, fn, n), M * (H2 * d2 * dv2 * 8 + C * 2 * 5 + H2 * dv2 * 4)), "linear_attn_step H=16 dv=64", lin1)
        del sts, ring
    ring = torch.zeros(M, 4, D, device=dev, dtype=bf)
    st = torch.zeros(M, D, device=dev)
    x, y, cw, cb, o = rnd(M, D), rnd(M, D), rnd(4, D), rnd(D), torch.empty(M, D, device=dev, dtype=bf)
    ms = _graph_ms(torch, lambda i: ops.rglru_step(x, y, cw, cb, ring, *gates, st, 8.0, pos, out=o), 8)
    u2, gst = rnd(M, 2 * D), torch.zeros(M, D, 4, device=dev, dtype=bf)
    gs = _entry(_graph_ms(torch, lambda i: ops.gated_conv_step(u2, gst, gw, gb), 8), M * D * (6 + 2 * 8) + D * 10)
    pair("rglru_step B=%d W=%d blocks=%d" % (M, D, blocks), _entry(ms, M * D * (6 + 8 + 8) + D * (2 * 2 * D // blocks + 16)),
         "gated_conv_step", gs)
    # projections of a single token
    M = 4
    Nw, n = 4096, 48
    ws = [rnd(Nw, D) for _ in range(n)]
    x, res, ro, nw = rnd(M, D), torch.randn(M, D, device=dev), torch.empty(M, D, device=dev), rnd(D)
    cw, ring = rnd(4, D), torch.zeros(M, 4, D, device=dev, dtype=bf)
    nbytes = Nw * D * 2
    for name, conv, epi in (("norm", None, ops.EPILOGUE_NONE), ("norm + input conv", (cw, ring, pos), ops.EPILOGUE_NONE),
                            ("norm + gate", None, ops.EPILOGUE_SWIGLU)):
        a = _graph_ms(torch, lambda i: ops.decode_linear(x, ws[i], prologue=ops.PROLOGUE_STREAM, residual_in=res, residual_out=ro,
                                                         norm_weight=nw, mult=0.7, norm_kind=ops.NORM_LAYER, input_conv=conv, epilogue=epi), n)
        b = _graph_ms(torch, lambda i: ops.decode_linear(x, ws[i], prologue=ops.PROLOGUE_ADD_RMS_NORM, residual_in=res, residual_out=ro,
                                                         norm_weight=nw, epilogue=epi), n)
        pair("decode_linear_stream 4096x1024 M=4, %s" % name, _entry(a, nbytes), "decode_linear (RMS norm)", _entry(b, nbytes))
    return out


def sozilix_config(D=1024, layers=27, vocab=50280, ff=2048):
    """A model of the Based-360m's width, depth and feed-forward: two recurrent layers, then a parallel one."""
    rec = {"type": "rglru", "mixer": {"width": D, "blocks": 8, "conv": 4}, "mlp": {"kind": "dense", "ff": ff}}
    par = {"type": "parallel", "mlp": {"kind": "dense", "ff": ff}, "mixer": {
        "left": {"heads": 16, "kv_heads": 4, "dim": 64, "vdim": 64, "mask": {"size": 129}, "rot": {"base": 10000.0, "dims": 32},
                 "scale": 0.125}, "left_scale": 0.7, "right_scale": 0.7,
        "right": {"heads": 8, "kv_heads": 8, "dim": 64, "vdim": 128, "conv": 4}}}
    return {"architecture": "Sozilix", "width": D, "vocab": vocab, "canon": {"taps": 4}, "norm": {"eps": 1e-5}, "residual_mult": 0.5,
            "layers": [par if i % 3 == 2 else rec for i in range(layers)]}


def model_configs():
    """Name -> function that makes the StackConfig of the two models."""
    from based_amd import architectures
    from based_amd.stack import StackConfig, based_360m_config

    raw = sozilix_config()
    return {"sozilix": lambda: StackConfig(**architectures.find(raw).stack_config(raw)), "based_360m": based_360m_config}


def bench_models(torch, makes, B=4, prefill_len=2048, new_tokens=128):
    """Prefill and greedy decoding (recorded graph) of every model, and decoding at batch 32."""
    from based_amd.stack import GPTLMHeadModel

    dev = torch.device("cuda:0")
    out = {"B": B, "prefill_len": prefill_len, "new_tokens": new_tokens}
    for name, make in makes.items():
        torch.manual_seed(0)
        model = GPTLMHeadModel(make(), device=dev, dtype=torch.bfloat16).eval()
        ids = torch.randint(0, 50000, (B, prefill_len), dtype=torch.long, device=dev)
        r = {"parameters_M": round(sum(p.numel() for p in model.parameters()) / 1e6, 1)}
        with torch.inference_mode():
            for _ in range(2):
                model(ids, num_last_tokens=1)
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            for _ in range(3):
                model(ids, num_last_tokens=1)
            torch.cuda.synchronize()
            r["prefill_ms"] = (time.perf_counter() - t0) * 1e3 / 3
            r["prefill_tok_s"] = B * prefill_len / (r["prefill_ms"] * 1e-3)
        for b in (B, 32):
            prompt = ids[:1, :64].expand(b, -1).contiguous()
            times = []
            for n in (8, 8 + new_tokens):  # the difference of two lengths: prefill and set-up drop out
                model.generate(prompt, max_length=64 + 8 + new_tokens, cg=True)
                torch.cuda.synchronize()
                t0 = time.perf_counter()
                model.generate(prompt, max_length=64 + n, cg=True)
                torch.cuda.synchronize()
                times.append(time.perf_counter() - t0)
            ms = (times[1] - times[0]) * 1e3 / new_tokens
            r[f"decode_B{b}_ms_per_token"], r[f"decode_B{b}_tok_s"] = ms, b / (ms * 1e-3)
        out[name] = {k: round(v, 3) for k, v in r.items()}
        del model
        torch.cuda.empty_cache()
    return out


def bench(torch):
    from based_amd import ops

    with torch.inference_mode():
        kernels = bench_kernels(torch, ops)
    torch.cuda.empty_cache()
    return {"kernels": kernels, "models": bench_models(torch, model_configs())}
