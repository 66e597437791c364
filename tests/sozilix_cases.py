"""Small configurations and random weights of the Sozilix design for the tests (made here, nothing is loaded)."""
import torch


def rglru(width, blocks, conv, ff=None):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}, "mlp": ff and {"kind": "dense", "ff": ff}}


def parallel(heads, kv, dim, vdim, window, rot, base, scale, rheads, rkv, rdim, rvdim, conv, ls, rs, ff=None):
    return {"type": "parallel", "mlp": ff and {"kind": "dense", "ff": ff}, "mixer": {
        "left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "mask": {"size": window},
                 "rot": {"base": base, "dims": rot}, "scale": scale},
        "left_scale": ls, "right_scale": rs,
        "right": {"heads": rheads, "kv_heads": rkv, "dim": rdim, "vdim": rvdim, "conv": conv}}}


def config(width, vocab, taps, eps, m, layers):
    return {"architecture": "Sozilix", "width": width, "vocab": vocab, "canon": {"taps": taps}, "norm": {"eps": eps},
            "residual_mult": m, "layers": layers}


CONFIGS = {
    # both kinds of layers, with and without a feed-forward; groups of 3 and 2; value sizes unlike key sizes
    "mixed": config(192, 331, 3, 1e-5, 0.6, [
        parallel(6, 2, 48, 32, 24, 32, 500.0, 0.2, 6, 3, 48, 96, 3, 1.3, 0.7, ff=200),
        rglru(96, 3, 4, ff=136),
        rglru(224, 1, 2),
        parallel(4, 1, 64, 64, 65, 64, 10000.0, 0.125, 2, 1, 128, 32, 4, 0.5, 1.5)]),
    # sizes and factors of 1
    "ones": config(64, 100, 1, 1e-6, 1.0, [
        parallel(1, 1, 16, 16, 1, 2, 10000.0, 1.0, 1, 1, 16, 16, 1, 1.0, 1.0, ff=8),
        rglru(64, 1, 1),
        rglru(8, 8, 3, ff=64)]),
    # rows that are no whole 16-byte pieces
    "odd": config(84, 77, 5, 1e-3, 0.9, [
        rglru(36, 3, 3, ff=52),
        parallel(6, 3, 20, 12, 9, 6, 100.0, 0.3, 4, 2, 12, 20, 5, 0.9, 1.1, ff=30),
        rglru(54, 2, 6)]),
    # larger heads, several heads per group, a window longer than a round of keys
    "wide": config(128, 96, 4, 1e-5, 0.5, [
        parallel(10, 2, 96, 160, 300, 48, 10000.0, 0.1, 3, 1, 160, 200, 4, 1.0, 0.8),
        rglru(640, 2, 4, ff=256)]),
}


def weights(cfg, seed=0):
    """bf16-representable float64 weights, scaled so that every mechanism reaches the logits."""
    g = torch.Generator().manual_seed(seed)
    D = cfg["width"]
    w = {}

    def put(name, *shape, std=None, mean=0.0):
        x = mean + torch.randn(*shape, generator=g) * (shape[-1] ** -0.5 if std is None else std)
        w[name] = x.bfloat16().double()

    put("embed", cfg["vocab"], D, std=1.0)
    put("head", cfg["vocab"], D)
    put("final.norm", D, std=0.2, mean=1.0)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}", layer["mixer"]
        put(f"{p}.norm1", D, std=0.2, mean=1.0)
        put(f"{p}.canon1", D, cfg["canon"]["taps"], std=0.3)
        if layer["type"] == "rglru":
            W, n = m["width"], m["width"] // m["blocks"]
            for name in "yx":
                put(f"{p}.mix.{name}", W, D)
                put(f"{p}.mix.{name}.b", W, std=0.2)
            put(f"{p}.mix.conv", W, m["conv"], std=0.6)
            put(f"{p}.mix.conv.b", W, std=0.1)
            for name in ("ra", "ri"):
                put(f"{p}.mix.{name}", m["blocks"], n, n)
                put(f"{p}.mix.{name}.b", m["blocks"], n, std=1.0)
            put(f"{p}.mix.lam", W, std=1.5, mean=-3.0)
            put(f"{p}.mix.o", D, W)
        else:
            l, r = m["left"], m["right"]
            put(f"{p}.mix.left.q", l["heads"] * l["dim"], D, std=2 * D ** -0.5)
            put(f"{p}.mix.left.k", l["kv_heads"] * l["dim"], D, std=2 * D ** -0.5)
            put(f"{p}.mix.left.v", l["kv_heads"] * l["vdim"], D)
            put(f"{p}.mix.left.o", D, l["heads"] * l["vdim"])
            for name, n in (("q", r["kv_heads"] * r["dim"]), ("k", r["kv_heads"] * r["dim"]), ("v", r["heads"] * r["vdim"])):
                put(f"{p}.mix.right.{name}", n, D)
                put(f"{p}.mix.right.{name}.conv", n, r["conv"], std=0.6)
            put(f"{p}.mix.right.b", r["heads"], D)
            put(f"{p}.mix.right.a", r["heads"], D)
            put(f"{p}.mix.right.A_log", r["heads"], std=1.0, mean=-2.0)
            put(f"{p}.mix.right.dt_bias", r["heads"], std=0.7, mean=-2.0)
            put(f"{p}.mix.right.norm", r["vdim"], std=0.2, mean=1.0)
            put(f"{p}.mix.right.g", r["heads"] * r["vdim"], D)
            put(f"{p}.mix.right.o", D, r["heads"] * r["vdim"])
        if layer["mlp"]:
            F = layer["mlp"]["ff"]
            put(f"{p}.norm2", D, std=0.2, mean=1.0)
            put(f"{p}.mlp.gate", F, D)
            put(f"{p}.mlp.up", F, D)
            put(f"{p}.mlp.down", D, F)
    return w


def tokens(cfg, n, seed=1):
    return torch.randint(cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def build(cfg, w, device, dtype):
    from based_amd import architectures
    from based_amd.stack import GPTLMHeadModel, StackConfig

    model = GPTLMHeadModel(StackConfig(**architectures.find(cfg).stack_config(cfg)), device=device, dtype=dtype)
    model.load_state_dict(architectures.find(cfg).convert_state(cfg, w))
    return model.eval()


def run_portions(model, toks, cuts, params=None):
    """Logits of every position, the tokens fed in portions of the sizes in `cuts` (the last one repeated)."""
    from based_amd.generation import InferenceParams

    dev = next(model.parameters()).device
    params = params or InferenceParams(max_seqlen=len(toks), max_batch_size=1)
    out, at, i = [], 0, 0
    with torch.inference_mode():
        while at < len(toks):
            n = min(cuts[min(i, len(cuts) - 1)], len(toks) - at)
            ids = torch.tensor([toks[at:at + n]], device=dev)
            out.append(model(ids, inference_params=params).logits[0].float())
            params.seqlen_offset += n
            at, i = at + n, i + 1
    return torch.cat(out).cpu().double()


def logit_error(got, ref):
    """Root mean square of the difference over the vocabulary, means taken off, per position, against the spread of ref."""
    d = got.double() - ref
    d = d - d.mean(-1, keepdim=True)
    return (d * d).mean(-1).sqrt() / (ref - ref.mean(-1, keepdim=True)).std()
