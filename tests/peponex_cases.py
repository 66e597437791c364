"""Small configurations and random weights of the Peponex design for the tests (made here, nothing is loaded)."""
import torch

from sozilix_cases import logit_error, run_portions, tokens  # noqa: F401  (the same for every design)


def wkv(heads, dim, mlp=None):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}, "mlp": mlp}


def lightning(heads, dim, vdim, decay, mlp=None):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, "mlp": mlp}


def latent(heads, dim, rot, vdim, rank, window, base, scale, mlp=None):
    return {"type": "latent_attention", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "mask": {"size": window},
        "rot": {"base": base, "dims": rot}, "scale": scale}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def config(width, vocab, eps, layers, loop=None, side=None, cap=None):
    cfg = {"architecture": "Peponex", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    if side:
        cfg["token_side"] = {"dim": side}
    if cap:
        cfg["logit_softcap"] = cap
    return cfg


CONFIGS = {
    # every kind of layer and feed-forward, a loop in the middle, value sizes unlike key sizes
    "mixed": config(192, 331, 1e-5, [
        lightning(3, 48, 80, [0.5, 0.97, 0.9995], dense(200)),
        latent(5, 40, 16, 24, 96, 33, 500.0, 0.21, moe(5, 2, 40)),
        wkv(3, 64, moe(6, 1, 72)),
        latent(2, 24, 32, 56, 64, 64, 10000.0, 0.125),
        wkv(5, 32)], loop=(1, 3, 3), side=24, cap=20.0),
    # sizes, counts and factors of 1
    "ones": config(64, 100, 1e-6, [
        wkv(1, 16, moe(1, 1, 8)),
        latent(1, 8, 2, 8, 8, 1, 10000.0, 1.0, dense(8)),
        lightning(1, 16, 16, [1.0])], loop=(0, 3, 1), side=8, cap=5.0),
    # rows that are no whole 16-byte pieces, a decay of zero, as many choices as experts
    "odd": config(84, 77, 1e-3, [
        wkv(3, 20, dense(30)),
        lightning(2, 10, 18, [0.0, 0.9], moe(3, 3, 22)),
        latent(3, 14, 6, 10, 36, 9, 100.0, 0.3, dense(52))], loop=(1, 2, 2), side=5, cap=30.0),
    # larger heads, more than sixteen of them, a window of several rounds of keys; no loop, token input or cap
    "wide": config(128, 96, 1e-5, [
        latent(18, 64, 64, 96, 256, 300, 10000.0, 0.09, moe(4, 2, 64)),
        wkv(1, 128, dense(256)),
        lightning(2, 112, 136, [0.8, 0.995])]),
}

W1_RANK = {"mixed": 24, "ones": 1, "odd": 7, "wide": 40}


def weights(name, seed=0):
    """bf16-representable float64 weights, scaled so that every mechanism reaches the logits.  Embeddings carry marks that the
    routers read: the choice of experts is no close call."""
    cfg = CONFIGS[name]
    g = torch.Generator().manual_seed(seed)
    D, V, dim = cfg["width"], cfg["vocab"], cfg["token_side"]["dim"] if "token_side" in cfg else 0
    w = {}

    def put(key, *shape, std=None, mean=0.0):
        x = mean + torch.randn(*shape, generator=g) * (shape[-1] ** -0.5 if std is None else std)
        w[key] = x.bfloat16().double()

    marks = torch.linalg.qr(torch.randn(D, 8, generator=g))[0].T  # orthonormal rows
    order = torch.stack([torch.randperm(8, generator=g) for _ in range(V)])
    strength = torch.tensor([2.6, 2.0, 1.4, 0.8, 0.2, -0.4, -1.0, -1.6])
    planted = (strength[None] * D ** 0.5 * 0.8)[:, :, None] * marks[order]
    w["embed"] = (0.7 * torch.randn(V, D, generator=g) + planted.sum(1)).bfloat16().double()
    put("head", V, D)
    put("final.norm", D, std=0.2, mean=1.0)
    if "loop" in cfg:
        put("loop.step", cfg["loop"]["times"], D, std=0.5)
    if dim:
        put("side.embed", V, len(cfg["layers"]) * dim, std=1.0)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}", layer["mixer"]
        put(f"{p}.norm1", D, std=0.2, mean=1.0)
        mix = f"{p}.mix"
        if layer["type"] == "wkv":
            n, rank = m["heads"] * m["dim"], W1_RANK[name]
            for s in "rkvgw":
                put(f"{mix}.mu.{s}", D, std=0.3, mean=0.5)
            for s in "rkvg":
                put(f"{mix}.{s}", n, D)
            put(f"{mix}.w1", rank, D)
            put(f"{mix}.w2", n, rank, std=1.5 * rank ** -0.5)
            put(f"{mix}.w0", n, std=2.5, mean=-2.0)
            put(f"{mix}.u", m["heads"], m["dim"], std=1.0)
            put(f"{mix}.norm", n, std=0.2, mean=1.0)
            put(f"{mix}.o", D, n)
        elif layer["type"] == "lightning":
            for s, n in (("q", m["dim"]), ("k", m["dim"]), ("v", m["vdim"]), ("g", m["vdim"])):
                put(f"{mix}.{s}", m["heads"] * n, D)
            put(f"{mix}.norm", m["heads"] * m["vdim"], std=0.2, mean=1.0)
            put(f"{mix}.o", D, m["heads"] * m["vdim"])
        else:
            put(f"{mix}.q", m["heads"] * (m["dim"] + m["rot_dim"]), D, std=2 * D ** -0.5)
            put(f"{mix}.dkv", m["kv_rank"] + m["rot_dim"], D, std=2 * D ** -0.5)
            put(f"{mix}.dkv.norm", m["kv_rank"], std=0.2, mean=1.0)
            put(f"{mix}.uk", m["heads"] * m["dim"], m["kv_rank"])
            put(f"{mix}.uv", m["heads"] * m["vdim"], m["kv_rank"])
            put(f"{mix}.o", D, m["heads"] * m["vdim"])
        mlp = layer["mlp"]
        if mlp:
            put(f"{p}.norm2", D, std=0.05, mean=1.0)
            parts = [f"{p}.mlp"] if mlp["kind"] == "dense" else [f"{p}.mlp.e{e}" for e in range(mlp["router"]["experts"])]
            F = mlp["ff"] if mlp["kind"] == "dense" else mlp["expert"]["ff"]
            for part in parts:
                put(f"{part}.gate", F, D)
                put(f"{part}.up", F, D)
                put(f"{part}.down", D, F)
            if mlp["kind"] == "moe":
                w[f"{p}.mlp.router"] = (marks[:mlp["router"]["experts"]] * 2.0 * D ** -0.5 * 1.5).bfloat16().double()
        if dim:
            put(f"{p}.side.gate", dim, D, std=0.5 * D ** -0.5)
            put(f"{p}.side.proj", D, dim)
            put(f"{p}.side.norm", D, std=0.1, mean=0.5)
    return w


def build(cfg, w, device, dtype):
    from based_amd import architectures
    from based_amd.stack import GPTLMHeadModel, StackConfig

    design = architectures.find(cfg)
    shapes = {name: tuple(t.shape) for name, t in w.items()}
    model = GPTLMHeadModel(StackConfig(**design.stack_config(cfg, shapes)), device=device, dtype=dtype)
    model.load_state_dict(design.convert_state(cfg, w))
    return model.eval()
