"""Whole Peponex models through the framework against the plain statement: prompts, decoding through the
caches, portions, batches, caches used again, long decoding, greedy generation eagerly and under the
decode graph, and the trace replay program."""
import json
import os
import subprocess

import pytest
import torch

import peponex_cases as cases
from oracle import peponex_oracle as O

pytestmark = pytest.mark.gpu
F32, BF16 = torch.float32, torch.bfloat16
LIMIT = {F32: 1e-4, BF16: 6e-2}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
LENGTHS = {"mixed": 150, "ones": 40, "odd": 60, "wide": 330}
CUTS = {"whole": [10 ** 6], "tokens": [1], "twos": [2], "mixed": [33, 2, 3, 31, 2, 5, 1, 1, 1, 17], "tail": [20, 1], "long": [100, 1]}
_made = {}


def case(name, dev, dtype):
    """(config, model, tokens, float64 logits), built once per process."""
    cfg = cases.CONFIGS[name]
    if name not in _made:
        w = cases.weights(name)
        toks = cases.tokens(cfg, LENGTHS[name])
        _made[name] = (w, toks, O.forward(cfg, w, torch.tensor(toks)))
    if (name, dtype) not in _made:
        _made[name, dtype] = cases.build(cfg, _made[name][0], dev, dtype)
    w, toks, ref = _made[name]
    return cfg, _made[name, dtype], toks, ref


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("cuts", sorted(CUTS))
@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_logits_for_every_cut(dev, name, cuts, dtype):
    cfg, model, toks, ref = case(name, dev, dtype)
    err = cases.logit_error(cases.run_portions(model, toks, CUTS[cuts]), ref)
    assert float(err.max()) < LIMIT[dtype], (int(err.argmax()), float(err.max()))


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_residual_after_every_layer_run(dev, dtype):
    cfg, model, toks, _ = case("mixed", dev, dtype)
    want, got = [], []
    O.forward(cfg, _made["mixed"][0], torch.tensor(toks[:50]), want)

    def hook(block, args, kwargs, out):
        hidden, residual = (t.double() for t in out)
        side = block.out_addends()
        if side is not None:
            hidden = O.rms(hidden, side.post_eps) * side.post_weight.double()
        got.append((hidden + residual)[0].cpu())

    handles = [layer.register_forward_hook(hook, with_kwargs=True) for layer in model.transformer.layers]
    try:
        with torch.inference_mode():
            model(torch.tensor([toks[:50]], device=dev))
    finally:
        for h in handles:
            h.remove()
    assert len(got) == len(want) == 9
    for i, (a, b) in enumerate(zip(got, want)):
        assert float((a - b).norm() / b.norm()) < (1e-5 if dtype == F32 else 2e-2), i


@pytest.mark.parametrize("name", ["mixed", "wide"])
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_without_caches_and_general_decode_path(dev, name, dtype):
    cfg, model, toks, ref = case(name, dev, dtype)
    with torch.inference_mode():
        y = model(torch.tensor([toks], device=dev)).logits[0]
    assert float(cases.logit_error(y.cpu(), ref).max()) < LIMIT[dtype]
    model.transformer.fused_decode = False
    try:
        err = cases.logit_error(cases.run_portions(model, toks, [90, 1]), ref)
    finally:
        model.transformer.fused_decode = True
    assert float(err.max()) < LIMIT[dtype]


def test_bf16_decoding_takes_the_fused_path(dev):
    from based_amd.generation import InferenceParams

    for name in ("mixed", "ones", "wide"):
        _, model, _, _ = case(name, dev, BF16)
        params = InferenceParams(max_seqlen=8, max_batch_size=1, seqlen_offset=3)
        with torch.inference_mode():
            assert model.transformer.decode_layers_ok(torch.zeros(1, 1, dtype=torch.long, device=dev), params), name


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_batch_rows_match_each_alone(dev, dtype):
    """Equal lengths together, then rows at unequal positions in one decoding step, few and many of them."""
    from based_amd.generation import InferenceParams

    cfg, model, _, _ = case("mixed", dev, dtype)
    w = _made["mixed"][0]
    seqs = [cases.tokens(cfg, 50, seed=s) for s in (5, 6, 7)]
    refs = [O.forward(cfg, w, torch.tensor(s)) for s in seqs]
    ids = torch.tensor(seqs, device=dev)
    params = InferenceParams(max_seqlen=50, max_batch_size=3)
    with torch.inference_mode():
        for lo, hi in ((0, 21), (21, 23), (23, 24), (24, 50)):
            y = model(ids[:, lo:hi], inference_params=params).logits
            params.seqlen_offset = hi
            for b in range(3):
                assert float(cases.logit_error(y[b].cpu(), refs[b][lo:hi]).max()) < LIMIT[dtype]
        # rows at 13, 40 and 27 tokens (and four of each): prompts one by one into their rows, then together
        for copies in (1, 4):
            B = 3 * copies
            params = InferenceParams(max_seqlen=50, max_batch_size=B)
            at = [13, 40, 27] * copies
            for b in range(B):
                params.seqlen_offset, params.batch_size_offset = 0, b
                model(ids[b % 3:b % 3 + 1, :at[b]], inference_params=params)
            params.batch_size_offset, params.seqlen_offset = 0, max(at)
            params.lengths_per_sample = torch.tensor(at, dtype=torch.int32, device=dev)
            for step in range(6):
                tok = torch.stack([ids[b % 3, at[b] + step] for b in range(B)])[:, None]
                y = model(tok, inference_params=params).logits[:, 0].cpu()
                params.lengths_per_sample += 1
                for b in range(B):
                    want = refs[b % 3][at[b] + step:at[b] + step + 1]
                    assert float(cases.logit_error(y[b:b + 1], want)[0]) < 2 * LIMIT[dtype]


@pytest.mark.parametrize("name", ["mixed", "odd"])
@pytest.mark.parametrize("dtype", [F32, BF16])
def test_caches_used_again(dev, name, dtype):
    """A second request on the caches of a longer first one, filled with values no request may see."""
    from based_amd.replay import Replay

    cfg, model, toks, ref = case(name, dev, dtype)
    n = LENGTHS[name]
    replay = Replay(model, n)
    replay.feed("a", cases.tokens(cfg, n - 10, seed=9), [])
    with torch.inference_mode():
        stores = replay.live["a"].key_value_memory_dict
        assert len(stores) == len(O.layer_runs(cfg))
        for store in stores.values():
            for t in store.values():
                t.fill_(float("nan"))
    replay.end("a")
    got = [replay.feed("b", toks[:2], [0, 1]), replay.feed("b", toks[2:3], [0]), replay.feed("b", toks[3:50], [0, 40])]
    assert len(replay.free) == 0
    err = cases.logit_error(torch.cat(got).cpu(), ref[[0, 1, 2, 3, 43]])
    assert float(err.max()) < LIMIT[dtype] * 1.5


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_long_decoding(dev, dtype):
    cfg, model, _, _ = case("ones", dev, dtype)
    toks = cases.tokens(cfg, 600, seed=12)
    ref = O.forward(cfg, _made["ones"][0], torch.tensor(toks))
    err = cases.logit_error(cases.run_portions(model, toks, [100, 1]), ref)
    assert float(err.max()) < LIMIT[dtype]


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_greedy_generation(dev, name):
    """generate() eagerly and with recorded graphs; float32 picks the tokens of the plain statement."""
    cfg, model, toks, _ = case(name, dev, F32)
    w = _made[name][0]
    prompt, n = toks[:19], 12
    seq = list(prompt)
    margin = []
    for _ in range(n):
        y = O.forward(cfg, w, torch.tensor(seq))[-1]
        top = y.topk(2).values
        margin.append(float(top[0] - top[1]))
        seq.append(int(y.argmax()))
    sure = next((i for i, m in enumerate(margin) if m < 1e-3), n)  # tokens before the first near-tie
    ids = torch.tensor([prompt], device=dev)
    for kw in (dict(cg=False), dict(cg=True, output_scores=True, return_dict_in_generate=True), dict(cg=True), dict(cg=True)):
        out = model.generate(ids, max_length=len(prompt) + n, **kw)
        out = out.sequences if kw.get("return_dict_in_generate") else out
        assert out[0, :len(prompt) + sure].tolist() == seq[:len(prompt) + sure], kw
    # a bf16 model: eager and recorded steps agree with each other, for small and large batches
    _, half, _, _ = case(name, dev, BF16)
    for rows in (2, 12):
        ids = torch.tensor([cases.tokens(cfg, 23, seed=s) for s in range(rows)], device=dev)
        eager = half.generate(ids, max_length=50, cg=False)
        for _ in range(2):
            assert torch.equal(half.generate(ids, max_length=50, cg=True), eager)
    torch.manual_seed(0)
    assert half.generate(ids, max_length=30, top_k=5, temperature=0.8).shape == (12, 30)


@pytest.mark.parametrize("name,dtype", [("mixed", "bfloat16"), ("mixed", "float32"), ("wide", "bfloat16")])
def test_trace_replay_program(dev, tmp_path, name, dtype):
    from safetensors.torch import save_file

    cfg, _, toks, ref = case(name, dev, F32)
    w = _made[name][0]
    model_dir, out_dir = tmp_path / "model", tmp_path / "out"
    model_dir.mkdir()
    out_dir.mkdir()
    (model_dir / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.to(BF16).contiguous() for k, v in w.items()}, str(model_dir / "model.safetensors"))
    steps, want = [], []
    for request in ("a", "b"):
        at = 0
        for n in (60, 2, 1, 1, 70, 1):
            places = [n - 1, 0] if n > 1 else ([0] if at != 62 else [])
            steps.append({"step": len(steps), "entries": [{"id": request, "tokens": toks[at:at + n], "want": places}],
                          "end": [request] if n == 1 and at == 134 else []})
            want.append([at + p for p in places])
            at += n
        steps.append({"step": len(steps), "entries": [{"id": "c" + request, "tokens": toks[:3], "want": []}], "end": ["c" + request]})
        want.append([])
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(model_dir), "--dtype", dtype, "--out", str(out_dir),
                        "--max-tokens", "160"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True,
                       timeout=110)
    assert p.returncode == 0, p.stderr[-2000:]
    done = [l for l in p.stdout.splitlines() if l.startswith("done")]
    assert done == [f"done {i}" for i in range(len(steps))]
    for i, places in enumerate(want):
        path = out_dir / f"{i}.f32"
        assert path.exists() == bool(places)
        if places:
            got = torch.frombuffer(bytearray(path.read_bytes()), dtype=torch.float32).view(len(places), cfg["vocab"])
            assert float(cases.logit_error(got, ref[places]).max()) < 1.5 * LIMIT[getattr(torch, dtype)], i
