"""Replays a trace of token portions through a model, step by step, and writes logits.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N < steps

Steps come from standard input, one JSON object per line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

Every entry is the next portion of a request; `want` lists the places in it whose logits are written,
as little-endian 32-bit floats [wanted, vocab] in the order of the entries, to DIR/<step>.f32.
Requests in `end` are finished and their caches go back to the pool.  "done <step>" follows every step.
Nothing is sampled; the model, its caches and its step function are those of `based_amd.generation`.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

DTYPES = ("bfloat16", "float32")


class Replay:
    """Live requests of one model, each with its inference parameters; finished ones are used again."""

    def __init__(self, model, max_tokens: int):
        self.model, self.max_tokens = model, max_tokens
        self.live, self.free = {}, []
        self.device = next(model.parameters()).device

    def _params(self, name):
        from .generation import InferenceParams

        if name not in self.live:
            if self.free:
                params = self.free.pop()
                params.reset(self.max_tokens, 1)
            else:
                params = InferenceParams(max_seqlen=self.max_tokens, max_batch_size=1)
            self.live[name] = params
        return self.live[name]

    def feed(self, name, tokens, want):
        """Runs the next portion of a request; the logits at `want`, (len(want), vocab) float32 on the device."""
        import torch

        params = self._params(name)
        if params.seqlen_offset + len(tokens) > self.max_tokens:
            raise ValueError(f"request {name!r} outgrows {self.max_tokens} tokens")
        ids = torch.tensor([tokens], dtype=torch.long, device=self.device)
        places = torch.tensor(want if len(tokens) > 1 else [0], dtype=torch.long, device=self.device)
        with torch.inference_mode():
            logits = self.model(ids, inference_params=params, logits_at=places).logits[0].float()
        params.seqlen_offset += len(tokens)
        return logits if len(tokens) > 1 else logits[want]

    def end(self, name):
        params = self.live.pop(name, None)
        if params is not None:
            self.free.append(params)


def _ready_kernels() -> None:
    """The whole library where it has been built, otherwise the part that streamed models need."""
    from . import _lib, build

    if not os.path.exists(_lib.LIB_PATH):
        if not os.path.exists(_lib.part_path("streaming")):
            build.build_part("streaming")
        _lib.use_part("streaming")


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="Replays a trace of token portions through a model and writes logits.")
    ap.add_argument("--model", required=True, help="folder with config.json and the weights")
    ap.add_argument("--dtype", required=True, choices=DTYPES)
    ap.add_argument("--out", required=True, help="folder for the <step>.f32 files")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time")
    args = ap.parse_args(argv)
    _ready_kernels()
    import torch

    from .stack import GPTLMHeadModel

    torch.set_float32_matmul_precision("highest")
    model = GPTLMHeadModel.from_pretrained_local(args.model, device="cuda:0", dtype=getattr(torch, args.dtype)).eval()
    replay = Replay(model, args.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = [replay.feed(e["id"], e["tokens"], e["want"]) for e in step["entries"]]
        wanted = [r for r in rows if r.shape[0]]
        if wanted:
            data = torch.cat(wanted).cpu().numpy().astype("<f4").tobytes()
            path = os.path.join(args.out, f"{step['step']}.f32")
            with open(path + ".part", "wb") as f:
                f.write(data)
            os.replace(path + ".part", path)
        else:
            torch.cuda.synchronize()
        for name in step["end"]:
            replay.end(name)
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
