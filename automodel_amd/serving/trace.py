"""Trace replay: feed given tokens through a model step by step, write logits.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

One JSON object per line on standard input:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}], "end": []}

``entries`` bring each request's next tokens, ``want`` the places among them
whose logits are written to ``DIR/<step>.f32`` (little-endian float32, [wanted,
vocab], in order); ``end`` names the requests that are finished after the step.
``done <step>`` is printed after every step. The requests of a step either all
start or all go on by one token.

Steps run through ``utils/generation.DecodeSession``, the same step function,
cache and kernels that generation uses. Kernels are compiled first if the
checkout holds no built library (inference kernels only).
"""

from __future__ import annotations

import argparse
import json
import os
import sys


def parse_args(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n")[0])
    ap.add_argument("--model", required=True, help="folder with config.json and safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, default=4096,
                    help="most tokens that live requests hold at any time")
    return ap.parse_args(argv)


class TraceReplay:
    """Requests by id on top of a DecodeSession."""

    def __init__(self, model, max_tokens: int):
        self.model, self.max_tokens = model, max_tokens
        self.session = None
        self.capacity = 0
        self.handles: dict[str, int] = {}

    def _start(self, entries) -> "torch.Tensor":
        from automodel_amd.utils.generation import DecodeSession

        if len(entries) + len(self.handles) > self.capacity:
            if self.handles:
                raise ValueError("a new batch starts only after the last one has ended")
            # no sequence can hold more than all of them together
            self.capacity = len(entries)
            self.session = None                     # free the old cache first
            self.session = DecodeSession(self.model, self.capacity, self.max_tokens)
        handles, logits = self.session.prefill([e["tokens"] for e in entries],
                                               [e["want"] for e in entries])
        self.handles.update((e["id"], h) for e, h in zip(entries, handles))
        return logits

    def _go_on(self, entries) -> "torch.Tensor":
        import torch

        if any(len(e["tokens"]) != 1 for e in entries):
            raise ValueError("requests start with their prompt, then go on by one token")
        tokens = torch.tensor([e["tokens"][0] for e in entries], device=self.session.device)
        logits = self.session.decode([self.handles[e["id"]] for e in entries], tokens)
        rows = [i for i, e in enumerate(entries) for _ in e["want"]]
        return logits[rows]

    def step(self, entries: list[dict], end: list[str]):
        """-> logits [wanted, vocab] of the step."""
        known = [e["id"] in self.handles for e in entries]
        if any(known) != all(known):
            raise ValueError("the requests of a step all start or all go on")
        logits = None
        if entries:
            logits = self._go_on(entries) if all(known) else self._start(entries)
        if end:
            self.session.release([self.handles.pop(i) for i in end])
        return logits


def main(argv=None) -> int:
    args = parse_args(argv)
    import torch

    if not torch.cuda.is_available():
        raise RuntimeError("trace_run needs a GPU: there is no CPU path")
    from automodel_amd.ops._backend import so_path

    if not os.path.exists(so_path()):
        from contextlib import redirect_stdout

        from automodel_amd.ops.build import build

        with redirect_stdout(sys.stderr):
            build(decode_only=True)
    from automodel_amd.models.registry import load_pretrained

    if args.dtype == "float32":
        torch.set_float32_matmul_precision("highest")
    model = load_pretrained(args.model, dtype=args.dtype, device="cuda")
    replay = TraceReplay(model, args.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        req = json.loads(line)
        logits = replay.step(req["entries"], req.get("end", []))
        if any(e["want"] for e in req["entries"]):
            path = os.path.join(args.out, f"{req['step']}.f32")
            logits.float().cpu().numpy().astype("<f4").tofile(path)
        print(f"done {req['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
