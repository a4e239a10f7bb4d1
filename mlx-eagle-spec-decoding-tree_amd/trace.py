"""Trace runner: replays given token ids through a model, step by step, and writes logits.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come on standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

`want`: places among an entry's tokens whose logits are asked for; `end`: requests that are finished
after the step.  Logits of a step go to OUT/<step>.f32 (little-endian fp32, [wanted, vocab], in the order
of the entries); after every step the line `done <step>` is printed.  Requests run on the streams that
`generate` uses; a finished request's stream is cleared and serves the next one.

Exit codes: 0 after the end of the input, 2 for bad arguments, 3 when the model's family does not run in
the asked storage type.
"""
import argparse
import json
import os
import sys


class Requests:
    """Streams of the live requests.  open_stream: () -> a new one."""

    def __init__(self, open_stream):
        self.open_stream, self.live, self.idle = open_stream, {}, []

    def stream(self, rid):
        if rid not in self.live:
            s = self.idle.pop() if self.idle else self.open_stream()
            s.clear()
            self.live[rid] = s
        return self.live[rid]

    def end(self, rid):
        s = self.live.pop(rid, None)
        if s is not None:
            self.idle.append(s)


def run_step(requests, step):
    """Feed a step's tokens; the wanted logits as one fp32 numpy array, or None."""
    import numpy as np

    parts = []
    for e in step["entries"]:
        want = e.get("want") or []
        logits = requests.stream(e["id"]).feed(e["tokens"], want=want)
        if want:
            parts.append(logits.float().cpu().numpy())
    for rid in step.get("end", ()):
        requests.end(rid)
    return np.concatenate(parts) if parts else None


def storage_type(family, name):
    """The family's name for a trace's dtype, or None: "bfloat16" stands for whatever 16-bit type the
    family is served in."""
    if name in family.dtypes:
        return name
    return family.dtypes[0] if name == "bfloat16" else None


def main(argv=None, stdin=None, stdout=None):
    ap = argparse.ArgumentParser(prog="trace_run", description="replay token ids and write logits")
    ap.add_argument("--model", required=True)
    ap.add_argument("--dtype", required=True, choices=("bfloat16", "float32"))
    ap.add_argument("--out", required=True)
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time")
    opt = ap.parse_args(argv)
    stdin, stdout = stdin or sys.stdin, stdout or sys.stdout

    from . import build, checkpoint, registry
    family = registry.resolve(checkpoint.load_config(opt.model))
    dtype = storage_type(family, opt.dtype)
    if dtype is None:
        print(f"the {family.name} family does not run in {opt.dtype}", file=sys.stderr)
        return 3
    build.build_missing(family.libraries)

    import torch
    from .generate import open_stream
    model, _ = checkpoint.load_model(opt.model, torch.device("cuda:0"), dtype=dtype)
    requests = Requests(lambda: open_stream(model, max(1, opt.max_tokens)))
    with torch.inference_mode():
        for line in stdin:
            if not line.strip():
                continue
            step = json.loads(line)
            logits = run_step(requests, step)
            if logits is not None:
                path = os.path.join(opt.out, f"{step['step']}.f32")
                logits.astype("<f4").tofile(path + ".part")
                os.replace(path + ".part", path)
            print(f"done {step['step']}", file=stdout, flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
