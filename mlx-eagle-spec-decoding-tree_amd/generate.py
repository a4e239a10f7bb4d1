"""Plain autoregressive generation, one token per pass, greedy, for every model family of the
registry: the entry point for a model that is served without a drafter (with one:
`spec.SpeculativeDecoder`).

    python -m mlx_eagle_spec_decoding_tree_amd.generate --model DIR --tokens 1,2,3 --max-tokens 32

Token ids in, token ids out (there is no tokenizer in this package).  A stream is one sequence:
`feed(ids, want)` appends tokens in portions of any size and returns logits at the wanted places,
`pick(logits)` selects a token, `greedy(token, n)` continues on the device, `clear()` starts the next sequence in the same buffers.
"""
import argparse
import json
import os
import sys
import time

import torch

from . import registry


class LlamaStream:
    """Stream over the quantised decoder: prompt passes of `spec.CausalPrefill` when only the last logits
    are wanted, the module path otherwise; one-row `spec.DecoderPass` for the continuation."""

    MAX_OUT = 8192

    def __init__(self, model, capacity, graphs=True):
        from .cache import make_prompt_cache

        # prompt passes are padded to 32 rows beyond the last token
        self.model, self.graphs, self.capacity = model, graphs, int(capacity)
        self.cache = make_prompt_cache(model, capacity=(self.capacity + 63) // 32 * 32)
        self.vocab_size = model.args.vocab_size
        self._prefill = self._pass = self._graph = None

    @property
    def length(self):
        return self.cache[0].offset

    def clear(self):
        self._set_length(0)

    def _set_length(self, n):
        for c in self.cache:
            c.offset = n
        self.cache[0].sync_len()

    def _check(self, n):
        if self.length + n > self.capacity:
            raise ValueError(f"a cache of {self.capacity} tokens has no room for {n} more at length {self.length}")

    def feed(self, ids, want=None):
        from . import spec

        ids = torch.as_tensor(ids).reshape(-1).to(self.model.device, torch.int64)
        n = ids.numel()
        if n == 0 or int(ids.min()) < 0 or int(ids.max()) >= self.vocab_size:
            raise ValueError(f"token ids must lie in 0..{self.vocab_size - 1}")
        self._check(n)
        if (want is None or list(want) == [n - 1]) and n > 1:
            if self._prefill is None:
                self._prefill = spec.CausalPrefill(self.model, self.cache, chunk=spec.MAX_CHUNK, graphs=False)
            return self._prefill(ids).float()
        rows = [n - 1] if want is None else [int(w) for w in want]
        logits = self.model(ids[None], cache=self.cache)[0]
        self.cache[0].sync_len()
        return logits[rows].float()

    def pick(self, logits):
        """Token id of the largest logit of the last row."""
        from . import ops
        return int(ops.argmax_rows(logits[-1:].half()).item())

    def _step(self):
        from . import _lib, ops

        L, st, length = _lib.lib(), torch.cuda.current_stream().cuda_stream, self.cache[0].len_dev
        _lib.check(L.eagle_tree_positions(self._zero.data_ptr(), length.data_ptr(), self._pos.data_ptr(), 1, st), "positions")
        logits = self._pass.forward(self._y, self._pos, length, length, self._mask, 1)
        ops.argmax_rows(logits, out=self._y)
        _lib.check(L.eagle_advance_len(length.data_ptr(), 1, st), "advance_len")

    def _prepare_step(self):
        from . import ops, spec

        i32 = dict(dtype=torch.int32, device=self.model.device)
        self._pass = spec.DecoderPass(self.model, self.cache, 1)
        self._y, self._zero, self._pos = torch.zeros(1, **i32), torch.zeros(1, **i32), torch.zeros(1, **i32)
        self._mask = ops.mask_to_words(torch.ones((1, 1), dtype=torch.bool, device=self.model.device))
        self._out = torch.zeros(self.MAX_OUT, **i32)
        if not self.graphs:
            return
        # the warm-up run writes one cache row beyond the length and advances the length
        length = self.cache[0].len_dev
        saved = length.clone()
        side = torch.cuda.Stream()
        side.wait_stream(torch.cuda.current_stream())
        with torch.cuda.stream(side):
            self._step()
        torch.cuda.current_stream().wait_stream(side)
        torch.cuda.synchronize()
        self._graph = torch.cuda.CUDAGraph()
        with torch.cuda.graph(self._graph):
            self._step()
        length.copy_(saved)

    def greedy(self, token, n):
        self._check(n)
        if n > self.MAX_OUT:
            return (first := self.greedy(token, self.MAX_OUT)) + self.greedy(first[-1], n - self.MAX_OUT)
        self.cache[0].sync_len()
        if self._pass is None:
            self._prepare_step()
        self._y.fill_(int(token))
        for i in range(n):
            if self._graph is not None:
                self._graph.replay()
            else:
                self._step()
            self._out[i:i + 1].copy_(self._y)
        self._set_length(self.length + n)
        return self._out[:n].tolist()


def open_stream(model, capacity, graphs=True):
    """A stream for one sequence of up to `capacity` tokens."""
    if hasattr(model, "stream"):
        return model.stream(capacity, graphs)
    return LlamaStream(model, capacity, graphs)


def generate(model, prompt, max_tokens, prefill_step_size=2048, stream=None):
    """Greedy continuation of `prompt` (token ids): the list of max_tokens tokens.  stream: an open one to
    reuse (cleared first)."""
    prompt = [int(t) for t in torch.as_tensor(prompt).reshape(-1).tolist()]
    if max_tokens < 1:
        return []
    if stream is None:
        stream = open_stream(model, len(prompt) + max_tokens)
    stream.clear()
    for s in range(0, len(prompt), prefill_step_size):
        logits = stream.feed(prompt[s:s + prefill_step_size])
    first = stream.pick(logits)
    return [first] + (stream.greedy(first, max_tokens - 1) if max_tokens > 1 else [])


def main(argv=None):
    from . import build, checkpoint

    ap = argparse.ArgumentParser(prog="generate", description="greedy generation from token ids")
    ap.add_argument("--model", required=True, help="folder with config.json and safetensors")
    ap.add_argument("--tokens", required=True, help="prompt token ids with commas between them, or @FILE")
    ap.add_argument("--max-tokens", type=int, default=32)
    ap.add_argument("--dtype", help=f"storage type (default: the one the family is served in; families: "
                                    f"{', '.join(registry.names())})")
    ap.add_argument("--prefill-step-size", type=int, default=2048)
    opt = ap.parse_args(argv)
    text = open(opt.tokens[1:]).read() if opt.tokens.startswith("@") else opt.tokens
    prompt = [int(t) for t in text.replace(",", " ").split()]
    build.build_missing(registry.resolve(checkpoint.load_config(opt.model)).libraries)
    model, _ = checkpoint.load_model(opt.model, torch.device("cuda:0"), dtype=opt.dtype)
    t0 = time.perf_counter()
    tokens = generate(model, prompt, opt.max_tokens, opt.prefill_step_size)
    torch.cuda.synchronize()
    print(json.dumps({"tokens": tokens, "prompt_tokens": len(prompt), "seconds": round(time.perf_counter() - t0, 4)}))
    return 0


if __name__ == "__main__":
    sys.exit(main())
