"""Decoder whose layers choose their mixer (linear attention, latent attention) and feed-forward, with
unquantised weights in bf16 or fp32, a fp32 residual stream, learned positions and a tied output
head; the passes it runs in and the runner that feeds a sequence through them.

`Model(inputs, cache)` has the call of `llama.Model`; caches come from `cache.make_prompt_cache(model)`.
"""
from dataclasses import dataclass, field
from typing import List, Optional

import torch

from . import hybrid_ops as hops
from .cache import PromptCache
from .hybrid_ops import round_up
from .llama import Module
from .mixers import MIXERS, STEP_ROWS, FeedForward, FeedForwardSpec, Layout

# Row counts passes are laid out for; a portion runs in the smallest that holds it (the rows that are
# not there cost a launch's idle workgroups).
PASS_ROWS = (1, 2, STEP_ROWS, 16, 64, 128, 256, 512, 1024, 2048)


@dataclass
class LayerSpec:
    mixer: object
    mlp: Optional[FeedForwardSpec]


@dataclass
class HybridArgs:
    model_type: str
    vocab_size: int
    width: int
    max_positions: int
    norm_eps: float
    embed_scale: float
    layers: List[LayerSpec] = field(default_factory=list)

    @property
    def num_hidden_layers(self):
        return len(self.layers)


class Layer(Module):
    """x <- x + mixer(norm1(x)), then x <- x + ff(norm2(x)) where there is a feed-forward."""

    def __init__(self, spec, tensors, layout):
        pick = lambda prefix: {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}
        self.mixer = MIXERS[type(spec.mixer)](spec.mixer, pick("mix."), layout)
        self.norm1 = layout.norm_around_one(tensors["norm1"])
        self.mlp = self.norm2 = None
        if spec.mlp is not None:
            self.mlp = FeedForward(spec.mlp, pick("mlp."), layout)
            self.norm2 = layout.norm_around_one(tensors["norm2"])

    @staticmethod
    def shapes(spec, width):
        out = {f"mix.{k}": v for k, v in MIXERS[type(spec.mixer)].shapes(spec.mixer, width).items()}
        out["norm1"] = (width,)
        if spec.mlp is not None:
            out.update({f"mlp.{k}": v for k, v in FeedForward.shapes(spec.mlp, width).items()})
            out["norm2"] = (width,)
        return out

    def emit(self, p, cache):
        self.mixer.emit(p, cache, self.norm1)
        if self.mlp is not None:
            self.mlp.emit(p, self.norm2)


class Model(Module):
    """tensors: {"embed", "pos", "final.norm", "layers": [per layer {"norm1", "mix.*", "norm2", "mlp.*"}]}."""

    def __init__(self, args: HybridArgs, tensors, device, dtype=torch.bfloat16):
        hops.code(dtype)
        self.args, self.device, self.dtype = args, torch.device(device), dtype
        self.model_type = args.model_type
        self.layout = layout = Layout(args.width, args.norm_eps, dtype, self.device)
        Dp = layout.padded_width
        # the table serves the embedding and, without its scale, the output head
        self.embed_tokens = layout.weight(tensors["embed"], round_up(args.vocab_size, 16), Dp)
        self.positions = layout.weight(tensors["pos"], args.max_positions, Dp)
        self.layers = [Layer(s, t, layout) for s, t in zip(args.layers, tensors["layers"])]
        self.norm = layout.norm_around_one(tensors["final.norm"])

    @staticmethod
    def shapes(args):
        """{"embed", ..., "layers": [{name: shape}]} of the tensors a checkpoint has to hold."""
        D = args.width
        return {"embed": (args.vocab_size, D), "pos": (args.max_positions, D), "final.norm": (D,),
                "layers": [Layer.shapes(s, D) for s in args.layers]}

    def make_cache(self, capacity):
        """One entry per layer; a layer that reads another layer's latents shares its entry."""
        capacity = min(int(capacity), self.args.max_positions)
        if capacity < 1:
            raise ValueError("capacity must be positive")
        len_dev = torch.zeros(1, dtype=torch.int32, device=self.device)
        out = PromptCache()
        for spec, layer in zip(self.args.layers, self.layers):
            src = getattr(spec.mixer, "kv_from", None)
            out.append(out[src] if src is not None else layer.mixer.new_cache(capacity, self.layout, len_dev))
        return out

    def stream(self, capacity, graphs=True):
        return HybridRunner(self, self.make_cache(capacity), graphs)

    def __call__(self, inputs, cache=None, mask=None, position_ids=None, flat_rope=False):
        """Logits [1, L, vocab] (fp32) of L tokens appended to `cache`, causal."""
        if cache is None:
            raise NotImplementedError("the decoder always runs with a cache")
        if mask is not None or position_ids is not None or flat_rope:
            raise NotImplementedError("a recurrent layer takes tokens in sequence order only")
        if inputs.dim() != 2 or inputs.shape[0] != 1:
            raise ValueError("batch size 1 only")
        if cache.runner is None:
            cache.runner = HybridRunner(self, cache, graphs=False)
        return cache.runner.feed(inputs[0], want=range(inputs.shape[1]))[None]


class HybridPass:
    """A pass of up to R rows: tokens -> residual stream `h` [R, width] and updated caches.  The
    buffers are static and the lengths live on the device, so the launches can be captured."""

    def __init__(self, model, cache, R):
        self.model, self.cache, self.R = model, cache, R
        self.rows = R if R <= STEP_ROWS else round_up(R, hops.CHUNK)
        dev = model.device
        self.len_dev = cache[0].len_dev
        self.n_dev = torch.zeros(1, dtype=torch.int32, device=dev)      # live rows
        self.tokens = torch.zeros(R, dtype=torch.int32, device=dev)
        self._buffers = {}
        Dp = model.layout.padded_width
        self.h = torch.zeros((self.rows, Dp), dtype=torch.float32, device=dev)
        self.hn = torch.zeros((self.rows, Dp), dtype=model.dtype, device=dev)
        self.graph, self.uses = None, 0

    def buffer(self, name, cols, dtype=None, rows=None):
        """A zero-initialised matrix owned by the pass; layers of one shape share it."""
        key = (name, cols, rows)
        if key not in self._buffers:
            self._buffers[key] = torch.zeros((rows or self.rows, cols), dtype=dtype or self.model.dtype,
                                             device=self.model.device)
        return self._buffers[key]

    def bytes(self, name, n):
        key = (name, n)
        if key not in self._buffers:
            self._buffers[key] = torch.zeros(max(n, 16), dtype=torch.uint8, device=self.model.device)
        return self._buffers[key]

    def project(self, w, norm, out, epilogue=hops.OUT_T):
        """out = epilogue(norm(h) w^T); the norm is part of the product where the form allows it."""
        m = self.model
        eps, d = m.args.norm_eps, m.args.width
        if self.R <= STEP_ROWS and hops.dense_form(m.dtype, self.R, w.shape[1], norm=True) == hops.ROWS:
            hops.dense(self.h, w, out, epilogue, M=self.R, n_dev=self.n_dev, norm=(norm, eps, d))
        else:
            hops.norm_rows(self.h, norm, eps, d, self.hn, n_dev=self.n_dev)
            hops.dense(self.hn, w, out, epilogue, M=self.R, n_dev=self.n_dev)

    def enqueue(self, tap=None):
        """tap(i, h): called after layer i (eager runs: tests that follow the residual stream)."""
        m = self.model
        hops.embed(self.tokens, m.embed_tokens, m.args.embed_scale, m.positions, self.len_dev, self.n_dev,
                   m.args.vocab_size, self.h[:self.R])
        for i, (layer, c) in enumerate(zip(m.layers, self.cache)):
            layer.emit(self, c)
            if tap is not None:
                tap(i, self.h)
        hops.advance_len(self.len_dev, self.n_dev, self.cache[0].capacity)

    def run(self, graphs):
        """Captured at its second use: a row count that comes up once is not worth a capture."""
        self.uses += 1
        if graphs and self.graph is None and self.uses > 1:
            self.graph = capture(self.enqueue, [self.n_dev])
        if self.graph is not None:
            self.graph.replay()
        else:
            self.enqueue()


def capture(enqueue, live):
    """HIP graph of `enqueue`.  The warm-up run happens with no live rows (`live`: the counters), so
    that it touches no cache or state."""
    saved = [t.clone() for t in live]
    for t in live:
        t.zero_()
    side = torch.cuda.Stream()
    side.wait_stream(torch.cuda.current_stream())
    with torch.cuda.stream(side):
        enqueue()
    torch.cuda.current_stream().wait_stream(side)
    torch.cuda.synchronize()
    graph = torch.cuda.CUDAGraph()
    with torch.cuda.graph(graph):
        enqueue()
    for t, s in zip(live, saved):
        t.copy_(s)
    return graph


class HybridRunner:
    """Feeds the tokens of one sequence through a model in portions of any size and continues it
    greedily (the stream interface of `generate`)."""

    MAX_OUT = 8192

    def __init__(self, model, cache, graphs=True):
        hops.check_device(model.device)
        self.model, self.cache, self.graphs = model, cache, graphs
        self.capacity = cache[0].capacity
        self.vocab_size = model.args.vocab_size
        self.passes = {}
        self._decode = None

    @property
    def length(self):
        return self.cache[0].offset

    def clear(self):
        """Forget the sequence; the buffers serve the next one."""
        self.cache.clear()

    def _pass(self, n):
        R = next(r for r in PASS_ROWS if r >= n)
        if R not in self.passes:
            self.passes[R] = HybridPass(self.model, self.cache, R)
        return self.passes[R]

    def _advance(self, n):
        for c in {id(c): c for c in self.cache}.values():
            c.offset = c.offset + n

    def _check_ids(self, ids):
        ids = torch.as_tensor(ids).reshape(-1).to(device="cpu", dtype=torch.int32)
        if ids.numel() == 0:
            raise ValueError("no tokens")
        if int(ids.min()) < 0 or int(ids.max()) >= self.vocab_size:
            raise ValueError(f"token ids must lie in 0..{self.vocab_size - 1}")
        if self.length + ids.numel() > self.capacity:
            raise ValueError(f"a cache of {self.capacity} tokens has no room for {ids.numel()} more at length {self.length}")
        return ids

    def feed(self, ids, want=None, tap=None):
        """Append tokens; fp32 logits [len(want), vocab] at the places `want` among them (default: the
        last), on the device.  tap(start, i, h): residual stream of the portion's rows after layer i."""
        ids = self._check_ids(ids)
        n = ids.numel()
        want = [n - 1] if want is None else [int(w) for w in want]
        if any(w < 0 or w >= n for w in want):
            raise ValueError("want must name places among the tokens")
        m = self.model
        Vp = m.embed_tokens.shape[0]
        logits = torch.empty((len(want), Vp), dtype=torch.float32, device=m.device)
        s = 0
        while s < n:
            part = ids[s:s + PASS_ROWS[-1]]
            k = part.numel()
            p = self._pass(k)
            p.tokens[:k].copy_(part)
            p.n_dev.fill_(k)
            if tap is not None:
                p.enqueue(lambda i, h: tap(s, i, h[:k]))
            else:
                p.run(self.graphs)
            here = [j for j, w in enumerate(want) if s <= w < s + k]
            if here:
                rows = torch.tensor([want[j] - s for j in here], dtype=torch.int32, device=m.device)
                got = self._head(p, rows)
                if len(here) == len(want):
                    logits = got
                else:
                    logits[torch.tensor(here, device=m.device)] = got
            self._advance(k)
            s += k
        return logits[:, :self.vocab_size]

    def _head(self, p, rows):
        """Final norm and output head of the given rows of a pass."""
        m = self.model
        hn = torch.empty((rows.numel(), p.hn.shape[1]), dtype=m.dtype, device=m.device)
        hops.norm_rows(p.h, m.norm, m.args.norm_eps, m.args.width, hn, rows=rows)
        out = torch.empty((rows.numel(), m.embed_tokens.shape[0]), dtype=torch.float32, device=m.device)
        return hops.dense(hn, m.embed_tokens, out, hops.OUT_F32)

    def pick(self, logits):
        """Token id of the largest logit of the last row."""
        out = torch.empty(1, dtype=torch.int32, device=self.model.device)
        return int(hops.argmax_rows(logits[-1:], out).item())

    def greedy(self, token, n):
        """The n tokens after `token` (not yet fed), each the argmax of the logits before it.  The loop
        state stays on the device: n graph replays and one copy back."""
        self._check_ids([token] * n)
        if n > self.MAX_OUT:
            return (first := self.greedy(token, self.MAX_OUT)) + self.greedy(first[-1], n - self.MAX_OUT)
        if self._decode is None:
            self._decode = DecodeStep(self._pass(1), self.MAX_OUT)
        tokens = self._decode.run(token, n, self.graphs)
        self._advance(n)
        return tokens


class DecodeStep:
    """One decoded token with everything on the device: pass of one row, final norm and head in one
    product, argmax, the token as the next input."""

    def __init__(self, p, max_out):
        self.p = p
        i32 = dict(dtype=torch.int32, device=p.model.device)
        self.next, self.count = torch.zeros(1, **i32), torch.zeros(1, **i32)
        self.out = torch.zeros(max_out, **i32)
        self.logits = torch.zeros((1, p.model.embed_tokens.shape[0]), dtype=torch.float32, device=p.model.device)
        self.graph = None

    def enqueue(self):
        p, m = self.p, self.p.model
        p.enqueue()
        p.project(m.embed_tokens, m.norm, self.logits, hops.OUT_F32)
        hops.argmax_rows(self.logits[:, :m.args.vocab_size], self.next)
        hops.token_advance(self.next, p.tokens, self.out, self.count)

    def run(self, token, n, graphs=True):
        self.p.n_dev.fill_(1)
        if graphs and self.graph is None:
            self.graph = capture(self.enqueue, [self.p.n_dev])
        self.p.tokens.fill_(int(token))
        self.count.zero_()
        for _ in range(n):
            if self.graph is not None:
                self.graph.replay()
            else:
                self.enqueue()
        return self.out[:n].tolist()
