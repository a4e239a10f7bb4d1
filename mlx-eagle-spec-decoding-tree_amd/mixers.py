"""Building blocks of decoders with unquantised weights: gated linear attention, latent attention and
a dense feed-forward, each with its sizes and constants as parameters, its own weight layout, its
own sequence state and its launch sequence on a pass object (`hybrid.HybridPass`).

Layout: inner dimensions are padded to 64, value heads to 16 and attention query / key heads to 32
columns with zero weights (exact: a pad column of every product is zero), and the projections that
read the same input are one matrix.
"""
from dataclasses import dataclass
from typing import Optional

import torch

from . import hybrid_ops as hops
from .cache import LatentCache, RecurrentState
from .hybrid_ops import round_up
from .llama import Module

STEP_ROWS = 4        # rows up to which the recurrence walks token by token and norms fold into products
ABSORB_ROWS = 16     # rows up to which latent attention runs on absorbed queries
UNBOUNDED = 1 << 30  # window size of plain causal attention
RANKS = [64 * n for n in (1, 2, 3, 4, 5, 6, 7, 8, 12, 16)]


@dataclass
class LinearAttentionSpec:
    """Gated linear attention: decay sigmoid(z)^(1 / tau) per key channel."""
    heads: int
    dim: int
    vdim: int
    tau: float


@dataclass
class LatentAttentionSpec:
    """Latent attention without positions; kv_from: layer whose cached latents it reads."""
    heads: int
    dim: int
    vdim: int
    rank: int
    scale: float
    window: int = UNBOUNDED
    kv_from: Optional[int] = None


@dataclass
class FeedForwardSpec:
    """down(relu(up x)^2)."""
    ff: int


@dataclass
class Layout:
    """Where and how a model's tensors live."""
    width: int
    eps: float
    dtype: torch.dtype
    device: torch.device

    @property
    def padded_width(self):
        return round_up(self.width, 64)

    def weight(self, w, rows, cols):
        """w [n, k] in the top left corner of a zero matrix of the storage type."""
        out = torch.zeros((rows, cols), dtype=self.dtype, device=self.device)
        out[:w.shape[0], :w.shape[1]] = w.to(self.device, self.dtype)
        return out

    def head_rows(self, w, heads, dim, padded, cols):
        """w [heads * dim, k] with every head's rows padded to `padded`."""
        out = torch.zeros((heads, padded, cols), dtype=self.dtype, device=self.device)
        out[:, :dim, :w.shape[1]] = w.to(self.device, self.dtype).reshape(heads, dim, -1)
        return out.reshape(heads * padded, cols)

    def head_cols(self, w, heads, dim, padded, rows):
        """w [n, heads * dim] with every head's columns padded to `padded`, columns padded to 64."""
        out = torch.zeros((rows, round_up(heads * padded, 64)), dtype=self.dtype, device=self.device)
        view = out[:, :heads * padded].reshape(rows, heads, padded)
        view[:w.shape[0], :, :dim] = w.to(self.device, self.dtype).reshape(-1, heads, dim)
        out[:, :heads * padded] = view.reshape(rows, heads * padded)
        return out

    def vector(self, v, n):
        """fp32 vector padded with zeros."""
        out = torch.zeros(n, dtype=torch.float32, device=self.device)
        out[:v.numel()] = v.to(self.device, torch.float32)
        return out

    def norm_around_one(self, w):
        """Norm weight stored as the difference from one."""
        return self.vector(1.0 + w.float(), self.padded_width)


class GatedLinearAttention(Module):
    """`hyb_gla_step` / `hyb_gla_chunks`: q, k, v, gate and the decay's first factor in one projection,
    the decay's second factor inside the step kernel (few rows) or as a product of its own."""

    def __init__(self, spec, tensors, layout):
        s, Dp = spec, layout.padded_width
        self.spec, self.eps = spec, layout.eps
        H = s.heads
        self.dkp, self.dvp = round_up(s.dim, 16), round_up(s.vdim, 16)
        if self.dkp > 512 or self.dvp > 512:
            raise ValueError(f"linear attention takes head sizes up to 512, got {s.dim} and {s.vdim}")
        rank = tensors["a1"].shape[0]
        rp = round_up(rank, 64)
        self.proj = torch.cat([layout.head_rows(tensors["q"], H, s.dim, self.dkp, Dp),
                               layout.head_rows(tensors["k"], H, s.dim, self.dkp, Dp),
                               layout.head_rows(tensors["v"], H, s.vdim, self.dvp, Dp),
                               layout.head_rows(tensors["g"], H, s.vdim, self.dvp, Dp),
                               layout.weight(tensors["a1"], rp, Dp)])
        K, V = H * self.dkp, H * self.dvp
        self.offsets = (0, K, 2 * K, 2 * K + V, 2 * K + 2 * V)
        self.a2 = layout.head_rows(tensors["a2"], H, s.dim, self.dkp, rp)
        bias = torch.zeros((H, self.dkp), dtype=torch.float32, device=layout.device)
        bias[:, :s.dim] = tensors["a2.b"].to(layout.device, torch.float32).reshape(H, s.dim)
        self.a2_bias = bias.reshape(-1)
        self.norm = layout.vector(tensors["norm"], self.dvp)
        self.o = layout.head_cols(tensors["o"], H, s.vdim, self.dvp, Dp)

    @staticmethod
    def shapes(spec, width):
        """Checkpoint tensors and their shapes (None: any size)."""
        K, V = spec.heads * spec.dim, spec.heads * spec.vdim
        return {"q": (K, width), "k": (K, width), "v": (V, width), "g": (V, width), "o": (width, V),
                "norm": (spec.vdim,), "a1": (None, width), "a2": (K, None), "a2.b": (K,)}

    def new_cache(self, capacity, layout, len_dev):
        return RecurrentState(self.spec.heads, self.dkp, self.dvp, capacity, layout.device, len_dev)

    def emit(self, p, cache, norm):
        s, R = self.spec, p.R
        x = p.buffer("proj", self.proj.shape[0])
        p.project(self.proj, norm, x)
        attn = p.buffer("attn", self.o.shape[1])
        args = (self.norm, cache.state, attn)
        consts = (s.vdim, s.dim ** -0.5, s.tau, self.eps)
        if R <= STEP_ROWS:
            hops.gla_step(x, self.offsets, self.a2, self.a2_bias, *args, R, *consts, n_dev=p.n_dev)
        else:
            z = p.buffer("z", self.a2.shape[0], dtype=torch.float32)
            oa = self.offsets[4]
            hops.dense(x[:, oa:oa + self.a2.shape[1]], self.a2, z, hops.OUT_F32, bias=self.a2_bias, M=R, n_dev=p.n_dev)
            ws = p.bytes("gla", hops.gla_chunk_workspace_bytes(p.rows, s.heads, self.dkp, self.dvp))
            hops.gla_chunks(x, self.offsets, z, *args, p.rows, *consts, ws, n_dev=p.n_dev)
        hops.dense(attn, self.o, p.h, hops.OUT_ADD, M=R, n_dev=p.n_dev)


class LatentAttention(Module):
    """Few rows: `hyb_latent_decode` on the cached latents.  Many rows: keys and values of the visible
    span (the window before the portion and the portion) projected from the cached latents, then
    `hyb_window_attention`."""

    def __init__(self, spec, tensors, layout):
        s, Dp = spec, layout.padded_width
        self.spec, self.eps = spec, layout.eps
        H = s.heads
        self.dp, self.dvp = round_up(s.dim, 32), round_up(s.vdim, 16)
        if self.dp > 256 or self.dvp > 256:
            raise ValueError(f"latent attention takes head sizes up to 256, got {s.dim} and {s.vdim}")
        if s.rank > RANKS[-1]:
            raise ValueError(f"latent attention takes ranks up to {RANKS[-1]}, got {s.rank}")
        self.rank = next(r for r in RANKS if r >= s.rank)
        parts = [layout.head_rows(tensors["q"], H, s.dim, self.dp, Dp),
                 layout.head_rows(tensors["g"], H, s.vdim, self.dvp, Dp)]
        self.dkv_norm = None
        if s.kv_from is None:
            parts.append(layout.weight(tensors["dkv"], self.rank, Dp))
            self.dkv_norm = layout.vector(tensors["dkv.norm"], self.rank)
        self.proj = torch.cat(parts)
        self.uk = layout.head_rows(tensors["uk"], H, s.dim, self.dp, self.rank)
        self.uv = layout.head_rows(tensors["uv"], H, s.vdim, self.dvp, self.rank)
        self.o = layout.head_cols(tensors["o"], H, s.vdim, self.dvp, Dp)

    @staticmethod
    def shapes(spec, width):
        K, V, r = spec.heads * spec.dim, spec.heads * spec.vdim, spec.rank
        own = {"dkv": (r, width), "dkv.norm": (r,)} if spec.kv_from is None else {}
        return {"q": (K, width), "g": (V, width), "uk": (K, r), "uv": (V, r), "o": (width, V), **own}

    def new_cache(self, capacity, layout, len_dev):
        return LatentCache(self.rank, capacity, layout.device, layout.dtype, len_dev)

    def emit(self, p, cache, norm):
        s, R, H = self.spec, p.R, self.spec.heads
        x = p.buffer("proj", self.proj.shape[0])
        p.project(self.proj, norm, x)
        og, oc = H * self.dp, H * (self.dp + self.dvp)
        q, gate = x[:, :og], x[:, og:oc]
        new = (x[:, oc:], self.dkv_norm, self.eps, s.rank) if s.kv_from is None else None
        attn = p.buffer("attn", self.o.shape[1])
        window = min(s.window, UNBOUNDED)
        if R <= ABSORB_ROWS:
            ws = p.bytes("latent", hops.latent_decode_workspace_bytes(R, H, self.rank, window, cache.capacity))
            hops.latent_decode(q, cache.latents, self.uk, self.uv, gate, attn, p.len_dev, p.n_dev, R, H, self.dp, self.dvp,
                               window, s.scale, ws, append=new)
        else:
            if new is not None:
                hops.latent_append(*new, cache.latents, p.len_dev, p.n_dev, R)
            back = min(window - 1, cache.capacity)
            span = back + R
            S = round_up(span, 128)
            k = p.buffer("keys", H * self.dp, rows=S)
            vt = p.buffer("values", S, rows=H * self.dvp)
            hops.dense(cache.latents, self.uk, k, M=span, n_dev=p.n_dev, len_dev=p.len_dev, back=back)
            hops.dense(cache.latents, self.uv, vt, hops.OUT_TRANSPOSED, M=span, n_dev=p.n_dev, len_dev=p.len_dev, back=back)
            hops.window_attention(q, k, vt, gate, attn, p.len_dev, p.n_dev, R, H, self.dp, self.dvp, window, back, s.scale)
        hops.dense(attn, self.o, p.h, hops.OUT_ADD, M=R, n_dev=p.n_dev)


class FeedForward(Module):
    """down(relu(up x)^2): the activation in the first product's epilogue, the residual in the second's."""

    def __init__(self, spec, tensors, layout):
        fp, Dp = round_up(spec.ff, 64), layout.padded_width
        self.spec = spec
        self.up = layout.weight(tensors["up"], fp, Dp)
        self.down = layout.weight(tensors["down"], Dp, fp)

    @staticmethod
    def shapes(spec, width):
        return {"up": (spec.ff, width), "down": (width, spec.ff)}

    def emit(self, p, norm):
        act = p.buffer("act", self.up.shape[0])
        p.project(self.up, norm, act, hops.OUT_RELU2)
        hops.dense(act, self.down, p.h, hops.OUT_ADD, M=p.R, n_dev=p.n_dev)


MIXERS = {LinearAttentionSpec: GatedLinearAttention, LatentAttentionSpec: LatentAttention}
