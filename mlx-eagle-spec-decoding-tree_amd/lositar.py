"""The Lositar design: config.json and tensor names -> `hybrid.HybridArgs` and `hybrid.Model`.

A small decoder: scaled token embedding plus learned positions, pre-norm layers (RMS norms whose
weight is stored around zero) of gated linear attention or windowed latent attention with an
optional squared-relu feed-forward, and the embedding table as the output head.
"""
import torch

from . import checkpoint, hybrid
from .mixers import FeedForwardSpec, LatentAttentionSpec, LinearAttentionSpec

ARCHITECTURE = "Lositar"


def _need(d, key, where):
    if key not in d:
        raise ValueError(f"config.json: {where} has no '{key}'")
    return d[key]


def _sizes(d, where, *keys):
    out = []
    for k in keys:
        v = _need(d, k, where)
        if not isinstance(v, int) or isinstance(v, bool) or v < 1:
            raise ValueError(f"config.json: {where}.{k} must be a positive integer, got {v!r}")
        out.append(v)
    return out


def _mixer(kind, m, where):
    if kind == "gla":
        heads, dim, vdim = _sizes(m, where, "heads", "dim", "vdim")
        tau = float(_need(m, "tau", where))
        if not tau > 0:
            raise ValueError(f"config.json: {where}.tau must be positive")
        return LinearAttentionSpec(heads, dim, vdim, tau)
    if kind == "latent_attention":
        heads, dim, vdim, rank = _sizes(m, where, "heads", "dim", "vdim", "kv_rank")
        mask = _need(m, "mask", where)
        (size,) = _sizes(mask, f"{where}.mask", "size")
        return LatentAttentionSpec(heads, dim, vdim, rank, float(_need(m, "scale", where)), size, m.get("kv_from"))
    raise ValueError(f"config.json: {where} has the unknown type {kind!r}")


def args_from_config(config):
    layers = []
    for i, entry in enumerate(_need(config, "layers", "the model")):
        where = f"layers[{i}]"
        mixer = _mixer(_need(entry, "type", where), _need(entry, "mixer", where), where)
        src = getattr(mixer, "kv_from", None)
        if src is not None:
            own = layers[src].mixer if isinstance(src, int) and 0 <= src < i else None
            if not isinstance(own, LatentAttentionSpec) or own.kv_from is not None or own.rank != mixer.rank:
                raise ValueError(f"config.json: {where}.kv_from must name an earlier latent-attention layer of the same "
                                 f"kv_rank with latents of its own, got {src!r}")
        mlp = entry.get("mlp")
        if mlp is not None:
            if mlp.get("kind") != "dense":
                raise ValueError(f"config.json: {where}.mlp has the unknown kind {mlp.get('kind')!r}")
            mlp = FeedForwardSpec(*_sizes(mlp, f"{where}.mlp", "ff"))
        layers.append(hybrid.LayerSpec(mixer, mlp))
    if not layers:
        raise ValueError("config.json: no layers")
    vocab, width, positions = _sizes(config, "the model", "vocab", "width", "max_positions")
    return hybrid.HybridArgs(model_type=ARCHITECTURE, vocab_size=vocab, width=width, max_positions=positions,
                             norm_eps=float(_need(_need(config, "norm", "the model"), "eps", "norm")),
                             embed_scale=float(_need(_need(config, "embedding", "the model"), "scale", "embedding")),
                             layers=layers)


def arrange(args, weights):
    """Checkpoint tensors (flat, `l<i>.` prefixes) in the form `hybrid.Model` takes, shapes checked."""
    shapes = hybrid.Model.shapes(args)

    def take(name, shape):
        t = weights.get(name)
        if t is None:
            raise ValueError(f"the checkpoint has no tensor '{name}'")
        if t.dim() != len(shape) or any(want is not None and got != want for got, want in zip(t.shape, shape)):
            raise ValueError(f"{name} has shape {tuple(t.shape)}, expected {shape}")
        return t

    out = {k: take(k, shapes[k]) for k in ("embed", "pos", "final.norm")}
    out["layers"] = [{k: take(f"l{i}.{k}", s) for k, s in layer.items()} for i, layer in enumerate(shapes["layers"])]
    for i, t in enumerate(out["layers"]):
        if "mix.a1" in t and t["mix.a1"].shape[0] != t["mix.a2"].shape[1]:
            raise ValueError(f"l{i}.mix.a1 and l{i}.mix.a2 do not fit together")
    return out


def build(config, weights, device, dtype=torch.bfloat16):
    """A model from a config dict and a flat dict of tensors."""
    args = args_from_config(config)
    return hybrid.Model(args, arrange(args, weights), device, dtype)


def load(path, config, device, dtype=None):
    return build(config, checkpoint.load_weights(path, "cpu", dtype=None), device, dtype or torch.bfloat16)
