"""Configurations, weights and comparisons shared by the Lositar tests."""
import copy
import functools

import numpy as np
import torch

from mlx_eagle_spec_decoding_tree_amd import synth
from oracle import lositar_oracle


def gla(heads=3, dim=24, vdim=40, tau=7.0, ff=70):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def latent(heads=2, dim=40, vdim=24, rank=72, window=50, scale=None, ff=70, kv_from=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank, "mask": {"size": window},
         "scale": dim ** -0.5 if scale is None else scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(*layers, width=88, vocab=203, positions=700, eps=1e-5, embed_scale=3.0):
    return {"architecture": "Lositar", "vocab": vocab, "width": width, "max_positions": positions,
            "norm": {"eps": eps}, "embedding": {"scale": embed_scale}, "layers": list(layers)}


CONFIGS = {
    # every branch at once: linear attention first, latents shared across layers with another window and
    # other heads, layers without a feed-forward, sizes that no padding unit divides
    "mixed": config(gla(), latent(), latent(heads=3, dim=16, vdim=56, window=93, kv_from=1, ff=None),
                    gla(heads=1, dim=100, vdim=8, tau=1.0, ff=130), latent(heads=1, dim=64, vdim=64, rank=64, window=7)),
    "linear_only": config(gla(heads=2, dim=16, vdim=136, tau=2.0), gla(heads=5, dim=72, vdim=16, tau=30.0, ff=None), width=64,
                          embed_scale=1.0, eps=1e-3),
    "latent_only": config(latent(window=1), latent(heads=4, dim=8, vdim=130, rank=200, window=128),
                          latent(heads=5, dim=33, vdim=17, rank=200, window=4000, kv_from=1), width=130, vocab=64,
                          eps=1e-6),
    # softmax so sharp that a query reads one or two keys: a wrong key or a window off by one changes everything
    "sharp": config(latent(scale=4.0, window=61, ff=None), latent(heads=3, scale=4.0, window=64, kv_from=0, ff=None),
                    gla(tau=16.0), width=96, embed_scale=1.0),
}


@functools.lru_cache(maxsize=None)
def weights(name, seed=5, memory=True):
    """bf16 tensors.  memory: decays close to one, so that the state's far past shows in the logits."""
    cfg = CONFIGS[name]
    w = synth.make_lositar_weights(cfg, seed=seed, decay_rank=5)
    for k in w:
        if memory and k.endswith("a2.b"):
            w[k] = w[k] + 4.0
        if k == "pos":
            w[k] = (w[k].float() * 2).to(torch.bfloat16)
    return w


def as_numpy(w):
    return {k: v.float().numpy() for k, v in w.items()}


@functools.lru_cache(maxsize=None)
def sequence(name, n, seed=0):
    return tuple(np.random.default_rng(seed).integers(0, CONFIGS[name]["vocab"], n).tolist())


@functools.lru_cache(maxsize=None)
def want_logits(name, n, seed=0, mistake=None):
    """float64 logits [n, vocab] of the oracle for `sequence`."""
    return lositar_oracle.forward(CONFIGS[name], as_numpy(weights(name)), sequence(name, n, seed),
                                  mistake=dict(mistake) if mistake else None)


def rms_err(got, want):
    """Worst row: root mean square of the difference over that of the reference (means taken off)."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    d = got - want
    d = d - d.mean(-1, keepdims=True)
    scale = np.sqrt(np.mean((want - want.mean(-1, keepdims=True)) ** 2))
    return float(np.sqrt(np.mean(d * d, axis=-1)).max() / scale)


def altered(name, **changes):
    cfg = copy.deepcopy(CONFIGS[name])
    cfg.update(changes)
    return cfg
