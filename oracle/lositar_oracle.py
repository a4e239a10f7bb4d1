"""Plain, slow restatement of the Lositar decoder (numpy, one token at a time where order
matters), one function per mechanism.  Shares no code with the package: tensors and sizes arrive
as a plain dict of arrays and the parsed config.json.

`dtype` is the type everything is computed in (float64 for the reference, float32 on request).
A forward over a whole sequence is defined position by position from the equations; there is no
cache, so prompts, portions and decoding all have the same right answer.
"""
import numpy as np


def sigmoid(z):
    z = np.asarray(z)
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e)).astype(z.dtype)


def log_sigmoid(z):
    z = np.asarray(z)
    return (np.minimum(z, 0) - np.log1p(np.exp(-np.abs(z)))).astype(z.dtype)


def silu(z):
    return z * sigmoid(z)


def relu_squared(z):
    return np.square(np.maximum(z, 0))


def unit_rms(x, eps):
    """x over its root mean square along the last axis, eps inside the root."""
    return x / np.sqrt(np.mean(np.square(x), axis=-1, keepdims=True) + x.dtype.type(eps))


def norm_around_one(x, w, eps):
    """RMS norm whose weight is stored as the difference from one."""
    return unit_rms(x, eps) * (1 + w)


def norm_plain(x, w, eps):
    return unit_rms(x, eps) * w


def embed(tokens, positions, table, pos_table, scale):
    """Scaled token row plus the (unscaled) learned row of its position."""
    return table[tokens] * table.dtype.type(scale) + pos_table[positions]


def gla_decay(z, tau):
    """Per-channel decay sigmoid(z) ** (1 / tau), taken through its logarithm."""
    return np.exp(log_sigmoid(z) / z.dtype.type(tau))


def gla_recurrence(q, k, v, alpha, state=None):
    """q, k, alpha [L,H,dk], v [L,H,dv]: S <- diag(alpha_t) S + k_t v_t^T, o_t = S^T q_t.
    Returns (o [L,H,dv], the state after the last token [H,dk,dv])."""
    L, H, dk = q.shape
    dv = v.shape[-1]
    S = np.zeros((H, dk, dv), q.dtype) if state is None else state.copy()
    o = np.empty((L, H, dv), q.dtype)
    for t in range(L):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = np.einsum("hkv,hk->hv", S, q[t])
    return o, S


def gla_mixer(h, w, cfg, eps, state=None):
    """Gated linear attention over the rows of h [L,D]; w: tensors by their short names."""
    L = h.shape[0]
    H, dk, dv = cfg["heads"], cfg["dim"], cfg["vdim"]
    q = (h @ w["q"].T * h.dtype.type(dk ** -0.5)).reshape(L, H, dk)
    k = (h @ w["k"].T).reshape(L, H, dk)
    v = (h @ w["v"].T).reshape(L, H, dv)
    z = (h @ w["a1"].T @ w["a2"].T + w["a2.b"]).reshape(L, H, dk)
    o, S = gla_recurrence(q, k, v, gla_decay(z, cfg["tau"]), state)
    o = norm_plain(o, w["norm"], eps).reshape(L, H * dv)
    return (o * silu(h @ w["g"].T)) @ w["o"].T, S


def latent(h, w, eps):
    """The cached vector of latent attention: down-projection and RMS norm."""
    return norm_plain(h @ w["dkv"].T, w["dkv.norm"], eps)


def window_visible(i, j, size):
    return 0 <= i - j < size


def window_softmax(scores, size):
    """scores [L,L]: softmax of every row over the positions its window shows."""
    L = scores.shape[0]
    p = np.zeros_like(scores)
    for i in range(L):
        vis = [j for j in range(L) if window_visible(i, j, size)]
        s = scores[i, vis]
        e = np.exp(s - s.max())
        p[i, vis] = e / e.sum()
    return p


def latent_attention(h, c, w, cfg):
    """Attention of the rows of h over the latents c [L,rank]."""
    L = h.shape[0]
    H, dim, vdim = cfg["heads"], cfg["dim"], cfg["vdim"]
    q = (h @ w["q"].T).reshape(L, H, dim)
    k = (c @ w["uk"].T).reshape(L, H, dim)
    v = (c @ w["uv"].T).reshape(L, H, vdim)
    out = np.empty((L, H, vdim), h.dtype)
    for a in range(H):
        p = window_softmax(q[:, a] @ k[:, a].T * h.dtype.type(cfg["scale"]), cfg["mask"]["size"])
        out[:, a] = p @ v[:, a]
    return (out.reshape(L, H * vdim) * sigmoid(h @ w["g"].T)) @ w["o"].T


def feed_forward(h, w):
    return relu_squared(h @ w["up"].T) @ w["down"].T


def short_names(weights, prefix):
    return {k[len(prefix):]: v for k, v in weights.items() if k.startswith(prefix)}


def forward(config, weights, tokens, dtype=np.float64, tap=None, mistake=None):
    """Logits [L, vocab] of one whole sequence.  tap(i, x): the residual stream after layer i.
    mistake: {name: value} changes the oracle on purpose (tests that a fault would show):
    "window" adds to every window size, "drop_state_at" forgets the recurrent state before that
    position, "pos_shift" shifts the learned positions."""
    mistake = mistake or {}
    W = {k: np.asarray(v).astype(dtype) for k, v in weights.items()}
    tokens = np.asarray(tokens)
    eps = config["norm"]["eps"]
    positions = np.arange(len(tokens)) + mistake.get("pos_shift", 0)
    x = embed(tokens, positions, W["embed"], W["pos"], config["embedding"]["scale"])
    latents = {}
    for i, layer in enumerate(config["layers"]):
        mix, cfg = short_names(W, f"l{i}.mix."), dict(layer["mixer"])
        h = norm_around_one(x, W[f"l{i}.norm1"], eps)
        if layer["type"] == "gla":
            cut = mistake.get("drop_state_at")
            if cut:
                y = np.concatenate([gla_mixer(h[:cut], mix, cfg, eps)[0], gla_mixer(h[cut:], mix, cfg, eps)[0]])
            else:
                y, _ = gla_mixer(h, mix, cfg, eps)
        elif layer["type"] == "latent_attention":
            cfg["mask"] = {"size": cfg["mask"]["size"] + mistake.get("window", 0)}
            if cfg.get("kv_from") is None:
                latents[i] = latent(h, mix, eps)
            y = latent_attention(h, latents[cfg["kv_from"] if cfg.get("kv_from") is not None else i], mix, cfg)
        else:
            raise ValueError(layer["type"])
        x = x + y
        if layer.get("mlp"):
            if layer["mlp"]["kind"] != "dense":
                raise ValueError(layer["mlp"]["kind"])
            x = x + feed_forward(norm_around_one(x, W[f"l{i}.norm2"], eps), short_names(W, f"l{i}.mlp."))
        if tap is not None:
            tap(i, x)
    return norm_around_one(x, W["final.norm"], eps) @ W["embed"].T
