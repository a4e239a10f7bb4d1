"""Operator front end of libhybrid_mi355x.so on torch tensors: dense layers, gated linear attention,
latent attention.  torch supplies device memory and the current stream; there is no eager or CPU
fallback.

`dtype` of weights, activations and cached latents is torch.bfloat16 or torch.float32; the residual
stream, norm weights, biases and recurrent states are float32.
"""
import ctypes

import torch

from . import _lib
from .ops import _need_cuda, _ptr, _stream, workspace

CODES = {torch.bfloat16: _lib.HYB_BF16, torch.float32: _lib.HYB_F32}
OUT_T, OUT_F32, OUT_ADD, OUT_RELU2, OUT_TRANSPOSED = range(5)
ROWS, SKINNY, GEMM = range(3)
CHUNK = _lib.HYB_GLA_CHUNK


def code(dtype):
    try:
        return CODES[dtype]
    except KeyError:
        raise TypeError(f"storage type must be bfloat16 or float32, got {dtype}") from None


def check_device(device):
    name = torch.cuda.get_device_properties(device).gcnArchName
    if not name.startswith("gfx950"):
        raise RuntimeError(f"the kernels are built for gfx950, this device is {name}")


def round_up(n, m):
    return (n + m - 1) // m * m


def _rows(t, what):
    """Row stride of a 2-d view whose rows are contiguous."""
    if t.dim() != 2 or t.stride(1) != 1:
        raise ValueError(f"{what} must be 2-d with contiguous rows")
    return t.stride(0)


def embed(tokens, table, scale, pos_table, len_dev, n_dev, vocab, out):
    """out[r] = table[tokens[r]] * scale + pos_table[*len_dev + r] (fp32)."""
    _need_cuda(tokens, table, pos_table, out)
    R, D = out.shape
    if tokens.numel() < R or tokens.dtype != torch.int32 or table.shape[1] != D or out.dtype != torch.float32 \
            or (pos_table is not None and (pos_table.shape[1] != D or pos_table.dtype != table.dtype)):
        raise ValueError("embed: shape or type mismatch")
    rc = _lib.hybrid().hyb_embed(code(table.dtype), _ptr(tokens), _ptr(table), float(scale), _ptr(pos_table),
                                 0 if pos_table is None else pos_table.shape[0], _ptr(len_dev), _ptr(n_dev), _ptr(out),
                                 R, D, int(vocab), _stream())
    _lib.check_hybrid(rc, "embed")
    return out


def norm_rows(x, weight, eps, d_true, out, rows=None, n_dev=None):
    """RMS norm of fp32 rows (those `rows` selects, or all) into `out`."""
    _need_cuda(x, weight, out, rows)
    R, D = out.shape
    if x.dtype != torch.float32 or not x.is_contiguous() or not out.is_contiguous() or x.shape[1] != D \
            or weight.numel() != D or (rows is None and x.shape[0] < R) or (rows is not None and rows.numel() < R):
        raise ValueError("norm_rows: shape or type mismatch")
    rc = _lib.hybrid().hyb_norm_rows(code(out.dtype), _ptr(x), _ptr(rows), _ptr(weight), float(eps), _ptr(out),
                                     _ptr(n_dev), R, D, int(d_true), _stream())
    _lib.check_hybrid(rc, "norm_rows")
    return out


def dense_form(dtype, M, K, norm=False, transposed=False):
    return _lib.hybrid().hyb_dense_form(code(dtype), int(M), int(K), int(norm), int(transposed))


def dense(x, w, out, epilogue=OUT_T, bias=None, M=None, n_dev=None, norm=None, len_dev=None, back=0, form=-1):
    """out = epilogue(x w^T + bias): the forms and epilogues of hyb_dense.  norm = (weight, eps, columns
    that count): x is the fp32 residual stream, normalised first (at most four rows).
    len_dev: x is indexed by token (a cache), the product's rows start at max(0, *len_dev - back)."""
    _need_cuda(x, w, out, bias)
    N, K = w.shape
    M = x.shape[0] if M is None else M
    if not w.is_contiguous() or x.shape[1] < K or (len_dev is None and x.shape[0] < M) \
            or x.dtype != (w.dtype if norm is None else torch.float32) \
            or out.dtype != (torch.float32 if epilogue in (OUT_F32, OUT_ADD) else w.dtype) \
            or (bias is not None and (bias.dtype != torch.float32 or bias.numel() != N)) \
            or (norm is not None and norm[0].numel() != K):
        raise ValueError(f"dense: shape or type mismatch (x {tuple(x.shape)} {x.dtype}, w {tuple(w.shape)} {w.dtype}, "
                         f"out {tuple(out.shape)} {out.dtype})")
    if (out.shape[0] < N or out.shape[1] < M) if epilogue == OUT_TRANSPOSED else (out.shape[0] < M or out.shape[1] < N):
        raise ValueError("dense: out is too small")
    a = _lib.HybDenseArgs(_ptr(x), _ptr(w), _ptr(bias), _ptr(out), _ptr(n_dev), _ptr(len_dev),
                          _ptr(norm[0]) if norm else None, _rows(x, "x"), _rows(out, "out"), code(w.dtype), M, N, K,
                          epilogue, int(back), int(norm[2]) if norm else 0, form, float(norm[1]) if norm else 0.0)
    _lib.check_hybrid(_lib.hybrid().hyb_dense(ctypes.byref(a), _stream()), "dense")
    return out


def gla_chunk_workspace_bytes(R, H, dkp, dvp):
    return _lib.hybrid().hyb_gla_chunk_workspace_bytes(R, H, dkp, dvp)


def _gla_args(x, offsets, norm_w, state, out, R, dv_true, qscale, tau, eps, n_dev, **more):
    H, dkp, dvp = state.shape
    oq, ok, ov, og, oa = offsets
    end = max(oq + H * dkp, ok + H * dkp, ov + H * dvp, og + H * dvp)
    if x.shape[0] < R or x.shape[1] < end or out.shape[0] < R or out.shape[1] < H * dvp or norm_w.numel() != dvp \
            or state.dtype != torch.float32 or not state.is_contiguous() or x.dtype != out.dtype:
        raise ValueError("gla: shape or type mismatch")
    a = _lib.HybGlaArgs(x=_ptr(x), norm_w=_ptr(norm_w), state=_ptr(state), out=_ptr(out), n_dev=_ptr(n_dev),
                        ldx=_rows(x, "x"), ldo=_rows(out, "out"), dtype=code(x.dtype), R=R, H=H, dkp=dkp, dvp=dvp,
                        dv_true=dv_true, off_q=oq, off_k=ok, off_v=ov, off_g=og, off_a=oa, qscale=float(qscale),
                        tau=float(tau), eps=float(eps))
    for k, v in more.items():
        setattr(a, k, v)
    return a


def gla_step(x, offsets, a2, a2_bias, norm_w, state, out, R, dv_true, qscale, tau, eps, n_dev=None):
    """Gated linear attention over few rows, one after the other; offsets: columns of q, k, v, gate
    and the decay's first factor in x."""
    _need_cuda(x, a2, a2_bias, norm_w, state, out)
    H, dkp, _ = state.shape
    if a2.shape[0] != H * dkp or a2.dtype != x.dtype or a2_bias.numel() != H * dkp or a2_bias.dtype != torch.float32 \
            or x.shape[1] < offsets[4] + a2.shape[1] or not a2.is_contiguous():
        raise ValueError("gla_step: shape or type mismatch")
    a = _gla_args(x, offsets, norm_w, state, out, R, dv_true, qscale, tau, eps, n_dev, a2=_ptr(a2), a2_bias=_ptr(a2_bias),
                  rp=a2.shape[1])
    _lib.check_hybrid(_lib.hybrid().hyb_gla_step(ctypes.byref(a), _stream()), "gla_step")
    return out


def gla_chunks(x, offsets, z, norm_w, state, out, R, dv_true, qscale, tau, eps, ws, n_dev=None):
    """Gated linear attention over a prompt portion laid out in R % 64 == 0 rows; z [R, H dkp] fp32 is
    the decay's argument and is overwritten."""
    _need_cuda(x, z, norm_w, state, out, ws)
    H, dkp, _ = state.shape
    if tuple(z.shape) != (R, H * dkp) or z.dtype != torch.float32 or not z.is_contiguous():
        raise ValueError("gla_chunks: z must be contiguous fp32 [R, H dkp]")
    a = _gla_args(x, offsets, norm_w, state, out, R, dv_true, qscale, tau, eps, n_dev, z=_ptr(z), workspace=_ptr(ws),
                  workspace_bytes=ws.numel())
    _lib.check_hybrid(_lib.hybrid().hyb_gla_chunks(ctypes.byref(a), _stream()), "gla_chunks")
    return out


def latent_rank_supported(rank):
    return bool(_lib.hybrid().hyb_latent_rank_supported(int(rank)))


def latent_append(x, norm_w, eps, rank_true, cache, len_dev, n_dev, R):
    """Norm R rows of x [., rank] and append them to `cache` [capacity, rank] at row *len_dev."""
    _need_cuda(x, norm_w, cache)
    cap, rank = cache.shape
    if x.shape[0] < R or x.shape[1] < rank or x.dtype != cache.dtype or norm_w.numel() != rank or not cache.is_contiguous():
        raise ValueError("latent_append: shape or type mismatch")
    rc = _lib.hybrid().hyb_latent_append(code(cache.dtype), _ptr(x), _rows(x, "x"), _ptr(norm_w), float(eps), _ptr(cache),
                                         cap, _ptr(len_dev), _ptr(n_dev), R, rank, int(rank_true), _stream())
    _lib.check_hybrid(rc, "latent_append")


def latent_decode_workspace_bytes(R, H, rank, window, cap):
    return _lib.hybrid().hyb_latent_decode_workspace_bytes(R, H, rank, window, cap)


def latent_decode(q, cache, uk, uv, gate, out, len_dev, n_dev, R, H, dp, dvp, window, scale, ws,
                  append=None):
    """Windowed attention of few rows over cached latents (absorbed key projection), gated.
    append = (rows [., rank], norm weight, eps, columns that count): the new rows, normed and appended
    first (None: they are in the cache)."""
    _need_cuda(q, cache, uk, uv, gate, out, ws)
    cap, rank = cache.shape
    new, new_norm, eps, rank_true = append if append is not None else (None, None, 0.0, 0)
    if new is not None and (new.shape[0] < R or new.shape[1] < rank or new.dtype != cache.dtype or new_norm.numel() != rank
                            or new_norm.dtype != torch.float32):
        raise ValueError("latent_decode: rows to append do not fit")
    if tuple(uk.shape) != (H * dp, rank) or tuple(uv.shape) != (H * dvp, rank) \
            or min(q.shape[0], gate.shape[0], out.shape[0]) < R or q.shape[1] < H * dp or gate.shape[1] < H * dvp \
            or out.shape[1] < H * dvp or len({t.dtype for t in (q, cache, uk, uv, gate, out)}) != 1 \
            or not (cache.is_contiguous() and uk.is_contiguous() and uv.is_contiguous()):
        raise ValueError("latent_decode: shape or type mismatch")
    a = _lib.HybLatentDecodeArgs(_ptr(q), _ptr(cache), _ptr(uk), _ptr(uv), _ptr(gate), _ptr(out), _ptr(len_dev), _ptr(n_dev),
                                 _ptr(ws), ws.numel(), _ptr(new), _ptr(new_norm), _rows(q, "q"), _rows(gate, "gate"),
                                 _rows(out, "out"), cap, 0 if new is None else _rows(new, "append"), code(q.dtype), R, H, dp,
                                 dvp, rank, int(window), int(rank_true), float(scale), float(eps))
    _lib.check_hybrid(_lib.hybrid().hyb_latent_decode(ctypes.byref(a), _stream()), "latent_decode")
    return out


def window_attention(q, k, vt, gate, out, len_dev, n_dev, R, H, dp, dvp, window, back, scale):
    """Windowed causal attention of a prompt portion over projected keys k [S, H dp] and transposed
    values vt [H dvp, S]; row s is position max(0, *len_dev - back) + s."""
    _need_cuda(q, k, vt, gate, out)
    S = vt.shape[1]
    if k.shape[0] < S or k.shape[1] < H * dp or vt.shape[0] < H * dvp or S < back + R \
            or min(q.shape[0], gate.shape[0], out.shape[0]) < R or q.shape[1] < H * dp or gate.shape[1] < H * dvp \
            or out.shape[1] < H * dvp or len({t.dtype for t in (q, k, vt, gate, out)}) != 1:
        raise ValueError("window_attention: shape or type mismatch")
    a = _lib.HybWindowArgs(_ptr(q), _ptr(k), _ptr(vt), _ptr(gate), _ptr(out), _ptr(len_dev), _ptr(n_dev), _rows(q, "q"),
                           _rows(k, "k"), _rows(vt, "vt"), _rows(gate, "gate"), _rows(out, "out"), code(q.dtype), R, H,
                           dp, dvp, int(window), int(back), float(scale))
    _lib.check_hybrid(_lib.hybrid().hyb_window_attention(ctypes.byref(a), _stream()), "window_attention")
    return out


def argmax_rows(logits, out):
    """Row argmax of fp32 logits (rows may be strided), lowest index among equal maxima."""
    _need_cuda(logits, out)
    R, V = logits.shape
    if logits.dtype != torch.float32 or out.dtype != torch.int32 or out.numel() < R:
        raise ValueError("argmax_rows: shape or type mismatch")
    L = _lib.hybrid()
    ws = workspace("hybrid_argmax", L.hyb_argmax_workspace_bytes(R), logits.device)
    rc = L.hyb_argmax_rows_f32(_ptr(logits), _rows(logits, "logits"), R, V, _ptr(out), _ptr(ws), ws.numel(), _stream())
    _lib.check_hybrid(rc, "argmax_rows")
    return out


def token_advance(token, nxt, out, count):
    rc = _lib.hybrid().hyb_token_advance(_ptr(token), _ptr(nxt), _ptr(out), _ptr(count), out.numel(), _stream())
    _lib.check_hybrid(rc, "token_advance")


def advance_len(len_dev, n_dev, capacity):
    _lib.check_hybrid(_lib.hybrid().hyb_advance_len(_ptr(len_dev), _ptr(n_dev), int(capacity), _stream()), "advance_len")
