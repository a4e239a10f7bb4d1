"""Kernels of libhybrid_mi355x.so against the plain implementation, each mechanism alone."""
import numpy as np
import pytest
import torch

from mlx_eagle_spec_decoding_tree_amd import hybrid_ops as hops
from oracle import lositar_oracle as lo

pytestmark = pytest.mark.gpu
DTYPES = [torch.bfloat16, torch.float32]


def tol(dtype, bf16=8e-3, f32=2e-5):
    return bf16 if dtype == torch.bfloat16 else f32


def rel(got, want):
    """Largest difference over the root mean square of the reference; for bf16 results, whose rounding
    grows with the element, the root mean square of the differences relative to max(|element|, rms)."""
    g, w = got.double().cpu().numpy(), np.asarray(want, np.float64)
    rms = np.sqrt(np.mean(w * w))
    if got.dtype == torch.bfloat16:
        d = np.abs(g - w) / np.maximum(np.abs(w), rms)
        return float(np.sqrt(np.mean(d * d))) if d.max() < 0.05 else float(d.max())
    return float(np.abs(g - w).max() / rms)


def i32(dev, *v):
    return torch.tensor(v, dtype=torch.int32, device=dev)


def rand(dev, dtype, *shape, seed=0, std=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(shape, generator=g) * std).to(dtype).to(dev)


# ---- dense ---------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,N,K", [(1, 16, 64), (1, 336, 704), (2, 80, 2112), (3, 48, 128), (4, 208, 4096), (5, 64, 192),
                                   (16, 48, 640), (33, 80, 64), (64, 96, 320), (65, 272, 128), (200, 112, 448), (300, 144, 64)])
def test_dense_forms_and_epilogues(dev, dtype, M, N, K):
    x, w = rand(dev, dtype, M, K + 64, seed=1), rand(dev, dtype, N, K, seed=2, std=K ** -0.5)
    want = x[:, :K].double().cpu().numpy() @ w.double().cpu().numpy().T
    live = i32(dev, M - 1 if M > 1 else 1)
    n = int(live)
    forms = {hops.dense_form(dtype, M, K)} | ({hops.SKINNY} if M <= 64 else set()) | {hops.GEMM}
    for form in forms:
        out = torch.full((M, N + 16), 7.0, dtype=dtype, device=dev)
        hops.dense(x[:, :K], w, out, form=form, n_dev=live)
        assert rel(out[:n, :N], want[:n]) < tol(dtype, 4e-3), form
        assert bool((out[:, N:] == 7).all()) and bool((out[n:] == 7).all()), "wrote outside its rows and columns"
        out = torch.full((M, N), 7.0, dtype=torch.float32, device=dev)
        bias = rand(dev, torch.float32, N, seed=3)
        hops.dense(x[:, :K], w, out, hops.OUT_F32, bias=bias, form=form)
        assert rel(out, want + bias.double().cpu().numpy()) < 2e-5
        h = rand(dev, torch.float32, M, N, seed=4)
        h0 = h.double().cpu().numpy()
        hops.dense(x[:, :K], w, h, hops.OUT_ADD, form=form)
        assert rel(h, h0 + want) < 2e-5
        out = torch.empty((M, N), dtype=dtype, device=dev)
        hops.dense(x[:, :K], w, out, hops.OUT_RELU2, form=form)
        assert rel(out, lo.relu_squared(want)) < tol(dtype, 4e-3, 5e-5)
    out = torch.full((N, hops.round_up(M, 128)), 7.0, dtype=dtype, device=dev)
    hops.dense(x[:, :K], w, out, hops.OUT_TRANSPOSED)
    assert rel(out[:, :M], want.T) < tol(dtype, 4e-3) and bool((out[:, hops.round_up(M, 4):] == 7).all())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,D,K,N", [(1, 250, 256, 32), (2, 64, 64, 96), (3, 100, 128, 16), (4, 1000, 1024, 48)])
def test_norm_folded_into_a_product(dev, dtype, M, D, K, N):
    x = torch.zeros(M, K, device=dev)
    x[:, :D] = rand(dev, torch.float32, M, D, std=3.0)
    g = torch.zeros(K, device=dev)
    g[:D] = 1 + 0.3 * rand(dev, torch.float32, D, seed=1)
    w = rand(dev, dtype, N, K, seed=2, std=K ** -0.5)
    normed = torch.empty(M, K, dtype=dtype, device=dev)
    hops.norm_rows(x, g, 1e-2, D, normed)
    want = lo.norm_plain(x[:, :D].double().cpu().numpy(), g[:D].double().cpu().numpy(), 1e-2)
    assert rel(normed[:, :D], want) < tol(dtype, 4e-3) and not normed[:, D:].any()
    a, b = torch.empty(M, N, device=dev), torch.empty(M, N, device=dev)
    hops.dense(x, w, a, hops.OUT_F32, norm=(g, 1e-2, D))
    hops.dense(normed, w, b, hops.OUT_F32)
    assert rel(a, b.double().cpu().numpy()) < 1e-4
    rows = i32(dev, *range(M - 1, -1, -1))
    back = torch.empty_like(normed)
    hops.norm_rows(x, g, 1e-2, D, back, rows=rows)
    assert torch.equal(back, normed.flip(0))


@pytest.mark.parametrize("dtype", DTYPES)
def test_dense_reads_a_window_of_a_token_buffer(dev, dtype):
    """Rows max(0, len - back) .. len + n - 1 of a cache, in every matrix form."""
    cache, w = rand(dev, dtype, 300, 128, seed=1), rand(dev, dtype, 48, 128, seed=2, std=0.1)
    full = cache.double().cpu().numpy() @ w.double().cpu().numpy().T
    for length, n, back, M in ((0, 5, 20, 25), (7, 9, 20, 40), (100, 30, 17, 60), (130, 100, 128, 256), (200, 100, 0, 100)):
        row0, live = max(0, length - back), min(length, back) + n
        for ep in (hops.OUT_T, hops.OUT_TRANSPOSED):
            out = torch.zeros((M, 48) if ep == hops.OUT_T else (48, hops.round_up(M, 128)), dtype=dtype, device=dev)
            hops.dense(cache, w, out, ep, M=M, n_dev=i32(dev, n), len_dev=i32(dev, length), back=back)
            got = out[:live] if ep == hops.OUT_T else out[:, :live].T
            assert rel(got, full[row0:row0 + live]) < tol(dtype, 4e-3), (length, n, back)


@pytest.mark.parametrize("dtype", DTYPES)
def test_embedding_adds_the_position_row(dev, dtype):
    table, pos = rand(dev, dtype, 32, 192, seed=1), rand(dev, dtype, 50, 192, seed=2)
    toks = i32(dev, 3, 31, 0, 7, 9)
    h = torch.full((5, 192), 7.0, device=dev)
    hops.embed(toks, table, 2.5, pos, i32(dev, 11), i32(dev, 4), 32, h)
    want = lo.embed(toks.cpu().numpy(), np.arange(5) + 11, table.double().cpu().numpy(), pos.double().cpu().numpy(), 2.5)
    assert rel(h[:4], want[:4]) < 1e-6 and bool((h[4] == 7).all())
    hops.embed(toks, table, 2.5, None, i32(dev, 11), i32(dev, 5), 32, h)
    assert rel(h, table.double().cpu().numpy()[toks.cpu().numpy()] * 2.5) < 1e-6


def test_argmax_takes_the_lowest_of_equal_maxima(dev):
    x = torch.zeros(3, 70016, device=dev)
    x[0, [69999, 123]] = 5.0
    x[1, 0] = -1.0
    x[2] = -3.0
    x[2, 65000] = -2.0
    out = torch.empty(3, dtype=torch.int32, device=dev)
    assert hops.argmax_rows(x[:, :70000], out).tolist() == [123, 1, 65000]


# ---- gated linear attention --------------------------------------------------------------------

def gla_case(dev, dtype, L, H, dk, dv, rank, tau, zscale, zshift, seed=0):
    """Fused projection rows with padded heads, and the oracle's inputs."""
    dkp, dvp, rp = hops.round_up(dk, 16), hops.round_up(dv, 16), hops.round_up(rank, 64)
    rng = np.random.default_rng(seed)
    q, k = rng.normal(size=(2, L, H, dk))
    v, gate = rng.normal(size=(2, L, H, dv))
    a1 = rng.normal(size=(L, rank))
    a2 = rng.normal(size=(H, dk, rank)) * zscale / np.sqrt(rank)
    bias = zshift + rng.normal(size=(H, dk))
    norm = 1 + 0.2 * rng.normal(size=dv)

    def pad(a, n):
        t = torch.zeros(*a.shape[:-1], n)
        t[..., :a.shape[-1]] = torch.from_numpy(a)
        return t.to(dtype)
    x = torch.cat([pad(q, dkp).reshape(L, -1), pad(k, dkp).reshape(L, -1), pad(v, dvp).reshape(L, -1),
                   pad(gate, dvp).reshape(L, -1), pad(a1, rp)], dim=1).to(dev)
    offs = np.cumsum([0, H * dkp, H * dkp, H * dvp, H * dvp])
    w = torch.zeros(H, dkp, rp, dtype=dtype)
    w[:, :dk, :rank] = torch.from_numpy(a2).to(dtype)
    b = torch.zeros(H, dkp)
    b[:, :dk] = torch.from_numpy(bias).float()
    nw = torch.zeros(dvp)
    nw[:dv] = torch.from_numpy(norm).float()
    # what the kernels see, in float64
    r = lambda a: torch.from_numpy(a).to(dtype).double().numpy()
    z = np.einsum("lr,hkr->lhk", r(a1), w[:, :dk, :rank].double().numpy()) + bias.astype(np.float32)
    ref = dict(q=r(q) * dk ** -0.5, k=r(k), v=r(v), alpha=lo.gla_decay(z, tau), gate=r(gate), norm=norm)
    return dict(x=x, offsets=[int(o) for o in offs], a2=w.reshape(H * dkp, rp).to(dev), a2_bias=b.reshape(-1).to(dev),
                norm_w=nw.to(dev), H=H, dk=dk, dv=dv, dkp=dkp, dvp=dvp, tau=tau), ref


def gla_want(ref, eps, state=None):
    o, S = lo.gla_recurrence(ref["q"], ref["k"], ref["v"], ref["alpha"], state)
    return lo.norm_plain(o, ref["norm"], eps) * lo.silu(ref["gate"]), S


def gla_run(dev, case, state, rows, form, eps):
    """Rows `rows` (a slice) through one form; the live count is below the layout's rows."""
    x = case["x"][rows]
    n = x.shape[0]
    R = n + 1 if form == "step" else hops.round_up(n + 1, 64)
    xp = torch.zeros(R, x.shape[1], dtype=x.dtype, device=dev)
    xp[:n] = x
    xp[n:] = 3.0                                       # rows that are not live
    out = torch.full((R, hops.round_up(case["H"] * case["dvp"], 64)), 7.0, dtype=x.dtype, device=dev)
    args = (case["norm_w"], state, out, R, case["dv"], case["dk"] ** -0.5, case["tau"], eps)
    if form == "step":
        hops.gla_step(xp, case["offsets"], case["a2"], case["a2_bias"], *args, n_dev=i32(dev, n))
    else:
        z = torch.empty(R, case["a2"].shape[0], device=dev)
        oa = case["offsets"][4]
        hops.dense(xp[:, oa:], case["a2"], z, hops.OUT_F32, bias=case["a2_bias"])
        ws = torch.full((hops.gla_chunk_workspace_bytes(R, case["H"], case["dkp"], case["dvp"]),), 255, dtype=torch.uint8,
                        device=dev)                    # NaN bit patterns: nothing stale may be used
        hops.gla_chunks(xp, case["offsets"], z, *args, ws, n_dev=i32(dev, n))
    assert bool((out[n:] == 7).all())
    return out[:n, :case["H"] * case["dvp"]].reshape(n, case["H"], case["dvp"])[..., :case["dv"]]


SHAPES = [(1, 16, 16, 3, 1.0), (3, 24, 40, 16, 16.0), (2, 100, 72, 70, 4.0), (2, 128, 128, 16, 16.0), (1, 48, 200, 8, 2.0),
          (1, 500, 24, 9, 16.0), (1, 40, 500, 9, 16.0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dk,dv,rank,tau", SHAPES)
def test_gla_step_and_chunks(dev, dtype, H, dk, dv, rank, tau):
    L, eps = 150, 1e-5
    case, ref = gla_case(dev, dtype, L, H, dk, dv, rank, tau, 2.0, 3.0)
    want, S = gla_want(ref, eps)
    for form in ("step", "chunk"):
        state = torch.zeros(H, case["dkp"], case["dvp"], device=dev)
        got, at = [], 0
        # portions around the chunk and sub-chunk sizes, single tokens in between
        for n in (1, 15, 2, 47, 64, 1, 20):
            got.append(gla_run(dev, case, state, slice(at, at + n), form, eps))
            at += n
        assert at == L
        assert rel(torch.cat(got), want) < tol(dtype, 4e-3, 2e-5), form
        assert rel(state[:, :dk, :dv], S) < 1e-5
        assert not state[:, dk:].any() and not state[:, :, dv:].any()
    state.zero_()
    assert rel(gla_run(dev, case, state, slice(0, L), "chunk", eps), want) < tol(dtype, 4e-3, 2e-5)


@pytest.mark.parametrize("zscale,zshift,tau", [(0.0, -60.0, 1.0), (25.0, 0.0, 1.0), (8.0, 20.0, 0.5), (0.0, 40.0, 16.0)])
def test_gla_extreme_decays(dev, zscale, zshift, tau):
    """Decays from e^-120 to 1 - 1e-18 in one tensor: no overflow, no loss of what is remembered."""
    # a large eps: without memory an output can be a cancelled k . q times v, which a small one would blow up
    eps = 0.1
    case, ref = gla_case(dev, torch.float32, 200, 2, 32, 32, 8, tau, zscale, zshift)
    want, S = gla_want(ref, eps)
    for form in ("step", "chunk"):
        state = torch.zeros(2, 32, 32, device=dev)
        got = torch.cat([gla_run(dev, case, state, slice(a, b), form, eps) for a, b in ((0, 130), (130, 200))])
        assert bool(torch.isfinite(got).all())
        assert rel(got, want) < 5e-5, form
        assert rel(state, S) < 5e-5, form


def test_gla_remembers_one_token(dev):
    """A key far back that one query alone asks for: with decays near one it dominates the output."""
    L, dk = 190, 32
    case, ref = gla_case(dev, torch.float32, L, 1, dk, 16, 8, 16.0, 0.0, 9.0)
    x, (oq, ok, ov, og, oa) = case["x"], case["offsets"]
    u = torch.ones(dk, device=dev)
    x[:, ok:ok + dk] *= 0.01
    ref["k"] *= 0.01
    for t in (0, 15, 16, 63, 64, 127):
        x2, r2 = x.clone(), {k: v.copy() for k, v in ref.items()}
        x2[t, ok:ok + dk], x2[-1, oq:oq + dk] = u, 5 * u
        r2["k"][t], r2["q"][-1] = 1.0, 5.0 * dk ** -0.5
        want, _ = gla_want(r2, 1e-6)
        gone, _ = gla_want({**r2, "v": np.where(np.arange(L)[:, None, None] == t, 0, r2["v"])}, 1e-6)
        assert np.abs(want[-1] - gone[-1]).max() > 0.3
        for form in ("step", "chunk"):
            state = torch.zeros(1, dk, 16, device=dev)
            got = gla_run(dev, {**case, "x": x2}, state, slice(0, L), form, 1e-6)
            assert rel(got[-1], want[-1]) < 1e-3, (t, form)


# ---- latent attention -----------------------------------------------------------------------------

def latent_case(dev, dtype, L, H, dim, vdim, rank, window, scale, seed=0, peak=None):
    """Queries, gates and cached latents of a sequence; peak (i, j): query i asks for key j alone."""
    rng = np.random.default_rng(seed)
    dp, dvp = hops.round_up(dim, 32), hops.round_up(vdim, 16)
    from mlx_eagle_spec_decoding_tree_amd.mixers import RANKS
    rp = next(r for r in RANKS if r >= rank)
    q = rng.normal(size=(L, H, dim))
    c = rng.normal(size=(L, rank))
    uk = rng.normal(size=(H, dim, rank)) / np.sqrt(rank)
    uv = rng.normal(size=(H, vdim, rank)) / np.sqrt(rank)
    gate = rng.normal(size=(L, H, vdim))
    if peak is not None:
        i, j = peak
        k = np.einsum("hdr,r->hd", uk, c[j])
        q[i] = 25.0 * k / np.sum(k * k, -1, keepdims=True) / scale
        c[:j] *= 0.3
        c[j + 1:] *= 0.3

    def pad(a, n, *shape):
        t = torch.zeros(*a.shape[:-1], n)
        t[..., :a.shape[-1]] = torch.from_numpy(a)
        return t.to(dtype)
    x = torch.cat([pad(q, dp).reshape(L, -1), pad(gate, dvp).reshape(L, -1)], dim=1).to(dev)

    def heads(a, n):
        t = torch.zeros(H, n, rp, dtype=dtype)
        t[:, :a.shape[1], :rank] = torch.from_numpy(a).to(dtype)
        return t.reshape(H * n, rp).to(dev)
    case = dict(x=x, c=pad(c, rp).to(dev), uk=heads(uk, dp), uv=heads(uv, dvp), H=H, dp=dp, dvp=dvp, vdim=vdim, window=window,
                scale=scale, rp=rp, rank=rank)
    r = lambda a: torch.from_numpy(a).to(dtype).double().numpy()
    q, c, uk, uv, gate = (r(a) for a in (q, c, uk, uv, gate))
    kk, vv = np.einsum("hdr,lr->lhd", uk, c), np.einsum("hdr,lr->lhd", uv, c)
    want = np.stack([lo.window_softmax(q[:, h] @ kk[:, h].T * scale, window) @ vv[:, h] for h in range(H)], 1)
    return case, want * lo.sigmoid(gate)


def latent_run(dev, case, start, n, form, capacity):
    """Positions start .. start + n - 1 with everything before them cached."""
    H, dp, dvp, dtype = case["H"], case["dp"], case["dvp"], case["x"].dtype
    R = n + 1
    x = torch.full((R, case["x"].shape[1]), 3.0, dtype=dtype, device=dev)
    x[:n] = case["x"][start:start + n]
    cache = torch.full((capacity, case["rp"]), 50.0, dtype=dtype, device=dev)      # rows past the length
    out = torch.full((R, hops.round_up(H * dvp, 64)), 7.0, dtype=dtype, device=dev)
    length, live = i32(dev, start), i32(dev, n)
    q, gate = x[:, :H * dp], x[:, H * dp:]
    cache[:start + n] = case["c"][:start + n]
    if form == "absorbed":
        ws = torch.full((hops.latent_decode_workspace_bytes(R, H, case["rp"], case["window"], capacity),), 255,
                        dtype=torch.uint8, device=dev)
        hops.latent_decode(q, cache, case["uk"], case["uv"], gate, out, length, live, R, H, dp, dvp, case["window"],
                           case["scale"], ws)
    else:
        back = min(case["window"] - 1, capacity)
        S = hops.round_up(back + R, 128)
        k = torch.zeros(S, H * dp, dtype=dtype, device=dev)
        vt = torch.zeros(H * dvp, S, dtype=dtype, device=dev)
        kw = dict(M=back + R, n_dev=live, len_dev=length, back=back)
        hops.dense(cache, case["uk"], k, **kw)
        hops.dense(cache, case["uv"], vt, hops.OUT_TRANSPOSED, **kw)
        hops.window_attention(q, k, vt, gate, out, length, live, R, H, dp, dvp, case["window"], back, case["scale"])
    assert bool((out[n:] == 7).all())
    return out[:n, :H * dvp].reshape(n, H, dvp)[..., :case["vdim"]]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dim,vdim,rank,window", [(1, 32, 16, 64, 1), (2, 40, 24, 72, 50), (3, 64, 64, 128, 64), (5, 16, 40, 100, 65),
                                                    (2, 128, 128, 512, 97), (17, 24, 16, 64, 129), (1, 200, 250, 600, 40), (2, 32, 48, 1000, 5000)])
def test_latent_attention_forms(dev, dtype, H, dim, vdim, rank, window):
    L = 230
    case, want = latent_case(dev, dtype, L, H, dim, vdim, rank, window, dim ** -0.5)
    for form, portions in (("absorbed", ((0, 1), (1, 2), (40, 16), (63, 3), (200, 7), (229, 1))),
                           ("window", ((0, 17), (0, L), (1, 64), (49, 70), (64, 128), (130, 100), (228, 2)))):
        for start, n in portions:
            got = latent_run(dev, case, start, n, form, capacity=L + 20)
            assert rel(got, want[start:start + n]) < tol(dtype, 5e-3, 3e-5), (form, start, n)


@pytest.mark.parametrize("window", [33, 64, 65, 100])
def test_latent_window_edges(dev, window):
    """One key stands out for one query: it decides the output just inside the window and is absent
    just outside, as the first and as the last row of a portion, wherever tiles and splits begin."""
    L = 210
    for i in (window - 1, window, 127, 128, 192, L - 1):
        for back in (0, 1, window - 1, window, window + 1):
            j = i - back
            if j < 0:
                continue
            case, want = latent_case(dev, torch.float32, L, 2, 24, 16, 64, window, 0.2, peak=(i, j))
            if back:        # with a window that shows the key where this one hides it, or the reverse, it shows
                moved = latent_case(dev, torch.float32, L, 2, 24, 16, 64, back + (back >= window), 0.2, peak=(i, j))[1]
                assert np.abs(moved[i] - want[i]).max() > 0.1
            for form, portions in (("absorbed", ((i, 1), (max(0, i - 5), min(6, i + 1)))),
                                   ("window", ((i, 1), (0, i + 1), (max(0, i - 40), min(41, i + 1))))):
                for start, n in portions:
                    got = latent_run(dev, case, start, n, form, capacity=L)
                    assert rel(got, want[start:start + n]) < 1e-4, (i, j, form, start)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rank,true", [(64, 64), (128, 100), (512, 500)])
def test_latent_append(dev, dtype, rank, true):
    x = torch.zeros(7, rank + 32, dtype=dtype, device=dev)
    x[:, :true] = rand(dev, dtype, 7, true, std=2.0)
    w = torch.zeros(rank, device=dev)
    w[:true] = 1 + 0.2 * rand(dev, torch.float32, true, seed=1)
    want = lo.norm_plain(x[:, :true].double().cpu().numpy(), w[:true].double().cpu().numpy(), 1e-3)
    cache = torch.full((20, rank), 7.0, dtype=dtype, device=dev)
    hops.latent_append(x[:, :rank], w, 1e-3, true, cache, i32(dev, 9), i32(dev, 6), 7)
    assert rel(cache[9:15, :true], want[:6]) < tol(dtype, 4e-3)
    assert bool((cache[:9] == 7).all()) and bool((cache[15:] == 7).all()) and not cache[9:15, true:].any()
    hops.latent_append(x[:, :rank], w, 1e-3, true, cache, i32(dev, 17), i32(dev, 7), 7)      # never past the buffer
    assert rel(cache[17:, :true], want[:3]) < tol(dtype, 4e-3)
    # the same rows appended by the absorbed form's own launch
    case, _ = latent_case(dev, dtype, 12, 2, 24, 16, min(true, 64), 9, 0.2)
    if rank == 64:
        a, b = (torch.zeros(20, 64, dtype=dtype, device=dev) for _ in range(2))
        out, ws = torch.zeros(3, 64, dtype=dtype, device=dev), torch.zeros(1 << 20, dtype=torch.uint8, device=dev)
        hops.latent_decode(case["x"][:, :64], a, case["uk"], case["uv"], case["x"][:, 64:], out, i32(dev, 4), i32(dev, 3), 3, 2, 32,
                           16, 9, 0.2, ws, append=(x[:, :64], w, 1e-3, true))
        hops.latent_append(x[:, :64], w, 1e-3, true, b, i32(dev, 4), i32(dev, 3), 3)
        assert torch.equal(a, b)
