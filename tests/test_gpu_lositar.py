"""The Lositar decoder as it is served, against the plain implementation: prompts, portions, decoding,
reused buffers, graphs, generation, the trace runner."""
import io
import json

import numpy as np
import pytest
import torch

from mlx_eagle_spec_decoding_tree_amd import cache, checkpoint, generate, hybrid, lositar, trace
from oracle import lositar_oracle as lo
from lositar_util import CONFIGS, as_numpy, config, gla, latent, rms_err, sequence, want_logits, weights

pytestmark = pytest.mark.gpu
TOL = {torch.float32: 2e-5, torch.bfloat16: 4e-2}


def build(dev, name, dtype=torch.float32):
    return lositar.build(CONFIGS[name], weights(name), dev, dtype)


def feed_all(stream, ids, portions):
    """Logits of every position, fed in portions (the last size repeats)."""
    out, at, k = [], 0, 0
    while at < len(ids):
        n = min(portions[min(k, len(portions) - 1)], len(ids) - at)
        out.append(stream.feed(ids[at:at + n], want=range(n)).double().cpu().numpy())
        at, k = at + n, k + 1
    return np.concatenate(out)


@pytest.mark.parametrize("dtype", list(TOL))
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_and_residual_stream(dev, name, dtype):
    n = 200
    model, ids = build(dev, name, dtype), sequence(name, n)
    stream = model.stream(300)
    tol = TOL[dtype] * (4 if name == "sharp" and dtype == torch.bfloat16 else 1)
    assert rms_err(stream.feed(ids, want=range(n)).cpu(), want_logits(name, n)) < tol
    # the residual stream after every layer
    taps, got = [], []
    lo.forward(CONFIGS[name], as_numpy(weights(name)), ids[:70], tap=lambda i, x: taps.append(x))
    stream.clear()
    stream.feed(ids[:70], tap=lambda s, i, h: got.append(h[:, :CONFIGS[name]["width"]].double().cpu().numpy()))
    assert len(got) == len(taps) == len(CONFIGS[name]["layers"])
    for i, (a, b) in enumerate(zip(got, taps)):
        assert np.abs(a - b).max() / np.sqrt(np.mean(b * b)) < 10 * tol, i


@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("portions", [(1,), (2,), (3,), (5, 17, 2, 1), (64,), (63, 2), (65, 1, 1, 66), (16, 130), (129,)])
def test_portions_give_the_same_logits(dev, name, portions):
    n = 200
    stream = build(dev, name).stream(256)
    assert rms_err(feed_all(stream, sequence(name, n), portions), want_logits(name, n)) < TOL[torch.float32]


@pytest.mark.parametrize("name", ["mixed", "sharp"])
def test_portions_in_bf16(dev, name):
    n = 200
    model = build(dev, name, torch.bfloat16)
    tol = TOL[torch.bfloat16] * (4 if name == "sharp" else 1)
    for portions in ((1,), (2, 3), (60, 1, 1, 40)):
        assert rms_err(feed_all(model.stream(256), sequence(name, n), portions), want_logits(name, n)) < tol, portions


@pytest.mark.parametrize("name", ["mixed", "linear_only", "latent_only"])
def test_first_tokens(dev, name):
    model = build(dev, name)
    stream = model.stream(64)
    for n in (1, 2, 3):
        stream.clear()
        assert rms_err(stream.feed(sequence(name, 9)[:n], want=range(n)).cpu(), want_logits(name, 9)[:n]) < TOL[torch.float32]
    stream.clear()
    assert rms_err(feed_all(stream, sequence(name, 9), (1,)), want_logits(name, 9)) < TOL[torch.float32]


def test_long_decoding_and_a_full_cache(dev):
    """Hundreds of decoded tokens, window and state passing over them, up to the last position."""
    name, n = "mixed", 420
    stream = build(dev, name).stream(n)
    ids = sequence(name, n)
    got = feed_all(stream, ids, (37, 1))
    assert rms_err(got, want_logits(name, n)) < TOL[torch.float32]
    assert stream.length == n
    with pytest.raises(ValueError):
        stream.feed([1])
    assert stream.length == n
    cfg = config(gla(), latent(), positions=20)
    short = hybrid.Model(lositar.args_from_config(cfg), lositar.arrange(lositar.args_from_config(cfg), _random(cfg)), dev)
    s = short.stream(1000)
    assert s.capacity == 20
    with pytest.raises(ValueError):
        s.feed([1] * 21)
    with pytest.raises(ValueError):
        s.feed([203])
    with pytest.raises(ValueError):
        s.feed([-1])
    with pytest.raises(ValueError):
        s.feed([])
    with pytest.raises(ValueError):
        s.feed([1, 2], want=[2])


def _random(cfg):
    from mlx_eagle_spec_decoding_tree_amd import synth
    return synth.make_lositar_weights(cfg)


@pytest.mark.parametrize("name", list(CONFIGS))
def test_buffers_serve_the_next_sequence(dev, name):
    """A cleared stream is as good as a new one, whatever lies in its buffers; streams that live at the
    same time do not touch each other."""
    model = build(dev, name)
    a, b = model.stream(256), model.stream(100)
    feed_all(a, sequence(name, 250, seed=9), (100, 1, 80))
    a.clear()
    ids = sequence(name, 90)
    got_a, got_b = [], []
    for at, n in ((0, 30), (30, 1), (31, 1), (32, 40), (72, 18)):
        got_a.append(a.feed(ids[at:at + n], want=range(n)).cpu().numpy())
        other = sequence(name, 90, seed=4)
        got_b.append(b.feed(other[at:at + n], want=range(n)).cpu().numpy())
    assert rms_err(np.concatenate(got_a), want_logits(name, 90)) < TOL[torch.float32]
    assert rms_err(np.concatenate(got_b), want_logits(name, 90, seed=4)) < TOL[torch.float32]
    a.clear()
    assert rms_err(a.feed(ids, want=[89]).cpu(), want_logits(name, 90)[89:]) < TOL[torch.float32]


@pytest.mark.parametrize("dtype", list(TOL))
def test_captured_passes_equal_eager_ones(dev, dtype):
    """A pass is captured at its second use: every replay, with other work in between, gives what the
    eager launches give, bit for bit."""
    model, ids = build(dev, "mixed", dtype), sequence("mixed", 330)
    portions = (40, 1, 1, 1, 40, 1, 40, 2, 2, 40, 1, 3, 3, 40, 70, 1)
    eager = feed_all(model.stream(400, graphs=False), ids, portions)
    s = model.stream(400)
    assert np.array_equal(feed_all(s, ids, portions), eager)
    assert s.passes[1].graph is not None and s.passes[64].graph is not None
    s.clear()
    torch.randn(1000, device=dev).sum().item()
    assert np.array_equal(feed_all(s, ids, portions), eager)


def test_module_call_matches_the_stream(dev):
    model, ids = build(dev, "mixed"), sequence("mixed", 80)
    c = cache.make_prompt_cache(model, capacity=128)
    t = torch.tensor(ids, device=dev)
    y = torch.cat([model(t[None, :50], cache=c), model(t[None, 50:51], cache=c), model(t[None, 51:], cache=c)], dim=1)
    assert y.shape == (1, 80, 203) and rms_err(y[0].cpu(), want_logits("mixed", 80)) < TOL[torch.float32]
    assert c[0].offset == c[1].offset == 80
    c.clear()
    assert rms_err(model(t[None, :5], cache=c)[0].cpu(), want_logits("mixed", 80)[:5]) < TOL[torch.float32]
    with pytest.raises(NotImplementedError):
        model(t[None], cache=c, mask=torch.zeros(1, device=dev))


@pytest.mark.parametrize("name", ["mixed", "latent_only", "linear_only"])
def test_greedy_generation(dev, name):
    """Every token is the oracle's argmax for the sequence so far (or within rounding of it)."""
    prompt, n = list(sequence(name, 45)), 40
    model = build(dev, name)
    tokens = generate.generate(model, prompt, n)
    assert len(tokens) == n
    y = lo.forward(CONFIGS[name], as_numpy(weights(name)), prompt + tokens)
    for i, t in enumerate(tokens):
        row = y[len(prompt) - 1 + i]
        assert row.max() - row[t] < 1e-4 * np.sqrt(np.mean(row * row)), i
    stream = model.stream(200)
    assert generate.generate(model, prompt, n, prefill_step_size=7, stream=stream) == tokens
    assert generate.generate(model, prompt, n, stream=stream) == tokens           # reused, decode graph captured
    assert stream.length == len(prompt) + n - 1
    # a generated sequence can be continued by feeding
    assert rms_err(stream.feed([tokens[-1]]).cpu(), y[-1:]) < TOL[torch.float32]


def test_generation_of_more_tokens_than_the_output_buffer(dev, monkeypatch):
    model, prompt = build(dev, "mixed"), list(sequence("mixed", 20))
    want = generate.generate(model, prompt, 60)
    monkeypatch.setattr(hybrid.HybridRunner, "MAX_OUT", 16)
    assert generate.generate(model, prompt, 60) == want


def save(tmp_path, name):
    from safetensors.torch import save_file
    (tmp_path / "config.json").write_text(json.dumps(CONFIGS[name]))
    save_file(weights(name), str(tmp_path / "model.safetensors"))
    return str(tmp_path)


@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_trace_runner(dev, tmp_path, dtype):
    path, ids = save(tmp_path, "mixed"), sequence("mixed", 120)
    other = sequence("mixed", 60, seed=3)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": ids[:70], "want": [0, 69]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": ids[70:71], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": ids[71:], "want": [48, 0]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": other, "want": [59, 2]}], "end": ["b"]}]
    out = io.StringIO()
    rc = trace.main(["--model", path, "--dtype", dtype, "--out", str(tmp_path), "--max-tokens", "120"],
                    stdin=io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n"), stdout=out)
    assert rc == 0 and out.getvalue().split("\n")[:4] == [f"done {i}" for i in range(4)]
    assert not (tmp_path / "1.f32").exists()
    tol = TOL[getattr(torch, dtype)]
    for s, (full, rows) in {0: (want_logits("mixed", 120), [0, 69]), 2: (want_logits("mixed", 120), [119, 71]),
                            3: (want_logits("mixed", 60, seed=3), [59, 2])}.items():
        got = np.fromfile(tmp_path / f"{s}.f32", "<f4").reshape(2, 203)
        assert rms_err(got, full[rows]) < tol, s


def test_generation_command(dev, tmp_path, capsys):
    path, prompt = save(tmp_path, "mixed"), list(sequence("mixed", 30))
    assert generate.main(["--model", path, "--dtype", "float32", "--tokens", ",".join(map(str, prompt)), "--max-tokens", "12"]) == 0
    line = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert line["prompt_tokens"] == 30
    model, _ = checkpoint.load_model(path, dev, dtype="float32")
    assert line["tokens"] == generate.generate(model, prompt, 12)


def test_llama_streams_generate_the_module_paths_tokens(dev):
    """The same entry point over the quantised decoder."""
    from mlx_eagle_spec_decoding_tree_amd import llama, ops, synth
    args = synth.tiny(layers=2, hidden=256, inter=512, heads=4, kv_heads=2, head_dim=64, vocab=1024)
    model = llama.Model.from_numpy(args, synth.make_model_weights(args, seed=3), dev)
    prompt = torch.from_numpy(np.random.default_rng(1).integers(0, 1024, 70)).to(dev)
    for graphs in (True, False):
        stream = generate.open_stream(model, 128, graphs)
        tokens = generate.generate(model, prompt, 20, stream=stream)
        ref = cache.make_prompt_cache(model, capacity=128)
        logits = model(prompt[None], cache=ref)[0, -1].float()
        for t in tokens:
            assert float(logits.max() - logits[t]) < 0.06
            logits = model(torch.tensor([[t]], device=dev), cache=ref)[0, -1].float()
        assert generate.generate(model, prompt, 20, stream=stream) == tokens
        assert stream.length == 89
    stream.clear()
    y = stream.feed(prompt[:40], want=[0, 39])
    assert y.shape == (2, 1024) and float((stream.feed(prompt[40:])[0] - model(prompt[None], cache=cache.make_prompt_cache(
        model, capacity=128))[0, -1].float()).abs().max()) < 0.1
    with pytest.raises(ValueError):
        stream.feed(prompt)
