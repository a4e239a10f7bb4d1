"""The plain Lositar implementation against properties that follow from its equations."""
import numpy as np
import pytest

from oracle import lositar_oracle as lo
from lositar_util import CONFIGS, as_numpy, rms_err, sequence, want_logits, weights


def test_norms_and_activations():
    x = np.array([[3.0, -4.0, 0.0, 0.0]])
    assert np.allclose(lo.unit_rms(x, 0.0), x / 2.5)
    assert np.allclose(lo.unit_rms(x, 2.75), x / 3.0)                 # eps inside the root
    assert np.allclose(lo.norm_around_one(x, np.zeros(4), 0.0), lo.norm_plain(x, np.ones(4), 0.0))
    assert np.allclose(lo.relu_squared(np.array([-2.0, 0.0, 3.0])), [0, 0, 9])
    z = np.array([-800.0, -3.0, 0.0, 3.0, 800.0])
    assert np.allclose(lo.sigmoid(z), [0, 1 / (1 + np.exp(3)), 0.5, 1 / (1 + np.exp(-3)), 1])
    assert np.allclose(lo.log_sigmoid(z)[[0, 4]], [-800, 0])
    assert np.allclose(lo.gla_decay(z[1:4], 4.0), lo.sigmoid(z[1:4]) ** 0.25)


def test_recurrence_equals_its_closed_form():
    """o_t = sum_{s <= t} (prod_{s < u <= t} alpha_u * k_s . q_t) v_s"""
    rng = np.random.default_rng(0)
    L, H, dk, dv = 9, 2, 3, 4
    q, k = rng.normal(size=(2, L, H, dk))
    v = rng.normal(size=(L, H, dv))
    a = rng.uniform(0.2, 1.0, size=(L, H, dk))
    o, S = lo.gla_recurrence(q, k, v, a)
    for t in range(L):
        want = np.zeros((H, dv))
        for s in range(t + 1):
            w = np.prod(a[s + 1:t + 1], axis=0) * k[s] * q[t]
            want += w.sum(-1)[:, None] * v[s]
        assert np.allclose(o[t], want)
    head, mid = lo.gla_recurrence(q[:4], k[:4], v[:4], a[:4])
    tail, end = lo.gla_recurrence(q[4:], k[4:], v[4:], a[4:], mid)
    assert np.allclose(np.concatenate([head, tail]), o) and np.allclose(end, S)


def test_window_sees_itself_and_the_tokens_before_it():
    for size in (1, 2, 5):
        p = lo.window_softmax(np.zeros((7, 7)), size)
        for i in range(7):
            n = min(size, i + 1)
            assert np.allclose(p[i], [(1 / n if i - n < j <= i else 0) for j in range(7)])


def test_logits_do_not_depend_on_what_follows():
    for name in CONFIGS:
        full = want_logits(name, 70)
        part = lo.forward(CONFIGS[name], as_numpy(weights(name)), sequence(name, 70)[:33])
        assert np.allclose(full[:33], part, atol=1e-9)


@pytest.mark.parametrize("name,mistake", [("sharp", (("window", 1),)), ("sharp", (("window", -1),)), ("mixed", (("window", 1),)),
                                          ("mixed", (("drop_state_at", 20),)), ("linear_only", (("drop_state_at", 20),)),
                                          ("sharp", (("pos_shift", 1),))])
def test_mistakes_would_show(name, mistake):
    """The tests' weights are such that a window off by one, a lost state or shifted positions move the
    logits by far more than the tolerances of the GPU tests."""
    n = 120
    assert rms_err(want_logits(name, n, mistake=mistake), want_logits(name, n)) > 0.05
