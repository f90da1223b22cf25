"""CPU: the Davasun oracle against itself and against facts its formulas imply (continuation, limits, other ways to write the
same sums), so that the GPU tests compare with something that has been looked at from a second side."""
import numpy as np
import pytest

from davasun_util import bits_and_values, config, latent, mlstm, tensors
from oracle import davasun_oracle as do


@pytest.fixture(scope="module")
def model(t12):
    cfg = config([mlstm(), latent(), mlstm(heads=3, dim=8, vdim=16, ff=24)], width=48, loop=(1, 3, 2))
    return cfg, {k: bits_and_values(v)[1] for k, v in tensors(cfg, 1).items()}


def test_portions_continue_a_sequence(model):
    cfg, t = model
    tok = np.random.default_rng(2).integers(0, 97, 40)
    whole = do.forward(cfg, t, tok)
    for cuts in ([1] * 40, [2, 7, 31], [39, 1]):
        st, at, parts = do.State(cfg), 0, []
        for c in cuts:
            parts.append(do.forward(cfg, t, tok[at:at + c], st))
            at += c
        assert np.allclose(np.concatenate(parts), whole, atol=1e-9)


def test_order_of_runs():
    layers = [mlstm()] * 5
    assert do.order(config(layers)) == [0, 1, 2, 3, 4]
    assert do.order(config(layers, loop=(1, 3, 3))) == [0, 1, 2, 1, 2, 1, 2, 3, 4]
    assert do.order(config(layers, loop=(0, 5, 2))) == [0, 1, 2, 3, 4] * 2
    assert do.order(config(layers, loop=(4, 5, 1))) == [0, 1, 2, 3, 4]


def test_every_run_of_a_looped_layer_has_a_past_of_its_own(model):
    cfg, t = model
    st = do.State(cfg)
    do.forward(cfg, t, [3, 5, 8], st)
    a, b = [r for r, i in zip(st.runs, do.order(cfg)) if i == 2]
    assert np.abs(a["S"] - b["S"]).max() > 1e-3


def test_memory_is_a_weighted_sum_of_its_tokens():
    """Unrolled: every past token enters with exp(its input gate + the forget gates behind it), over the same scale."""
    rng = np.random.default_rng(3)
    T, d, e = 12, 5, 4
    q, k, v = rng.standard_normal((T, 1, d)), rng.standard_normal((T, 1, d)), rng.standard_normal((T, 1, e))
    i, f = 3 * rng.standard_normal((T, 1)), do.log_sigmoid(2 * rng.standard_normal((T, 1)))
    o, *_ = do.memory_scan(q, k, v, i, f, np.zeros((1, d, e)), np.zeros((1, d)), np.zeros(1))
    m = 0.0
    for t in range(T):
        m = max(f[t, 0] + m, i[t, 0])
        w = np.array([np.exp(i[s, 0] + f[s + 1:t + 1, 0].sum()) for s in range(t + 1)]) * (k[:t + 1, 0] @ q[t, 0])
        want = w @ v[:t + 1, 0] / (max(abs(w.sum()), 1.0) + 1e-6 * np.exp(m))
        assert np.allclose(o[t, 0], want, rtol=1e-10)


def test_the_running_maximum_starts_at_zero():
    """A first token with a small input gate is scaled against e^0, not against itself."""
    one = np.ones(1)
    S, n, m, o = do.memory_step(np.zeros((1, 1)), np.zeros(1), 0.0, one, one, one, -5.0, -0.1)
    assert m == -0.1 and np.isclose(S[0, 0], np.exp(-4.9)) and np.isclose(o[0], np.exp(-4.9) / (np.exp(0.1) + 1e-6))


def test_rotation_keeps_lengths_and_depends_on_distance():
    rng = np.random.default_rng(4)
    q, k = rng.standard_normal((2, 1, 10))
    dot = lambda a, b: float(np.sum(do.rotate_half(q, [a], 50.0) * do.rotate_half(k, [b], 50.0)))
    assert np.isclose(dot(9, 4), dot(105, 100)) and not np.isclose(dot(9, 4), dot(9, 5))
    assert np.isclose(np.linalg.norm(do.rotate_half(q, [77], 50.0)), np.linalg.norm(q))
    x = np.zeros((1, 4))
    x[0, 0] = 1.0                                              # partner of coordinate 0 is coordinate 2
    y = do.rotate_half(x, [1], 50.0)[0]
    assert np.isclose(y[0], np.cos(1)) and np.isclose(y[2], np.sin(1)) and y[1] == y[3] == 0


def test_attention_is_causal_and_normalised():
    rng = np.random.default_rng(5)
    q, k, v = rng.standard_normal((6, 2, 4)), rng.standard_normal((6, 2, 4)), np.ones((6, 2, 3))
    assert np.allclose(do.causal_attention(q, k, v, 0.7, 0), 1.0)
    v = rng.standard_normal((6, 2, 3))
    assert np.allclose(do.causal_attention(q, k, v, 0.7, 0)[0], v[0])
    assert np.allclose(do.causal_attention(q[5:], k, v, 0.7, 5), do.causal_attention(q, k, v, 0.7, 0)[5:])


def test_clamped_unit():
    assert np.allclose(do.clamped_glu(np.array([9.0]), np.array([-9.0]), 2.0), 2.0 * do.sigmoid(3.404) * -1.0)
    assert np.allclose(do.clamped_glu(np.array([-9.0]), np.array([9.0]), 2.0), -9.0 * do.sigmoid(-9 * 1.702) * 3.0)
    assert np.allclose(do.clamped_glu(np.array([0.5]), np.array([0.25]), 2.0), 0.5 * do.sigmoid(0.851) * 1.25)
