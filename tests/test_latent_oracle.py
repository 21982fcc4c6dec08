"""The plain statement of the latent-attention decoder held to facts that do not
come from it: closed forms, hand-made cases, recurrences cut at any token."""
import math

import numpy as np
import pytest

import latent_model as lm
import latent_oracle as lo
import mixed_model as mm


def test_norm_of_a_constant_row():
    x = np.full((2, 8), 3.0)
    assert np.allclose(lo.root_mean_square_norm(x, np.arange(8.0), 0.0), np.arange(8.0))
    # the epsilon is added to the mean of the squares
    assert np.allclose(lo.root_mean_square_norm(x, np.ones(8), 16.0), 3.0 / 5.0)


def test_rotation_pairs_halves_and_depends_on_distance_only():
    rng = np.random.default_rng(1)
    rot = {"dims": 8, "base": 100.0}
    x = rng.standard_normal((1, 12))
    assert np.allclose(lo.rotate_halves(x, [0], rot), x)
    turned = lo.rotate_halves(x, [1], rot)[0]
    assert np.allclose(turned[0], x[0, 0] * math.cos(1) - x[0, 4] * math.sin(1))
    assert np.allclose(turned[4], x[0, 4] * math.cos(1) + x[0, 0] * math.sin(1))
    assert np.array_equal(turned[8:], x[0, 8:])
    k = rng.standard_normal((1, 12))
    scores = [float(lo.rotate_halves(x, [p + 5], rot)[0] @ lo.rotate_halves(k, [p], rot)[0])
              for p in (0, 3, 40)]
    assert np.allclose(scores, scores[0])


def test_stretched_frequencies():
    plain, one = lo.frequencies(32, 10000.0)
    assert one == 1.0 and plain[0] == 1.0
    scaling = {"factor": 8.0, "original": 512, "fast": 32.0, "slow": 1.0}
    stretched, magnitude = lo.frequencies(32, 10000.0, scaling)
    assert magnitude == pytest.approx(1.0 + 0.1 * math.log(8.0))
    # the fastest dimensions stay, the slowest are divided, no ratio rises on the way
    ratio = stretched / plain
    assert ratio[0] == 1.0 and ratio[-1] == pytest.approx(1.0 / 8.0)
    assert np.all(np.diff(ratio) <= 1e-15)
    # a dimension that turns once over the original length ends the ramp
    last = math.ceil(16 * math.log(512 / (2 * math.pi)) / math.log(10000.0))
    assert ratio[last - 1] > 1.0 / 8.0 and ratio[last] == pytest.approx(1.0 / 8.0)
    # a factor of one changes nothing
    same, magnitude = lo.frequencies(32, 10000.0, dict(scaling, factor=1.0))
    assert np.allclose(same, plain) and magnitude == 1.0


@pytest.mark.parametrize("window", [None, 1, 4, 100])
def test_what_a_position_sees(window):
    seen = lo.visible(9, window)
    for i in range(9):
        for j in range(9):
            assert seen[i, j] == (j <= i and (window is None or i - j < window))


def test_attention_over_one_key_returns_its_value():
    rng = np.random.default_rng(2)
    q, k, v = (rng.standard_normal((5, n)) for n in (6, 6, 3))
    assert np.allclose(lo.attend(q, k, v, 0.7, lo.visible(5, 1)), v)
    # equal scores: the mean of what is seen
    assert np.allclose(lo.attend(0 * q, k, v, 0.7, lo.visible(5, 2))[3], v[2:4].mean(0))


def test_decay_is_a_power_of_the_logistic():
    z = np.array([-40.0, -2.0, 0.0, 3.0, 40.0])
    assert np.allclose(lo.channel_decay(z, 1.0), 1.0 / (1.0 + np.exp(-z)))
    assert np.allclose(lo.channel_decay(z, 4.0) ** 4, 1.0 / (1.0 + np.exp(-z)))


@pytest.mark.parametrize("cut", [1, 4, 9])
def test_recurrence_in_closed_form_and_cut_anywhere(cut):
    rng = np.random.default_rng(cut)
    q, k = rng.standard_normal((2, 10, 4))
    v = rng.standard_normal((10, 6))
    alpha = rng.uniform(0.5, 1.0, (10, 4))
    out, end = lo.gated_recurrence(q, k, v, alpha, np.zeros((4, 6)))
    for t in range(10):
        want = sum(np.sum(q[t] * k[s] * np.prod(alpha[s + 1:t + 1], axis=0)) * v[s]
                   for s in range(t + 1))
        assert np.allclose(out[t], want)
    head, middle = lo.gated_recurrence(q[:cut], k[:cut], v[:cut], alpha[:cut],
                                       np.zeros((4, 6)))
    tail, last = lo.gated_recurrence(q[cut:], k[cut:], v[cut:], alpha[cut:], middle)
    assert np.allclose(out, np.concatenate([head, tail])) and np.allclose(end, last)


def test_prefix_of_a_sequence_does_not_see_the_rest():
    config = lm.configuration(
        40, 24, [lm.gla(2, 5, 3), lm.windowed_latent(2, 6, 4, 5, 7, 9, 4), lm.latent(3, 8, 4, 6)],
        [0, 20, 12])
    weights = mm.float64(lm.random_weights(config, 3))
    tokens = np.random.default_rng(0).integers(0, 40, 14)
    whole, streams = lo.forward(config, weights, tokens)
    part, _ = lo.forward(config, weights, tokens[:9])
    assert np.allclose(whole[:9], part) and streams.shape == (3, 14, 24)


def test_every_sublayer_adds_a_row_of_known_size():
    """The norm behind a sublayer makes what it adds independent of the scale of
    its output projection."""
    config = lm.configuration(40, 24, [lm.latent(3, 8, 4, 6)], [12], eps=1e-12, residual=0.5)
    weights = mm.float64(lm.random_weights(config, 3))
    tokens = [3, 9, 1]
    _, plain = lo.forward(config, weights, tokens)
    weights["l0.mix.o"] *= 7.0
    weights["l0.mlp.down"] *= 0.2
    assert np.allclose(lo.forward(config, weights, tokens)[1], plain)
