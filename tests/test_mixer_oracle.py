"""The plain statement of the mixed-layer decoder held to facts that do not come
from it: closed forms, hand-made cases, and agreement of its own recurrences
with their definitions cut at any token."""
import numpy as np
import pytest

import mixed_model as mm
import mixer_oracle as mo


def test_rotation_turns_pairs_and_depends_on_distance_only():
    rng = np.random.default_rng(1)
    q, k = rng.standard_normal((2, 1, 1, 12))
    unturned = mo.rotate_interleaved(q, np.array([0.0]), 8, 100.0)
    assert np.array_equal(unturned, q)
    one = mo.rotate_interleaved(q, np.array([1.0]), 8, 100.0)[0, 0]
    u, v = q[0, 0, :2]
    assert np.allclose(one[:2], [u * np.cos(1) - v * np.sin(1), v * np.cos(1) + u * np.sin(1)])
    assert np.array_equal(one[8:], q[0, 0, 8:])
    scores = [np.sum(mo.rotate_interleaved(q, np.array([p + 5.0]), 8, 100.0) *
                     mo.rotate_interleaved(k, np.array([float(p)]), 8, 100.0))
              for p in (0, 3, 40)]
    assert np.allclose(scores, scores[0])


@pytest.mark.parametrize("window,sinks", [(1, 0), (4, 0), (4, 2), (3, 5), (100, 1)])
def test_window_with_kept_first_tokens(window, sinks):
    seen = mo.visible_window(np.arange(12), np.arange(12), window, sinks)
    for i in range(12):
        for j in range(12):
            assert seen[i, j] == (j <= i and (i - j < window or j < sinks))


def test_head_mixing_with_the_identity_is_plain_attention():
    rng = np.random.default_rng(2)
    q, k, v = (rng.standard_normal(s) for s in ((6, 4, 8), (6, 2, 8), (6, 2, 5)))
    at = np.arange(6)
    plain = mo.attention_core(q, k, v, at, at, 0.5, 3, 1, np.eye(4))
    swapped = mo.attention_core(q, k, v, at, at, 0.5, 3, 1, np.eye(4)[[1, 0, 3, 2]])
    # heads 0 and 1 share a key/value head: their weights change places
    assert np.allclose(plain[:, [1, 0, 3, 2]], swapped)
    assert np.allclose(plain[0, 0], v[0, 0])


@pytest.mark.parametrize("cut", [1, 4, 9])
def test_recurrences_may_be_cut_anywhere(cut):
    rng = np.random.default_rng(cut)
    r, k, v = rng.standard_normal((3, 10, 6))
    w, a = rng.uniform(0.5, 1.0, (2, 10, 6))
    zero = np.zeros((6, 6))
    whole, end = mo.delta_recurrence(r, k, v, w, a, zero)
    head, middle = mo.delta_recurrence(r[:cut], k[:cut], v[:cut], w[:cut], a[:cut], zero)
    tail, last = mo.delta_recurrence(r[cut:], k[cut:], v[cut:], w[cut:], a[cut:], middle)
    assert np.allclose(whole, np.concatenate([head, tail])) and np.allclose(end, last)
    bonus = rng.standard_normal(6)
    whole, end = mo.wkv_recurrence(r, k, v, w, bonus, zero)
    head, middle = mo.wkv_recurrence(r[:cut], k[:cut], v[:cut], w[:cut], bonus, zero)
    tail, last = mo.wkv_recurrence(r[cut:], k[cut:], v[cut:], w[cut:], bonus, middle)
    assert np.allclose(whole, np.concatenate([head, tail])) and np.allclose(end, last)


def test_recurrences_in_closed_form():
    rng = np.random.default_rng(7)
    r, k, v = rng.standard_normal((3, 5, 4))
    # no removal, constant decay: a geometric sum of outer products
    decay = np.full((5, 4), 0.9)
    out, _ = mo.delta_recurrence(r, k, v, decay, np.zeros((5, 4)), np.zeros((4, 4)))
    for t in range(5):
        want = sum(0.9 ** (t - s) * np.dot(r[t], k[s]) * v[s] for s in range(t + 1))
        assert np.allclose(out[t], want)
    # the same with a bonus of 1 leaves the current token's weight at 1
    out, _ = mo.wkv_recurrence(r, k, v, decay, np.ones(4), np.zeros((4, 4)))
    for t in range(5):
        want = np.dot(r[t], k[t]) * v[t] + sum(
            0.9 ** (t - 1 - s) * np.dot(r[t], k[s]) * v[s] for s in range(t))
        assert np.allclose(out[t], want)
    # full removal along a repeated key: the old value is replaced
    key = np.array([[2.0, 0, 0, 0]] * 2)
    out, state = mo.delta_recurrence(key, key, v[:2], np.ones((2, 4)), np.ones((2, 4)),
                                     np.zeros((4, 4)))
    assert np.allclose(state[0], 2.0 * v[1], atol=1e-5)


def test_prefix_of_a_sequence_does_not_see_the_rest():
    config = mm.configuration(
        40, 24, [mm.attention(2, 1, 8, 6, 5, 2), mm.wkv(2, 5), mm.general_delta(3, 4)],
        [20, 0, 12])
    weights = mm.float64(mm.random_weights(config, 3))
    tokens = np.random.default_rng(0).integers(0, 40, 14)
    whole, streams = mo.forward(config, weights, tokens)
    part, _ = mo.forward(config, weights, tokens[:9])
    assert np.allclose(whole[:9], part) and streams.shape == (3, 14, 24)
