"""The float64 oracle of the Kamelorn tests against properties of the equations themselves (no GPU): rotation in halves depends on distance
only, the state space equals its closed form and can be cut anywhere, the convolution sees nothing before the start, the gate stands in front
of a norm in parts, the streams' update reads the old streams only, router weights sum to the scale, ties, run order, causality; plus mistakes
planted in the oracle, each of which the comparisons of the GPU tests would show."""
import math

import numpy as np
import pytest

from tests import kamelorn_fixtures as fx
from tests import kamelorn_oracle as orc


def test_rotation_in_halves_depends_on_distance_only_and_leaves_the_rest():
    rng = np.random.default_rng(0)
    a, b = rng.standard_normal((1, 10)), rng.standard_normal((1, 10))
    dots = [float((orc.turn_halves(a, [i], 8, 50.0) * orc.turn_halves(b, [i - 7], 8, 50.0)).sum()) for i in (7, 20, 300)]
    assert max(dots) - min(dots) < 1e-12
    z = orc.turn_halves(a, [3], 8, 50.0)
    assert np.array_equal(z[:, 8:], a[:, 8:])
    # the pair (i, i + dims / 2): a vector in dimension 1 turns into dimension 5 and stays out of all others
    e = np.zeros((1, 10)); e[0, 1] = 1.0
    t = orc.turn_halves(e, [2], 8, 50.0)[0]
    ang = 2 * 50.0 ** (-2.0 / 8)
    assert abs(t[1] - math.cos(ang)) < 1e-15 and abs(t[5] - math.sin(ang)) < 1e-15 and np.abs(np.delete(t, [1, 5])).max() == 0


def test_state_space_closed_form_and_cuts():
    rng = np.random.default_rng(1)
    T, n, v, a, D = 11, 4, 3, 0.7, -0.4
    x, B, C, dt = rng.standard_normal((T, v)), rng.standard_normal((T, n)), rng.standard_normal((T, n)), rng.uniform(0.01, 2.0, T)
    y, S = orc.ssm_scan(x, B, C, dt, a, D)
    l = np.cumsum(-a * dt)
    for t in range(T):
        want = sum(math.exp(l[t] - l[j]) * dt[j] * (B[j] @ C[t]) * x[j] for j in range(t + 1)) + D * x[t]
        assert np.abs(y[t] - want).max() < 1e-12
    y1, S1 = orc.ssm_scan(x[:4], B[:4], C[:4], dt[:4], a, D)
    y2, S2 = orc.ssm_scan(x[4:], B[4:], C[4:], dt[4:], a, D, S1)
    assert np.abs(np.concatenate([y1, y2]) - y).max() < 1e-12 and np.abs(S2 - S).max() < 1e-12


def test_convolution_bias_and_start():
    rng = np.random.default_rng(2)
    x, w, b = rng.standard_normal((6, 5)), rng.standard_normal((5, 3)), rng.standard_normal(5)
    y = orc.causal_conv(x, w, b)
    assert np.abs(y[0] - (w[:, 2] * x[0] + b)).max() < 1e-15
    assert np.abs(y[4] - (w[:, 0] * x[2] + w[:, 1] * x[3] + w[:, 2] * x[4] + b)).max() < 1e-15


def test_norm_in_parts_and_softplus():
    y = np.array([[3.0, 4.0, 30.0, 40.0]])
    z = orc.rms_parts(y, np.ones(4), 2, 0.0)
    assert np.allclose(z[0, :2], z[0, 2:])          # each part by its own root mean square
    assert not np.allclose(orc.rms_parts(y, np.ones(4), 1, 0.0)[0, :2], z[0, :2])
    s = orc.softplus(np.array([-800.0, 0.0, 800.0]))
    assert s[0] == 0.0 and abs(s[1] - math.log(2.0)) < 1e-15 and s[2] == 800.0


def test_streams_update_reads_the_old_streams_and_indexes_from_to():
    W = {"p.in": np.array([1.0, 0.0]), "p.out": np.array([0.0, 2.0]), "p.mix": np.array([[0.0, 1.0], [5.0, 0.0]])}
    X = np.stack([np.full((1, 4), 1.0), np.full((1, 4), 7.0)])
    Y = orc.sublayer(X, W, "p.", np.ones(4), 0.0, 0.5, lambda h: h)
    # new stream 0 = 5 x old stream 1; new stream 1 = old stream 0 + 0.5 * 2 * rms(stream 0)
    assert np.allclose(Y[0], 35.0) and np.allclose(Y[1], 2.0)


def test_router_weights_sum_to_the_scale_and_ties_take_the_lower_index():
    rng = np.random.default_rng(3)
    h, r = rng.standard_normal((5, 8)), rng.standard_normal((6, 8))
    r[4] = r[1]
    idx, w = orc.route(h, r, 3, 2.5)
    assert np.allclose(w.sum(-1), 2.5)
    for row in idx:
        assert not (4 in row and 1 not in row)
    i1, w1 = orc.route(h, r, 1, 1.0)
    assert np.allclose(w1, 1.0)


def test_run_order():
    cfg = fx.config([fx.ssm_layer(mlp=None)] * 5, loop=(1, 3, 3))
    assert orc.run_order(cfg) == [0, 1, 2, 1, 2, 1, 2, 3, 4]
    assert orc.run_order(fx.config([fx.ssm_layer(mlp=None)] * 3)) == [0, 1, 2]


SMALL = fx.config([fx.latent_layer(), fx.ssm_layer(), fx.ssm_layer(conv=3, mlp=fx.dense(16)), fx.latent_layer(mlp=None)], width=32, vocab=31, loop=(1, 3, 2))


def test_causality():
    w = fx.oracle_weights(fx.random_weights(SMALL, 1))
    toks = [int(t) for t in np.random.default_rng(4).integers(0, 31, 20)]
    full = orc.forward(SMALL, w, toks)
    assert np.abs(orc.forward(SMALL, w, toks[:13]) - full[:13]).max() < 1e-10
    other = list(toks); other[12] = (toks[12] + 1) % 31
    assert np.abs(orc.forward(SMALL, w, other)[:12] - full[:12]).max() < 1e-10 and np.abs(orc.forward(SMALL, w, other)[12] - full[12]).max() > 1e-3


MISTAKES = {
    "mix_transposed": ("sublayer", lambda f: lambda X, W, p, *r: f(X, {**W, p + "mix": W[p + "mix"].T}, p, *r)),
    "pairs_interleaved": ("turn_halves", lambda f: lambda z, pos, d, b: f(z[..., np.r_[0:d:2, 1:d:2, d:z.shape[-1]]], pos, d, b)),
    "no_skip": ("ssm_scan", lambda f: lambda x, B, C, dt, a, D: f(x, B, C, dt, a, 0.0)),
    "step_size_not_in_the_input": ("ssm_scan", lambda f: lambda x, B, C, dt, a, D: f(x, B / dt[:, None], C, dt, a, D)),
    "one_norm_part": ("rms_parts", lambda f: lambda y, w, parts, eps: f(y, w, 1, eps)),
    "no_conv_bias": ("causal_conv", lambda f: lambda x, w, b: f(x, w, 0 * b)),
    "weights_not_scaled": ("route", lambda f: lambda h, r, top, s: f(h, r, top, 1.0)),
    "one_pass": ("run_order", lambda f: lambda cfg: f({**cfg, "loop": {**cfg["loop"], "times": 1}})),
}


@pytest.mark.parametrize("name", sorted(MISTAKES))
def test_planted_mistakes_show(monkeypatch, name):
    w = fx.oracle_weights(fx.random_weights(SMALL, 5))
    toks = [int(t) for t in np.random.default_rng(6).integers(0, 31, 24)]
    want = orc.forward(SMALL, w, toks)
    fn, wrap = MISTAKES[name]
    monkeypatch.setattr(orc, fn, wrap(getattr(orc, fn)))
    assert fx.rel_err(orc.forward(SMALL, w, toks), want).max() > 1e-2
