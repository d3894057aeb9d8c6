"""The float64 oracle of the Rosilix tests against properties of the equations themselves (no GPU): rotation in pairs depends on distance only, chunks
are counted from position 0, a sink is one more key without a value, two equal maps cancel, a head's output has a fixed size, shared cache rows are the
source layer's, causality; plus mistakes planted in the oracle, each of which the comparisons of the GPU tests would show.  (The factor 1 - diff behind the head's norm cancels in the norm behind
the mixer, but for eps: it shows in the op-level comparisons only.)"""
import math

import numpy as np
import pytest

from tests import rosilix_fixtures as fx
from tests import rosilix_oracle as orc


def test_rotation_in_pairs_depends_on_distance_only_and_leaves_the_rest():
    rng = np.random.default_rng(0)
    a, b = rng.standard_normal((1, 10)), rng.standard_normal((1, 10))
    dots = [float((orc.turn_pairs(a, [i], 8, 50.0) * orc.turn_pairs(b, [i - 7], 8, 50.0)).sum()) for i in (7, 20, 300)]
    assert max(dots) - min(dots) < 1e-12
    assert np.array_equal(orc.turn_pairs(a, [3], 8, 50.0)[:, 8:], a[:, 8:])
    # the pair (2, 3): a vector in dimension 2 turns into dimension 3 and stays out of all others
    e = np.zeros((1, 10)); e[0, 2] = 1.0
    t = orc.turn_pairs(e, [2], 8, 50.0)[0]
    ang = 2 * 50.0 ** (-2.0 / 8)
    assert abs(t[2] - math.cos(ang)) < 1e-15 and abs(t[3] - math.sin(ang)) < 1e-15 and np.abs(np.delete(t, [2, 3])).max() == 0


def test_chunks_are_counted_from_position_0():
    v = orc.visible(10, 4)
    assert v[3].tolist() == [True] * 4 + [False] * 6 and v[4].tolist() == [False] * 4 + [True] + [False] * 5 and v[9, 8] and not v[9, 7]
    assert orc.visible(5, 1).tolist() == np.eye(5, dtype=bool).tolist()
    assert orc.visible(6).tolist() == np.tril(np.ones((6, 6), bool)).tolist()
    assert orc.visible(10, 4, 2)[7].tolist() == [False] * 6 + [True] * 2 + [False] * 2 and orc.visible(10, 4, 3)[8].sum() == 1


def test_sink_is_one_more_key_without_a_value():
    rng = np.random.default_rng(1)
    s = rng.standard_normal((3, 5))
    for z in (-4.0, 0.3, 30.0):
        assert np.allclose(orc.softmax(s, z), orc.softmax(np.concatenate([s, np.full((3, 1), z)], 1))[:, :5], atol=1e-15)
    assert np.allclose(orc.softmax(s).sum(-1), 1.0)


def test_difference_of_maps():
    rng = np.random.default_rng(2)
    a, lq, lk = rng.standard_normal((4, 3, 8)), rng.standard_normal(6), rng.standard_normal(6)
    assert abs(orc.mixing_factor(lq, lk, lq, lk, 0.4) - 0.4) < 1e-15
    assert abs(orc.mixing_factor(lq, lk, 0 * lq, lk, 0.0) - (math.exp(lq @ lk) - 1.0)) < 1e-15
    assert np.abs(orc.difference(a, a, 1.0, 0.2, 1e-6)).max() == 0.0
    o = orc.difference(a, 0.5 * a, 0.7, 0.2, 0.0)
    assert np.allclose((o * o).mean(-1), 0.8 ** 2)          # every head by its own size
    assert np.allclose(o, orc.difference(3.0 * a, 1.5 * a, 0.7, 0.2, 0.0))


def test_feed_forward_is_the_square_of_relu():
    y = orc.feed_forward(np.array([[1.0, -2.0]]), np.eye(2), np.array([[1.0, 0.0], [0.0, 1.0]]) * 3.0)
    assert y.tolist() == [[3.0, 0.0]]
    assert orc.feed_forward(np.array([[2.0]]), np.eye(1), np.eye(1))[0, 0] == 4.0


SMALL = fx.config([fx.latent_layer(), fx.attention_layer(chunk=7), fx.latent_layer(heads=2, dim=8, vdim=16, kv_from=0), fx.attention_layer(heads=3, kv_heads=1, chunk=10, mlp=None)],
                  width=32, vocab=31)


def test_causality_and_chunk_reach():
    w = fx.oracle_weights(fx.random_weights(SMALL, 1))
    toks = [int(t) for t in np.random.default_rng(4).integers(0, 31, 20)]
    full = orc.forward(SMALL, w, toks)
    assert np.abs(orc.forward(SMALL, w, toks[:13]) - full[:13]).max() < 1e-10
    other = list(toks); other[12] = (toks[12] + 1) % 31
    assert np.abs(orc.forward(SMALL, w, other)[:12] - full[:12]).max() < 1e-10 and np.abs(orc.forward(SMALL, w, other)[12] - full[12]).max() > 1e-3
    # attention layers alone: a token never reaches another chunk
    cfg = fx.config([fx.attention_layer(chunk=6), fx.attention_layer(chunk=6)], width=32, vocab=31)
    w = fx.oracle_weights(fx.random_weights(cfg, 2))
    full, alt = orc.forward(cfg, w, toks), orc.forward(cfg, w, other)
    d = np.abs(full - alt).max(-1)
    assert d[:12].max() < 1e-10 and d[12] > 1e-3 and d[13:18].min() > 1e-7 and d[18:].max() < 1e-10


def test_shared_rows_are_the_source_layers():
    """a reader with the source's projections, on the source's input, gives the source's output"""
    rng = np.random.default_rng(5)
    L = fx.latent_layer()
    cfg = fx.config([L, fx.latent_layer(kv_from=0)], width=32, vocab=31)
    w = fx.oracle_weights(fx.random_weights(cfg, 3))
    for n in ("q", "uk", "uv", "sink", "g", "o"):
        w["l1.mix." + n] = w["l0.mix." + n]
    h = rng.standard_normal((9, 32))
    rows = orc.latent_rows(h, w, "l0.mix.", L["mixer"], 1e-5)
    assert np.array_equal(orc.latent_attention(h, rows, w, "l0.mix.", L["mixer"]), orc.latent_attention(h, rows, w, "l1.mix.", L["mixer"]))
    assert "l1.mix.dkv" not in w


MISTAKES = {
    "pairs_in_halves": ("turn_pairs", lambda f: lambda z, pos, d, b: f(z[..., np.r_[np.arange(d).reshape(2, -1).T.reshape(-1), d:z.shape[-1]]], pos, d, b)),
    "no_sink": ("softmax", lambda f: lambda s, sink=None: f(s)),
    "chunk_one_longer": ("visible", lambda f: lambda T, chunk=None, window=None: f(T, chunk + 1 if chunk else chunk)),
    "window_for_chunk": ("visible", lambda f: lambda T, chunk=None, window=None: f(T, None, chunk)),
    "factor_without_diff": ("mixing_factor", lambda f: lambda a, b, c, d, diff: f(a, b, c, d, 0.0)),
    "second_exponential_lost": ("mixing_factor", lambda f: lambda a, b, c, d, diff: f(a, b, 0 * c, d, diff)),
    "difference_not_normed": ("difference", lambda f: lambda a, b, lam, diff, eps: (a - lam * b) * (1 - diff)),
    "relu_not_squared": ("feed_forward", lambda f: lambda h, u, d: np.maximum(h @ u.T, 0) @ d.T),
    "latent_not_normed": ("latent_rows", lambda f: lambda h, W, p, mx, eps: ((h @ W[p + "dkv"].T)[:, :mx["kv_rank"]], f(h, W, p, mx, eps)[1])),
    "norm_one_plus": ("norm", lambda f: lambda y, w, eps: f(y, 1.0 + w, eps)),
}


@pytest.mark.parametrize("name", sorted(MISTAKES))
def test_planted_mistakes_show(monkeypatch, name):
    w = fx.oracle_weights(fx.random_weights(SMALL, 5))
    toks = [int(t) for t in np.random.default_rng(6).integers(0, 31, 24)]
    want = orc.forward(SMALL, w, toks)
    fn, wrap = MISTAKES[name]
    monkeypatch.setattr(orc, fn, wrap(getattr(orc, fn)))
    assert fx.rel_err(orc.forward(SMALL, w, toks), want).max() > 1e-2
