"""Host-side checks of the Zusuvik design (no GPU): the registry, the order of looped layers, and the float64 restatement against closed
forms and against itself -- rotation and its rescaled frequencies (also the product's own table), the short convolution, retention, the
matrix memory's stabilised recurrence, routing, the gated shared unit."""
import math

import numpy as np
import pytest

from oracle import zusuvik as oz
from tests.conftest import load_pkg


def test_the_registry_resolves_the_architecture():
    load_pkg()
    from dash_infer_amd import models
    assert "Zusuvik" in models.known()
    cls = models.resolve({"architecture": "Zusuvik"})
    assert cls.engine == "sequence" and cls.__name__ == "Zusuvik"


def test_order_of_looped_layers():
    load_pkg()
    from dash_infer_amd import models
    runs = models.layer_runs(5, {"start": 1, "stop": 3, "times": 3})
    assert [r[0] for r in runs] == [0, 1, 2, 1, 2, 1, 2, 3, 4] and [r[1] for r in runs] == [0, 0, 0, 1, 1, 2, 2, 0, 0]
    cfg = {"layers": [None] * 5, "loop": {"start": 1, "stop": 3, "times": 3}}
    assert [(i, bool(p)) for i, _, p in runs] == oz.layer_order(cfg)       # x0 joins before the later passes' first layer alone
    assert oz.layer_order({"layers": [None] * 2}) == [(0, False), (1, False)]
    with pytest.raises(ValueError):
        models.layer_runs(3, {"start": 2, "stop": 4, "times": 2})


@pytest.mark.parametrize("layout", ["pairs", "halves"])
def test_rotation_is_relative_and_leaves_the_rest(layout):
    rng = np.random.default_rng(0)
    q, k = rng.normal(size=12), rng.normal(size=12)
    for sc in (None, oz.TURNS):
        rot = {"dims": 8, "base": 100.0, "scaling": sc}
        dots = [oz.rotate(q, p + 5, rot, layout) @ oz.rotate(k, p, rot, layout) for p in (0, 3, 40)]
        assert np.allclose(dots, dots[0], rtol=1e-5)
        assert np.array_equal(oz.rotate(q, 9, rot, layout)[8:], q[8:]) and np.allclose(oz.rotate(q, 0, rot, layout), q)
    r = oz.rotate(np.array([1.0, 0.0, 0.0, 1.0]), 1, {"dims": 4, "base": 100.0}, layout)
    if layout == "pairs":          # dimension 0 turns with 1 by 1 radian, 2 with 3 by 0.1
        assert np.allclose(r, [np.cos(1.0), np.sin(1.0), -np.sin(0.1), np.cos(0.1)], atol=1e-6)
    else:                          # 0 turns with 2 by 1 radian, 1 with 3 by 0.1
        assert np.allclose(r, [np.cos(1.0), -np.sin(0.1), np.sin(1.0), np.cos(0.1)], atol=1e-6)


@pytest.mark.parametrize("dims,base", [(8, 5000.0), (64, 10000.0), (2, 20.0), (20, 1e6)])
def test_frequencies_rescaled_by_the_number_of_turns(dims, base):
    load_pkg()
    from dash_infer_amd.mixers import rotary_frequencies
    plain = oz.frequencies(dims, base)
    seen = set()
    for sc in (oz.TURNS, dict(factor=8.0, low=1.0, high=4.0, original=8192), dict(factor=2.0, low=0.5, high=16.0, original=64),
               dict(factor=1.0, low=1.0, high=2.0, original=100)):
        f = oz.frequencies(dims, base, sc)
        for i in range(dims // 2):
            turns = sc["original"] * plain[i] / (2 * math.pi)
            if turns > sc["high"]:
                assert f[i] == plain[i]
                seen.add("kept")
            elif turns < sc["low"]:
                assert np.isclose(f[i], plain[i] / sc["factor"], rtol=1e-12)
                seen.add("slowed")
            else:
                part = (turns - sc["low"]) / (sc["high"] - sc["low"])
                assert np.isclose(f[i], plain[i] * (part + (1 - part) / sc["factor"]), rtol=1e-12)
                seen.add("between")
        got, mag = rotary_frequencies(dims, base, sc)                              # the table the kernels read
        assert np.allclose(got.numpy(), f.astype(np.float32), rtol=1e-6) and mag == 1.0
    assert "kept" in seen


def test_short_convolution_is_causal_and_starts_on_zeros():
    rng = np.random.default_rng(1)
    u, w = rng.normal(size=(6, 3)), rng.normal(size=(3, 4))
    y = oz.causal_conv(u, w)
    assert np.allclose(y[0], u[0] * w[:, 3]) and np.allclose(y[2], u[2] * w[:, 3] + u[1] * w[:, 2] + u[0] * w[:, 1])
    assert np.allclose(y[5], sum(u[5 - d] * w[:, 3 - d] for d in range(4)))
    assert np.allclose(oz.causal_conv(u[:3], w), y[:3])
    assert np.allclose(oz.causal_conv(u, w[:, :1]), u * w[:, 0])


def test_retention_against_its_closed_form():
    rng = np.random.default_rng(2)
    q, k, v = rng.normal(size=(9, 2, 4)), rng.normal(size=(9, 2, 4)), rng.normal(size=(9, 2, 3))
    decay = [0.9, 0.5]
    got = oz.retention_scan(q, k, v, decay)
    for t in range(9):
        for h in range(2):
            assert np.allclose(got[t, h], sum(decay[h] ** (t - s) * (q[t, h] @ k[s, h]) * v[s, h] for s in range(t + 1)))


def test_matrix_memory_against_its_unscaled_recurrence():
    rng = np.random.default_rng(3)
    n, H, D, V = 12, 2, 4, 3
    q, k, v = rng.normal(size=(n, H, D)), rng.normal(size=(n, H, D)), rng.normal(size=(n, H, V))
    li, lf = rng.normal(0, 2.0, (n, H)), oz.log_sigmoid(rng.normal(1.0, 2.0, (n, H)))
    got = oz.matrix_memory_scan(q, k, v, li, lf)
    S, N = np.zeros((H, D, V)), np.zeros((H, D))
    m = np.zeros(H)
    for t in range(n):                     # the true sums; the running maximum only scales numerator and divisor (and the small constant)
        S = np.exp(lf[t])[:, None, None] * S + np.exp(li[t])[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        N = np.exp(lf[t])[:, None] * N + np.exp(li[t])[:, None] * k[t]
        m = np.maximum(lf[t] + m, li[t])
        den = np.maximum(np.abs((N * q[t]).sum(1)), 1.0) + 1e-6 * np.exp(m)
        assert np.allclose(got[t], np.einsum("hdv,hd->hv", S, q[t]) / den[:, None])


def test_matrix_memory_starts_at_zero_not_at_minus_infinity():
    """with small input gates the maximum stays at 0 decayed, and the divisor's floor with it"""
    q = k = v = np.ones((1, 1, 1))
    low = oz.matrix_memory_scan(q, k, v, np.full((1, 1), -5.0), np.full((1, 1), -0.5))
    assert np.allclose(low, np.exp(-5.0) / (1.0 + 1e-6 * np.exp(-0.5)))        # floor 1 of the true sum |n . q| = exp(-5)
    high = oz.matrix_memory_scan(q, k, v, np.full((1, 1), 3.0), np.full((1, 1), -0.5))
    assert np.allclose(high, 1.0 / (1.0 + 1e-6))


def test_routing_and_the_gated_shared_unit():
    rng = np.random.default_rng(4)
    fc, w = oz.ff_parts(rng, 16, dict(experts=5, top=3, ff=4, shared=6))
    h = rng.normal(size=(40, 16))
    chosen = []
    got = oz.moe_ff(h, w, fc, chosen)
    z = h @ w["router"].T.astype(np.float64) + w["router.b"]
    assert all(set(c) == set(np.argsort(-z[t])[:3]) for t, c in enumerate(chosen))
    _, ws = oz.route(z, 3)
    assert np.allclose(ws.sum(1), 1.0)
    alone = oz.moe_ff(h, w, dict(fc, shared=None))
    gate = 1.0 / (1.0 + np.exp(-(h @ w["shared.sg"].T.astype(np.float64))))
    assert np.allclose(got - alone, gate * oz.clamped_unit(h, w, "shared.", 2.0))
    far = oz.clamped_unit(h * 100.0, w, "shared.", 2.0)                          # both clamps bind
    g, u = np.minimum(h @ w["shared.gate"].T * 100.0, 2.0), np.clip(h @ w["shared.up"].T * 100.0, -2.0, 2.0)
    assert np.allclose(far, (g / (1.0 + np.exp(-1.702 * g)) * (u + 1.0)) @ w["shared.down"].T)


def test_a_random_model_runs_and_its_loop_passes_differ():
    rng = np.random.default_rng(5)
    cfg, t = oz.random_zusuvik(rng, [("parallel", None, {}), ("retention", None, {}), ("retention", None, None)], loop=(1, 2, 3))
    streams = []
    lg = oz.forward(cfg, t, [3, 1, 4, 1, 5], streams)
    assert lg.shape == (5, cfg["vocab"]) and len(streams) == 5 and np.isfinite(lg).all()
    assert np.allclose(oz.forward(cfg, t, [3, 1, 4])[:3], lg[:3])               # causal
    plain = oz.forward(dict(cfg, loop=None), t, [3, 1, 4, 1, 5])
    assert np.abs(plain - lg).max() > 1e-2
