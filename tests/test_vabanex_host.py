"""Host-side checks of the Vabanex design (no GPU): the registry, and the float64 restatement against closed forms and against itself
-- rotation and its rescaled frequencies (also the product's own table), the gated latent attention, routing, the clamped unit."""
import math

import numpy as np
import pytest

from oracle import vabanex as ov
from tests.conftest import load_pkg


def test_the_registry_resolves_the_architecture():
    load_pkg()
    from dash_infer_amd import models
    assert "Vabanex" in models.known()
    cls = models.resolve({"architecture": "Vabanex"})
    assert cls.engine == "sequence" and cls.__name__ == "Vabanex"


def test_rotation_is_relative_and_pairs_neighbours():
    rng = np.random.default_rng(0)
    q, k = rng.normal(size=12), rng.normal(size=12)
    for sc in (None, ov.YARN):
        dots = [ov.rotate_pairs(q, p + 5, 8, 100.0, sc) @ ov.rotate_pairs(k, p, 8, 100.0, sc) for p in (0, 3, 40)]
        assert np.allclose(dots, dots[0], rtol=1e-5)
    assert np.array_equal(ov.rotate_pairs(q, 9, 8, 100.0)[8:], q[8:]) and np.allclose(ov.rotate_pairs(q, 0, 8, 100.0), q)
    r = ov.rotate_pairs(np.array([1.0, 0.0, 0.0, 1.0]), 1, 4, 100.0)            # dimension 0 turns with 1 by 1 radian, 2 with 3 by 0.1
    assert np.allclose(r, [np.cos(1.0), np.sin(1.0), -np.sin(0.1), np.cos(0.1)], atol=1e-6)


SCALINGS = [ov.YARN, dict(factor=40.0, original=4096, fast=32.0, slow=1.0), dict(factor=2.0, original=16, fast=1.0, slow=1.0),
            dict(factor=4.0, original=8, fast=64.0, slow=2.0), dict(factor=1.0, original=100, fast=9.0, slow=2.0)]


@pytest.mark.parametrize("dims,base", [(8, 5000.0), (64, 10000.0), (2, 20.0), (20, 1e6)])
def test_rescaled_frequencies(dims, base):
    load_pkg()
    from dash_infer_amd.mixers import rotary_frequencies
    plain, one = ov.pair_frequencies(dims, base)
    assert one == 1.0 and np.allclose(plain, [base ** (-2.0 * i / dims) for i in range(dims // 2)])
    for sc in SCALINGS:
        f, mag = ov.pair_frequencies(dims, base, sc)
        assert abs(mag - (1.0 + 0.1 * math.log(sc["factor"]))) < 1e-12
        assert ((f <= plain * (1 + 1e-12)) & (f >= plain / sc["factor"] * (1 - 1e-12))).all()     # between slowed down and as it was
        for i in range(dims // 2):
            turns = sc["original"] * plain[i] / (2 * math.pi)
            if turns > sc["fast"] * base ** (2.0 / dims):                       # clearly above (the ramp's ends are whole indices)
                assert np.isclose(f[i], plain[i])
            if turns < sc["slow"] / base ** (4.0 / dims) and i > 0:
                assert np.isclose(f[i], plain[i] / sc["factor"])
        pf, pm = rotary_frequencies(dims, base, sc)                             # the table the kernels read
        assert np.allclose(pf.numpy(), f.astype(np.float32), rtol=1e-6) and abs(pm - mag) < 1e-12


def test_latent_attention_of_one_token_and_its_gate():
    rng = np.random.default_rng(1)
    o = dict(ov.LATENT, heads=2, vdim=3)
    w = ov.latent_weights(rng, 20, o)
    h = rng.normal(size=(4, 20))
    got = ov.latent_attention(h, w, ov.latent_config(o), 1e-5)
    c = ov.unit_rms(h[:1] @ w["dkv"][: o["kv_rank"]].T.astype(np.float64), 1e-5) * w["dkv.norm"]
    v = (c @ w["uv"].T.astype(np.float64)).reshape(2, 3)                        # one key: its value
    gate = 1 / (1 + np.exp(-(h[0] @ w["g"].T.astype(np.float64))))
    assert np.allclose(got[0], (v * gate[:, None]).reshape(-1) @ w["o"].T.astype(np.float64))
    assert np.allclose(ov.latent_attention(h[:2], w, ov.latent_config(o), 1e-5), got[:2])      # causal


def test_routing_by_brute_force():
    rng = np.random.default_rng(2)
    fc = ov.ff_config(("moe", dict(experts=8, count=4, keep=2, top=3, ff=4, scale=1.7)))
    w = ov.ff_weights(rng, 16, fc)
    h = rng.normal(size=(200, 16))
    idx, ws = ov.route(h, w, fc)
    s = ov.sigmoid(h @ w["router"].T.astype(np.float64))
    choice = s + w["correction"]
    assert (choice < 0).any() and (choice > 0).any()
    for t in range(200):
        pair = choice[t].reshape(4, 2).sum(1)                                   # two experts a group: both count
        best = sorted(range(4), key=lambda g: -pair[g])[:2]
        allowed = sorted((e for e in range(8) if e // 2 in best), key=lambda e: -choice[t, e])[:3]
        assert list(idx[t]) == allowed
    assert np.allclose(ws, np.take_along_axis(s, idx, 1) * 1.7)                 # not renormalised, the correction left out
    assert ov.moe_ff(h[:5], w, fc).shape == (5, 16)


def test_clamped_unit():
    w = {"gate": np.array([[1.0], [1.0], [1.0]]), "up": np.array([[1.0], [-5.0], [0.0]]), "down": np.eye(3)}
    y = ov.dense_ff(np.array([[2.0]]), w, {"limit": 1.5})
    g = 1.5 / (1 + np.exp(-1.702 * 1.5))
    assert np.allclose(y, [[g * 2.5, g * -0.5, g]])
    low = ov.dense_ff(np.array([[-9.0]]), w, {"limit": 1.5})                    # the gate has no lower limit
    assert np.allclose(low[0, 2], -9.0 / (1 + np.exp(1.702 * 9.0)))


def test_a_random_model_runs_and_its_logits_are_capped():
    rng = np.random.default_rng(4)
    cfg, t = ov.random_vabanex(rng, [(None, ("dense",)), ({"scaling": None}, ("moe",)), ({"heads": 1}, None)], softcap=2.0)
    assert "l2.norm2" not in t and "l1.norm2.b" in t and "scaling" not in cfg["layers"][1]["mixer"]["rot"]
    streams = []
    lg = ov.forward(cfg, t, [3, 1, 4, 1, 5], streams)
    assert lg.shape == (5, cfg["vocab"]) and len(streams) == 3 and np.isfinite(lg).all()
    assert np.abs(lg).max() < 2.0
    assert np.allclose(ov.forward(cfg, t, [3, 1, 4])[:3], lg[:3])               # causal
    free = dict(cfg)
    del free["logit_softcap"]
    assert np.abs(ov.forward(free, t, [3, 1, 4])).max() > 2.0
