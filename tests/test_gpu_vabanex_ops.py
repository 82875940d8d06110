"""The mechanisms of the Vabanex design, each alone, against the float64 restatement in oracle/vabanex.py: the biased layer norm fused
with the residual step, scaled embedding rows, products with one multiplier per group and with capped outputs, rotation of
neighbouring dimensions with rescaled frequencies, attention through a latent with a gate per head, the clamped gated unit, sigmoid
routing limited to groups that count by two choice scores, experts without a gate."""
import numpy as np
import pytest
import torch

from oracle import vabanex as ov
from tests.conftest import load_pkg
from tests.seq_helpers import MixerRig, dev_weights, rel_err

pytestmark = pytest.mark.gpu
bf = ov.bf16_values
EPS = 1e-5


@pytest.fixture(scope="module")
def so():
    load_pkg()
    from dash_infer_amd import seq_ops
    return seq_ops


def mixers():
    load_pkg()
    from dash_infer_amd import mixers as m
    return m


def dev(a, dt=torch.float32):
    return torch.from_numpy(np.ascontiguousarray(a, dtype=np.float32)).to(dt).cuda()


def i32(a):
    return torch.tensor(a, dtype=torch.int32, device="cuda")


def rows(rng, n, width, scale=1.0):
    """hidden rows whose values are 16-bit ones, so that both engines read the same numbers"""
    return bf(rng.normal(0, scale, (n, width)))


# ---------------------------------------------------------------------------------------------------------------- row operators
@pytest.mark.parametrize("K", [50, 1024 + 41, 3000, 4096 + 8, 9001, 16384 + 40])
def test_biased_layer_norm_fused_with_the_residual_step(so, K):
    rng = np.random.default_rng(0)
    T = 11
    x, a = (rng.normal(0, 1.5, (T, K)) + 0.7).astype(np.float32), rng.normal(0, 0.5, (T, K)).astype(np.float32)
    w, b = bf(1.0 + 0.3 * rng.normal(size=K)), bf(rng.normal(size=K))
    xo = x.astype(np.float64) + a
    xd = dev(x)
    h = so.residual_layernorm(xd, dev(w, torch.bfloat16), a=dev(a), eps=1e-4, x_out=xd, bias=dev(b, torch.bfloat16))
    assert rel_err(xd.cpu().numpy(), xo) < 1e-6 and rel_err(h.cpu().numpy(), ov.layer_norm(xo, w, b, 1e-4)) < 3e-6
    pick = [5, 0, 10, 5]
    hr = so.residual_layernorm(dev(x), dev(w), eps=1e-4, row_idx=i32(pick), bias=dev(b))
    assert rel_err(hr.cpu().numpy(), ov.layer_norm(x, w, b, 1e-4)[pick]) < 3e-6
    assert rel_err(hr.cpu().numpy(), ov.layer_norm(x, w, 0.0 * b, 1e-4)[pick]) > 1e-2      # the bias shows


@pytest.mark.parametrize("K", [72, 3000, 17000])
@pytest.mark.parametrize("top", [1, 3])
def test_routed_rows_summed_inside_the_residual_step(so, K, top):
    """the bits of the separate sum, beside another sublayer's rows or alone"""
    rng = np.random.default_rng(2)
    T = 9
    x, a, rows = (rng.normal(0, 1.0, (n, K)).astype(np.float32) for n in (T, T, T * top))
    wts, dst = rng.uniform(0, 2, (T, top)).astype(np.float32), rng.permutation(T * top)
    w, b = dev(bf(1.0 + 0.3 * rng.normal(size=K))), dev(bf(rng.normal(size=K)))
    y = so.moe_combine(dev(rows), i32(dst), dev(wts), T, top)
    assert rel_err(y.cpu().numpy(), (wts[:, :, None] * rows[dst].reshape(T, top, K).astype(np.float64)).sum(1)) < 1e-6
    for other in (None, dev(a)):
        x1, x2 = dev(x), dev(x)
        h1 = so.residual_layernorm(x1, w, a=other if other is not None else y, b=y if other is not None else None, mult=0.5, eps=1e-5, x_out=x1, bias=b)
        h2 = so.residual_layernorm(x2, w, a=other, routed=(dev(rows), i32(dst), dev(wts)), mult=0.5, eps=1e-5, x_out=x2, bias=b)
        assert torch.equal(x1, x2) and torch.equal(h1, h2)


def test_scaled_embedding_rows(so):
    rng = np.random.default_rng(1)
    table = bf(rng.normal(size=(37, 50)))
    ids = [3, 36, 0, 3]
    got = so.embed_rows(i32(ids), dev(table, torch.bfloat16), scale=0.3)
    assert rel_err(got.cpu().numpy(), table[ids].astype(np.float64) * 0.3) < 1e-6


@pytest.mark.parametrize("T", [1, 3, 40])
@pytest.mark.parametrize("K,N", [(64, 48), (30, 21)])
def test_products_with_a_multiplier_per_group_and_capped_outputs(so, T, K, N):
    """every kernel of the linear layer: f32 tiles, streamed weights for few rows, matrix cores; odd sizes without vector loads"""
    rng = np.random.default_rng(2)
    G = 3
    x, w = rows(rng, T, G * K), bf(rng.normal(0, 0.3, (G, N, K)))
    gate = rng.uniform(0, 1, (T, G)).astype(np.float32)
    want = np.concatenate([(x[:, g * K:(g + 1) * K].astype(np.float64) @ w[g].astype(np.float64).T) * gate[:, g:g + 1] for g in range(G)], 1)
    wide = dev(np.concatenate([np.ones((T, 5), np.float32), gate], 1))                     # the gates are a column slice of a wider row
    for math in (so.MATH_F32, so.MATH_BF16):
        got = so.linear(dev(x), dev(w, torch.bfloat16), groups=G, mul=wide[:, 5:], mul_group=True, math=math)
        assert rel_err(got.cpu().numpy(), want) < 2e-6
    w1 = bf(rng.normal(0, 0.8, (N, K)))
    z = x[:, :K].astype(np.float64) @ w1.astype(np.float64).T
    for cap in (4.0, 1.0):
        for math in (so.MATH_F32, so.MATH_BF16):
            got = so.linear(dev(x)[:, :K], dev(w1, torch.bfloat16), act="softcap", act_param=cap, math=math)
            assert rel_err(got.cpu().numpy(), ov.soft_cap(z, cap)) < 5e-6
    assert np.abs(z).max() > 4.0                                                           # values beyond the cap were there
    with pytest.raises(Exception):
        so.linear(dev(x)[:, :K], dev(w1, torch.bfloat16), act="softcap", act_param=0.0)


# ---------------------------------------------------------------------------------------------------------------- rotation
@pytest.mark.parametrize("rot,base,scaling", [(8, 5000.0, ov.YARN), (2, 100.0, None), (64, 10000.0, dict(factor=40.0, original=4096, fast=32.0, slow=1.0)),
                                              (6, 50.0, dict(factor=2.0, original=16, fast=1.0, slow=1.0)), (16, 30.0, dict(factor=1.0, original=100, fast=9.0, slow=2.0))])
def test_rotation_of_neighbouring_dimensions_with_rescaled_frequencies(so, rot, base, scaling):
    load_pkg()
    from dash_infer_amd.mixers import rotary_frequencies
    from dash_infer_amd.seq_state import SequenceStateManager
    rng = np.random.default_rng(3)
    R, H, n = 20, 3, 150
    Rp = R + rot + 3                                                                       # padding behind the rotated part
    f, mag = rotary_frequencies(rot, base, scaling)
    st = SequenceStateManager(256, 1, 64, "cuda")
    tab = st.add_span_cache("c", Rp, torch.float32)
    st.admit("a")
    s = st.reserve("a", n)
    st.upload()
    ckv, qr = rng.normal(size=(n, R + rot)).astype(np.float32), rng.normal(size=(n, H * rot)).astype(np.float32)
    gam = bf(1 + 0.2 * rng.normal(size=R))
    ql = torch.full((n, H * Rp), 7.0, device="cuda")
    so.latent_rope_append(tab, dev(ckv), dev(gam, torch.bfloat16), EPS, R, rot, f.cuda(), dev(qr), ql, H, i32([s.index] * n), i32(list(range(n))),
                          layout=so.ROTARY_LAYOUTS["pairs"], mag=mag)
    page = tab.rows(s.index, s.pages, n).cpu().numpy()
    assert rel_err(page[:, :R], ov.unit_rms(ckv[:, :R], EPS) * gam) < 3e-6
    want_k = np.stack([ov.rotate_pairs(ckv[p, R:], p, rot, base, scaling) for p in range(n)])
    want_q = np.stack([ov.rotate_pairs(qr[p].reshape(H, rot), p, rot, base, scaling) for p in range(n)])
    q = ql.cpu().numpy().reshape(n, H, Rp)
    assert rel_err(page[:, R:R + rot], want_k) < 3e-6 and (page[:, R + rot:] == 0).all()
    assert rel_err(q[:, :, R:R + rot], want_q) < 3e-6
    assert (q[:, :, :R] == 7.0).all() and (q[:, :, R + rot:] == 7.0).all()                 # nothing else of the queries is touched


# ---------------------------------------------------------------------------------------------------------------- latent attention
def latent_rig(w, o, dtype, max_tokens=2048):
    m = mixers()
    mc = ov.latent_config(o)
    return MixerRig(lambda st, dt: m.LatentWindowAttention("mine", o["heads"], o["dim"], o["vdim"], o["kv_rank"], o["q_rank"], 0, mc["scale"], dev_weights(w),
                                                           st, dt, rot_dim=o["rot_dim"], rot_base=o["base"], rot_layout="pairs", rot_scaling=o["scaling"],
                                                           head_gate=True), dtype, max_tokens=max_tokens)


LATENT_SHAPES = {
    "plain": {},
    "one_head_odd": dict(heads=1, dim=12, rot_dim=2, vdim=9, kv_rank=11, q_rank=5, scaling=None),
    "one_row_of_64": dict(heads=4, dim=32, rot_dim=16, vdim=32, kv_rank=48, q_rank=40, base=100.0),
    "padded_row": dict(heads=5, dim=8, rot_dim=24, vdim=16, kv_rank=80, q_rank=16, scale=0.7),
    "value_not_in_16s": dict(heads=2, dim=10, rot_dim=4, vdim=7, kv_rank=90, q_rank=33),
    "many_heads": dict(heads=24, dim=8, rot_dim=8, vdim=8, kv_rank=120, q_rank=16),
    "row_of_256": dict(heads=2, dim=16, rot_dim=32, vdim=24, kv_rank=200, q_rank=24),
    "row_of_512": dict(heads=3, dim=16, rot_dim=64, vdim=16, kv_rank=448, q_rank=24),
    "row_of_576": dict(heads=3, dim=16, rot_dim=64, vdim=16, kv_rank=512, q_rank=24),       # wider than its value of 512
    "row_of_640": dict(heads=2, dim=8, rot_dim=128, vdim=16, kv_rank=500, q_rank=24),
    "beyond_the_matrix_core_rows": dict(heads=2, dim=8, rot_dim=16, vdim=16, kv_rank=530, q_rank=24),
}


@pytest.mark.parametrize("shape", list(LATENT_SHAPES))
def test_latent_attention_whole_portions_and_decoding(shape):
    rng = np.random.default_rng(4)
    o = dict(ov.LATENT, **LATENT_SHAPES[shape])
    w = ov.latent_weights(rng, 72, o)
    n = 150
    h = rows(rng, n, 72)
    want = ov.latent_attention(h, w, ov.latent_config(o), EPS)
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 0.05)):
        rig = latent_rig(w, o, dtype)
        assert rel_err(rig.step([("a", h)])[0], want) < tol
        cuts = [0, 3, 5, 64, 65, 70, 128, 130, n]                              # portions that end inside a page, at its border, one row after
        got = np.concatenate([rig.step([("b", h[a:b])])[0] for a, b in zip(cuts, cuts[1:])])
        assert rel_err(got, want) < tol
        dec = np.concatenate([rig.step([("c", h[i:i + 1])])[0] for i in range(80)])
        assert rel_err(dec, want[:80]) < tol


def test_the_gate_is_one_number_per_head_and_reads_the_mixers_input():
    rng = np.random.default_rng(5)
    o = dict(ov.LATENT, heads=4, vdim=6)
    w = ov.latent_weights(rng, 72, o)
    w["g"][:] = 0.0
    h = rows(rng, 30, 72)
    half = ov.latent_attention(h, w, ov.latent_config(o), EPS)                   # a gate of one half everywhere
    w2 = dict(w, g=w["g"].copy())
    w2["g"][2] = bf(rng.normal(0, 0.5, 72))
    want = ov.latent_attention(h, w2, ov.latent_config(o), EPS)
    assert rel_err(half, want) > 0.05
    only = dict(w2, o=w["o"].copy())
    only["o"][:, 2 * 6: 3 * 6] = 0.0                                            # without head 2's columns the gate of head 2 does not matter
    assert rel_err(latent_rig(only, o, torch.float32).step([("a", h)])[0], latent_rig(dict(only, g=w["g"]), o, torch.float32).step([("a", h)])[0]) < 1e-6
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 0.05)):
        assert rel_err(latent_rig(w2, o, dtype).step([("a", h)])[0], want) < tol


def test_latent_attention_reads_one_far_key_across_pages():
    """sharp scores: the last rows put most of their weight on single keys, hundreds of positions and several pages back; the rotated
    part, its rescaled frequencies and its magnitude decide too (shown by oracles without them)"""
    rng = np.random.default_rng(6)
    o = dict(ov.LATENT, scale=3.0, rot_dim=16, base=50.0, scaling=dict(factor=8.0, original=128, fast=8.0, slow=1.0))
    w = ov.latent_weights(rng, 72, o)
    n = 400
    h = rows(rng, n, 72)
    m = ov.latent_config(o)
    want = ov.latent_attention(h, w, m, EPS)
    moved = h.copy()
    moved[:100] = rows(rng, 100, 72)                                            # other far keys: the last rows change
    assert rel_err(ov.latent_attention(moved, w, m, EPS)[-40:], want[-40:]) > 0.05
    unscaled = dict(m, rot={"base": 50.0, "dims": 16})
    assert rel_err(ov.latent_attention(h, w, unscaled, EPS)[-40:], want[-40:]) > 0.05
    w0 = dict(w, uq=w["uq"].copy())
    w0["uq"].reshape(o["heads"], o["dim"] + o["rot_dim"], -1)[:, o["dim"]:] = 0.0  # no rotated query part
    assert rel_err(ov.latent_attention(h, w0, m, EPS)[-40:], want[-40:]) > 0.05
    for dtype, tol in ((torch.float32, 5e-5), (torch.bfloat16, 0.08)):
        rig = latent_rig(w, o, dtype)
        got = np.concatenate([rig.step([("a", h[:360])])[0]] + [rig.step([("a", h[i:i + 1])])[0] for i in range(360, n)])
        assert rel_err(got[:360], want[:360]) < tol and rel_err(got[360:], want[360:]) < tol


@pytest.mark.parametrize("at", [0, 1, 63, 64, 127, 128, 191])
def test_one_key_that_stands_out_at_every_page_border(at):
    """one row's latent points along the last query: with sharp scores the last row's result is that row's value, wherever it lies"""
    rng = np.random.default_rng(7)
    o = dict(ov.LATENT, heads=1, scale=4.0)
    w = ov.latent_weights(rng, 72, o)
    w["uq"][o["dim"]:] *= 2.0 ** -4                                             # the rotated part stays in the background
    m = ov.latent_config(o)
    n = 260
    h = rows(rng, n, 72)
    cq = ov.unit_rms(h[-1].astype(np.float64) @ w["dq"].T, EPS) * w["dq.norm"]
    q = (cq @ w["uq"].T)[: o["dim"]] @ w["uk"].astype(np.float64)                # the last query against the latents
    h[at] = bf(30.0 * np.linalg.pinv(w["dkv"][: o["kv_rank"]].astype(np.float64)) @ (q / w["dkv.norm"]) / np.linalg.norm(q))
    want = ov.latent_attention(h, w, m, EPS)[-1:]
    c, _ = ov.latent_keys(h, w, m, EPS)
    alone = (ov.sigmoid(h[-1:].astype(np.float64) @ w["g"].T) * (c[at:at + 1] @ w["uv"].T.astype(np.float64))) @ w["o"].T
    assert rel_err(alone, want) < 0.2                                           # nearly all weight on that key
    for dtype, tol in ((torch.float32, 5e-5), (torch.bfloat16, 0.08)):
        rig = latent_rig(w, o, dtype)
        whole = rig.step([("w", h)])[0][-1:]
        rig.step([("d", h[:-1])])
        dec = rig.step([("d", h[-1:])])[0]
        assert rel_err(whole, want) < tol and rel_err(dec, want) < tol


def test_unequal_portions_in_one_batch_and_pages_used_again():
    rng = np.random.default_rng(8)
    o = dict(ov.LATENT)
    w = ov.latent_weights(rng, 72, o)
    m = ov.latent_config(o)
    hs = [rows(rng, n, 72) for n in (130, 1, 77)]
    want = [ov.latent_attention(x, w, m, EPS) for x in hs]
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 0.05)):
        rig = latent_rig(w, o, dtype, max_tokens=384)                            # 6 pages
        for rnd in range(3):                                                     # pages and slots come back dirty
            first = rig.step([("a", hs[0][:60]), ("b", hs[1]), ("c", hs[2][:2])])
            second = rig.step([("a", hs[0][60:]), ("c", hs[2][2:])])
            assert rel_err(np.concatenate([first[0], second[0]]), want[0]) < tol
            assert rel_err(first[1], want[1]) < tol and rel_err(np.concatenate([first[2], second[1]]), want[2]) < tol
            for name in "abc":
                rig.release(name)


# ---------------------------------------------------------------------------------------------------------------- feed-forward
@pytest.mark.parametrize("limit", [0.4, 1.0, 7.0])
def test_clamped_gated_feed_forward(limit):
    rng = np.random.default_rng(9)
    fc = ov.ff_config(("dense", dict(ff=50, limit=limit)))
    w = ov.ff_weights(rng, 72, fc)
    h = rows(rng, 40, 72)
    want = ov.dense_ff(h, w, fc)
    free = ov.dense_ff(h, w, dict(fc, limit=1e9))
    assert (rel_err(want, free) > 0.05) == (limit < 5.0)                        # the clamp binds, except the widest
    m, d = mixers(), dev_weights(w)
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 0.03)):
        rig = MixerRig(lambda st, dt: m.GatedMlp(d["gate"], d["up"], d["down"], ("clamped", limit)), dtype)
        assert rel_err(rig.step([("a", h)])[0], want) < tol and rel_err(rig.step([("b", h[3:4])])[0], want[3:4]) < tol


ROUTES = [(6, 3, 2, 2), (8, 4, 1, 2), (4, 1, 1, 4), (9, 3, 1, 3), (8, 4, 2, 3), (5, 5, 2, 1), (5, 5, 3, 2), (70, 7, 3, 6), (256, 8, 4, 8), (320, 64, 5, 9), (1024, 16, 3, 32)]


@pytest.mark.parametrize("experts,count,keep,top", ROUTES)
def test_sigmoid_routing_limited_to_the_best_groups(so, experts, count, keep, top):
    """many rows and few rows (the one-launch form); groups of one expert, one group, as many choices as the kept groups hold"""
    rng = np.random.default_rng(10)
    n = 300
    z = rng.normal(0, 1.5, (n, experts)).astype(np.float32)
    corr = bf(rng.normal(-0.7, 0.4, experts))                                   # choice scores of both signs
    s = ov.sigmoid(z)
    idx, ws = ov.route_scores(s, corr, top, count, keep, 2.5)
    kw = dict(scoring=so.ROUTE_SIGMOID, correction=dev(corr, torch.bfloat16), groups=(count, keep), group_top2=True, renorm=False, factor=2.5)
    ids, wts, seg, src_row, dst = so.moe_route(dev(z), top, **kw)
    same = (ids.cpu().numpy() == idx).all(1)
    assert same.mean() > 0.99                                                   # (float64 against f32: a tie of the last bit may fall the other way)
    assert rel_err(wts.cpu().numpy()[same], ws[same]) < 1e-6
    few, fw, fseg, fsrc, fdst = so.moe_route(dev(z[:20]), top, **kw)
    assert torch.equal(few, ids[:20]) and torch.equal(fw, wts[:20])
    for i, sg, src, d, m in ((ids, seg, src_row, dst, n), (few, fseg, fsrc, fdst, 20)):   # the pairs grouped by expert, every pair once
        i, sg, src, d = i.cpu().numpy().reshape(-1), sg.cpu().numpy(), src.cpu().numpy(), d.cpu().numpy()
        order = np.argsort(i, kind="stable")
        assert np.array_equal(src[: m * top], order // top) and np.array_equal(d[order], np.arange(m * top))
        assert np.array_equal(sg[: experts + 1], np.concatenate([[0], np.cumsum(np.bincount(i, minlength=experts))]))
    if count > keep and experts > count:                                        # (kept groups of one expert hold the best experts anyway)
        plain = np.argsort(-(s + corr), axis=1, kind="stable")[:, :top]
        assert any(set(a) != set(b) for a, b in zip(plain.tolist(), idx.tolist()))
    if experts // count > 1 and 1 < count and keep < count:                     # a group by its best expert alone would choose otherwise
        best = np.argsort(-(s + corr).reshape(n, count, -1).max(2), axis=1, kind="stable")[:, :keep]
        assert any(set(i // (experts // count)) - set(b) for i, b in zip(idx, best))


def test_closed_groups_count_as_minus_infinity_and_ties_go_to_the_lower_index(so):
    z = torch.zeros(3, 6, device="cuda")                                        # all scores one half
    corr = dev([-3.0, -3.0, -2.0, -2.0, -3.0, -3.0])                            # every choice score is negative
    ids, wts, *_ = so.moe_route(z, 2, so.ROUTE_SIGMOID, corr, (3, 1), group_top2=True, renorm=False, factor=3.0)
    assert ids.tolist() == [[2, 3]] * 3 and torch.equal(wts, torch.full((3, 2), 1.5, device="cuda"))
    ids, wts, *_ = so.moe_route(z, 3, so.ROUTE_SIGMOID, None, (3, 2), group_top2=True, renorm=True, factor=3.0)
    assert ids.tolist() == [[0, 1, 2]] * 3 and rel_err(wts.cpu().numpy(), np.ones((3, 3))) < 1e-6


@pytest.mark.parametrize("spec", [{}, dict(experts=5, count=0, top=1, ff=7, scale=1.0), dict(experts=8, count=4, keep=2, top=4, ff=32, scale=0.5)])
def test_routed_experts_without_a_gate(spec):
    rng = np.random.default_rng(11)
    n = 200
    fc = ov.ff_config(("moe", spec))
    w = ov.ff_weights(rng, 72, fc)
    h = rows(rng, n, 72)
    want = ov.moe_ff(h, w, fc)
    r = fc["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    m, d = mixers(), dev_weights(w)
    E = r["experts"]
    for dtype, tol, share in ((torch.float32, 2e-5, 1.0), (torch.bfloat16, 0.05, 0.9)):
        rig = MixerRig(lambda st, dt: m.ExpertMlp(d["router"], None, None, [d[f"e{e}.up"] for e in range(E)], [d[f"e{e}.down"] for e in range(E)], r["top"],
                                                  unit="gelu_erf", scoring="sigmoid", correction=d["correction"], groups=(g["count"], g["keep"]),
                                                  group_score="top2", renorm=False, factor=r["scale"]), dtype)
        got = rig.step([("a", h)])[0]
        err = np.abs(got - want).max(1) / np.abs(want).max()
        assert np.mean(err < tol) >= share
        alone = rig.step([("b", h[7:8])])[0]                                    # a token alone (the one-launch routing) against the batch
        assert rel_err(alone, got[7:8]) < (1e-6 if dtype == torch.float32 else 0.05)
