"""The mechanisms of the Zusuvik design, each alone, against the float64 restatement in oracle/zusuvik.py: the residual step with two
input norms, retention, the matrix memory, attention with short convolutions and row norms, the weighted pair, the routed experts with a
gated shared one."""
import numpy as np
import pytest
import torch

from oracle import zusuvik as oz
from tests.conftest import load_pkg
from tests.seq_helpers import MixerRig, dev_weights, rel_err

pytestmark = pytest.mark.gpu
bf = oz.bf16_values
EPS = 1e-5
WIDTH = 72


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


def rows(rng, n, width=WIDTH, scale=1.0):
    """hidden rows whose values are 16-bit ones, so that both engines read the same numbers"""
    return bf(rng.normal(0, scale, (n, width)))


# ---------------------------------------------------------------------------------------------------------------- residual step
@pytest.mark.parametrize("K", [50, 72, 1024 + 41, 3000, 4096 + 8, 9001, 16384 + 40])      # every form of the row kernel
def test_residual_step_with_two_input_norms(so, K):
    rng = np.random.default_rng(0)
    T, top, R = 11, 3, 40
    r = lambda *s: rng.normal(0, 0.7, s).astype(np.float32)
    x, a, b, again, bias, routed = r(T, K), r(T, K), r(T, K), r(T, K), r(K), r(R, K)
    w1, w2 = bf(0.3 * rng.normal(size=K)), bf(0.3 * rng.normal(size=K))
    dst, wts = rng.integers(0, R, (T, top)), rng.random((T, top)).astype(np.float32)
    total = x.astype(np.float64) + a + b + bias + (wts[:, :, None].astype(np.float64) * routed[dst]).sum(1) + again
    wide = dev(np.concatenate([b, b], 1))                                       # a sublayer's output as a column slice
    xd = dev(x)
    kw = dict(a=dev(a), b=wide[:, K:], bias=dev(bias), again=dev(again), routed=(dev(routed), i32(dst.reshape(-1).tolist()), dev(wts)), eps=1e-4)
    h1, h2 = so.residual_rmsnorm(xd, dev(w1, torch.bfloat16), dev(w2, torch.bfloat16), x_out=xd, **kw)
    assert rel_err(xd.cpu().numpy(), total) < 1e-6
    assert rel_err(h1.cpu().numpy(), oz.offset_norm(total, w1, 1e-4)) < 3e-6 and rel_err(h2.cpu().numpy(), oz.offset_norm(total, w2, 1e-4)) < 3e-6
    x2, out = dev(x), torch.empty(T, K, device="cuda")                          # not in place, f32 weights, 16-bit norms, the second norm alone
    n1, g2 = so.residual_rmsnorm(x2, None, dev(w2), x_out=out, out_dtype=torch.bfloat16, **kw)
    assert n1 is None and torch.equal(out, xd) and torch.equal(x2, dev(x)) and torch.equal(g2, h2.to(torch.bfloat16))
    x3 = dev(x)
    assert so.residual_rmsnorm(x3, a=dev(a), x_out=x3) == (None, None)          # a step without a norm
    assert rel_err(x3.cpu().numpy(), x.astype(np.float64) + a) < 1e-6
    pick = [5, 0, 10, 5]
    hr, _ = so.residual_rmsnorm(dev(x), dev(w1), scale=0.3, eps=1e-4, row_idx=i32(pick))
    assert rel_err(hr.cpu().numpy(), 0.3 * oz.offset_norm(x, w1, 1e-4)[pick]) < 3e-6


@pytest.mark.parametrize("H,V", [(3, 20), (1, 200), (9, 64)])
def test_per_head_norm_with_its_options(so, H, V):
    rng = np.random.default_rng(1)
    T = 6
    x, mul, div = rng.normal(0, 2.0, (T, H * V)).astype(np.float32), rng.random((T, H * V)).astype(np.float32), rng.random((T, H)).astype(np.float32)
    per_head, shared = bf(1 + 0.2 * rng.normal(size=H * V)), bf(1 + 0.2 * rng.normal(size=V))
    unit = lambda d: oz.unit_rms(x.reshape(T, H, V).astype(np.float64) * d[:, :, None], EPS).reshape(T, H * V)
    got = so.head_rmsnorm_mul(dev(x), dev(per_head, torch.bfloat16), EPS, H, V, mul=dev(mul), div=dev(div), out_scale=0.4)
    assert rel_err(got.cpu().numpy(), unit(div) * per_head * mul * 0.4) < 3e-6
    one = np.ones((T, H))
    assert rel_err(so.head_rmsnorm_mul(dev(x), None, EPS, H, V, mul=dev(mul)).cpu().numpy(), unit(one) * mul) < 3e-6
    assert rel_err(so.head_rmsnorm_mul(dev(x), dev(shared), EPS, H, V).cpu().numpy(), unit(one) * np.tile(shared, H)) < 3e-6


# ---------------------------------------------------------------------------------------------------------------- the two recurrences
def retention_rig(w, m, dtype, slots=4):
    mx, rot = mixers(), m["rot"]
    return MixerRig(lambda st, dt: mx.Retention("r", m["heads"], m["dim"], m["vdim"], m["decay"], dev_weights(w), st, rot_dims=rot["dims"],
                                                rot_base=rot["base"]), dtype, slots=slots)


def memory_rig(w, m, dtype, slots=4):
    mx = mixers()
    return MixerRig(lambda st, dt: mx.MatrixMemory("m", m["heads"], m["dim"], m["vdim"], m["gate_cap"], dev_weights(w), st), dtype, slots=slots)


RETENTION_SHAPES = {
    "plain": {},
    "odd": dict(heads=1, dim=6, vdim=9, rot_dims=2, decay=[0.97]),
    "no_rotation": dict(heads=2, dim=7, vdim=5, rot_dims=0, decay=[0.3, 1.0]),
    "tiles": dict(heads=4, dim=64, vdim=128, rot_dims=64),
    "many_channels": dict(heads=2, dim=160, vdim=70, rot_dims=100),
    "most_channels": dict(heads=1, dim=400, vdim=200, rot_dims=400, decay=[0.99]),
}
MEMORY_SHAPES = {
    "plain": {},
    "odd": dict(heads=1, dim=5, vdim=9, gate_cap=4.0),
    "tiles": dict(heads=4, dim=64, vdim=64, gate_cap=15.0),
    "wide_values": dict(heads=2, dim=36, vdim=200),
    "many_channels": dict(heads=2, dim=130, vdim=132),
    "most_channels": dict(heads=1, dim=300, vdim=66),
}
CUTS = [0, 2, 3, 64, 65, 66, 200, 202, 329, 330]


def portions(rig, name, h, cuts):
    return np.concatenate([rig.step([(name, h[a:b])])[0] for a, b in zip(cuts, cuts[1:])])


@pytest.mark.parametrize("shape", list(RETENTION_SHAPES))
def test_retention_whole_rows_and_portions(shape):
    rng = np.random.default_rng(2)
    m, w = oz.retention_parts(rng, WIDTH, RETENTION_SHAPES[shape])
    h = rows(rng, 330)
    want = oz.retention(h, w, m, EPS)
    for dtype, tol in ((torch.float32, 3e-5), (torch.bfloat16, 0.05)):
        rig = retention_rig(w, m, dtype)
        assert rel_err(rig.step([("a", h)])[0], want) < tol                     # chunks side by side
        assert rel_err(portions(rig, "b", h, range(331)), want) < tol           # row by row
        assert rel_err(portions(rig, "c", h, CUTS), want) < tol


@pytest.mark.parametrize("shape", list(MEMORY_SHAPES))
def test_matrix_memory_whole_rows_and_portions(shape):
    rng = np.random.default_rng(3)
    m, w = oz.memory_parts(rng, WIDTH, MEMORY_SHAPES[shape])
    h = rows(rng, 330)
    want = oz.matrix_memory(h, w, m, EPS)
    for dtype, tol in ((torch.float32, 3e-5), (torch.bfloat16, 0.05)):
        rig = memory_rig(w, m, dtype)
        assert rel_err(rig.step([("a", h)])[0], want) < tol
        assert rel_err(portions(rig, "b", h, range(331)), want) < tol
        assert rel_err(portions(rig, "c", h, CUTS), want) < tol


@pytest.mark.parametrize("ib,fb", [(-8.0, 6.0), (9.0, -9.0), (0.0, 12.0), (-9.0, -9.0), (0.0, 0.0)])
def test_matrix_memory_gates_at_their_ends(so, ib, fb):
    """gates that hold the state for good, forget it at once, write almost nothing (the divisor is its floor exp(-m), m still what it was at
    the start) or as much as the cap allows; long enough that the running maximum crosses the blocks of the gates' scan"""
    rng = np.random.default_rng(4)
    n, H, D, V, cap = 1300, 2, 12, 20, 8.0
    r = lambda *s: rng.normal(size=s).astype(np.float32)
    q, k, v = r(n, H * D), r(n, H * D), r(n, H * V)
    gi, gf = (ib + r(n, H)).astype(np.float32), (fb + r(n, H)).astype(np.float32)
    want = oz.matrix_memory_scan(q.reshape(n, H, D).astype(np.float64) * D ** -0.5, k.reshape(n, H, D), v.reshape(n, H, V), oz.soft_cap(gi, cap),
                                 oz.log_sigmoid(oz.soft_cap(gf, cap)))
    late = oz.matrix_memory_scan(q.reshape(n, H, D).astype(np.float64) * D ** -0.5, k.reshape(n, H, D), v.reshape(n, H, V), oz.soft_cap(gi, cap) + 4.0,
                                 oz.log_sigmoid(oz.soft_cap(gf, cap)))
    if ib < 0:
        assert rel_err(late, want) > 0.05                                       # the input gate's size matters where the floor is the divisor
    for chunked, cuts in ((True, [0, n]), (False, [0, n]), (True, [0, 1100, 1164, n]), (False, [0, 5, 7, n])):
        S, N, M = torch.zeros(3, H, D, V, device="cuda"), torch.zeros(3, H, D, device="cuda"), torch.zeros(3, H, so.memory_copies(V), device="cuda")
        got = []
        for a, b in zip(cuts, cuts[1:]):
            o, den = so.matrix_memory(dev(q[a:b]), dev(k[a:b]), dev(v[a:b]), dev(gi[a:b]), dev(gf[a:b]), cap, D ** -0.5, S, N, M, i32([1]), i32([0]),
                                      i32([b - a]), b - a, H, D, V, chunked=chunked)
            got.append((o.view(b - a, H, V) * den[:, :, None]).cpu().numpy())
        assert rel_err(np.concatenate(got), want) < 5e-5
        assert not S[0].any() and not S[2].any() and not N[2].any() and not M[0].any()      # the other slots are untouched


def test_retention_remembers_one_far_key():
    """one row's key and value are large, the slow head still holds them hundreds of rows on; a decay that is a little off would show"""
    rng = np.random.default_rng(5)
    n, H, D, V = 700, 2, 16, 24
    r = lambda *s: rng.normal(size=s).astype(np.float32)
    x = np.concatenate([r(n, H * D), r(n, H * D), r(n, H * V)], 1)
    x[3, H * D:] *= 40.0
    decay = [0.998, 0.9]
    split = lambda a: (a[:, : H * D].reshape(n, H, D), a[:, H * D: 2 * H * D].reshape(n, H, D), a[:, 2 * H * D:].reshape(n, H, V))
    q, k, v = split(x)
    want = oz.retention_scan(q, k * 0.25, v, decay)
    q0, k0, v0 = split(np.where(np.arange(n)[:, None] == 3, 0.0, x))
    assert rel_err(oz.retention_scan(q, k0 * 0.25, v0, decay)[-1], want[-1]) > 0.1
    assert rel_err(oz.retention_scan(q, k * 0.25, v, [0.9985, 0.9])[-1], want[-1]) > 0.01
    load_pkg()
    from dash_infer_amd import seq_ops as so
    logs = torch.tensor(decay, dtype=torch.float64).log().cuda()
    for chunked, step in ((True, n), (False, n), (True, 130), (False, 1)):
        S, got = torch.zeros(1, H, D, V, device="cuda"), []
        for a in range(0, n, step):
            b = min(n, a + step)
            got.append(so.retention(dev(x[a:b]), 0, H * D, 2 * H * D, 0.25, logs, None, 0, 1, S, i32(list(range(a, b))), i32([0]), i32([0]), i32([b - a]),
                                    b - a, H, D, V, chunked=chunked).cpu().numpy().reshape(b - a, H, V))
        assert rel_err(np.concatenate(got), want) < 3e-5


@pytest.mark.parametrize("kind", ["retention", "memory"])
def test_sequences_side_by_side_and_a_slot_used_again(kind):
    rng = np.random.default_rng(6)
    if kind == "retention":
        (m, w), oracle, make = oz.retention_parts(rng, WIDTH), oz.retention, retention_rig
    else:
        (m, w), oracle, make = oz.memory_parts(rng, WIDTH), oz.matrix_memory, memory_rig
    hs = [rows(rng, n) for n in (90, 140, 7)]
    want = [oracle(x, w, m, EPS) for x in hs]
    rig = make(w, m, torch.float32, slots=3)
    for _ in range(2):                                                           # the second round takes slots that hold old state
        first = rig.step([("a", hs[0][:50]), ("b", hs[1][:1]), ("c", hs[2])])
        second = rig.step([("b", hs[1][1:131]), ("a", hs[0][50:])])
        third = rig.step([("b", hs[1][131:])])
        assert rel_err(np.concatenate([first[0], second[1]]), want[0]) < 3e-5
        assert rel_err(np.concatenate([first[1], second[0], third[0]]), want[1]) < 3e-5 and rel_err(first[2], want[2]) < 3e-5
        for name in "abc":
            rig.release(name)


# ---------------------------------------------------------------------------------------------------------------- attention
def attention_rig(w, m, dtype, max_tokens=2048, out_scale=1.0):
    mx, rot = mixers(), m["rot"]
    return MixerRig(lambda st, dt: mx.GroupedQueryAttention("att", m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], dev_weights(w), st, dt,
                                                            rot_dims=rot["dims"], rot_base=rot["base"], rot_layout="pairs", rot_scaling=rot.get("scaling"),
                                                            qk_norm="row", softcap=m["softcap"], conv=m["conv"], out_scale=out_scale), dtype,
                    max_tokens=max_tokens)


ATTENTION_SHAPES = {
    "plain": {},
    "odd_one_kv_head": dict(heads=3, kv_heads=1, dim=10, vdim=7, rot_dims=6, conv=2, scaling=None, softcap=3.0),
    "one_tap": dict(heads=4, kv_heads=4, dim=32, vdim=64, rot_dims=32, conv=1, scale=0.3),
    "many_taps": dict(heads=2, kv_heads=2, dim=88, vdim=104, rot_dims=20, conv=7, scaling=dict(factor=2.0, low=1.0, high=4.0, original=256)),
    "wide_rows": dict(heads=10, kv_heads=5, dim=128, vdim=16, rot_dims=128, conv=3),
    "no_rotation_no_cap": dict(heads=1, kv_heads=1, dim=9, vdim=200, rot_dims=0, softcap=None),
}


@pytest.mark.parametrize("shape", list(ATTENTION_SHAPES))
def test_attention_with_short_convolutions(shape):
    rng = np.random.default_rng(7)
    m, w = oz.attention_parts(rng, WIDTH, ATTENTION_SHAPES[shape])
    n = 150
    h = rows(rng, n)
    want = oz.conv_attention(h, w, m, EPS)
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 0.05)):
        rig = attention_rig(w, m, dtype)
        assert rel_err(rig.step([("a", h)])[0], want) < tol
        cuts = [0, 1, 2, 4, 6, 64, 65, 70, 128, 130, n]                          # portions shorter than the taps, pages' borders
        assert rel_err(portions(rig, "b", h, cuts), want) < tol
        dec = np.concatenate([rig.step([("c", h[i:i + 1])])[0] for i in range(90)])
        assert rel_err(dec, want[:90]) < tol
    rig = attention_rig(w, m, torch.float32, out_scale=0.3)
    assert rel_err(rig.step([("a", h)])[0] - w["o.b"], 0.3 * (want - w["o.b"])) < 2e-5     # the scale is on the heads, not on the output's bias


def test_attention_reads_one_far_key_across_pages():
    """one row's key has a large share of the query direction: the last rows put their weight on it, five pages on; cut out of the oracle's
    keys it would show, and so would a rotation by positions that are one off"""
    rng = np.random.default_rng(8)
    m, w = oz.attention_parts(rng, WIDTH, dict(scale=1.2, softcap=30.0, base=50.0, scaling=None))
    n = 400
    h = rows(rng, n)
    want = oz.conv_attention(h, w, m, EPS)
    moved = h.copy()
    moved[:100] = rows(rng, 100)
    assert rel_err(oz.conv_attention(moved, w, m, EPS)[-40:], want[-40:]) > 0.05
    assert rel_err(oz.conv_attention(h, w, dict(m, rot={"dims": 0}), EPS)[-40:], want[-40:]) > 0.05
    for dtype, tol in ((torch.float32, 5e-5), (torch.bfloat16, 0.08)):
        rig = attention_rig(w, m, dtype)
        got = np.concatenate([rig.step([("a", h[:360])])[0]] + [rig.step([("a", h[i:i + 1])])[0] for i in range(360, n)])
        assert rel_err(got[:360], want[:360]) < tol and rel_err(got[360:], want[360:]) < tol


def test_attention_unequal_portions_in_one_batch_and_pages_used_again():
    rng = np.random.default_rng(9)
    m, w = oz.attention_parts(rng, WIDTH)
    hs = [rows(rng, n) for n in (130, 1, 77)]
    want = [oz.conv_attention(x, w, m, EPS) for x in hs]
    rig = attention_rig(w, m, torch.float32, max_tokens=384)                     # 6 pages
    for _ in range(3):                                                           # pages, slots and convolution tails come back dirty
        first = rig.step([("a", hs[0][:60]), ("b", hs[1]), ("c", hs[2][:2])])
        one = rig.step([("c", hs[2][2:3]), ("a", hs[0][60:61])])
        second = rig.step([("a", hs[0][61:]), ("c", hs[2][3:])])
        assert rel_err(np.concatenate([first[0], one[1], second[0]]), want[0]) < 2e-5
        assert rel_err(first[1], want[1]) < 2e-5 and rel_err(np.concatenate([first[2], one[0], second[1]]), want[2]) < 2e-5
        for name in "abc":
            rig.release(name)


# ---------------------------------------------------------------------------------------------------------------- pair, experts
@pytest.mark.parametrize("left,right", [({}, {}), (dict(heads=3, kv_heads=3, dim=10, vdim=7, conv=1), dict(heads=1, dim=6, vdim=5))])
def test_weighted_pair(left, right):
    rng = np.random.default_rng(10)
    (lm, lw), (rm, rw) = oz.attention_parts(rng, WIDTH, left), oz.memory_parts(rng, WIDTH, right)
    cfg = {"left": lm, "right": rm, "left_scale": 0.7, "right_scale": 1.3}
    w = {**{"left." + k: v for k, v in lw.items()}, **{"right." + k: v for k, v in rw.items()}}
    h = rows(rng, 100)
    want = oz.parallel_mixer(h, w, cfg, EPS)
    mx = mixers()
    def build(st, dt):
        rot = lm["rot"]
        return mx.WeightedPair(mx.GroupedQueryAttention("att", lm["heads"], lm["kv_heads"], lm["dim"], lm["vdim"], lm["scale"], dev_weights(lw), st, dt,
                                                        rot_dims=rot["dims"], rot_base=rot["base"], rot_scaling=rot["scaling"], qk_norm="row",
                                                        softcap=lm["softcap"], conv=lm["conv"], out_scale=0.7),
                               mx.MatrixMemory("mem", rm["heads"], rm["dim"], rm["vdim"], rm["gate_cap"], dev_weights(rw), st, out_scale=1.3))
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 0.05)):
        rig = MixerRig(build, dtype)
        assert rel_err(portions(rig, "a", h, [0, 37, 38, 100]), want) < tol


@pytest.mark.parametrize("over", [{}, dict(experts=3, top=3, ff=9, shared=5), dict(experts=9, top=1, shared=0), dict(experts=70, top=4, ff=8, shared=16, limit=0.3)])
def test_routed_experts_with_a_gated_shared_one(over):
    rng = np.random.default_rng(11)
    fc, w = oz.ff_parts(rng, WIDTH, over)
    E, top = fc["router"]["experts"], fc["router"]["top"]
    h = rows(rng, 120)
    want = oz.moe_ff(h, w, fc)
    mx, d = mixers(), dev_weights(w)
    def build(st, dt):
        shared = mx.GatedMlp(d["shared.gate"], d["shared.up"], d["shared.down"], ("clamped", fc["shared"]["limit"])) if fc["shared"] else None
        return mx.ExpertMlp(d["router"], d["router.b"], [d[f"e{e}.gate"] for e in range(E)], [d[f"e{e}.up"] for e in range(E)],
                            [d[f"e{e}.down"] for e in range(E)], top, fc["expert"]["limit"], shared=shared, shared_gate=d.get("shared.sg"))
    for dtype, tol, few in ((torch.float32, 2e-5, 1.0), (torch.bfloat16, 0.05, 0.9)):
        rig = MixerRig(build, dtype)
        got = rig.step([("a", h)])[0]
        assert np.mean(np.abs(got - want).max(1) / np.abs(want).max() < tol) >= few
        (rws, dst, wts), add = rig.mixer.parts(rig.ctx, dev(h), dev(h, torch.bfloat16) if dtype == torch.bfloat16 else None)
        x = torch.zeros(120, WIDTH, device="cuda")
        rig.so.residual_rmsnorm(x, b=add, routed=(rws, dst, wts), x_out=x)       # summed inside the residual step
        assert rel_err(x.cpu().numpy(), got) < 1e-6
        alone = rig.step([("b", h[7:8])])[0]
        assert rel_err(alone, got[7:8]) < (1e-6 if dtype == torch.float32 else 0.05)
