"""bench.py --workload zusuvik_layers: prefill and decode throughput of the sequence engine on random Zusuvik models of layer sizes that
resemble real models', per-operator times of the design's kernels against their rooflines, and Vogusun models of equal width, heads and
active feed-forward size (the closest design the engine serves: parallel layers, grouped-query attention with capped scores, gated linear
attention, routed clamped units) with their like operators beside them."""
import math
import sys

import torch

from . import vogusun_bench
from .seq_bench import HBM_BW, MFMA_BF16, VALU_F32, _time, engine_throughput

SIZES = {
    # attention: heads / kv heads of 128, 4 taps; matrix memory: heads of 128 x 128; retention: heads of 64 x 128; experts: 8 of which 2 per
    # token, with the shared one as many active parameters as the Vogusun model's two
    "2k": dict(width=2048, heads=16, kv_heads=4, dim=128, vdim=128, taps=4, mem_heads=8, mem_dim=128, mem_vdim=128, ret_heads=16, ret_dim=64, ret_vdim=128,
               experts=8, top=2, expert_ff=3072, shared_ff=2048, vocab=32000),
    "4k": dict(width=4096, heads=32, kv_heads=8, dim=128, vdim=128, taps=4, mem_heads=16, mem_dim=128, mem_vdim=128, ret_heads=32, ret_dim=64, ret_vdim=128,
               experts=8, top=2, expert_ff=5120, shared_ff=4096, vocab=32000),
}
PATTERN = ("parallel", "retention") * 3
LIKE_PATTERN = ("attention_2+moe", "gla+moe") * 3


def random_model(size, device="cuda", seed=0, pattern=PATTERN, loop=None):
    """config + bf16 tensors on the device (torch generator: nothing of it is trained or loaded)"""
    s = SIZES[size] if isinstance(size, str) else size
    g = torch.Generator(device=device).manual_seed(seed)
    W = s["width"]

    def r(*shape, sd=None):
        sd = sd if sd is not None else 1.0 / math.sqrt(shape[-1])
        return (torch.randn(*shape, generator=g, device=device) * sd).to(torch.bfloat16)

    one = lambda n: 1 + r(n, sd=0.1)
    cfg = {"architecture": "Zusuvik", "width": W, "vocab": s["vocab"], "norm": {"eps": 1e-6}, "logit_scale": 0.02, "layers": []}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    t = {"embed": r(s["vocab"], W, sd=1.0), "final.norm": r(W, sd=0.1)}
    for i, kind in enumerate(pattern):
        p, q = f"l{i}.", f"l{i}.mix."
        t[p + "norm1"], t[p + "norm2"] = r(W, sd=0.1), r(W, sd=0.1)
        if kind == "retention":
            H, D, V = s["ret_heads"], s["ret_dim"], s["ret_vdim"]
            m = {"heads": H, "dim": D, "vdim": V, "decay": [1.0 - 2.0 ** (-5.0 - 7.0 * h / H) for h in range(H)], "rot": {"base": 10000.0, "dims": D}}
            t[q + "q"], t[q + "k"], t[q + "v"], t[q + "g"], t[q + "o"] = r(H * D, W), r(H * D, W), r(H * V, W), r(H * V, W), r(W, H * V)
        else:
            H, G, D, V, taps = s["heads"], s["kv_heads"], s["dim"], s["vdim"], s["taps"]
            left = {"heads": H, "kv_heads": G, "dim": D, "vdim": V, "conv": taps, "scale": 1.0 / math.sqrt(D), "softcap": 50.0,
                    "rot": {"base": 500000.0, "dims": D // 2, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
            for n, rows in (("q", H * D), ("k", G * D), ("v", G * V)):
                t[q + f"left.{n}"], t[q + f"left.{n}.b"], t[q + f"left.{n}.conv"] = r(rows, W), r(rows, sd=0.1), r(rows, taps, sd=0.5)
            t[q + "left.q.norm"], t[q + "left.k.norm"], t[q + "left.o"], t[q + "left.o.b"] = one(H * D), one(G * D), r(W, H * V), r(W, sd=0.1)
            H, D, V = s["mem_heads"], s["mem_dim"], s["mem_vdim"]
            for n, rows in (("q", H * D), ("k", H * D), ("v", H * V), ("g", H * V), ("i", H), ("f", H)):
                t[q + f"right.{n}"] = r(rows, W)
            t[q + "right.o"], t[q + "right.norm"], t[q + "right.i.b"], t[q + "right.f.b"] = r(W, H * V), one(H * V), r(H, sd=1.0), 4 + r(H, sd=1.0)
            m = {"left": left, "right": {"heads": H, "dim": D, "vdim": V, "gate_cap": 15.0}, "left_scale": 0.75, "right_scale": 0.6}
        E, F, FS = s["experts"], s["expert_ff"], s["shared_ff"]
        for e, f in [(f"e{e}", F) for e in range(E)] + [("shared", FS)]:
            t[p + f"mlp.{e}.gate"], t[p + f"mlp.{e}.up"], t[p + f"mlp.{e}.down"] = r(f, W), r(f, W), r(W, f)
        t[p + "mlp.router"], t[p + "mlp.router.b"], t[p + "mlp.shared.sg"] = r(E, W), r(E, sd=0.1), r(1, W)
        cfg["layers"].append({"type": kind, "mixer": m, "mlp": {"kind": "moe", "expert": {"ff": F, "limit": 7.0}, "router": {"experts": E, "top": s["top"]},
                                                                "shared": {"ff": FS, "limit": 7.0}}})
    return cfg, t


def vogusun_equal_size(size):
    s = SIZES[size]
    v = dict(vogusun_bench.SIZES[size], heads=s["heads"], kv_heads=s["kv_heads"], dim=s["dim"], vdim=s["vdim"], gla_heads=s["ret_heads"], gla_dim=s["ret_dim"],
             gla_vdim=s["ret_vdim"], experts=s["experts"], top=s["top"], expert_ff=s["expert_ff"] + s["shared_ff"] // s["top"], vocab=s["vocab"])
    return vogusun_bench.random_model(v, pattern=LIKE_PATTERN)


def _seconds(fn, T):
    """seconds per call on the device: few-row calls are shorter than their launch from Python, so twenty of them replay as one graph"""
    if T > 1:
        return _time(fn, 5)
    fn()
    torch.cuda.synchronize()
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        for _ in range(20):
            fn()
    return _time(g.replay, 5) / 20


def operator_table(size, prompt_len):
    """the design's kernels and the Vogusun design's like ones at the same sizes, at the prompt's row count and at one row: seconds and the
    fraction of their bound (the largest of matrix work at the bf16 peak, f32 recurrences at the vector units' peak -- each key-value element
    of the state read and written by two multiply-adds per row -- and the bytes at 8 TB/s)"""
    from . import seq_ops as so
    from .seq_state import SequenceStateManager
    s = SIZES[size]
    W, H, G, D, V, taps = s["width"], s["heads"], s["kv_heads"], s["dim"], s["vdim"], s["taps"]
    E, top, F, FS = s["experts"], s["top"], s["expert_ff"], s["shared_ff"]
    dev = "cuda"
    out = []
    bf = lambda *sh: (torch.randn(*sh, device=dev) * 0.05).to(torch.bfloat16)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)

    def add(name, T, fn, nbytes, mfma=0.0, valu=0.0, like=None):
        """like: (name, fn, bytes, mfma, valu) of the Vogusun design's form of the step"""
        def one(fn, nbytes, mfma, valu):
            sec = _seconds(fn, T)
            return round(sec * 1e6, 1), round(max(nbytes / HBM_BW, mfma / MFMA_BF16, valu / VALU_F32) / sec, 4)
        row = {"op": f"{name} T={T}"}
        row["us"], row["of_bound"] = one(fn, nbytes, mfma, valu)
        if like is not None:
            row["vogusun_op"] = like[0]
            row["vogusun_us"], row["vogusun_of_bound"] = one(*like[1:])
        out.append(row)
    for T in (prompt_len, 1):
        st = SequenceStateManager(prompt_len + 64, 1, 64, dev)
        kt, vt = st.add_span_cache("k", G * D, torch.bfloat16), st.add_span_cache("v", G * V, torch.bfloat16)
        st.admit("a")
        st.reserve("a", prompt_len)
        st.upload()
        for tab in (kt, vt):
            tab.pool.pool.view(torch.bfloat16).normal_(0, 0.3)
        pos = torch.arange(T, dtype=torch.int32, device=dev) if T > 1 else i32([prompt_len - 1])
        slot, off = torch.zeros(T, dtype=torch.int32, device=dev), torch.arange(T, dtype=torch.int32, device=dev)
        es, er, ec, max_pos = i32([0]), i32([0]), i32([T]), int(pos[-1])
        # -- attention
        C = (H + G) * D + G * V
        a = torch.randn(T, C + H, device=dev) * 0.3
        conv, tail = bf(taps, C), torch.zeros(1, taps - 1, C, device=dev)
        qn, kn, hn, freq = bf(H * D) + 1, bf(G * D) + 1, bf(D) + 1, torch.rand(D // 2, device=dev)
        prep_bytes = 4.0 * T * C + 4.0 * T * H * D + 2.0 * T * G * (D + V)
        add(f"convolution of {taps} taps + row norms + rotation + page append", T,
            lambda: so.qkv_conv_prep_append(a, conv, tail, T == 1, H, G, D, V, qn, kn, 1e-6, freq, D // 2, 0, 1.0, kt, vt, slot, pos, off),
            prep_bytes + (0 if T > 1 else 8.0 * (taps - 1) * C),
            like=("norms per head + rotation + page append",
                  lambda: so.qkv_prep_append(a, 0, H * D, (H + G) * D, H, G, D, V, hn, hn, 1e-6, freq, D, 0, 1.0, 0.0, None, None, kt, vt, slot, pos), prep_bytes, 0.0, 0.0))
        q, gain, o = torch.randn(T, H * D, device=dev), torch.full((1, H), 0.8, device=dev).expand(T, H), torch.empty(T, H * V, dtype=torch.bfloat16, device=dev)
        keys = sum(int(p) + 1 for p in pos.tolist())
        att = (2.0 * G * (D + V) * prompt_len + T * H * (4.0 * D + 2.0 * V), 2.0 * keys * H * (D + V), 0.0)
        attend = lambda **kw: so.gqa_attn_mc(q, kt, vt, pos, es, er, ec, T, max_pos, H, G, D, V, 0.09, softcap=50.0, out=o, **kw)
        add(f"attention, capped scores, scaled result H={H} G={G}", T, lambda: attend(gate=gain), *att, like=("attention, capped scores", attend, *att))
        # -- recurrences, beside gated linear attention of the same state size
        def gla(h, d, v):
            x, z = torch.randn(T, 3 * h * d + h * v, device=dev) * 0.3, torch.zeros(1, h, d, v, device=dev)
            oo = torch.empty(T, h * v, device=dev)
            return lambda: so.gla(x, x[:, h * d:], x[:, 3 * h * d:], x[:, 2 * h * d:], 0.125, 8.0, z, es, er, ec, T, h, d, v, out=oo)
        rec = lambda h, d, v, extra: (4.0 * T * (extra + 2 * h * d + 2 * h * v) + 8.0 * h * d * v, 0.0, 4.0 * T * h * d * v)
        h, d, v = s["ret_heads"], s["ret_dim"], s["ret_vdim"]
        x = torch.randn(T, 2 * h * d + 2 * h * v, device=dev) * 0.3
        logs, S, fr, ro = torch.full((h,), -0.01, dtype=torch.float64, device=dev), torch.zeros(1, h, d, v, device=dev), torch.rand(d // 2, device=dev), torch.empty(T, h * v, device=dev)
        add(f"retention with its rotation, heads={h} D={d} V={v}", T,
            lambda: so.retention(x, 0, h * d, 2 * h * d, d ** -0.5, logs, fr, d, 1, S, pos, es, er, ec, T, h, d, v, out=ro), *rec(h, d, v, 0),
            like=("gated linear attention", gla(h, d, v), *rec(h, d, v, h * d)))
        mul, y16 = torch.rand(T, h * v, device=dev), torch.empty(T, h * v, dtype=torch.bfloat16, device=dev)
        gam = bf(v) + 1
        nb = 10.0 * T * h * v
        add("per-head norm x gate (retention)", T, lambda: so.head_rmsnorm_mul(ro, None, 1e-6, h, v, mul=mul, out=y16), nb,
            like=("per-head norm x gate", lambda: so.head_rmsnorm_mul(ro, gam, 1e-6, h, v, mul=mul, out=y16), nb, 0.0, 0.0))
        h2, d2, v2 = s["mem_heads"], s["mem_dim"], s["mem_vdim"]
        x2 = torch.randn(T, 2 * h2 * d2 + h2 * v2 + 2 * h2, device=dev) * 0.3
        S2, N2, M2 = torch.zeros(1, h2, d2, v2, device=dev), torch.zeros(1, h2, d2, device=dev), torch.zeros(1, h2, so.memory_copies(v2), device=dev)
        mo, gi = torch.empty(T, h2 * v2, device=dev), 2 * h2 * d2 + h2 * v2
        add(f"matrix memory with its gates, heads={h2} D={d2} V={v2}", T,
            lambda: so.matrix_memory(x2, x2[:, h2 * d2:], x2[:, 2 * h2 * d2:], x2[:, gi:], x2[:, gi + h2:], 15.0, d2 ** -0.5, S2, N2, M2, es, er, ec, T, h2, d2, v2, out=mo),
            *rec(h2, d2, v2, 3 * h2), like=("gated linear attention", gla(h2, d2, v2), *rec(h2, d2, v2, h2 * d2)))
        # -- the residual step
        xs, m1, m2, w1, w2 = torch.randn(T, W, device=dev), torch.randn(T, W, device=dev), torch.randn(T, W, device=dev), bf(W), bf(W)
        h16 = (torch.randn(T, W, device=dev) * 0.5).to(torch.bfloat16)
        R = T * top
        logits = torch.randn(T, E, device=dev)
        _, wts, seg, src, dst = so.moe_route(logits, top)
        dn = torch.randn(R, W, device=dev)
        nw = (0.75, bf(W) + 1, bf(W))

        def vogusun_step():
            so.add_dyt(xs, m1, so.moe_combine(dn, dst, wts, T, top), norm=nw, x_out=xs, want16=True)
        add(f"residual of two sublayers and {top} routed rows + two norms", T,
            lambda: so.residual_rmsnorm(xs, w1, w2, a=m1, b=m2, routed=(dn, dst, wts), eps=1e-6, x_out=xs, out_dtype=torch.bfloat16), 20.0 * T * W + 4.0 * R * W,
            like=("weighted sum of routed rows; residual of two sublayers + norm", vogusun_step, 14.0 * T * W + 4.0 * R * W, 0.0, 0.0))
        # -- feed-forward
        wx, rb = bf(((E + 3) & ~3) + 4 + 2 * FS, W), bf(E, W)
        zx = torch.empty(T, wx.shape[0], device=dev)
        lin = lambda n, k, xe: (2.0 * n * k + 4.0 * T * n + xe * T * k, 2.0 * T * n * k, 0.0)
        wv = bf(2 * FS, W)
        zv = torch.empty(T, 2 * FS, device=dev)

        def vogusun_two():
            so.linear(h16, rb, out=logits, math=so.MATH_F32_STREAM)
            so.linear(h16, wv, out=zv, math=so.MATH_BF16)
        few = ((E + 3) & ~3) + 4
        zr = torch.empty(T, few, device=dev)

        def zusuvik_x():       # few rows: one product; many: the few columns apart
            if T <= 16:
                return so.linear(h16, wx, out=zx, math=so.MATH_BF16)
            so.linear(h16, wx[:few], out=zr, math=so.MATH_F32_STREAM)
            so.linear(h16, wx[few:], out=zv, math=so.MATH_BF16)
        add(f"router, shared gate and shared [gate | up], {wx.shape[0]} columns", T, zusuvik_x, *lin(wx.shape[0], W, 2.0),
            like=("router logits; a dense [gate | up] product", vogusun_two, *lin(2 * FS + E, W, 2.0)))
        w_gu, w_dn, used = bf(E, 2 * F, W), bf(E, W, F), min(E, R)
        gu, y = torch.empty(R, 2 * F, device=dev), torch.empty(R, F, dtype=torch.bfloat16, device=dev)
        add(f"routing: top-{top} of {E}, grouping by expert", T, lambda: so.moe_route(logits, top), 4.0 * T * E + 16.0 * R)
        add(f"experts' [gate | up] [{R}x{W}]x[{E}x{2 * F}]", T, lambda: so.linear_segmented(h16, w_gu, seg, src, T, R, out=gu, math=so.MATH_BF16),
            4.0 * used * F * W + 8.0 * R * F + 2.0 * R * W, 4.0 * R * F * W)
        add(f"experts' clamped unit [{R}x{F}]", T, lambda: so.moe_glu(gu, F, 7.0, 1.702, y), 10.0 * R * F)
        add(f"experts' down [{R}x{F}]x[{E}x{W}]", T, lambda: so.linear_segmented(y, w_dn, seg, None, T, R, out=dn, math=so.MATH_BF16),
            2.0 * used * F * W + 2.0 * R * F + 4.0 * R * W, 2.0 * R * F * W)
        del w_gu, w_dn, wx, wv
        # -- the pair's products
        n_in, k_out = C + 2 * h2 * d2 + 2 * h2 * v2 + 2 * h2, H * V + h2 * v2
        wi, wo = bf(n_in, W), bf(W, k_out)
        yi, both, yo = torch.empty(T, n_in, device=dev), torch.randn(T, k_out, device=dev).to(torch.bfloat16), torch.empty(T, W, device=dev)
        add(f"both mixers' input product, {n_in} columns", T, lambda: so.linear(h16, wi, out=yi, math=so.MATH_BF16), *lin(n_in, W, 2.0))
        add(f"both mixers' output product over {k_out}", T, lambda: so.linear(both, wo, out=yo, math=so.MATH_BF16), *lin(W, k_out, 2.0))
    return out


def run(args):
    from . import models
    from .engine import SeqEngine
    prompt_len = 2048
    res = {"metric": "prefill / decode throughput of the sequence engine (random Zusuvik models) beside Vogusun models of equal size",
           "unit": "tokens/s", "n_gpus": 1, "dtype": "bf16", "data": "synthetic", "prompt_len": prompt_len, "sizes": {}}
    for size in SIZES:
        entry = {"layers": list(PATTERN), "vogusun_layers": list(LIKE_PATTERN), **SIZES[size]}
        for name, make in (("engine", random_model), ("vogusun_equal_size", vogusun_equal_size)):
            cfg, t = make(size)
            eng = SeqEngine(models.resolve(cfg), cfg, t, dtype=torch.bfloat16, max_tokens=4 * (prompt_len + 128), max_slots=4)
            entry[name] = engine_throughput(eng, cfg["vocab"], prompt_len)
            entry[name]["weight_bytes"] = int(sum(v.numel() * v.element_size() for k, v in t.items() if k != "embed" or "head" not in t))
            del eng, t
            torch.cuda.empty_cache()
            print(f"# {size} {name} {entry[name]}", file=sys.stderr, flush=True)
        entry["operators"] = operator_table(size, prompt_len)
        res["sizes"][size] = entry
    res["value"] = res["sizes"]["4k"]["engine"]["prefill_tokens_per_s"]
    return res
