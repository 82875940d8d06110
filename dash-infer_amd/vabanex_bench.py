"""bench.py --workload vabanex_layers: prefill and decode throughput of the sequence engine on random Vabanex models of layer sizes
that resemble real models', per-operator times of the design's kernels against their rooflines, and Filipel models of equal width,
heads, latent sizes and parameter count (the closest design the engine serves: the same latent attention with a gate per element,
group-limited routed experts, a dense feed-forward) with their like operators beside them."""
import math

import torch

from . import filipel_bench
from .seq_bench import HBM_BW, MFMA_BF16, _time, engine_throughput

SIZES = {
    # latent 512 + 64 rotated (a 576-element page row), frequencies rescaled by 40; experts: 32 in 8 groups of which 4 are kept, 4 per token
    "2k": dict(width=2048, heads=16, dim=128, rot=64, vdim=128, kv_rank=512, q_rank=768, ff=5376, experts=32, groups=8, keep=4, top=4, expert_ff=960,
               vocab=32000),
    "4k": dict(width=4096, heads=32, dim=128, rot=64, vdim=128, kv_rank=512, q_rank=1536, ff=9216, experts=32, groups=8, keep=4, top=4, expert_ff=1920,
               vocab=32000),
}
PATTERN = ("dense", "moe", "moe", "moe", "moe", "moe")


def random_model(size, device="cuda", seed=0, pattern=PATTERN):
    """config + bf16 tensors on the device (torch generator: nothing of it is trained or loaded)"""
    s = SIZES[size]
    g = torch.Generator(device=device).manual_seed(seed)
    W = s["width"]

    def r(*shape, sd=None):
        sd = sd if sd is not None else 1.0 / math.sqrt(shape[-1])
        return (torch.randn(*shape, generator=g, device=device) * sd).to(torch.bfloat16)

    def one(n):
        return (1 + 0.1 * torch.randn(n, generator=g, device=device)).to(torch.bfloat16)
    cfg = {"architecture": "Vabanex", "width": W, "vocab": s["vocab"], "norm": {"eps": 1e-6}, "embedding": {"scale": 1.0}, "logit_softcap": 20.0, "layers": []}
    t = {"embed": r(s["vocab"], W, sd=1.0), "head": r(s["vocab"], W)}

    def norm(name):
        t[name], t[name + ".b"] = one(W), r(W, sd=0.1)
    norm("final.norm")
    H, D, LR, V, R, Q = s["heads"], s["dim"], s["rot"], s["vdim"], s["kv_rank"], s["q_rank"]
    for i, ff in enumerate(pattern):
        p, q = f"l{i}.", f"l{i}.mix."
        norm(p + "norm1")
        norm(p + "norm2")
        m = {"heads": H, "dim": D, "rot_dim": LR, "vdim": V, "kv_rank": R, "q_rank": Q, "scale": 1.0 / math.sqrt(D + LR),
             "rot": {"base": 10000.0, "dims": LR, "scaling": {"factor": 40.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
        t[q + "dq"], t[q + "dq.norm"], t[q + "uq"] = r(Q, W), one(Q), r(H * (D + LR), Q)
        t[q + "dkv"], t[q + "dkv.norm"] = r(R + LR, W), one(R)
        t[q + "uk"], t[q + "uv"], t[q + "g"], t[q + "o"] = r(H * D, R), r(H * V, R), r(H, W), r(W, H * V)
        if ff == "dense":
            fc = {"kind": "dense", "ff": s["ff"], "limit": 7.0}
            t[p + "mlp.gate"], t[p + "mlp.up"], t[p + "mlp.down"] = r(s["ff"], W), r(s["ff"], W), r(W, s["ff"])
        else:
            E, F = s["experts"], s["expert_ff"]
            fc = {"kind": "moe", "expert": {"ff": F}, "router": {"experts": E, "top": s["top"], "scale": 2.5, "groups": {"count": s["groups"], "keep": s["keep"]}}}
            for e in range(E):
                t[p + f"mlp.e{e}.up"], t[p + f"mlp.e{e}.down"] = r(F, W), r(W, F)
            t[p + "mlp.router"], t[p + "mlp.correction"] = r(E, W), r(E, sd=0.2)
        cfg["layers"].append({"type": "latent_attention", "mixer": m, "mlp": fc})
    return cfg, t


def filipel_size(size):
    """the like sizes of a Filipel model: the same attention; its experts have three matrices of 2/3 the width where Vabanex experts have
    two, its dense feed-forward two of 3/2 the width where Vabanex has three"""
    s = SIZES[size]
    return dict(filipel_bench.SIZES[size], lat_heads=s["heads"], lat_dim=s["dim"], lat_rot=s["rot"], lat_vdim=s["vdim"], kv_rank=s["kv_rank"], q_rank=s["q_rank"],
                ff=s["ff"] * 3 // 2, experts=s["experts"], top=s["top"], expert_ff=s["expert_ff"] * 2 // 3, groups=s["groups"], keep=s["keep"], vocab=s["vocab"])


def _with_filipel_size(size, fn):
    saved = filipel_bench.SIZES[size]
    filipel_bench.SIZES[size] = filipel_size(size)
    try:
        return fn()
    finally:
        filipel_bench.SIZES[size] = saved


def filipel_equal_size(size):
    return _with_filipel_size(size, lambda: filipel_bench.random_model(size, pattern=tuple("latent+" + ff for ff in PATTERN)))


def operator_table(size, prompt_len, like=False):
    """the design's kernels alone, at the prompt's row count and at one row: seconds and the fraction of their bound (the larger of the
    matrix-core time at the bf16 peak and the bytes at 8 TB/s).  like: the Filipel design's form of the same step at equal size."""
    from . import seq_ops as so
    from .seq_state import SequenceStateManager
    s = SIZES[size]
    W, H, D, LR, V, R, Q = s["width"], s["heads"], s["dim"], s["rot"], s["vdim"], s["kv_rank"], s["q_rank"]
    Rp = -(-(R + LR) // 32) * 32
    E, top = s["experts"], s["top"]
    F = s["expert_ff"] * 2 // 3 if like else s["expert_ff"]
    ff = s["ff"] * 3 // 2 if like else s["ff"]
    dev = "cuda"
    out = []
    bf = lambda *sh: (torch.randn(*sh, device=dev) * 0.05).to(torch.bfloat16)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)

    def add(name, fn, flops, nbytes, reps=5):
        sec = _time(fn, reps)
        bound = max(flops / MFMA_BF16, nbytes / HBM_BW)
        row = {"op": name, "us": round(sec * 1e6, 1), "of_bound": round(bound / sec, 4)}
        if flops:
            row["tflops"] = round(flops / sec / 1e12, 1)
        out.append(row)
    for T in (prompt_len, 1):
        st = SequenceStateManager(prompt_len + 64, 1, 64, dev)
        lt = st.add_span_cache("c", Rp, torch.bfloat16)
        st.admit("a")
        st.reserve("a", prompt_len)
        st.upload()
        lt.pool.pool.view(torch.bfloat16).normal_(0, 0.3)
        pos = torch.arange(T, dtype=torch.int32, device=dev) if T > 1 else i32([prompt_len - 1])
        slot = torch.zeros(T, dtype=torch.int32, device=dev)
        e_slot, e_row0, e_cnt = i32([0]), i32([0]), i32([T])
        max_pos = int(pos[-1])
        # attention
        gcols = H * V if like else H
        a = torch.randn(T, Q + R + LR + gcols, device=dev)
        ckv, qrot, ql = a[:, Q:Q + R + LR], torch.randn(T, H * LR, device=dev), torch.randn(T, H * Rp, device=dev) * 0.1
        gam, freq = bf(R), torch.rand(LR // 2, device=dev)
        add(f"latent norm + rotated key part -> page, rotated query parts T={T}",
            lambda: so.latent_rope_append(lt, ckv, gam, 1e-6, R, LR, freq, qrot, ql, H, slot, pos, layout=1 if like else 0, mag=1.0 if like else 1.37),
            0, 4.0 * T * (R + LR) + 2.0 * T * Rp + 8.0 * T * H * LR)
        keys = sum(int(p) + 1 for p in pos.tolist())
        add(f"latent attention, all keys, row {Rp} (latent {R} + rotated {LR}) T={T} H={H}",
            lambda: so.latent_window_attn_mc(ql, lt, None, pos, e_slot, e_row0, e_cnt, T, max_pos, H, 0, 0.07, value=R),
            2.0 * keys * H * (R + LR + R), 2.0 * Rp * prompt_len + 4.0 * T * H * (Rp + R), 3)
        ol, uv = torch.randn(T, H * R, device=dev), bf(H, V, R)
        og = torch.empty(T, H * V, dtype=torch.bfloat16, device=dev)
        add(f"values per head x {'element' if like else 'head'} gate T={T}",
            lambda: so.linear(ol, uv, groups=H, mul=a[:, Q + R + LR:], mul_group=not like, math=so.MATH_BF16, out=og),
            2.0 * T * H * V * R, 4.0 * T * H * R + 2.0 * H * V * R + 2.0 * T * H * V + 4.0 * T * gcols)
        # norms and residual
        x, m1, m2, nw, nb = torch.randn(T, W, device=dev), torch.randn(T, W, device=dev), torch.randn(T, W, device=dev), bf(W), bf(W)
        if like:
            add(f"residual of two sublayers + layer norm T={T}",
                lambda: so.residual_layernorm(x, nw, a=m1, b=m2, mult=0.5, eps=1e-6, x_out=x, out_dtype=torch.bfloat16), 0, 18.0 * T * W)
        else:
            add(f"residual + biased layer norm T={T}",
                lambda: so.residual_layernorm(x, nw, a=m1, eps=1e-6, x_out=x, bias=nb, out_dtype=torch.bfloat16), 0, 14.0 * T * W)
        # dense feed-forward's activation
        act = torch.empty(T, ff, dtype=torch.bfloat16, device=dev)
        if like:
            zz, coef = torch.randn(T, ff, device=dev), bf(4)
            add(f"cubic of normalised powers T={T} x {ff}", lambda: so.polynorm(zz, coef, 1e-6, act), 0, 6.0 * T * ff)
        else:
            gu = torch.randn(T, 2 * ff, device=dev)
            add(f"clamped sigmoid-gated unit T={T} x {ff}", lambda: so.moe_glu(gu, ff, 7.0, 1.702, act), 0, 10.0 * T * ff)
        # routed experts
        h16 = (torch.randn(T, W, device=dev) * 0.5).to(torch.bfloat16)
        wr, corr = bf(E, W), bf(E)
        logits = torch.empty(T, E, device=dev)
        add(f"router logits (f32 products) T={T} x {E}", lambda: so.linear(h16, wr, out=logits, math=so.MATH_F32_STREAM), 0, 2.0 * T * W + 2.0 * E * W + 4.0 * T * E)
        if like:
            route = lambda: so.moe_route(logits, top, so.ROUTE_SCORES, None, (s["groups"], s["keep"]))
        else:
            route = lambda: so.moe_route(logits, top, so.ROUTE_SIGMOID, corr, (s["groups"], s["keep"]), group_top2=True, renorm=False, factor=2.5)
        name = "softmax, groups by their best" if like else "sigmoid + correction, groups by their two best"
        add(f"routing: {name}, {s['keep']} of {s['groups']} groups, top-{top} of {E}, grouping by expert T={T}", route, 0, 4.0 * T * E + 16.0 * T * top)
        _, wts, seg, src, dst = route()
        P = T * top
        used = min(E, P)      # experts whose weights a step of T rows reads, at most
        n_up = 2 * F if like else F
        w_up, w_dn = bf(E, n_up, W), bf(E, W, F)
        gu2, y, d = torch.empty(P, n_up, device=dev), torch.empty(P, F, dtype=torch.bfloat16, device=dev), torch.empty(P, W, device=dev)

        def units():
            if like:
                so.linear_segmented(h16, w_up, seg, src, T, P, out=gu2, math=so.MATH_BF16)
                so.moe_glu(gu2, F, 0.0, 1.702, y, unit=so.UNIT_SILU)
            else:
                so.linear_segmented(h16, w_up, seg, src, T, P, act="gelu_erf", out=y, math=so.MATH_BF16)
        add(f"experts' {'[gate | up] product + silu unit' if like else 'up product + gelu'} {P} pairs x {F}", units, 2.0 * P * n_up * W, 2.0 * used * n_up * W + 2.0 * P * (W + F))
        add(f"experts' down product {P} pairs", lambda: so.linear_segmented(y, w_dn, seg, None, T, P, out=d, math=so.MATH_BF16), 2.0 * P * F * W,
            2.0 * used * F * W + 2.0 * P * F + 4.0 * P * W)
        if like:
            add(f"residual of a sublayer + {top} routed rows per token + layer norm T={T}",
                lambda: so.residual_layernorm(x, nw, a=m1, routed=(d, dst, wts), mult=0.5, eps=1e-6, x_out=x, out_dtype=torch.bfloat16), 0,
                4.0 * P * W + 14.0 * T * W)
        else:
            add(f"residual of {top} routed rows per token + biased layer norm T={T}",
                lambda: so.residual_layernorm(x, nw, routed=(d, dst, wts), eps=1e-6, x_out=x, bias=nb, out_dtype=torch.bfloat16), 0, 4.0 * P * W + 10.0 * T * W)
        if T == 1:
            head = bf(s["vocab"], W)
            add(f"head {'' if like else '+ cap '}{s['vocab']} x {W}", lambda: so.linear(h16, head, act=None if like else "softcap", act_param=20.0, math=so.MATH_BF16),
                2.0 * s["vocab"] * W, 2.0 * s["vocab"] * W)
    return out


def run(args):
    from . import models
    from .engine import SeqEngine
    prompt_len = 2048
    res = {"metric": "prefill / decode throughput of the sequence engine (random Vabanex models) beside Filipel models of equal size",
           "unit": "tokens/s", "n_gpus": 1, "dtype": "bf16", "data": "synthetic", "prompt_len": prompt_len, "sizes": {}}
    for size in SIZES:
        entry = {"layers": ["latent_attention+" + ff for ff in PATTERN], **SIZES[size]}
        for name, make in (("engine", random_model), ("filipel_equal_size", filipel_equal_size)):
            cfg, t = make(size)
            eng = SeqEngine(models.resolve(cfg), cfg, t, dtype=torch.bfloat16, max_tokens=4 * (prompt_len + 128), max_slots=4)
            entry[name] = engine_throughput(eng, cfg["vocab"], prompt_len)
            entry[name]["weight_bytes"] = int(sum(v.numel() * v.element_size() for k, v in t.items() if k != "embed"))
            del eng, t
            torch.cuda.empty_cache()
        entry["operators"] = operator_table(size, prompt_len)
        entry["filipel_operators"] = operator_table(size, prompt_len, like=True)
        res["sizes"][size] = entry
    res["value"] = res["sizes"]["4k"]["engine"]["prefill_tokens_per_s"]
    return res
