"""Plain, slow float64 restatement of the Vabanex design, one function per mechanism, row by row.  Test infrastructure only:
numpy, no kernels, no code shared with the product path.

Notation: h [n, width] the rows of ONE sequence in order (row p is position p); weights as the checkpoint stores them
([out, in]); w maps the names below '<layer>.mix.' / '<layer>.mlp.' to arrays."""
import math

import numpy as np


def f64(a):
    return np.asarray(a, np.float64)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-f64(z)))


def gelu_exact(z):
    z = f64(z)
    return 0.5 * z * (1.0 + np.vectorize(math.erf)(z / math.sqrt(2.0)))


def unit_rms(x, eps):
    x = f64(x)
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def layer_norm(x, w, b, eps):
    """mean and variance over the row, a weight and a bias"""
    x = f64(x)
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * f64(w) + f64(b)


def soft_cap(z, cap):
    return cap * np.tanh(f64(z) / cap) if cap else f64(z)


# -- rotary positions -----------------------------------------------------------------------------------------------------
def pair_frequencies(dims, base, scaling=None):
    """-> (frequency per pair, magnitude of cos and sin).  With scaling: pairs that turn often within the original context keep their
    frequency, pairs that hardly turn are slowed down by the factor, a linear ramp over the pair's index between."""
    i = np.arange(dims // 2, dtype=np.float64)
    f = float(base) ** (-2.0 * i / dims)
    if not scaling:
        return f, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def index_of(turns):     # the (fractional) index of the pair that turns `turns` times over the original context
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(index_of(float(scaling["fast"]))), 0)
    hi = min(math.ceil(index_of(float(scaling["slow"]))), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / factor * ramp + f * (1.0 - ramp), 0.1 * math.log(factor) + 1.0


def rotate_pairs(x, pos, dims, base, scaling=None):
    """x [.., dim] of the token at position pos: dimension 2i turns with dimension 2i + 1; the dimensions from dims on stay.  The
    angle is the 32-bit product of position and frequency."""
    f, mag = pair_frequencies(dims, base, scaling)
    ang = (np.float32(pos) * f.astype(np.float32)).astype(np.float64)
    c, s = mag * np.cos(ang), mag * np.sin(ang)
    out = f64(x).copy()
    u, v = f64(x)[..., 0:dims:2], f64(x)[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def softmax_weights(scores):
    e = np.exp(scores - scores.max())
    return e / e.sum()


# -- attention through a latent with a shared rotated key part ------------------------------------------------------------
def latent_keys(h, w, m, eps):
    """what the layer caches: (latent c [n, kv_rank], rotated key part [n, rot_dim])"""
    R, Rd, rot = int(m["kv_rank"]), int(m["rot_dim"]), m["rot"]
    kv = f64(h) @ f64(w["dkv"]).T
    c = unit_rms(kv[:, :R], eps) * f64(w["dkv.norm"])
    kr = np.stack([rotate_pairs(kv[p, R: R + Rd], p, int(rot["dims"]), float(rot["base"]), rot.get("scaling")) for p in range(h.shape[0])])
    return c, kr


def latent_attention(h, w, m, eps):
    n = h.shape[0]
    H, D, Rd, V, rot = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), m["rot"]
    h = f64(h)
    cq = unit_rms(h @ f64(w["dq"]).T, eps) * f64(w["dq.norm"])
    q = (cq @ f64(w["uq"]).T).reshape(n, H, D + Rd)
    c, kr = latent_keys(h, w, m, eps)
    k = (c @ f64(w["uk"]).T).reshape(n, H, D)
    v = (c @ f64(w["uv"]).T).reshape(n, H, V)
    gate = sigmoid(h @ f64(w["g"]).T)                        # [n, H]: one number per head
    out = np.zeros((n, H, V))
    for i in range(n):
        qr = rotate_pairs(q[i, :, D:], i, int(rot["dims"]), float(rot["base"]), rot.get("scaling"))
        for hd in range(H):
            s = (k[: i + 1, hd] @ q[i, hd, :D] + kr[: i + 1] @ qr[hd]) * float(m["scale"])
            out[i, hd] = gate[i, hd] * (softmax_weights(s) @ v[: i + 1, hd])
    return out.reshape(n, H * V) @ f64(w["o"]).T


# -- feed-forward -----------------------------------------------------------------------------------------------------------
def dense_ff(h, w, fc):
    lim = float(fc["limit"])
    g = np.minimum(f64(h) @ f64(w["gate"]).T, lim)
    u = np.clip(f64(h) @ f64(w["up"]).T, -lim, lim)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ f64(w["down"]).T


def route_scores(s, correction, top, count, keep, factor):
    """s [n, E] in (0, 1) -> (chosen experts [n, top], weights [n, top])"""
    n, E = s.shape
    gsz = E // count
    idx, ws = np.zeros((n, top), np.int64), np.zeros((n, top))
    for t in range(n):
        choice = f64(s[t]) + f64(correction)
        groups = np.array([np.sort(choice[g * gsz: (g + 1) * gsz])[::-1][:2].sum() for g in range(count)])
        kept = np.argsort(-groups, kind="stable")[:keep]
        open_ = np.full(E, -np.inf)
        for g in kept:
            open_[g * gsz: (g + 1) * gsz] = choice[g * gsz: (g + 1) * gsz]
        idx[t] = np.argsort(-open_, kind="stable")[:top]
        ws[t] = s[t, idx[t]] * factor
    return idx, ws


def route(h, w, fc):
    r = fc["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    return route_scores(sigmoid(f64(h) @ f64(w["router"]).T), w["correction"], int(r["top"]), int(g["count"]), int(g["keep"]), float(r["scale"]))


def moe_ff(h, w, fc, chosen=None):
    h = f64(h)
    idx, ws = route(h, w, fc)
    if chosen is not None:
        chosen.extend(idx.tolist())
    out = np.zeros_like(h)
    for e in np.unique(idx):
        t, k = np.nonzero(idx == e)
        y = gelu_exact(h[t] @ f64(w[f"e{e}.up"]).T) @ f64(w[f"e{e}.down"]).T
        np.add.at(out, t, ws[t, k][:, None] * y)
    return out


# -- the model --------------------------------------------------------------------------------------------------------------
def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def forward(cfg, tensors, tokens, streams=None):
    """tokens of ONE sequence from position 0 -> logits [n, vocab]; streams: a list that receives the residual stream after every layer"""
    eps = float(cfg["norm"]["eps"])
    x = f64(tensors["embed"])[np.asarray(tokens)] * float(cfg["embedding"]["scale"])
    for i, lc in enumerate(cfg["layers"]):
        w = sub(tensors, f"l{i}.")
        if lc["type"] != "latent_attention":
            raise ValueError(lc["type"])
        x = x + latent_attention(layer_norm(x, w["norm1"], w["norm1.b"], eps), sub(w, "mix."), lc["mixer"], eps)
        fc = lc.get("mlp")
        if fc is not None:
            h = layer_norm(x, w["norm2"], w["norm2.b"], eps)
            x = x + (dense_ff(h, sub(w, "mlp."), fc) if fc["kind"] == "dense" else moe_ff(h, sub(w, "mlp."), fc))
        if streams is not None:
            streams.append(x.copy())
    z = layer_norm(x, tensors["final.norm"], tensors["final.norm.b"], eps) @ f64(tensors["head"]).T
    return soft_cap(z, float(cfg.get("logit_softcap") or 0.0))


# -- small random models (tests) --------------------------------------------------------------------------------------------
def bf16_values(a):
    """float32 array whose values are exactly representable in bfloat16 (round to nearest even)"""
    u = np.asarray(a, np.float32).view(np.uint32)
    u = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16) << 16
    return u.astype(np.uint32).view(np.float32)


YARN = dict(factor=3.0, original=64, fast=6.0, slow=0.5)
LATENT = dict(heads=3, dim=16, rot_dim=8, vdim=20, kv_rank=24, q_rank=28, base=5000.0, scaling=YARN, scale=None)
DENSE = dict(ff=50, limit=1.5)
MOE = dict(experts=6, count=3, keep=2, top=2, ff=20, scale=2.5)


def latent_weights(rng, width, o):
    bf = bf16_values
    r = lambda *s: bf(rng.normal(0, 1.0 / math.sqrt(s[-1]), s))
    H, D, Rd, V, R, Q = o["heads"], o["dim"], o["rot_dim"], o["vdim"], o["kv_rank"], o["q_rank"]
    return {"dq": r(Q, width), "dq.norm": bf(1.0 + 0.2 * rng.normal(size=Q)), "uq": r(H * (D + Rd), Q), "dkv": r(R + Rd, width),
            "dkv.norm": bf(1.0 + 0.2 * rng.normal(size=R)), "uk": r(H * D, R), "uv": r(H * V, R), "g": bf(rng.normal(0, 2.0 / math.sqrt(width), (H, width))),
            "o": r(width, H * V)}


def latent_config(o):
    rot = {"base": o["base"], "dims": o["rot_dim"]}
    if o["scaling"]:
        rot["scaling"] = dict(o["scaling"])
    return {"heads": o["heads"], "dim": o["dim"], "rot_dim": o["rot_dim"], "vdim": o["vdim"], "kv_rank": o["kv_rank"], "q_rank": o["q_rank"],
            "rot": rot, "scale": o["scale"] if o["scale"] is not None else (o["dim"] + o["rot_dim"]) ** -0.5}


def ff_config(spec):
    """spec: None, ("dense", overrides of DENSE) or ("moe", overrides of MOE)"""
    if spec is None:
        return None
    over = spec[1] if len(spec) > 1 else {}
    if spec[0] == "dense":
        return {"kind": "dense", **dict(DENSE, **over)}
    o = dict(MOE, **over)
    r = {"experts": o["experts"], "top": o["top"], "scale": o["scale"]}
    if o["count"]:
        r["groups"] = {"count": o["count"], "keep": o["keep"]}
    return {"kind": "moe", "expert": {"ff": o["ff"]}, "router": r}


def ff_weights(rng, width, fc):
    bf = bf16_values
    r = lambda *s: bf(rng.normal(0, 1.0 / math.sqrt(s[-1]), s))
    if fc["kind"] == "dense":
        return {"gate": r(fc["ff"], width), "up": r(fc["ff"], width), "down": r(width, fc["ff"])}
    E, F = fc["router"]["experts"], fc["expert"]["ff"]
    w = {"router": bf(rng.normal(0, 2.0 / math.sqrt(width), (E, width))), "correction": bf(rng.normal(-0.6, 0.4, E))}   # choice scores of both signs
    for e in range(E):
        w[f"e{e}.up"], w[f"e{e}.down"] = r(F, width), r(width, F)
    return w


def random_vabanex(rng, layers, width=72, vocab=97, eps=1e-5, embed_scale=0.7, softcap=9.0):
    """A small random model -> (config, tensors as float32 arrays of bf16 values).  layers: a list of (overrides of LATENT, ff spec as
    ff_config takes it); softcap None: the configuration has no cap."""
    bf = bf16_values
    cfg = {"architecture": "Vabanex", "width": width, "vocab": vocab, "norm": {"eps": eps}, "embedding": {"scale": embed_scale}, "layers": []}
    if softcap is not None:
        cfg["logit_softcap"] = softcap
    t = {"embed": bf(rng.normal(size=(vocab, width))), "head": bf(rng.normal(0, 3.0 / math.sqrt(width), (vocab, width)))}

    def norm(name):
        t[name], t[name + ".b"] = bf(1.0 + 0.2 * rng.normal(size=width)), bf(0.3 * rng.normal(size=width))
    norm("final.norm")
    for i, (over, ff) in enumerate(layers):
        p, o, fc = f"l{i}.", dict(LATENT, **(over or {})), ff_config(ff)
        norm(p + "norm1")
        for k, v in latent_weights(rng, width, o).items():
            t[p + "mix." + k] = v
        if fc is not None:
            norm(p + "norm2")
            for k, v in ff_weights(rng, width, fc).items():
                t[p + "mlp." + k] = v
        cfg["layers"].append({"type": "latent_attention", "mixer": latent_config(o), "mlp": fc})
    return cfg, t
