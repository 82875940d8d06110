"""Plain, slow float64 restatement of the Zusuvik design, one function per mechanism, row by row.  Test infrastructure only: numpy,
no kernels, no code shared with the product path.

Notation: h [n, width] the rows of ONE sequence in order (row p is position p); weights as the checkpoint stores them ([out, in]); w maps
the names below '<layer>.mix.' / '<layer>.mlp.' to arrays."""
import math

import numpy as np


def f64(a):
    return np.asarray(a, np.float64)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-f64(z)))


def silu(z):
    return f64(z) * sigmoid(z)


def log_sigmoid(z):
    return -np.logaddexp(0.0, -f64(z))


def soft_cap(z, cap):
    return cap * np.tanh(f64(z) / cap) if cap else f64(z)


def unit_rms(x, eps):
    x = f64(x)
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def offset_norm(x, w, eps):
    """the stored weight is the deviation from one"""
    return unit_rms(x, eps) * (1.0 + f64(w))


# -- rotary positions -----------------------------------------------------------------------------------------------------
def frequencies(dims, base, scaling=None):
    """one frequency per rotated pair.  With scaling: a pair that turns more than `high` times over the original context keeps its
    frequency, one that turns fewer than `low` times is slowed down by the factor, a blend by the number of turns between."""
    f = float(base) ** (-2.0 * np.arange(dims // 2, dtype=np.float64) / dims)
    if not scaling:
        return f
    factor, low, high, original = (float(scaling[k]) for k in ("factor", "low", "high", "original"))
    out = f.copy()
    for i in range(len(f)):
        wavelength = 2.0 * math.pi / f[i]
        if wavelength < original / high:
            continue
        if wavelength > original / low:
            out[i] = f[i] / factor
        else:
            s = (original / wavelength - low) / (high - low)
            out[i] = (1.0 - s) * f[i] / factor + s * f[i]
    return out


def rotate(x, pos, rot, layout):
    """x [.., dim] of the token at position pos; layout 'pairs': dimension 2i turns with 2i + 1, 'halves': i with i + dims / 2; the
    dimensions from rot.dims on stay.  The angle is the 32-bit product of position and frequency."""
    out = f64(x).copy()
    dims = int((rot or {}).get("dims", 0))
    if not dims:
        return out
    f = frequencies(dims, float(rot["base"]), rot.get("scaling"))
    ang = (np.float32(pos) * f.astype(np.float32)).astype(np.float64)
    c, s = np.cos(ang), np.sin(ang)
    first, second = (slice(0, dims, 2), slice(1, dims, 2)) if layout == "pairs" else (slice(0, dims // 2), slice(dims // 2, dims))
    u, v = f64(x)[..., first], f64(x)[..., second]
    out[..., first] = u * c - v * s
    out[..., second] = v * c + u * s
    return out


# -- retention ------------------------------------------------------------------------------------------------------------
def retention_scan(q, k, v, decay):
    """q, k [n, H, D], v [n, H, V], decay [H] -> outputs [n, H, V]: S <- decay S + k v^T, o = S^T q"""
    n, H, D = q.shape
    S, out = np.zeros((H, D, v.shape[2])), np.zeros((n, H, v.shape[2]))
    for t in range(n):
        S = f64(decay)[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hdv,hd->hv", S, q[t])
    return out


def retention(h, w, m, eps):
    n = h.shape[0]
    H, D, V = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    h = f64(h)
    q, k = (h @ f64(w["q"]).T).reshape(n, H, D), (h @ f64(w["k"]).T).reshape(n, H, D)
    v = (h @ f64(w["v"]).T).reshape(n, H, V)
    q = np.stack([rotate(q[p], p, m.get("rot"), "halves") for p in range(n)])
    k = np.stack([rotate(k[p], p, m.get("rot"), "halves") for p in range(n)]) * D ** -0.5
    o = unit_rms(retention_scan(q, k, v, m["decay"]), eps).reshape(n, H * V)
    return (o * silu(h @ f64(w["g"]).T)) @ f64(w["o"]).T


# -- the two halves of a parallel mixer -----------------------------------------------------------------------------------
def causal_conv(u, taps_w):
    """u [n, channels], taps_w [channels, taps]: y_t = sum over the last `taps` rows, the newest with the last tap; zeros before row 0"""
    u, taps_w = f64(u), f64(taps_w)
    taps = taps_w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, u.shape[1])), u])
    return sum(padded[j: j + u.shape[0]] * taps_w[:, j] for j in range(taps))


def softmax_weights(scores):
    e = np.exp(scores - scores.max())
    return e / e.sum()


def attention_qkv(h, w, m, eps):
    """-> (q [n, H, D], k [n, G, D], v [n, G, V]) as the scores and the cache see them"""
    n = h.shape[0]
    H, G, D, V = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    h = f64(h)
    q, k, v = (causal_conv(h @ f64(w[x]).T + f64(w[x + ".b"]), w[x + ".conv"]) for x in ("q", "k", "v"))
    q = (unit_rms(q, eps) * f64(w["q.norm"])).reshape(n, H, D)
    k = (unit_rms(k, eps) * f64(w["k.norm"])).reshape(n, G, D)
    turn = lambda a: np.stack([rotate(a[p], p, m.get("rot"), "pairs") for p in range(n)])
    return turn(q), turn(k), v.reshape(n, G, V)


def conv_attention(h, w, m, eps):
    n = h.shape[0]
    H, G, V = int(m["heads"]), int(m["kv_heads"]), int(m["vdim"])
    q, k, v = attention_qkv(h, w, m, eps)
    out = np.zeros((n, H, V))
    for i in range(n):
        for hd in range(H):
            g = hd // (H // G)
            s = soft_cap(k[: i + 1, g] @ q[i, hd] * float(m["scale"]), m.get("softcap"))
            out[i, hd] = softmax_weights(s) @ v[: i + 1, g]
    return out.reshape(n, H * V) @ f64(w["o"]).T + f64(w["o.b"])


def matrix_memory_scan(q, k, v, log_in, log_forget):
    """q, k [n, H, D], v [n, H, V], log gates [n, H] -> [n, H, V].  The state is held divided by exp(m), m the running maximum of the
    accumulated log gates (0 at the start)."""
    n, H, D = q.shape
    S, N, m = np.zeros((H, D, v.shape[2])), np.zeros((H, D)), np.zeros(H)
    out = np.zeros((n, H, v.shape[2]))
    for t in range(n):
        new = np.maximum(log_forget[t] + m, log_in[t])
        keep, write = np.exp(log_forget[t] + m - new), np.exp(log_in[t] - new)
        S = keep[:, None, None] * S + write[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        N = keep[:, None] * N + write[:, None] * k[t]
        m = new
        den = np.maximum(np.abs(np.einsum("hd,hd->h", N, q[t])), np.exp(-m)) + 1e-6
        out[t] = np.einsum("hdv,hd->hv", S, q[t]) / den[:, None]
    return out


def matrix_memory(h, w, m, eps):
    n = h.shape[0]
    H, D, V, cap = int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["gate_cap"])
    h = f64(h)
    q, k = (h @ f64(w["q"]).T).reshape(n, H, D) * D ** -0.5, (h @ f64(w["k"]).T).reshape(n, H, D)
    v = (h @ f64(w["v"]).T).reshape(n, H, V)
    log_in = soft_cap(h @ f64(w["i"]).T + f64(w["i.b"]), cap)
    log_forget = log_sigmoid(soft_cap(h @ f64(w["f"]).T + f64(w["f.b"]), cap))
    o = unit_rms(matrix_memory_scan(q, k, v, log_in, log_forget), eps).reshape(n, H * V)
    return (o * f64(w["norm"]) * sigmoid(h @ f64(w["g"]).T)) @ f64(w["o"]).T


def parallel_mixer(h, w, m, eps):
    left = conv_attention(h, sub(w, "left."), m["left"], eps)
    right = matrix_memory(h, sub(w, "right."), m["right"], eps)
    return float(m["left_scale"]) * left + float(m["right_scale"]) * right


# -- feed-forward -----------------------------------------------------------------------------------------------------------
def clamped_unit(h, w, p, limit):
    g = np.minimum(f64(h) @ f64(w[p + "gate"]).T, limit)
    u = np.clip(f64(h) @ f64(w[p + "up"]).T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ f64(w[p + "down"]).T


def route(z, top):
    """z [n, E] logits -> (chosen [n, top], weights [n, top]: a softmax over the chosen logits)"""
    idx = np.argsort(-f64(z), axis=1, kind="stable")[:, :top]
    return idx, np.stack([softmax_weights(f64(z)[t, idx[t]]) for t in range(len(z))])


def moe_ff(h, w, fc, chosen=None):
    h = f64(h)
    idx, ws = route(h @ f64(w["router"]).T + f64(w["router.b"]), int(fc["router"]["top"]))
    if chosen is not None:
        chosen.extend(idx.tolist())
    out = np.zeros_like(h)
    for e in np.unique(idx):
        t, k = np.nonzero(idx == e)
        np.add.at(out, t, ws[t, k][:, None] * clamped_unit(h[t], w, f"e{e}.", float(fc["expert"]["limit"])))
    if fc.get("shared"):
        out = out + sigmoid(h @ f64(w["shared.sg"]).T) * clamped_unit(h, w, "shared.", float(fc["shared"]["limit"]))
    return out


# -- the model --------------------------------------------------------------------------------------------------------------
def sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def layer_order(cfg):
    """[(layer, a later pass of the loop starts here)]"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = int(loop["start"]), int(loop["stop"])
    order = [(i, False) for i in range(a)]
    for t in range(int(loop["times"])):
        order += [(i, t > 0 and i == a) for i in range(a, b)]
    return order + [(i, False) for i in range(b, n)]


def forward(cfg, tensors, tokens, streams=None):
    """tokens of ONE sequence from position 0 -> logits [n, vocab]; streams: a list that receives the residual stream after every layer run"""
    eps = float(cfg["norm"]["eps"])
    x0 = f64(tensors["embed"])[np.asarray(tokens)]
    x = x0
    for i, again in layer_order(cfg):
        if again:
            x = x + x0
        lc, w = cfg["layers"][i], sub(tensors, f"l{i}.")
        mixer = {"retention": retention, "parallel": parallel_mixer}[lc["type"]]
        y = mixer(offset_norm(x, w["norm1"], eps), sub(w, "mix."), lc["mixer"], eps)
        if lc.get("mlp") is not None:
            y = y + moe_ff(offset_norm(x, w["norm2"], eps), sub(w, "mlp."), lc["mlp"])
        x = x + y
        if streams is not None:
            streams.append(x.copy())
    return offset_norm(x, tensors["final.norm"], eps) @ f64(tensors["embed"]).T * float(cfg["logit_scale"])


# -- small random models (tests) --------------------------------------------------------------------------------------------
def bf16_values(a):
    """float32 array whose values are exactly representable in bfloat16 (round to nearest even)"""
    u = np.asarray(a, np.float32).view(np.uint32)
    u = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16) << 16
    return u.astype(np.uint32).view(np.float32)


TURNS = dict(factor=3.0, low=1.0, high=5.0, original=90)
RETENTION = dict(heads=3, dim=16, vdim=20, decay=None, rot_dims=12, base=900.0)
LEFT = dict(heads=6, kv_heads=2, dim=16, vdim=24, conv=4, rot_dims=8, base=500.0, scaling=TURNS, scale=None, softcap=7.0)
RIGHT = dict(heads=2, dim=12, vdim=28, gate_cap=9.0)
MOE = dict(experts=6, top=2, ff=20, limit=1.25, shared=30, shared_limit=2.0)


def _matrix(rng):
    return lambda *s, sd=None: bf16_values(rng.normal(0, sd if sd is not None else 1.0 / math.sqrt(s[-1]), s))


def rot_config(o):
    rot = {"base": o["base"], "dims": o["rot_dims"]}
    if o.get("scaling"):
        rot["scaling"] = dict(o["scaling"])
    return rot


def retention_parts(rng, width, over=None):
    """-> (mixer configuration, weights)"""
    o, r = dict(RETENTION, **(over or {})), _matrix(rng)
    H, D, V = o["heads"], o["dim"], o["vdim"]
    decay = o["decay"] or [1.0 - 2.0 ** (-2.0 - 1.5 * i) for i in range(H)]
    return ({"heads": H, "dim": D, "vdim": V, "decay": list(decay), "rot": rot_config(o)},
            {"q": r(H * D, width), "k": r(H * D, width), "v": r(H * V, width), "g": r(H * V, width), "o": r(width, H * V)})


def attention_parts(rng, width, over=None):
    o, r = dict(LEFT, **(over or {})), _matrix(rng)
    H, G, D, V = o["heads"], o["kv_heads"], o["dim"], o["vdim"]
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": V, "conv": o["conv"], "rot": rot_config(o), "scale": o["scale"] or D ** -0.5,
         "softcap": o["softcap"]}
    w = {"o": r(width, H * V), "o.b": r(width, sd=0.2)}
    for name, rows in (("q", H * D), ("k", G * D), ("v", G * V)):
        w[name], w[name + ".b"], w[name + ".conv"] = r(rows, width), r(rows, sd=0.2), r(rows, o["conv"], sd=0.6)
    w["q.norm"], w["k.norm"] = bf16_values(1.0 + 0.2 * rng.normal(size=H * D)), bf16_values(1.0 + 0.2 * rng.normal(size=G * D))
    return m, w


def memory_parts(rng, width, over=None):
    o, r = dict(RIGHT, **(over or {})), _matrix(rng)
    H, D, V = o["heads"], o["dim"], o["vdim"]
    w = {"q": r(H * D, width), "k": r(H * D, width), "v": r(H * V, width), "g": r(H * V, width), "o": r(width, H * V),
         "norm": bf16_values(1.0 + 0.2 * rng.normal(size=H * V)), "i": r(H, width), "f": r(H, width), "i.b": r(H, sd=1.0),
         "f.b": bf16_values(3.0 + rng.normal(size=H))}
    return {"heads": H, "dim": D, "vdim": V, "gate_cap": o["gate_cap"]}, w


def ff_parts(rng, width, over=None):
    o, r = dict(MOE, **(over or {})), _matrix(rng)
    fc = {"kind": "moe", "expert": {"ff": o["ff"], "limit": o["limit"]}, "router": {"experts": o["experts"], "top": o["top"]},
          "shared": {"ff": o["shared"], "limit": o["shared_limit"]} if o["shared"] else None}
    w = {"router": r(o["experts"], width, sd=2.0 / math.sqrt(width)), "router.b": r(o["experts"], sd=0.3)}
    for p, F in [(f"e{e}.", o["ff"]) for e in range(o["experts"])] + ([("shared.", o["shared"])] if o["shared"] else []):
        w[p + "gate"], w[p + "up"], w[p + "down"] = r(F, width), r(F, width), r(width, F)
    if o["shared"]:
        w["shared.sg"] = r(1, width)
    return fc, w


def random_zusuvik(rng, layers, width=72, vocab=97, eps=1e-5, logit_scale=0.6, loop=None):
    """A small random model -> (config, tensors as float32 arrays of bf16 values).  layers: a list of (type, overrides, ff overrides):
    overrides of RETENTION, or {"left": .., "right": .., "scales": (l, r)} of a parallel layer; ff overrides of MOE, or None for a layer
    without a feed-forward.  loop: (start, stop, times) or None."""
    bf = bf16_values
    cfg = {"architecture": "Zusuvik", "width": width, "vocab": vocab, "norm": {"eps": eps}, "logit_scale": logit_scale, "layers": []}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    t = {"embed": bf(rng.normal(size=(vocab, width))), "final.norm": bf(0.2 * rng.normal(size=width))}
    for i, (kind, over, ff) in enumerate(layers):
        p, over = f"l{i}.", over or {}
        t[p + "norm1"] = bf(0.2 * rng.normal(size=width))
        if kind == "retention":
            m, w = retention_parts(rng, width, over)
        else:
            lm, lw = attention_parts(rng, width, over.get("left"))
            rm, rw = memory_parts(rng, width, over.get("right"))
            ls, rs = over.get("scales", (0.7, 1.2))
            m = {"left": lm, "right": rm, "left_scale": ls, "right_scale": rs}
            w = {**{"left." + k: v for k, v in lw.items()}, **{"right." + k: v for k, v in rw.items()}}
        t.update({p + "mix." + k: v for k, v in w.items()})
        fc = None
        if ff is not None:
            t[p + "norm2"] = bf(0.2 * rng.normal(size=width))
            fc, w = ff_parts(rng, width, ff)
            t.update({p + "mlp." + k: v for k, v in w.items()})
        cfg["layers"].append({"type": kind, "mixer": m, "mlp": fc})
    return cfg, t
