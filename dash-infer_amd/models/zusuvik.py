"""Zusuvik: a decoder-only model whose layers run their token mixer and their routed feed-forward side by side, each behind a norm of its
own, with a looped block of layers.

  embedding   x0 = embed[token]
  layer i     x <- x + (mixer(norm1(x)) + ff(norm2(x)));  norm(v) = v / rms(v) * (1 + w): the stored weight is the deviation from one
              mixer 'retention': linear attention with a constant decay per head, rotary positions on the two halves of the rotated part,
                    unit-RMS norm per head, silu output gate
              mixer 'parallel': two mixers on the same input, added with a constant each --
                    left:  grouped-query attention with biases, a short causal convolution on every channel of q, k and v, norms over the
                           whole query / key row, rotary positions on neighbouring dimensions (frequencies rescaled for longer
                           contexts), capped scores
                    right: a matrix memory (mLSTM): exponential input and forget gates held in range by a running maximum, a key sum that
                           divides the output, unit-RMS norm per head, sigmoid output gate
              ff:   top-k routed clamped sigmoid-gated units, weights = softmax over the chosen logits; a shared unit behind a sigmoid gate
                    per token
  loop        layers start .. stop - 1 run `times` times in a row with the same weights and caches / states of their own per pass; every
              pass but the first starts with x <- x + x0
  head        logits = embed . norm(x; final.norm) * logit_scale
Sizes, layer order and constants come from config.json; tensor names are those of the checkpoint ('l<i>.mix.*', 'l<i>.mix.left.*',
'l<i>.mix.right.*', 'l<i>.mlp.*').
"""
import torch

from .. import mixers
from .. import seq_ops as so
from . import layer_runs, register


def _sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


class _Layer:
    __slots__ = ("norm1", "norm2", "mixer", "bias", "ff")


@register("Zusuvik")
class Zusuvik:
    engine = "sequence"

    def __init__(self, config, tensors, state, dtype):
        self.width, self.vocab = int(config["width"]), int(config["vocab"])
        self.eps = float(config["norm"]["eps"])
        self.logit_scale = float(config.get("logit_scale", 1.0))
        self.math = so.MATH_BF16 if dtype == torch.bfloat16 else so.MATH_F32
        self.act_dtype = torch.bfloat16 if self.math == so.MATH_BF16 else torch.float32     # what products read
        self.embed, self.final_norm = tensors["embed"].contiguous(), tensors["final.norm"].contiguous()
        assert self.embed.shape == (self.vocab, self.width)
        n = len(config["layers"])
        self.runs = layer_runs(n, config.get("loop") or None)
        times = [sum(1 for r in self.runs if r[0] == i) for i in range(n)]
        self.layers = []
        for i, lc in enumerate(config["layers"]):
            w, m, kind = _sub(tensors, f"l{i}."), lc["mixer"], lc["type"]
            L = _Layer()
            L.norm1, L.bias = w["norm1"].contiguous(), None
            if kind == "retention":
                L.mixer = self._retention(i, m, _sub(w, "mix."), state, times[i])
            elif kind == "parallel":
                L.mixer = mixers.WeightedPair(self._attention(i, m["left"], _sub(w, "mix.left."), state, dtype, times[i], float(m["left_scale"])),
                                              self._memory(i, m["right"], _sub(w, "mix.right."), state, times[i], float(m["right_scale"])))
                L.bias = L.mixer.bias
            else:
                raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
            L.ff = self._feed_forward(i, lc.get("mlp"), _sub(w, "mlp."))
            L.norm2 = w["norm2"].contiguous() if L.ff is not None else None
            self.layers.append(L)

    # -- the parts of a layer, each from its piece of the configuration ---------------------------------------------------------
    def _retention(self, i, m, mw, state, runs):
        rot = m.get("rot") or {}
        return mixers.Retention(f"l{i}.retention", int(m["heads"]), int(m["dim"]), int(m["vdim"]), m["decay"], mw, state, rot_dims=int(rot.get("dims", 0)),
                                rot_base=float(rot.get("base", 10000.0)), rot_layout="halves", rot_scaling=rot.get("scaling"), runs=runs)

    def _attention(self, i, m, lw, state, dtype, runs, out_scale):
        rot = m.get("rot") or {}
        return mixers.GroupedQueryAttention(f"l{i}.attn", int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), float(m["scale"]), lw,
                                            state, dtype, rot_dims=int(rot.get("dims", 0)), rot_base=float(rot.get("base", 10000.0)),
                                            rot_layout="pairs", rot_scaling=rot.get("scaling"), qk_norm="row", softcap=m.get("softcap"),
                                            conv=int(m["conv"]), runs=runs, out_scale=out_scale)

    def _memory(self, i, m, rw, state, runs, out_scale):
        return mixers.MatrixMemory(f"l{i}.memory", int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["gate_cap"]), rw, state, runs=runs,
                                   out_scale=out_scale)

    def _feed_forward(self, i, fc, fw):
        if fc is None:
            return None
        if fc.get("kind", "moe") != "moe":
            raise ValueError(f"layer {i}: unknown feed-forward kind {fc['kind']!r}")
        n, shared, gate = int(fc["router"]["experts"]), None, None
        if fc.get("shared") is not None:
            shared = mixers.GatedMlp(fw["shared.gate"], fw["shared.up"], fw["shared.down"], ("clamped", float(fc["shared"]["limit"])))
            gate = fw["shared.sg"]
            assert fw["shared.gate"].shape == (int(fc["shared"]["ff"]), self.width)
        assert fw["e0.gate"].shape == (int(fc["expert"]["ff"]), self.width)
        return mixers.ExpertMlp(fw["router"], fw.get("router.b"), [fw[f"e{e}.gate"] for e in range(n)], [fw[f"e{e}.up"] for e in range(n)],
                                [fw[f"e{e}.down"] for e in range(n)], int(fc["router"]["top"]), float(fc["expert"]["limit"]), shared=shared,
                                shared_gate=gate)

    @classmethod
    def from_config(cls, config, tensors, state, dtype):
        return cls(config, tensors, state, dtype)

    def second_rows(self, prev, tokens):
        return None      # one embedding table

    def forward(self, ctx):
        """-> the residual stream after the last layer, [T, width] f32.  The residual step of a layer (the mixer's rows, the routed rows'
        weighted sum, the shared expert's rows, x0 where a later pass starts) and both input norms of the next one are one launch."""
        x0 = so.embed_rows(ctx.ids, self.embed)
        x = torch.empty_like(x0)
        split = (lambda h: (None, h)) if self.act_dtype == torch.bfloat16 else (lambda h: (h, None))

        def enter(r):       # what the residual step before run r also does: its norms, and x0 at the start of a later pass
            if r >= len(self.runs):
                return {}
            L, first = self.layers[self.runs[r][0]], self.runs[r][2]
            return dict(w1=L.norm1, w2=L.norm2, again=x0 if first else None)

        src = x0            # the first residual step reads x0 and leaves it as it is
        h1, h2 = so.residual_rmsnorm(src, eps=self.eps, out_dtype=self.act_dtype, **enter(0))
        for r, (li, run, _) in enumerate(self.runs):
            L = self.layers[li]
            mo = L.mixer.rows(ctx, *split(h1), run=run) if isinstance(L.mixer, mixers.WeightedPair) else L.mixer(ctx, *split(h1), run=run)
            routed = add = None
            if L.ff is not None:
                routed, add = L.ff.parts(ctx, *split(h2))
            step = dict(a=mo, b=add, bias=L.bias, routed=routed)
            if ctx.taps is not None:      # the stream between a layer's sum and what the next pass adds
                so.residual_rmsnorm(src, x_out=x, **step)
                ctx.taps[r], src, step = x.clone(), x, {}
            h1, h2 = so.residual_rmsnorm(src, eps=self.eps, x_out=x, out_dtype=self.act_dtype, **step, **enter(r + 1))
            src = x
        return src

    def logits(self, ctx, x, rows):
        """rows: int32 device tensor of the row indices whose logits are wanted -> f32 [len(rows), vocab]"""
        hn, _ = so.residual_rmsnorm(x, self.final_norm, scale=self.logit_scale, eps=self.eps, row_idx=rows, out_dtype=self.act_dtype)
        return so.linear(hn, self.embed, math=ctx.math)
