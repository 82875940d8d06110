"""Vabanex: a decoder-only model of pre-norm layers (layer norms with weight and bias) whose only token mixer is attention through a
low-rank latent.

  embedding   x = embed[token] * embedding.scale
  layer i     x <- x + mixer(layer_norm(x; norm1)),  then  x <- x + ff(layer_norm(x; norm2))   (no second step where mlp is null)
              mixer 'latent_attention': causal attention through a low-rank latent; queries through a normed latent of their own; every
                    head's query is [dim plain | rot_dim rotated], the key is [W_uk c | one rotated part shared by the heads]; only the
                    normed latent c and the rotated key part are cached; rotary positions on neighbouring dimensions, optionally with
                    frequencies rescaled for longer contexts; one sigmoid gate per head
              ff:   dense: down of the clamped sigmoid-gated unit; or routed experts down(gelu(up h)): scores = sigmoid of the router's
                    logits, the choice by score + correction among the best groups (a group counts by its two largest choice scores),
                    weights = the chosen scores times a factor
  head        logits = cap * tanh(head . layer_norm(x; final.norm) / cap)
Sizes, the order of the layers and every constant come from config.json; tensor names are those of the checkpoint
('l<i>.norm1', 'l<i>.norm1.b', 'l<i>.mix.*', 'l<i>.mlp.*', 'l<i>.mlp.e<j>.*').
"""
import torch

from .. import mixers
from .. import seq_ops as so
from . import register


def _sub(tensors, prefix):
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def _norm(tensors, name):
    return tensors[name].contiguous(), tensors[name + ".b"].contiguous()


@register("Vabanex")
class Vabanex:
    engine = "sequence"

    def __init__(self, config, tensors, state, dtype):
        self.width, self.vocab = int(config["width"]), int(config["vocab"])
        self.eps = float(config["norm"]["eps"])
        self.embed_scale = float((config.get("embedding") or {}).get("scale", 1.0))
        self.softcap = float(config.get("logit_softcap") or 0.0)
        self.math = so.MATH_BF16 if dtype == torch.bfloat16 else so.MATH_F32
        self.act_dtype = torch.bfloat16 if self.math == so.MATH_BF16 else torch.float32     # what products read
        self.embed = tensors["embed"].contiguous()
        assert self.embed.shape == (self.vocab, self.width)
        self.final_norm, self.head = _norm(tensors, "final.norm"), tensors["head"].contiguous()
        self.layers = []
        for i, lc in enumerate(config["layers"]):
            w = _sub(tensors, f"l{i}.")
            if lc["type"] != "latent_attention":
                raise ValueError(f"layer {i}: unknown mixer type {lc['type']!r}")
            ff = self._feed_forward(i, lc.get("mlp"), _sub(w, "mlp."))
            self.layers.append((_norm(w, "norm1"), self._latent(i, lc["mixer"], _sub(w, "mix."), state, dtype),
                                _norm(w, "norm2") if ff is not None else None, ff))

    # -- the parts of a layer, each from its piece of the configuration ---------------------------------------------------------
    def _latent(self, i, m, mw, state, dtype):
        rot = m.get("rot") or {}
        if int(rot.get("dims", m.get("rot_dim", 0))) != int(m.get("rot_dim", 0)):
            raise ValueError(f"layer {i}: the rotated part is rot_dim wide")
        return mixers.LatentWindowAttention(f"l{i}.latent", int(m["heads"]), int(m["dim"]), int(m["vdim"]), int(m["kv_rank"]), int(m["q_rank"]), 0,
                                            float(m["scale"]), mw, state, dtype, rot_dim=int(m.get("rot_dim", 0)),
                                            rot_base=float(rot.get("base", 10000.0)), rot_layout="pairs", rot_scaling=rot.get("scaling"),
                                            head_gate=True)

    def _feed_forward(self, i, fc, fw):
        if fc is None:
            return None
        if fc["kind"] == "dense":
            assert fw["up"].shape == (int(fc["ff"]), self.width)
            return mixers.GatedMlp(fw["gate"], fw["up"], fw["down"], ("clamped", float(fc["limit"])))
        if fc["kind"] == "moe":
            r = fc["router"]
            n, g = int(r["experts"]), r.get("groups") or {}
            assert fw["e0.up"].shape == (int(fc["expert"]["ff"]), self.width)
            return mixers.ExpertMlp(fw["router"], None, None, [fw[f"e{e}.up"] for e in range(n)], [fw[f"e{e}.down"] for e in range(n)],
                                    int(r["top"]), unit="gelu_erf", scoring="sigmoid", correction=fw["correction"],
                                    groups=(int(g.get("count", 1)), int(g.get("keep", g.get("count", 1)))), group_score="top2", renorm=False,
                                    factor=float(r.get("scale", 1.0)))
        raise ValueError(f"layer {i}: unknown feed-forward kind {fc['kind']!r}")

    @classmethod
    def from_config(cls, config, tensors, state, dtype):
        return cls(config, tensors, state, dtype)

    def second_rows(self, prev, tokens):
        return None      # one embedding table

    def _residual(self, x, norm, y=None):
        """x += y (the rows of a sublayer, or the parts of a routed feed-forward's sum); the layer norm of the result for what comes next
        (None: no norm), one launch"""
        w, b = norm if norm is not None else (None, None)
        a, routed = (None, y) if isinstance(y, tuple) else (y, None)
        return so.residual_layernorm(x, w, a=a, routed=routed, eps=self.eps, x_out=x if y is not None else None, bias=b, out_dtype=self.act_dtype)

    def forward(self, ctx):
        """-> the residual stream after the last layer, [T, width] f32.  A sublayer's residual step and the next sublayer's input norm
        are one launch; bf16 products read a bf16 copy of the norm's output (the same bits at half the traffic)."""
        x = so.embed_rows(ctx.ids, self.embed, scale=self.embed_scale)
        split = (lambda h: (None, h)) if self.act_dtype == torch.bfloat16 else (lambda h: (h, None))
        h = self._residual(x, self.layers[0][0]) if self.layers else None
        for i, (_, mixer, norm2, ff) in enumerate(self.layers):
            nxt = self.layers[i + 1][0] if i + 1 < len(self.layers) else None
            mo = mixer(ctx, *split(h))
            if ff is not None:
                h = self._residual(x, norm2, mo)
                mo = ff(ctx, *split(h), **({"defer": True} if isinstance(ff, mixers.ExpertMlp) else {}))
            h = self._residual(x, nxt, mo)
            if ctx.taps is not None:
                ctx.taps[i] = x.clone()
        return x

    def logits(self, ctx, x, rows):
        """rows: int32 device tensor of the row indices whose logits are wanted -> f32 [len(rows), vocab]"""
        w, b = self.final_norm
        hn = so.residual_layernorm(x, w, eps=self.eps, row_idx=rows, bias=b, out_dtype=self.act_dtype)
        return so.linear(hn, self.head, act="softcap" if self.softcap else None, act_param=self.softcap, math=ctx.math)
