"""Sagupel: a decoder-only model whose norms come after the sums, x <- norm1(alpha x + mixer(h)), x <- norm2(alpha x + ff(x)) (RMS
norms, one gain per coordinate); the residual stream is float.

config.json: {architecture, width, vocab, norm: {eps}, postln_alpha, canon: {taps}, layers: [{type, mixer: {...}, mlp: {...} | null}]}.
* Embedding: rows of `embed`, normed by `embed.norm`; the output is `final.norm` and the same matrix `embed`.
* A mixer reads h = x + a causal convolution of x over time per channel (l<i>.canon1 [width, taps]); the last taps - 1 rows of x are
  state of the sequence in every layer.  The feed-forward reads x itself.
* Mixers: `retention` = qserve_amd.layers.recurrent.Retention; `attention` = qserve_amd.layers.softmax_attention.SinkWindowAttention
  with per-head norms, values tied to the keys and distance slopes; `parallel` = TalkingHeadsAttention (left) beside GatedDeltaRule with
  one decay per head (right), joined by ParallelMixer.
* Feed-forward: clamped gated units (qserve_amd.layers.moe.GatedFeedForward).
Tensor names: embed, embed.norm, final.norm, l<i>.norm1 / norm2 / canon1, l<i>.mix.{q, k, v, g, o} (retention), l<i>.mix.{q, k, q.norm,
k.norm, sink, o} (attention), l<i>.mix.left.{q, q.b, k, k.b, q.norm, k.norm, talk, temp, g, o, out} + l<i>.mix.right.{q, k, v, q.conv,
k.conv, v.conv, b, A_log, norm, a, dt_bias, g, o, out} (parallel), l<i>.mlp.{gate, up, down}.
"""
import torch

from ..layers.moe import GatedFeedForward
from ..layers.ops import linear
from ..layers.recurrent import GatedDeltaRule, ParallelMixer, Retention
from ..layers.rotary import RotaryTable
from ..layers.softmax_attention import SinkWindowAttention, TalkingHeadsAttention, distance_slopes
from ..serving.cache import StateSpec
from ..serving.registry import register_model


@register_model("Sagupel")
class Sagupel:
    def __init__(self, ops, width, vocab, eps, alpha, embed, embed_norm, final_norm, layers, taps, rotaries):
        self.ops, self.width, self.vocab, self.eps, self.alpha, self.taps = ops, width, vocab, eps, alpha, taps
        self.embed, self.embed_norm, self.final_norm, self.layers, self.rotaries = embed, embed_norm, final_norm, layers, rotaries
        # a layer's states: [the convolution's inputs, with more than one tap | the mixer's]
        self.cache_rows, self.state_specs, self.slices = [], [], []
        for L in layers:
            m = L["mixer"]
            p0, s0 = len(self.cache_rows), len(self.state_specs)
            self.cache_rows += m.cache_rows
            self.state_specs += ([StateSpec((taps - 1, width), copies=2)] if taps > 1 else []) + m.state_specs
            self.slices.append((p0, len(self.cache_rows), s0 + (taps > 1), len(self.state_specs)))

    def reserve_positions(self, n):
        for r in self.rotaries:
            r.reserve(n)

    def graph_signature(self):
        return tuple(r.table.data_ptr() for r in self.rotaries)

    @classmethod
    def from_config(cls, config, weights, ops, device, dtype, page=64):
        D, V, eps = int(config["width"]), int(config["vocab"]), float(config["norm"]["eps"])
        taps = int(config["canon"]["taps"])
        if taps < 1:
            raise ValueError(f"canon: {taps} taps")

        def w(name, *shape):
            if name not in weights:
                raise KeyError(f"checkpoint has no tensor {name!r}")
            if shape and tuple(weights[name].shape) != shape:
                raise ValueError(f"{name}: shape {tuple(weights[name].shape)}, expected {shape}")
            return weights[name].to(device=device, dtype=dtype).contiguous()

        tables = {}

        def table(rot):
            if not rot or not int(rot["dims"]):
                return None
            t = RotaryTable(int(rot["dims"]), float(rot["base"]), rot.get("scaling"), device)
            return tables.setdefault(t.key(), t)

        def kv(m):
            return int(m.get("kv_heads") or m["heads"])

        def tied(i, m):
            if int(m.get("vdim", m["dim"])) != int(m["dim"]):
                raise ValueError(f"layer {i}: values are the projected keys, but vdim {m['vdim']} is not dim {m['dim']}")

        layers = []
        for i, spec in enumerate(config["layers"]):
            kind, m, p = spec["type"], spec["mixer"], f"l{i}.mix."
            if kind == "retention":
                mixer = Retention(ops, heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), decay=m["decay"], rotary=table(m.get("rot")),
                                  eps=eps, weights={k: w(p + k) for k in ("q", "k", "v", "g", "o")})
            elif kind == "attention":
                tied(i, m)
                names = (("q", "q"), ("k", "k"), ("o", "o"), ("q_norm", "q.norm"), ("k_norm", "k.norm"), ("sink", "sink"))
                mixer = SinkWindowAttention(ops, heads=int(m["heads"]), kv_heads=kv(m), dim=int(m["dim"]), vdim=int(m["dim"]),
                                            scale=float(m["scale"]), eps=eps, window=int(m["mask"]["size"]), norm="head", tied_values=True,
                                            slopes=distance_slopes(int(m["heads"])), weights={k: w(p + n) for k, n in names}, page=page)
            elif kind == "parallel":
                a, b, q = m["left"], m["right"], p + "left."
                tied(i, a)
                names = (("q", "q"), ("q_b", "q.b"), ("k", "k"), ("k_b", "k.b"), ("q_norm", "q.norm"), ("k_norm", "k.norm"), ("temp", "temp"),
                         ("talk", "talk"), ("g", "g"), ("o", "o"))
                left = TalkingHeadsAttention(ops, heads=int(a["heads"]), kv_heads=kv(a), dim=int(a["dim"]), scale=float(a["scale"]),
                                             softcap=a.get("softcap"), rotary=table(a.get("rot")), eps=eps,
                                             weights={k: w(q + n) for k, n in names}, page=page)
                q = p + "right."
                wr = {k: w(q + k) for k in ("q", "k", "v", "b", "A_log", "norm", "a", "dt_bias", "g", "o")}
                wr.update(q_conv=w(q + "q.conv"), k_conv=w(q + "k.conv"), v_conv=w(q + "v.conv"))
                right = GatedDeltaRule(ops, heads=int(b["heads"]), kv_heads=kv(b), dim=int(b["dim"]), vdim=int(b["vdim"]), taps=int(b["conv"]),
                                       eps=eps, weights=wr, gate="silu")
                mixer = ParallelMixer(ops, left, right, w(p + "left.out", D), w(p + "right.out", D), eps)
            else:
                raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
            L = {"mixer": mixer, "norm1": w(f"l{i}.norm1", D), "conv": w(f"l{i}.canon1", D, taps).float().t().contiguous(), "ff": None}
            mlp, q = spec.get("mlp"), f"l{i}.mlp."
            if mlp:
                if mlp["kind"] != "dense":
                    raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
                ff = int(mlp["ff"])
                L["ff"] = GatedFeedForward(ops, gate=w(q + "gate", ff, D), up=w(q + "up", ff, D), down=w(q + "down", D, ff), act="clamped",
                                           limit=float(mlp["limit"]))
                L["norm2"] = w(f"l{i}.norm2", D)
            layers.append(L)
        return cls(ops, D, V, eps, float(config["postln_alpha"]), w("embed", V, D), w("embed.norm", D), w("final.norm", D), layers, taps,
                   list(tables.values()))

    def forward(self, batch, pools, states=(), tap=None):
        """-> the float residual stream [T, width] after the last layer; tap(i, x) is called after every layer (tests)."""
        ops, n = self.ops, len(self.layers)
        x = ops.embed_rms_norm(batch.tokens, self.embed, self.embed_norm, self.eps)

        def conv(i):                                          # the convolution in front of layer i and its state
            return self.layers[i]["conv"], (states[self.slices[i][2] - 1] if self.taps > 1 else None)

        # steps of one token per sequence: a norm's launch also makes the next mixer's input (no row needs another row's new x)
        single = all(cnt == 1 for _, _, cnt in batch.items)
        h = None
        for i, L in enumerate(self.layers):
            p0, p1, s0, s1 = self.slices[i]
            if h is None:
                h = ops.residual_conv(x, *conv(i), batch)
            y = L["mixer"](h, batch, pools[p0:p1], states[s0:s1])
            nxt = dict(then_conv=conv(i + 1), batch=batch) if single and i + 1 < n else dict(want_h=False)
            if L["ff"] is not None:
                h = ops.scaled_add_rms_norm(x, y, self.alpha, L["norm1"], self.eps)
                h = ops.scaled_add_rms_norm(x, L["ff"](h), self.alpha, L["norm2"], self.eps, **nxt)
            else:
                h = ops.scaled_add_rms_norm(x, y, self.alpha, L["norm1"], self.eps, **nxt)
            if tap is not None:
                tap(i, x)
        return x

    def logits(self, x, rows):
        return linear(self.ops.rms_norm_rows(x, rows, self.final_norm, self.eps), self.embed).float()
