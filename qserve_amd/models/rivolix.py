"""Rivolix: a decoder-only model of parallel layers with a norm and a scale of its own for each side, x <- x + (ls1 * mixer(norm1(x)) + ls2 *
ff(norm2(x))); norm(x) = x / rms(x) * (1 + w) (weights stored around zero), ls1 and ls2 one factor per coordinate; the residual stream
is float.

config.json: {architecture, width, vocab, norm: {eps}, layers: [{type, mixer: {...}, mlp: {...} | null}]}.
* Mixers: `attention` = qserve_amd.layers.softmax_attention.DifferentialAttention (two softmax maps over the same values, short convolutions on
  q, k and v, a query temperature that grows with the position, an output gate); with `kv_from: j` the layer has queries only and reads layer
  j's cache.  `attention_2` = TiedRotaryAttention (values are the projected keys, rotation with YaRN scaling, norms behind the rotation).
* Feed-forward: qserve_amd.layers.moe.SigmoidMoE with the router's weight on the expert's input, and a shared expert.
* Output: `final.norm`, then the embedding matrix.
Tensor names: embed, final.norm, l<i>.norm1 / ls1 / norm2 / ls2, l<i>.mix.{q, k, v, q.conv, k.conv, v.conv, lq1, lk1, lq2, lk2, g, o} (attention; no k,
v and their convolutions with kv_from) or l<i>.mix.{q, k, o} (attention_2), l<i>.mlp.{router, e<k>.{gate, up, down}, shared.{gate, up, down}}.
"""
from ..layers.moe import GatedFeedForward, SigmoidMoE
from ..layers.ops import linear
from ..layers.rotary import RotaryTable
from ..layers.softmax_attention import DifferentialAttention, TiedRotaryAttention
from ..serving.registry import register_model


@register_model("Rivolix")
class Rivolix:
    def __init__(self, ops, width, vocab, eps, embed, final_gain, layers, rotaries):
        self.ops, self.width, self.vocab, self.eps = ops, width, vocab, eps
        self.embed, self.final_gain, self.layers, self.rotaries = embed, final_gain, layers, rotaries
        self.cache_rows, self.state_specs, self.slices = [], [], []
        for L in layers:
            m = L["mixer"]
            p0, s0 = len(self.cache_rows), len(self.state_specs)
            self.cache_rows += m.cache_rows
            self.state_specs += m.state_specs
            self.slices.append((p0, len(self.cache_rows), s0, len(self.state_specs)))
        for i, L in enumerate(layers):                        # a layer without keys and values of its own reads its source's pools
            if L["kv_from"] is not None:
                self.slices[i] = self.slices[L["kv_from"]][:2] + self.slices[i][2:]

    def reserve_positions(self, n):
        for r in self.rotaries:
            r.reserve(n)

    def graph_signature(self):
        return tuple(r.table.data_ptr() for r in self.rotaries)

    @classmethod
    def from_config(cls, config, weights, ops, device, dtype, page=64):
        D, V, eps = int(config["width"]), int(config["vocab"]), float(config["norm"]["eps"])

        def w(name, *shape):
            if name not in weights:
                raise KeyError(f"checkpoint has no tensor {name!r}")
            if shape and tuple(weights[name].shape) != shape:
                raise ValueError(f"{name}: shape {tuple(weights[name].shape)}, expected {shape}")
            return weights[name].to(device=device, dtype=dtype).contiguous()

        def gain(name):
            return 1.0 + w(name, D).float()                    # (float: 1 + w does not fit the storage type)

        tables = {}

        def table(rot):
            if not rot or not int(rot["dims"]):
                return None
            t = RotaryTable(int(rot["dims"]), float(rot["base"]), rot.get("scaling"), device)
            return tables.setdefault(t.key(), t)

        def unit(prefix, ff):
            return GatedFeedForward(ops, gate=w(prefix + "gate", ff, D), up=w(prefix + "up", ff, D), down=w(prefix + "down", D, ff), act="silu")

        layers = []
        for i, spec in enumerate(config["layers"]):
            kind, m, p = spec["type"], spec["mixer"], f"l{i}.mix."
            heads, dim, vdim = int(m["heads"]), int(m["dim"]), int(m.get("vdim") or m["dim"])
            kv_heads, src = int(m.get("kv_heads") or heads), None
            if kind == "attention":
                names = ["q", "g", "o", "lq1", "lk1", "lq2", "lk2"]
                wm = {k: w(p + k) for k in names}
                wm["q_conv"] = w(p + "q.conv")
                if m.get("kv_from") is not None:
                    src = int(m["kv_from"])
                    if not 0 <= src < i or layers[src]["kv_from"] is not None or config["layers"][src]["type"] != kind:
                        raise ValueError(f"layer {i}: keys and values from layer {src}, which has none of this kind before this layer")
                    other = layers[src]["mixer"]
                    if (other.G, other.dim, other.vdim) != (kv_heads, dim, vdim):
                        raise ValueError(f"layer {i}: layer {src}'s keys and values have other sizes")
                else:
                    wm.update(k=w(p + "k"), v=w(p + "v"), k_conv=w(p + "k.conv"), v_conv=w(p + "v.conv"))
                t = m.get("q_temp")
                mixer = DifferentialAttention(ops, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=float(m["scale"]), taps=int(m["conv"]),
                                              diff=float(m["diff"]), eps=eps, weights=wm, shared_kv=src is not None, page=page,
                                              temperature=(float(t["coef"]), float(t["every"])) if t else None)
            elif kind == "attention_2":
                if vdim != dim:
                    raise ValueError(f"layer {i}: values are the projected keys, but vdim {vdim} is not dim {dim}")
                mixer = TiedRotaryAttention(ops, heads=heads, kv_heads=kv_heads, dim=dim, scale=float(m["scale"]), rotary=table(m.get("rot")), eps=eps,
                                            weights={k: w(p + k) for k in ("q", "k", "o")}, page=page)
            else:
                raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
            L = {"mixer": mixer, "kv_from": src, "norm1": gain(f"l{i}.norm1"), "ls1": w(f"l{i}.ls1", D), "ff": None}
            mlp, q = spec.get("mlp"), f"l{i}.mlp."
            if mlp:
                if mlp["kind"] != "moe":
                    raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
                E, ff, shared = int(mlp["router"]["experts"]), int(mlp["expert"]["ff"]), mlp.get("shared")
                L["ff"] = SigmoidMoE(ops, router=w(q + "router", E, D), gate=[w(f"{q}e{e}.gate", ff, D) for e in range(E)],
                                     up=[w(f"{q}e{e}.up", ff, D) for e in range(E)], down=[w(f"{q}e{e}.down", D, ff) for e in range(E)],
                                     top_k=int(mlp["router"]["top"]), weigh="input", shared=unit(q + "shared.", int(shared["ff"])) if shared else None)
                L["norm2"], L["ls2"] = gain(f"l{i}.norm2"), w(f"l{i}.ls2", D)
            layers.append(L)
        return cls(ops, D, V, eps, w("embed", V, D), gain("final.norm"), layers, list(tables.values()))

    def forward(self, batch, pools, states=(), tap=None):
        """-> the float residual stream [T, width] after the last layer; tap(i, x) is called after every layer (tests)."""
        ops, n = self.ops, len(self.layers)

        def gains(i):                                          # the norms in front of layer i
            if i >= n:
                return []
            L = self.layers[i]
            return [L["norm1"]] + ([L["norm2"]] if L["ff"] is not None else [])

        x, hs = ops.scaled_sum_rms_norms(None, [], gains(0), self.eps, tokens=batch.tokens, table=self.embed)
        for i, L in enumerate(self.layers):
            p0, p1, s0, s1 = self.slices[i]
            parts = [(L["mixer"](hs[0], batch, pools[p0:p1], states[s0:s1]), L["ls1"])]
            if L["ff"] is not None:
                parts += [(y, L["ls2"]) for y in L["ff"](hs[1])]
            # the next layer's two inputs come out of the pass that adds this layer's outputs to the stream
            _, hs = ops.scaled_sum_rms_norms(x, parts, gains(i + 1), self.eps)
            if tap is not None:
                tap(i, x)
        return x

    def logits(self, x, rows):
        return linear(self.ops.rms_norm_rows(x, rows, self.final_gain, self.eps), self.embed).float()
