"""A plain, slow statement of the Sagupel design in float64 numpy: one function per mechanism, whole sequences at once, no cache,
no batching.  It shares nothing with the served model; the tests compare the engine against it.

Notation: T tokens of one sequence at positions 0 .. T - 1 (or `pos`), D the model width, H query heads over G key / value heads.
"""
import math

import numpy as np


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def causal_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start."""
    T, C = u.shape
    taps = w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, C)), u])
    return sum(padded[j:j + T] * w[:, j] for j in range(taps))


def rotate_halves(x, pos, dims, base, factor=1.0):
    """x [T, heads, dim]: dimensions i and i + dims / 2 of each head turn by pos * base^(-2i / dims) / factor."""
    out = x.copy()
    half = dims // 2
    for i in range(half):
        a = np.asarray(pos, dtype=np.float64) * base ** (-2.0 * i / dims) / factor
        c, s = np.cos(a)[:, None], np.sin(a)[:, None]
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def slopes(H):
    return np.array([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)])


def capped_scores(q, k, scale, temp, cap):
    """q [T, H, d], k [T, G, d] -> [H, T, T]: cap tanh(q . k scale temp_h / cap) (cap None: not capped)."""
    T, H, _ = q.shape
    G = k.shape[1]
    s = np.stack([q[:, h] @ k[:, h // (H // G)].T * scale * temp[h] for h in range(H)])
    return s if cap is None else cap * np.tanh(s / cap)


def softmax_weights(s, visible, sink=None):
    """s [T, T], visible bool [T, T]; the denominator also holds exp(sink)."""
    z = np.where(visible, s, -np.inf)
    m = z.max(-1, keepdims=True)
    if sink is not None:
        m = np.maximum(m, sink)
    e = np.exp(z - m)
    den = e.sum(-1, keepdims=True) + (0.0 if sink is None else np.exp(sink - m))
    return e / den


def window_mask(T, size=None):
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) if size is None else (j <= i) & (i - j < size)


def slope_attention(q, k, v, scale, size, sink):
    """Distance bias -slope_h (i - j) after the scale, a window of `size` tokens, a sink per head.  -> [T, H, dv]."""
    T, H, _ = q.shape
    G = k.shape[1]
    dist = np.arange(T)[:, None] - np.arange(T)[None, :]
    s = capped_scores(q, k, scale, np.ones(H), None)
    out = []
    for h in range(H):
        w = softmax_weights(s[h] - slopes(H)[h] * dist, window_mask(T, size), sink[h])
        out.append(w @ v[:, h // (H // G)])
    return np.stack(out, axis=1)


def talking_attention(q, k, v, scale, temp, cap, talk):
    """Softmax per head over j <= i, the heads' weights mixed by talk [H, H], mixed weights on each head's own values."""
    T, H, _ = q.shape
    G = k.shape[1]
    s = capped_scores(q, k, scale, temp, cap)
    w = np.stack([softmax_weights(s[h], window_mask(T)) for h in range(H)])
    mixed = np.einsum("hg,gij->hij", talk, w)
    return np.stack([mixed[h] @ v[:, h // (H // G)] for h in range(H)], axis=1)


def attention_mixer(h, w, m, eps):
    """w: q, k, q_norm, k_norm, sink, o.  The values are the projected keys before their norm."""
    T = h.shape[0]
    H, G, d = m["heads"], m.get("kv_heads", m["heads"]), m["dim"]
    q, k = (h @ w["q"].T).reshape(T, H, d), (h @ w["k"].T).reshape(T, G, d)
    o = slope_attention(rms(q, eps) * w["q_norm"], rms(k, eps) * w["k_norm"], k, m["scale"], m["mask"]["size"], w["sink"])
    return o.reshape(T, -1) @ w["o"].T


def left_mixer(h, w, m, eps):
    """w: q, q_b, k, k_b, q_norm, k_norm, temp, talk, g, o."""
    T = h.shape[0]
    H, G, d, rot = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["rot"]
    q, k = (h @ w["q"].T + w["q_b"]).reshape(T, H, d), (h @ w["k"].T + w["k_b"]).reshape(T, G, d)
    factor = rot["scaling"]["factor"] if rot.get("scaling") else 1.0
    qr, kr = (rotate_halves(rms(u, eps) * w[n], np.arange(T), rot["dims"], rot["base"], factor) for u, n in ((q, "q_norm"), (k, "k_norm")))
    o = talking_attention(qr, kr, k, m["scale"], w["temp"], m["softcap"], w["talk"])
    return (o * sigmoid(h @ w["g"].T)[:, :, None]).reshape(T, -1) @ w["o"].T


def delta_rule(q, k, v, g, beta):
    """q, k [T, H, d], v [T, H, dv], g, beta [T, H] -> [T, H, dv]; the state starts at zero, o reads the updated state."""
    T, H, d = q.shape
    S, out = np.zeros((H, d, v.shape[2])), np.zeros_like(v)
    for t in range(T):
        for h in range(H):
            S[h] *= g[t, h]
            u = beta[t, h] * (v[t, h] - S[h].T @ k[t, h])
            S[h] += np.outer(k[t, h], u)
            out[t, h] = S[h].T @ q[t, h]
    return out


def right_mixer(h, w, m, eps):
    """w: q, k, v, q_conv, k_conv, v_conv, b, A_log, a, dt_bias, norm, g, o."""
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    G = m.get("kv_heads", H)
    q, k, v = (silu(causal_conv(h @ w[n].T, w[n + "_conv"])) for n in ("q", "k", "v"))
    q, k = q.reshape(T, G, d), k.reshape(T, G, d)
    q, k = (x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6) for x in (q, k))
    q, k = (np.repeat(x, H // G, axis=1) for x in (q * d ** -0.5, k))
    g = np.exp(-np.exp(w["A_log"]) * softplus(h @ w["a"].T + w["dt_bias"]))
    o = delta_rule(q, k, v.reshape(T, H, dv), g, sigmoid(h @ w["b"].T))
    return (rms(o, eps) * w["norm"] * silu(h @ w["g"].T).reshape(T, H, dv)).reshape(T, -1) @ w["o"].T


def retention(q, k, v, decay):
    """S <- decay_h S + k v^T, o = S^T q; no denominator."""
    T, H, d = q.shape
    S, out = np.zeros((H, d, v.shape[2])), np.zeros_like(v)
    for t in range(T):
        for h in range(H):
            S[h] = decay[h] * S[h] + np.outer(k[t, h], v[t, h])
            out[t, h] = S[h].T @ q[t, h]
    return out


def retention_mixer(h, w, m, eps):
    """w: q, k, v, g, o."""
    T = h.shape[0]
    H, d, dv, rot = m["heads"], m["dim"], m["vdim"], m["rot"]
    q, k = (rotate_halves((h @ w[n].T).reshape(T, H, d), np.arange(T), rot["dims"], rot["base"]) for n in ("q", "k"))
    o = retention(q, k * d ** -0.5, (h @ w["v"].T).reshape(T, H, dv), m["decay"])
    return (rms(o, eps).reshape(T, -1) * silu(h @ w["g"].T)) @ w["o"].T


def clamped_ff(h, gate, up, down, limit):
    g, u = np.minimum(h @ gate.T, limit), np.clip(h @ up.T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ down.T


LEFT = {"q": "q", "q_b": "q.b", "k": "k", "k_b": "k.b", "q_norm": "q.norm", "k_norm": "k.norm", "temp": "temp", "talk": "talk", "g": "g", "o": "o"}
RIGHT = {"q": "q", "k": "k", "v": "v", "q_conv": "q.conv", "k_conv": "k.conv", "v_conv": "v.conv", "b": "b", "A_log": "A_log", "a": "a",
         "dt_bias": "dt_bias", "norm": "norm", "g": "g", "o": "o"}
ATT = {"q": "q", "k": "k", "q_norm": "q.norm", "k_norm": "k.norm", "sink": "sink", "o": "o"}
RET = {n: n for n in ("q", "k", "v", "g", "o")}


def pick(W, prefix, names):
    return {k: W[prefix + n] for k, n in names.items()}


def mixer(kind, h, W, p, m, eps):
    """The mixer whose tensors start with p."""
    if kind == "attention":
        return attention_mixer(h, pick(W, p, ATT), m, eps)
    if kind == "retention":
        return retention_mixer(h, pick(W, p, RET), m, eps)
    left, right = left_mixer(h, pick(W, p + "left.", LEFT), m["left"], eps), right_mixer(h, pick(W, p + "right.", RIGHT), m["right"], eps)
    return 0.5 * (rms(left, eps) * W[p + "left.out"] + rms(right, eps) * W[p + "right.out"])


def forward(config, W, tokens, taps=None):
    """W: name -> float64 array (the checkpoint's names).  -> logits [T, vocab]; taps (a list) receives the stream after each layer."""
    eps, alpha = config["norm"]["eps"], config["postln_alpha"]
    x = rms(W["embed"][np.asarray(tokens)], eps) * W["embed.norm"]
    for i, L in enumerate(config["layers"]):
        p = f"l{i}."
        h = x + causal_conv(x, W[p + "canon1"])
        x = rms(alpha * x + mixer(L["type"], h, W, p + "mix.", L["mixer"], eps), eps) * W[p + "norm1"]
        mlp = L.get("mlp")
        if mlp:
            y = clamped_ff(x, W[p + "mlp.gate"], W[p + "mlp.up"], W[p + "mlp.down"], mlp["limit"])
            x = rms(alpha * x + y, eps) * W[p + "norm2"]
        if taps is not None:
            taps.append(x.copy())
    return (rms(x, eps) * W["final.norm"]) @ W["embed"].T


def tensor_shapes(config):
    """name -> shape of every tensor a checkpoint of this config holds."""
    D, V = config["width"], config["vocab"]
    out = {"embed": (V, D), "embed.norm": (D,), "final.norm": (D,)}
    for i, L in enumerate(config["layers"]):
        p, m = f"l{i}.", L["mixer"]
        out[p + "norm1"], out[p + "canon1"] = (D,), (D, config["canon"]["taps"])
        if L["type"] == "attention":
            H, G, d, dv, q = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"], p + "mix."
            out.update({q + "q": (H * d, D), q + "k": (G * d, D), q + "q.norm": (d,), q + "k.norm": (d,), q + "sink": (H,), q + "o": (D, H * dv)})
        elif L["type"] == "retention":
            H, d, dv, q = m["heads"], m["dim"], m["vdim"], p + "mix."
            out.update({q + "q": (H * d, D), q + "k": (H * d, D), q + "v": (H * dv, D), q + "g": (H * dv, D), q + "o": (D, H * dv)})
        else:
            a, b, q = m["left"], m["right"], p + "mix.left."
            H, G, d, dv = a["heads"], a.get("kv_heads", a["heads"]), a["dim"], a["vdim"]
            out.update({q + "q": (H * d, D), q + "q.b": (H * d,), q + "k": (G * d, D), q + "k.b": (G * d,), q + "q.norm": (d,), q + "k.norm": (d,),
                        q + "talk": (H, H), q + "temp": (H,), q + "g": (H, D), q + "o": (D, H * dv), q + "out": (D,)})
            H, d, dv, q = b["heads"], b["dim"], b["vdim"], p + "mix.right."
            G, taps = b.get("kv_heads", H), b["conv"]
            out.update({q + "q": (G * d, D), q + "q.conv": (G * d, taps), q + "k": (G * d, D), q + "k.conv": (G * d, taps), q + "v": (H * dv, D),
                        q + "v.conv": (H * dv, taps), q + "b": (H, D), q + "A_log": (H,), q + "norm": (dv,), q + "a": (H, D), q + "dt_bias": (H,),
                        q + "g": (H * dv, D), q + "o": (D, H * dv), q + "out": (D,)})
        if L.get("mlp"):
            ff = L["mlp"]["ff"]
            out.update({p + "norm2": (D,), p + "mlp.gate": (ff, D), p + "mlp.up": (ff, D), p + "mlp.down": (D, ff)})
    return out


def random_weights(config, seed=0):
    """Random tensors (numpy float64, every value a bfloat16 number) with scales that keep every mechanism awake."""
    import torch
    g = torch.Generator().manual_seed(seed)
    W = {}
    for name, shape in tensor_shapes(config).items():
        last = name.rsplit(".", 1)[-1]
        t = torch.randn(shape, generator=g)
        if last in ("norm", "norm1", "norm2", "out", "temp"):
            t = 1.0 + 0.3 * t
        elif last in ("sink", "embed"):
            pass
        elif last in ("b", "A_log", "dt_bias") and len(shape) == 1:
            t = 0.5 * t
        elif last == "talk":
            t = torch.eye(shape[0]) + 0.5 * t
        elif last in ("conv", "canon1"):
            t = t / math.sqrt(shape[1])
        else:
            t = t / math.sqrt(shape[-1])
        W[name] = t.bfloat16().double().numpy()
    return W
