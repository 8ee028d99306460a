"""A plain, slow statement of the Rivolix design in float64 numpy: one function per mechanism, whole sequences at once, no cache,
no batching.  It shares nothing with the served model; the tests compare the engine against it.

Notation: T tokens of one sequence at positions 0 .. T - 1 (or `pos`), D the model width, H query heads over G key / value heads.
"""
import math

import numpy as np


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm(x, w, eps):
    """The weight is stored around zero."""
    return rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def causal_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_(t - taps + 1 + j), zeros before the start."""
    T, C = u.shape
    taps = w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, C)), u])
    return sum(padded[j:j + T] * w[:, j] for j in range(taps))


def temperature(pos, coef, every):
    return 1.0 + coef * np.log(np.floor((np.asarray(pos, dtype=np.float64) + 1.0) / every) + 1.0)


def frequencies(rot):
    """-> (frequency per pair, magnitude of cos and sin)."""
    n, base = rot["dims"], rot["base"]
    f = np.array([base ** (-2.0 * i / n) for i in range(n // 2)])
    s = rot.get("scaling")
    if not s:
        return f, 1.0

    def dim_of(turns):
        return n * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(dim_of(s["fast"])), 0), min(math.ceil(dim_of(s["slow"])), n - 1)
    ramp = np.clip((np.arange(n // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / s["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(s["factor"]) + 1.0


def rotate(x, pos, rot):
    """x [T, heads, dim]: dimensions i and i + dims / 2 of each head turn by the position."""
    out = x.copy()
    f, mag = frequencies(rot)
    half = rot["dims"] // 2
    for i in range(half):
        a = np.asarray(pos, dtype=np.float64) * f[i]
        c, s = mag * np.cos(a)[:, None], mag * np.sin(a)[:, None]
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * c - v * s
        out[..., i + half] = v * c + u * s
    return out


def causal_softmax(s):
    """s [T, n] scores of queries that are the last T of n positions."""
    T, n = s.shape
    s = np.where(np.arange(n)[None, :] <= np.arange(n - T, n)[:, None], s, -np.inf)
    e = np.exp(s - s.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


def attention(q, k, v, scale):
    """q [T, H, d], k [n, G, d], v [n, G, dv] -> [T, H, dv]; the queries are the last T positions."""
    H, G = q.shape[1], k.shape[1]
    return np.stack([causal_softmax(q[:, h] @ k[:, h // (H // G)].T * scale) @ v[:, h // (H // G)] for h in range(H)], axis=1)


def lambda_of(lq1, lk1, lq2, lk2, diff):
    return math.exp(float(np.sum(lq1 * lk1))) - math.exp(float(np.sum(lq2 * lk2))) + diff


def differential(q, k, v, scale, lam, diff, eps):
    """q [T, H, 2, d], k [n, G, 2, d], v [n, G, dv] -> [T, H, dv]."""
    a1, a2 = (attention(q[:, :, m], k[:, :, m], v, scale) for m in (0, 1))
    return rms(a1 - lam * a2, eps) * (1.0 - diff)


def differential_kv(h, w, m):
    """The layer's own keys and values after their convolutions."""
    T = h.shape[0]
    G, d, dv = m["kv_heads"], m["dim"], m["vdim"]
    return (causal_conv(h @ w["k"].T, w["k_conv"]).reshape(T, G, 2, d), causal_conv(h @ w["v"].T, w["v_conv"]).reshape(T, G, dv))


def differential_mixer(h, w, m, eps, kv=None):
    """w: q, q_conv, lq1, lk1, lq2, lk2, g, o and, without kv (another layer's keys and values), k, v, k_conv, v_conv."""
    T = h.shape[0]
    H, d = m["heads"], m["dim"]
    k, v = kv if kv is not None else differential_kv(h, w, m)
    q = causal_conv(h @ w["q"].T, w["q_conv"]).reshape(T, H, 2, d)
    t = m.get("q_temp")
    if t:
        q = q * temperature(np.arange(T), t["coef"], t["every"])[:, None, None, None]
    o = differential(q, k, v, m["scale"], lambda_of(w["lq1"], w["lk1"], w["lq2"], w["lk2"], m["diff"]), m["diff"], eps)
    return (o.reshape(T, -1) * sigmoid(h @ w["g"].T)) @ w["o"].T


def tied_mixer(h, w, m, eps):
    """w: q, k, o.  Values are the projected keys; q and k are normed after their rotation."""
    T = h.shape[0]
    H, G, d, pos = m["heads"], m["kv_heads"], m["dim"], np.arange(h.shape[0])
    q, k = (h @ w["q"].T).reshape(T, H, d), (h @ w["k"].T).reshape(T, G, d)
    o = attention(rms(rotate(q, pos, m["rot"]), eps), rms(rotate(k, pos, m["rot"]), eps), k, m["scale"])
    return o.reshape(T, -1) @ w["o"].T


def unit(x, gate, up, down):
    return (silu(x @ gate.T) * (x @ up.T)) @ down.T


def route(h, router, top):
    """-> (indices [T, top], weights [T, top]): plain sigmoid scores, not divided by their sum."""
    s = sigmoid(h @ router.T)
    idx = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    return idx, np.take_along_axis(s, idx, axis=-1)


def experts(h, idx, wt, gate, up, down):
    """The weight scales the expert's INPUT."""
    y = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(idx[t], wt[t]):
            y[t] += unit(w * h[t], gate[e], up[e], down[e])
    return y


def feed_forward(h, W, p, mlp):
    E, top = mlp["router"]["experts"], mlp["router"]["top"]
    idx, wt = route(h, W[p + "router"], top)
    y = experts(h, idx, wt, *([W[f"{p}e{e}.{n}"] for e in range(E)] for n in ("gate", "up", "down")))
    if mlp.get("shared"):
        y = y + unit(h, *(W[f"{p}shared.{n}"] for n in ("gate", "up", "down")))
    return y


def mixer(kind, h, W, p, m, eps, kv=None):
    def take(names):
        return {n.replace(".", "_"): W[p + n] for n in names}

    if kind == "attention":
        names = ["q", "q.conv", "lq1", "lk1", "lq2", "lk2", "g", "o"]
        return differential_mixer(h, take(names + ([] if kv is not None else ["k", "v", "k.conv", "v.conv"])), m, eps, kv)
    assert kind == "attention_2"
    return tied_mixer(h, take(["q", "k", "o"]), m, eps)


def forward(cfg, W, tokens, taps=None):
    """-> logits [T, vocab]; the residual stream after every layer is appended to `taps`."""
    W = {k: np.asarray(v, dtype=np.float64) for k, v in W.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][np.asarray(tokens)]
    kvs = {}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        h, kv = norm(x, W[p + "norm1"], eps), None
        if L["type"] == "attention":
            if m.get("kv_from") is None:
                kvs[i] = differential_kv(h, {n.replace(".", "_"): W[f"{p}mix.{n}"] for n in ("k", "v", "k.conv", "v.conv")}, m)
            else:
                kv = kvs[m["kv_from"]]
        y = mixer(L["type"], h, W, p + "mix.", m, eps, kv) * W[p + "ls1"]
        if L.get("mlp"):
            y = y + feed_forward(norm(x, W[p + "norm2"], eps), W, p + "mlp.", L["mlp"]) * W[p + "ls2"]
        x = x + y
        if taps is not None:
            taps.append(x.copy())
    return norm(x, W["final.norm"], eps) @ W["embed"].T


def random_weights(cfg, seed=0):
    """Random weights of the config's shapes, rounded to bfloat16 (so that every storage type holds them exactly)."""
    import torch
    g = torch.Generator().manual_seed(seed)

    def rnd(*shape, s=1.0, mean=0.0):
        return (mean + s * torch.randn(shape, generator=g)).bfloat16().double().numpy()

    def mat(o, i, s=1.0):
        return rnd(o, i, s=s / math.sqrt(i))

    D, V = cfg["width"], cfg["vocab"]
    W = {"embed": rnd(V, D), "final.norm": rnd(D, s=0.2)}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        W[p + "norm1"], W[p + "ls1"] = rnd(D, s=0.2), rnd(D, s=0.3, mean=0.7)
        q = p + "mix."
        H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        if L["type"] == "attention":
            W.update({q + "q": mat(2 * H * d, D, 1.5), q + "q.conv": rnd(2 * H * d, m["conv"], s=0.5), q + "g": mat(H * dv, D), q + "o": mat(D, H * dv)})
            W.update({q + n: rnd(d, s=0.6 / d ** 0.25) for n in ("lq1", "lk1", "lq2", "lk2")})
            if m.get("kv_from") is None:
                W.update({q + "k": mat(2 * G * d, D, 1.5), q + "v": mat(G * dv, D), q + "k.conv": rnd(2 * G * d, m["conv"], s=0.5),
                          q + "v.conv": rnd(G * dv, m["conv"], s=0.5)})
        else:
            W.update({q + "q": mat(H * d, D), q + "k": mat(G * d, D), q + "o": mat(D, H * dv)})
        mlp = L.get("mlp")
        if mlp:
            W[p + "norm2"], W[p + "ls2"] = rnd(D, s=0.2), rnd(D, s=0.3, mean=0.7)
            q = p + "mlp."
            E, ff = mlp["router"]["experts"], mlp["expert"]["ff"]
            W[q + "router"] = mat(E, D)
            units = [(f"{q}e{e}.", ff) for e in range(E)] + ([(q + "shared.", mlp["shared"]["ff"])] if mlp.get("shared") else [])
            for name, n in units:
                W.update({name + "gate": mat(n, D, 1.5), name + "up": mat(n, D, 1.5), name + "down": mat(D, n)})
    return W
