"""Plain implementation of the Netanex design in numpy float64: one function per mechanism, whole sequences only (no
cache), written from the design's equations and sharing no code with the package.  `weights` maps checkpoint names to
arrays; `cfg` is the config.json dictionary."""
import math

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def unit_rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm(x, w, eps):
    """RMS norm whose stored weight is the distance from one."""
    return unit_rms(x, eps) * (1.0 + w)


def visible(i, j, size):
    return j <= i and (size <= 0 or i - j < size)


def weights_over(scores, extra):
    """Softmax of the visible scores whose denominator also holds exp(extra) (None: nothing)."""
    top = scores.max() if extra is None else max(scores.max(), extra)
    e = np.exp(scores - top)
    return e / (e.sum() + (0.0 if extra is None else math.exp(extra - top)))


def query_factor(position, coef, every):
    return 1.0 + coef * math.log((position + 1) // every + 1)


def two_map_lambda(W, p, diff):
    dot = lambda a, b: float(np.dot(W[p + a].astype(np.float64), W[p + b].astype(np.float64)))
    return math.exp(dot("lq1", "lk1")) - math.exp(dot("lq2", "lk2")) + diff


def differential_attention(W, p, m, h, eps):
    """Two attention maps per head over the same values, the second one subtracted; queries and keys normed per head and
    map; queries that grow with the position; no rotation."""
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ W[p + "q"].T + W[p + "q.b"]).reshape(T, H, 2, d)
    k = (h @ W[p + "k"].T + W[p + "k.b"]).reshape(T, G, 2, d)
    v = (h @ W[p + "v"].T + W[p + "v.b"]).reshape(T, G, dv)
    q, k = unit_rms(q, eps) * W[p + "q.norm"], unit_rms(k, eps) * W[p + "k.norm"]
    temp = m.get("q_temp")
    if temp:
        q = q * np.array([query_factor(i, temp["coef"], temp["every"]) for i in range(T)])[:, None, None, None]
    lam = two_map_lambda(W, p, m["diff"])
    out = np.zeros((T, H, dv))
    for i in range(T):
        for hd in range(H):
            c = hd // (H // G)
            a = [weights_over((k[:i + 1, c, x] @ q[i, hd, x]) * m["scale"], None) @ v[:i + 1, c] for x in (0, 1)]
            out[i, hd] = unit_rms(a[0] - lam * a[1], eps) * (1.0 - m["diff"])
    return out.reshape(T, H * dv) @ W[p + "o"].T + W[p + "o.b"]


def turning(rot):
    """(frequencies, factor on cosine and sine) of a rotation, with YaRN's scaling where it has one."""
    n, base, s = rot["dims"], rot["base"], rot.get("scaling")
    f = np.array([base ** (-2.0 * i / n) for i in range(n // 2)])
    if not s:
        return f, 1.0
    place = lambda turns: n * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(place(s["fast"])), 0), min(math.ceil(place(s["slow"])), n - 1)
    ramp = np.array([min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0) for i in range(n // 2)])
    return f / s["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(s["factor"]) + 1.0


def turn(x, rot):
    """x [T, ..., lanes], row t at position t."""
    f, factor = turning(rot)
    half, out = rot["dims"] // 2, x.copy()
    for t in range(x.shape[0]):
        c, s = np.cos(t * f) * factor, np.sin(t * f) * factor
        u, v = x[t, ..., :half], x[t, ..., half:2 * half]
        out[t, ..., :half], out[t, ..., half:2 * half] = u * c - v * s, v * c + u * s
    return out


def latent_attention(W, p, m, h, eps):
    """Keys and values expanded from one normed latent per token beside one turned key part for all heads; a window, a
    sink per head, an output gate."""
    T = h.shape[0]
    H, dn, dr, dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (h @ W[p + "q"].T).reshape(T, H, dn + dr)
    qn, qr = q[:, :, :dn], turn(q[:, :, dn:], m["rot"])
    down = h @ W[p + "dkv"].T
    c, kr = unit_rms(down[:, :R], eps) * W[p + "dkv.norm"], turn(down[:, R:], m["rot"])
    kn, v = (c @ W[p + "uk"].T).reshape(T, H, dn), (c @ W[p + "uv"].T).reshape(T, H, dv)
    size = (m.get("mask") or {}).get("size", 0)
    out = np.zeros((T, H, dv))
    for i in range(T):
        see = [j for j in range(i + 1) if visible(i, j, size)]
        for hd in range(H):
            s = (kn[see, hd] @ qn[i, hd] + kr[see] @ qr[i, hd]) * m["scale"]
            out[i, hd] = weights_over(s, float(W[p + "sink"][hd])) @ v[see, hd]
    return (out.reshape(T, H * dv) * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def gated_attention(W, p, m, h, eps):
    """Grouped queries, queries and keys normed over their whole rows, a denominator with one added, a gate per head."""
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (unit_rms(h @ W[p + "q"].T + W[p + "q.b"], eps) * W[p + "q.norm"]).reshape(T, H, d)
    k = (unit_rms(h @ W[p + "k"].T + W[p + "k.b"], eps) * W[p + "k.norm"]).reshape(T, G, d)
    v = (h @ W[p + "v"].T + W[p + "v.b"]).reshape(T, G, dv)
    gate = sigmoid(h @ W[p + "g"].T)
    out = np.zeros((T, H, dv))
    for i in range(T):
        for hd in range(H):
            c = hd // (H // G)
            out[i, hd] = gate[i, hd] * (weights_over((k[:i + 1, c] @ q[i, hd]) * m["scale"], 0.0) @ v[:i + 1, c])
    return out.reshape(T, H * dv) @ W[p + "o"].T


MIXERS = {"attention": differential_attention, "latent_attention": latent_attention, "attention_2": gated_attention}


def table_experts(W, p, h, tokens):
    """Every token's experts are those its row of the table names, equally weighted."""
    table, out = W[p + "table"], np.zeros_like(h)
    for t, tok in enumerate(tokens):
        for e in table[int(tok)]:
            w = lambda r: W[f"{p}e{int(e)}.{r}"]
            out[t] += (w("down") @ (silu(w("gate") @ h[t]) * (w("up") @ h[t]))) / table.shape[1]
    return out


def owner(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def residuals(W, cfg, tokens):
    """The residual stream behind every layer, [layers, tokens, width]."""
    eps, tokens = cfg["norm"]["eps"], [int(t) for t in tokens]
    x = norm(W["embed"][tokens].astype(np.float64), W["embed.norm"], eps)
    out = []
    for i in range(len(cfg["layers"])):
        j = owner(cfg, i)
        L, l = cfg["layers"][j], f"l{j}."
        a = MIXERS[L["type"]](W, l + "mix.", L["mixer"], norm(x, W[l + "norm1"], eps), eps)
        x = x + norm(a, W[l + "norm1b"], eps)
        if L.get("mlp") is not None:
            x = x + norm(table_experts(W, l + "mlp.", norm(x, W[l + "norm2"], eps), tokens), W[l + "norm2b"], eps)
        out.append(x)
    return np.stack(out)


def forward(W, cfg, tokens):
    """Logits of every position, [tokens, vocab]."""
    x = residuals(W, cfg, tokens)[-1]
    return norm(x, W["final.norm"], cfg["norm"]["eps"]) @ W["embed"].astype(np.float64).T
