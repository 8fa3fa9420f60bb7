"""Plain implementation of the Belelorn design in numpy float64: one function per mechanism, whole sequences
only (no cache; the recurrences may be given a state), written from the design's equations and sharing no code with
the package.  `weights` maps checkpoint names to arrays; `cfg` is the config.json dictionary."""
import math

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


def unit_rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm(x, w, eps):
    """RMS norm whose stored weight is the distance from one."""
    return unit_rms(x, eps) * (1.0 + w)


def position_vectors(positions, width):
    out = np.zeros((len(positions), width))
    for j in range(width):
        angle = np.asarray(positions, dtype=np.float64) * 10000.0 ** (-2.0 * (j // 2) / width)
        out[:, j] = np.sin(angle) if j % 2 == 0 else np.cos(angle)
    return out


def embedding(W, cfg, tokens):
    tokens = np.asarray(tokens)
    return W["embed"][tokens].astype(np.float64) + position_vectors(np.arange(len(tokens)), cfg["width"])


def visible(i, j, size, keep_first):
    return j <= i and (size <= 0 or i - j < size or j < keep_first)


def softmax_attention(W, p, m, h, eps):
    """Grouped queries; unit-RMS queries and keys; values are the keys as projected; capped scores; a sliding window
    beside which the first tokens stay visible."""
    T = h.shape[0]
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    q = (h @ W[p + "q"].T + W[p + "q.b"]).reshape(T, H, d)
    k = (h @ W[p + "k"].T + W[p + "k.b"]).reshape(T, G, d)
    v = k.copy()
    q, k = unit_rms(q, eps), unit_rms(k, eps)
    mask = m.get("mask") or {}
    size, first = mask.get("size", 0), mask.get("keep_first", 0)
    cap = m.get("softcap")
    out = np.zeros((T, H, d))
    for i in range(T):
        see = [j for j in range(i + 1) if visible(i, j, size, first)]
        for hd in range(H):
            c = hd // (H // G)
            s = (k[see, c] @ q[i, hd]) * m["scale"]
            if cap:
                s = cap * np.tanh(s / cap)
            e = np.exp(s - s.max())
            out[i, hd] = (e @ v[see, c]) / e.sum()
    return out.reshape(T, H * d) @ W[p + "o"].T


def lightning_attention(W, p, m, h, eps, state=None):
    """S_t = decay_h S_(t-1) + k_t v_t^T, o_t = S_t^T q_t with SiLU on q, k and v; norm over all heads together, a
    sigmoid gate, the output projection.  Returns (result, last states)."""
    T = h.shape[0]
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    q = silu(h @ W[p + "q"].T).reshape(T, H, dk)
    k = silu(h @ W[p + "k"].T).reshape(T, H, dk)
    v = silu(h @ W[p + "v"].T).reshape(T, H, dv)
    decay = m["decay"] if isinstance(m["decay"], (list, tuple)) else [m["decay"]] * H
    S = np.zeros((H, dk, dv)) if state is None else state.copy()
    o = np.zeros((T, H, dv))
    for t in range(T):
        for hd in range(H):
            S[hd] = decay[hd] * S[hd] + np.outer(k[t, hd], v[t, hd])
            o[t, hd] = S[hd].T @ q[t, hd]
    o = unit_rms(o.reshape(T, H * dv), eps) * W[p + "norm"] * sigmoid(h @ W[p + "g"].T)
    return o @ W[p + "o"].T, S


def two_mixers(W, p, m, h, eps):
    left = softmax_attention(W, p + "left.", m["left"], h, eps)
    right, _ = lightning_attention(W, p + "right.", m["right"], h, eps)
    return 0.5 * (unit_rms(left, eps) * W[p + "left.out"] + unit_rms(right, eps) * W[p + "right.out"])


def matrix_memory(q, k, v, log_i, log_f, state=None):
    """The stabilised recurrence over q, k [T, H, dk] (q scaled), v [T, H, dv] and the logarithms of the gates [T, H].
    state: (S [H, dk, dv], n [H, dk], m [H]).  Returns (o [T, H, dv], last state)."""
    T, H, dk = q.shape
    dv = v.shape[-1]
    S, n, m = (np.zeros((H, dk, dv)), np.zeros((H, dk)), np.zeros(H)) if state is None else (a.copy() for a in state)
    o = np.zeros((T, H, dv))
    for t in range(T):
        for hd in range(H):
            top = max(log_f[t, hd] + m[hd], log_i[t, hd])
            keep, take = math.exp(log_f[t, hd] + m[hd] - top), math.exp(log_i[t, hd] - top)
            S[hd] = keep * S[hd] + take * np.outer(k[t, hd], v[t, hd])
            n[hd] = keep * n[hd] + take * k[t, hd]
            m[hd] = top
            o[t, hd] = (S[hd].T @ q[t, hd]) / (max(abs(n[hd] @ q[t, hd]), math.exp(-top)) + 1e-6)
    return o, (S, n, m)


def log_gates(W, p, m, h):
    cap = m["gate_cap"]
    z = lambda r: cap * np.tanh((h @ W[p + r].T + W[p + r + ".b"]) / cap)
    return z("i"), log_sigmoid(z("f"))


def mlstm(W, p, m, h, eps, state=None):
    T = h.shape[0]
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    q = (h @ W[p + "q"].T).reshape(T, H, dk) * dk ** -0.5
    k = (h @ W[p + "k"].T).reshape(T, H, dk)
    v = (h @ W[p + "v"].T).reshape(T, H, dv)
    log_i, log_f = log_gates(W, p, m, h)
    o, state = matrix_memory(q, k, v, log_i, log_f, state)
    o = unit_rms(o, eps).reshape(T, H * dv) * W[p + "norm"] * sigmoid(h @ W[p + "g"].T)
    return o @ W[p + "o"].T, state


def dense(W, p, f, h):
    return np.maximum(h @ W[p + "up"].T, 0.0) ** 2 @ W[p + "down"].T


def expert(W, p, h, limit):
    g = np.minimum(h @ W[p + "gate"].T, limit)
    u = np.clip(h @ W[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ W[p + "down"].T


def route(W, p, f, h):
    """-> (chosen [T, top], their weights [T, top])."""
    s = sigmoid(h @ W[p + "router"].T)
    chosen = np.argsort(-s, axis=-1, kind="stable")[:, : f["router"]["top"]]
    return chosen, np.take_along_axis(s, chosen, axis=-1)


def experts(W, p, f, h):
    """Each chosen expert reads its share of the token: the weight is on its input."""
    chosen, w = route(W, p, f, h)
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(chosen[t], w[t]):
            out[t] += expert(W, f"{p}e{e}.", a * h[t], f["expert"]["limit"])
    if f.get("shared"):
        out = out + expert(W, p + "shared.", h, f["shared"]["limit"])
    return out


def layer(W, cfg, i, x):
    L, l = cfg["layers"][i], f"l{i}."
    eps = cfg["norm"]["eps"]
    h = norm(x, W[l + "norm1"], eps)
    if L["type"] == "parallel":
        y = two_mixers(W, l + "mix.", L["mixer"], h, eps)
    else:
        y, _ = mlstm(W, l + "mix.", L["mixer"], h, eps)
    x = x + norm(y, W[l + "norm1b"], eps)
    f = L.get("mlp")
    if f is not None:
        h = norm(x, W[l + "norm2"], eps)
        y = dense(W, l + "mlp.", f, h) if f["kind"] == "dense" else experts(W, l + "mlp.", f, h)
        x = x + norm(y, W[l + "norm2b"], eps)
    return x


def runs(cfg):
    """The layers in the order they run: (layer, number of the pass or None, whether it is a pass's first)."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None, False) for i in range(n)]
    out = [(i, None, False) for i in range(loop["start"])]
    for t in range(loop["times"]):
        out += [(i, t, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return out + [(i, None, False) for i in range(loop["stop"], n)]


def enter_pass(W, x, x0, t):
    return np.concatenate([x, x0], axis=-1) @ W["loop.in"].T + W["loop.step"][t]


def forward(W, cfg, tokens, residuals=None):
    """Logits [T, vocab] of one whole sequence; residuals (a list) receives the stream after every layer run."""
    x0 = embedding(W, cfg, tokens)
    x = x0
    for i, t, first in runs(cfg):
        if first:
            x = enter_pass(W, x, x0, t)
        x = layer(W, cfg, i, x)
        if residuals is not None:
            residuals.append(x.copy())
    return (norm(x, W["final.norm"], cfg["norm"]["eps"]) @ W["head"].T) * cfg["logit_scale"]
