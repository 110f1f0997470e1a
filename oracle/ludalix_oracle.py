"""Plain, slow statement of the Ludalix decoder in numpy float64: one function per mechanism, whole sequences at
a time, no cache, recurrences token by token. Test infrastructure; it shares no code with the library and reads
nothing but arrays.

Notation: x_t is the residual row of token t = 0, 1, ... of its sequence, all weights are [out, in].

  stem        x = scale * E[token] + wave(t)
  layer       x += mu n1(mixer(x)); with a feed-forward also x += mu n2(ff(x))
  head        logits = W_head n_final(x)
"""
from __future__ import annotations

import numpy as np


# ── elementary pieces ────────────────────────────────────────────────────────

def unit_rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def log_sigmoid(z):
    return np.minimum(z, 0.0) - np.log1p(np.exp(-np.abs(z)))


def soft_cap(z, cap):
    return cap * np.tanh(z / cap)


def position_waves(positions, width):
    """Row t: columns 2i and 2i + 1 are the sine and cosine of t / 10000^(2i / width)."""
    c = np.arange(width)
    angle = np.asarray(positions, np.float64)[:, None] * 10000.0 ** (-(c - c % 2) / width)
    return np.where(c % 2 == 0, np.sin(angle), np.cos(angle))


# ── matrix memory ────────────────────────────────────────────────────────────

def matrix_memory(q, k, v, log_in, log_forget):
    """One head: q, k [T, dim], v [T, vdim], gates [T]. Memory C and normaliser z are kept divided by e^m, m the
    running maximum of the log weights (0 at the start)."""
    T, dim = q.shape
    C, z, m = np.zeros((dim, v.shape[1])), np.zeros(dim), 0.0
    out = np.zeros((T, v.shape[1]))
    for t in range(T):
        top = max(log_forget[t] + m, log_in[t])
        keep, take = np.exp(log_forget[t] + m - top), np.exp(log_in[t] - top)
        C = keep * C + take * np.outer(k[t], v[t])
        z = keep * z + take * k[t]
        m = top
        out[t] = (q[t] @ C) / (max(abs(z @ q[t]), np.exp(-m)) + 1e-6)
    return out


def mlstm(h, m, t, eps):
    """m: the mixer's sizes, t: suffix -> tensor."""
    T, H, dim, vdim, cap = len(h), m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q = (h @ t["q"].T).reshape(T, H, dim) / np.sqrt(dim)
    k = (h @ t["k"].T).reshape(T, H, dim)
    v = (h @ t["v"].T).reshape(T, H, vdim)
    log_in = soft_cap(h @ t["i"].T + t["i.b"], cap)
    log_forget = log_sigmoid(soft_cap(h @ t["f"].T + t["f.b"], cap))
    o = np.stack([unit_rms(matrix_memory(q[:, a], k[:, a], v[:, a], log_in[:, a], log_forget[:, a]), eps) for a in range(H)], axis=1)
    return (o.reshape(T, H * vdim) * t["norm"] * sigmoid(h @ t["g"].T)) @ t["o"].T


# ── attention ────────────────────────────────────────────────────────────────

def visible(T, window, kept):
    """[T, T] (row = query): which keys a query sees."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    near = i - j < window if window else np.ones((T, T), bool)
    return (j <= i) & (near | (j < kept))


def masked_softmax(score, seen):
    s = np.where(seen, score, -np.inf)
    p = np.exp(s - s.max(axis=-1, keepdims=True))
    return p / p.sum(axis=-1, keepdims=True)


def attention_keys(h, m, t, eps):
    """Normed keys [T, G, dim] and values [T, G, vdim]."""
    T, G = len(h), m["kv_heads"]
    k = unit_rms((h @ t["k"].T).reshape(T, G, m["dim"]), eps) * t["k.norm"]
    return k, (h @ t["v"].T).reshape(T, G, m["vdim"])


def attention(h, m, t, eps, k, v):
    T, H, G = len(h), m["heads"], m["kv_heads"]
    q = unit_rms((h @ t["q"].T).reshape(T, H, m["dim"]), eps) * t["q.norm"]
    mask = m.get("mask") or {}
    seen = visible(T, mask.get("size") or 0, mask.get("keep_first") or 0)
    out = np.zeros((T, H, m["vdim"]))
    for a in range(H):
        g = a // (H // G)
        out[:, a] = masked_softmax((q[:, a] @ k[:, g].T) * m["scale"], seen) @ v[:, g]
    return out.reshape(T, -1) @ t["o"].T


# ── feed-forward ─────────────────────────────────────────────────────────────

def clamped_glu(h, gate, up, down, limit):
    g = np.minimum(h @ gate.T, limit)
    u = np.clip(h @ up.T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def route(h, router, top):
    """Chosen experts [T, top] and their weights, the scores themselves."""
    s = sigmoid(h @ router.T)
    chosen = np.argsort(-s, axis=1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, axis=1)


def expert(h, gate, up, down):
    z = h @ gate.T
    return (z * sigmoid(z) * (h @ up.T)) @ down.T


def mixture(h, mlp, t):
    """t: suffix -> tensor ("router", "e0.gate", ...). An expert sees its weight on its input."""
    chosen, weight = route(h, t["router"], mlp["router"]["top"])
    y = np.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        rows, place = np.nonzero(chosen == e)
        if len(rows):
            y[rows] += expert(weight[rows, place][:, None] * h[rows], t[f"e{e}.gate"], t[f"e{e}.up"], t[f"e{e}.down"])
    return y


# ── the model ────────────────────────────────────────────────────────────────

def forward(cfg, weights, tokens):
    """(logits [T, vocab], residual after every layer [layers, T, width]) of one sequence, float64."""
    w = {k: np.asarray(v, np.float64) for k, v in weights.items()}
    eps, mu = cfg["norm"]["eps"], cfg["residual_mult"]
    x = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"] + position_waves(np.arange(len(tokens)), cfg["width"])
    trail, keys = [], {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        t = {k[len(p) + 4:]: v for k, v in w.items() if k.startswith(p + "mix.")}
        if layer["type"] == "mlstm":
            y = mlstm(x, m, t, eps)
        else:
            source = m.get("kv_from")
            if source is None:
                keys[i] = attention_keys(x, m, t, eps)
            y = attention(x, m, t, eps, *keys[i if source is None else source])
        x = x + mu * unit_rms(y, eps) * w[p + "norm1"]
        mlp = layer.get("mlp")
        if mlp:
            t = {k[len(p) + 4:]: v for k, v in w.items() if k.startswith(p + "mlp.")}
            y = clamped_glu(x, t["gate"], t["up"], t["down"], mlp["limit"]) if mlp["kind"] == "dense" else mixture(x, mlp, t)
            x = x + mu * unit_rms(y, eps) * w[p + "norm2"]
        trail.append(x)
    return unit_rms(x, eps) * w["final.norm"] @ w["head"].T, np.stack(trail)
