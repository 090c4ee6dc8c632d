"""Plain float64 implementation of the Sadodra equations: one function per mechanism, no cache, no
batching, no state carried between calls.  It shares no code with the package; the tests compare
the engine with it.

Notation: ``sd`` maps checkpoint names to float64 arrays, ``cfg`` is the config.json dictionary,
``h`` is a sublayer's input [T, W] for ONE sequence that starts at position 0, ``p`` a tensor-name
prefix such as ``"l3.mix."``.
"""
import math

import numpy as np


def to_f64(sd):
    return {k: v.double().numpy() for k, v in sd.items()}


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rms(x, w, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def layer_norm(x, w, b, eps):
    d = x - x.mean(-1, keepdims=True)
    return d / np.sqrt((d * d).mean(-1, keepdims=True) + eps) * w + b


def embedding(sd, tokens):
    """Token row plus the learned row of its position."""
    return sd["embed"][np.asarray(tokens)] + sd["pos"][:len(tokens)]


def softmax(s):
    w = np.exp(s - s.max())
    return w / w.sum()


# ------------------------------------------------------------------ windowed attention with a capped, distance-biased score
def temperature(m, t):
    """Factor of the query at position t."""
    qt = m.get("q_temp")
    return 1.0 if not qt else 1.0 + qt["coef"] * math.log((t + 1) // qt["every"] + 1.0)


def slope(h, H):
    return 2.0 ** (-8.0 * (h + 1) / H)


def scores(m, h, q, keys, i, first):
    """Scores of query q (position i, head h; temperature applied) on the keys at positions first, first + 1, ..."""
    s = keys @ q * m["scale"]
    if m.get("softcap"):
        s = m["softcap"] * np.tanh(s / m["softcap"])
    return s - slope(h, m["heads"]) * (i - (first + np.arange(len(keys))))


def attention(sd, p, m, h, eps):
    """GQA attention whose values are the keys as projected, q / k normed over all heads at once."""
    T = h.shape[0]
    H, d = m["heads"], m["dim"]
    G = m.get("kv_heads", H)
    k_raw = h @ sd[p + "k"].T
    q = rms(h @ sd[p + "q"].T, sd[p + "q.norm"], eps).reshape(T, H, d)
    k = rms(k_raw, sd[p + "k.norm"], eps).reshape(T, G, d)
    v = k_raw.reshape(T, G, d)
    size = (m.get("mask") or {}).get("size", 0)
    out = np.zeros((T, H, d))
    for i in range(T):
        first = max(0, i - size + 1) if size else 0
        for a in range(H):
            g = a // (H // G)
            s = scores(m, a, q[i, a] * temperature(m, i), k[first:i + 1, g], i, first)
            out[i, a] = softmax(s) @ v[first:i + 1, g]
    return out.reshape(T, H * d) @ sd[p + "o"].T


# ------------------------------------------------------------------ latent attention without positions
def latent(sd, p, h, eps):
    """The normed latent of every token, [T, kv_rank]."""
    return rms(h @ sd[p + "dkv"].T, sd[p + "dkv.norm"], eps)


def latent_attention(sd, p, m, h, c):
    """Causal softmax attention over per-head keys and values expanded from the latents ``c``
    (this layer's own or an earlier layer's), one sigmoid gate per head."""
    T = h.shape[0]
    H, d, vd = m["heads"], m["dim"], m["vdim"]
    q = (h @ sd[p + "q"].T).reshape(T, H, d)
    k = (c @ sd[p + "uk"].T).reshape(T, H, d)
    v = (c @ sd[p + "uv"].T).reshape(T, H, vd)
    gate = sigmoid(h @ sd[p + "g"].T)
    out = np.zeros((T, H, vd))
    for i in range(T):
        for a in range(H):
            s = k[:i + 1, a] @ q[i, a] * m["scale"]
            out[i, a] = softmax(s) @ v[:i + 1, a] * gate[i, a]
    return out.reshape(T, H * vd) @ sd[p + "o"].T


# ------------------------------------------------------------------ feed-forward, whole model
def feed_forward(sd, p, h):
    return (gelu_tanh(h @ sd[p + "gate"].T) * (h @ sd[p + "up"].T)) @ sd[p + "down"].T


def forward(sd, cfg, tokens, trace=None):
    """Logits [T, vocab] of one sequence; ``trace`` receives the residual stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = embedding(sd, tokens)
    latents = {}
    for i, l in enumerate(cfg["layers"]):
        p, m = f"l{i}.", l["mixer"]
        if l["type"] == "attention":
            y = attention(sd, p + "mix.", m, x, eps)
        else:
            src = m.get("kv_from")
            if src is None:
                latents[i] = latent(sd, p + "mix.", x, eps)
            y = latent_attention(sd, p + "mix.", m, x, latents[i if src is None else src])
        x = x + layer_norm(y, sd[p + "norm1"], sd[p + "norm1.b"], eps)
        if l.get("mlp"):
            x = x + layer_norm(feed_forward(sd, p + "mlp.", x), sd[p + "norm2"], sd[p + "norm2.b"], eps)
        if trace is not None:
            trace.append(x.copy())
    return layer_norm(x, sd["final.norm"], sd["final.norm.b"], eps) @ sd["head"].T
