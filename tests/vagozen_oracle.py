"""Plain float64 implementation of the Vagozen equations: one function per mechanism, no cache, no
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


def unit_rms(x, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def rms(x, w, eps):
    return unit_rms(x, eps) * w


def softmax(s):
    w = np.exp(s - s.max(-1, keepdims=True))
    return w / w.sum(-1, keepdims=True)


# ------------------------------------------------------------------ rotary positions
def frequencies(rot):
    """(frequency of every pair, factor of cos and sin): base^(-2i / dims), with the ramp between two
    turn counts of the original context when the config scales them."""
    dims, base = rot["dims"], float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if not s:
        return np.array(f), 1.0

    def pair_of(turns):
        return dims * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo = max(math.floor(pair_of(s["fast"])), 0)
    hi = min(math.ceil(pair_of(s["slow"])), dims - 1)
    for i in range(dims // 2):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        f[i] = r * f[i] / s["factor"] + (1.0 - r) * f[i]
    return np.array(f), 1.0 + 0.1 * math.log(s["factor"])


def turn(x, rot, layout):
    """x [T, ..., d]: row t is the vector at position t.  layout "pairs": features 2i and 2i + 1 turn
    together, "halves": features i and i + dims / 2."""
    if not rot or not rot["dims"]:
        return x
    n = rot["dims"] // 2
    f, amp = frequencies(rot)
    a = np.arange(x.shape[0]).reshape((-1,) + (1,) * (x.ndim - 1)) * f
    c, s = np.cos(a) * amp, np.sin(a) * amp
    y = x.copy()
    if layout == "pairs":
        u, v = x[..., 0:2 * n:2], x[..., 1:2 * n:2]
        y[..., 0:2 * n:2], y[..., 1:2 * n:2] = u * c - v * s, v * c + u * s
    else:
        u, v = x[..., :n], x[..., n:2 * n]
        y[..., :n], y[..., n:2 * n] = u * c - v * s, v * c + u * s
    return y


# ------------------------------------------------------------------ window attention with kept first keys
def sees(mask, i, T):
    """[T] bool: the keys that position i sees."""
    j = np.arange(T)
    see = j <= i
    if mask:
        see &= (i - j < mask["size"]) | (j < mask.get("keep_first", 0))
    return see


def attention(sd, p, m, h):
    T = h.shape[0]
    H, d, vd = m["heads"], m["dim"], m["vdim"]
    G = m.get("kv_heads", H)
    q = turn((h @ sd[p + "q"].T + sd[p + "q.b"]).reshape(T, H, d), m.get("rot"), "pairs")
    k = turn((h @ sd[p + "k"].T + sd[p + "k.b"]).reshape(T, G, d), m.get("rot"), "pairs")
    v = (h @ sd[p + "v"].T + sd[p + "v.b"]).reshape(T, G, vd)
    see = np.stack([sees(m.get("mask"), i, T) for i in range(T)])
    out = np.zeros((T, H, vd))
    for a in range(H):
        g = a // (H // G)
        s = np.where(see, q[:, a] @ k[:, g].T * m["scale"], -np.inf)
        out[:, a] = softmax(s) @ v[:, g]
    return out.reshape(T, H * vd) @ sd[p + "o"].T


# ------------------------------------------------------------------ retention
def retention_states(m, k, v):
    """Yields S_t [H, dim, vdim] for t = 0, 1, ...: S_t = decay S_(t-1) + k_t v_t^T from S = 0."""
    H, vd = v.shape[1:]
    S = np.zeros((H, k.shape[2], vd))
    for t in range(k.shape[0]):
        S = np.asarray(m["decay"], dtype=np.float64)[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        yield S


def retention(sd, p, m, h, eps):
    T = h.shape[0]
    H, d, vd = m["heads"], m["dim"], m["vdim"]
    q = turn((h @ sd[p + "q"].T).reshape(T, H, d), m.get("rot"), "halves")
    k = turn((h @ sd[p + "k"].T).reshape(T, H, d), m.get("rot"), "halves") / math.sqrt(d)
    v = (h @ sd[p + "v"].T).reshape(T, H, vd)
    o = np.stack([np.einsum("hde,hd->he", S, q[t]) for t, S in enumerate(retention_states(m, k, v))])
    z = h @ sd[p + "g"].T
    return (unit_rms(o, eps).reshape(T, H * vd) * (z * sigmoid(z))) @ sd[p + "o"].T


# ------------------------------------------------------------------ latent attention
def latent_attention(sd, p, m, h, eps):
    """Causal softmax attention over per-head keys and values expanded from one latent per token,
    plus one rotated key part for all heads."""
    T = h.shape[0]
    H, d, rd, vd, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (rms(h @ sd[p + "dq"].T, sd[p + "dq.norm"], eps) @ sd[p + "uq"].T).reshape(T, H, d + rd)
    q_plain, q_rot = q[..., :d], turn(q[..., d:], m.get("rot"), "pairs")
    y = h @ sd[p + "dkv"].T
    c, k_rot = rms(y[:, :r], sd[p + "dkv.norm"], eps), turn(y[:, r:], m.get("rot"), "pairs")
    k = (c @ sd[p + "uk"].T).reshape(T, H, d)
    v = (c @ sd[p + "uv"].T).reshape(T, H, vd)
    see = np.tril(np.ones((T, T), dtype=bool))
    out = np.zeros((T, H, vd))
    for a in range(H):
        s = (q_plain[:, a] @ k[:, a].T + q_rot[:, a] @ k_rot.T) * m["scale"]
        out[:, a] = softmax(np.where(see, s, -np.inf)) @ v[:, a]
    return out.reshape(T, H * vd) @ sd[p + "o"].T


def mixer(sd, p, l, h, eps):
    if l["type"] == "attention":
        return attention(sd, p, l["mixer"], h)
    if l["type"] == "retention":
        return retention(sd, p, l["mixer"], h, eps)
    return latent_attention(sd, p, l["mixer"], h, eps)


# ------------------------------------------------------------------ feed-forwards
def clamped_glu(g, u, limit):
    g, u = np.minimum(g, limit), np.clip(u, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


def gated(sd, p, h, limit):
    return clamped_glu(h @ sd[p + "gate"].T, h @ sd[p + "up"].T, limit) @ sd[p + "down"].T


def route(sd, p, h, top):
    """(chosen experts [T, top], weights [T, top])."""
    z = h @ sd[p + "router"].T + sd[p + "router.b"]
    idx = np.argsort(-z, axis=-1, kind="stable")[:, :top]
    return idx, softmax(np.take_along_axis(z, idx, 1))


def experts(sd, p, f, h):
    idx, w = route(sd, p, h, f["router"]["top"])
    out = np.zeros_like(h)
    for e in range(f["router"]["experts"]):
        t, j = np.nonzero(idx == e)
        if len(t):
            out[t] += w[t, j][:, None] * gated(sd, f"{p}e{e}.", h[t], f["expert"]["limit"])
    return out


def feed_forward(sd, p, f, h):
    return gated(sd, p, h, f["limit"]) if f["kind"] == "dense" else experts(sd, p, f, h)


# ------------------------------------------------------------------ layers, loop, whole model
def layer(sd, i, l, x, eps):
    n = f"l{i}."
    y = mixer(sd, n + "mix.", l, rms(x, sd[n + "norm1"], eps), eps)
    x = x + rms(y, sd[n + "norm1b"], eps) * sd[n + "ls1"]
    if l.get("mlp"):
        y = feed_forward(sd, n + "mlp.", l["mlp"], rms(x, sd[n + "norm2"], eps))
        x = x + rms(y, sd[n + "norm2b"], eps) * sd[n + "ls2"]
    return x


def schedule(cfg):
    """[(layer, pass it opens or None)] in running order."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop or loop["stop"] <= loop["start"]:
        return [(i, None) for i in range(n)]
    runs = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        runs += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return runs + [(i, None) for i in range(loop["stop"], n)]


def enter_pass(sd, t, x, x0):
    """The stream as pass t starts: from the second pass on the embedding comes in again, then the
    pass's own vector."""
    return (x if t == 0 else x + x0) + sd["loop.step"][t]


def forward(sd, cfg, tokens, trace=None):
    """Logits [T, vocab] of one sequence; ``trace`` receives the residual stream after every layer run."""
    eps = cfg["norm"]["eps"]
    x0 = sd["embed"][np.asarray(tokens)]
    x = x0
    for i, opens in schedule(cfg):
        if opens is not None:
            x = enter_pass(sd, opens, x, x0)
        x = layer(sd, i, cfg["layers"][i], x, eps)
        if trace is not None:
            trace.append(x.copy())
    return rms(x, sd["final.norm"], eps) @ sd["embed"].T * cfg.get("logit_scale", 1.0)
