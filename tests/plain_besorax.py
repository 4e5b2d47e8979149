"""The Besorax decoder written plainly: NumPy float64, whole sequences, no cache, no batches, one function per
mechanism, each from its equations.  It shares no code with the package; the tests compare the engine with it.

Notation: T tokens, W the model's width.  Weights are a dict name -> array, linear weights [out, in], applied as
y = x @ w.T.  `cfg` is the parsed config.json.
"""
import math

import numpy as np
from scipy.special import erf


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu(z):
    return 0.5 * z * (1.0 + erf(z / math.sqrt(2.0)))


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def tanh_norm(x, w, name):
    """The layers' norm: no statistics, an elementwise tanh with a gain, a weight and a bias."""
    return np.tanh(float(np.asarray(w[name + ".alpha"]).reshape(())) * x) * w[name] + w[name + ".b"]


# ------------------------------------------------------------------------------------------ rotation
def rotate_pairs(x, positions, base, dims):
    """x [T, heads, d]: among the first `dims` columns, columns 2i and 2i + 1 are turned by p * base^(-2i/dims)."""
    out = x.copy()
    for i in range(dims // 2):
        a = np.asarray(positions, dtype=np.float64) * base ** (-2.0 * i / dims)
        c, s = np.cos(a)[:, None], np.sin(a)[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i] = u * c - v * s
        out[:, :, 2 * i + 1] = v * c + u * s
    return out


# ------------------------------------------------------------------------------------------ softmax attention
def attend(q, k, v, scale, sink, chunk=0):
    """q [T, H, D], k [T, G, D], v [T, G, V].  Query i sees key j when j <= i and (no chunk size, or both lie in the same
    run of `chunk` positions counted from 0); exp(sink_h) joins the denominator."""
    T, H, _ = q.shape
    G, V = k.shape[1], v.shape[2]
    out = np.zeros((T, H, V))
    for h in range(H):
        g = h // (H // G)
        for i in range(T):
            lo = (i // chunk) * chunk if chunk else 0
            s = (k[lo:i + 1, g] @ q[i, h]) * scale
            m = max(s.max(), sink[h])
            e = np.exp(s - m)
            out[i, h] = (e @ v[lo:i + 1, g]) / (e.sum() + math.exp(sink[h] - m))
    return out


def keys_and_values(h, w, p, m, positions):
    T, G, D, V = h.shape[0], m["kv_heads"], m["dim"], m["vdim"]
    k = rotate_pairs((h @ w[p + "k"].T).reshape(T, G, D), positions, m["rot"]["base"], m["rot"]["dims"])
    return k, (h @ w[p + "v"].T).reshape(T, G, V)


def chunked_attention(h, w, p, m, positions, kv):
    T, H, D = h.shape[0], m["heads"], m["dim"]
    q = rotate_pairs((h @ w[p + "q"].T).reshape(T, H, D), positions, m["rot"]["base"], m["rot"]["dims"])
    o = attend(q, kv[0], kv[1], m["scale"], w[p + "sink"], m["mask"]["size"])
    return o.reshape(T, -1) @ w[p + "o"].T


def latent_attention(h, w, p, m, eps, positions):
    T, H, D, R, V = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    rank, base = m["kv_rank"], m["rot"]["base"]
    cq = rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]
    q = (cq @ w[p + "uq"].T).reshape(T, H, D + R)
    q = np.concatenate([q[:, :, :D], rotate_pairs(q[:, :, D:], positions, base, R)], axis=2)
    down = h @ w[p + "dkv"].T
    c = rms(down[:, :rank], eps) * w[p + "dkv.norm"]
    shared = rotate_pairs(down[:, None, rank:], positions, base, R)
    k = np.concatenate([(c @ w[p + "uk"].T).reshape(T, H, D), np.repeat(shared, H, axis=1)], axis=2)
    v = (c @ w[p + "uv"].T).reshape(T, H, V)
    return attend(q, k, v, m["scale"], w[p + "sink"]).reshape(T, -1) @ w[p + "o"].T


# ------------------------------------------------------------------------------------------ lightning attention
def decayed_sum(q, k, v, decay):
    """q, k [T, H, D], v [T, H, V].  Per head: S <- decay_h S + k v^T; o = S^T q."""
    T, H, D = q.shape
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        S = np.zeros((D, v.shape[2]))
        for t in range(T):
            S = decay[h] * S + np.outer(k[t, h], v[t, h])
            out[t, h] = S.T @ q[t, h]
    return out


def lightning_mixer(h, w, p, m, eps):
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = silu(h @ w[p + "q"].T).reshape(T, H, D)
    k = silu(h @ w[p + "k"].T).reshape(T, H, D)
    v = silu(h @ w[p + "v"].T).reshape(T, H, V)
    o = rms(decayed_sum(q, k, v, m["decay"]).reshape(T, H * V), eps) * w[p + "norm"]
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# ------------------------------------------------------------------------------------------ feed-forward
def dense_ff(h, w, p, limit):
    g = np.minimum(h @ w[p + "gate"].T, limit)
    u = np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def gelu_ff(h, w, p):
    return gelu(h @ w[p + "up"].T) @ w[p + "down"].T


def route(h, w, p, top):
    """(chosen experts [T, top], their weights): sigmoid scores, the largest win, the weights are the scores."""
    s = sigmoid(h @ w[p + "router"].T)
    idx = np.argsort(-s, axis=1, kind="stable")[:, :top]
    return idx, np.take_along_axis(s, idx, axis=1)


def routed_ff(h, w, p, top, has_shared):
    idx, wt = route(h, w, p, top)
    y = gelu_ff(h, w, p + "shared.") if has_shared else np.zeros((h.shape[0], w[p + "e0.down"].shape[0]))
    for t in range(h.shape[0]):
        for e, s in zip(idx[t], wt[t]):
            y[t] += gelu_ff(s * h[t], w, p + f"e{e}.")          # the weight multiplies the expert's INPUT
    return y


def feed_forward(h, w, p, mlp):
    if mlp["kind"] == "dense":
        return dense_ff(h, w, p, mlp["limit"])
    return routed_ff(h, w, p, mlp["router"]["top"], mlp.get("shared") is not None)


# ------------------------------------------------------------------------------------------ model
def forward(cfg, w, ids, taps=None, rounding=None):
    """Logits [T, vocab] of a whole sequence.  `taps`, a list, receives the residual stream after every layer.
    `rounding`, a function, is applied to every sublayer's normed input (to see how far a rounding there is carried)."""
    eps, mult = cfg["norm"]["eps"], cfg.get("residual_mult", 1.0)
    x = w["embed"][np.asarray(ids)] * (cfg.get("embedding") or {}).get("scale", 1.0)
    positions = np.arange(len(ids))
    kvs = {}
    rounding = rounding or (lambda u: u)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        h = rounding(tanh_norm(x, w, p + "norm1"))
        if L["type"] == "attention":
            kvs[i] = kvs[m["kv_from"]] if m.get("kv_from") is not None else keys_and_values(h, w, p + "mix.", m, positions)
            y = chunked_attention(h, w, p + "mix.", m, positions, kvs[i])
        elif L["type"] == "latent_attention":
            y = latent_attention(h, w, p + "mix.", m, eps, positions)
        elif L["type"] == "lightning":
            y = lightning_mixer(h, w, p + "mix.", m, eps)
        else:
            raise ValueError(L["type"])
        x = x + mult * y
        if L.get("mlp") is not None:
            x = x + mult * feed_forward(rounding(tanh_norm(x, w, p + "norm2")), w, p + "mlp.", L["mlp"])
        if taps is not None:
            taps.append(x)
    return tanh_norm(x, w, "final.norm") @ w["head"].T
