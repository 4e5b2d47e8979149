"""The Dimelix decoder written plainly: NumPy float64, whole sequences, no cache, no batches, one function per
mechanism, each from its equations.  It shares no code with the package; the tests compare the engine with it.

Notation: T tokens, W the model's width.  Weights are a dict name -> array, linear weights [out, in], applied as
y = x @ w.T.  `cfg` is the parsed config.json.
"""
import math

import numpy as np

UNIT_EPS = 1e-6
DECAY_FACTOR = math.exp(-0.5)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def softplus(z):
    return np.logaddexp(0.0, z)


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def offset_norm(x, w, eps):
    """The layers' norm: the weight is stored around zero, y = rms(x) * (1 + w)."""
    return rms(x, eps) * (1.0 + w)


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
def attend(q, k, v, scale, sink=None, window=0, slopes=None):
    """q [T, H, D], k [T, G, D], v [T, G, V].  Query i sees key j when j <= i and (no window, or i - j < window);
    score (q . k) * scale - slope_h (i - j); a sink adds exp(sink_h) to the denominator."""
    T, H, _ = q.shape
    G, V = k.shape[1], v.shape[2]
    out = np.zeros((T, H, V))
    for h in range(H):
        g = h // (H // G)
        for i in range(T):
            lo = max(0, i - window + 1) if window else 0
            s = (k[lo:i + 1, g] @ q[i, h]) * scale
            if slopes is not None:
                s = s - slopes[h] * (i - np.arange(lo, i + 1))
            m = s.max() if sink is None else max(s.max(), sink[h])
            e = np.exp(s - m)
            out[i, h] = (e @ v[lo:i + 1, g]) / (e.sum() + (0.0 if sink is None else math.exp(sink[h] - m)))
    return out


def heads_out(o, h, w, p):
    """The gate, element by element, and the output projection."""
    o = o.reshape(o.shape[0], -1) * sigmoid(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def rotary_attention(h, w, p, m, eps, positions):
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms((h @ w[p + "q"].T).reshape(T, H, D), eps) * w[p + "q.norm"]
    k = rms((h @ w[p + "k"].T).reshape(T, G, D), eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].T).reshape(T, G, V)
    q = rotate_pairs(q, positions, m["rot"]["base"], m["rot"]["dims"])
    k = rotate_pairs(k, positions, m["rot"]["base"], m["rot"]["dims"])
    return heads_out(attend(q, k, v, m["scale"], sink=w[p + "sink"]), h, w, p)


def latent_attention(h, w, p, m, eps):
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).reshape(T, H, D)
    c = rms(h @ w[p + "dkv"].T, eps) * w[p + "dkv.norm"]
    k = (c @ w[p + "uk"].T).reshape(T, H, D)
    v = (c @ w[p + "uv"].T).reshape(T, H, V)
    return heads_out(attend(q, k, v, m["scale"]), h, w, p)


def distance_attention(h, w, p, m, eps):
    """The keys before their norm are the values; no rotation; every score loses slope_h times the distance."""
    T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = rms((h @ w[p + "q"].T).reshape(T, H, D), eps) * w[p + "q.norm"]
    raw = (h @ w[p + "k"].T).reshape(T, G, D)
    k = rms(raw, eps) * w[p + "k.norm"]
    slopes = [2.0 ** (-8.0 * (hh + 1) / H) for hh in range(H)]
    return heads_out(attend(q, k, raw, m["scale"], window=m["mask"]["size"], slopes=slopes), h, w, p)


# ------------------------------------------------------------------------------------------ delta rule, decay a channel
def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + UNIT_EPS)


def channel_delta_rule(r, k, v, decay, removal):
    """All [T, H, D].  Per head, S of D x D, u = unit(k): S <- diag(decay) S - (removal * u) (u^T S) + k v^T with the
    old S in both terms; o = S^T r."""
    T, H, D = r.shape
    out = np.zeros((T, H, v.shape[2]))
    u = unit(k)
    for h in range(H):
        S = np.zeros((D, v.shape[2]))
        for t in range(T):
            S = decay[t, h][:, None] * S - np.outer(removal[t, h] * u[t, h], u[t, h] @ S) + np.outer(k[t, h], v[t, h])
            out[t, h] = r[t, h] @ S
    return out


def channel_delta_mixer(h, w, p, m, eps):
    T, H, D = h.shape[0], m["heads"], m["dim"]
    r, k, v = ((h @ w[p + x].T).reshape(T, H, D) for x in "rkv")
    low = np.tanh(h @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]
    decay = np.exp(-DECAY_FACTOR * sigmoid(low)).reshape(T, H, D)
    removal = sigmoid(h @ w[p + "a"].T + w[p + "a.b"]).reshape(T, H, D)
    o = rms(channel_delta_rule(r, k, v, decay, removal), eps).reshape(T, H * D) * w[p + "norm"]
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel_mixer(h, w, p, m, eps):
    return (m["left_scale"] * distance_attention(h, w, p + "left.", m["left"], eps)
            + m["right_scale"] * channel_delta_mixer(h, w, p + "right.", m["right"], eps))


# ------------------------------------------------------------------------------------------ feed-forward
def xielu(z, p, q):
    neg = np.minimum(z, 0.0)
    return np.where(z > 0, softplus(p) * z * z + 0.5 * z, (0.5 + softplus(q)) * (np.exp(neg) - 1.0 - neg) + 0.5 * z)


def dense_ff(h, w, p):
    a = w[p + "act"]
    return xielu(h @ w[p + "up"].T, a[0], a[1]) @ w[p + "down"].T


# ------------------------------------------------------------------------------------------ streams
def read_streams(xs, w, p):
    return sum(w[p + "in"][s] * xs[s] for s in range(len(xs)))


def write_streams(xs, y, w, p):
    mix, out = w[p + "mix"], w[p + "out"]
    return [sum(mix[s, t] * xs[s] for s in range(len(xs))) + out[t] * y for t in range(len(xs))]


# ------------------------------------------------------------------------------------------ model
def mixer(L, u, w, p, eps, positions):
    if L["type"] == "attention":
        return rotary_attention(u, w, p, L["mixer"], eps, positions)
    if L["type"] == "latent_attention":
        return latent_attention(u, w, p, L["mixer"], eps)
    if L["type"] == "parallel":
        return parallel_mixer(u, w, p, L["mixer"], eps)
    raise ValueError(L["type"])


def order(cfg):
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    return list(range(loop["start"])) + loop["times"] * list(range(loop["start"], loop["stop"])) + list(range(loop["stop"], n))


def forward(cfg, w, ids, taps=None, rounding=None):
    """Logits [T, vocab] of a whole sequence.  `taps`, a list, receives the sum of the streams after every layer run.
    `rounding`, a function, is applied to every sublayer's normed input (to see how far a rounding there is carried)."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(ids)] * cfg["embedding"]["scale"]
    xs = [x.copy() for _ in range(cfg["streams"])]
    positions = np.arange(len(ids))
    for i in order(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        u = offset_norm(read_streams(xs, w, p + "hc1."), w[p + "norm1"], eps)
        u = rounding(u) if rounding else u
        xs = write_streams(xs, mixer(L, u, w, p + "mix.", eps, positions), w, p + "hc1.")
        if L.get("mlp") is not None:
            u = offset_norm(read_streams(xs, w, p + "hc2."), w[p + "norm2"], eps)
            u = rounding(u) if rounding else u
            xs = write_streams(xs, dense_ff(u, w, p + "mlp."), w, p + "hc2.")
        if taps is not None:
            taps.append(sum(xs))
    return head(cfg, w, sum(xs))


def head(cfg, w, x):
    logits = offset_norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["embed"].T
    cap = cfg.get("logit_softcap") or 0.0
    return cap * np.tanh(logits / cap) if cap else logits
