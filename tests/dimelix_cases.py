"""Tiny Dimelix configurations and weights for the tests, made here: sizes that differ in everything from each other, and
weights with gains near one, so that every mechanism moves the logits (the framework's own random weights are N(0, 0.02):
a mixer's fault would hardly show through them)."""
import json
from pathlib import Path

import numpy as np
import torch


def dense(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def attention(heads, kv_heads, dim, vdim, scale, base, dims, ff):
    return {"type": "attention", "mlp": dense(ff),
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"base": base, "dims": dims}}}


def latent(heads, dim, vdim, kv_rank, scale, ff):
    return {"type": "latent_attention", "mlp": dense(ff),
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale}}


def parallel(left, right, left_scale, right_scale, ff):
    """left = (heads, kv_heads, dim, scale, window); right = (heads, dim)."""
    lh, lkv, ld, ls, win = left
    return {"type": "parallel", "mlp": dense(ff),
            "mixer": {"left": {"heads": lh, "kv_heads": lkv, "dim": ld, "vdim": ld, "scale": ls, "mask": {"size": win}},
                      "right": {"heads": right[0], "dim": right[1]}, "left_scale": left_scale, "right_scale": right_scale}}


# A: small odd sizes, two streams; the windowed layer first and a layer without feed-forward; the last two passed twice
CONFIG_A = {"architecture": "Dimelix", "vocab": 203, "width": 88, "norm": {"eps": 1e-4}, "streams": 2, "embedding": {"scale": 1.7},
            "logit_softcap": 11.0, "loop": {"start": 2, "stop": 4, "times": 2},
            "layers": [parallel((6, 3, 20, 0.25, 9), (3, 12), 0.6, 1.1, 100), attention(6, 2, 12, 28, 0.35, 700.0, 8, None),
                       latent(3, 20, 12, 28, 0.21, 72), parallel((2, 2, 10, 0.4, 33), (1, 30), 1.3, 0.8, None)]}
# B: five streams, no loop, no cap, one kv head, rotation of the whole head, a window of one token (only the token itself)
CONFIG_B = {"architecture": "Dimelix", "vocab": 310, "width": 120, "norm": {"eps": 1e-6}, "streams": 5, "embedding": {"scale": 0.8},
            "layers": [attention(8, 1, 16, 48, 0.25, 1e6, 16, 136), parallel((4, 1, 16, 0.3, 1), (5, 8), 0.9, 0.7, 56),
                       latent(5, 8, 24, 48, 0.4, None)]}
# C: sizes that reach the matrix-core kernels (heads of 64 and 128 columns, latents of 64 and 128 columns, widths in
# multiples of 32), states of 64 and of 128 values a column, four streams, the whole model passed twice
CONFIG_C = {"architecture": "Dimelix", "vocab": 416, "width": 256, "norm": {"eps": 1e-5}, "streams": 4, "embedding": {"scale": 1.0},
            "logit_softcap": 25.0, "loop": {"start": 0, "stop": 3, "times": 2},
            "layers": [parallel((8, 2, 128, 0.09, 48), (2, 128), 0.9, 0.8, 512), latent(8, 64, 32, 128, 0.125, 384),
                       attention(4, 2, 64, 128, 0.12, 5000.0, 32, None), latent(4, 32, 64, 64, 0.17, 320),
                       parallel((4, 4, 64, 0.125, 130), (4, 64), 0.5, 1.2, 256)]}
# D: ones everywhere: one stream, one head, two rotated columns, one layer of each kind
CONFIG_D = {"architecture": "Dimelix", "vocab": 64, "width": 40, "norm": {"eps": 1e-6}, "streams": 1, "embedding": {"scale": 3.0},
            "logit_softcap": 6.0, "loop": {"start": 1, "stop": 2, "times": 1},
            "layers": [latent(1, 8, 8, 16, 0.35, None), attention(1, 1, 8, 8, 0.35, 100.0, 2, 24), parallel((1, 1, 8, 0.3, 5), (1, 16), 1.0, 1.0, 48)]}
# name -> (configuration, page size, seed, rank of the decays' low-rank pair)
CASES = {"A": (CONFIG_A, 8, 41, 6), "B": (CONFIG_B, 16, 42, 20), "C": (CONFIG_C, 32, 43, 32), "D": (CONFIG_D, 4, 44, 1)}


def tensor_shapes(config, rank):
    """name -> shape of every tensor, from the configuration, written out here again."""
    W, s, out = config["width"], config["streams"], {"embed": (config["vocab"], config["width"]), "final.norm": (config["width"],)}
    for i, L in enumerate(config["layers"]):
        p, m = f"l{i}.", L["mixer"]
        for q in (1, 2) if L["mlp"] else (1,):
            out.update({f"{p}norm{q}": (W,), f"{p}hc{q}.in": (s,), f"{p}hc{q}.out": (s,), f"{p}hc{q}.mix": (s, s)})
        if L["mlp"]:
            ff = L["mlp"]["ff"]
            out.update({p + "mlp.up": (ff, W), p + "mlp.down": (W, ff), p + "mlp.act": (2,)})

        def heads(at, a, values):
            H, G, D, V = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            out.update({at + "q": (H * D, W), at + "k": (G * D, W), at + "q.norm": (D,), at + "k.norm": (D,), at + "g": (H * V, W), at + "o": (W, H * V)})
            if values:
                out[at + "v"] = (G * V, W)
        x = p + "mix."
        if L["type"] == "attention":
            heads(x, m, True)
            out[x + "sink"] = (m["heads"],)
        elif L["type"] == "latent_attention":
            H, D, V, R = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
            out.update({x + "q": (H * D, W), x + "dkv": (R, W), x + "dkv.norm": (R,), x + "uk": (H * D, R), x + "uv": (H * V, R),
                        x + "g": (H * V, W), x + "o": (W, H * V)})
        else:
            heads(x + "left.", m["left"], False)
            n, x = m["right"]["heads"] * m["right"]["dim"], x + "right."
            out.update({x + t: (n, W) for t in ("r", "k", "v", "a", "g")})
            out.update({x + "a.b": (n,), x + "w0": (n,), x + "norm": (n,), x + "w1": (rank, W), x + "w2": (n, rank), x + "o": (W, n)})
    return out


def draw_weights(config, seed, rank, long_memory=False):
    """name -> float32 array, gains near one.  `long_memory`: decays near one and small removal rates."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in sorted(tensor_shapes(config, rank).items()):
        leaf = name.split(".")[-1]
        if name == "embed":
            a = rng.normal(0.0, 1.0, shape)
        elif leaf in ("norm1", "norm2") or name == "final.norm":                     # stored around zero
            a = rng.normal(0.0, 0.1, shape)
        elif leaf == "norm":                                                         # plain weights
            a = rng.normal(1.0, 0.1, shape)
        elif ".hc" in name and leaf == "mix":
            a = 0.8 * np.eye(shape[0]) + rng.normal(0.0, 0.25 / shape[0], shape)
        elif ".hc" in name:
            a = rng.normal(0.7, 0.3, shape) if leaf == "in" else rng.normal(0.9, 0.3, shape)
        elif leaf == "w0":
            a = np.full(shape, -6.0) if long_memory else rng.normal(-1.0, 1.5, shape)
        elif name.endswith("a.b"):
            a = np.full(shape, -4.0) if long_memory else rng.normal(0.0, 1.0, shape)
        elif leaf == "act":
            a = rng.normal(-0.5, 0.5, shape)
        elif leaf == "sink":
            a = rng.normal(0.5, 1.0, shape)
        else:                                                                        # a matrix [out, in]
            a = rng.normal(0.0, 1.0 / np.sqrt(shape[-1]), shape)
        out[name] = a.astype(np.float32)
    return out


def write_model(folder, config, weights, dtype=torch.float32):
    """config.json and model.safetensors with these weights, stored in `dtype`."""
    from litinfer_amd.weights.safetensors_io import write_safetensors
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(config))
    write_safetensors(folder / "model.safetensors", ((n, torch.from_numpy(a).to(dtype)) for n, a in sorted(weights.items())),
                      metadata={"format": "pt"})
    return folder


def stored(weights, dtype):
    """The weights as a checkpoint of `dtype` holds them, float64."""
    return {n: torch.from_numpy(a).to(dtype).to(torch.float64).numpy() for n, a in weights.items()}


def random_config(seed):
    """(configuration, rank): every size, the order of layers, the loop, the windows and the constants vary."""
    rng = np.random.default_rng(1000 + seed)
    pick = lambda *xs: xs[int(rng.integers(0, len(xs)))]
    layers = []
    for _ in range(int(rng.integers(2, 6))):
        ff, kv, dim = pick(None, 24, 100, 264, 500), pick(1, 2, 3), pick(8, 12, 32, 64, 128)
        kind = pick("attention", "latent", "parallel", "parallel")
        if kind == "attention":
            dims = pick(*[d for d in (2, 4, 8, 32, 64) if d <= dim])
            layers.append(attention(kv * pick(1, 2, 5), kv, dim, dim if dim >= 64 else pick(8, 20, 64), float(rng.uniform(0.5, 1.5)) / dim ** 0.5,
                                    pick(50.0, 3000.0, 1e5), dims, ff))
        elif kind == "latent":
            layers.append(latent(pick(1, 3, 4, 8), pick(8, 16, 32, 64), pick(8, 24, 32, 64), pick(16, 40, 64, 128, 256), float(rng.uniform(0.1, 0.4)), ff))
        else:
            layers.append(parallel((kv * pick(1, 2, 4), kv, dim, float(rng.uniform(0.5, 1.5)) / dim ** 0.5, pick(1, 2, 7, 16, 31, 64, 100)),
                                   (pick(1, 2, 3, 6), pick(4, 8, 10, 16, 24, 32, 64, 96, 128)), float(rng.uniform(0.3, 1.5)), float(rng.uniform(0.3, 1.5)), ff))
    cfg = {"architecture": "Dimelix", "vocab": pick(61, 200, 450, 515), "width": pick(48, 72, 96, 128, 200, 256), "norm": {"eps": pick(1e-6, 1e-5, 1e-3)},
           "streams": int(rng.integers(1, 7)), "embedding": {"scale": float(rng.uniform(0.5, 4.0))}, "layers": layers}
    if rng.random() < 0.7:
        cfg["logit_softcap"] = pick(5.0, 20.0, 50.0)
    if rng.random() < 0.7:
        start = int(rng.integers(0, len(layers)))
        cfg["loop"] = {"start": start, "stop": int(rng.integers(start + 1, len(layers) + 1)), "times": int(rng.integers(1, 4))}
    return cfg, pick(2, 5, 8, 16, 24, 40)
