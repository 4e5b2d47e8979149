"""Tiny Besorax configurations and weights for the tests, made here: sizes that differ in everything from each other, and
weights with gains near one, so that every mechanism moves the logits (the framework's own random weights are N(0, 0.02):
a mixer's fault would hardly show through them)."""
import json
from pathlib import Path

import numpy as np
import torch


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(ff, experts, top, shared):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}, **({"shared": {"ff": shared}} if shared else {})}


def lightning(heads, dim, vdim, decay, mlp):
    return {"type": "lightning", "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}}


def attention(heads, kv_heads, dim, vdim, scale, base, dims, chunk, mlp, kv_from=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"base": base, "dims": dims},
                      "mask": {"size": chunk}, **({"kv_from": kv_from} if kv_from is not None else {})}}


def latent(heads, dim, rot_dim, vdim, kv_rank, q_rank, scale, base, mlp):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale,
                      "rot": {"base": base, "dims": rot_dim}}}


# A: small odd sizes; keys of layer 1 read twice, once with a longer and once with a shorter chunk that does not divide it;
# three choices among five experts; a layer without feed-forward
CONFIG_A = {"architecture": "Besorax", "vocab": 211, "width": 84, "norm": {"eps": 1e-4}, "residual_mult": 0.7, "embedding": {"scale": 1.6},
            "layers": [lightning(3, 12, 20, (0.4, 0.93, 0.998), moe(36, 5, 3, 28)),
                       attention(6, 2, 20, 12, 0.3, 900.0, 8, 13, dense(100, 0.9)),
                       attention(6, 2, 20, 12, 0.4, 900.0, 8, 30, None, kv_from=1),
                       latent(3, 20, 6, 28, 24, 36, 0.25, 5000.0, moe(20, 3, 1, None)),
                       attention(6, 2, 20, 12, 0.25, 900.0, 8, 7, moe(24, 4, 2, 60), kv_from=1),
                       lightning(2, 10, 6, (0.75, 0.5), dense(40, 2.5))]}
# B: one kv head, rotation of whole heads, chunks of one token and of a page, the residual factor absent, wide values
CONFIG_B = {"architecture": "Besorax", "vocab": 300, "width": 120, "norm": {"eps": 1e-6}, "embedding": {"scale": 2.3},
            "layers": [attention(8, 1, 16, 48, 0.25, 1e6, 16, 1, dense(136, 7.0)), lightning(5, 8, 24, (0.99, 0.2, 0.95, 0.6, 1.0), dense(56, 1.2)),
                       latent(5, 8, 4, 24, 48, 20, 0.4, 100.0, moe(48, 7, 2, 16)), attention(4, 4, 12, 12, 0.35, 50.0, 2, 16, moe(52, 2, 2, 44))]}
# C: sizes that reach the matrix-core kernels: heads of 64 and 128 columns, latent rows of 160 and 192 columns of which 128 are
# values, states of 64 x 64 and 128 x 128 values, widths in multiples of 64, experts in multiples of 32
CONFIG_C = {"architecture": "Besorax", "vocab": 420, "width": 256, "norm": {"eps": 1e-5}, "residual_mult": 0.5, "embedding": {"scale": 1.0},
            "layers": [latent(8, 64, 32, 32, 128, 96, 0.1, 8000.0, moe(96, 8, 2, 160)), lightning(2, 128, 128, (0.97, 0.8), dense(512, 1.0)),
                       attention(8, 2, 128, 128, 0.09, 4e4, 64, 48, moe(64, 6, 2, 128)), latent(4, 32, 64, 64, 128, 160, 0.12, 300.0, dense(320, 3.0)),
                       attention(4, 2, 64, 64, 0.125, 5000.0, 32, 100, moe(128, 4, 1, None)), lightning(4, 64, 64, (0.9, 0.99, 0.7, 0.999), moe(32, 16, 4, 64)),
                       attention(4, 2, 64, 64, 0.15, 5000.0, 32, 64, dense(256, 1.6), kv_from=4)]}
# D: ones everywhere: one head, one expert, two rotated columns, one layer of each kind
CONFIG_D = {"architecture": "Besorax", "vocab": 64, "width": 40, "norm": {"eps": 1e-6}, "residual_mult": 1.0, "embedding": {"scale": 1.0},
            "layers": [latent(1, 8, 2, 8, 16, 8, 0.35, 100.0, moe(16, 1, 1, 8)), attention(1, 1, 8, 8, 0.35, 100.0, 2, 5, dense(24, 1.0)),
                       lightning(1, 16, 16, (0.9,), None)]}
# name -> (configuration, page size, seed)
CASES = {"A": (CONFIG_A, 8, 51), "B": (CONFIG_B, 16, 52), "C": (CONFIG_C, 32, 53), "D": (CONFIG_D, 4, 54)}


def tensor_shapes(config):
    """name -> shape of every tensor, from the configuration, written out here again."""
    W, out = config["width"], {"embed": (config["vocab"], config["width"]), "head": (config["vocab"], config["width"])}

    def norm(name):
        out.update({name: (W,), name + ".b": (W,), name + ".alpha": ()})
    norm("final.norm")
    for i, L in enumerate(config["layers"]):
        p, m = f"l{i}.", L["mixer"]
        x = p + "mix."
        norm(p + "norm1")
        H, V = m["heads"], m["vdim"]
        if L["type"] == "lightning":
            D = m["dim"]
            out.update({x + "q": (H * D, W), x + "k": (H * D, W), x + "v": (H * V, W), x + "g": (H * V, W), x + "norm": (H * V,), x + "o": (W, H * V)})
        elif L["type"] == "attention":
            G, D = m["kv_heads"], m["dim"]
            out.update({x + "q": (H * D, W), x + "sink": (H,), x + "o": (W, H * V)})
            if m.get("kv_from") is None:
                out.update({x + "k": (G * D, W), x + "v": (G * V, W)})
        else:
            D, R, K, Q = m["dim"], m["rot_dim"], m["kv_rank"], m["q_rank"]
            out.update({x + "dq": (Q, W), x + "dq.norm": (Q,), x + "uq": (H * (D + R), Q), x + "dkv": (K + R, W), x + "dkv.norm": (K,),
                        x + "uk": (H * D, K), x + "uv": (H * V, K), x + "sink": (H,), x + "o": (W, H * V)})
        mlp = L["mlp"]
        if mlp is None:
            continue
        norm(p + "norm2")
        y = p + "mlp."
        if mlp["kind"] == "dense":
            out.update({y + "gate": (mlp["ff"], W), y + "up": (mlp["ff"], W), y + "down": (W, mlp["ff"])})
            continue
        out[y + "router"] = (mlp["router"]["experts"], W)
        pairs = [(f"e{e}.", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])]
        if mlp.get("shared"):
            pairs.append(("shared.", mlp["shared"]["ff"]))
        for e, ff in pairs:
            out.update({y + e + "up": (ff, W), y + e + "down": (W, ff)})
    return out


def draw_weights(config, seed):
    """name -> float32 array, gains near one."""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in sorted(tensor_shapes(config).items()):
        leaf = name.split(".")[-1]
        if name == "embed":
            a = rng.normal(0.0, 1.0, shape)
        elif leaf == "alpha":
            a = np.asarray(rng.uniform(0.4, 1.3))
        elif leaf == "b":
            a = rng.normal(0.0, 0.2, shape)
        elif leaf in ("norm", "norm1", "norm2"):
            a = rng.normal(1.0, 0.2, shape)
        elif leaf == "sink":
            a = rng.normal(0.5, 1.0, shape)
        elif leaf == "router":
            a = rng.normal(0.0, 2.0 / np.sqrt(shape[-1]), shape)             # (scores far apart: few close calls)
        else:                                                                # a matrix [out, in]
            a = rng.normal(0.0, 1.0 / np.sqrt(shape[-1]), shape)
        out[name] = np.asarray(a).astype(np.float32)
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
    """Every size, the order of layers, who reads whose keys, the chunks, the feed-forwards and the constants vary."""
    rng = np.random.default_rng(2000 + seed)
    pick = lambda *xs: xs[int(rng.integers(0, len(xs)))]

    def ff():
        kind = pick("none", "dense", "moe", "moe")
        if kind == "none":
            return None
        if kind == "dense":
            return dense(pick(24, 100, 264, 512), float(rng.uniform(0.5, 7.0)))
        n = pick(1, 2, 3, 5, 8, 17)
        return moe(pick(12, 32, 50, 64, 96), n, int(rng.integers(1, min(n, 4) + 1)), pick(None, 16, 33, 64, 128))
    layers, owners = [], []
    for i in range(int(rng.integers(2, 7))):
        kind = pick("lightning", "attention", "attention", "latent")
        if kind == "lightning":
            h = pick(1, 2, 3, 6)
            layers.append(lightning(h, pick(4, 8, 10, 16, 32, 64, 96, 128), pick(4, 7, 16, 24, 64, 128),
                                    [float(d) for d in rng.choice([0.0, 0.3, 0.6, 0.9, 0.97, 0.995, 1.0], h)], ff()))
        elif kind == "latent":
            layers.append(latent(pick(1, 3, 4, 8), pick(8, 16, 32, 64), pick(2, 4, 16, 32, 64), pick(8, 24, 32, 64), pick(16, 40, 64, 128),
                                 pick(8, 20, 64, 100), float(rng.uniform(0.1, 0.4)), pick(50.0, 3000.0, 1e5), ff()))
        elif owners and rng.random() < 0.5:
            j = pick(*owners)
            m = layers[j]["mixer"]
            layers.append(attention(m["heads"], m["kv_heads"], m["dim"], m["vdim"], float(rng.uniform(0.5, 1.5)) / m["dim"] ** 0.5, m["rot"]["base"],
                                    m["rot"]["dims"], pick(1, 2, 7, 16, 31, 64, 100), ff(), kv_from=j))
        else:
            kv, dim = pick(1, 2, 3), pick(8, 12, 32, 64, 128)
            dims = pick(*[d for d in (2, 4, 8, 32, 64) if d <= dim])
            owners.append(i)
            layers.append(attention(kv * pick(1, 2, 5), kv, dim, dim if dim >= 64 else pick(8, 20, 64), float(rng.uniform(0.5, 1.5)) / dim ** 0.5,
                                    pick(50.0, 3000.0, 1e5), dims, pick(1, 2, 7, 16, 31, 64, 100), ff()))
    cfg = {"architecture": "Besorax", "vocab": pick(61, 200, 450, 515), "width": pick(48, 72, 96, 128, 200, 256), "norm": {"eps": pick(1e-6, 1e-5, 1e-3)},
           "residual_mult": float(rng.uniform(0.2, 1.2)), "embedding": {"scale": float(rng.uniform(0.5, 4.0))}, "layers": layers}
    return cfg
