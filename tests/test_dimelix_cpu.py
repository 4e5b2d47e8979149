"""Dimelix without a GPU: pins of the plain implementation (tests/plain_dimelix.py) against closed forms written another
way, the typed configuration and its errors, the model as data (order, tensors), and what the entries ask of the cache."""
import copy
import math

import numpy as np
import pytest
import torch

import dimelix_cases as cases
import plain_dimelix as plain


# ------------------------------------------------------------------------------------- the plain implementation
def test_rotation_of_neighbouring_pairs_is_a_complex_multiplication():
    rng = np.random.default_rng(0)
    v, pos = rng.normal(size=(5, 2, 9)), np.array([0, 1, 7, 100, 3])
    out = plain.rotate_pairs(v, pos, 40.0, 6)
    z = (v[..., 0:6:2] + 1j * v[..., 1:6:2]) * np.exp(1j * pos[:, None, None] * 40.0 ** (-2.0 * np.arange(3) / 6))
    assert np.allclose(out[..., 0:6:2], z.real) and np.allclose(out[..., 1:6:2], z.imag) and np.array_equal(out[..., 6:], v[..., 6:])


def test_softmax_with_sink_window_and_slopes_by_hand():
    rng = np.random.default_rng(1)
    T, D, V = 9, 4, 3
    q, k, v = rng.normal(size=(T, 2, D)), rng.normal(size=(T, 1, D)), rng.normal(size=(T, 1, V))
    sink, slopes = np.array([0.4, -1.0]), [0.5, 0.03]
    out = plain.attend(q, k, v, 0.7, sink=sink, window=4, slopes=slopes)
    for h in range(2):
        for i in range(T):
            seen = [j for j in range(T) if 0 <= i - j < 4]
            e = {j: math.exp(0.7 * float(q[i, h] @ k[j, 0]) - slopes[h] * (i - j)) for j in seen}
            want = sum(e[j] * v[j, 0] for j in seen) / (sum(e.values()) + math.exp(sink[h]))
            assert np.allclose(out[i, h], want)
    assert np.allclose(plain.attend(q, k, v, 0.7, window=1)[:, 0], v[:, 0])           # a window of one: the token itself
    assert np.abs(plain.attend(q, k, v, 0.7, sink=np.array([60.0, 60.0]))).max() < 1e-12


def test_channel_delta_rule_as_a_product_of_matrices():
    rng = np.random.default_rng(2)
    T, D = 7, 5
    r, k, v = (rng.normal(size=(T, 1, D)) for _ in range(3))
    w, a = rng.uniform(0.5, 1.0, (T, 1, D)), rng.uniform(0.0, 1.0, (T, 1, D))
    out = plain.channel_delta_rule(r, k, v, w, a)
    S = np.zeros((D, D))
    for t in range(T):
        u = k[t, 0] / math.sqrt(k[t, 0] @ k[t, 0] + 1e-6)
        A = np.diag(w[t, 0]) - (a[t, 0] * u)[:, None] @ u[None]
        S = A @ S + k[t, 0][:, None] @ v[t, 0][None]
        assert np.allclose(out[t, 0], S.T @ r[t, 0])


def test_channel_delta_rule_stores_removes_and_decays():
    """No decay and full removal: a second write under the same key replaces the first; half removal keeps half; a decay
    acts on the channel it belongs to only; a key at a right angle removes nothing."""
    e1, e2 = np.array([1.0, 0.0]), np.array([0.0, 1.0])
    one, v1, v2 = np.ones(2), np.array([2.0, -1.0]), np.array([0.5, 4.0])
    run = lambda r, k, v, w, a: plain.channel_delta_rule(*(np.stack(x)[:, None] for x in (r, k, v, w, a)))[:, 0]
    o = run([e1, e1], [e1, e1], [v1, v2], [one, one], [one, one])
    assert np.allclose(o, [v1, v2], atol=1e-5)
    o = run([e1, e1], [e1, e1], [v1, v2], [one, one], [one, 0.5 * one])
    assert np.allclose(o[1], 0.5 * v1 + v2, atol=1e-5)
    o = run([e1, e1], [e1, e2], [v1, v2], [one, np.array([0.25, 1.0])], [one, one])
    assert np.allclose(o[1], 0.25 * v1, atol=1e-5)
    o = run([e2, e2], [e2, e1], [v1, v2], [one, np.array([0.25, 1.0])], [one, one])
    assert np.allclose(o[1], v1, atol=1e-5)
    assert np.allclose(run([e1], [3.0 * e1], [v1], [one], [one])[0], 3.0 * v1)        # the key that is written is not normed


def test_decays_and_removal_rates_of_the_mixer():
    """With low-rank weights of zero the decay is exp(-exp(-1/2) / 2) for w0 = 0, near one for w0 -> -inf, and at least
    exp(-exp(-1/2)) whatever w0."""
    sig = lambda z: 1.0 / (1.0 + math.exp(-z))
    assert abs(math.exp(-plain.DECAY_FACTOR * sig(0.0)) - 0.7384) < 1e-4 and abs(math.exp(-plain.DECAY_FACTOR) - 0.5452) < 1e-4
    cfg = cases.CONFIG_D
    W = {n: x.astype(np.float64) for n, x in cases.draw_weights(cfg, 5, 1).items()}
    p, m = "l2.mix.right.", cfg["layers"][2]["mixer"]["right"]
    W[p + "w2"][:] = 0.0
    W[p + "w0"][:] = -60.0                   # no decay,
    W[p + "a"][:], W[p + "a.b"][:] = 0.0, -60.0          # no removal: plain linear attention
    h = np.random.default_rng(3).normal(size=(6, cfg["width"]))
    r, k, v = (h @ W[p + x].T for x in "rkv")
    o = np.stack([sum((r[t] @ k[j]) * v[j] for j in range(t + 1)) for t in range(6)])
    want = (plain.rms(o, 1e-6) * W[p + "norm"] * plain.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T
    assert np.allclose(plain.channel_delta_mixer(h, W, p, m, 1e-6), want)


def test_xielu_values():
    f = lambda z: float(plain.xielu(np.array(z), 0.0, 0.0))
    ln2 = math.log(2.0)
    assert f(0.0) == 0.0
    assert abs(f(2.0) - (4.0 * ln2 + 1.0)) < 1e-12
    assert abs(f(-1.5) - ((0.5 + ln2) * (math.exp(-1.5) - 1.0 + 1.5) - 0.75)) < 1e-12
    assert abs((f(1e-6) - f(-1e-6)) / 2e-6 - 0.5) < 1e-5                        # smooth at zero, slope 1/2
    assert plain.xielu(np.array(3.0), 1.0, -9.0) == plain.xielu(np.array(3.0), 1.0, 5.0)      # p on one side, q on the other
    assert plain.xielu(np.array(-3.0), 1.0, 0.2) == plain.xielu(np.array(-3.0), -4.0, 0.2)


def test_streams_are_mixed_from_the_old_ones_with_rows_as_sources():
    w = {"h.in": np.array([2.0, -1.0]), "h.out": np.array([0.5, 3.0]), "h.mix": np.array([[1.0, 10.0], [100.0, 0.0]])}
    xs, y = [np.array([1.0]), np.array([2.0])], np.array([4.0])
    assert np.allclose(plain.read_streams(xs, w, "h."), 0.0)
    new = plain.write_streams(xs, y, w, "h.")
    assert np.allclose(new[0], 1.0 * 1 + 100.0 * 2 + 0.5 * 4) and np.allclose(new[1], 10.0 * 1 + 0.0 * 2 + 3.0 * 4)


def test_one_stream_with_ones_is_the_plain_residual_sum():
    cfg = copy.deepcopy(cases.CONFIG_D)
    W = {n: x.astype(np.float64) for n, x in cases.draw_weights(cfg, 6, 2).items()}
    for n in W:
        if ".hc" in n:
            W[n] = np.ones_like(W[n])
    ids, eps = [3, 9, 11, 3], cfg["norm"]["eps"]
    x = W["embed"][ids] * cfg["embedding"]["scale"]
    for i, L in enumerate(cfg["layers"]):
        x = x + plain.mixer(L, plain.offset_norm(x, W[f"l{i}.norm1"], eps), W, f"l{i}.mix.", eps, np.arange(4))
        if L["mlp"]:
            x = x + plain.dense_ff(plain.offset_norm(x, W[f"l{i}.norm2"], eps), W, f"l{i}.mlp.")
    assert np.allclose(plain.forward(cfg, W, ids), plain.head(cfg, W, x))
    assert np.abs(plain.head(cfg, W, x)).max() <= cfg["logit_softcap"]


def test_the_order_of_a_loop():
    assert plain.order(cases.CONFIG_A) == [0, 1, 2, 3, 2, 3] and plain.order(cases.CONFIG_B) == [0, 1, 2]
    assert plain.order(cases.CONFIG_C) == [0, 1, 2, 0, 1, 2, 3, 4]


# ------------------------------------------------------------------------------------------------ configuration
def test_configuration_reads_every_key():
    from litinfer_amd.config import DimelixConfig
    c = DimelixConfig.from_dict(cases.CONFIG_A)
    assert (c.vocab, c.width, c.eps, c.streams, c.embedding_scale, c.logit_softcap, c.loop) == (203, 88, 1e-4, 2, 1.7, 11.0, (2, 4, 2))
    p, a, l = c.layers[0], c.layers[1], c.layers[2]
    assert (p.mixer.left.heads, p.mixer.left.kv_heads, p.mixer.left.dim, p.mixer.left.scale, p.mixer.left.window) == (6, 3, 20, 0.25, 9)
    assert (p.mixer.right.heads, p.mixer.right.dim, p.mixer.left_scale, p.mixer.right_scale, p.ff) == (3, 12, 0.6, 1.1, 100)
    assert (a.mixer.dim, a.mixer.vdim, a.mixer.rot_base, a.mixer.rot_dims, a.ff) == (12, 28, 700.0, 8, 0)
    assert (l.mixer.heads, l.mixer.dim, l.mixer.vdim, l.mixer.kv_rank, l.mixer.scale) == (3, 20, 12, 28, 0.21)
    b = DimelixConfig.from_dict(cases.CONFIG_B)
    assert b.loop is None and b.logit_softcap == 0.0
    d = copy.deepcopy(cases.CONFIG_B)                     # keys that may be absent
    del d["embedding"], d["layers"][0]["mixer"]["kv_heads"], d["layers"][0]["mixer"]["vdim"], d["layers"][1]["mixer"]["left"]["mask"]
    d = DimelixConfig.from_dict(d)
    assert d.embedding_scale == 1.0 and (d.layers[0].mixer.kv_heads, d.layers[0].mixer.vdim) == (8, 16) and d.layers[1].mixer.left.window == 0


@pytest.mark.parametrize("path,value", [
    (("layers", 0, "type"), "delta"), (("layers", 0, "mixer", "left", "kv_heads"), 4), (("layers", 0, "mixer", "left", "vdim"), 16),
    (("layers", 0, "mixer", "right", "dim"), 0), (("layers", 0, "mixer", "left_scale"), None), (("layers", 0, "mixer", "left", "mask", "size"), 0),
    (("layers", 1, "mixer", "rot", "dims"), 7), (("layers", 1, "mixer", "rot", "dims"), 14), (("layers", 1, "mixer", "rot"), None),
    (("layers", 1, "mixer", "rot", "base"), 0), (("layers", 2, "mixer", "kv_rank"), None), (("layers", 2, "mixer", "scale"), "x"),
    (("layers", 2, "mlp", "kind"), "moe"), (("layers", 2, "mlp", "ff"), 0), (("loop", "stop"), 5), (("loop", "times"), 0),
    (("norm", "eps"), -1.0), (("streams",), 0), (("streams",), None), (("vocab",), 0), (("layers",), []), (("logit_softcap",), -2.0)])
def test_configuration_errors(path, value):
    from litinfer_amd.config import ConfigError, DimelixConfig
    cfg = copy.deepcopy(cases.CONFIG_A)
    node = cfg
    for k in path[:-1]:
        node = node[k]
    node[path[-1]] = value
    with pytest.raises(ConfigError):
        DimelixConfig.from_dict(cfg)


def _model(cfg):
    from litinfer_amd.config import architecture_name, lookup
    from litinfer_amd.engine.model import Model
    from litinfer_amd.parts import Runtime
    arch = lookup(architecture_name(cfg))
    spec = arch.model_spec(arch.config_from_dict(cfg))
    spec.validate()
    return spec, Model(spec, Runtime(torch.device("cpu"), torch.float32))


@pytest.mark.parametrize("name", list(cases.CASES))
def test_model_as_data(name):
    cfg, _, _, rank = cases.CASES[name]
    spec, model = _model(cfg)
    assert spec.architecture == "Dimelix" and spec.streams == cfg["streams"] and [e.layer for e in spec.order] == plain.order(cfg)
    assert all(l.block == "hyper" for l in spec.layers) and model.graph_safe
    names, want = model.expected_params(), cases.tensor_shapes(cfg, rank)
    assert set(names) == set(want)
    assert all(names[n].matches(s) for n, s in want.items())
    assert not names["embed"].matches((cfg["vocab"] + 1, cfg["width"]))


def test_a_dimension_that_the_stored_tensor_decides():
    from litinfer_amd.weights.loader import ParamSpec, WeightError, check_entries
    p = ParamSpec((64, 5), free_dims=(0,))
    assert p.matches((3, 5)) and p.matches((64, 5)) and not p.matches((0, 5)) and not p.matches((3, 6)) and not p.matches((3, 5, 1))
    check_entries({"w": p}, {"w": ("BF16", (7, 5))})
    with pytest.raises(WeightError):
        check_entries({"w": p}, {"w": ("BF16", (7, 4))})


def test_low_rank_tensors_that_do_not_fit_each_other_are_refused(tmp_path):
    from litinfer_amd.weights.loader import load_into
    cfg, _, seed, rank = cases.CASES["D"]
    w = cases.draw_weights(cfg, seed, rank)
    w["l2.mix.right.w1"] = np.zeros((3, cfg["width"]), dtype=np.float32)
    _, model = _model(cfg)
    with pytest.raises(ValueError, match="w2 has 1 columns"):
        load_into(model, cases.write_model(tmp_path / "m", cfg, w))


def test_weights_load_as_the_parts_hold_them(tmp_path):
    from litinfer_amd.weights.loader import load_into
    cfg, _, seed, rank = cases.CASES["A"]
    w = cases.draw_weights(cfg, seed, rank)
    spec, model = _model(cfg)
    assert load_into(model, cases.write_model(tmp_path / "m", cfg, w), strict=True) == []
    b = model.layers[0]
    assert np.allclose(b.reader1.weights.numpy(), w["l0.hc1.in"]) and np.allclose(b.mix2.numpy(), w["l0.hc2.mix"])
    assert np.allclose(b.norm1.weight.numpy(), 1.0 + w["l0.norm1"])
    assert b.mixer.right.rank == rank and np.allclose(b.mixer.left.slopes, [2.0 ** (-8.0 * (h + 1) / 6) for h in range(6)])
    assert abs(b.ffn.sp - np.log1p(np.exp(float(w["l0.mlp.act"][0])))) < 1e-6
    assert abs(b.ffn.sq - 0.5 - np.log1p(np.exp(float(w["l0.mlp.act"][1])))) < 1e-6
    assert model.layers[3].ffn is None and model.layers[3].reader2 is None


def test_what_the_entries_ask_of_the_cache():
    from litinfer_amd.parts import needs_of
    _, model = _model(cases.CONFIG_A)
    needs, sources = model.cache_needs()
    assert sources == [None] * 6 and needs[2] == needs[4] and needs[3] == needs[5]         # each pass keeps its own
    paged, states = needs_of(needs[0])
    assert paged.window == 9 and [(t.name, t.shape) for t in paged.tensors] == [("k", (3, 20)), ("v", (3, 20))]
    assert [(s.name, s.shape, s.dtype) for s in states] == [("channel_delta", (3, 12, 12), torch.float32)]
    paged, states = needs_of(needs[1])
    assert paged.window == 0 and [t.shape for t in paged.tensors] == [(2, 12), (2, 28)] and not states
    paged, states = needs_of(needs[2])
    assert [(t.name, t.shape) for t in paged.tensors] == [("latent", (1, 28))] and not states


def test_what_the_parts_refuse():
    from litinfer_amd.config import PartSpec
    from litinfer_amd.parts import Runtime, build_part
    rt = Runtime(torch.device("cpu"), torch.float32)
    att = {"hidden_size": 8, "num_heads": 2, "head_dim": 4, "qk_norm": "heads"}
    for bad in ({"keys_are_values": True, "value_dim": 8}, {"keys_are_values": True, "qk_norm": True}, {"keys_are_values": True, "bias": True},
                {"slopes": [0.5]}, {"head_gate": True, "column_gate": True}):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("masked_attention", "x.", {**att, **bad}), rt)
    with pytest.raises(ValueError):
        build_part("mixer", PartSpec("channel_delta", "x.", {"hidden_size": 8, "num_heads": 1, "head_dim": 300}), rt)
    norm = PartSpec("rmsnorm", "x.", {"size": 8, "eps": 1e-5})
    with pytest.raises(ValueError):
        build_part("block", PartSpec("hyper"), rt, parts={"hyper": PartSpec("hyper", "x.", {"streams": 17}), "norm1": norm,
                                                         "mixer": PartSpec("masked_attention", "x.", att)})
    from litinfer_amd.parts import HyperStream
    with pytest.raises(NotImplementedError):
        HyperStream(torch.zeros(2, 8), None, 3).tensor()
