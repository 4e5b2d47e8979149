"""Besorax without a GPU: pins of the plain implementation (tests/plain_besorax.py) against closed forms written another
way, the typed configuration and its errors, the model as data (order, tensors), what the entries ask of the cache, pages
that go back at a chunk's end, and what parts refuse."""
import copy
import math

import numpy as np
import pytest
import torch

import besorax_cases as cases
import plain_besorax as plain


# ------------------------------------------------------------------------------------- the plain implementation
def test_rotation_of_neighbouring_pairs_is_a_complex_multiplication():
    rng = np.random.default_rng(0)
    v, pos = rng.normal(size=(5, 2, 9)), np.array([0, 1, 7, 100, 3])
    out = plain.rotate_pairs(v, pos, 40.0, 6)
    z = (v[..., 0:6:2] + 1j * v[..., 1:6:2]) * np.exp(1j * pos[:, None, None] * 40.0 ** (-2.0 * np.arange(3) / 6))
    assert np.allclose(out[..., 0:6:2], z.real) and np.allclose(out[..., 1:6:2], z.imag) and np.array_equal(out[..., 6:], v[..., 6:])


def test_softmax_with_a_sink_inside_a_chunk_by_hand():
    rng = np.random.default_rng(1)
    T, D, V = 11, 4, 3
    q, k, v = rng.normal(size=(T, 2, D)), rng.normal(size=(T, 1, D)), rng.normal(size=(T, 1, V))
    sink = np.array([0.4, -1.0])
    out = plain.attend(q, k, v, 0.7, sink, chunk=4)
    for h in range(2):
        for i in range(T):
            seen = [j for j in range(T) if j <= i and j // 4 == i // 4]
            e = {j: math.exp(0.7 * float(q[i, h] @ k[j, 0])) for j in seen}
            assert np.allclose(out[i, h], sum(e[j] * v[j, 0] for j in seen) / (sum(e.values()) + math.exp(sink[h])))
    low = np.array([-80.0, -80.0])
    assert np.allclose(plain.attend(q, k, v, 0.7, low, chunk=1)[:, 0], v[:, 0])                # a chunk of one: the token itself
    assert np.allclose(plain.attend(q, k, v, 0.7, sink, chunk=64), plain.attend(q, k, v, 0.7, sink))     # one chunk: all keys
    assert np.abs(plain.attend(q, k, v, 0.7, np.array([60.0, 60.0]))).max() < 1e-12


def test_decayed_sums_by_their_closed_form():
    rng = np.random.default_rng(2)
    T, D, V, a = 9, 5, 3, [0.8, 1.0]
    q, k, v = rng.normal(size=(T, 2, D)), rng.normal(size=(T, 2, D)), rng.normal(size=(T, 2, V))
    out = plain.decayed_sum(q, k, v, a)
    for h in range(2):
        for t in range(T):
            assert np.allclose(out[t, h], sum(a[h] ** (t - j) * (q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1)))
    none = plain.decayed_sum(q, k, v, [0.0, 0.0])                                   # nothing is remembered
    assert np.allclose(none[4, 0], (q[4, 0] @ k[4, 0]) * v[4, 0])


def test_the_lightning_mixer_norms_all_heads_together_and_gates_by_a_sigmoid():
    cfg = cases.CONFIG_A
    W = {n: x.astype(np.float64) for n, x in cases.draw_weights(cfg, 5).items()}
    p, m = "l0.mix.", cfg["layers"][0]["mixer"]
    h = np.random.default_rng(3).normal(size=(4, cfg["width"]))
    z = lambda x: (h @ W[p + x].T) / (1.0 + np.exp(-(h @ W[p + x].T)))
    o = np.zeros((4, 60))
    for t in range(4):
        for hh in range(3):
            for j in range(t + 1):
                o[t, 20 * hh:20 * hh + 20] += (m["decay"][hh] ** (t - j) * (z("q")[t, 12 * hh:12 * hh + 12] @ z("k")[j, 12 * hh:12 * hh + 12])
                                               * z("v")[j, 20 * hh:20 * hh + 20])
    o = o / np.sqrt((o ** 2).mean(axis=1, keepdims=True) + 1e-4) * W[p + "norm"]
    assert np.allclose(plain.lightning_mixer(h, W, p, m, 1e-4), (o / (1.0 + np.exp(-(h @ W[p + "g"].T)))) @ W[p + "o"].T)


def test_the_norm_has_no_statistics():
    w = {"n": np.array([2.0, 1.0]), "n.b": np.array([0.5, -1.0]), "n.alpha": np.array(0.3)}
    x = np.array([[4.0, -7.0], [4.0, 100.0]])
    out = plain.tanh_norm(x, w, "n")
    assert np.allclose(out[:, 0], 2.0 * math.tanh(1.2) + 0.5) and np.allclose(out[1, 1], 0.0)      # a column does not see the others
    assert np.allclose(out[0, 1], math.tanh(-2.1) - 1.0)


def test_clamped_feed_forward_and_gelu_values():
    eye = {"m.gate": np.eye(3), "m.up": np.eye(3)[[2, 0, 1]], "m.down": np.eye(3)}
    sg = lambda z: 1.0 / (1.0 + math.exp(-z))
    out = plain.dense_ff(np.array([[3.0, -5.0, 0.5]]), eye, "m.", 2.0)[0]
    assert np.allclose(out, [2.0 * sg(3.404) * 1.5, -5.0 * sg(-8.51) * 3.0, 0.5 * sg(0.851) * -1.0])
    assert np.allclose(plain.gelu(np.array([0.0, 1.0, -1.0, 3.0])), [0.0, 0.8413447460685429, -0.15865525393145707, 2.99595030590511])


def test_a_choices_weight_multiplies_the_experts_input():
    cfg = cases.CONFIG_A
    W = {n: x.astype(np.float64) for n, x in cases.draw_weights(cfg, 5).items()}
    h = np.random.default_rng(4).normal(size=(6, cfg["width"]))
    idx, wt = plain.route(h, W, "l0.mlp.", 3)
    s = 1.0 / (1.0 + np.exp(-h @ W["l0.mlp.router"].T))
    y = plain.routed_ff(h, W, "l0.mlp.", 3, True)
    for t in range(6):
        best = sorted(range(5), key=lambda e: -s[t, e])[:3]
        assert list(idx[t]) == best and np.allclose(wt[t], s[t, best])               # (not divided by their sum)
        want = plain.gelu(W["l0.mlp.shared.up"] @ h[t]) @ W["l0.mlp.shared.down"].T
        for e in best:
            want = want + W[f"l0.mlp.e{e}.down"] @ plain.gelu(s[t, e] * (W[f"l0.mlp.e{e}.up"] @ h[t]))
        assert np.allclose(y[t], want)


def test_shared_keys_are_the_owners_and_the_first_token_sees_itself():
    cfg = copy.deepcopy(cases.CONFIG_A)
    W = {n: x.astype(np.float64) for n, x in cases.draw_weights(cfg, 6).items()}
    a = plain.forward(cfg, W, [3, 9, 11])
    assert np.allclose(a[0], plain.forward(cfg, W, [3, 1, 2])[0])
    W["l1.mix.k"] = W["l1.mix.k"] * 3.0                                              # moves every layer that reads them
    cfg["layers"][1]["mlp"] = None
    streams, other = [], []
    plain.forward(cfg, W, [3, 9, 11], streams)
    W["l1.mix.o"] = W["l1.mix.o"] * 0.0                                              # layer 1 adds nothing, layer 2 still reads its keys
    b = plain.forward(cfg, W, [3, 9, 11], other)
    W["l1.mix.v"] = W["l1.mix.v"] * 0.0
    assert np.allclose(other[1], other[0]) and np.abs(plain.forward(cfg, W, [3, 9, 11]) - b).max() > 1e-2


# ------------------------------------------------------------------------------------------------ configuration
def test_configuration_reads_every_key():
    from litinfer_amd.config import BesoraxConfig
    c = BesoraxConfig.from_dict(cases.CONFIG_A)
    assert (c.vocab, c.width, c.eps, c.residual_mult, c.embedding_scale) == (211, 84, 1e-4, 0.7, 1.6)
    l, a, s, z = c.layers[0], c.layers[1], c.layers[2], c.layers[3]
    assert (l.mixer.heads, l.mixer.dim, l.mixer.vdim, l.mixer.decay) == (3, 12, 20, (0.4, 0.93, 0.998))
    assert (l.mlp.kind, l.mlp.ff, l.mlp.experts, l.mlp.top, l.mlp.shared_ff) == ("moe", 36, 5, 3, 28)
    assert (a.mixer.heads, a.mixer.kv_heads, a.mixer.dim, a.mixer.vdim, a.mixer.scale, a.mixer.rot_base, a.mixer.rot_dims, a.mixer.chunk,
            a.mixer.kv_from) == (6, 2, 20, 12, 0.3, 900.0, 8, 13, None)
    assert (a.mlp.kind, a.mlp.ff, a.mlp.limit) == ("dense", 100, 0.9)
    assert (s.mixer.kv_from, s.mixer.chunk, s.mlp) == (1, 30, None) and c.layers[3].mlp.shared_ff == 0
    assert (z.mixer.heads, z.mixer.dim, z.mixer.rot_dim, z.mixer.vdim, z.mixer.kv_rank, z.mixer.q_rank, z.mixer.scale, z.mixer.rot_base) == \
        (3, 20, 6, 28, 24, 36, 0.25, 5000.0)
    d = copy.deepcopy(cases.CONFIG_B)                     # keys that may be absent
    del d["embedding"], d["layers"][0]["mixer"]["mask"], d["layers"][0]["mixer"]["rot"], d["layers"][3]["mixer"]["kv_heads"]
    del d["layers"][1]["mixer"]["vdim"]
    d = BesoraxConfig.from_dict(d)
    assert (d.embedding_scale, d.residual_mult) == (1.0, 1.0) and (d.layers[0].mixer.chunk, d.layers[0].mixer.rot_dims) == (0, 0)
    assert d.layers[3].mixer.kv_heads == 4 and d.layers[1].mixer.vdim == 8


@pytest.mark.parametrize("path,value", [
    (("layers", 0, "type"), "delta"), (("layers", 0, "mixer", "decay"), [0.5, 0.5]), (("layers", 0, "mixer", "decay"), 0.9),
    (("layers", 0, "mixer", "dim"), 0), (("layers", 0, "mlp", "kind"), "gated"), (("layers", 0, "mlp", "router", "top"), 6),
    (("layers", 0, "mlp", "expert"), None), (("layers", 0, "mlp", "shared", "ff"), 0), (("layers", 1, "mlp", "limit"), 0),
    (("layers", 1, "mlp", "limit"), None), (("layers", 1, "mixer", "kv_heads"), 4), (("layers", 1, "mixer", "mask", "size"), 0),
    (("layers", 1, "mixer", "rot", "dims"), 22), (("layers", 1, "mixer", "rot", "dims"), 3), (("layers", 1, "mixer", "scale"), None),
    (("layers", 2, "mixer", "kv_from"), 2), (("layers", 2, "mixer", "kv_from"), 0), (("layers", 4, "mixer", "kv_from"), 2),
    (("layers", 2, "mixer", "kv_from"), -1), (("layers", 2, "mixer", "kv_heads"), 3), (("layers", 2, "mixer", "rot", "base"), 901.0),
    (("layers", 3, "mixer", "rot", "dims"), 4), (("layers", 3, "mixer", "rot"), None), (("layers", 3, "mixer", "q_rank"), None),
    (("residual_mult",), 0), (("norm", "eps"), -1.0), (("vocab",), 0), (("layers",), [])])
def test_configuration_errors(path, value):
    from litinfer_amd.config import BesoraxConfig, ConfigError
    cfg = copy.deepcopy(cases.CONFIG_A)
    node = cfg
    for k in path[:-1]:
        node = node[k]
    node[path[-1]] = value
    with pytest.raises(ConfigError):
        BesoraxConfig.from_dict(cfg)


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
    cfg = cases.CASES[name][0]
    spec, model = _model(cfg)
    assert spec.architecture == "Besorax" and [e.layer for e in spec.order] == list(range(len(cfg["layers"])))
    assert [e.cache_from for e in spec.order] == [L["mixer"].get("kv_from") for L in cfg["layers"]]
    assert spec.residual_scale == cfg.get("residual_mult", 1.0)
    assert {n: tuple(p.shape) for n, p in model.expected_params().items()} == {n: tuple(s) for n, s in cases.tensor_shapes(cfg).items()}


def test_what_the_entries_ask_of_the_cache():
    """An owner keeps its pages as long as any reader sees them: the chunks 13, 30 and 7 do not divide one another, so the
    last 30 positions stay; chunks of which one divides the other stay chunks."""
    from litinfer_amd.parts import PagedNeed, needs_of
    needs, sources = _model(cases.CONFIG_A)[1].cache_needs()
    assert sources == [None, None, 1, None, 1, None]
    paged, states = needs_of(needs[0])
    assert paged is None and [(s.name, s.shape, s.dtype) for s in states] == [("lightning", (3, 12, 20), torch.float32)]
    assert isinstance(needs[1], PagedNeed) and [(t.name, t.shape) for t in needs[1].tensors] == [("k", (2, 20)), ("v", (2, 12))]
    assert (needs[1].window, needs[1].chunk, needs[1].reach) == (30, 0, 30)
    assert [(t.name, t.shape) for t in needs[3].tensors] == [("latent", (1, 30))] and needs[3].reach == 0
    k = needs[1].tensors
    assert PagedNeed(k, chunk=8).covering(PagedNeed(k, chunk=24)) == PagedNeed(k, chunk=24)
    assert PagedNeed(k, chunk=8).covering(PagedNeed(k)) == PagedNeed(k) and PagedNeed(k).covering(PagedNeed(k, chunk=8)) == PagedNeed(k)
    assert PagedNeed(k, window=5, keep_first=2).covering(PagedNeed(k, chunk=8)) == PagedNeed(k, window=8, keep_first=2)
    with pytest.raises(ValueError):
        PagedNeed(k).covering(PagedNeed(k[:1]))


def test_pages_go_back_when_a_chunk_ends():
    """Chunks of 10 positions on pages of 4: what a request holds after every committed token is exactly the pages from
    the chunk's first position on; a rewind past a page that went back is refused."""
    from litinfer_amd.cache import CacheManager
    from litinfer_amd.parts import PagedNeed, PagedTensor
    need = PagedNeed((PagedTensor("k", (1, 4)),), chunk=10)
    m = CacheManager([need], [None], page_size=4, num_pages=6, max_seqs=2, dtype=torch.float32, device="cpu")
    m.admit("a")
    for n in range(1, 64):
        m.reserve("a", 1)
        m.commit("a", 1)
        lo = n // 10 * 10                                  # the next query's chunk begins here
        table = m.block_table("a", 0)
        assert [b >= 0 for b in table] == [4 * i + 4 > lo for i in range(len(table))] and len(table) == -(-n // 4), n
        m.check_invariants()
    with pytest.raises(ValueError):
        m.rewind("a", 5)
    m.reserve("a", 9)                                      # a portion across two chunk ends is held whole until it is over
    m.commit("a", 9)
    m.release("a")
    assert m.free_pages() == [6]


def test_parts_refuse_what_they_do_not_have():
    from litinfer_amd.config import ModelSpec, PartSpec
    from litinfer_amd.parts import Runtime, build_part
    rt = Runtime(torch.device("cpu"), torch.float32)
    attn = {"hidden_size": 8, "num_heads": 2, "head_dim": 4, "scale": 1.0}
    for bad in ({"chunk": 4, "window": 4}, {"shared_keys": True, "qk_norm": "heads"}, {"chunk": -1}):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("masked_attention", "", {**attn, **bad}), rt)
    shared = build_part("mixer", PartSpec("masked_attention", "", {**attn, "shared_keys": True}), rt)
    with pytest.raises(ValueError):                        # a mixer without keys of its own given a cache of its own
        from types import SimpleNamespace
        shared.forward(None, None, None, SimpleNamespace(owned=True))
    ret = {"hidden_size": 8, "num_heads": 1, "head_dim": 4, "decay": [0.5]}
    rope = PartSpec("rope_pairs", "", {"head_dim": 4, "theta": 10.0})
    for bad in ({"activation": "relu"}, {"norm": "rows"}, {"gate": "tanh"}, {"activation": "silu", "position": rope}):
        with pytest.raises(ValueError):
            build_part("mixer", PartSpec("retention", "", {**ret, **bad}), rt)
    mlp = {"hidden_size": 8, "intermediate_size": 8}
    for bad in ({"activation": "clamped"}, {"activation": "silu", "limit": 2.0}, {"activation": "relu"}):
        with pytest.raises(ValueError):
            build_part("feed_forward", PartSpec("gated_mlp", "", {**mlp, **bad}), rt)
    moe = {**mlp, "experts": 4, "top": 2, "scores": "sigmoid"}
    for bad in ({"weigh_input": True, "identity": 1, "activation": "gelu"}, {"activation": "gelu_tanh"}, {"activation": "swiglu", "shared_intermediate_size": 8}):
        with pytest.raises(ValueError):
            build_part("feed_forward", PartSpec("routed_mlp", "", {**moe, **bad}), rt)
    spec, _ = _model(cases.CONFIG_D)
    from dataclasses import replace
    with pytest.raises(ValueError):
        replace(spec, residual_scale=0.5, streams=2).validate()


def test_a_stream_with_a_factor():
    """What a sublayer adds is multiplied; arrangements that norm a sublayer's output refuse a factor."""
    from litinfer_amd.parts.stream import BranchStream, ResidualStream
    x = torch.zeros(2, 3)
    s = ResidualStream(x, None, 0.25)

    def add(out, factor, tanh_norm):
        assert tanh_norm is None
        out += factor * 4.0
    s.add_by(add)
    assert torch.all(x == 1.0)
    b = BranchStream(torch.full((2, 3), 9.0), None)
    b.add_by(add)                                          # (a branch starts from zero and has no factor yet)
    assert torch.all(b.result() == 4.0)

    class N:
        def as_scaling(self):
            return object()
    with pytest.raises(NotImplementedError):
        s.add_normed(N(), x)
