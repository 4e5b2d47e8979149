"""The Besorax decoder on the GPU against the plain implementation (tests/plain_besorax.py): whole models of four tiny
configurations and of configurations drawn at random through the engine's step function (whole prompts, tails decoded one
by one, portions down to two tokens, mixed batches with pages and slots used again), every layer against the plain stream,
a standout key far away, at page borders and just inside and outside a chunk (of the layer's own keys and of another
layer's), a state that hardly forgets across portions, slots used again, long decoding through recorded steps, greedy
generation through the entry point, the scheduler, the command line and the trace replay; then every mechanism alone at the
level of its kernels."""
import json
import math
import os
import subprocess
import sys
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import besorax_cases as cases
import helpers
import plain_besorax as plain
import schedules

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
TOL = {"float32": 2e-5, "bfloat16": 4e-2}
LENGTHS = [5, 17, 33, 70, 150, 41, 64, 2, 1]
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def row_errs(out, ref):
    return np.concatenate([np.abs(out[r].astype(np.float64) - ref[r]).max(axis=-1) / np.abs(ref[r]).max() for r in ref])


def check_rows(out, ref, dt, what, noise=None):
    """float32: nine rows in ten within half the limit and every row within five times it.  bfloat16: nine rows in ten
    within the limit and half of them within half of it (a router's choice between two experts whose scores differ by less
    than the rounding may fall the other way, and moves that token's rows).  `noise`: the rows' deviations when the plain
    implementation rounds the sublayers' inputs to bfloat16 and nothing else; where that alone comes near the limits, three
    times it counts."""
    e = row_errs(out, ref)
    worst, q90, q50 = float(e.max()), float(np.quantile(e, 0.9)), float(np.quantile(e, 0.5))
    print(f"[observed] {what} {dt}: worst {worst:.3e}, nine in ten below {q90:.3e}, half below {q50:.3e}")
    assert np.isfinite(e).all()
    if dt == "float32":
        assert q90 < TOL[dt] / 2 and worst < 5 * TOL[dt], (what, worst, q90)
    else:
        n90, n50 = (np.quantile(noise, 0.9), np.quantile(noise, 0.5)) if noise is not None else (0.0, 0.0)
        assert q90 < max(TOL[dt], 3 * n90) and q50 < max(TOL[dt] / 2, 3 * n50), (what, worst, q90, q50, n90, n50)


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, (cfg, page, seed) in cases.CASES.items():
        w = cases.draw_weights(cfg, seed)
        for dt in ("float32", "bfloat16"):
            d = cases.write_model(tmp_path_factory.mktemp(f"b{name}{dt}"), cfg, w, DT[dt])
            reqs = helpers.random_requests(cfg["vocab"], LENGTHS, seed + 10)
            wd = cases.stored(w, DT[dt])
            out[(name, dt)] = (d, reqs, {r: plain.forward(cfg, wd, t) for r, t in reqs.items()}, wd)
    return out


def _engine(d, dt, page, max_tokens, **kw):
    from litinfer_amd.engine import Engine
    return Engine.from_dir(d, dtype=dt, device=DEV, page_size=page, max_tokens=max_tokens, max_seqs=4, page_order_seed=5, **kw)


def _rows(eng, rid, toks, cuts):
    from litinfer_amd.engine import StepEntry
    return np.concatenate([eng.step([StepEntry(rid, toks[a:b], list(range(b - a)))]).float().cpu().numpy().copy()
                           for a, b in zip(cuts, cuts[1:]) if b > a])


# ------------------------------------------------------------------------------------------ whole models
@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(cases.CASES))
@pytest.mark.parametrize("kind", ["whole", "tail", "chunks", "mixed"])
def test_schedules_match_the_plain_implementation(models, name, dt, kind):
    page = cases.CASES[name][1]
    d, reqs, ref, _ = models[(name, dt)]
    steps = getattr(schedules, kind)(reqs)
    eng = _engine(d, dt, page, schedules.max_live_tokens(reqs, steps, page if kind == "mixed" else 64))
    out = schedules.run(eng, reqs, steps)
    eng.cache.check_invariants()
    assert all(f == g.pool.capacity for f, g in zip(eng.cache.free_pages(), eng.cache.groups)) and eng.cache.free_slots() == 4
    if kind == "mixed":
        assert all(g.pool.total_allocations > g.pool.capacity for g in eng.cache.groups), "no page was used again"
    check_rows(out, ref, dt, f"{name} {kind}")


@pytest.mark.parametrize("seed", range(20))
def test_configurations_drawn_at_random(tmp_path, seed):
    """Sizes, order of layers, shared keys, chunks, experts and constants drawn from a seed: a mixed schedule on few pages."""
    cfg = cases.random_config(seed)
    w32 = cases.draw_weights(cfg, 100 + seed)
    reqs = helpers.random_requests(cfg["vocab"], [3, 40, 18, 105, 1, 29], 200 + seed)
    page = (4, 8, 16, 32)[seed % 4]
    for dt in ("float32", "bfloat16"):
        d = cases.write_model(tmp_path / dt, cfg, w32, DT[dt])
        w = cases.stored(w32, DT[dt])
        ref = {r: plain.forward(cfg, w, t) for r, t in reqs.items()}
        steps = schedules.mixed(reqs, seed=seed)
        eng = _engine(d, dt, page, schedules.max_live_tokens(reqs, steps, page))
        out = schedules.run(eng, reqs, steps)
        eng.cache.check_invariants()
        noise = None
        if dt == "bfloat16":
            noise = row_errs({r: plain.forward(cfg, w, t, rounding=helpers.round_to_bfloat16) for r, t in reqs.items()}, ref)
        check_rows(out, ref, dt, f"random configuration {seed}", noise)


@pytest.mark.parametrize("name", list(cases.CASES))
def test_float32_logits_do_not_depend_on_the_schedule(models, name):
    page = cases.CASES[name][1]
    d, reqs, _, _ = models[(name, "float32")]
    outs = {}
    for kind in ("whole", "tail", "chunks", "mixed"):
        steps = getattr(schedules, kind)(reqs)
        outs[kind] = schedules.run(_engine(d, "float32", page, schedules.max_live_tokens(reqs, steps)), reqs, steps)
    for kind in ("tail", "chunks", "mixed"):
        for r in reqs:
            assert schedules.rel_err(outs[kind][r], outs["whole"][r].astype(np.float64)) < 2e-5, (kind, r)


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(cases.CASES))
def test_every_layer_against_the_plain_stream(models, name, dt):
    from litinfer_amd.engine import StepEntry
    cfg, page = cases.CASES[name][:2]
    d, reqs, _, w = models[(name, dt)]
    toks, streams, taps = reqs["r3"], [], []
    plain.forward(cfg, w, toks, streams)
    eng = _engine(d, dt, page, 256)
    eng.model.tap = lambda i, x: taps.append(x.detach().cpu().numpy().copy())
    eng.step([StepEntry("a", toks, [0])])
    assert len(taps) == len(streams) == len(cfg["layers"])
    for i, (got, ref) in enumerate(zip(taps, streams)):
        e = np.abs(got - ref).max(axis=-1) / np.abs(ref).max()
        assert (e.max() if dt == "float32" else np.quantile(e, 0.9)) < TOL[dt], (i, e.max())


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_long_decoding_through_recorded_steps(models, dt):
    from litinfer_amd.engine import StepEntry
    cfg, page = cases.CASES["A"][:2]
    d, _, _, w = models[("A", dt)]
    toks = np.random.default_rng(3).integers(0, cfg["vocab"], 170).tolist()
    ref = plain.forward(cfg, w, toks)
    eng = _engine(d, dt, page, 256)
    rows = [eng.step([StepEntry("a", toks[:20], list(range(20)))]).float().cpu().numpy()]
    rows += [eng.step([StepEntry("a", [toks[i]], [0])]).float().cpu().numpy().copy() for i in range(20, 170)]
    assert eng.graph_replays > 100
    check_rows({"a": np.concatenate(rows)}, {"a": ref}, dt, "150 tokens decoded")


def test_slots_that_are_used_again_start_from_zero(models):
    """Requests follow each other on the same slots; two requests that take turns keep their own states."""
    from litinfer_amd.engine import StepEntry
    page = cases.CASES["B"][1]
    d, reqs, ref, _ = models[("B", "float32")]
    eng = _engine(d, "float32", page, 1024)
    for rnd in range(3):
        for r in ("r0", "r1", "r2", "r5", "r7"):
            out = _rows(eng, r, reqs[r], [0, 1, len(reqs[r])])
            eng.finish(r)
            assert schedules.rel_err(out, ref[r]) < TOL["float32"], (rnd, r)
    got = {"r1": [], "r2": []}
    for i in range(12):
        for r in got:
            got[r].append(eng.step([StepEntry(r, [reqs[r][i]], [0])]).float().cpu().numpy().copy())
    for r in got:
        assert schedules.rel_err(np.concatenate(got[r]), ref[r][:12]) < TOL["float32"]


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_a_state_that_hardly_forgets_across_portions(tmp_path, dt):
    """Decays near one: what the first tokens wrote still counts hundreds of tokens later, across portions cut at 1, 63, 64,
    65, 128, 129 tokens."""
    cfg = {"architecture": "Besorax", "vocab": 97, "width": 64, "norm": {"eps": 1e-6}, "residual_mult": 1.3, "embedding": {"scale": 1.0},
           "layers": [cases.lightning(3, 20, 12, (1.0, 0.9995, 0.999), None)]}
    w32 = cases.draw_weights(cfg, 9)
    d = cases.write_model(tmp_path / "m", cfg, w32, DT[dt])
    w = cases.stored(w32, DT[dt])
    toks = np.random.default_rng(6).integers(0, 97, 330).tolist()
    ref = plain.forward(cfg, w, toks)
    other = [(t + 1) % 97 for t in toks[:4]] + toks[4:]
    moved = np.abs(plain.forward(cfg, w, other)[-1] - ref[-1]).max() / np.abs(ref[-1]).max()
    assert moved > 200 * TOL["float32"], moved           # the first tokens still count at the end
    for cuts in ([0, 330], [0, 1, 64, 127, 192, 257, 330], [0, 128, 257, 258, 330], [0, 65, 66, 68, 330]):
        out = _rows(_engine(d, dt, 16, 512), "a", toks, cuts)
        check_rows({"a": out}, {"a": ref}, dt, f"slow decay, cuts {cuts}")


def test_greedy_generation_through_the_entry_point(models):
    from litinfer_amd import models as entry
    cfg, page = cases.CASES["A"][:2]
    d, reqs, _, w = models[("A", "float32")]
    lm = entry.load(d, dtype="float32", device=DEV, page_size=page, max_tokens=512, max_seqs=4)
    seq = list(reqs["r1"])
    new = list(lm.generate(seq, max_new_tokens=12, top_k=1, top_p=1.0, temperature=1.0))
    assert len(new) == 12
    for t in new:
        logits = plain.forward(cfg, w, seq)[-1]
        assert t == np.argmax(logits) or logits.max() - logits[t] < 1e-4 * np.abs(logits).max(), (len(seq), t)
        seq.append(int(t))


def test_several_requests_through_the_scheduler(models):
    """Continuous batching of five prompts on four state slots (tokens are fed back on the device, the scheduler looks
    ahead): each request's greedy tokens are those of the request alone."""
    from litinfer_amd import models as entry
    page = cases.CASES["C"][1]
    d, reqs, _, _ = models[("C", "float32")]
    lm = entry.load(d, dtype="float32", device=DEV, page_size=page, max_tokens=1024, max_seqs=4)
    prompts = [reqs[r] for r in ("r0", "r1", "r2", "r5", "r7")]
    alone = [list(lm.generate(p, max_new_tokens=8)) for p in prompts]
    lm.engine_start()
    ids = [lm.engine_add_request(p, 8) for p in prompts]
    while lm.engine_has_unfinished():
        lm.engine_step()
    assert [list(lm.engine_get_output(i)) for i in ids] == alone


def test_generate_through_the_command_line(models):
    cfg = cases.CASES["D"][0]
    d, reqs, _, w = models[("D", "float32")]
    seq = list(reqs["r1"])
    r = subprocess.run([sys.executable, "-m", "litinfer_amd", "generate", "--model", str(d), "--dtype", "float32", "--prompt-ids",
                        ",".join(map(str, seq)), "--max-new-tokens", "6", "--top-k", "1"], cwd=ROOT, capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    new = []
    for _ in range(6):
        new.append(int(np.argmax(plain.forward(cfg, w, seq + new)[-1])))
    assert ",".join(map(str, new)) in r.stdout.replace(" ", ""), r.stdout[-500:]


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_trace_replay_in_a_subprocess(models, tmp_path, dt):
    cfg = cases.CASES["A"][0]
    d, reqs, ref, _ = models[("A", dt)]
    use = {r: reqs[r] for r in ("r0", "r1", "r3", "r5", "r7")}
    steps = schedules.mixed(use, seed=2)
    lines = [json.dumps({"step": n, "entries": [{"id": r, "tokens": use[r][i:i + k], "want": list(range(k))} for r, i, k in entries], "end": end})
             for n, (entries, end) in enumerate(steps)]
    out = tmp_path / "out"
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(d), "--dtype", dt, "--out", str(out), "--max-tokens",
                        str(schedules.max_live_tokens(use, steps, 64))], input="\n".join(lines) + "\n", cwd=ROOT, capture_output=True,
                       text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {n}" for n in range(len(steps))]
    rows = {r_: [] for r_ in use}
    for n, (entries, end) in enumerate(steps):
        a, o = np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, cfg["vocab"]), 0
        for r_, i, k in entries:
            rows[r_].append(a[o:o + k])
            o += k
    check_rows({r_: np.concatenate(v) for r_, v in rows.items()}, {r_: ref[r_] for r_ in use}, dt, "trace replay")


# ------------------------------------------------------------------------------------------- a standout key
CHUNK = 21
A_TOK, B_TOK = 63, 62


def _standout_model(tmp, dt, kind, sizes, sink=0.0, owner_chunk=8):
    """Weights that make ONE key win: token A's key meets token B's query in every head with a score of 16, far above all
    others, and A's value is large.  Whether B sees A decides B's logits.  `sizes` = (heads, kv heads, dim).  "shared": the
    queries stand in layer 1, which reads layer 0's keys with a chunk of its own; layer 0 itself adds nothing."""
    H, G, D = sizes
    scale, rank, mlp = 16.0 / D, 32 if D == 16 else 64, cases.dense(48, 2.0)
    layers = {"attention": lambda: [cases.attention(H, G, D, D, scale, 1e4, 4, CHUNK, mlp)],
              "whole": lambda: [cases.attention(H, G, D, D, scale, 1e4, 4, 4096, mlp)],
              "shared": lambda: [cases.attention(H, G, D, D, scale, 1e4, 4, owner_chunk, None),
                                 cases.attention(H, G, D, D, scale, 1e4, 4, CHUNK, mlp, kv_from=0)],
              "latent": lambda: [cases.latent(H, D, 16 if D == 16 else 32, D, rank, 24, scale, 1e4, mlp)]}[kind]()
    cfg = {"architecture": "Besorax", "vocab": 64, "width": 64, "norm": {"eps": 1e-6}, "residual_mult": 0.9, "embedding": {"scale": 1.0}, "layers": layers}
    w = cases.draw_weights(cfg, 5)
    w["embed"][:, :2] = 0.0
    w["embed"][A_TOK] = w["embed"][B_TOK] = 0.0
    w["embed"][A_TOK, 0] = w["embed"][B_TOK, 1] = 3.0
    for n in w:
        if ".norm1" in n and not n.endswith(("alpha", ".b")):
            w[n][:], w[n + ".b"][:], w[n + ".alpha"] = 1.0, 0.0, np.float32(1.0)
    w = {n: np.asarray(a) for n, a in w.items()}
    rng = np.random.default_rng(1)
    pq, pk = ("l1.mix.", "l0.mix.") if kind == "shared" else ("l0.mix.", "l0.mix.")
    u = np.ones(D) if kind == "latent" else np.r_[np.zeros(4), np.full(D - 4, (D / (D - 4.0)) ** 0.5)]      # (columns that are not rotated)
    if kind == "latent":
        Q, R = 24, rank
        dq, d = np.where(np.arange(Q) % 3 == 0, -1.0, 1.0), np.where(np.arange(R) % 2 == 0, 1.0, -1.0)
        for n, scale_ in (("dq", 0.1), ("dkv", 0.1), ("uq", 0.05), ("uk", 0.05)):
            w[pq + n] *= scale_
        w[pq + "dq"][:, 1], w[pq + "dkv"][:R, 0], w[pq + "dq.norm"][:], w[pq + "dkv.norm"][:] = 6.0 * dq, 6.0 * d, 1.0, 1.0
        for h in range(H):
            at = h * (D + cfg["layers"][0]["mixer"]["rot_dim"])
            w[pq + "uq"][at:at + D] += np.outer(u, dq) / Q
            w[pq + "uk"][h * D:(h + 1) * D] += np.outer(u, d) / R
        w[pq + "uv"] += 6.0 * rng.normal(size=(H * D, 1)) * d[None] / R
    else:
        w[pq + "q"] *= 0.02
        w[pk + "k"] *= 0.02
        for h in range(H):
            w[pq + "q"][h * D:(h + 1) * D, 1] = u
        for g in range(G):
            w[pk + "k"][g * D:(g + 1) * D, 0] = u
        w[pk + "v"][:, 0] += 6.0 * rng.normal(size=G * D)
    if kind == "shared":
        w["l0.mix.o"] *= 0.0
    w[pq + "sink"][:] = sink
    d = cases.write_model(tmp, cfg, w, DT[dt])
    return cfg, cases.stored(w, DT[dt]), d


def _run_how(eng, toks, lo, hi, how):
    from litinfer_amd.engine import StepEntry
    n = len(toks)
    if how == "prompt":
        return _rows(eng, "a", toks, [0, n])
    if how == "portions":                                  # a cut between the two, one right at the later one, portions of two
        return _rows(eng, "a", toks, sorted({0, lo + 1, hi, min(hi + 2, n), n}))
    rows = [eng.step([StepEntry("a", toks[:lo + 1], list(range(lo + 1)))]).float().cpu().numpy()]
    rows += [eng.step([StepEntry("a", [toks[i]], [0])]).float().cpu().numpy().copy() for i in range(lo + 1, n)]
    return np.concatenate(rows)


def _moved(cfg, w, toks, pa, pb, ref):
    without = list(toks)
    without[pa] = 7
    return np.abs(plain.forward(cfg, w, without)[pb] - ref[pb]).max() / np.abs(ref[pb]).max()


SIZES = [(4, 2, 16), (4, 4, 64), (8, 1, 64)]        # the general kernels; the matrix-core tiles; many heads a kv head


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", SIZES)
@pytest.mark.parametrize("kind", ["whole", "latent"])
def test_a_far_key_among_hundreds(tmp_path, dt, kind, sizes):
    cfg, w, d = _standout_model(tmp_path / "m", dt, kind, sizes)
    toks = np.random.default_rng(4).integers(0, 60, 420).tolist()
    toks[3], toks[400] = A_TOK, B_TOK
    ref = plain.forward(cfg, w, toks)
    assert _moved(cfg, w, toks, 3, 400, ref) > 0.1
    for cuts in ([0, 420], [0, 390, 420], [0, 2, 5, 399, 401, 420], [0, 398, 399, 400, 401, 402, 420]):
        out = _rows(_engine(d, dt, 16, 512), "a", toks, cuts)
        assert schedules.rel_err(out[395:], ref[395:]) < TOL[dt], cuts


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("how", ["prompt", "portions", "decoded"])
@pytest.mark.parametrize("kind", ["whole", "latent"])
def test_a_key_at_page_borders_at_the_query_and_behind_it(tmp_path, dt, how, kind):
    """The key at the last and the first row of a page and at position 0; the query right behind the key, many pages
    later, and BEFORE it (the key must not be seen)."""
    cfg, w, d = _standout_model(tmp_path / "m", dt, kind, (4, 2, 16))
    moved = []
    for pa, pb in ((0, 70), (7, 8), (8, 71), (15, 16), (16, 95), (31, 33), (40, 39)):
        toks = np.random.default_rng(3).integers(0, 60, max(pa, pb) + 4).tolist()
        toks[pa], toks[pb] = A_TOK, B_TOK
        ref = plain.forward(cfg, w, toks)
        moved.append(_moved(cfg, w, toks, pa, pb, ref))
        out = _run_how(_engine(d, dt, 8, 128), toks, min(pa, pb), max(pa, pb), how)
        assert schedules.rel_err(out, ref) < TOL[dt], (pa, pb)
    assert min(moved[:-1]) > 0.1 and moved[-1] < 1e-12, moved


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("how", ["prompt", "portions", "decoded"])
@pytest.mark.parametrize("sizes", SIZES)
@pytest.mark.parametrize("kind,owner_chunk", [("attention", 0), ("shared", 8), ("shared", 64), ("shared", 2 * CHUNK)])
def test_a_key_just_inside_and_just_outside_the_chunk(tmp_path, dt, how, sizes, kind, owner_chunk):
    """Key and query at the first and last position of a chunk, in one chunk and in two that follow each other, the first
    tokens, far on; the keys are the layer's own or another layer's, whose own chunk is shorter, longer or a multiple."""
    cfg, w, d = _standout_model(tmp_path / "m", dt, kind, sizes, owner_chunk=owner_chunk)
    C = CHUNK
    for pa, pb in ((0, 1), (0, C - 1), (0, C), (C - 1, C), (C, C + 1), (C, 2 * C - 1), (C, 2 * C), (2 * C - 1, 2 * C), (3 * C, 4 * C - 1), (4 * C - 2, 4 * C)):
        toks = np.random.default_rng(pa).integers(0, 60, pb + 3).tolist()
        toks[pa], toks[pb] = A_TOK, B_TOK
        ref = plain.forward(cfg, w, toks)
        moved = _moved(cfg, w, toks, pa, pb, ref)
        assert (moved > 0.1) if pa // C == pb // C else (moved < 1e-12), (pa, pb, moved)
        out = _run_how(_engine(d, dt, 8, 192), toks, pa, pb, how)
        assert schedules.rel_err(out, ref) < TOL[dt], (pa, pb)


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", SIZES[:2])
@pytest.mark.parametrize("kind", ["attention", "latent"])
def test_a_sink_that_outweighs_every_key(tmp_path, dt, sizes, kind):
    """With a large sink nearly all weight goes to the term without a value.  Leaving it out, or counting it once a split
    of the keys, changes the logits by far more than the tolerance."""
    cfg, w, d = _standout_model(tmp_path / "m", dt, kind, sizes, sink=9.0)
    toks = np.random.default_rng(8).integers(0, 60, 300).tolist()
    ref = plain.forward(cfg, w, toks)
    w0 = {**w, "l0.mix.sink": w["l0.mix.sink"] - 50.0}
    assert np.abs(plain.forward(cfg, w0, toks) - ref).max() > 0.1 * np.abs(ref).max()
    for cuts in ([0, 300], [0, 290, 291, 292, 300], [0, 33, 35, 300]):
        check_rows({"a": _rows(_engine(d, dt, 16, 512), "a", toks, cuts)}, {"a": ref}, dt, f"large sink, cuts {cuts}")


# ------------------------------------------------------------------------------------------ mechanisms alone
def _ctx(q_lens, slots):
    q_len = np.asarray(q_lens, dtype=np.int32)
    q_start = np.concatenate([[0], np.cumsum(q_len)[:-1]]).astype(np.int32)
    dev = lambda a: torch.from_numpy(np.ascontiguousarray(a, dtype=np.int32)).to(DEV)
    return SimpleNamespace(num_tokens=int(q_len.sum()), num_segments=len(q_len), host_state_slots=np.asarray(slots, dtype=np.int32),
                           seg_of_token=dev(np.repeat(np.arange(len(q_len)), q_len)), q_start=dev(q_start), q_len=dev(q_len),
                           state_slots=dev(slots), max_q_len=int(q_len.max()))


def _f32(a):
    return torch.tensor(np.asarray(a), dtype=torch.float32, device=DEV)


STEPS = ([(0, 1), (2, 5)], [(2, 100), (0, 1)], [(0, 199), (2, 64)], [(2, 65)], [(0, 1), (2, 1)], [(0, 700), (2, 130)], [(2, 33), (0, 2)])


@pytest.mark.parametrize("silu_in", [False, True])
@pytest.mark.parametrize("heads,N,vdim", [(3, 12, 12), (2, 8, 40), (4, 64, 64), (1, 128, 128), (2, 100, 20), (1, 256, 12), (2, 64, 160), (1, 36, 132),
                                          (2, 256, 256), (3, 30, 30), (2, 5, 7)])
def test_retention_across_steps_and_slots(heads, N, vdim, silu_in):
    """Two requests on slots 0 and 2 take turns with portions of 1 to 700 tokens (token after token, and as products over
    chunks side by side); slot 1 is nobody's and stays as it is.  Decays 0, 1 and in between."""
    from litinfer_amd.engine.workspace import Workspace
    from litinfer_amd.kernels import ops
    ws, rng = Workspace(DEV), np.random.default_rng(N + vdim)
    decay = rng.uniform(0.3, 1.0, heads)
    decay[0] = 0.9995
    if heads > 2:
        decay[1:3] = 0.0, 1.0
    state = torch.zeros(3, heads, N, vdim, device=DEV)
    state[1] = 7.0
    dec32 = decay.astype(np.float32).astype(np.float64)
    S, H, V = {0: np.zeros((heads, N, vdim)), 2: np.zeros((heads, N, vdim))}, heads, vdim
    for step in STEPS:
        x = rng.normal(size=(sum(n for _, n in step), H * V + 2 * H * N))
        wide = torch.zeros(len(x), x.shape[1] + 4, device=DEV)                    # (the rows lie inside a wider buffer)
        wide[:, 4:] = _f32(x)
        y = torch.empty(len(x), H * V, device=DEV)
        ops.ssm_scan(wide[:, 4:], None, None, None, None, state, _ctx([n for _, n in step], [s for s, _ in step]), y, H, V, N, H, ws,
                     fixed_decay=_f32(decay), fixed_step=0.7, silu_in=silu_in)
        g, want, o = plain.silu(x) if silu_in else x, np.zeros((len(x), H * V)), 0
        for s, n in step:
            for t in range(o, o + n):
                v, k, q = g[t, :H * V].reshape(H, V), g[t, H * V:H * V + H * N].reshape(H, N), g[t, H * V + H * N:].reshape(H, N)
                S[s] = dec32[:, None, None] * S[s] + 0.7 * k[:, :, None] * v[:, None, :]
                want[t] = np.matmul(q[:, None], S[s])[:, 0].reshape(-1)
            o += n
        assert np.abs(y.cpu().numpy() - want).max() < 2e-5 * max(1.0, np.abs(want).max()), step
        for s in (0, 2):
            assert np.abs(state[s].cpu().numpy() - S[s]).max() < 2e-5 * max(1.0, np.abs(S[s]).max()), step
    assert torch.all(state[1] == 7.0)


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_small_kernels_of_the_design(dt):
    from litinfer_amd.kernels import ops
    rng = np.random.default_rng(0)
    tol = 1e-5 if dt == "float32" else 1e-2
    for T, H in ((37, 100), (3, 33), (1, 1536), (300, 64)):
        x, out = rng.normal(0, 3, size=(T, H)), torch.empty(T, H, dtype=DT[dt], device=DEV)
        w = {"n": rng.normal(1, 0.3, H), "n.b": rng.normal(0, 0.3, H), "n.alpha": 0.6}
        ops.tanh_norm(_f32(x), 0.6, _f32(w["n"]), _f32(w["n.b"]), out)
        want = plain.tanh_norm(x, w, "n")
        assert np.abs(out.float().cpu().numpy() - want).max() < tol * np.abs(want).max()
        ops.gelu_erf(_f32(x), out)
        assert np.abs(out.float().cpu().numpy() - plain.gelu(x)).max() < tol * np.abs(x).max()
        if H % 2 == 0:
            half = torch.empty(T, H // 2, dtype=DT[dt], device=DEV)
            ops.gated_act(_f32(x), half, "clamped", 1.3)
            g, u = np.minimum(x[:, :H // 2], 1.3), np.clip(x[:, H // 2:], -1.3, 1.3)
            assert np.abs(half.float().cpu().numpy() - g * plain.sigmoid(1.702 * g) * (u + 1)).max() < tol * 4


PRODUCTS = [(1, 96, 64), (5, 1536, 256), (20, 200, 1024), (31, 520, 72), (48, 256, 2048), (64, 130, 4096), (70, 256, 1024), (200, 384, 2048), (300, 512, 128),
            (130, 72, 40), (7, 50, 33), (90, 64, 50), (600, 1024, 64)]


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("M,N,K", PRODUCTS)
@pytest.mark.parametrize("biased", [False, True])
def test_products_that_join_the_sum_with_a_factor(dt, M, N, K, biased):
    """out += factor * (x w^T + b) in every form that the library picks by size; then with the tanh norm of the new sum
    beside it, and with the RMS norm, where the library has those in one go."""
    from litinfer_amd.engine.workspace import Workspace
    from litinfer_amd.kernels import ops
    rng, ws = np.random.default_rng(M + N), Workspace(DEV)
    x, w = torch.tensor(rng.normal(size=(M, K)), dtype=torch.float32).to(DT[dt]), torch.tensor(rng.normal(size=(N, K)) / K ** 0.5, dtype=torch.float32).to(DT[dt])
    b, o, gm, bt = rng.normal(size=N), rng.normal(size=(M, N)), rng.normal(1, 0.2, N), rng.normal(0, 0.2, N)
    bias = _f32(b) if biased else None
    sums = o - 0.37 * (x.double().numpy() @ w.double().numpy().T + (b if biased else 0.0))
    out = _f32(o)
    ops.linear(x.to(DEV), w.to(DEV), bias, out, True, ws=ws, factor=-0.37)
    near = lambda got, want, tol: np.abs(got.float().cpu().numpy() - want).max() < tol * np.abs(want).max()
    assert near(out, sums, 1e-5)
    out, xn = _f32(o), torch.zeros(M, N, dtype=DT[dt], device=DEV)
    took = ops.linear_tanh_norm(x.to(DEV), w.to(DEV), bias, out, 0.8, _f32(gm), _f32(bt), xn, ws, factor=-0.37)
    assert took == (dt == "bfloat16" and (M <= 32 and K % 8 == 0 or M in (48, 64, 200) or (M, K) == (70, 1024))), took
    if took:
        assert near(out, sums, 1e-5) and near(xn, np.tanh(0.8 * sums) * gm + bt, 1e-2)
    else:
        assert near(out, o, 1e-6)
    if dt == "bfloat16":
        out = _f32(o)
        if ops.linear_then_norm(x.to(DEV), w.to(DEV), bias, out, _f32(gm), 1e-5, xn, ws, factor=-0.37):
            assert near(out, sums, 1e-5) and near(xn, plain.rms(sums, 1e-5) * gm, 1e-2)
        if ops.residual_norm_takes(M, N, K, torch.bfloat16) and ops.few_rows_preferred(M, N, K):
            out, parts = _f32(o), torch.zeros(ops.RESIDUAL_NORM_MAX_PARTS * ops.RESIDUAL_NORM_MAX_ROWS, device=DEV)
            ops.linear_residual_norm(x.to(DEV), w.to(DEV), bias, out, _f32(gm), xn, parts, factor=-0.37)
            assert near(out, sums, 1e-5) and near(xn, sums * gm, 1e-2)


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("M,I,K", [(1, 96, 64), (9, 700, 256), (16, 64, 1024), (30, 96, 128), (50, 160, 64), (64, 8192, 128), (200, 192, 256), (700, 640, 64)])
def test_clamped_activation_as_the_products_epilogue(dt, M, I, K):
    from litinfer_amd.kernels import ops
    if not ops.swiglu_takes(M, K, DT[dt]):
        pytest.skip("this dtype has no such epilogue at this size")
    rng = np.random.default_rng(I)
    x, w = torch.tensor(rng.normal(size=(M, K)), dtype=torch.float32).to(DT[dt]), torch.tensor(2.0 * rng.normal(size=(2 * I, K)) / K ** 0.5, dtype=torch.float32).to(DT[dt])
    out = torch.empty(M, I, dtype=DT[dt], device=DEV)
    ops.linear_swiglu(x.to(DEV), w.to(DEV), out, limit=1.1)
    z = x.double().numpy() @ w.double().numpy().T
    g, u = np.minimum(z[:, :I], 1.1), np.clip(z[:, I:], -1.1, 1.1)
    want = g * plain.sigmoid(1.702 * g) * (u + 1.0)
    assert np.abs(out.float().cpu().numpy() - want).max() < (1e-5 if dt == "float32" else 1e-2) * np.abs(want).max()


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("T,K,E,top,ff,shared", [(1, 64, 5, 1, 32, 48), (7, 96, 12, 3, 64, 0), (33, 50, 3, 2, 30, 20), (100, 128, 4, 1, 96, 64), (5, 256, 8, 2, 128, 0),
                                                 (40, 512, 6, 2, 64, 256), (300, 256, 16, 4, 64, 128), (600, 64, 2, 2, 32, 32), (900, 128, 2, 1, 160, 0), (3, 48, 1, 1, 16, 8)])
@pytest.mark.parametrize("norm", [False, True])
def test_routed_feed_forward_with_weights_on_the_input(dt, T, K, E, top, ff, shared, norm):
    """The part alone, against the plain one: every form of the routed products, the factor of the stream and, with `norm`,
    the tanh norm of the new sum beside it."""
    from litinfer_amd.config import PartSpec
    from litinfer_amd.engine.workspace import Workspace
    from litinfer_amd.parts import Runtime, build_part
    from litinfer_amd.parts.stream import ResidualStream
    rng, ws = np.random.default_rng(T + K), Workspace(DEV)
    names = {"m.router": (E, K), **{f"m.e{e}.{s}": ((ff, K) if s == "up" else (K, ff)) for e in range(E) for s in ("up", "down")}}
    if shared:
        names.update({"m.shared.up": (shared, K), "m.shared.down": (K, shared)})
    w = {n: torch.tensor(rng.normal(size=s) * (2.0 if "router" in n else 1.5) / s[1] ** 0.5, dtype=torch.float32).to(DT[dt]) for n, s in names.items()}
    wn = {"n": rng.normal(1, 0.2, K), "n.b": rng.normal(0, 0.2, K), "n.alpha": np.array(0.7)}
    rt = Runtime(torch.device(DEV), DT[dt])
    part = build_part("feed_forward", PartSpec("routed_mlp", "m.", {
        "hidden_size": K, "intermediate_size": ff, "experts": E, "top": top, "activation": "gelu", "scores": "sigmoid", "normalize": False,
        "router_bias": False, "weigh_input": True, "shared_intermediate_size": shared, "shared_gate": False}), rt)
    part.load_params(lambda n: w[n])
    h, x = torch.tensor(rng.normal(size=(T, K)), dtype=torch.float32).to(DT[dt]), rng.normal(size=(T, K))
    stream = ResidualStream(_f32(x), ws, 0.6)
    stream.ws_dtype = DT[dt]
    nrm = build_part("norm", PartSpec("dynamic_tanh", "", {"size": K, "param": "n"}), rt)
    nrm.load_params(lambda n: torch.tensor(wn[n], dtype=torch.float32))
    stream.next_norm = nrm if norm else None
    part.forward(h.to(DEV), stream, SimpleNamespace(ws=ws))
    want = x + 0.6 * plain.routed_ff(h.double().numpy(), {n: a.double().numpy() for n, a in w.items()}, "m.", top, shared > 0)
    e = np.abs(stream.total().cpu().numpy() - want).max(axis=1) / np.abs(want).max()
    assert (e.max() if dt == "float32" else np.quantile(e, 0.95)) < (1e-5 if dt == "float32" else 1.5e-2), e.max()
    if norm:
        rows = stream.normed(nrm, None)                       # left by the kernel that adds
        wn32 = {n: a.astype(np.float32).astype(np.float64) for n, a in wn.items()}
        e = np.abs(rows.float().cpu().numpy() - plain.tanh_norm(stream.total().double().cpu().numpy(), wn32, "n")).max()
        assert e < (1e-5 if dt == "float32" else 2e-2), e


def _attention_case(dtype, seg_specs, nh, nkv, dk, dv, page, chunk, seed, heads_kernel=None):
    """Random queries, keys and values for segments (context, queries) in shuffled pages, a sink a head, chunks whose older
    pages have been given back; returns the kernel's output and the plain one."""
    from litinfer_amd.engine.batch import AttentionMeta
    from litinfer_amd.engine.workspace import Workspace
    from litinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(seed)
    blocks = [-(-c // page) for c, _ in seg_specs]
    num_pages = sum(blocks) + 2
    perm = torch.randperm(num_pages, generator=g).tolist()
    kc, vc = torch.randn(num_pages, nkv, page, dk, generator=g).to(dtype), torch.randn(num_pages, nkv, page, dv, generator=g).to(dtype)
    tab = np.full((len(seg_specs), max(blocks)), -1, dtype=np.int32)
    T = sum(q for _, q in seg_specs)
    q = torch.randn(T, nh, dk, generator=g)
    sink = torch.randn(nh, generator=g) * 2.0
    scale, refs, o = 1.0 / math.sqrt(dk), [], 0
    for s, (c, ql) in enumerate(seg_specs):
        k, v = torch.randn(c, nkv, dk, generator=g).to(dtype), torch.randn(c, nkv, dv, generator=g).to(dtype)
        for b in range(blocks[s]):
            n = min(page, c - b * page)
            if not chunk or b * page + n > (c - ql) // chunk * chunk:           # (older pages have been given back)
                tab[s, b] = perm.pop()
                kc[tab[s, b], :, :n] = k[b * page:b * page + n].transpose(0, 1)
                vc[tab[s, b], :, :n] = v[b * page:b * page + n].transpose(0, 1)
        qq = np.zeros((c, nh, dk))
        qq[c - ql:] = q[o:o + ql].double().numpy()
        kk, vv, sk = k.double().numpy(), v.double().numpy(), sink.double().numpy()
        out = np.zeros((ql, nh, dv))
        for i in range(ql):
            p = c - ql + i
            lo = p // chunk * chunk if chunk else 0
            for h in range(nh):
                sc = kk[lo:p + 1, h // (nh // nkv)] @ qq[p, h] * scale
                mx = max(sc.max(), sk[h])
                e = np.exp(sc - mx)
                out[i, h] = (e @ vv[lo:p + 1, h // (nh // nkv)]) / (e.sum() + math.exp(sk[h] - mx))
        refs.append(out.reshape(ql, -1))
        o += ql
    q_len, ctx_len = np.array([x for _, x in seg_specs], dtype=np.int32), np.array([c for c, _ in seg_specs], dtype=np.int32)
    q_start = np.concatenate([[0], np.cumsum(q_len)[:-1]]).astype(np.int32)
    seg_of = np.repeat(np.arange(len(seg_specs), dtype=np.int32), q_len)
    dev = lambda a: torch.from_numpy(a).to(DEV)
    single, multi = np.nonzero(q_len[seg_of] == 1)[0].astype(np.int32), np.nonzero(q_len[seg_of] != 1)[0].astype(np.int32)
    tiles = np.asarray([(i, int(q_start[i]) + a, min(32, int(q_len[i]) - a), 0) for i in range(len(seg_specs))
                        if q_len[i] > 1 for a in range(0, int(q_len[i]), 32)], dtype=np.int32).reshape(-1, 4)
    meta = AttentionMeta(block_table=dev(tab), max_blocks=tab.shape[1], seg_of_token=dev(seg_of), q_start=dev(q_start), q_len=dev(q_len),
                         ctx_len=dev(ctx_len), num_segments=len(seg_specs), num_tokens=T, max_q_len=int(q_len.max()),
                         max_ctx_len=int(ctx_len.max()), host_q_start=q_start, host_q_len=q_len, host_ctx_len=ctx_len,
                         single_tokens=dev(single) if len(multi) else None, num_single=len(single),
                         multi_tokens=dev(multi) if len(single) else None, num_multi=len(multi),
                         tiles=dev(tiles), num_tiles=len(tiles), tile_rows=32)
    out, was = torch.empty(T, nh * dv, dtype=dtype, device=DEV), ops._heads_kernel_pays
    if heads_kernel is not None:
        ops._heads_kernel_pays = lambda *a: bool(heads_kernel)
    try:
        ops.masked_attention(q.to(DEV).contiguous(), nh * dk, dk, out, kc.to(DEV), vc.to(DEV), meta, nh, nkv, dk, dv, page, 0, 0, 0.0,
                             scale, ws=Workspace(DEV), sink=sink.to(DEV), chunk=chunk)
    finally:
        ops._heads_kernel_pays = was
    return out.float().cpu().numpy(), np.concatenate(refs)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("chunk", [1, 40, 64, 1000, 0])
@pytest.mark.parametrize("segs,nh,nkv,dk,dv,page,heads_kernel", [
    ([(2, 2)], 1, 1, 4, 4, 16, None),                                          # the general kernel, one wave
    ([(100, 37), (33, 2), (300, 1), (70, 70)], 6, 3, 24, 40, 8, None),         # ... four and eight waves a (token, head)
    ([(700, 3), (5, 5)], 2, 1, 24, 16, 16, None),
    ([(100, 37), (33, 2), (300, 1), (70, 70), (64, 64), (1, 1)], 6, 3, 64, 64, 8, None),   # tiles of queries beside single tokens
    ([(1100, 1100)], 8, 2, 64, 64, 16, None),                                  # one long prompt: tiles whose keys are cut into splits
    ([(900, 1), (81, 1), (80, 1), (2500, 1), (2001, 1)], 8, 4, 64, 64, 16, False),         # single tokens, rows over lanes, splits and their join
    ([(900, 1), (41, 1), (40, 1), (2500, 1)], 8, 2, 128, 128, 16, True),       # single tokens with the heads as a tile's columns
    ([(300, 1), (7, 1)], 6, 1, 256, 256, 16, False),                           # long rows
])
def test_chunks_and_sinks_in_every_attention_kernel(dtype, segs, nh, nkv, dk, dv, page, heads_kernel, chunk):
    got, ref = _attention_case(dtype, segs, nh, nkv, dk, dv, page, chunk, seed=dk + nh, heads_kernel=heads_kernel)
    err = float(np.abs(got - ref).max() / np.abs(ref).max())
    assert err < (2e-5 if dtype is torch.float32 else 1.2e-2), err
