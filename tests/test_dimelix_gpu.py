"""The Dimelix decoder on the GPU against the plain implementation (tests/plain_dimelix.py): whole models of four tiny
configurations and of configurations drawn at random through the engine's step function (whole prompts, tails decoded one
by one, portions down to two tokens, mixed batches with pages and slots used again), every layer run against the plain
stream, a standout key far away, at page borders and just inside and outside the window, a state that forgets slowly
across portions, slots used again, long decoding through recorded steps, greedy generation through the entry point, the
scheduler, the command line and the trace replay; then every mechanism alone at the level of its kernels."""
import json
import math
import os
import subprocess
import sys
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import dimelix_cases as cases
import helpers
import plain_dimelix as plain
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
    within the limit, half of them within half of it, and every row within three times the limit.  `noise`: the rows'
    deviations when the plain implementation rounds the sublayers' inputs to bfloat16 and nothing else; where that alone
    comes near the limits (a stream that nearly cancels is divided by its small root mean square), three times it counts."""
    e = row_errs(out, ref)
    worst, q90, q50 = float(e.max()), float(np.quantile(e, 0.9)), float(np.quantile(e, 0.5))
    print(f"[observed] {what} {dt}: worst {worst:.3e}, nine in ten below {q90:.3e}, half below {q50:.3e}")
    assert np.isfinite(e).all()
    if dt == "float32":
        assert q90 < TOL[dt] / 2 and worst < 5 * TOL[dt], (what, worst, q90)
    else:
        n90, n50, nw = (np.quantile(noise, 0.9), np.quantile(noise, 0.5), noise.max()) if noise is not None else (0.0, 0.0, 0.0)
        assert q90 < max(TOL[dt], 3 * n90) and q50 < max(TOL[dt] / 2, 3 * n50) and worst < max(3 * TOL[dt], 3 * nw), (what, worst, q90, q50, nw, n90, n50)


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, (cfg, page, seed, rank) in cases.CASES.items():
        w = cases.draw_weights(cfg, seed, rank)
        for dt in ("float32", "bfloat16"):
            d = cases.write_model(tmp_path_factory.mktemp(f"d{name}{dt}"), cfg, w, DT[dt])
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


@pytest.mark.parametrize("seed", range(16))
def test_configurations_drawn_at_random(tmp_path, seed):
    """Sizes, order of layers, loop, windows, streams and constants drawn from a seed: a mixed schedule on few pages."""
    cfg, rank = cases.random_config(seed)
    w32 = cases.draw_weights(cfg, 100 + seed, rank)
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
def test_every_layer_run_against_the_plain_stream(models, name, dt):
    from litinfer_amd.engine import StepEntry
    cfg, page = cases.CASES[name][:2]
    d, reqs, _, w = models[(name, dt)]
    toks, streams, taps = reqs["r3"], [], []
    plain.forward(cfg, w, toks, streams)
    eng = _engine(d, dt, page, 256)
    eng.model.tap = lambda i, x: taps.append(x.detach().cpu().numpy().copy())
    eng.step([StepEntry("a", toks, [0])])
    assert len(taps) == len(streams) == len(plain.order(cfg))
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
def test_states_that_forget_slowly_across_portions(tmp_path, dt):
    """Decays near one and small removal rates: what the first tokens wrote still counts hundreds of tokens later, across
    portions cut at 1, 63, 64, 65, 128, 129 tokens."""
    cfg = {"architecture": "Dimelix", "vocab": 97, "width": 64, "norm": {"eps": 1e-6}, "streams": 2, "embedding": {"scale": 1.0},
           "layers": [cases.parallel((2, 1, 16, 0.25, 7), (3, 20), 0.2, 1.5, 96)]}
    w32 = cases.draw_weights(cfg, 9, 8, long_memory=True)
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
WINDOW = 21
A_TOK, B_TOK = 63, 62


def _standout_model(tmp, dt, kind, sizes, sink=None):
    """One layer whose weights make ONE key win: token A's key meets token B's query in every head with a score far above
    all others, and A's value is large.  Whether B sees A decides B's logits.  `sizes` = (heads, kv heads, dim)."""
    H, G, D = sizes
    scale = 40.0 / D if kind == "left" else 16.0 / D            # (a score of 40 or 16; the distance costs at most 1/2 a token)
    layer = {"attention": lambda: cases.attention(H, G, D, D, scale, 1e4, 4, 48),
             "latent": lambda: cases.latent(H, D, D, 32 if D == 16 else 64, scale, 48),
             "left": lambda: cases.parallel((H, G, D, scale, WINDOW), (2, 8), 1.0, 0.02, 48)}[kind]()
    cfg = {"architecture": "Dimelix", "vocab": 64, "width": 64, "norm": {"eps": 1e-6}, "streams": 3, "embedding": {"scale": 1.0}, "layers": [layer]}
    w = cases.draw_weights(cfg, 5, 4)
    w["embed"][:, :2] = 0.0
    w["embed"][A_TOK] = w["embed"][B_TOK] = 0.0
    w["embed"][A_TOK, 0] = w["embed"][B_TOK, 1] = 3.0
    for q in (1, 2):
        w[f"l0.hc{q}.in"][:], w[f"l0.norm{q}"][:] = np.abs(w[f"l0.hc{q}.in"]), 0.0
    p = "l0.mix.left." if kind == "left" else "l0.mix."
    rng = np.random.default_rng(1)
    for n in ("q", "k"):
        if p + n in w:
            w[p + n] *= 0.02
        if p + n + ".norm" in w:
            w[p + n + ".norm"][:] = 1.0
    u = np.ones(D) if kind != "attention" else np.r_[np.zeros(4), np.ones(D - 4)]          # (columns that are not rotated)
    if kind == "left":
        u = np.where(np.arange(D) % 3 == 0, -1.0, 1.0)
    for h in range(H):
        w[p + "q"][h * D:(h + 1) * D, 1] = u / 8.0 if kind == "latent" else u
    if kind == "latent":
        R = w[p + "dkv"].shape[0]
        d = np.where(np.arange(R) % 2 == 0, 1.0, -1.0)
        w[p + "dkv"] *= 0.5
        w[p + "dkv"][:, 0] = d                                  # A's latent is d
        w[p + "dkv.norm"][:] = 1.0
        w[p + "uk"] *= 0.05
        for h in range(H):
            w[p + "uk"][h * D:(h + 1) * D] += np.outer(u, d) / R
        w[p + "uv"] += 5.0 * rng.normal(size=(H * D, 1)) * d[None] / R
    else:
        for g in range(G):
            w[p + "k"][g * D:(g + 1) * D, 0] = u
        if kind == "attention":
            w[p + "v"][:, 0] += 6.0 * rng.normal(size=G * D)
            w[p + "sink"][:] = 0.0 if sink is None else sink
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
@pytest.mark.parametrize("kind", ["attention", "latent"])
def test_a_far_key_among_hundreds(tmp_path, dt, kind, sizes):
    cfg, w, d = _standout_model(tmp_path / "m", dt, kind, sizes)
    toks = np.random.default_rng(4).integers(0, 60, 420).tolist()
    toks[3], toks[400] = A_TOK, B_TOK
    ref = plain.forward(cfg, w, toks)
    assert _moved(cfg, w, toks, 3, 400, ref) > 0.2
    for cuts in ([0, 420], [0, 390, 420], [0, 2, 5, 399, 401, 420], [0, 398, 399, 400, 401, 402, 420]):
        out = _rows(_engine(d, dt, 16, 512), "a", toks, cuts)
        assert schedules.rel_err(out[395:], ref[395:]) < TOL[dt], cuts


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("how", ["prompt", "portions", "decoded"])
@pytest.mark.parametrize("kind", ["attention", "latent"])
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
    assert min(moved[:-1]) > 0.2 and moved[-1] < 1e-12, moved


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("how", ["prompt", "portions", "decoded"])
@pytest.mark.parametrize("sizes", SIZES)
def test_a_key_just_inside_and_just_outside_the_window(tmp_path, dt, how, sizes):
    """Distances window - 1 (seen) and window (not seen), the pair at page borders, the sequence's first tokens, far on."""
    cfg, w, d = _standout_model(tmp_path / "m", dt, "left", sizes)
    for pa in (0, 1, 7, 8, 30, 64, 90):
        for dist in (1, WINDOW - 1, WINDOW):
            pb = pa + dist
            toks = np.random.default_rng(pa).integers(0, 60, pb + 3).tolist()
            toks[pa], toks[pb] = A_TOK, B_TOK
            ref = plain.forward(cfg, w, toks)
            moved = _moved(cfg, w, toks, pa, pb, ref)
            assert (moved > 0.2) if dist < WINDOW else (moved < 0.05), (pa, dist, moved)
            out = _run_how(_engine(d, dt, 8, 192), toks, pa, pb, how)
            assert schedules.rel_err(out, ref) < TOL[dt], (pa, dist)


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", SIZES[:2])
def test_a_sink_that_outweighs_every_key(tmp_path, dt, sizes):
    """With a large sink nearly all weight goes to the term without a value.  Leaving it out, or counting it once a split
    of the keys, changes the logits by far more than the tolerance."""
    cfg, w, d = _standout_model(tmp_path / "m", dt, "attention", sizes, sink=9.0)
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


STEPS = ([(0, 1), (2, 5)], [(2, 1), (0, 2)], [(0, 1)], [(0, 20), (2, 2)], [(2, 15), (0, 16)], [(2, 100), (0, 1)], [(0, 199), (2, 64)], [(2, 65)])


@pytest.mark.parametrize("heads,N,vdim", [(3, 12, 12), (2, 8, 40), (4, 64, 64), (1, 128, 128), (2, 100, 20), (1, 256, 12), (3, 30, 30), (2, 5, 7),
                                          (1, 200, 6), (5, 16, 16), (1, 66, 66)])
@pytest.mark.parametrize("chunked", [False, True])
def test_channel_delta_rule_across_steps_and_slots(heads, N, vdim, chunked):
    """Two requests on slots 0 and 2 take turns with portions of 1 to 199 tokens; slot 1 is nobody's and stays as it is.
    `chunked`: portions of more than 64 tokens run as chunks side by side; else token after token."""
    from litinfer_amd.engine.workspace import Workspace
    from litinfer_amd.kernels import ops
    ws, rng = Workspace(DEV), np.random.default_rng(N + vdim)
    seqs, ref = {}, {}
    for s in (0, 2):
        L = sum(n for step in STEPS for sl, n in step if sl == s)
        r, k, a, low = (rng.normal(size=(L, heads, N)) for _ in range(4))
        v, k, low = rng.normal(size=(L, heads, vdim)), k * rng.uniform(0.2, 3.0, (L, heads, 1)), 3.0 * low
        k[L // 2] = 0.0                                                       # (a key of zeros has a unit key of zeros)
        flat = lambda x: x.reshape(L, -1)
        seqs[s] = (np.concatenate([flat(r), flat(k), flat(v), flat(a)], axis=1), flat(low))
        ref[s] = plain.channel_delta_rule(r, k, v, np.exp(-plain.DECAY_FACTOR * plain.sigmoid(low)), plain.sigmoid(a)).reshape(L, -1)
    state = torch.zeros(3, heads, N, vdim, device=DEV)
    state[1] = 7.0
    at = {0: 0, 2: 0}
    for step in STEPS:
        x = np.concatenate([seqs[s][0][at[s]:at[s] + n] for s, n in step])
        low = np.concatenate([seqs[s][1][at[s]:at[s] + n] for s, n in step])
        wide = torch.zeros(len(x), x.shape[1] + 3, device=DEV)                # (the rows lie inside a wider buffer)
        wide[:, 3:] = _f32(x)
        y = torch.empty(len(x), heads * vdim, device=DEV)
        ops.channel_delta(wide[:, 3:], _f32(low), state, _ctx([n for _, n in step], [s for s, _ in step]), y, heads, vdim, N,
                          ws=ws if chunked else None)
        want = np.concatenate([ref[s][at[s]:at[s] + n] for s, n in step])
        assert np.abs(y.cpu().numpy() - want).max() < 2e-5 * max(1.0, np.abs(want).max()), step
        for s, n in step:
            at[s] += n
    assert torch.all(state[1] == 7.0)


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,T,H", [(1, 3, 40), (2, 37, 72), (3, 300, 96), (4, 5, 1536), (4, 260, 5000), (5, 9, 33), (7, 2, 4104), (16, 11, 64), (3, 2, 9001)])
def test_streams_step(dt, n, T, H):
    """Read from equal streams, write from equal streams, write in place with two outputs and factors, read alone; the
    norm of the next reader beside the write; the sum over streams at chosen tokens."""
    from litinfer_amd.kernels import ops
    rng = np.random.default_rng(n + H)
    tol = 1e-5 if dt == "float32" else 1e-2
    x, y1, y2 = rng.normal(size=(T, H)), rng.normal(size=(T, H)), rng.normal(size=(T, H))
    w = {"h.in": rng.normal(size=n), "h.out": rng.normal(size=n), "h.mix": rng.normal(size=(n, n)) / n ** 0.5}
    nw, eps, rows = rng.normal(1, 0.2, H), 1e-4, torch.empty(T, H, dtype=DT[dt], device=DEV)
    win, wout, wmix, nwd = _f32(w["h.in"]), _f32(w["h.out"]), _f32(w["h.mix"]), _f32(nw)
    read = dict(read=win, weight=nwd, eps=eps, xn=rows)

    def rows_are(xs):
        want = plain.rms(plain.read_streams(xs, w, "h."), eps) * nw
        assert np.abs(rows.float().cpu().numpy() - want).max() < tol * np.abs(want).max()
    xs, xd = [x] * n, _f32(x)
    ops.hyper_step(xd, None, n, **read)
    rows_are(xs)
    st = torch.empty(T, n, H, device=DEV)
    ops.hyper_step(xd, st, n, _f32(y1), None, (1.0, 1.0), wmix, wout, **read)
    xs = plain.write_streams(xs, y1, w, "h.")
    rows_are(xs)
    ops.hyper_step(st, st, n, _f32(y1), _f32(y2), (0.6, -1.5), wmix, wout, **read)
    xs = plain.write_streams(xs, 0.6 * y1 - 1.5 * y2, w, "h.")
    rows_are(xs)
    ops.hyper_step(st, st, n, _f32(y2), None, (2.0, 1.0), wmix, wout)          # nobody reads
    xs = plain.write_streams(xs, 2.0 * y2, w, "h.")
    want = np.stack(xs, axis=1)
    assert np.abs(st.cpu().numpy() - want).max() < 1e-5 * np.abs(want).max()
    ops.hyper_step(st, None, n, **read)
    rows_are(xs)
    pick = rng.integers(0, T, 6).astype(np.int32)
    out = torch.empty(6, H, device=DEV)
    ops.stream_sum(st, out, torch.tensor(pick, device=DEV))
    assert np.abs(out.cpu().numpy() - sum(xs)[pick]).max() < 1e-5 * np.abs(sum(xs)).max()


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_small_kernels_of_the_design(dt):
    from litinfer_amd.kernels import ops
    rng = np.random.default_rng(0)
    tol = 1e-5 if dt == "float32" else 1e-2
    for T, I in ((37, 100), (3, 33)):
        u, out = rng.normal(0, 3, size=(T, I)), torch.empty(T, I, dtype=DT[dt], device=DEV)
        u[0, :3] = (0.0, 1e-7, -1e-7)
        ops.xielu(_f32(u), out, float(plain.softplus(0.3)), 0.5 + float(plain.softplus(-1.2)))
        want = plain.xielu(u, 0.3, -1.2)
        assert np.abs(out.float().cpu().numpy() - want).max() < tol * np.abs(want).max()
    x, out = rng.normal(0, 2, size=(9, 50)), torch.empty(9, 20, dtype=DT[dt], device=DEV)
    ops.tanh_rows(_f32(x)[:, 7:27], out)
    assert np.abs(out.float().cpu().numpy() - np.tanh(x[:, 7:27])).max() < tol
    for heads, dim in ((5, 24), (2, 300), (3, 1)):
        y, z, w = rng.normal(size=(19, heads * dim)), rng.normal(size=(19, heads * dim)), rng.normal(1, 0.2, heads * dim)
        out = torch.empty(19, heads * dim, dtype=DT[dt], device=DEV)
        ops.gated_group_norm(_f32(y), _f32(z), _f32(w), 1e-3, heads, out, gate_after=True, gate="sigmoid")
        want = plain.rms(y.reshape(19, heads, dim), 1e-3).reshape(19, -1) * w * plain.sigmoid(z)
        assert np.abs(out.float().cpu().numpy() - want).max() < tol * np.abs(want).max()
    table = torch.randn(30, 24).to(DT[dt])
    out = torch.empty(4, 24, device=DEV)
    ops.embedding(torch.tensor([3, 29, 0, 3], dtype=torch.int32, device=DEV), table.to(DEV), out, scale=1.75)
    assert torch.allclose(out.cpu(), 1.75 * table[[3, 29, 0, 3]].float(), rtol=1e-6)


@pytest.mark.parametrize("nh,nkv,dk,dv,rot", [(4, 2, 24, 16, 8), (8, 4, 64, 64, 64), (1, 1, 8, 8, 2), (6, 6, 10, 10, 0), (3, 1, 128, 128, 32), (2, 2, 260, 30, 4)])
@pytest.mark.parametrize("keys_are_values", [False, True])
def test_a_norm_for_every_head(nh, nkv, dk, dv, rot, keys_are_values):
    from litinfer_amd.kernels import ops
    if keys_are_values:
        dv = dk
    rng = np.random.default_rng(dk)
    T, page, n = 19, 8, nh * dk + nkv * dk + (0 if keys_are_values else nkv * dv)
    qkv = rng.normal(size=(T, n + 4))                                           # (the gates' columns ride behind)
    wq, wk, pos = rng.normal(1, 0.2, dk), rng.normal(1, 0.2, dk), np.arange(40, 40 + T)
    freq = np.array([300.0 ** (-2.0 * i / rot) for i in range(rot // 2)])
    cos, sin = (_f32(np.cos(pos[:, None] * freq)), _f32(np.sin(pos[:, None] * freq))) if rot else (None, None)
    slots = rng.permutation(5 * page)[:T].astype(np.int32)
    kc, vc = torch.zeros(5, nkv, page, dk, device=DEV), torch.zeros(5, nkv, page, dv, device=DEV)
    d = _f32(qkv)
    ops.qk_head_norm_store(d, nh, nkv, dk, dv, rot, _f32(wq), _f32(wk), 1e-5, cos, sin, torch.tensor(slots, device=DEV), kc, vc, page,
                           keys_are_values=keys_are_values)
    raw = qkv[:, nh * dk:(nh + nkv) * dk].reshape(T, nkv, dk)
    q = plain.rotate_pairs(plain.rms(qkv[:, :nh * dk].reshape(T, nh, dk), 1e-5) * wq, pos, 300.0, rot)
    k = plain.rotate_pairs(plain.rms(raw, 1e-5) * wk, pos, 300.0, rot)
    v = raw if keys_are_values else qkv[:, (nh + nkv) * dk:n].reshape(T, nkv, dv)
    assert np.abs(d[:, :nh * dk].cpu().numpy().reshape(T, nh, dk) - q).max() < 1e-5
    assert np.abs(d[:, n:].cpu().numpy() - qkv[:, n:]).max() < 1e-6
    for t in range(T):
        assert np.abs(kc[slots[t] // page, :, slots[t] % page].cpu().numpy() - k[t]).max() < 1e-5
        assert np.abs(vc[slots[t] // page, :, slots[t] % page].cpu().numpy() - v[t]).max() < 1e-6


def _attention_case(dtype, seg_specs, nh, nkv, dk, dv, page, window, seed, heads_kernel=None, sinks=True):
    """Random queries, keys and values for segments (context, queries) in shuffled pages, a gate an element, slopes, a
    window and, with `sinks`, a sink a head; returns the kernel's output and the plain one."""
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
    sink = torch.randn(nh, generator=g) * 2.0 if sinks else None
    slopes = torch.tensor([0.7 * 2.0 ** -h for h in range(nh)], dtype=torch.float32)
    gate = torch.randn(T, nh * dv + 8, generator=g)                             # (a view of columns inside wider rows)
    scale, refs, o = 1.0 / math.sqrt(dk), [], 0
    for s, (c, ql) in enumerate(seg_specs):
        k, v = torch.randn(c, nkv, dk, generator=g).to(dtype), torch.randn(c, nkv, dv, generator=g).to(dtype)
        for b in range(blocks[s]):
            n = min(page, c - b * page)
            if not window or b * page + n > c - ql - window + 1:                # (older pages have been given back)
                tab[s, b] = perm.pop()
                kc[tab[s, b], :, :n] = k[b * page:b * page + n].transpose(0, 1)
                vc[tab[s, b], :, :n] = v[b * page:b * page + n].transpose(0, 1)
        qq = np.zeros((c, nh, dk))
        qq[c - ql:] = q[o:o + ql].double().numpy()
        kk, vv = k.double().numpy(), v.double().numpy()
        out = np.zeros((ql, nh, dv))
        for i in range(ql):
            p = c - ql + i
            lo = max(0, p - window + 1) if window else 0
            for h in range(nh):
                sc = kk[lo:p + 1, h // (nh // nkv)] @ qq[p, h] * scale - float(slopes[h]) * (p - np.arange(lo, p + 1))
                mx = max(sc.max(), float(sink[h])) if sinks else sc.max()
                e = np.exp(sc - mx)
                out[i, h] = (e @ vv[lo:p + 1, h // (nh // nkv)]) / (e.sum() + (math.exp(float(sink[h]) - mx) if sinks else 0.0))
        refs.append(out.reshape(ql, -1) * plain.sigmoid(gate[o:o + ql, 4:4 + nh * dv].double().numpy()))
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
    out, gd, was = torch.empty(T, nh * dv, dtype=dtype, device=DEV), gate.to(DEV), ops._heads_kernel_pays
    if heads_kernel is not None:
        ops._heads_kernel_pays = lambda *a: bool(heads_kernel)
    try:
        ops.masked_attention(q.to(DEV).contiguous(), nh * dk, dk, out, kc.to(DEV), vc.to(DEV), meta, nh, nkv, dk, dv, page, window, 0, 0.0,
                             scale, ws=Workspace(DEV), sink=sink.to(DEV) if sinks else None, column_gate=gd[:, 4:4 + nh * dv], slopes=slopes.to(DEV))
    finally:
        ops._heads_kernel_pays = was
    return out.float().cpu().numpy(), np.concatenate(refs)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("window", [0, 40])
@pytest.mark.parametrize("segs,nh,nkv,dk,dv,page,heads_kernel", [
    ([(2, 2)], 1, 1, 4, 4, 16, None),                                          # the general kernel, one wave
    ([(100, 37), (33, 2), (300, 1), (70, 70)], 6, 3, 24, 40, 8, None),         # ... four and eight waves a (token, head)
    ([(700, 3), (5, 5)], 2, 1, 24, 16, 16, None),
    ([(100, 37), (33, 2), (300, 1), (70, 70), (64, 64), (1, 1)], 6, 3, 64, 64, 8, None),   # tiles of queries beside single tokens
    ([(700, 700)], 8, 2, 64, 64, 16, None),                                    # one long prompt: tiles whose keys are cut into splits
    ([(900, 1), (90, 1), (3, 1), (2500, 1)], 8, 4, 64, 64, 16, False),         # single tokens, rows over lanes, splits and their join
    ([(900, 1), (90, 1), (3, 1), (2500, 1)], 8, 2, 128, 128, 16, True),        # single tokens with the heads as a tile's columns
    ([(40, 1)], 4, 4, 128, 64, 8, False),                                      # no splits: the finishing step inside the kernel
    ([(40, 1)], 32, 1, 64, 64, 8, True),
    ([(300, 1), (7, 1)], 6, 1, 256, 256, 16, False),                           # long rows
])
def test_slopes_gates_and_sinks_in_every_attention_kernel(dtype, segs, nh, nkv, dk, dv, page, heads_kernel, window):
    got, ref = _attention_case(dtype, segs, nh, nkv, dk, dv, page, window, seed=dk + nh, heads_kernel=heads_kernel, sinks=window == 0)
    err = float(np.abs(got - ref).max() / np.abs(ref).max())
    assert err < (2e-5 if dtype is torch.float32 else 1.2e-2), err


@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
@pytest.mark.parametrize("T,nh,n_out,n_in", [(1, 3, 12, 28), (40, 2, 64, 96), (33, 5, 20, 16), (70, 4, 128, 64), (17, 1, 7, 5)])
def test_per_head_products_with_a_gate_an_element(dt, T, nh, n_out, n_in):
    from litinfer_amd.kernels import ops
    rng = np.random.default_rng(n_in)
    m = torch.tensor(rng.normal(size=(nh, n_out, n_in)) / n_in ** 0.5, dtype=torch.float32).to(DT[dt])
    x = torch.tensor(rng.normal(size=(T, nh * n_in)), dtype=torch.float32).to(DT[dt])
    gate = rng.normal(size=(T, nh * n_out + 4))
    out = torch.empty(T, nh * n_out, dtype=DT[dt], device=DEV)
    ops.headwise_linear(x.to(DEV), nh * n_in, n_in, m.to(DEV), out, nh * n_out, n_out, T, gate=_f32(gate)[:, 4:], gate_columns=True)
    want = np.einsum("hjk,thk->thj", m.double().numpy(), x.double().numpy().reshape(T, nh, n_in)).reshape(T, -1) * plain.sigmoid(gate[:, 4:])
    assert np.abs(out.float().cpu().numpy() - want).max() < (1e-5 if dt == "float32" else 1e-2) * np.abs(want).max()
