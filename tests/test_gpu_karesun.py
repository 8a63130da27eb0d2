"""Karesun models on the GPU against the plain implementation (tests/plain_karesun.py): every way of cutting requests into
steps, in float32 and bfloat16, on small configurations that differ in every size; mixed batches with pages used again, with and
without graphs; long decoding past every window; a key made to stand out in either map so that the query at the window's last
position sees it and the next one does not, read by the layer that made it or by one that looks farther back; a far key among
hundreds; batches of many single tokens; a batch against each request alone; pages that are used again; generation through the
entry point and the command line; bin/trace_run as a subprocess."""
import json
import os
import random
import subprocess
import sys

import numpy as np
import pytest
import torch

import helpers as H
import karesun_models as KM
import plain_karesun as P

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# as fractions of the largest logit: float32 is the rounding of float32 sums in another order; bfloat16 rounds activations
# between kernels (never the stream, statistics, scores, the maps' difference, the router or partial sums)
TOL = {"float32": 3e-5, "bfloat16": 4e-2}
# under bfloat16 a router's choice between two experts whose scores nearly tie may turn: a few rows may lie beyond the line
STRAY = {"float32": 0.0, "bfloat16": 0.03}


def match(rows, ref, dtype, what):
    H.assert_rows_match(rows, ref, TOL[dtype], what, may_exceed=STRAY[dtype])


# sizes of a real model's kind: maps of 64 and 32 with values of 128 and 64, windows of 96 and 130, a reader that looks farther back
CONFIG_E = KM.config(523, 320, 1700, 1e-6, 2.5, [
    (KM.mixer(4, 2, 64, 128, 0.06, 0.3, 96, 20.0), KM.dense(512)),
    (KM.mixer(4, 2, 64, 128, 0.07, 0.55, 200, 30.0, kv_from=0), KM.moe(96, 14, 4, 1.5, 2, (4, 2))),
    (KM.mixer(10, 2, 32, 64, 0.12, 0.7, 130, 15.0), KM.moe(64, 8, 2, 1.0)),
    (KM.mixer(10, 2, 32, 64, 0.1, 0.4, 130, 25.0, kv_from=2), None),
])
ALL = dict(KM.CONFIGS, E=(CONFIG_E, 9))


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    return {name: KM.write_model(str(tmp_path_factory.mktemp(f"karesun_{name}")), cfg, seed) for name, (cfg, seed) in ALL.items()}


@pytest.fixture(autouse=True)
def product_kernels():
    from easy_gpt.cpp_amd import kernels

    kernels.use_backend(None)
    assert kernels.backend().name == "hip-gfx950"


def engine(model_dir, dtype, **kw):
    from easy_gpt.cpp_amd.engine import Engine

    return Engine.from_dir(model_dir, dtype=dtype, device="cuda:0", **kw)


def plain_rows(model_dir, reqs):
    cfg, w = P.read_model(model_dir)
    return {rid: P.forward(cfg, w, ids) for rid, ids in reqs.items()}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C", "D", "E", "F"])
def test_every_cutting_agrees_with_plain(models, name, dtype):
    cfg = ALL[name][0]
    reqs = H.make_requests(cfg["vocab"], [150, 1, 47, 2, 96], seed=21)
    ref = plain_rows(models[name], reqs)
    cuttings = {"whole": H.trace_whole(reqs), "last decoded": H.trace_last_decoded(reqs, 40), "portions": H.trace_portions(reqs),
                "mixed": H.trace_mixed(reqs, seed=5, decode_tail=20)}
    for what, trace in cuttings.items():
        for page_size in (16, 32, 48) if what == "whole" else (16, 48) if what == "mixed" else (16,):
            eng = engine(models[name], dtype, page_size=page_size, max_tokens=H.max_live_tokens(trace, 64), max_requests=4)
            rows = H.replay(eng, trace)
            assert len(rows) == sum(len(v) for v in reqs.values())
            match(rows, ref, dtype, f"{name} {dtype} {what} pages of {page_size}")
            if name == "F":
                H.assert_rows_match(rows, ref, TOL[dtype], f"{name} {dtype} {what}")
            assert eng.cache.free_pages() == [p.num_pages for p in eng.cache.pools]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("use_graphs", [True, False])
@pytest.mark.parametrize("name", ["A", "F"])
def test_mixed_batches_with_pages_used_again(models, dtype, use_graphs, name):
    """Ten requests, four of them live, in a pool that holds a third of their tokens; with the decode steps replayed from graphs
    and kernel by kernel."""
    cfg = ALL[name][0]
    reqs = H.make_requests(cfg["vocab"], [70, 23, 110, 64, 37, 90, 5, 130, 49, 81], seed=33)
    ref = plain_rows(models[name], reqs)
    trace = H.trace_mixed(reqs, seed=9, decode_tail=24)
    eng = engine(models[name], dtype, page_size=16, max_tokens=H.max_live_tokens(trace, 16), max_requests=4, use_graphs=use_graphs)
    match(H.replay(eng, trace), ref, dtype, f"mixed {name} {dtype}")
    assert sum(-(-len(v) // 16) for v in reqs.values()) > 2 * max(p.num_pages for p in eng.cache.pools)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name, n", [("A", 300), ("C", 340), ("E", 340)])
def test_long_decoding_passes_every_window(models, name, n, dtype):
    """Three tokens as a prompt, then hundreds one by one, to the last row of the position table in the first model: windows of
    5 to 200 tokens pass over decoded tokens alone."""
    cfg = ALL[name][0]
    reqs = H.make_requests(cfg["vocab"], [n], seed=44)
    ref = plain_rows(models[name], reqs)
    eng = engine(models[name], dtype, page_size=16, max_tokens=384, max_requests=2)
    rows = H.replay(eng, H.trace_last_decoded(reqs, n - 3))
    assert len(rows) == n
    match(rows, ref, dtype, f"long decoding {name} {dtype}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["E", "F"])
def test_steps_of_many_single_tokens(models, name, dtype):
    """Twenty-one requests decode together (more rows than the fused kernels take), then fewer and fewer."""
    cfg = ALL[name][0]
    reqs = H.make_requests(cfg["vocab"], [20 + 3 * i for i in range(21)], seed=51)
    ref = plain_rows(models[name], reqs)
    trace = [H.step_record(0, [(rid, ids[:15], [14]) for rid, ids in reqs.items()])]
    for p in range(15, max(map(len, reqs.values()))):
        live = [(rid, [ids[p]], [0]) for rid, ids in reqs.items() if p < len(ids)]
        trace.append(H.step_record(p, live, [rid for rid, _, _ in live if len(reqs[rid]) == p + 1]))
    eng = engine(models[name], dtype, page_size=16, max_tokens=H.max_live_tokens(trace, 64), max_requests=21)
    match(H.replay(eng, trace), ref, dtype, f"many single tokens {name} {dtype}")


def _one_loud_key(cfg, loud):
    """Weights with which token 7 has a key that the queries of token 9 weigh far above all others in one of the maps: channel 0 of
    the embedding marks token 7 and channel 1 token 9, no layer writes those channels, and the first feature of map `loud` of every
    query and key head reads them alone."""

    def change(w):
        g = torch.Generator().manual_seed(1)
        width = w["embed"].shape[1]
        w["embed"][:] = 0.3 * torch.randn(w["embed"].shape, generator=g)
        w["pos"][:] *= 0.3
        w["embed"][:, :2] = 0.0
        w["pos"][:, :2] = 0.0
        for token, channel in ((7, 0), (9, 1)):
            w["embed"][token, :] = 0.0
            w["embed"][token, channel] = 6.0
        for i, entry in enumerate(cfg["layers"]):
            m, q = entry["mixer"], f"l{i}.mix."
            w[f"l{i}.norm1"][:] = 0.0
            w[q + "o"][:2, :] = 0.0
            for name, heads, channel in (("k", m["kv_heads"], 0), ("q", m["heads"], 1)):
                if q + name not in w:
                    continue
                proj = w[q + name]
                proj[:] = 0.3 * torch.randn(proj.shape, generator=g) / width ** 0.5
                proj[:, :2] = 0.0
                for head in range(heads):
                    row = (2 * head + loud) * m["dim"]
                    proj[row, :] = 0.0
                    proj[row, channel] = 0.6
        for name in w:
            w[name] = w[name].to(torch.bfloat16).to(torch.float32)

    return change


def _edge_cuts(reqs, rid, edges):
    n = len(reqs[rid])
    cut = list(zip([0] + edges, edges + [n]))
    return [H.step_record(s, [(rid, reqs[rid][a:b], list(range(b - a)))], [rid] if b == n else []) for s, (a, b) in enumerate(cut)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("loud", [0, 1])
@pytest.mark.parametrize("window, dim, vdim, reader", [(5, 16, 16, False), (64, 16, 16, False), (100, 12, 20, False), (33, 64, 48, False),
                                                       (64, 16, 32, True), (41, 11, 13, True)])
def test_a_loud_key_is_seen_to_the_windows_last_position_and_not_beyond(tmp_path, dtype, loud, window, dim, vdim, reader):
    """One key stands out at position `window`.  Asking tokens at the last position whose window holds it and at the next
    one: as a whole prompt, in portions cut just before and just after the edge, and decoded one by one; against the plain
    implementation, which also shows that the two rows differ by far more than the tolerance.  With `reader` the window is that of
    a layer that reads the keys of an earlier one whose own window is 6."""
    mixers = [(KM.mixer(4, 2, dim, vdim, 1.0, 0.5, window, 12.0), None)]
    if reader:
        mixers = [(KM.mixer(4, 2, dim, vdim, 1.0, 0.4, 6, 12.0), None), (KM.mixer(4, 2, dim, vdim, 1.0, 0.5, window, 12.0, kv_from=0), None)]
    cfg = KM.config(64, 48, 400, 1e-5, 1.0, mixers)
    path = KM.write_model(str(tmp_path / "m"), cfg, 3, change=_one_loud_key(cfg, loud))
    n = 3 * window + 2
    tokens = torch.randint(10, 64, (n,), generator=torch.Generator().manual_seed(window)).tolist()
    tokens[window] = 7
    for p in (2 * window - 1, 2 * window, 2 * window - 2, 2 * window + 1, window - 1):
        tokens[p] = 9
    c, w = P.read_model(path)
    want = P.forward(c, w, tokens)
    without = P.forward(c, w, tokens[:window] + [11] + tokens[window + 1 :])
    moved = (want - without).abs().amax(-1) / want.abs().max()
    assert float(moved[2 * window - 1]) > 0.2 and (reader or float(moved[2 * window]) < 1e-9)
    reqs = {"r0": tokens}
    for what, trace in [("whole", H.trace_whole(reqs)), ("decoded", H.trace_last_decoded(reqs, n - window - 1)),
                        ("portions", _edge_cuts(reqs, "r0", [2 * window - 1, 2 * window + 1])), ("small portions", H.trace_portions(reqs))]:
        eng = engine(path, dtype, page_size=16, max_tokens=-(-n // 64) * 64, max_requests=1)
        H.assert_rows_match(H.replay(eng, trace), {"r0": want}, TOL[dtype], f"window {window} {dtype} {what}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("dim, vdim, loud", [(12, 20, 0), (32, 32, 1)])
def test_a_far_token_among_hundreds_reaches_the_queries(tmp_path, dtype, dim, vdim, loud):
    """One token stands out at position 3 of 700 (and then the first one of all), without a window.  Asking tokens at positions 650
    to 699, as a whole prompt, in portions and decoded one by one, against the plain implementation, which also shows that the
    rows differ by far more than the tolerance from those of the same prompt without that token."""
    cfg = KM.config(64, 48, 700, 1e-5, 1.0, [(KM.mixer(3, 1, dim, vdim, 1.0, 0.3, None, 14.0), None)])
    path = KM.write_model(str(tmp_path / "m"), cfg, 4, change=_one_loud_key(cfg, loud))
    n = 700
    for far in (3, 0):
        tokens = torch.randint(10, 64, (n,), generator=torch.Generator().manual_seed(5)).tolist()
        tokens[far] = 7
        asks = [650, 677, 698, 699]
        for p in asks:
            tokens[p] = 9
        c, w = P.read_model(path)
        want = P.forward(c, w, tokens)
        without = P.forward(c, w, tokens[:far] + [11] + tokens[far + 1 :])
        for p in asks:
            assert float((want[p] - without[p]).abs().max()) > 0.2 * float(want[p].abs().max())
        reqs = {"r0": tokens}
        for what, trace in [("whole", H.trace_whole(reqs)), ("decoded", H.trace_last_decoded(reqs, 60)), ("portions", H.trace_portions(reqs))]:
            eng = engine(path, dtype, page_size=16, max_tokens=704, max_requests=1)
            rows = {key: row for key, row in H.replay(eng, trace).items() if key[1] in asks or key[1] < 4}
            H.assert_rows_match(rows, {"r0": want}, TOL[dtype], f"far token {dtype} {what}")


def test_pages_that_are_used_again_hold_nothing_of_before(models):
    """A request on the pages of a finished one gets what it gets in a new engine, bit for bit (float32)."""
    from easy_gpt.cpp_amd.engine import StepEntry

    name = "C"
    reqs = H.make_requests(ALL[name][0]["vocab"], [60, 45], seed=12)
    first = engine(models[name], "float32", page_size=16, max_tokens=64, max_requests=1)
    first.add_request("b")
    first.step([StepEntry("b", reqs["r1"][:20], [])])
    alone = first.step([StepEntry("b", reqs["r1"][20:], [24])]).cpu().clone()
    eng = engine(models[name], "float32", page_size=16, max_tokens=64, max_requests=1)
    eng.add_request("a")
    eng.step([StepEntry("a", reqs["r0"], [59])])
    eng.finish("a")
    eng.add_request("b")
    eng.step([StepEntry("b", reqs["r1"][:20], [])])
    assert torch.equal(eng.step([StepEntry("b", reqs["r1"][20:], [24])]).cpu(), alone)


def test_a_batch_gives_each_request_what_it_gets_alone(models):
    """float32: the logits of a request in a batch of unequal requests against the same request alone."""
    from easy_gpt.cpp_amd.engine import StepEntry

    name = "E"
    reqs = H.make_requests(ALL[name][0]["vocab"], [90, 7, 33, 64], seed=55)
    eng = engine(models[name], "float32", page_size=16, max_tokens=512, max_requests=4)
    for rid in reqs:
        eng.add_request(rid)
    together = eng.step([StepEntry(rid, ids, [len(ids) - 1]) for rid, ids in reqs.items()]).cpu().clone()
    scale = float(together.abs().max())
    for i, (rid, ids) in enumerate(reqs.items()):
        eng.finish(rid)
        eng.add_request(rid)
        alone = eng.step([StepEntry(rid, ids, [len(ids) - 1])]).cpu()
        assert float((alone[0] - together[i]).abs().max()) <= 2e-6 * scale, rid


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_prompt_of_1500_tokens_in_one_step_then_single_tokens(models, dtype):
    name = "E"
    reqs = H.make_requests(ALL[name][0]["vocab"], [1510], seed=88)
    ref = plain_rows(models[name], reqs)
    eng = engine(models[name], dtype, page_size=16, max_tokens=1536, max_requests=1)
    trace = H.trace_last_decoded(reqs, 10)
    for rec in trace:                     # the logits of the last 200 tokens of the prompt and of the decoded ones
        for e in rec["entries"]:
            e["want"] = [i for i in e["want"] if len(e["tokens"]) == 1 or i >= len(e["tokens"]) - 200]
    rows = H.replay(eng, trace)
    assert len(rows) == 210
    H.assert_rows_match(rows, ref, 1e-4 if dtype == "float32" else TOL[dtype], f"long prompt {dtype}", may_exceed=STRAY[dtype])


def draw_config(seed: int) -> dict:
    """A configuration drawn at random: head counts, sizes that are multiples of 16 and of nothing, windows of readers and
    writers, experts, groups and constants that no hand-made configuration has."""
    r = random.Random(seed)
    round16 = r.random() < 0.5                                   # half of them with sizes that the matrix-core kernels take
    size = (lambda lo, hi: 16 * r.randint(max(1, lo // 16), hi // 16)) if round16 else (lambda lo, hi: r.randint(lo, hi))
    width = 8 * r.randint(6, 40) if r.random() < 0.7 else r.randint(40, 200)
    window = lambda: r.choice([None, 1, 2, r.randint(3, 40), r.randint(41, 130), 1000])
    layers = []
    for i in range(r.randint(2, 6)):
        own = [j for j, (m, _) in enumerate(layers) if "kv_from" not in m]
        diff, cap = r.choice([0.0, 0.1, 0.3, 0.5, 0.8]), r.choice([None, 3.0, 10.0, 50.0])
        if own and r.random() < 0.5:
            j = r.choice(own)
            src = layers[j][0]
            mixer = KM.mixer(src["kv_heads"] * r.choice([1, 2, 3]), src["kv_heads"], src["dim"], src["vdim"], src["scale"] * r.choice([1.0, 0.7]),
                             diff, window(), cap, kv_from=j)
        else:
            kv, dim = r.choice([1, 2, 3, 4]), size(4, 96)
            mixer = KM.mixer(kv * r.choice([1, 1, 2, 3]), kv, dim, size(8, 128), dim ** -0.5 * r.choice([1.0, 1.5]), diff, window(), cap)
        if r.random() < 0.2:
            ff = None
        elif r.random() < 0.4:
            ff = KM.dense(r.randint(16, 300))
        else:
            outputs = r.randint(2, 24)
            groups = r.choice([g for g in range(1, outputs + 1) if outputs % g == 0])
            keep = r.randint(1, groups)
            ff = KM.moe(r.randint(8, 90), r.randint(1, outputs), r.randint(1, min(6, outputs // groups * keep)), r.choice([0.5, 1.0, 2.5]), 0,
                        (groups, keep) if r.random() < 0.8 else None)
            ff["router"]["identity"] = outputs - ff["router"]["experts"]
        layers.append((mixer, ff))
    return KM.config(r.randint(60, 700), width, r.randint(140, 600), r.choice([1e-6, 1e-5, 1e-3]), r.choice([0.5, 1.0, 4.0]), layers)


@pytest.mark.parametrize("seed", list(range(300, 316)))
def test_a_configuration_drawn_at_random(tmp_path, seed):
    cfg = draw_config(seed)
    path = KM.write_model(str(tmp_path / "m"), cfg, seed)
    reqs = H.make_requests(cfg["vocab"], [140, 1, 37, 2, 75], seed=seed)
    ref = plain_rows(path, reqs)
    cuttings = {"whole": H.trace_whole(reqs), "last decoded": H.trace_last_decoded(reqs, 33), "portions": H.trace_portions(reqs, seed),
                "mixed": H.trace_mixed(reqs, seed=seed, decode_tail=16)}
    for what, trace in cuttings.items():
        eng = engine(path, "float32", page_size=16, max_tokens=H.max_live_tokens(trace, 64), max_requests=4)
        H.assert_rows_match(H.replay(eng, trace), ref, 5e-5, f"seed {seed} {what}: {cfg['layers']}")
    eng = engine(path, "bfloat16", page_size=16, max_tokens=H.max_live_tokens(cuttings["mixed"], 64), max_requests=4)
    H.assert_rows_match(H.replay(eng, cuttings["mixed"]), ref, 5e-2, f"seed {seed} bfloat16 mixed", may_exceed=0.05)


@pytest.mark.parametrize("name, dtype", [("A", "float32"), ("F", "float32"), ("F", "bfloat16")])
def test_greedy_generation_through_the_entry_point(models, name, dtype):
    """(bfloat16 on a model without routers, where every token must be a near best one)"""
    from easy_gpt.cpp_amd.generate import LLM

    prompts = list(H.make_requests(ALL[name][0]["vocab"], [5, 40, 17, 1, 33, 8], seed=66).values())
    llm = LLM(models[name], dtype=dtype, cache_tokens=1024, prefill_chunk=16)
    outs = llm.generate(prompts, max_new_tokens=24, greedy=True, ignore_eos=True)
    c, w = P.read_model(models[name])
    for prompt, out in zip(prompts, outs):
        assert len(out) == 24
        logits = P.forward(c, w, prompt + out)
        for i, tok in enumerate(out):
            row = logits[len(prompt) + i - 1]
            gap = float(row.max() - row[tok])
            assert gap <= (1e-4 if dtype == "float32" else 5e-2) * float(row.abs().max()), (dtype, i, tok, gap)


def test_generation_under_page_pressure_gives_the_tokens_of_a_run_with_room(models):
    """Requests that are preempted and computed again: what they generate is the plain model's choice."""
    from easy_gpt.cpp_amd.generate import LLM

    name = "A"
    prompts = list(H.make_requests(ALL[name][0]["vocab"], [50, 70, 30, 90, 20, 60, 45, 80], seed=67).values())
    tight = LLM(models[name], dtype="float32", cache_tokens=400, prefill_chunk=32)
    c, w = P.read_model(models[name])
    for prompt, out in zip(prompts, tight.generate(prompts, max_new_tokens=40, greedy=True, ignore_eos=True)):
        assert len(out) == 40
        logits = P.forward(c, w, prompt + out)
        for i, tok in enumerate(out):
            row = logits[len(prompt) + i - 1]
            assert float(row.max() - row[tok]) <= 1e-4 * float(row.abs().max()), (i, tok)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run_as_a_subprocess(models, tmp_path, dtype):
    name = "B" if dtype == "float32" else "C"
    cfg = ALL[name][0]
    reqs = H.make_requests(cfg["vocab"], [70, 23, 110, 37, 55], seed=77)
    ref = plain_rows(models[name], reqs)
    trace = H.trace_mixed(reqs, seed=4, decode_tail=32, want_all=False)
    out_dir = str(tmp_path / "out")
    cmd = [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", models[name], "--dtype", dtype, "--out", out_dir,
           "--max-tokens", str(H.max_live_tokens(trace, 64))]
    p = subprocess.Popen(cmd, stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
    rows, fed = {}, {}
    for rec in trace:
        p.stdin.write(json.dumps(rec) + "\n")
        p.stdin.flush()
        assert p.stdout.readline().strip() == f"done {rec['step']}"
        wanted = sum(len(e["want"]) for e in rec["entries"])
        if wanted:
            data = np.fromfile(os.path.join(out_dir, f"{rec['step']}.f32"), dtype="<f4").reshape(wanted, cfg["vocab"])
            r = 0
            for e in rec["entries"]:
                for want in e["want"]:
                    rows[(e["id"], fed.get(e["id"], 0) + want)] = torch.from_numpy(data[r].copy())
                    r += 1
        for e in rec["entries"]:
            fed[e["id"]] = fed.get(e["id"], 0) + len(e["tokens"])
    p.stdin.close()
    assert p.wait(timeout=60) == 0
    assert len(rows) > 60
    match(rows, ref, dtype, f"trace_run {dtype}")


def test_the_command_line_generates_with_a_karesun_folder(models):
    name = "A"
    prompt = [5, 17, 3, 250, 9, 44, 1]
    cmd = [sys.executable, os.path.join(ROOT, "bin", "easy_llm"), "--model", models[name], "--dtype", "float32", "--greedy",
           "--ignore-eos", "--max-new-tokens", "12"]
    p = subprocess.run(cmd + [" ".join(map(str, prompt))], capture_output=True, text=True, timeout=110, cwd=ROOT)
    assert p.returncode == 0, p.stderr[-2000:]
    c, w = P.read_model(models[name])
    out = [int(t) for t in p.stdout.split()]
    assert len(out) == 12
    logits = P.forward(c, w, prompt + out)
    for i, tok in enumerate(out):
        row = logits[len(prompt) + i - 1]
        assert float(row.max() - row[tok]) <= 1e-4 * float(row.abs().max()), (i, tok)
