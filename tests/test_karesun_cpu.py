"""Karesun on the CPU: configuration and registry, the model's description (tensor names, cache groups, who writes and who reads
which), pins of the plain implementation's mechanisms (tests/plain_karesun.py), and the engine's bookkeeping (pages, windows of
readers and writers, ragged batches) with the tests' slow stand-in for the kernels against the plain implementation."""
import copy
import math

import pytest
import torch

import helpers as H
import karesun_models as KM
import plain_karesun as P
from emulated_kernels import EmulatedKernels
from easy_gpt.cpp_amd import kernels
from easy_gpt.cpp_amd.config import ConfigError, KaresunConfig, resolve_architecture
from easy_gpt.cpp_amd.engine import Engine
from easy_gpt.cpp_amd.parts import LayerSpec, ModelSpec, PartSpec, RunSpec, build_model
from easy_gpt.cpp_amd.parts.base import CacheNeed, make_part
from easy_gpt.cpp_amd.weights import WeightsError, write_random_model

F64 = torch.float64


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    return {name: KM.write_model(str(tmp_path_factory.mktemp(f"karesun_{name}")), cfg, seed) for name, (cfg, seed) in KM.CONFIGS.items()}


@pytest.fixture()
def emulated():
    kernels.use_backend(EmulatedKernels())
    yield
    kernels.use_backend(None)


def plain_rows(model_dir, reqs):
    cfg, w = P.read_model(model_dir)
    return {rid: P.forward(cfg, w, ids) for rid, ids in reqs.items()}


# ----------------------------------------------------------------------------- configuration and description
def test_the_design_is_found_by_its_name_and_every_size_is_read():
    assert resolve_architecture(KM.CONFIG_A).name == "Karesun"
    cfg = KaresunConfig.from_dict(KM.CONFIG_A)
    assert (cfg.vocab, cfg.width, cfg.max_positions, cfg.eps, cfg.embedding_scale, len(cfg.layers)) == (300, 64, 300, 1e-6, 1.5, 5)
    m = cfg.layers[1].mixer
    assert (m.heads, m.kv_heads, m.dim, m.vdim, m.scale, m.diff, m.softcap, m.window, m.kv_from) == (4, 2, 16, 24, 0.3, 0.2, 8.0, 7, 0)
    f = cfg.layers[1].mlp
    assert (f.kind, f.ff, f.experts, f.top, f.scale, f.identities, f.groups, f.keep_groups) == ("moe", 40, 6, 2, 1.7, 2, 4, 2)
    f = cfg.layers[3].mlp
    assert (f.identities, f.groups, f.keep_groups) == (0, 1, 1)
    assert cfg.layers[2].mlp is None and cfg.layers[0].mlp.kind == "dense" and cfg.layers[0].mixer.kv_from is None
    open_ended = KaresunConfig.from_dict(KM.CONFIG_B).layers
    assert open_ended[0].mixer.softcap is None and open_ended[1].mixer.window is None
    bare = copy.deepcopy(KM.CONFIG_A)
    del bare["embedding"], bare["layers"][1]["mlp"]["router"]["scale"], bare["layers"][1]["mlp"]["router"]["identity"]
    bare["layers"][1]["mlp"]["router"]["groups"] = None
    bare = KaresunConfig.from_dict(bare)
    assert bare.embedding_scale == 1.0 and bare.layers[1].mlp.scale == 1.0 and bare.layers[1].mlp.identities == 0


@pytest.mark.parametrize("edit, key", [
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.pop("max_positions"), "max_positions"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c["embedding"].update(scale="x"), "scale"),
    (lambda c: c["layers"][0].update(type="retention"), "type"),
    (lambda c: c["layers"][0]["mixer"].pop("diff"), "diff"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mixer"].update(heads=3), "kv_heads"),
    (lambda c: c["layers"][0]["mixer"].update(softcap=0.0), "softcap"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][1]["mixer"].update(kv_from=1), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=1), "kv_from"),
    (lambda c: c["layers"][1]["mixer"].update(dim=8), "equal"),
    (lambda c: c["layers"][0]["mlp"].update(kind="glu"), "kind"),
    (lambda c: c["layers"][0]["mlp"].pop("ff"), "ff"),
    (lambda c: c["layers"][1]["mlp"]["router"].pop("experts"), "experts"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(identity=1), "count"),
    (lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=5), "keep"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=5), "top"),
    (lambda c: c["layers"][1]["mlp"].pop("expert"), "expert"),
])
def test_a_wrong_configuration_is_refused_by_name(edit, key):
    cfg = copy.deepcopy(KM.CONFIG_A)
    edit(cfg)
    with pytest.raises(ConfigError, match=key):
        KaresunConfig.from_dict(cfg)


def test_the_description_names_every_tensor_and_caches_live_as_long_as_their_farthest_reader():
    model = build_model(resolve_architecture(KM.CONFIG_A).build_spec(KaresunConfig.from_dict(KM.CONFIG_A)))
    declared = {s.name: tuple(s.shape) for s in model.param_specs()}
    assert declared == {k: tuple(v.shape) for k, v in KM.draw_weights(KM.CONFIG_A, 1).items()}
    assert declared["l0.mix.q"] == (128, 64) and declared["l0.mix.k"] == (64, 64) and declared["l0.mix.lq1"] == (16,)
    assert "l1.mix.k" not in declared and "l1.mix.v" not in declared and declared["l1.mix.lk2"] == (16,)
    assert declared["l1.mlp.router"] == (8, 64) and declared["l1.mlp.correction"] == (8,) and "l1.mlp.e6.up" not in declared
    # layer 0 looks back 12 tokens, its readers 7 and 21; layer 2 looks back 33, its reader 5
    needs = {g.cache_ids: (g.need.window, tuple((t.name, t.dims) for t in g.need.tensors)) for g in model.cache_groups}
    assert needs == {(0,): (21, (("k", (2, 32)), ("v", (2, 24)))), (2,): (33, (("k", (3, 16)), ("v", (3, 16))))}
    assert [(r.cache, r.writes_cache) for r in model.spec.run_order] == [(0, True), (0, False), (2, True), (0, False), (2, False)]
    assert model.graph_safe and not model.state_needs


def test_a_cache_serves_readers_of_any_reach_but_not_of_other_tensors():
    a = CacheNeed.keys_and_values(2, 16, 12, 24, keep_first=3)
    b = CacheNeed.keys_and_values(2, 16, 30, 24, keep_first=1)
    assert a.joined(b) == CacheNeed.keys_and_values(2, 16, 30, 24, keep_first=3)
    assert a.joined(CacheNeed.keys_and_values(2, 16, None, 24)) == CacheNeed.keys_and_values(2, 16, None, 24)
    assert a.joined(CacheNeed.keys_and_values(2, 16, 12, 32)) is None


def test_a_head_of_two_maps_goes_without_what_it_does_not_take():
    base = dict(n_heads=4, n_kv_heads=2, key_dim=16, value_dim=16, scale=0.25, eps=1e-6, norm_queries_keys=False, difference=0.3)
    make = lambda **kw: make_part("mixer", PartSpec("normed_attention", {**base, **kw}), hidden_size=64)
    m = make()
    assert (m.key_dim, m.map_dim, m.q_width, m.k_width, m.v_width) == (32, 16, 128, 64, 32)
    reader = make(shares_cache=True)
    assert reader.cache_need() == m.cache_need() and (reader.k_width, reader.v_width) == (0, 0)
    for kw in (dict(sink=True), dict(sink=0.0), dict(gated="heads"), dict(gated=True), dict(norm_queries_keys=True), dict(key_dim=520)):
        with pytest.raises(ValueError):
            make(**kw)
    for kw in (dict(mixes_values=True), dict(norm_values=True)):
        with pytest.raises(ValueError, match="none of its own"):
            make(shares_cache=True, **kw)


def test_choices_must_fit_the_groups():
    base = dict(n_experts=6, top=3, intermediate_size=8, router_bias=False, routing="softmax_all", identities=2, normalized=False)
    make = lambda **kw: make_part("feed_forward", PartSpec("expert_mixture", {**base, **kw}), hidden_size=64)
    assert make(groups=4, keep_groups=2).outputs == 8
    for kw in (dict(groups=3), dict(groups=4, keep_groups=1), dict(groups=2, keep_groups=3), dict(top=9), dict(routing="softmax_top")):
        with pytest.raises(ValueError):
            make(**kw)


def test_a_missing_tensor_is_named_and_one_too_many_too(tmp_path, emulated):
    path = KM.write_model(str(tmp_path / "m"), KM.CONFIG_A, 3, change=lambda w: w.pop("l1.mix.lk1"))
    with pytest.raises(WeightsError) as e:
        Engine.from_dir(path, dtype="float32", device="cpu", page_size=4, max_tokens=32, max_requests=1)
    assert e.value.missing == ["l1.mix.lk1"]
    path = KM.write_model(str(tmp_path / "n"), KM.CONFIG_A, 3, change=lambda w: w.update({"l1.mix.k": w["l0.mix.k"]}))
    with pytest.raises(WeightsError) as e:
        Engine.from_dir(path, dtype="float32", device="cpu", page_size=4, max_tokens=32, max_requests=1)
    assert e.value.unexpected == ["l1.mix.k"]


def test_random_weights_run(tmp_path, emulated):
    path = write_random_model(str(tmp_path / "m"), KM.CONFIG_C, seed=4, device="cpu")
    reqs = H.make_requests(411, [9], seed=1)
    ref = plain_rows(path, reqs)
    assert bool(torch.isfinite(ref["r0"]).all())
    eng = Engine.from_dir(path, dtype="float32", device="cpu", page_size=4, max_tokens=16, max_requests=1)
    H.assert_rows_match(H.replay(eng, H.trace_whole(reqs)), ref, 1e-5, "random weights")


def test_a_request_does_not_outgrow_the_position_table(models, emulated):
    from easy_gpt.cpp_amd.engine import StepEntry

    eng = Engine.from_dir(models["A"], dtype="float32", device="cpu", page_size=16, max_tokens=400, max_requests=1)
    eng.add_request("a")
    with pytest.raises(ValueError):
        eng.step([StepEntry("a", [1] * 301, [])])


# ----------------------------------------------------------------------------- pins of the plain mechanisms
def test_a_norms_weight_is_its_distance_from_one():
    x = torch.tensor([[3.0, 4.0]], dtype=F64)
    y = P.offset_norm(x, torch.tensor([0.0, -0.5], dtype=F64), 0.0)
    assert torch.allclose(y, torch.tensor([[3.0, 2.0]], dtype=F64) / math.sqrt(12.5))
    assert torch.allclose(P.unit_rms(torch.zeros(1, 2, dtype=F64), 1e-6), torch.zeros(1, 2, dtype=F64))


def test_a_window_ends_where_it_says_and_scores_are_capped():
    t, w = 7, 3
    k = torch.zeros(t, 1, 2, dtype=F64)
    v = torch.eye(t, dtype=F64)[:, None, :]               # the value of token j is the j-th unit vector: outputs are weights
    out = P.capped_window_map(torch.zeros(t, 1, 2, dtype=F64), k, v, 1.0, 5.0, w)[:, 0]
    for i in range(t):
        seen = range(max(0, i - w + 1), i + 1)
        for j in range(t):
            assert abs(float(out[i, j]) - (1.0 / len(seen) if j in seen else 0.0)) < 1e-12
    # two keys with raw scores of 8 and 0: the weights are those of 2 tanh(8 / 2) and 0
    q = torch.tensor([[[0.0, 0.0]], [[4.0, 0.0]]], dtype=F64)
    key = torch.tensor([[[4.0, 0.0]], [[0.0, 4.0]]], dtype=F64)
    got = P.capped_window_map(q, key, torch.eye(2, dtype=F64)[:, None, :], 0.5, 2.0)[1, 0]
    s = 2.0 * math.tanh(4.0)
    assert abs(float(got[0]) - math.exp(s) / (math.exp(s) + 1.0)) < 1e-12


def test_lambda_is_one_number_made_of_four_vectors():
    w = {"lq1": [1.0, 2.0], "lk1": [0.5, -0.25], "lq2": [0.0, 1.0], "lk2": [3.0, -1.0]}
    w = {name: torch.tensor(v, dtype=F64) for name, v in w.items()}
    assert abs(P.map_weight(w, "", 0.3) - (math.exp(0.0) - math.exp(-1.0) + 0.3)) < 1e-12


def test_the_maps_share_values_and_their_difference_is_divided_by_its_root_mean_square():
    """Map 1 looks at the first of two tokens alone, map 2 at both alike: v0 - lambda (v0 + v1) / 2."""
    q = torch.zeros(2, 1, 2, 1, dtype=F64)
    k = torch.zeros(2, 1, 2, 1, dtype=F64)
    q[1, 0, 0, 0], k[0, 0, 0, 0] = 1.0, 1000.0
    v = torch.tensor([[[1.0, 0.0]], [[0.0, 3.0]]], dtype=F64)
    lam, diff = 0.5, 0.25
    raw = torch.tensor([1.0 - 0.25, -0.75], dtype=F64)
    got = P.two_maps(q, k, v, 1.0, None, None, lam, diff, 1e-5)[1, 0]
    assert torch.allclose(got, raw / math.sqrt(float((raw ** 2).mean()) + 1e-5) * 0.75)


def test_groups_choose_by_corrected_scores_and_weigh_by_plain_ones():
    z = torch.log(torch.tensor([[0.30, 0.05, 0.10, 0.15, 0.25, 0.15]], dtype=F64))          # scores are these numbers
    router = {"experts": 5, "top": 2, "scale": 3.0, "identity": 1, "groups": {"count": 3, "keep": 1}}
    idx, wt = P.route_scores(z, torch.zeros(6, dtype=F64), router)
    assert idx.tolist() == [[0, 1]]                               # within group 0, though 4 scores higher than 1
    assert torch.allclose(wt, torch.tensor([[0.9, 0.15]], dtype=F64))
    shift = torch.tensor([-1.0, -1.0, -0.5, -0.6, -0.9, -0.5], dtype=F64)                    # choice scores below zero
    idx, wt = P.route_scores(z, shift, router)
    assert idx.tolist() == [[5, 4]] and torch.allclose(wt, torch.tensor([[0.45, 0.75]], dtype=F64))      # not the masked ones
    idx, _ = P.route_scores(z, shift, {**router, "groups": {"count": 3, "keep": 2}})
    assert idx.tolist() == [[5, 2]]
    idx, _ = P.route_scores(z, shift, {**router, "groups": None})
    assert idx.tolist() == [[5, 2]]


def test_an_identity_expert_hands_its_input_on():
    g = torch.Generator().manual_seed(0)
    h = torch.randn(3, 4, generator=g, dtype=F64)
    w = {"router": torch.zeros(3, 4, dtype=F64), "correction": torch.tensor([0.0, 0.5, 1.0], dtype=F64)}
    for e in range(2):
        for name, shape in (("gate", (5, 4)), ("up", (5, 4)), ("down", (4, 5))):
            w[f"e{e}.{name}"] = torch.randn(shape, generator=g, dtype=F64)
    mlp = {"router": {"experts": 2, "top": 2, "scale": 1.5, "identity": 1}}
    assert torch.allclose(P.expert_mixture(h, w, "", mlp), 0.5 * h + 0.5 * P.gated_expert(h, w, "e1."))


def test_a_layer_reads_the_keys_it_names_with_its_own_queries_and_mask(models):
    """Changing layer 0's keys moves the output of its readers; layer 2's reader does not see them but through the stream."""
    cfg, w = P.read_model(models["A"])
    tokens = H.make_requests(300, [30], seed=2)["r0"]
    base = P.forward(cfg, w, tokens)
    narrower = copy.deepcopy(cfg)
    narrower["layers"][3]["mixer"]["mask"]["size"] = 20
    assert torch.equal(P.forward(narrower, w, tokens)[:20], base[:20])
    assert float((P.forward(narrower, w, tokens)[20:] - base[20:]).abs().max()) > 1e-3
    other = copy.deepcopy(cfg)
    other["layers"] = other["layers"][:4]
    moved = P.forward(other, {**w, "l3.mix.q": w["l3.mix.q"] * 0.5}, tokens)
    assert float((moved - P.forward(other, w, tokens)).abs().max()) > 1e-3


# ----------------------------------------------------------------------------- the engine's bookkeeping
@pytest.mark.parametrize("name", ["A", "B", "D"])
def test_cuttings_agree_with_plain(models, emulated, name):
    cfg = KM.CONFIGS[name][0]
    reqs = H.make_requests(cfg["vocab"], [5, 41, 1, 23], seed=11)
    ref = plain_rows(models[name], reqs)
    for page_size, trace in [(4, H.trace_whole(reqs)), (16, H.trace_last_decoded(reqs, 9)), (3, H.trace_portions(reqs))]:
        eng = Engine.from_dir(models[name], dtype="float32", device="cpu", page_size=page_size, max_tokens=64, max_requests=2)
        rows = H.replay(eng, trace)
        assert len(rows) == sum(len(v) for v in reqs.values())
        H.assert_rows_match(rows, ref, 1e-5, f"{name} page {page_size}")
        assert eng.cache.free_pages() == [p.num_pages for p in eng.cache.pools]


@pytest.mark.parametrize("name", ["A", "C"])
def test_mixed_batches_with_pages_used_again(models, emulated, name):
    """(the stand-in asserts that no page is read that was given back: a reader's window is wider than the writer's)"""
    cfg = KM.CONFIGS[name][0]
    reqs = H.make_requests(cfg["vocab"], [23, 9, 37, 30, 14, 26, 3, 19], seed=3)
    ref = plain_rows(models[name], reqs)
    trace = H.trace_mixed(reqs, seed=1, max_live=3, decode_tail=5)
    need = H.max_live_tokens(trace, round_to=4)
    eng = Engine.from_dir(models[name], dtype="float32", device="cpu", page_size=4, max_tokens=need, max_requests=3)
    H.assert_rows_match(H.replay(eng, trace), ref, 1e-5, name)


def test_readers_and_writers_of_one_cache_in_a_row_of_layers(emulated):
    """A reader before its writer, and two writers, are refused."""
    spec = resolve_architecture(KM.CONFIG_A).build_spec(KaresunConfig.from_dict(KM.CONFIG_A))
    with pytest.raises(ValueError, match="before any entry writes"):
        build_model(ModelSpec(**{**spec.__dict__, "run_order": (RunSpec(1, cache=0, writes_cache=False), RunSpec(0, cache=0))}))
    with pytest.raises(ValueError, match="two run-order entries"):
        build_model(ModelSpec(**{**spec.__dict__, "run_order": (RunSpec(0, cache=0), RunSpec(0, cache=0))}))
    with pytest.raises(ValueError, match="different needs"):
        build_model(ModelSpec(**{**spec.__dict__, "run_order": (RunSpec(0, cache=0), RunSpec(2, cache=0, writes_cache=False))}))


def test_parallel_streams_take_no_norm_whose_weight_is_a_distance():
    spec = resolve_architecture(KM.CONFIG_A).build_spec(KaresunConfig.from_dict(KM.CONFIG_A))
    layer = spec.layers[2]
    link = PartSpec("hyper_connection", dict(streams=2, names=dict(read="in", write="out", mix="mix")), prefix="x.")
    odd = LayerSpec(block="connected_mixer_only", mixer=layer.mixer, feed_forward=None, norms=layer.norms, connections={"mixer": link})
    with pytest.raises(ValueError, match="RMS norm"):
        build_model(ModelSpec(**{**spec.__dict__, "layers": spec.layers[:2] + (odd,) + spec.layers[3:]}))
