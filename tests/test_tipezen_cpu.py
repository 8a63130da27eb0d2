"""Tipezen on the CPU: configuration and registry, the model's description (tensor names, cache groups, states), pins of
the plain implementation's mechanisms (tests/plain_tipezen.py), and the engine's bookkeeping (pages, state slots, streams,
ragged batches) with the tests' slow stand-in for the kernels against the plain implementation."""
import copy
import math

import pytest
import torch

import helpers as H
import plain_tipezen as P
import tipezen_models as TM
from emulated_kernels import EmulatedKernels
from easy_gpt.cpp_amd import kernels
from easy_gpt.cpp_amd.config import ConfigError, TipezenConfig, resolve_architecture
from easy_gpt.cpp_amd.engine import Engine
from easy_gpt.cpp_amd.parts import LayerSpec, PartSpec, build_model
from easy_gpt.cpp_amd.weights import WeightsError, write_random_model

F64 = torch.float64


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    return {name: TM.write_model(str(tmp_path_factory.mktemp(f"tipezen_{name}")), cfg, seed) for name, (cfg, seed) in TM.CONFIGS.items()}


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
    assert resolve_architecture(TM.CONFIG_A).name == "Tipezen"
    cfg = TipezenConfig.from_dict(TM.CONFIG_A)
    assert (cfg.vocab, cfg.width, cfg.eps, cfg.streams, len(cfg.layers)) == (300, 64, 1e-6, 2, 5)
    m = cfg.layers[0].mixer
    assert cfg.layers[0].type == "retention" and cfg.layers[0].ff == 96
    assert (m.heads, m.dim, m.vdim, m.decay, m.rotation.base, m.rotation.dims) == (3, 16, 24, (0.9, 0.97, 0.6), 10000.0, 8)
    m = cfg.layers[1].mixer
    assert (m.heads, m.kv_heads, m.dim, m.vdim, m.scale, m.softcap, m.window, m.mixes_values) == (4, 2, 16, 24, 0.25, 5.0, 12, True)
    assert (m.rotation.factor, m.rotation.original, m.rotation.fast, m.rotation.slow) == (4.0, 64.0, 8.0, 1.0)
    assert cfg.layers[2].ff is None and cfg.layers[4].mixer.window is None
    plain = TipezenConfig.from_dict(TM.CONFIG_B)
    assert plain.layers[0].mixer.softcap is None and not plain.layers[0].mixer.mixes_values and plain.layers[2].mixer.rotation is None
    alone = copy.deepcopy(TM.CONFIG_A)
    del alone["layers"][4]["mixer"]["kv_heads"]
    assert TipezenConfig.from_dict(alone).layers[4].mixer.kv_heads == 2


@pytest.mark.parametrize("edit, key", [
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.pop("streams"), "streams"),
    (lambda c: c.update(streams=0), "streams"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c["layers"][0].update(type="mamba"), "type"),
    (lambda c: c["layers"][0]["mixer"].update(decay=[0.5]), "decay"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18), "dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(scaling={"factor": 2, "original": 8, "fast": 2, "slow": 1}), "scaling"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "kind"),
    (lambda c: c["layers"][0]["mlp"].pop("ff"), "ff"),
    (lambda c: c["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][1]["mixer"].update(heads=3), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"].update(softcap=-1.0), "softcap"),
    (lambda c: c["layers"][1]["mixer"].update(v_mix=3), "v_mix"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=7), "dims"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].pop("original"), "original"),
    (lambda c: c["layers"][2]["mixer"].update(vdim=20), "mixed"),
])
def test_a_wrong_configuration_is_refused_by_name(edit, key):
    cfg = copy.deepcopy(TM.CONFIG_A)
    edit(cfg)
    with pytest.raises(ConfigError, match=key):
        TipezenConfig.from_dict(cfg)


def test_the_description_names_every_tensor_groups_the_caches_and_sizes_the_states():
    model = build_model(resolve_architecture(TM.CONFIG_A).build_spec(TipezenConfig.from_dict(TM.CONFIG_A)))
    declared = {s.name: tuple(s.shape) for s in model.param_specs()}
    assert declared == {k: tuple(v.shape) for k, v in TM.draw_weights(TM.CONFIG_A, 1).items()}
    assert declared["l1.mix.g"] == (4, 64) and declared["l0.mix.g"] == (72, 64) and declared["l1.mix.vmix"] == ()
    assert declared["l2.hc1.mix"] == (2, 2) and "l2.hc2.mix" not in declared and "l2.ls2" not in declared and "l0.mix.norm" not in declared
    needs = {g.cache_ids: (g.need.window, tuple((t.name, t.dims) for t in g.need.tensors)) for g in model.cache_groups}
    assert needs == {(1,): (12, (("k", (2, 16)), ("v", (2, 24)))), (2,): (33, (("k", (2, 24)), ("v", (2, 24)))),
                     (4,): (None, (("k", (2, 8)), ("v", (2, 24))))}
    assert {i: s.shape for i, s in model.state_needs.items()} == {0: (3, 16, 24), 3: (2, 20, 8)}
    assert model.graph_safe


def test_a_layer_must_give_the_connections_that_its_arrangement_has():
    spec = resolve_architecture(TM.CONFIG_A).build_spec(TipezenConfig.from_dict(TM.CONFIG_A))
    bare = LayerSpec(block="connected", mixer=spec.layers[0].mixer, feed_forward=spec.layers[0].feed_forward, norms=spec.layers[0].norms)
    with pytest.raises(ValueError, match="connects the branches"):
        build_model(type(spec)(**{**spec.__dict__, "layers": (bare,) + spec.layers[1:]}))
    odd = LayerSpec(block="connected_mixer_only", mixer=spec.layers[2].mixer, feed_forward=None, connections=spec.layers[2].connections,
                    norms={"mixer": PartSpec("layernorm", dict(eps=1e-5, name="norm1", bias_name=None), prefix="l2.")})
    with pytest.raises(ValueError, match="RMS norm"):
        build_model(type(spec)(**{**spec.__dict__, "layers": spec.layers[:2] + (odd,) + spec.layers[3:]}))


def test_a_missing_tensor_is_named(tmp_path, emulated):
    path = TM.write_model(str(tmp_path / "m"), TM.CONFIG_A, 3, change=lambda w: w.pop("l2.hc1.out"))
    with pytest.raises(WeightsError) as e:
        Engine.from_dir(path, dtype="float32", device="cpu", page_size=4, max_tokens=32, max_requests=1)
    assert e.value.missing == ["l2.hc1.out"]


def test_random_weights_run_and_keep_the_streams_in_size(tmp_path, emulated):
    path = write_random_model(str(tmp_path / "m"), TM.CONFIG_C, seed=4, device="cpu")
    reqs = H.make_requests(411, [9], seed=1)
    ref = plain_rows(path, reqs)
    assert bool(torch.isfinite(ref["r0"]).all())
    eng = Engine.from_dir(path, dtype="float32", device="cpu", page_size=4, max_tokens=16, max_requests=1)
    H.assert_rows_match(H.replay(eng, H.trace_whole(reqs)), ref, 1e-5, "random weights")


# ----------------------------------------------------------------------------- pins of the plain mechanisms
def test_slow_frequencies_are_divided_along_a_ramp_and_the_rotation_grows():
    base, dims, factor, original = 100.0, 8, 4.0, 60.0
    f = [base ** (-2.0 * i / dims) for i in range(4)]
    place = lambda turns: dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = math.floor(place(4.0)), math.ceil(place(0.7))
    assert (lo, hi) == (0, 3)                            # pair 0 stays, pair 3 is divided, two lie on the ramp
    got, magnitude = P.rotation_frequencies(TM.rotation(base, dims, (factor, original, 4.0, 0.7)))
    for i in range(4):
        assert abs(got[i] - (f[i] * (1 - i / 3) + f[i] / factor * (i / 3))) < 1e-15
    assert abs(magnitude - (0.1 * math.log(4.0) + 1.0)) < 1e-15
    x = torch.randn(2, 1, dims, dtype=F64)
    y = P.rotate(x, torch.tensor([0, 5]), TM.rotation(base, dims, (factor, original, 4.0, 0.7)), "interleaved")
    assert torch.allclose(y[0], x[0] * magnitude) and torch.allclose(y.norm(dim=-1), x.norm(dim=-1) * magnitude)


def test_the_two_pairings_turn_their_places_by_the_positions_angle():
    rot = {"base": 1.0, "dims": 4}                       # base 1: every frequency is 1, the angle is the position
    x = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 5.0]]], dtype=F64).repeat(2, 1, 1)
    pos, c, s = torch.tensor([0, 1]), math.cos(1.0), math.sin(1.0)
    inter, half = P.rotate(x, pos, rot, "interleaved"), P.rotate(x, pos, rot, "half")
    assert torch.equal(inter[0], x[0]) and torch.equal(half[0], x[0])
    assert torch.allclose(inter[1, 0], torch.tensor([1 * c - 2 * s, 2 * c + 1 * s, 3 * c - 4 * s, 4 * c + 3 * s, 5.0], dtype=F64))
    assert torch.allclose(half[1, 0], torch.tensor([1 * c - 3 * s, 2 * c - 4 * s, 3 * c + 1 * s, 4 * c + 2 * s, 5.0], dtype=F64))


def test_one_joins_the_denominator_a_window_ends_where_it_says_and_scores_are_capped():
    t, w = 7, 3
    k = torch.zeros(t, 1, 2, dtype=F64)
    v = torch.eye(t, dtype=F64)[:, None, :]               # the value of token j is the j-th unit vector: outputs are weights
    out = P.capped_window_attention(torch.zeros(t, 1, 2, dtype=F64), k, v, 1.0, 5.0, w)[:, 0]
    for i in range(t):
        seen = range(max(0, i - w + 1), i + 1)
        for j in range(t):
            assert abs(float(out[i, j]) - (1.0 / (len(seen) + 1.0) if j in seen else 0.0)) < 1e-12
    # one key with a raw score of 8: its weight is e^s / (1 + e^s) with s = 2 tanh(8 / 2)
    q = torch.tensor([[[4.0, 0.0]]], dtype=F64)
    key = torch.tensor([[[4.0, 0.0]]], dtype=F64)
    s = 2.0 * math.tanh(4.0)
    assert abs(float(P.capped_window_attention(q, key, torch.ones(1, 1, 1, dtype=F64), 0.5, 2.0)) - math.exp(s) / (1 + math.exp(s))) < 1e-12
    # scores far below zero leave the denominator's one alone: the output vanishes
    assert float(P.capped_window_attention(q, -key, torch.ones(1, 1, 1, dtype=F64), 40.0)) < 1e-200


def test_the_constant_decay_scan_has_its_closed_form_and_goes_on_from_a_carried_state():
    t = 9
    ones = torch.ones(t, 2, 1, dtype=F64)
    o, s = P.constant_decay_scan(ones, ones, ones, (0.5, 0.9))
    for h, d in enumerate((0.5, 0.9)):
        for i in range(t):
            assert abs(float(o[i, h, 0]) - sum(d ** n for n in range(i + 1))) < 1e-12
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(t, 2, 3, generator=g, dtype=F64) for _ in range(3))
    whole, last = P.constant_decay_scan(q, k, v, (0.5, 0.9))
    first, carried = P.constant_decay_scan(q[:4], k[:4], v[:4], (0.5, 0.9))
    second, end = P.constant_decay_scan(q[4:], k[4:], v[4:], (0.5, 0.9), carried)
    assert torch.allclose(torch.cat([first, second]), whole) and torch.allclose(end, last)


def test_the_gates_activation_is_the_tanh_form_of_gelu():
    z = torch.linspace(-6, 6, 25, dtype=F64)
    assert torch.allclose(P.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    assert float((P.gelu_tanh(z) - torch.nn.functional.gelu(z)).abs().max()) > 1e-4


def test_streams_are_rewritten_at_once_from_the_old_ones_and_mixed_from_row_to_column():
    x = torch.tensor([[[1.0]], [[10.0]]], dtype=F64)
    y = torch.tensor([[100.0]], dtype=F64)
    w = {"in": torch.tensor([2.0, 0.5], dtype=F64), "out": torch.tensor([1.0, 3.0], dtype=F64),
         "mix": torch.tensor([[0.0, 1.0], [2.0, 0.0]], dtype=F64)}
    assert float(P.read_streams(x, w, "")) == 7.0
    new = P.write_streams(x, y, w, "")
    assert new[:, 0, 0].tolist() == [2 * 10 + 100, 1 + 300]


def test_the_first_layer_that_mixes_keeps_its_values_and_later_ones_mix_them(models):
    """The first mixing layer's lambda does nothing, a later one's does."""
    cfg, w = P.read_model(models["A"])
    tokens = H.make_requests(300, [9], seed=2)["r0"]
    base = P.forward(cfg, w, tokens)
    for name, moves in (("l1.mix.vmix", False), ("l2.mix.vmix", True), ("l4.mix.vmix", True)):
        changed = P.forward(cfg, {**w, name: w[name] + 0.4}, tokens)
        assert bool(float((changed - base).abs().max()) > 1e-3) == moves, name


# ----------------------------------------------------------------------------- the engine's bookkeeping
@pytest.mark.parametrize("name", ["A", "B", "D", "F"])
def test_cuttings_agree_with_plain(models, emulated, name):
    cfg = TM.CONFIGS[name][0]
    reqs = H.make_requests(cfg["vocab"], [5, 41, 1, 23], seed=11)
    ref = plain_rows(models[name], reqs)
    for page_size, trace in [(4, H.trace_whole(reqs)), (16, H.trace_last_decoded(reqs, 9)), (3, H.trace_portions(reqs))]:
        eng = Engine.from_dir(models[name], dtype="float32", device="cpu", page_size=page_size, max_tokens=64, max_requests=2)
        rows = H.replay(eng, trace)
        assert len(rows) == sum(len(v) for v in reqs.values())
        H.assert_rows_match(rows, ref, 1e-5, f"{name} page {page_size}")
        assert eng.cache.free_pages() == [p.num_pages for p in eng.cache.pools]


@pytest.mark.parametrize("name", ["A", "B"])
def test_mixed_batches_with_pages_and_state_slots_used_again(models, emulated, name):
    cfg = TM.CONFIGS[name][0]
    reqs = H.make_requests(cfg["vocab"], [23, 9, 37, 30, 14, 26, 3, 19], seed=3)
    ref = plain_rows(models[name], reqs)
    trace = H.trace_mixed(reqs, seed=1, max_live=3, decode_tail=5)
    need = H.max_live_tokens(trace, round_to=4)
    eng = Engine.from_dir(models[name], dtype="float32", device="cpu", page_size=4, max_tokens=need, max_requests=3)
    H.assert_rows_match(H.replay(eng, trace), ref, 1e-5, name)
    assert max(len(r["entries"]) for r in trace) == 3          # eight requests went through three state slots
