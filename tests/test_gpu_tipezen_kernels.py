"""The kernels and operands that the Tipezen design brought, each alone against the plain functions of
tests/plain_tipezen.py: heads that are rotated and stored without a norm, with values mixed and handed on and a gate per
head; the attention with capped scores, a constant sink and a gate per head; parallel residual streams rewritten, summed and
normed; a linear attention with a constant decay, in chunks, token by token and by the general state scan; the gelu gate in
every kernel of the gated feed-forward."""
import math

import pytest
import torch

import plain_tipezen as P
from test_gpu_bubetar_kernels import dev_ints, product, scan_setup
from test_gpu_head_kernels import close, paged, rnd

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F64 = torch.float64
I32 = torch.int32


@pytest.fixture(scope="module")
def k():
    from easy_gpt.cpp_amd import kernels

    kernels.use_backend(None)
    return kernels.backend()


def rope(k, rot, positions):
    """(the step's table on the device, the factor on cosines and sines)"""
    f, magnitude = P.rotation_frequencies(rot)
    return k.rope_table(positions.to(DEV), torch.tensor(f, dtype=torch.float32, device=DEV)), magnitude


# ----------------------------------------------------------------------------- head preparation
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nq, nkv, dk, dv, rot, pairing, splits, n_gates, t", [
    (4, 2, 16, 24, 8, "interleaved", 2, 4, 9),
    (6, 3, 11, 13, 10, "interleaved", 1, 6, 9),                  # an odd head: one place passes alone
    (3, 1, 32, 8, 32, "half", 0, 0, 9),
    (2, 2, 9, 5, 0, "half", 3, 2, 1),                            # no rotation at all
    (6, 2, 64, 48, 64, "interleaved", 1, 6, 301),                # a prompt: eight tokens side by side, the last ones fewer
    (5, 1, 7, 17, 4, "half", 0, 3, 262),
])
@pytest.mark.parametrize("normed", [False, True])
def test_heads_are_rotated_stored_mixed_and_gated(k, dtype, nq, nkv, dk, dv, rot, pairing, splits, n_gates, t, normed):
    page_size, eps, lam = 16, 1e-5, 0.375
    used = (nq + nkv) * dk + nkv * dv
    width = used + 3 + n_gates + 2
    given, x = product(rnd(t, width, seed=1, scale=2.0), dtype, splits)
    positions = (torch.arange(t) * 7 % 61).to(I32)          # (float32 angles: their error grows with the position)
    table = {"base": 1000.0, "dims": rot, "scaling": {"factor": 3.0, "original": 50, "fast": 4.0, "slow": 0.5}} if rot else {"base": 1.0, "dims": 0}
    unit = (lambda a: P.rms_norm(a, None, eps)) if normed else (lambda a: a)
    turn = lambda a: P.rotate(unit(a), positions, table, pairing)
    q = turn(x[:, : nq * dk].view(t, nq, dk))
    key = turn(x[:, nq * dk : (nq + nkv) * dk].view(t, nkv, dk))
    val = x[:, (nq + nkv) * dk : used].view(t, nkv, dv)
    first = rnd(t, nkv * dv, seed=4)
    mixed = (1 - lam) * val + lam * first.to(F64).view(t, nkv, dv)
    pages = -(-t // page_size) + 2
    slots = torch.randperm(pages * page_size, generator=torch.Generator().manual_seed(5))[:t].to(I32)
    page, off = (slots // page_size).long().to(DEV), (slots % page_size).long().to(DEV)
    rotation = {}
    if rot:
        cos_sin, magnitude = rope(k, table, positions)
        rotation = dict(cos_sin=cos_sin, rotary_dim=rot, pairing=pairing, magnitude=magnitude)
    for mix_with in (None, first.to(DEV)):
        k_cache = torch.full((pages, nkv, page_size, dk), 7.0, dtype=dtype, device=DEV)
        v_cache = torch.full((pages, nkv, dv, page_size), 7.0, dtype=dtype, device=DEV)
        q_out = torch.empty((t, nq * dk), dtype=dtype, device=DEV)
        values = torch.empty((t, nkv * dv), dtype=torch.float32, device=DEV)
        gates = torch.empty((t, n_gates), dtype=torch.float32, device=DEV) if n_gates else None
        k.head_norm_store(given, q_out, None, None, eps, False, slots.to(DEV), k_cache, v_cache, nq, nkv, dk, dv, page_size,
                          row_width=width, norm_plain=normed, values_out=values, mix_with=mix_with, mix=lam, gates_out=gates,
                          gate_offset=used + 3, **rotation)
        close(q_out, q.reshape(t, nq * dk), dtype, "queries")
        close(k_cache[page, :, off, :], key, dtype, "keys in their pages")
        close(v_cache[page, :, :, off], val if mix_with is None else mixed, dtype, "values in their pages")
        close(values, val.reshape(t, nkv * dv), torch.float32, "values handed on")
        if n_gates:
            close(gates, torch.sigmoid(x[:, used + 3 : used + 3 + n_gates]), torch.float32, "gates")
        held = torch.zeros((pages, page_size), dtype=torch.bool)
        held[page.cpu(), off.cpu()] = True
        free = (~held).nonzero()
        assert bool((k_cache[free[:, 0], :, free[:, 1], :] == 7.0).all()) and bool((v_cache[free[:, 0], :, :, free[:, 1]] == 7.0).all())


# ----------------------------------------------------------------------------- attention
def run(k, q, k_cache, v_cache, table, kv_len, page_size, scale, window, softcap, sink, gate, dv):
    m, nq, dk = q.shape
    nkv = k_cache.shape[1]
    out = torch.empty((m, nq * dv), dtype=q.dtype, device=DEV)
    k.window_attention(q.reshape(m, nq * dk).to(DEV).contiguous(), out, k_cache, v_cache, table, dev_ints([0]), dev_ints([m]), dev_ints([kv_len]),
                       nq, nkv, dk, dv, page_size, scale, window, 0, sink, m, kv_len, softcap=softcap, head_gate=gate)
    return out.view(m, nq, dv)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nq, nkv, dk, dv", [(4, 2, 16, 32), (8, 2, 64, 64), (6, 1, 128, 96), (3, 3, 11, 13), (2, 1, 40, 24)])
@pytest.mark.parametrize("window, softcap", [(0, 3.0), (70, 1.5), (12, None), (1, 30.0)])
def test_attention_with_capped_scores_a_constant_sink_and_gates(k, dtype, nq, nkv, dk, dv, window, softcap):
    n, ps = 150, 16
    keys, values = rnd(n, nkv, dk, seed=11).to(dtype), rnd(n, nkv, dv, seed=12).to(dtype)
    q = rnd(n, nq, dk, seed=13, scale=2.5).to(dtype)
    gate = torch.rand(n, nq, generator=torch.Generator().manual_seed(14))
    scale = 1.7 / math.sqrt(dk)
    k_cache, v_cache, table = paged(keys, values, ps, dtype, seed=15)
    want = P.capped_window_attention(q.to(F64), keys.to(F64), values.to(F64), scale, softcap, window or None)
    if softcap:                                           # the cap bends the large scores: without it rows differ visibly
        bare = P.capped_window_attention(q.to(F64), keys.to(F64), values.to(F64), scale, None, window or None)
        assert window == 1 or softcap > 10 or float((bare - want).abs().max()) > 0.1
    want = want * gate.to(F64)[:, :, None]
    sink = torch.zeros(nq, dtype=torch.float32, device=DEV)
    for first, m in [(0, n), (37, 50), (95, 2), (0, 1), (149, 1), (63, 1), (64, 1)]:
        got = run(k, q[first : first + m], k_cache, v_cache, table, first + m, ps, scale, window, softcap, sink,
                  gate[first : first + m].contiguous().to(DEV), dv)
        close(got, want[first : first + m], dtype, f"rows {first}..{first + m}")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_far_key_stands_out_below_its_cap_and_is_lost_behind_the_window(k, dtype):
    """Key 3 of 900 fits the query with a raw score of 36, capped at 15: far above the noise."""
    n, ps, dk, dv = 900, 16, 64, 48
    keys, values = rnd(n, 1, dk, seed=16, scale=0.05), rnd(n, 1, dv, seed=17)
    q = rnd(1, 2, dk, seed=18, scale=0.05)
    keys[3, 0, 0], q[0, :, 0] = 6.0, 6.0
    keys, values, q = keys.to(dtype), values.to(dtype), q.to(dtype)
    k_cache, v_cache, table = paged(keys, values, ps, dtype, seed=19)
    sink, gate = torch.zeros(2, device=DEV), torch.full((1, 2), 0.5, device=DEV)
    want = P.capped_window_attention(torch.cat([torch.zeros(n - 1, 2, dk), q.float()]).to(F64), keys.to(F64), values.to(F64), 1.0, 15.0)[-1:]
    got = run(k, q, k_cache, v_cache, table, n, ps, 1.0, 0, 15.0, sink, gate, dv)
    close(got, want * 0.5, dtype, "far key")
    assert float((got[0, 0].cpu().to(F64) * 2 - values[3, 0].to(F64)).abs().max()) < 0.02
    for window, seen in ((n - 3, True), (n - 4, False)):
        got = run(k, q, k_cache, v_cache, table, n, ps, 1.0, window, 15.0, sink, gate, dv)
        assert (float((got[0, 0].cpu().to(F64) * 2 - values[3, 0].to(F64)).abs().max()) < 0.02) == seen


def test_a_cap_and_a_bias_by_distance_are_not_taken_together(k):
    q = torch.zeros((1, 16), device=DEV)
    cache = torch.zeros((1, 1, 16, 16), device=DEV)
    with pytest.raises(ValueError, match="cap"):
        k.window_attention(q, q.clone(), cache, cache, dev_ints([[0]]), dev_ints([0]), dev_ints([1]), dev_ints([1]), 1, 1, 16, 16, 16, 1.0, 0,
                           0, None, 1, 1, slopes=torch.ones(1, device=DEV), softcap=2.0)


# ----------------------------------------------------------------------------- streams
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n, hidden, splits", [(1, 64, 1), (2, 100, 3), (3, 288, 0), (4, 1030, 1), (5, 72, 12), (8, 2048, 2), (10, 36, 1), (9, 33, 0)])
@pytest.mark.parametrize("scaled", [True, False])
def test_streams_are_rewritten_summed_and_normed(k, dtype, n, hidden, splits, scaled):
    from easy_gpt.cpp_amd.kernels import StreamUpdate

    t, eps = 7, 1e-5
    x = rnd(n, t, hidden, seed=31)
    given, y = product(rnd(t, hidden, seed=32, scale=2.0), dtype, splits)
    weight = rnd(hidden, seed=33, dtype=dtype) + 1
    scale = rnd(hidden, seed=34) if scaled else None
    w = {"in": rnd(n, seed=35), "out": rnd(n, seed=36), "mix": rnd(n, n, seed=37)}
    wd = {name: v.to(DEV) for name, v in w.items()}
    w64 = {name: v.to(F64) for name, v in w.items()}
    yy = y if scale is None else y * scale.to(F64)
    update = StreamUpdate(given, None if scale is None else scale.to(DEV), wd["mix"], wd["out"])
    norm = lambda u: P.rms_norm(u, weight.to(F64), eps)
    new = P.write_streams(x.to(F64), yy, w64, "")
    rows = dev_ints([5, 0, 3])
    streams = x.to(DEV)
    # nothing pending: a weighted sum; the sum of all with the update, for some rows, nothing kept
    out, kept = k.connect_streams(streams, None, wd["in"], n, None, weight.to(DEV), eps)
    assert kept is streams and torch.equal(streams.cpu(), x)
    close(out, norm(P.read_streams(x.to(F64), w64, "")), dtype, "read")
    out, kept = k.connect_streams(streams, update, None, n, rows, weight.to(DEV), eps)
    assert kept is streams and torch.equal(streams.cpu(), x)
    close(out, norm(new.sum(0))[[5, 0, 3]], dtype, "summed rows")
    out, kept = k.connect_streams(streams, update, None, n, None, weight.to(DEV), eps, keep=False)
    assert kept is streams and torch.equal(streams.cpu(), x)
    close(out, norm(new.sum(0)), dtype, "summed")
    # rewritten and read by the next branch
    out, kept = k.connect_streams(streams, update, wd["in"], n, None, weight.to(DEV), eps)
    close(kept, new, torch.float32, "streams")
    close(out, norm(P.read_streams(new, w64, "")), dtype, "read behind the update")
    # all streams equal: one tensor
    one = x[0].to(DEV)
    same = x[:1].to(F64).expand(n, -1, -1)
    out, kept = k.connect_streams(one, None, wd["in"], n, None, weight.to(DEV), eps)
    assert kept is one
    close(out, norm(P.read_streams(same, w64, "")), dtype, "read from equal streams")
    out, kept = k.connect_streams(one, update, wd["in"], n, None, weight.to(DEV), eps)
    assert torch.equal(one.cpu(), x[0])
    new = P.write_streams(same, yy, w64, "")
    close(kept, new, torch.float32, "streams from one")
    close(out, norm(P.read_streams(new, w64, "")), dtype, "read behind the first update")


# ----------------------------------------------------------------------------- constant decay
DECAYS = (0.5, 0.97, 1.0, 0.0, 0.9995, 0.9)


def decay_case(heads, dk, dv, rot, lengths, dtype, splits, seed=16):
    t = sum(lengths)
    width = 2 * heads * dk + 2 * heads * dv + 5
    raw = rnd(t, width, seed=seed)
    # keys lean towards the queries: a sum that nearly cancels (a decay of 0 leaves one key) is divided by its small root mean
    # square, and its rounding with it
    raw[:, 3 + heads * dk : 3 + 2 * heads * dk] = 0.8 * raw[:, 3 : 3 + heads * dk] + 0.6 * raw[:, 3 + heads * dk : 3 + 2 * heads * dk]
    given, x = product(raw, dtype, splits)
    decay = (DECAYS * 3)[:heads]
    powers = torch.pow(torch.tensor(decay, dtype=torch.float32).to(F64)[:, None], torch.arange(65, dtype=F64)[None]).to(torch.float32)
    return t, width, given, x, decay, powers.to(DEV)


def plain_heads(x, s0, n, first_pos, heads, dk, dv, rot, layout, decay, k_scale, state, weight, eps, gate_act):
    """(gated heads [n, heads * dv], raw heads, state behind) of the rows s0 .. s0 + n whose positions begin at first_pos"""
    rows = x[s0 : s0 + n, 3:]
    positions = torch.arange(first_pos, first_pos + n)
    qk, vw = heads * dk, heads * dv
    q = P.rotate(rows[:, :qk].view(n, heads, dk), positions, rot, layout)
    key = P.rotate(rows[:, qk : 2 * qk].view(n, heads, dk), positions, rot, layout) * k_scale
    val = rows[:, 2 * qk : 2 * qk + vw].view(n, heads, dv)
    o, last = P.constant_decay_scan(q, key, val, torch.tensor(decay, dtype=torch.float32).to(F64), state)
    g = rows[:, 2 * qk + vw : 2 * qk + 2 * vw]
    g = P.silu(g) if gate_act == "silu" else torch.sigmoid(g)
    return (P.rms_norm(o, weight, eps).reshape(n, vw) * g), o.reshape(n, vw), last


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads, dk, dv, rot, layout, weighted, gate_act, splits", [
    (4, 24, 40, 24, "half", False, "silu", 1),
    (2, 16, 32, 8, "half", True, "sigmoid", 2),
    (5, 64, 48, 64, "half", False, "silu", 1),
    (1, 36, 20, 6, "interleaved", False, "silu", 0),
    (3, 8, 130, 0, "half", False, "silu", 3),
    (2, 64, 128, 64, "half", False, "silu", 1),
    (2, 9, 7, 4, "half", True, "silu", 1),                       # neither is a multiple of four
    (1, 128, 256, 128, "half", False, "silu", 1),                # chunks of 32
    (1, 256, 256, 64, "half", False, "silu", 1),
    (2, 33, 251, 32, "interleaved", False, "silu", 2),
])
def test_constant_decay_heads_in_chunks_and_token_by_token(k, dtype, heads, dk, dv, rot, layout, weighted, gate_act, splits):
    """Requests in one step: portions behind a carried state (of several chunks, one token short of and one beyond a chunk's
    edge), single tokens, and a new prompt in a slot that held another's state."""
    from easy_gpt.cpp_amd.kernels.hip import HipKernels

    eps, k_scale = 1e-6, dk ** -0.5
    table = {"base": 500.0, "dims": rot}
    pairing = layout
    w = (rnd(dv, seed=18, dtype=dtype) + 1) if weighted else None
    for lengths, first_pos in (([150, 1, 64, 65, 31, 2], [40, 7, 0, 100, 3, 11]), ([1, 3, 1, 4], [9, 0, 200, 64])):
        slots = [4, 0, 2, 6, 7, 1][: len(lengths)]
        q_start, q_len, slot_t, starts = scan_setup(lengths, slots, 9)
        t, width, given, x, decay, powers = decay_case(heads, dk, dv, rot, lengths, dtype, splits)
        fresh = torch.tensor([p == 0 for p in first_pos])
        positions = torch.cat([torch.arange(p, p + n) for p, n in zip(first_pos, lengths)]).to(I32)
        states = rnd(9, heads, dk, dv, seed=17)
        rotation = {}
        if rot:
            cos_sin, _ = rope(k, table, positions)
            rotation = dict(cos_sin=cos_sin, rotary_dim=rot, pairing=pairing)
        at = (3, 3 + heads * dk, 3 + 2 * heads * dk, 3 + 2 * heads * dk + heads * dv)
        want = [plain_heads(x, s0, n, p, heads, dk, dv, table, layout, decay, k_scale, None if p == 0 else states[slot].to(F64),
                            None if w is None else w.to(F64), eps, gate_act)
                for s0, n, p, slot in zip(starts, lengths, first_pos, slots)]
        before = HipKernels.decay_step_tokens
        try:
            # by the longest portion as it is, and the other way: chunks for few tokens, steps for many
            for limit in (4, 0, 10000):
                HipKernels.decay_step_tokens = limit
                states_dev = states.to(DEV).clone()
                got = k.constant_decay_heads(given, dtype, *at, k_scale, powers, states_dev, slot_t, fresh.to(DEV), q_start, q_len, max(lengths),
                                             heads, dk, dv, None if w is None else w.to(DEV), eps, gate_act=gate_act, **rotation)
                for b, (s0, n, slot) in enumerate(zip(starts, lengths, slots)):
                    close(got[s0 : s0 + n], want[b][0], dtype, f"limit {limit}: outputs of request {b}")
                    close(states_dev[slot], want[b][2], torch.float32, f"limit {limit}: state of request {b}")
                for slot in set(range(9)) - set(slots):
                    assert torch.equal(states_dev[slot].cpu(), states[slot])
        finally:
            HipKernels.decay_step_tokens = before
        # the general scan and the norm behind it
        states_dev = states.to(DEV).clone()
        o = k.decayed_state_scan(given, dtype, *at[:3], 1.0, None, states_dev, slot_t, fresh.to(DEV), q_start, q_len, heads, dk, dv,
                                 head_decay=powers[:, 1].contiguous(), k_scale=k_scale, **rotation)
        gated = torch.empty((t, heads * dv), dtype=dtype, device=DEV)
        k.head_norm_gate(o, None if w is None else w.to(DEV), eps, given, at[3], gated, heads, dv, gate_act=gate_act)
        for b, (s0, n, slot) in enumerate(zip(starts, lengths, slots)):
            close(o.sum(0)[s0 : s0 + n], want[b][1], torch.float32, f"scan: raw outputs of request {b}")
            close(gated[s0 : s0 + n], want[b][0], dtype, f"scan: outputs of request {b}")
            close(states_dev[slot], want[b][2], torch.float32, f"scan: state of request {b}")


def test_wider_heads_than_the_chunks_take_are_left_to_the_scan(k):
    assert k.constant_decay_heads(torch.zeros((1, 1, 4), device=DEV), torch.float32, 0, 0, 0, 0, 1.0, None, None, None, None, None, None, 1, 1, 300,
                                  16, None, 1e-5) is None


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_first_token_that_stands_out_is_still_there_after_hundreds(k, dtype):
    """With a decay near one, what the first token of 700 wrote comes back to the last one's query, whatever the cut."""
    heads, dk, dv, n = 1, 32, 16, 700
    x = 0.01 * rnd(n, 2 * dk + 2 * dv, seed=40)
    x[0, dk] = 50.0                                             # the first key's first place, and the last query's
    x[n - 1, 0] = 50.0
    x[0, 2 * dk : 2 * dk + dv] = rnd(dv, seed=41)
    x[:, 2 * dk + dv :] = 8.0                                   # gates open
    given = x[None].to(DEV)
    powers = torch.pow(torch.tensor(0.999, dtype=F64), torch.arange(65, dtype=F64))[None].to(torch.float32).to(DEV)
    want = P.rms_norm(x[0, 2 * dk : 2 * dk + dv].to(F64), None, 1e-6)
    for cut in ([n], [n - 1, 1], [64, 64, n - 128], [333, 2, n - 335]):
        states = torch.full((1, heads, dk, dv), 3.0, device=DEV)
        done = 0
        for m in cut:
            part = given[:, done : done + m].contiguous()
            out = k.constant_decay_heads(part, dtype, 0, dk, 2 * dk, 2 * dk + dv, 1.0, powers, states, dev_ints([0]),
                                         torch.tensor([done == 0], device=DEV), dev_ints([0]), dev_ints([m]), m, heads, dk, dv, None, 1e-6)
            done += m
        close(out[-1] / (8.0 / (1 + math.exp(-8.0))), want, torch.bfloat16, f"cut {cut}")


# ----------------------------------------------------------------------------- the gate's activation
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("inter, splits, rows", [(64, 0, 9), (50, 0, 9), (64, 1, 9), (33, 3, 4), (416, 1, 300)])
def test_the_gelu_gate_of_a_product(k, dtype, inter, splits, rows):
    given, x = product(rnd(rows, 2 * inter, seed=50, scale=3.0), dtype, splits)
    out = torch.empty((rows, inter), dtype=dtype, device=DEV)
    k.swiglu(given, out, activation="gelu_tanh")
    want = P.gelu_tanh(x[:, :inter]) * x[:, inter:]
    close(out, want, dtype, "gelu gate")
    assert float((want - P.silu(x[:, :inter]) * x[:, inter:]).abs().max()) > 0.1
    big = torch.tensor([[-1e4, 1e4, -60.0, 0.0] * 2 + [1.0] * 8], dtype=dtype, device=DEV)      # no overflow to NaN
    o = torch.empty((1, 8), dtype=dtype, device=DEV)
    k.swiglu(big, o, activation="gelu_tanh")
    assert torch.equal(o.cpu(), torch.relu(big[:, :8].cpu()))


def test_the_gelu_gate_folded_into_products(k):
    t, inter, n, hidden, eps = 7, 328, 192, 77, 1e-5
    gu = rnd(3, t, 2 * inter, seed=51, scale=1.5).to(DEV)
    ss = (torch.rand(3, t, generator=torch.Generator().manual_seed(2)) * 50 + 1).to(DEV)
    w = rnd(n, inter, dtype=torch.bfloat16, seed=52, scale=0.05)
    z = gu.double().sum(0).cpu() * (1.0 / torch.sqrt(ss.double().sum(0).cpu() / hidden + eps))[:, None]
    act = P.gelu_tanh(z[:, :inter]) * z[:, inter:]
    got = k.product_swiglu(gu, ss, hidden, eps, w.to(DEV), activation="gelu_tanh")
    close(got.sum(0), act @ w.to(F64).T, torch.bfloat16, "folded into the down product")
    alone = torch.empty((t, inter), dtype=torch.float32, device=DEV)
    k.swiglu(gu, alone, row_ss=ss, hidden=hidden, eps=eps, activation="gelu_tanh")
    close(alone, act, torch.float32, "with the rows' pending factor")
    x, wg = rnd(40, 96, dtype=torch.bfloat16, seed=53), rnd(2 * 80, 96, dtype=torch.bfloat16, seed=54, scale=0.15)
    p = x.to(F64) @ wg.to(F64).T
    for groups in (1, 2):
        got = k.gate_up_swiglu(x.to(DEV), wg.to(DEV), groups=groups, activation="gelu_tanh")
        close(got, P.gelu_tanh(p[:, :80]) * p[:, 80:], torch.bfloat16, f"with the gate and up product, {groups} groups")
