"""The kernels and operands that the Karesun design brought, each alone against the plain functions of tests/plain_karesun.py: the
attention whose heads are the difference of two maps (prompts, portions, single tokens with split keys, batches of unequal
requests, sizes for the matrix cores and sizes that are multiples of nothing), rows of queries alone, norms whose weights are stored
around zero in every kernel that norms or folds a norm, a scaled embedding with positions on either kind of stream, the
squared relu with a pending row factor and folded into the product behind it, and experts chosen within groups with identity
experts, added into the stream."""
import math

import pytest
import torch

import plain_karesun as P
from test_gpu_bubetar_kernels import dev_ints, product
from test_gpu_head_kernels import close, paged, rnd

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F64 = torch.float64
I32 = torch.int32
FIXED = 4294967296.0


@pytest.fixture(scope="module")
def k():
    from easy_gpt.cpp_amd import kernels

    kernels.use_backend(None)
    return kernels.backend()


def fixed(x):
    return torch.round(x.double() * FIXED).to(torch.int64)


# ----------------------------------------------------------------------------- attention
def two_maps(q, keys, values, scale, softcap, window, lam, diff, eps):
    """The plain function on heads laid out [map 1 | map 2]."""
    split = lambda a: a.to(F64).view(*a.shape[:2], 2, -1)
    return P.two_maps(split(q), split(keys), values.to(F64), scale, softcap, window or None, lam, diff, eps)


def run(k, q, k_cache, v_cache, table, kv_len, page_size, scale, window, softcap, lam, diff, eps, dv):
    m, nq, dk = q.shape
    out = torch.empty((m, nq * dv), dtype=q.dtype, device=DEV)
    k.window_attention(q.reshape(m, nq * dk).to(DEV).contiguous(), out, k_cache, v_cache, table, dev_ints([0]), dev_ints([m]), dev_ints([kv_len]),
                       nq, k_cache.shape[1], dk, dv, page_size, scale, window, 0, None, m, kv_len, softcap=softcap, difference=(lam, eps, 1 - diff))
    return out.view(m, nq, dv)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nq, nkv, dim, dv", [
    (4, 2, 16, 32), (8, 2, 64, 64), (6, 1, 128, 96), (4, 1, 40, 48), (5, 5, 24, 16), (2, 1, 96, 256), (14, 2, 32, 64), (3, 1, 8, 176),   # the matrix cores
    (3, 3, 11, 13), (2, 1, 20, 24), (2, 2, 1, 1), (2, 1, 150, 70), (1, 1, 4, 300),                      # any sizes
])
@pytest.mark.parametrize("window, softcap, lam", [(0, 3.0, 0.6), (70, 1.5, -0.4), (12, None, 0.8), (1, 30.0, 0.3), (64, 6.0, 1.7)])
def test_attention_by_the_difference_of_two_maps(k, dtype, nq, nkv, dim, dv, window, softcap, lam):
    n, ps, diff, eps = 150, 16, 0.35, 1e-5
    keys, values = rnd(n, nkv, 2 * dim, seed=11).to(dtype), rnd(n, nkv, dv, seed=12).to(dtype)
    q = rnd(n, nq, 2 * dim, seed=13, scale=2.5).to(dtype)
    scale = 1.7 / math.sqrt(dim)
    k_cache, v_cache, table = paged(keys, values, ps, dtype, seed=15)
    want = two_maps(q, keys, values, scale, softcap, window, lam, diff, eps)
    if softcap and softcap < 10 and window != 1 and dv > 1:         # the cap bends the large scores
        assert float((two_maps(q, keys, values, scale, None, window, lam, diff, eps) - want).abs().max()) > 0.05
    for first, m in [(0, n), (37, 50), (95, 2), (0, 1), (149, 1), (63, 1), (64, 1)]:
        got = run(k, q[first : first + m], k_cache, v_cache, table, first + m, ps, scale, window, softcap, lam, diff, eps, dv)
        # (one value alone divided by its root mean square is a sign: near zero any rounding turns it)
        if dv > 1:
            close(got, want[first : first + m], dtype, f"rows {first}..{first + m}")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nq, nkv, dim, dv, ps", [(6, 2, 32, 64, 32), (4, 2, 64, 128, 48), (4, 4, 13, 9, 5)])
def test_a_batch_of_portions_and_single_tokens_against_each_request_alone(k, dtype, nq, nkv, dim, dv, ps):
    """Unequal requests in one launch, some of them single tokens far behind others, against the plain function per request."""
    lam, diff, eps, scale, cap, window = 0.55, 0.2, 1e-6, 0.9 / math.sqrt(dim), 8.0, 90
    lengths, brought = [300, 1, 77, 640, 129], [1, 1, 2, 1, 40]
    caches, tables, qs, wants = [], [], [], []
    base = 0
    for i, (n, m) in enumerate(zip(lengths, brought)):
        keys, values = rnd(n, nkv, 2 * dim, seed=50 + i).to(dtype), rnd(n, nkv, dv, seed=60 + i).to(dtype)
        q = rnd(n, nq, 2 * dim, seed=70 + i, scale=2.0).to(dtype)
        kc, vc, table = paged(keys, values, ps, dtype, seed=i)
        caches.append((kc, vc))
        tables.append(table[0] + base)
        base += kc.shape[0]
        qs.append(q[n - m :])
        wants.append(two_maps(q, keys, values, scale, cap, window, lam, diff, eps)[n - m :])
    width = max(len(t) for t in tables)
    table = torch.full((len(lengths), width), -1, dtype=I32, device=DEV)
    for i, t in enumerate(tables):
        table[i, : len(t)] = t
        gone = max(0, lengths[i] - brought[i] - window + 1) // ps        # pages that the window gave back
        table[i, :gone] = -1
    q = torch.cat(qs)
    t = q.shape[0]
    starts = [sum(brought[:i]) for i in range(len(brought))]
    out = torch.empty((t, nq * dv), dtype=dtype, device=DEV)
    k.window_attention(q.reshape(t, -1).to(DEV).contiguous(), out, torch.cat([c[0] for c in caches]), torch.cat([c[1] for c in caches]), table,
                       dev_ints(starts), dev_ints(brought), dev_ints(lengths), nq, nkv, 2 * dim, dv, ps, scale, window, 0, None, max(brought),
                       max(lengths), softcap=cap, difference=(lam, eps, 1 - diff))
    close(out.view(t, nq, dv), torch.cat(wants), dtype, "batch")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("loud", [0, 1])
def test_a_far_key_stands_out_in_one_map_and_is_lost_behind_the_window(k, dtype, loud):
    """Key 3 of 900 fits one map's query with a raw score of 36, capped at 15: far above the noise.  The other map spreads over all
    keys.  In map 2 the key's value comes out with the sign turned."""
    n, ps, dim, dv, lam = 900, 16, 64, 48, 0.7
    keys, values = rnd(n, 1, 2 * dim, seed=16, scale=0.05), rnd(n, 1, dv, seed=17)
    q = rnd(1, 2, 2 * dim, seed=18, scale=0.05)
    keys[3, 0, loud * dim], q[0, :, loud * dim] = 6.0, 6.0
    keys, values, q = keys.to(dtype), values.to(dtype), q.to(dtype)
    k_cache, v_cache, table = paged(keys, values, ps, dtype, seed=19)
    direction = P.unit_rms(values[3, 0].to(F64), 1e-6) * (1.0 if loud == 0 else -1.0)
    whole_q = torch.cat([torch.zeros(n - 1, 2, 2 * dim, dtype=dtype), q])
    for window, seen in ((0, True), (n - 3, True), (n - 4, False)):
        want = two_maps(whole_q, keys, values, 1.0, 15.0, window, lam, 0.0, 1e-6)[-1:]
        got = run(k, q, k_cache, v_cache, table, n, ps, 1.0, window, 15.0, lam, 0.0, 1e-6, dv)
        if seen:
            close(got, want, dtype, f"far key, window {window}")
        assert (float((got[0, 0].cpu().to(F64) - direction).abs().max()) < 0.25) == seen


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_pages_beyond_the_window_are_not_touched_and_the_two_maps_are_not_mixed_up(k, dtype):
    """Pages that lie wholly behind the window are -1 in the table; swapping the maps turns the sign where lambda is 1 / lambda."""
    n, ps, nq, nkv, dim, dv, window, lam = 200, 16, 4, 2, 32, 32, 30, 0.5
    keys, values = rnd(n, nkv, 2 * dim, seed=21).to(dtype), rnd(n, nkv, dv, seed=22).to(dtype)
    q = rnd(2, nq, 2 * dim, seed=23, scale=2.0).to(dtype)
    k_cache, v_cache, table = paged(keys, values, ps, dtype, seed=24)
    table = table.clone()
    table[0, : (n - 2 - window + 1) // ps] = -1
    got = run(k, q, k_cache, v_cache, table, n, ps, 0.2, window, 9.0, lam, 0.0, 0.0, dv)
    whole_q = torch.cat([torch.zeros(n - 2, nq, 2 * dim, dtype=dtype), q])
    close(got, two_maps(whole_q, keys, values, 0.2, 9.0, window, lam, 0.0, 0.0)[-2:], dtype, "window")
    turn = lambda a: torch.cat([a[..., dim:], a[..., :dim]], dim=-1).contiguous()
    kt, vt, tt = paged(turn(keys), values, ps, dtype, seed=24)
    close(run(k, turn(q), kt, vt, tt, n, ps, 0.2, window, 9.0, 1.0 / lam, 0.0, 0.0, dv), -got.cpu().to(F64), dtype, "swapped")


def test_what_two_maps_do_not_go_with_is_refused(k):
    q = torch.zeros((1, 16), device=DEV)
    cache = torch.zeros((1, 1, 16, 16), device=DEV)
    args = (q, q.clone(), cache, cache, dev_ints([[0]]), dev_ints([0]), dev_ints([1]), dev_ints([1]), 1, 1, 16, 16, 16, 1.0, 0, 0)
    for sink, kw in ((torch.zeros(1, device=DEV), {}), (None, dict(head_gate=torch.ones(1, 1, device=DEV))), (None, dict(slopes=torch.ones(1, device=DEV)))):
        with pytest.raises(ValueError, match="two maps"):
            k.window_attention(*args, sink, 1, 1, difference=(0.5, 1e-6, 1.0), **kw)
    odd = torch.zeros((1, 15), device=DEV)
    cache15 = torch.zeros((1, 1, 16, 15), device=DEV)
    with pytest.raises(ValueError, match="even"):
        k.window_attention(odd, q.clone(), cache15, cache, dev_ints([[0]]), dev_ints([0]), dev_ints([1]), dev_ints([1]), 1, 1, 15, 16, 16, 1.0, 0, 0,
                           None, 1, 1, difference=(0.5, 1e-6, 1.0))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("t, nq, dk, splits, normed", [(9, 4, 32, 2, False), (3, 5, 22, 0, False), (301, 6, 48, 1, False), (7, 3, 20, 3, True)])
def test_rows_of_queries_alone(k, dtype, t, nq, dk, splits, normed):
    given, x = product(rnd(t, nq * dk, seed=1, scale=2.0), dtype, splits)
    q_out = torch.empty((t, nq * dk), dtype=dtype, device=DEV)
    cache = torch.zeros((1, 2, 16, dk), dtype=dtype, device=DEV)
    k.head_norm_store(given, q_out, None, None, 1e-5, False, None, cache, cache, nq, 0, dk, 8, 16, norm_plain=normed)
    want = x.view(t, nq, dk)
    close(q_out, (P.unit_rms(want, 1e-5) if normed else want).reshape(t, -1), dtype, "queries")
    with pytest.raises(ValueError, match="nothing to store"):
        k.head_norm_store(given, q_out, None, None, 1e-5, False, torch.zeros(t, dtype=I32, device=DEV), cache, cache, nq, 0, dk, 8, 16)


# ----------------------------------------------------------------------------- norms whose weights are distances from one
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("t, hidden, splits", [(7, 64, 0), (7, 100, 3), (40, 288, 1), (40, 288, 0), (5, 1030, 2), (33, 4096, 1), (3, 9000, 0)])
def test_a_norms_offset_is_added_in_float32(k, dtype, t, hidden, splits):
    """Weights of a few thousandths: one added to them in bfloat16 would lose them."""
    eps = 1e-5
    x = rnd(t, hidden, seed=2, scale=3.0)
    given, y = product(rnd(t, hidden, seed=3), dtype, splits)
    w = rnd(hidden, seed=4, scale=3e-3).to(dtype)
    want = P.offset_norm(x.to(F64) + y, w.to(F64), eps)
    bare = P.unit_rms(x.to(F64) + y, eps)
    rows = dev_ints([t - 1, 0, 2])
    for stream in (x.to(DEV), fixed(x).to(DEV)):
        h = stream.clone()
        out = torch.empty((t, hidden), dtype=dtype, device=DEV)
        k.add_rmsnorm(h, given, w.to(DEV), eps, out, weight_offset=1.0)
        close(out, want, dtype, "norm")
        some = torch.empty((3, hidden), dtype=dtype, device=DEV)
        k.rows_add_rmsnorm(stream.clone(), given, rows, w.to(DEV), eps, some, weight_offset=1.0)
        close(some, want[[t - 1, 0, 2]], dtype, "norm of rows")
        if dtype == torch.float32:
            assert float((out.cpu().to(F64) - bare).abs().max()) > 100 * float((out.cpu().to(F64) - want).abs().max())
    # what the sum of many values keeps of the weights shows that bfloat16 keeps them too: projected on the weights
    gain = ((out.cpu().to(F64) - bare) * w.to(F64) * bare).sum() / ((w.to(F64) * bare) ** 2).sum()
    assert t * hidden < 3000 or abs(float(gain) - 1.0) < 0.35


@pytest.mark.parametrize("t, n, hidden", [(1, 64, 64), (8, 200, 896), (16, 320, 256), (3, 1000, 1536)])
@pytest.mark.parametrize("as_fixed", [True, False])
def test_a_product_with_the_norm_folded_in_takes_the_offset(k, t, n, hidden, as_fixed):
    eps, dtype = 1e-6, torch.bfloat16
    x, w = rnd(t, hidden, seed=5, scale=2.0), rnd(hidden, seed=6, scale=0.2).to(dtype)
    m = rnd(n, hidden, seed=7, scale=hidden ** -0.5).to(dtype)
    stream = fixed(x).to(DEV) if as_fixed else x.to(DEV)
    fused = k.product_normed(stream, None, w.to(DEV), m.to(DEV), weight_offset=1.0, waves=4, splits=min(2, -(-hidden // 128)))
    assert fused is not None
    parts, row_ss, _ = fused
    factor = 1.0 / torch.sqrt(row_ss.double().sum(0) / hidden + eps)
    got = parts.double().sum(0) * factor[:, None]
    close(got, P.offset_norm(x.to(F64), w.to(F64), eps) @ m.to(F64).T, dtype, "folded norm")


# ----------------------------------------------------------------------------- embedding
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("as_fixed", [True, False])
def test_a_scaled_embedding_with_a_vector_per_position(k, dtype, as_fixed):
    hidden, scale = 150, 3.7
    table, pos = rnd(40, hidden, seed=8).to(dtype), rnd(30, hidden, seed=9).to(dtype)
    ids, positions = dev_ints([3, 39, 0, 3, 12]), dev_ints([0, 29, 7, 8, 1])
    out = torch.empty((5, hidden), dtype=torch.int64 if as_fixed else torch.float32, device=DEV)
    k.embed_positions(ids, positions, table.to(DEV), pos.to(DEV), out, factor=scale)
    got = out.double() / FIXED if as_fixed else out
    close(got, table.to(F64)[ids.cpu().long()] * scale + pos.to(F64)[positions.cpu().long()], torch.float32, "embedding")


# ----------------------------------------------------------------------------- squared relu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("t, cols, splits, mode, gate", [(9, 96, 2, "relu2", False), (3, 50, 1, "relu2", True), (8, 320, 1, "relu2", False),
                                                         (5, 64, 3, "polynorm", True), (4, 200, 1, "polynorm", False)])
def test_an_activation_applies_the_rows_pending_factor(k, dtype, t, cols, splits, mode, gate):
    width, hidden, eps = cols + (1 if gate else 0), 77, 1e-5
    given, z = product(rnd(t, width, seed=10, scale=2.0), dtype, splits)
    row_ss = torch.rand(2, t, generator=torch.Generator().manual_seed(11)) * 40
    z = z / torch.sqrt(row_ss.to(F64).sum(0) / hidden + eps)[:, None]
    coef = torch.tensor([0.5, -0.3, 0.7, 0.1])
    out = torch.empty((t, cols), dtype=dtype, device=DEV)
    k.ff_activation(given, cols, mode, out, coef=coef.to(DEV) if mode == "polynorm" else None, eps=1e-6, gate_col=cols if gate else -1,
                    row_ss=row_ss.to(DEV), hidden=hidden, norm_eps=eps)
    v = z[:, :cols]
    want = torch.relu(v) ** 2 if mode == "relu2" else (0.5 * P.unit_rms(v, 1e-6) - 0.3 * P.unit_rms(v ** 2, 1e-6) + 0.7 * P.unit_rms(v ** 3, 1e-6) + 0.1)
    close(out, want * torch.sigmoid(z[:, cols:]) if gate else want, dtype, mode)


@pytest.mark.parametrize("t, n, inter, splits, waves", [(1, 64, 96, 1, 4), (8, 896, 1024, 3, 8), (16, 200, 328, 9, 4), (5, 100, 1000, 2, 16)])
@pytest.mark.parametrize("pending", [True, False])
def test_a_product_begins_with_the_squared_relu(k, t, n, inter, splits, waves, pending):
    dtype, hidden, eps = torch.bfloat16, 300, 1e-6
    given, z = product(rnd(t, inter, seed=12, scale=2.0), dtype, splits)
    row_ss = (torch.rand(3, t, generator=torch.Generator().manual_seed(13)) * 200).to(DEV) if pending else None
    if pending:
        z = z / torch.sqrt(row_ss.cpu().to(F64).sum(0) / hidden + eps)[:, None]
    w = rnd(n, inter, seed=14, scale=inter ** -0.5).to(dtype)
    want = (torch.relu(z) ** 2) @ w.to(F64).T
    got = k.product_swiglu(given, row_ss, hidden, eps, w.to(DEV), waves=waves, activation="relu2")
    close(got.double().sum(0), want, dtype, "squared relu, then the product")
    stream = torch.zeros((t, n), dtype=torch.int64, device=DEV)
    assert k.product_swiglu(given, row_ss, hidden, eps, w.to(DEV), waves=waves, residual=stream, activation="relu2") is stream
    close(stream.double() / FIXED, want, dtype, "added into the stream")


# ----------------------------------------------------------------------------- experts
def expert_case(t, experts, identity, hidden, ff, seed=16):
    outputs = experts + identity
    x = rnd(t, hidden, seed=seed)
    w = {"router": rnd(outputs, hidden, seed=seed + 1, scale=2.0 / hidden ** 0.5), "correction": rnd(outputs, seed=seed + 2, scale=0.4) - 0.5}
    for e in range(experts):
        w[f"e{e}.gate"], w[f"e{e}.up"] = (rnd(ff, hidden, seed=100 * i + e, scale=hidden ** -0.5) for i in (1, 2))
        w[f"e{e}.down"] = rnd(hidden, ff, seed=300 + e, scale=ff ** -0.5)
    gate_up = torch.stack([torch.cat([w[f"e{e}.gate"], w[f"e{e}.up"]]) for e in range(experts)])
    down = torch.stack([w[f"e{e}.down"] for e in range(experts)])
    return x, w, gate_up, down


@pytest.mark.parametrize("experts, identity, top, groups, keep, hidden, ff, scale", [
    (6, 2, 3, 4, 2, 64, 48, 1.5), (8, 1, 3, 3, 1, 100, 50, 2.0), (6, 0, 4, 3, 2, 100, 30, 1.0), (12, 4, 6, 2, 2, 128, 32, 0.7), (7, 2, 3, None, None, 60, 20, 2.5),
    (3, 3, 2, 2, 1, 72, 40, 1.0),                       # one group holds identity experts alone
    (90, 38, 9, 16, 4, 96, 24, 1.1), (100, 60, 3, 80, 70, 64, 16, 1.0), (1, 1, 1, 2, 1, 48, 16, 1.0),
])
@pytest.mark.parametrize("t", [1, 70])
def test_experts_within_groups_and_identity_experts(k, experts, identity, top, groups, keep, hidden, ff, scale, t):
    x, w, gate_up, down = expert_case(t, experts, identity, hidden, ff)
    w64 = {n: v.to(F64) for n, v in w.items()}
    router = {"experts": experts, "top": top, "scale": scale, "identity": identity, "groups": {"count": groups, "keep": keep} if groups else None}
    want = P.expert_mixture(x.to(F64), w64, "", {"router": router})
    chosen, _ = P.route_scores(x.to(F64) @ w64["router"].T, w64["correction"], router)
    if t > 1:                                            # both kinds of output are chosen, and the groups change who is
        assert bool((chosen < experts).any()) and (identity == 0 or bool((chosen >= experts).any()))
        # (with as many groups as choices the best choices lie in the best groups anyway)
        if groups and keep < min(groups, top) and experts < 90:
            free, _ = P.route_scores(x.to(F64) @ w64["router"].T, w64["correction"], {**router, "groups": None})
            assert bool((free.sort(-1).values != chosen.sort(-1).values).any())
    options = dict(score_all=True, correction=w["correction"].to(DEV), weight_scale=scale, identities=identity, groups=groups or 1,
                   keep_groups=keep or 1, normalized=False)
    args = (x.to(DEV), w["router"].to(DEV), None, gate_up.to(DEV), down.to(DEV), top)
    got = k.expert_mixture(*args, **options)
    close(got, want, torch.float32, "experts")
    start = rnd(t, hidden, seed=40)
    stream = fixed(start).to(DEV)
    assert k.expert_mixture(*args, **options, residual=stream) is stream
    close(stream.double() / FIXED, want + start.to(F64), torch.float32, "added into the stream")
    # every token of the batch gets what it gets alone, bit for bit
    alone = k.expert_mixture(x[-1:].to(DEV), *args[1:], **options)
    assert torch.equal(alone[0], got[-1])


def test_bfloat16_experts_and_tokens_that_are_all_identity(k):
    """The identity experts' corrections are so large that nothing else is chosen: the input times the sum of two scores."""
    t, experts, identity, hidden = 20, 4, 2, 64
    x, w, gate_up, down = expert_case(t, experts, identity, hidden, 16)
    w["correction"][experts:] = 5.0
    b = {n: v.to(torch.bfloat16) for n, v in w.items()}
    xb = x.to(torch.bfloat16)
    s = torch.softmax(xb.to(F64) @ b["router"].to(F64).T, dim=-1)[:, experts:].sum(-1, keepdim=True)
    got = k.expert_mixture(xb.to(DEV), b["router"].to(DEV), None, gate_up.to(torch.bfloat16).to(DEV), down.to(torch.bfloat16).to(DEV), 2, score_all=True,
                           correction=w["correction"].to(DEV), weight_scale=1.5, identities=identity, normalized=False)
    close(got, 1.5 * s * xb.to(F64), torch.float32, "identity alone")


def test_equal_choice_scores_go_to_the_lower_index_and_group(k):
    """A router of zeros: all scores are equal, groups and experts are taken from the first on."""
    x, w, gate_up, down = expert_case(3, 6, 2, 32, 16)
    w["router"][:] = 0.0
    w["correction"][:] = 0.25
    args = (x.to(DEV), w["router"].to(DEV), None, gate_up.to(DEV), down.to(DEV), 3)
    got = k.expert_mixture(*args, score_all=True, correction=w["correction"].to(DEV), identities=2, groups=4, keep_groups=2, normalized=False)
    w64 = {n: v.to(F64) for n, v in w.items()}
    close(got, sum(P.gated_expert(x.to(F64), w64, f"e{e}.") for e in range(3)) / 8, torch.float32, "ties")


def test_choices_that_do_not_fit_are_refused(k):
    x, w, gate_up, down = expert_case(3, 6, 2, 32, 16)
    args = (x.to(DEV), w["router"].to(DEV), None, gate_up.to(DEV), down.to(DEV))
    options = dict(score_all=True, correction=w["correction"].to(DEV), identities=2, normalized=False)
    for top, kw in ((3, dict(groups=4, keep_groups=1)), (2, dict(groups=3)), (2, dict(groups=2, keep_groups=3)), (9, {})):
        with pytest.raises(ValueError):
            k.expert_mixture(*args, top, **options, **kw)
    with pytest.raises(ValueError, match="groups"):
        k.expert_mixture(*args, 2, identities=2, groups=2)
    with pytest.raises(ValueError):
        k.expert_mixture(*args, 2, score_all=True, identities=3)
