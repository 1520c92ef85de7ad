"""Lurirax in the engine against its plain implementation (tests/plain_lurirax.py): each mechanism alone at the
kernels, then whole models in every way of cutting the work."""
import math
import types

import numpy as np
import pytest
import torch

import helpers
import lurirax_helpers as lh
import plain_lurirax as pl
from test_gitasun_gpu import compare_for, paged_rows, rel_err, state_step
from test_kernels_gpu import FakeCache, FakeStep, dev, from_value_layout, ints, rounded

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
# Largest |logit difference| from the float64 plain implementation, as a fraction of the request's largest |logit|.
# fp32: the rounding of fused multiply-adds and exponentials; a lost state, a window that is one token off, a sink, a gate or a
# distance term left out show as 1e-2 and more.
# bf16: activations and cache rounded to 8 bits of mantissa at every part, residual stream, norms and scores in 32-bit. Retention's
# read-outs and differences of two maps are divided by their root mean square, which a rounding turns where they are nearly zero
# (at a first token the read-out's sign is the sign of one product), and a close call of a router may fall to the other side: whole
# models are compared as a distribution (``compare_for``: the median within half the tolerance, at most one position in twelve
# beyond it and none beyond ten times it). The plain implementation with the bf16 engine's roundings put in differs from itself by
# as much, at the same positions but for the routers' close calls: 0.46 at a first token (small), 0.78 at one position (ones).
TOL = {"float32": 1e-4, "bfloat16": 6e-2}
TOL_OF = {("small", "bfloat16"): 8e-2, ("ones", "bfloat16"): 8e-2}


def tol_of(name, dtype):
    return TOL_OF.get((name, dtype), TOL[dtype])


# ---- mechanisms alone ----------------------------------------------------------------------------------------------

@pytest.mark.parametrize("R,E,top,shared", [(1, 7, 2, True), (5, 40, 3, False), (9, 44, 4, True), (3, 2048, 8, True), (300, 256, 4, True), (600, 1028, 1, False),
                                            (2, 20000, 5, True), (4, 333, 6, True)])
def test_experts_and_a_gated_shared_expert_normed_into_the_stream(ops32, ops16, R, E, top, shared):
    """The sum that the norm's kernel forms on its way, the stream it adds to, and the copy it leaves; the same sum on demand."""
    rng = np.random.default_rng(R + E)
    pairs, ys = rng.standard_normal((R * top, E)).astype(np.float32), rng.standard_normal((R, E)).astype(np.float32)
    x0, z = rng.standard_normal((R, E)).astype(np.float32), rng.standard_normal((R, 3)).astype(np.float32)
    w = (1.0 + 0.2 * rng.standard_normal(E)).astype(np.float32)
    b = pairs.astype(np.float64).reshape(R, top, E).sum(1)
    if shared:
        b = b + pl.sigmoid(z[:, 1:2].astype(np.float64)) * ys
    want = x0 + pl.unit_rms(b, 1e-5) * w
    for ops in (ops32, ops16):
        y, x, gate = torch.full((R, E), float("nan"), dtype=torch.float32, device="cuda"), dev(x0), dev(z)
        keep = dev(pairs), dev(ys), dev(w)
        ops.branch_sum(y, keep[0], top, extra=keep[1] if shared else None, extra_gate=gate[:, 1:2] if shared else None)
        ops.rmsnorm_add(y, keep[2], 1e-5, x, copy=True)
        assert np.max(np.abs(x.cpu().numpy() - want)) <= 3e-6 * np.max(np.abs(want))
        h = ops.rounded(x)
        assert h.dtype == ops.act_dtype and torch.equal(h, x.to(ops.act_dtype))
        ops.scale_add(dev(x0), x, scale=1.0)                       # the stream moves on: the copy is no longer its own
        assert torch.equal(ops.rounded(x), x.to(ops.act_dtype))
        ops.branch_sum(y, keep[0], top, extra=keep[1] if shared else None, extra_gate=gate[:, 1:2] if shared else None)
        ops.settle()                                               # a sum that nobody takes along is formed on demand
        assert np.max(np.abs(y.cpu().numpy() - b)) <= 3e-6 * np.max(np.abs(b))


@pytest.mark.parametrize("T,E,F", [(3, 256, 4096), (8, 1024, 2048), (48, 512, 2048), (130, 256, 1024), (700, 512, 512), (5, 44, 40)])
def test_a_sublayers_result_as_partial_sums(ops16, T, E, F):
    """A product whose K was split hands its partial sums to the norm's kernel, alone and as the shared expert of a sum."""
    rng = np.random.default_rng(T)
    a, w = dev(rng.standard_normal((T, F)), torch.bfloat16), dev(rng.standard_normal((E, F)) / math.sqrt(F), torch.bfloat16)
    x0, norm, z, pairs = dev(rng.standard_normal((T, E))), dev(1.0 + 0.1 * rng.standard_normal(E)), dev(rng.standard_normal((T, 1))), dev(rng.standard_normal((2 * T, E)))
    prod = a.double().cpu().numpy() @ w.double().cpu().numpy().T
    for branch in (False, True):
        x, y, ys = x0.clone(), torch.empty((T, E), dtype=torch.float32, device="cuda"), torch.empty((T, E), dtype=torch.float32, device="cuda")
        ops16.gemm(a, w, ys if branch else y, defer=True)
        b = prod
        if branch:
            ops16.branch_sum(y, pairs, 2, extra=ys, extra_gate=z)
            b = pl.sigmoid(z.double().cpu().numpy()) * prod + pairs.double().cpu().numpy().reshape(T, 2, E).sum(1)
        ops16.rmsnorm_add(y, norm, 1e-6, x)
        want = x0.double().cpu().numpy() + pl.unit_rms(b, 1e-6) * norm.double().cpu().numpy()
        assert rel_err(x.cpu().numpy(), want) <= 1e-4


@pytest.mark.parametrize("in_dtype,out_dtype", [(torch.float32, torch.float32), (torch.float32, torch.bfloat16), (torch.bfloat16, torch.bfloat16)])
@pytest.mark.parametrize("T,H,G,D,GV,Dv,rot,page", [(5, 3, 1, 10, 1, 6, 6, 8), (9, 6, 2, 5, 1, 7, 0, 4), (1, 1, 1, 2, 1, 1, 2, 4), (70, 8, 2, 64, 2, 64, 32, 16), (3, 4, 4, 128, 4, 64, 128, 16),
                                                    (17, 8, 4, 32, 2, 64, 0, 16), (600, 4, 2, 96, 2, 96, 48, 16), (530, 5, 1, 64, 1, 128, 64, 32), (4, 2, 2, 200, 2, 20, 100, 8), (600, 3, 3, 64, 3, 64, 20, 8)])
def test_heads_normed_before_or_after_a_rotation_and_stored(ops32, ops16, in_dtype, out_dtype, T, H, G, D, GV, Dv, rot, page):
    ops = ops32 if out_dtype == torch.float32 else ops16
    rng = np.random.default_rng(T + D)
    rows = rng.standard_normal((T, (H + G) * D + GV * Dv)).astype(np.float32)
    x = rounded(rows, in_dtype)
    positions = rng.integers(0, 900, T)
    freqs = pl.rotary_frequencies(rot, 500.0) if rot else None
    weights = [(1.0 + 0.3 * rng.standard_normal(D)).astype(np.float32) for _ in range(2)]
    n_pages = T // page + 3
    # mostly runs of consecutive rows of pages, as a prompt has, with a few rows elsewhere
    slots = (rng.permutation(n_pages)[np.arange(T) // page] * page + np.arange(T) % page).astype(np.int32)
    q0, k0 = x[:, :H * D].reshape(T, H, D), x[:, H * D:(H + G) * D].reshape(T, G, D)
    wide = torch.zeros((T, rows.shape[1] + 8), dtype=in_dtype, device="cuda")          # rows that lie apart
    wide[:, :rows.shape[1]] = dev(rows, in_dtype)
    for weighted in (True, False):
        for after in (True, False):
            def norm(y, w):
                return pl.unit_rms(y, 1e-5) * (w if weighted else 1.0)

            def ref(y, w):
                y = y.astype(np.float64)
                if rot and after:
                    return norm(pl.rotate(y, positions, freqs), w)
                return pl.rotate(norm(y, w), positions, freqs) if rot else norm(y, w)
            cache = FakeCache(group=0, k=torch.full((n_pages * page, G * D), 7.0, dtype=out_dtype, device="cuda"),
                              v=torch.full((n_pages * page, GV * Dv), 7.0, dtype=out_dtype, device="cuda"), page_tokens=page, window=0)
            q = torch.empty((T, H * D), dtype=out_dtype, device="cuda")
            ops.head_norm_store(wide[:, :rows.shape[1]], H, G, D, Dv, dev(weights[0]) if weighted else None, dev(weights[1]) if weighted else None, 1e-5, q, cache,
                                ints(slots), n_v_heads=GV, norm=True, after=after, positions=ints(positions),
                                inv_freq=dev(freqs) if rot else None, rot_dim=rot)
            tol = 3e-4 if out_dtype == torch.float32 else 2e-2          # (angles of hundreds of radians are fp32 products)
            assert np.max(np.abs(q.float().cpu().numpy() - ref(q0, weights[0]).reshape(T, -1))) <= tol * 4
            assert np.max(np.abs(cache.k.float().cpu().numpy()[slots] - ref(k0, weights[1]).reshape(T, -1))) <= tol * 4
            v = from_value_layout(cache.v.float().cpu().numpy(), page)
            assert np.array_equal(v[slots], rounded(x[:, (H + G) * D:], out_dtype))
            untouched = np.setdiff1d(np.arange(n_pages * page), slots)
            assert (cache.k.float().cpu().numpy()[untouched] == 7.0).all() and (v[untouched] == 7.0).all()
            # without a cache: queries and values to rows
            q2, v2 = (torch.empty((T, n), dtype=out_dtype, device="cuda") for n in (H * D, GV * Dv))
            ops.head_norm_store(dev(np.concatenate([rows[:, :H * D], rows[:, (H + G) * D:]], axis=1), in_dtype), H, 0, D, Dv, dev(weights[0]) if weighted else None,
                                None, 1e-5, q2, None, None, n_v_heads=GV, norm=True, after=after, positions=ints(positions),
                                inv_freq=dev(freqs) if rot else None, rot_dim=rot, v_rows=v2)
            assert float((q2.float() - q.float()).abs().max()) <= tol and np.array_equal(v2.float().cpu().numpy(), rounded(x[:, (H + G) * D:], out_dtype))


@pytest.mark.parametrize("T,E,H,G,D,GV,Dv,rot,n_extra", [(3, 256, 4, 2, 64, 2, 64, 32, 4), (20, 2048, 8, 2, 128, 2, 128, 128, 8), (48, 512, 4, 4, 32, 2, 64, 0, 2),
                                                        (600, 2048, 8, 2, 64, 2, 64, 64, 8), (700, 512, 4, 2, 128, 2, 64, 32, 5), (130, 1024, 6, 2, 40, 2, 24, 8, 3)])
def test_heads_from_a_product_that_is_still_pending(ops16, T, E, H, G, D, GV, Dv, rot, n_extra):
    """Projections with a bias, their sums finished by the kernel that norms, turns and stores, which also hands out the columns
    behind the values: as from the finished product, and as in fp64."""
    rng = np.random.default_rng(T + E)
    N = (H + G) * D + GV * Dv + n_extra
    a, w = dev(rng.standard_normal((T, E)), torch.bfloat16), dev(rng.standard_normal((N, E)) / math.sqrt(E), torch.bfloat16)
    bias = rng.standard_normal(N).astype(np.float32) * 0.3
    rows = a.double().cpu().numpy() @ w.double().cpu().numpy().T + bias
    positions, freqs, page = np.arange(T), pl.rotary_frequencies(rot, 500.0) if rot else None, 16
    n_pages = T // page + 2
    slots = np.arange(T, dtype=np.int32) + page
    for defer in (True, False):
        cache = FakeCache(group=0, k=torch.zeros((n_pages * page, G * D), dtype=torch.bfloat16, device="cuda"),
                          v=torch.zeros((n_pages * page, GV * Dv), dtype=torch.bfloat16, device="cuda"), page_tokens=page, window=0)
        proj, q = torch.empty((T, N), dtype=torch.bfloat16, device="cuda"), torch.empty((T, H * D), dtype=torch.bfloat16, device="cuda")
        b = dev(bias)
        ops16.gemm(a, w, proj, bias=b, defer=defer)
        more = ops16.head_norm_store(proj, H, G, D, Dv, None, None, 1e-5, q, cache, ints(slots), n_v_heads=GV, norm=True, after=True, positions=ints(positions),
                                     inv_freq=dev(freqs) if rot else None, rot_dim=rot, extra="a test's columns")
        for got, first, heads in ((q, 0, H), (cache.k[page:page + T], H * D, G)):
            ref = rows[:, first:first + heads * D].reshape(T, heads, D)
            ref = pl.unit_rms(pl.rotate(ref, positions, freqs) if rot else ref, 1e-5).reshape(T, -1)
            assert np.max(np.abs(got.float().cpu().numpy() - ref)) <= 6e-2, defer
        v = from_value_layout(cache.v.float().cpu().numpy(), page)[slots]
        assert np.max(np.abs(v - rows[:, (H + G) * D:N - n_extra])) <= 3e-2
        assert np.max(np.abs(more.float().cpu().numpy() - rows[:, N - n_extra:])) <= 3e-2


def masked_case(rng, H, G, share, D, Dv, page, window, chunk, keep, rel_n, lengths, q_lens, dtype, gate_dtype):
    """Requests whose queries are the last positions; keys just inside and just outside the window or chunk, the last kept first
    token and the one behind it, and the query's own stand out for some queries."""
    GV = G // share
    ks, vs, cache, table = paged_rows(rng, lengths, G * D, GV * Dv, page, dtype)
    scale = 1.5 / math.sqrt(D)
    rel = (rng.standard_normal((H, rel_n)) * 1.5).astype(np.float32) if rel_n else None
    sinks = (rng.standard_normal(H) * 1.5).astype(np.float32)
    gates = rng.standard_normal((sum(q_lens), H + 3)).astype(np.float32)
    grp = np.arange(H) // (H // G)
    qs, wants, positions, slots = [], [], [], []
    for s, (n, ql) in enumerate(zip(lengths, q_lens)):
        q = rng.standard_normal((ql, H, D)).astype(np.float32)
        k, v = rounded(ks[s], dtype).reshape(n, G, D), rounded(vs[s], dtype).reshape(n, GV, Dv)
        for i in range(ql):
            p = n - ql + i
            far = [p - window + 1, p - window, keep - 1, keep, p][i % 5] if window else [p - p % chunk, p - p % chunk - 1, p][i % 3] if chunk else [2, page - 1, p][i % 3]
            if 0 <= far <= p:
                q[i] += 4.0 * ks[s][far].reshape(G, D)[grp] / math.sqrt(D)
        qr = rounded(q, dtype)
        want = np.zeros((ql, H, Dv))
        for i in range(ql):
            p = n - ql + i
            j = np.arange(p + 1)
            vis = np.ones(p + 1, bool)
            if window:
                vis &= p - j < window
            if chunk:
                vis &= j // chunk == p // chunk
            if window or chunk:
                vis |= j < keep
            sc = np.einsum("hd,jhd->hj", qr[i], k[:p + 1][:, grp]) * scale
            if rel_n:
                sc = sc + rel.astype(np.float64)[:, np.minimum(p - j, rel_n - 1)]
            sc = np.where(vis[None], sc, -np.inf)
            e = np.exp(sc - sc.max(axis=1, keepdims=True))
            a = e / (e.sum(axis=1, keepdims=True) + np.exp(sinks.astype(np.float64) - sc.max(axis=1))[:, None])
            want[i] = np.einsum("hj,jhd->hd", a, v[:p + 1][:, grp // share])
        qs.append(q.reshape(ql, H * D))
        wants.append(want.reshape(ql, H * Dv))
        positions += list(range(n - ql, n))
        slots += [s] * ql
    factor = 0.8 * pl.sigmoid(rounded(gates, gate_dtype)[:, 2:2 + H].astype(np.float64))
    want = (np.concatenate(wants).reshape(-1, H, Dv) * factor[:, :, None]).reshape(-1, H * Dv)
    step = FakeStep(ints(positions), ints(slots), table, None)
    args = dict(v_head_dim=Dv, mask_chunk=chunk, sink=True, sink_scores=dev(sinks), v_share=share, keep_first=keep,
                rel=dev(rel) if rel_n else None, gate=dev(gates, gate_dtype)[:, 2:2 + H], out_scale=0.8)
    return dev(np.concatenate(qs), dtype), cache, step, scale, args, want


MASKED = [
    # H, G, share, D, Dv, page, window, chunk, keep, table, lengths, q_lens
    (4, 2, 1, 10, 7, 8, 11, 0, 3, 0, [1, 5, 64, 130], [1, 3, 20, 1]),                      # sizes for the plain kernel
    (6, 6, 2, 5, 4, 4, 9, 0, 20, 0, [30, 77], [30, 9]),
    (6, 2, 1, 9, 12, 4, 0, 13, 0, 6, [30, 77], [30, 9]),
    (4, 2, 1, 12, 12, 8, 9, 0, 5, 7, [30, 90], [30, 9]),                                   # kept keys and a table: the plain kernel
    (8, 2, 1, 64, 64, 16, 61, 0, 20, 0, [1, 40, 203, 320], [1, 3, 17, 1]),                 # a portion: four waves a tile
    (8, 2, 1, 64, 64, 16, 61, 0, 33, 0, [700, 1500, 62, 61, 95], [1, 1, 1, 1, 1]),         # single tokens
    (8, 4, 2, 32, 64, 16, 83, 0, 27, 0, [700, 300, 30], [1, 1, 1]),                        # two maps on one head of values, twice their size
    (8, 4, 2, 32, 64, 16, 83, 0, 27, 0, [700, 300, 30], [200, 64, 30]),
    (16, 8, 2, 64, 128, 16, 1000, 0, 64, 0, [3000, 999, 1070, 1], [1, 1, 1, 1]),           # keys cut into chunks, the kept ones a chunk of their own
    (16, 8, 2, 64, 128, 16, 600, 0, 64, 0, [1500, 40], [200, 40]),
    (4, 2, 2, 32, 32, 8, 600, 0, 700, 0, [1500], [64]),                                    # more kept keys than the window has; few blocks of a portion
    (4, 1, 1, 32, 32, 8, 600, 0, 33, 0, [1500], [1]),
    (2, 2, 1, 96, 96, 32, 32, 0, 32, 0, [400, 33], [130, 33]),
    (4, 4, 1, 64, 64, 64, 100, 0, 70, 0, [500], [300]),                                    # pages of 64 tokens
    (4, 4, 1, 64, 64, 128, 100, 0, 1, 0, [900], [3]),
    (2, 2, 2, 128, 64, 16, 40, 0, 10, 0, [200, 60], [50, 1]),                              # value heads of half the size
    (3, 1, 1, 64, 32, 16, 40, 0, 10, 0, [200, 60], [2, 1]),
    (8, 2, 1, 64, 64, 16, 0, 50, 0, 33, [1, 49, 50, 51, 203, 320], [1, 1, 1, 3, 60, 1]),   # chunks and a table in LDS
    (8, 2, 1, 64, 64, 16, 0, 600, 0, 230, [700, 1500, 600, 601, 599], [1, 1, 1, 1, 1]),
    (16, 4, 1, 128, 128, 16, 0, 1024, 0, 1024, [3000, 1025, 1024], [1, 1, 1]),
    (16, 4, 1, 128, 128, 16, 0, 1024, 0, 100, [1500, 40], [300, 40]),
    (8, 1, 1, 32, 32, 16, 0, 2000, 0, 1500, [1900], [70]),                                 # a table too large for LDS
    (8, 1, 1, 32, 32, 16, 0, 2000, 0, 1500, [1900, 3], [1, 1]),
    (6, 2, 1, 32, 64, 16, 0, 64, 0, 40, [130, 64], [40, 1]),
    (4, 4, 1, 96, 96, 8, 0, 7, 0, 2, [90, 17], [40, 1]),
    (4, 2, 1, 64, 128, 16, 33, 0, 0, 0, [90, 170], [40, 1]),                               # a window alone with wide values
    (4, 2, 1, 128, 64, 16, 0, 0, 0, 50, [90, 170], [40, 1]),                               # no mask
    (6, 1, 1, 64, 64, 16, 1, 0, 2, 0, [90, 17], [40, 1]),                                  # a window of the token itself
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,share,D,Dv,page,window,chunk,keep,rel_n,lengths,q_lens", MASKED)
def test_attention_with_kept_keys_distance_tables_shared_values_and_gates(ops16, ops32, dtype, H, G, share, D, Dv, page, window, chunk, keep, rel_n, lengths, q_lens):
    ops = ops16 if dtype == torch.bfloat16 else ops32
    rng = np.random.default_rng(H + D + sum(lengths) + rel_n)
    for gate_dtype, out_dtype in ((torch.float32, torch.float32), (dtype, dtype)):
        q, cache, step, scale, args, want = masked_case(rng, H, G, share, D, Dv, page, window, chunk, keep, rel_n, lengths, q_lens, dtype, gate_dtype)
        for plain in (False, True):
            out = torch.full((q.shape[0], H * Dv + 16), float("nan"), dtype=out_dtype, device="cuda")      # rows that lie apart
            ops.force_plain_attention = plain
            try:
                ops.paged_attention(q, H, G, D, cache, step, window, scale, out[:, 8:8 + H * Dv], **args)
            finally:
                ops.force_plain_attention = False
            err = np.max(np.abs(out[:, 8:8 + H * Dv].float().cpu().numpy() - want))
            assert err <= (3e-5 if dtype == torch.float32 else 0.03), f"plain {plain} {out_dtype}: {err:.3e}"
            assert torch.isnan(out[:, :8]).all() and torch.isnan(out[:, 8 + H * Dv:]).all()


def test_attention_refuses_what_does_not_go_together(ops16):
    from hf_cpu_amd.status import EngineError
    rng = np.random.default_rng(0)
    q, cache, step, scale, _, _ = masked_case(rng, 4, 2, 1, 32, 32, 16, 7, 0, 0, 0, [20], [1], torch.bfloat16, torch.float32)
    out = torch.empty((1, 128), dtype=torch.bfloat16, device="cuda")
    for bad in (dict(rel=dev(np.ones((3, 5)))), dict(gate=dev(np.ones((1, 3)))), dict(v_share=3), dict(rel=dev(np.ones((4, 5))), weights="sigmoid"),
                dict(cross_values=True, keep_first=3), dict(v_share=2)):
        with pytest.raises(EngineError):
            ops16.paged_attention(q, 4, 2, 32, cache, step, 7, scale, out, **bad)


@pytest.mark.parametrize("T,H,G,Dv", [(1, 1, 1, 1), (5, 6, 3, 7), (3, 4, 1, 64), (300, 16, 4, 128), (9, 2, 2, 200), (2, 8, 2, 300)])
def test_two_maps_as_one(ops32, ops16, T, H, G, Dv):
    rng = np.random.default_rng(T + Dv)
    a = rng.standard_normal((T, G, 2, H // G, Dv)).astype(np.float32)
    d = (a[:, :, 0].astype(np.float64) - 0.75 * a[:, :, 1]).reshape(T, H, Dv)
    want = (pl.unit_rms(d, 1e-5) * 0.6).reshape(T, -1)
    for ops in (ops32, ops16):
        wide = torch.zeros((T, H * Dv + 8), dtype=ops.act_dtype, device="cuda")
        ops.diff_mix(dev(a.reshape(T, -1)), dev([0.75]), 0.6, 1e-5, H, G, Dv, wide[:, 8:])
        assert np.max(np.abs(wide[:, 8:].float().cpu().numpy() - want)) <= (1e-5 if ops is ops32 else 1e-2)
        assert (wide[:, :8] == 0).all()


@pytest.mark.parametrize("M,E,F", [(1, 256, 96), (8, 128, 320), (20, 512, 64), (48, 256, 512), (100, 128, 96), (300, 256, 224), (1100, 512, 512), (5, 40, 32), (7, 44, 20)])
def test_gated_units_with_the_tanh_gelu(ops16, ops32, M, E, F):
    """In the product's last lines where gate and up rows are interleaved, and as a kernel of its own; z from -6 to 6."""
    from hf_cpu_amd.parts.mlp import GatedMLP
    rng = np.random.default_rng(M + F)
    x = rng.standard_normal((M, E)).astype(np.float32)
    w = {n: helpers.bf16_round(rng.standard_normal(s) * sd) for n, s, sd in (("gate", (F, E), 2.0 / math.sqrt(E)), ("up", (F, E), 1.0 / math.sqrt(E)), ("down", (E, F), 1.0 / math.sqrt(F)))}
    for ops in (ops16, ops32):
        h = rounded(x, ops.act_dtype).astype(np.float64)
        for act, fn in (("gelu_tanh", pl.gelu_tanh), ("silu", pl.silu)):
            part = GatedMLP(E, F, activation=act, names=dict(gate="gate", up="up", down="down"))
            part.bind({k: dev(v, ops.act_dtype) for k, v in w.items()}, ops)
            want = (fn(h @ w["gate"].T.astype(np.float64)) * (h @ w["up"].T.astype(np.float64))) @ w["down"].T.astype(np.float64)
            y = torch.full((M, E), 3.0, dtype=torch.float32, device="cuda")
            part.forward(ops, None, dev(x, ops.act_dtype), y, accumulate=False)
            ops.settle()
            assert rel_err(y.cpu().numpy(), want) <= (1e-5 if ops is ops32 else 1e-2), (act, ops.act_dtype)
            part.forward(ops, None, dev(x, ops.act_dtype), y)
            ops.settle()
            assert rel_err(y.cpu().numpy(), 2.0 * want) <= (1e-5 if ops is ops32 else 1e-2)
    part = GatedMLP(E, F, activation="gelu_tanh", names=dict(gate="gate", up="up", down="down"))
    big = {"gate": dev(np.full((F, E), 4.0)), "up": dev(np.ones((F, E))), "down": dev(np.ones((E, F)))}
    part.bind(big, ops32)
    for sign in (1.0, -1.0):                                       # far from zero: z itself, or nothing
        y = torch.empty((1, E), dtype=torch.float32, device="cuda")
        part.forward(ops32, None, dev(np.full((1, E), sign)), y, accumulate=False)
        ops32.settle()
        assert np.allclose(y.cpu().numpy(), F * E * 4.0 * E if sign > 0 else 0.0, rtol=1e-6, atol=1e-3)


@pytest.mark.parametrize("T,E,top", [(1, 1, 1), (7, 5, 3), (64, 14, 3), (130, 64, 8), (3, 300, 6), (2000, 32, 4)])
def test_router_with_a_correction_for_the_choice_alone(ops32, T, E, top):
    rng = np.random.default_rng(T + E)
    z, c = rng.standard_normal((T, E)).astype(np.float32), (rng.standard_normal(E) * 0.4).astype(np.float32)
    if E >= 5:
        z[0] = 0.5                                                 # equal scores: the correction decides, among equals the lower index
        c[1] = c[3] = float(c.max()) + 0.25
    ids, w = ops32.moe_route(dev(z), top, 1, 1, "sigmoid", False, 2.25, correction=dev(c))
    s = pl.sigmoid(z.astype(np.float64))
    order = np.argsort(-(1.0 / (1.0 + np.exp(-z)) + c), axis=1, kind="stable")[:, :top]
    got = ids.cpu().numpy()
    clear = np.array([np.min(np.abs(np.diff(np.sort(s[t] + c)))) > 1e-6 if E > 1 and t else True for t in range(T)])
    assert clear.mean() >= 0.9 or E >= 300
    assert np.array_equal(got[clear], order[clear])
    assert np.allclose(w.cpu().numpy(), 2.25 * np.take_along_axis(s, got, axis=1), rtol=1e-6)


@pytest.mark.parametrize("T,E,X,top,F,shared", [(1, 44, 5, 3, 12, 8), (9, 64, 4, 1, 32, 6), (60, 128, 8, 2, 64, 64), (300, 256, 6, 6, 96, 128), (700, 128, 3, 1, 64, None)])
def test_experts_with_a_gated_shared_expert_as_a_part(ops32, ops16, T, E, X, top, F, shared):
    from hf_cpu_amd.parts.moe import MixtureOfExperts
    from hf_cpu_amd.plan import PartSpec
    rng = np.random.default_rng(T + F)
    f = lh.moe(X, top, F, shared=shared, scale=1.7)
    cfg = lh.config(10, E, layers=[lh.layer(lh.attention(1, 1, 2, 2, 4, 2), f)])
    w = {k[len("l0.mlp."):]: v for k, v in lh.make_weights(cfg, T).items() if k.startswith("l0.mlp.")}
    w["correction"] = helpers.bf16_round(rng.permutation(X) * 2.0)            # (far apart: no rounding changes a choice)
    x = helpers.bf16_round(rng.standard_normal((T, E)))
    want = pl.feed_forward(x.astype(np.float64), {k: np.asarray(v, np.float64) for k, v in w.items()}, "", f)
    for ops in (ops32, ops16):
        names = dict(gate="gate", up="up", down="down")
        part = MixtureOfExperts(E, F, X, top, scoring="sigmoid", renormalize=False, weight_scale=1.7, gated=dict(alpha=1.0), correction=True,
                                shared=PartSpec("gated_mlp", dict(hidden_size=E, intermediate_size=shared, prefix="shared.", names=names)) if shared else None,
                                shared_gate=bool(shared), names=dict(router="router", correction="correction", shared_gate="shared.sg",
                                                                     gate="e{e}.gate", up="e{e}.up", down="e{e}.down"))
        part.bind_all({k: dev(v, torch.float32 if k == "correction" else ops.act_dtype) for k, v in w.items()}, ops)
        h = dev(x, ops.act_dtype)
        y = torch.full((T, E), 5.0, dtype=torch.float32, device="cuda")
        part.forward(ops, None, h, y, accumulate=False)
        ops.settle()
        assert rel_err(y.cpu().numpy(), want) <= (1e-5 if ops is ops32 else 2e-2)
        part.forward(ops, None, h, y)
        ops.settle()
        assert rel_err(y.cpu().numpy(), 2.0 * want) <= (1e-5 if ops is ops32 else 2e-2)


@pytest.mark.parametrize("H,D,P,rot", [(1, 2, 1, 2), (3, 7, 5, 4), (2, 20, 12, 20), (4, 32, 64, 32), (2, 128, 128, 64), (1, 256, 17, 256)])
def test_retention_in_portions_and_single_tokens(ops32, ops16, H, D, P, rot):
    """Three requests in portions of changing size down to one token, their states carried between them; the second pass runs
    in state rows that others have used and that were cleared."""
    from hf_cpu_amd.parts.recurrent import Retention
    from hf_cpu_amd.plan import PartSpec
    E = 64
    rng = np.random.default_rng(D + P)
    m = lh.right(H, D, P, rot, base=50.0, decay=[1.0 - 0.3 * 0.1 ** h for h in range(H)])
    w = {n: helpers.bf16_round(rng.standard_normal(s) / math.sqrt(s[1])) for n, s in (("q", (H * D, E)), ("k", (H * D, E)), ("v", (H * P, E)), ("g", (H * P, E)), ("o", (E, H * P)))}
    lengths, slots = [90, 11, 40], [1, 3, 0]
    cuts = [[1, 2, 70, 1, 1, 15], [2, 1, 1, 5, 1, 1], [16, 1, 1, 1, 20, 1]]
    xs = [helpers.bf16_round(rng.standard_normal((n, E))) for n in lengths]
    ref = [pl.retention(x.astype(np.float64), {k: v.astype(np.float64) for k, v in w.items()}, "", m, 1e-5, np.arange(len(x))) for x in xs]
    for ops in (ops32, ops16):
        part = Retention(E, H, D, P, m["decay"], 1e-5, PartSpec("rotary", dict(head_dim=D, rot_dim=rot, theta=50.0)), names={n: n for n in "qkvgo"})
        part.bind_all({k: dev(v, ops.act_dtype) for k, v in w.items()}, ops)
        state = torch.zeros((5, part.cache_need().n_floats), dtype=torch.float32, device="cuda")
        cache = types.SimpleNamespace(state=state)
        for again in range(2):
            at = [0, 0, 0]
            for turn in range(6):
                take = [xs[s][at[s]:at[s] + cuts[s][turn]] for s in range(3)]
                step = state_step([len(t) for t in take], slots)
                step.positions = ints(np.concatenate([np.arange(at[s], at[s] + len(take[s])) for s in range(3)]))
                y = torch.empty((step.n_tokens, E), dtype=torch.float32, device="cuda")
                with ops.on_current_stream():
                    part.forward(ops, step, dev(np.concatenate(take), ops.act_dtype), cache, y, accumulate=False)
                    ops.settle()
                got, r0 = y.cpu().numpy(), 0
                for s in range(3):
                    c = len(take[s])
                    want = ref[s][at[s]:at[s] + c]
                    err = np.abs(got[r0:r0 + c] - want)
                    scale = np.max(np.abs(ref[s]))
                    # (a token's read-out is normed: where it is nearly zero, sixteen-bit inputs turn it)
                    assert np.max(err) <= 1e-4 * scale if ops is ops32 else np.median(err) <= 2e-2 * scale, (again, turn, s)
                    at[s], r0 = at[s] + c, r0 + c
            assert at == lengths
            state[torch.tensor(slots, device="cuda")] = 0.0
        assert float(state.abs().max()) == 0.0


# ---- whole models --------------------------------------------------------------------------------------------------

@pytest.fixture(scope="module", params=list(lh.CONFIGS))
def tiny(request, tmp_path_factory, gpu):
    cfg = lh.CONFIGS[request.param]
    d = lh.make_model_dir(str(tmp_path_factory.mktemp(request.param) / "model"), cfg, seed=7, stored=lh.STORED[request.param])
    reqs = lh.random_requests(cfg, [61, 97, 130, 7, 5, 9, 24, 57, 2], seed=11)
    return request.param, cfg, d, reqs, lh.plain_logits(d, reqs)


def engine_for(d, dtype, name, max_tokens, max_seqs=4, **kw):
    import hf_cpu_amd
    return hf_cpu_amd.load_engine(d, dtype=dtype, page_tokens=lh.PAGE[name], max_tokens=max_tokens, max_seqs=max_seqs, **kw)


def run_against_plain(name, d, want, dtype, steps, what, **kw):
    engine = engine_for(d, dtype, name, helpers.max_live_tokens(steps), **kw)
    got = helpers.run_trace_in_engine(engine, steps)
    worst = compare_for(dtype, got, want, tol_of(name, dtype), what)
    engine.manager.check()
    assert engine.manager.stats()["requests"] == 0
    return engine, got, worst


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_stream_after_every_layer(gpu, tiny, dtype):
    """One prompt's stream after each layer, then of its last tokens decoded one by one."""
    name, cfg, d, reqs, _ = tiny
    toks = reqs["r6"]
    pcfg, w = pl.read_model(d)
    want = []
    pl.forward(pcfg, w, toks, want)
    engine = engine_for(d, dtype, name, 64, graphs=False)
    seen = []
    for l in engine.model.layers:
        def wrapped(ops, step, x, parts, caches, write_cache=True, inner=l.block.forward):
            inner(ops, step, x, parts, caches, write_cache)
            ops.settle()
            seen.append(x.cpu().numpy())
        l.block.forward = wrapped
    at = 0
    for n in [19, 1, 1, 2, 1]:
        seen.clear()
        engine.step([("a", toks[at:at + n], [0])])
        for l, got in enumerate(seen):
            ref = want[l][at:at + n]
            err = np.max(np.abs(got - ref), axis=1) / np.max(np.abs(want[l]))
            assert np.max(err) <= 2e-5 if dtype == "float32" else np.median(err) <= 4e-2, f"layer {l}, tokens from {at}: {err}"
        at += n


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("cutting", ["whole", "tail", "portions", "mixed"])
def test_cuttings(gpu, tiny, dtype, cutting):
    """Whole prompts; most of a prompt and then token by token; portions of changing size down to two tokens; up to
    four requests live, portions beside single tokens, pages and state rows used again."""
    name, cfg, d, reqs, want = tiny
    steps = {"whole": helpers.trace_whole, "tail": lambda r: helpers.trace_tail(r, tail=90),
             "portions": helpers.trace_portions, "mixed": lambda r: helpers.trace_mixed(r, seed=3)}[cutting](reqs)
    engine, got, worst = run_against_plain(name, d, want, dtype, steps, f"{name} {dtype} {cutting}")
    assert len(got) == sum(len(t) for t in reqs.values())
    print(f"{name} {dtype} {cutting}: worst |diff| {worst:.3e}")
    if cutting == "mixed":
        assert any(p.reused > 0 for p in engine.manager.pools), "the trace was meant to use pages again"


def test_cuttings_agree_with_each_other(gpu, tiny):
    """In fp32 the cuttings agree among themselves: the same values are computed, only in other launches."""
    name, cfg, d, reqs, _ = tiny
    results = []
    for make in (helpers.trace_whole, helpers.trace_portions, lambda r: helpers.trace_tail(r, tail=60),
                 lambda r: helpers.trace_mixed(r, seed=5), lambda r: helpers.trace_portions(r, sizes=(2, 2, 3, 2, 64, 2, 7))):
        steps = make(reqs)
        engine = engine_for(d, "float32", name, helpers.max_live_tokens(steps))
        results.append(helpers.run_trace_in_engine(engine, steps))
    for other in results[1:]:
        for key, row in results[0].items():
            err = float(np.max(np.abs(row - other[key])))
            assert err <= 5e-5 * max(1.0, float(np.max(np.abs(row)))), f"{name}: {key}: cuttings differ by {err:.3e}"


def test_a_batch_of_unequal_requests_against_each_alone(gpu, tiny):
    name, cfg, d, reqs, want = tiny
    engine = engine_for(d, "float32", name, 64 * len(reqs) + sum(len(t) for t in reqs.values()), max_seqs=len(reqs))
    together = engine.step([(r, toks, list(range(len(toks)))) for r, toks in reqs.items()]).cpu().numpy()
    at = 0
    for r, toks in reqs.items():
        engine.release(r)
        alone = engine.step([(r + "'", toks, list(range(len(toks))))]).cpu().numpy()
        engine.release(r + "'")
        assert np.max(np.abs(alone - together[at:at + len(toks)])) <= 5e-5 * np.max(np.abs(want[r]))
        assert np.max(np.abs(alone - want[r])) <= TOL["float32"] * np.max(np.abs(want[r]))
        at += len(toks)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_in_a_small_pool(gpu, tiny, dtype):
    """Three requests decoded token by token together from their second token on, in a pool that holds them and no
    more, then three more in the pages and state rows that they gave back: what the first left there must be gone."""
    name, cfg, d, reqs, want = tiny
    long = {r: t for r, t in reqs.items() if len(t) >= 57}
    names = list(long)[:3]
    order = [names, names[::-1]]                    # the second turn's requests land in other state rows than the first's
    steps = []
    for turn in range(2):
        ids = {r: f"{r}/{turn}" for r in names}
        steps.append(helpers._step(len(steps), [(ids[r], long[r][:2], [0, 1]) for r in order[turn]]))
        for i in range(2, max(len(long[r]) for r in names)):
            live = [r for r in order[turn] if i < len(long[r])]
            steps.append(helpers._step(len(steps), [(ids[r], long[r][i:i + 1], [0]) for r in live],
                                       [ids[r] for r in live if i == len(long[r]) - 1]))
    want2 = {f"{r}/{turn}": want[r] for r in names for turn in range(2)}
    engine, got, _ = run_against_plain(name, d, want2, dtype, steps, f"{name} {dtype} long decoding")
    assert all(p.reused > 0 for p in engine.manager.pools)
    assert engine.graph_replays > 0, "decode steps were meant to replay captured graphs"


def test_trace_replay_program(gpu, tiny, tmp_path):
    """bin/trace_run as a user calls it (pages of 16, four state rows, a pool for the live requests only): a mixed trace
    against the plain implementation in both dtypes."""
    import json
    import os
    import subprocess
    import sys
    name, cfg, d, reqs, want = tiny
    steps = helpers.trace_mixed(reqs, seed=21)
    places = helpers.wanted_places(steps)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    for dtype in ("float32", "bfloat16"):
        out = tmp_path / dtype
        r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", d, "--dtype", dtype, "--out", str(out),
                            "--max-tokens", str(helpers.max_live_tokens(steps))],
                           input="".join(json.dumps(st) + "\n" for st in steps), text=True, capture_output=True, timeout=300)
        assert r.returncode == 0, r.stderr
        assert [w for w in r.stdout.split() if w != "done"] == [str(st["step"]) for st in steps]
        got = {}
        for st in steps:
            if st["step"] in places:
                rows = np.fromfile(out / f"{st['step']}.f32", dtype="<f4").reshape(len(places[st["step"]]), -1)
                got.update(zip(places[st["step"]], rows))
        assert len(got) == sum(len(t) for t in reqs.values())
        compare_for(dtype, got, want, tol_of(name, dtype), "trace_run " + dtype)


def test_greedy_generation_through_the_session(gpu, tiny):
    """Greedy continuation of three prompts through Session.generate (the scheduler, the sampler, graphs): every token
    is the plain implementation's best, or within rounding of it."""
    import hf_cpu_amd.session as S
    name, cfg, d, reqs, _ = tiny
    prompts = [reqs["r3"], reqs["r4"], reqs["r5"]]
    pcfg, w = pl.read_model(d)
    s = S.Session(d, dtype="float32", ctx_max=256, batch=16, page_size=lh.PAGE[name], max_seqs=4)
    gens = s.generate(prompts, temp=0.0, max_tokens=40)
    for g, p in zip(gens, prompts):
        assert len(g.tokens) == 40
        rows = pl.forward(pcfg, w, list(p) + g.tokens)
        for i, t in enumerate(g.tokens):
            row = rows[len(p) - 1 + i]
            assert row[int(np.argmax(row))] - row[t] <= 1e-4 * max(1.0, float(np.max(np.abs(row)))), \
                f"token {i} = {t}, plain picks {int(np.argmax(row))}"


def test_command_line_generates_and_forks(gpu, tiny):
    """bin/hfamd on a folder of this design: greedy tokens are the plain implementation's; two continuations of one prompt
    (the second forks the first's pages, the kept ones among them, and state rows after the prompt) are the same; sampled runs
    with one seed repeat themselves."""
    import os
    import subprocess
    import sys
    name, cfg, d, reqs, _ = tiny
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    prompt = reqs["r7"]

    def run(extra):
        r = subprocess.run([sys.executable, os.path.join(root, "bin", "hfamd"), "--stdin-mode", "none", "--model", d, "--dtype", "float32",
                            "--ctx-max", "128", "--page-size", str(lh.PAGE[name]), "--max-seqs", "4", "--log-level", "error",
                            "--prompt-ids", " ".join(map(str, prompt))] + extra, text=True, capture_output=True, timeout=300)
        assert r.returncode == 0, r.stderr
        toks = {}
        for line in r.stdout.replace("\x1e", "\n").splitlines():
            if line.startswith("@token "):
                f = dict(x.split("=", 1) for x in line.split(" ")[1:] if "=" in x)
                toks.setdefault(f.get("seq", "0"), []).append(int(f["id"]))
        return toks
    greedy = run(["--temp", "0", "--max-tokens", "6"])["0"]
    pcfg, w = pl.read_model(d)
    rows = pl.forward(pcfg, w, prompt + greedy)
    for i, t in enumerate(greedy):
        row = rows[len(prompt) - 1 + i]
        assert row[int(np.argmax(row))] - row[t] <= 1e-4 * max(1.0, float(np.max(np.abs(row))))
    both = run(["--temp", "0", "--max-tokens", "5", "--n", "2"])
    assert both["0"] == greedy[:5] and both["1"] == greedy[:5]
    drawn = run(["--temp", "0.9", "--seed", "11", "--max-tokens", "8", "--n", "2"])
    assert drawn == run(["--temp", "0.9", "--seed", "11", "--max-tokens", "8", "--n", "2"]) and len(drawn["0"]) == 8 and len(drawn["1"]) == 8


def edge_model(kind, size, keep=0):
    """One layer that shows a single key. Token 1 alone has an entry in the table's column before the last, every token the same
    entry in the last column. Queries are a fixed direction, keys another one at right angles to it, token 1's key the queries' own
    with a large multiple: after the per-head norms every query that sees token 1 gives it nearly all its weight, and the values of
    all other tokens are zero, so that nothing is left where it is not seen. The rotated dimensions hold nothing."""
    E, D = 64, 32
    rng = np.random.default_rng(5)
    mix = {"window": lambda: lh.attention(2, 1, D, 32, size, 2, scale=0.4),
           "chunk": lambda: lh.parallel(lh.left(2, 1, D, 32, size, 40, 16, scale=0.4), lh.right(1, 8, 8, 8, decay=[0.5]), 1.0, 0.0),
           "kept": lambda: lh.diff(2, 1, D, 32, size, keep, 0.3, scale=0.4)}[kind]()
    cfg = lh.config(50, E, [lh.layer(mix, None)], embedding_scale=1.0)
    w = lh.make_weights(cfg, seed=1)
    p = "l0.mix.left." if kind == "chunk" else "l0.mix."
    u, r = np.zeros(D), np.zeros(D)
    u[2:16], r[16:] = np.sign(rng.standard_normal(14)), np.sign(rng.standard_normal(16))
    maps = 2 if kind == "kept" else 1
    for n in ("q", "k", "v"):
        w[p + n][:] = 0.0
        if p + n + ".b" in w:
            w[p + n + ".b"][:] = 0.0
    for hd in range(2 * maps):
        w[p + "q"][hd * D:(hd + 1) * D, E - 1] = u if hd % maps == 0 else r      # (a second map that looks elsewhere)
    for hd in range(maps):
        w[p + "k"][hd * D:(hd + 1) * D, E - 1], w[p + "k"][hd * D:(hd + 1) * D, E - 2] = r, 8.0 * u
    w[p + "v"][:, E - 2] = helpers.bf16_round(rng.standard_normal(32) * 2.0)
    w["embed"][:, E - 2:] = 0.0
    w["embed"][:, E - 1] = 1.0
    w["embed"][1, E - 2] = 4.0
    w["l0.norm1"][:] = 1.0
    return cfg, w


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind,size,keep", [("window", 20, 0), ("window", 129, 0), ("window", 600, 0), ("chunk", 33, 0), ("chunk", 128, 0), ("chunk", 700, 0),
                                            ("kept", 24, 16), ("kept", 70, 17), ("kept", 300, 98), ("kept", 40, 3)])
def test_a_key_just_inside_and_just_outside_its_mask(gpu, tmp_path, dtype, kind, size, keep):
    """The marked token at a page's first and last place and in between: the last query that sees it and the first that does not,
    inside a prompt's first portion, in a second portion, and among decoded tokens; kept first tokens that are seen for good and
    the one behind them that is not."""
    import hf_cpu_amd
    cfg, w = edge_model(kind, size, keep)
    d = lh.make_model_dir(str(tmp_path / "m"), cfg, seed=0, weights=w, stored="BF16")
    rng = np.random.default_rng(9)
    n = size + 240
    base = [int(t) for t in rng.integers(2, cfg["vocab"], n)]
    reqs = {f"at{at}": base[:at] + [1] + base[at + 1:] for at in sorted({2, 15, 16, 97, 150, 215, max(0, keep - 1), keep})}
    reqs["none"] = base
    want = lh.plain_logits(d, reqs)
    size_of = float(np.max(np.abs(want["none"])))
    steps = []
    for r, t in reqs.items():
        if r != "none":
            at = int(r[2:])
            last = (at // size + 1) * size - 1 if kind == "chunk" else n - 1 if at < keep else at + size - 1
            diffs = np.max(np.abs(want[r] - want["none"]), axis=1)
            assert diffs[min(last, n - 1)] >= 0.1 * size_of, "the plain logits do not show the key"
            assert last + 1 >= n or diffs[last + 1] <= 1e-9 * size_of
        cut, head = size + 60, size + 130
        steps.append(helpers._step(len(steps), [(r, t[:cut], range(cut))]))
        steps.append(helpers._step(len(steps), [(r, t[cut:head], range(head - cut))]))
        for i in range(head, n):
            steps.append(helpers._step(len(steps), [(r, t[i:i + 1], [0])], [r] if i == n - 1 else []))
    engine = hf_cpu_amd.load_engine(d, dtype=dtype, page_tokens=16, max_tokens=helpers.max_live_tokens(steps), max_seqs=1)
    got = helpers.run_trace_in_engine(engine, steps)
    helpers.compare(got, want, TOL[dtype], f"{kind} {size} {dtype}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_long_prompt_decoded_token_by_token(gpu, tmp_path, dtype):
    """Two requests of 700 and 1,300 tokens: the prompt in two portions (the second begins in the middle of a page),
    then 45 tokens decoded together; windows and chunks of hundreds of tokens whose keys a decoded token cuts over many waves."""
    import hf_cpu_amd
    cfg = lh.config(300, 128, layers=[
        lh.layer(lh.attention(4, 2, 32, 32, 500, 16), lh.dense(128)),
        lh.layer(lh.parallel(lh.left(4, 2, 32, 32, 640, 300, 32), lh.right(2, 32, 32, 32, decay=[0.999, 0.98])), None),
        lh.layer(lh.diff(4, 2, 32, 64, 300, 70), lh.moe(4, 2, 32, shared=64))])
    d = lh.make_model_dir(str(tmp_path / "m"), cfg, seed=4, stored="BF16")
    reqs = lh.random_requests(cfg, [700, 1300], seed=2)
    want = lh.plain_logits(d, reqs)
    steps = []
    heads = {r: len(t) - 45 for r, t in reqs.items()}
    for r, t in reqs.items():
        steps.append(helpers._step(len(steps), [(r, t[:heads[r] - 201], [heads[r] - 202])]))
        steps.append(helpers._step(len(steps), [(r, t[heads[r] - 201:heads[r]], [0, 200])]))
    for i in range(45):
        steps.append(helpers._step(len(steps), [(r, t[heads[r] + i:heads[r] + i + 1], [0]) for r, t in reqs.items()],
                                   list(reqs) if i == 44 else []))
    engine = hf_cpu_amd.load_engine(d, dtype=dtype, page_tokens=16, max_tokens=helpers.max_live_tokens(steps), max_seqs=2)
    got = helpers.run_trace_in_engine(engine, steps)
    assert len(got) == 2 * 48
    helpers.compare(got, want, TOL[dtype], f"long prompts {dtype}")
    engine.manager.check()


def test_graphs_of_decode_steps_survive_a_longer_prompt(gpu, tmp_path):
    """Decode steps of a short request are captured into graphs; then a prompt arrives that is longer than anything before
    (work buffers grow); the short request's next steps, replayed or captured anew, still give the plain logits."""
    import hf_cpu_amd
    cfg = lh.config(120, 64, layers=[lh.layer(lh.diff(4, 2, 32, 32, 25, 6), lh.dense(64)), lh.layer(lh.attention(2, 2, 32, 32, 30, 32), lh.moe(3, 2, 32, shared=32)),
                                     lh.layer(lh.parallel(lh.left(2, 1, 32, 32, 48, 20, 8), lh.right(1, 32, 32, 16)), None)])
    d = lh.make_model_dir(str(tmp_path / "m"), cfg, seed=2, stored="BF16")
    reqs = lh.random_requests(cfg, [40, 1300], seed=5)
    want = lh.plain_logits(d, reqs)
    a, b = reqs["r0"], reqs["r1"]
    steps = [helpers._step(0, [("r0", a[:20], [19])])]
    steps += [helpers._step(len(steps) + i, [("r0", a[20 + i:21 + i], [0])]) for i in range(8)]
    steps.append(helpers._step(len(steps), [("r1", b, [0, 1299])], ["r1"]))
    steps += [helpers._step(len(steps) + i, [("r0", a[28 + i:29 + i], [0])], ["r0"] if i == 11 else []) for i in range(12)]
    for dtype in ("float32", "bfloat16"):
        engine = hf_cpu_amd.load_engine(d, dtype=dtype, page_tokens=16, max_tokens=helpers.max_live_tokens(steps), max_seqs=2)
        got = helpers.run_trace_in_engine(engine, steps)
        assert engine.graph_replays > 0
        helpers.compare(got, want, TOL[dtype], f"graphs and a longer prompt {dtype}")


def test_a_checkpoint_may_hold_the_norm_of_a_sublayer_that_a_layer_lacks(gpu, tmp_path):
    import hf_cpu_amd
    cfg = lh.config(60, 32, layers=[lh.layer(lh.attention(2, 1, 8, 8, 6, 4), None)])
    w = lh.make_weights(cfg, 0)
    toks = [3, 9, 27, 50, 1, 4, 5, 6, 7, 8]
    rows = []
    for extra in (False, True):
        if extra:
            w["l0.norm2"] = np.ones(32)
        d = lh.make_model_dir(str(tmp_path / f"m{extra}"), cfg, 0, weights=w, stored="BF16")
        engine = hf_cpu_amd.load_engine(d, dtype="float32", page_tokens=4, max_tokens=64, max_seqs=1)
        rows.append(engine.step([("a", toks, list(range(10)))]).cpu().numpy())
    assert np.array_equal(rows[0], rows[1])


def test_random_weights_and_other_orders_of_layers(gpu, tmp_path):
    """``write_random_model`` makes a folder for this design too, and the engine reads it back: models of one kind of layer only,
    without masks and rescaled frequencies, and with widths that are no multiple of 8."""
    import copy
    import hf_cpu_amd
    from hf_cpu_amd.config import config_from_dict
    one = lh.config(90, 64, layers=[lh.layer(lh.attention(2, 1, 32, 32, 12, 32), lh.dense(16))] * 2)
    two = lh.config(90, 64, layers=[lh.layer(lh.parallel(lh.left(2, 1, 32, 32, 9, 20, 8), lh.right(2, 32, 32, 32)), None)])
    odd = lh.config(77, 100, eps=1e-3, layers=[lh.layer(lh.diff(3, 1, 20, 28, 8, 5), lh.moe(3, 2, 12)), lh.layer(lh.diff(5, 5, 4, 3, 1, 0), None)])
    bare = copy.deepcopy(lh.config(90, 64, layers=[lh.layer(lh.attention(2, 1, 32, 32, 100, 16), None), lh.layer(lh.diff(2, 1, 32, 32, 100, 0), None),
                                                   lh.layer(lh.parallel(lh.left(2, 2, 16, 32, 100, 20, 8), lh.right(2, 32, 32, 32)), None)]))
    unmasked = copy.deepcopy(bare)                               # the plain implementation wants a mask: one that hides nothing
    for lc in unmasked["layers"]:
        (lc["mixer"]["left"] if lc["type"] == "parallel" else lc["mixer"]).pop("mask")
    for k, (c, e) in enumerate(((one, one), (two, two), (odd, odd), (bare, unmasked))):
        d = str(tmp_path / f"m{k}")
        hf_cpu_amd.write_random_model(d, config_from_dict(e), seed=3, dtype="bfloat16")
        _, w = pl.read_model(d)
        toks = [int(t) for t in np.random.default_rng(0).integers(0, c["vocab"], 45)]
        want = pl.forward(c, w, toks)
        for dtype in ("float32", "bfloat16"):
            engine = hf_cpu_amd.load_engine(d, dtype=dtype, page_tokens=4, max_tokens=64, max_seqs=1)
            got = engine.step([("a", toks[:31], list(range(31)))]).cpu().numpy()
            rows = {("a", i): row for i, row in enumerate(got)}
            for i in range(31, 45):
                rows[("a", i)] = engine.step([("a", toks[i:i + 1], [0])]).cpu().numpy()[0]
            helpers.compare(rows, {"a": want}, TOL[dtype], f"random weights {k} {dtype}")


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(gpu, tmp_path, seed):
    """Layers of every kind in any order with sizes drawn at random (even seeds: sizes for the matrix cores): a prompt, a
    portion that starts in the middle of a page, then single tokens, in fp32 and in bf16."""
    import hf_cpu_amd
    rng = np.random.default_rng(100 + seed)
    cfg = lh.random_config(rng, big=seed % 2 == 0)
    d = lh.make_model_dir(str(tmp_path / "m"), cfg, seed=seed, stored="BF16" if seed % 2 == 0 else "F32")
    toks = [int(t) for t in rng.integers(0, cfg["vocab"], 110)]
    pcfg, w = pl.read_model(d)
    want = pl.forward(pcfg, w, toks)
    steps = [helpers._step(0, [("a", toks[:55], range(55))]), helpers._step(1, [("a", toks[55:88], range(33))])]
    steps += [helpers._step(2 + i, [("a", toks[88 + i:89 + i], [0])], ["a"] if i == 21 else []) for i in range(22)]
    for dtype in ("float32", "bfloat16"):
        engine = hf_cpu_amd.load_engine(d, dtype=dtype, page_tokens=16, max_tokens=128, max_seqs=2, graphs=dtype == "float32")
        got = helpers.run_trace_in_engine(engine, steps)
        compare_for(dtype, got, {"a": want}, TOL[dtype] if dtype == "float32" else 8e-2, f"random configuration {seed} {dtype}: {cfg}")
