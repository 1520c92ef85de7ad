"""Fugevik in the engine against its plain implementation (tests/plain_fugevik.py): each mechanism alone at the
kernels, then whole models in every way of cutting the work."""
import math
import types

import numpy as np
import pytest
import torch

import fugevik_helpers as fh
import helpers
import plain_fugevik as pf
from test_gitasun_gpu import paged_rows, rel_err, state_step
from test_kernels_gpu import FakeStep, dev, from_value_layout, ints, rounded

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
# Largest |logit difference| from the float64 plain implementation, as a fraction of the request's largest |logit|.
# fp32: the rounding of fused multiply-adds and exponentials; a lost state, a window that is one token off, a sink or a
# distance term left out, streams mixed in the other direction show as 1e-2 and more.
# bf16: activations and cache rounded to 8 bits of mantissa at every part, residual streams, norms and scores in 32-bit.
TOL = {"float32": 1e-4, "bfloat16": 4e-2}
# What rounding alone does to these models was measured on the plain implementation with the activations that the bf16 engine
# holds in 16 bits rounded there too: up to 3.2e-2 (cores) and 5.1e-2 (ones, at the same position as the engine).
TOL_OF = {("small", "bfloat16"): 8e-2, ("cores", "bfloat16"): 6e-2, ("ones", "bfloat16"): 7e-2}


# ---- mechanisms alone ----------------------------------------------------------------------------------------------

@pytest.mark.parametrize("S,E,T", [(1, 7, 3), (2, 40, 5), (3, 42, 1), (4, 256, 9), (4, 2048, 300), (5, 36, 11), (8, 64, 2), (9, 30, 4), (6, 5000, 3),
                                   (7, 12, 6), (2, 12288, 2), (11, 64, 270)])
def test_streams_updated_read_and_summed(ops32, S, E, T):
    """Copies of the embedding, two sublayers' updates and inputs, then the sum at chosen rows, as the kernels chain them."""
    rng = np.random.default_rng(S * E + T)
    e = rng.standard_normal((T, E)).astype(np.float32)
    ys = [rng.standard_normal((T, E)).astype(np.float32) for _ in range(2)]
    mix = [(rng.standard_normal((S, S)) * 0.6).astype(np.float32) for _ in range(2)]
    out_w = [rng.standard_normal(S).astype(np.float32) for _ in range(2)]
    in_w = [rng.standard_normal(S).astype(np.float32) for _ in range(2)]
    norm = (1.0 + 0.2 * rng.standard_normal(E)).astype(np.float32)
    x = torch.full((T, S, E), float("nan"), dtype=torch.float32, device="cuda")
    ops32.stream_update(x, dev(e))
    want = np.repeat(e[:, None].astype(np.float64), S, axis=1)
    keep = []
    for k in range(2):
        for dtype in DTYPES:                                  # (the second call finds the update done)
            n = torch.empty((T, E), dtype=dtype, device="cuda")
            ops32.stream_input(x, dev(in_w[k]), dev(norm), 1e-5, n)
            ref = pf.rms_norm(pf.stream_input(want, in_w[k].astype(np.float64)), norm.astype(np.float64), 1e-5)
            assert np.max(np.abs(n.float().cpu().numpy() - ref) / (np.abs(ref) + 1.0)) <= (2e-5 if dtype == torch.float32 else 1e-2), (k, dtype)
        assert rel_err(x.cpu().numpy(), want) <= 3e-6
        keep.append(tuple(dev(a) for a in (ys[k], mix[k], out_w[k])))
        ops32.stream_update(x, *keep[-1])
        want = pf.stream_update(want, ys[k].astype(np.float64), mix[k].astype(np.float64), out_w[k].astype(np.float64))
    before = x.clone()
    rows = [T - 1, 0, T // 2]
    total = torch.empty((3, E), dtype=torch.float32, device="cuda")
    ops32.stream_sum(x, total, ints(rows))
    assert np.max(np.abs(total.cpu().numpy() - want.sum(1)[rows])) <= 1e-5 * S * np.max(np.abs(want))
    assert torch.equal(x, before), "the sum leaves the streams alone"
    ops32.stream_update(x, *keep[-1])
    ops32.settle()                                            # an update that nobody takes along is done on demand
    assert rel_err(x.cpu().numpy(), want) <= 3e-6
    total = torch.empty((T, E), dtype=torch.float32, device="cuda")
    ops32.stream_sum(x, total)
    assert np.max(np.abs(total.cpu().numpy() - want.sum(1))) <= 1e-5 * S * np.max(np.abs(want))


@pytest.mark.parametrize("T,E,F", [(3, 256, 4096), (48, 512, 2048), (130, 256, 1024)])
def test_a_sublayers_result_as_partial_sums(ops16, T, E, F):
    """A product whose K was split hands its partial sums to the streams' kernel: the same as the finished product."""
    rng = np.random.default_rng(T)
    a, w = dev(rng.standard_normal((T, F)), torch.bfloat16), dev(rng.standard_normal((E, F)) / math.sqrt(F), torch.bfloat16)
    S = 4
    x0 = dev(rng.standard_normal((T, S, E)))
    mix, out_w, in_w = (dev(rng.standard_normal(s)) for s in ((S, S), (S,), (S,)))
    norm = dev(np.ones(E))
    res = []
    for defer in (True, False):
        y, x, n = torch.empty((T, E), dtype=torch.float32, device="cuda"), x0.clone(), torch.empty((T, E), dtype=torch.float32, device="cuda")
        ops16.gemm(a, w, y, defer=defer)
        ops16.stream_update(x, y, mix, out_w)
        ops16.stream_input(x, in_w, norm, 1e-6, n)
        res.append((x.cpu().numpy(), n.cpu().numpy()))
    for got, want in zip(*res):
        assert np.max(np.abs(got - want)) <= 1e-4 * np.max(np.abs(want))
    ref = a.double().cpu().numpy() @ w.double().cpu().numpy().T
    ref = pf.stream_update(x0.double().cpu().numpy(), ref, mix.double().cpu().numpy(), out_w.double().cpu().numpy())
    assert rel_err(res[0][0], ref) <= 1e-4


@pytest.mark.parametrize("out_dtype", DTYPES)
@pytest.mark.parametrize("E,K", [(42, 4), (256, 2), (40, 3), (64, 1), (7, 5), (132, 6), (20, 8), (2048, 4)])
def test_input_convolution_in_portions_and_single_tokens(ops32, out_dtype, E, K):
    """Three requests whose inputs come in portions of changing size (down to one token, portions longer than a block's run of
    tokens) and as single tokens through the streams' kernel, the state carried between them; a state row that another request
    has used and that was cleared."""
    from hf_cpu_amd.parts.inputs import InputConv
    rng = np.random.default_rng(E + K)
    lengths, slots = [70, 9, 31], [1, 3, 0]
    cuts = [[1, 2, 33, 1, 1, 32], [2, 1, 1, 3, 1, 1], [16, 1, 1, 1, 11, 1]]
    h = [rng.standard_normal((n, E)).astype(np.float32) for n in lengths]
    w = helpers.bf16_round(rng.standard_normal((E, K)) * 0.5)
    part = InputConv(E, K)
    part.bind({part.name: dev(w)}, ops32)
    # rows whose norm is what we want: weights divide the root mean square out again
    cache = types.SimpleNamespace(state=torch.zeros((5, max(1, (K - 1) * E)), dtype=torch.float32, device="cuda"))
    ones, one = dev(np.ones(E)), dev(np.ones(1))
    ref = []
    for s in range(3):
        n = pf.rms_norm(h[s].astype(np.float64), 1.0, 1e-6)
        ref.append(pf.input_conv(n, w.astype(np.float64)))
    tol = 2e-5 if out_dtype == torch.float32 else 1e-2
    for again in range(2):
        at = [0, 0, 0]
        for turn in range(6):
            take = [h[s][at[s]:at[s] + cuts[s][turn]] for s in range(3)]
            step = state_step([cuts[s][turn] for s in range(3)], slots)
            step.token_slot = ints(np.repeat(slots, [len(t) for t in take]))
            x = dev(np.concatenate(take))[:, None, :].contiguous()
            out = torch.empty((step.n_tokens, E), dtype=out_dtype, device="cuda")
            if step.max_q_len == 1:
                ops32.stream_input(x, one, ones, 1e-6, out, **part.single_token(step, cache))
            else:
                n = torch.empty((step.n_tokens, E), dtype=torch.float32, device="cuda")
                ops32.stream_input(x, one, ones, 1e-6, n)
                part.forward(ops32, step, n, cache, out)
            got = out.float().cpu().numpy()
            r0 = 0
            for s in range(3):
                c = cuts[s][turn]
                want = ref[s][at[s]:at[s] + c]
                assert np.max(np.abs(got[r0:r0 + c] - want) / (np.abs(want) + 1.0)) <= tol, (again, turn, s)
                at[s], r0 = at[s] + c, r0 + c
        assert at == lengths
        cache.state[torch.tensor(slots, device="cuda")] = 0.0       # as at admission: the second pass must find nothing of the first
    assert K == 1 or float(cache.state.abs().max()) == 0.0


def shaped_case(rng, H, G, D, Dv, page, cap, window, lengths, q_lens, dtype, dist=True, sink=False):
    """Requests whose queries are the last positions; keys just inside and just outside the window, at a page's last place and the
    query's own stand out for some queries. Returns (q, cache, step, args of paged_attention, the float64 result)."""
    ks, vs, cache, table = paged_rows(rng, lengths, G * D, G * Dv, page, dtype)
    scale = 1.5 / math.sqrt(D)
    r1, r2 = rng.uniform(0.2, 1.5, H).astype(np.float32), rng.uniform(0.01, 1.2, H).astype(np.float32)
    sinks = (rng.standard_normal(H) * 1.5).astype(np.float32)
    grp = np.arange(H) // (H // G)
    qs, wants, positions, slots = [], [], [], []
    for s, (n, ql) in enumerate(zip(lengths, q_lens)):
        q = rng.standard_normal((ql, H, D)).astype(np.float32)
        k, v = rounded(ks[s], dtype).reshape(n, G, D), rounded(vs[s], dtype).reshape(n, G, Dv)
        for i in range(ql):
            p = n - ql + i
            far = [p - window + 1, p - window, page - 1, p][i % 4] if window else [2, page - 1, p, 0][i % 4]
            if 0 <= far <= p:
                q[i] += 4.0 * ks[s][far].reshape(G, D)[grp] / math.sqrt(D)
        qr = rounded(q, dtype)
        want = np.zeros((ql, H, Dv))
        for i in range(ql):
            p = n - ql + i
            lo = max(0, p - window + 1) if window else 0
            sc = np.einsum("hd,jhd->hj", qr[i], k[lo:p + 1][:, grp]) * scale
            if cap:
                sc = pf.soft_cap(sc, cap)
            if dist:
                sc = sc - r1[:, None].astype(np.float64) * np.log(1.0 + r2[:, None].astype(np.float64) * (p - np.arange(lo, p + 1))[None])
            a = pf.softmax_weights(sc[:, None, :], np.ones((1, p + 1 - lo), bool), sinks.astype(np.float64) if sink else None)[:, 0]
            want[i] = np.einsum("hj,jhd->hd", a, v[lo:p + 1][:, grp])
        qs.append(q.reshape(ql, H * D))
        wants.append(want.reshape(ql, H * Dv))
        positions += list(range(n - ql, n))
        slots += [s] * ql
    step = FakeStep(ints(positions), ints(slots), table, None)
    args = dict(v_head_dim=Dv, softcap=cap)
    if dist:
        args["distance"] = (dev(r1), dev(r2))
    if sink:
        args.update(sink=True, sink_scores=dev(sinks))
    return dev(np.concatenate(qs), dtype), cache, step, scale, args, np.concatenate(wants)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,Dv,page,cap,window,lengths,q_lens", [
    (4, 2, 10, 7, 8, 4.0, 11, [1, 5, 64, 130], [1, 3, 20, 1]),                     # sizes for the plain kernel
    (6, 6, 16, 16, 4, 0.0, 0, [30, 77], [30, 9]),
    (8, 2, 64, 64, 16, 15.0, 61, [1, 40, 203, 320], [1, 3, 17, 1]),                # a portion: four waves a tile
    (8, 2, 64, 64, 16, 15.0, 61, [700, 1500, 62, 61, 60], [1, 1, 1, 1, 1]),        # single tokens, lengths at the window's edge
    (16, 4, 128, 128, 16, 50.0, 1000, [3000, 999, 1001, 1], [1, 1, 1, 1]),         # keys cut into chunks inside a window
    (16, 4, 128, 128, 16, 50.0, 300, [1500, 40], [200, 40]),
    (4, 1, 32, 32, 8, 10.0, 600, [1500], [64]),                                    # few blocks of a portion: each cut into chunks
    (4, 1, 32, 32, 8, 10.0, 0, [1500], [64]),
    (2, 2, 96, 96, 32, 6.0, 32, [400, 33], [130, 33]),
    (4, 4, 64, 64, 64, 20.0, 100, [500], [300]),                                   # pages of 64 tokens
    (3, 1, 32, 32, 16, 0.0, 5, [50, 200], [50, 1]),                                # a distance term without a cap
    (8, 8, 64, 64, 16, 25.0, 1, [90, 17], [40, 1]),                                # a window of the token itself
])
def test_attention_with_capped_scores_and_a_distance_term(ops16, ops32, dtype, H, G, D, Dv, page, cap, window, lengths, q_lens):
    ops = ops16 if dtype == torch.bfloat16 else ops32
    for dist, sink in ((True, False), (True, True), (False, True)):
        rng = np.random.default_rng(H + D + sum(lengths) + 2 * dist + sink)
        q, cache, step, scale, args, want = shaped_case(rng, H, G, D, Dv, page, cap, window, lengths, q_lens, dtype, dist, sink)
        for plain in (False, True):
            out = torch.empty((q.shape[0], H * Dv), dtype=dtype, device="cuda")
            ops.force_plain_attention = plain
            try:
                ops.paged_attention(q, H, G, D, cache, step, window, scale, out, **args)
            finally:
                ops.force_plain_attention = False
            err = np.max(np.abs(out.float().cpu().numpy() - want))
            assert err <= (3e-5 if dtype == torch.float32 else 0.03), f"dist {dist} sink {sink} plain {plain}: {err:.3e}"


@pytest.mark.parametrize("H,DK,C,page,window,lengths,q_lens", [
    (4, 112, 96, 16, 37, [1, 36, 37, 38, 130, 203], [1, 3, 37, 1, 64, 1]),
    (16, 576, 512, 16, 1000, [1700, 999, 1001], [1, 1, 1]),             # single tokens: the window's keys cut into chunks
    (16, 576, 512, 16, 100, [300, 77], [300, 77]),
    (2, 128, 64, 8, 9, [1100, 17, 2], [300, 17, 2]),
    (40, 96, 32, 4, 33, [150, 1], [9, 1]),                              # more heads than a tile has columns
    (12, 320, 256, 32, 640, [900], [33]),
    (1, 48, 32, 16, 1, [70, 200], [70, 1]),
    (6, 224, 160, 16, 80, [500, 81, 80], [1, 1, 1]),
    (5, 80, 64, 16, 0, [500, 81, 300], [1, 30, 2]),
    (3, 17, 11, 8, 6, [40, 20], [9, 1]),                                # sizes for the plain kernel
])
def test_many_heads_on_one_wide_key_value_head_with_a_window_and_sinks(ops16, H, DK, C, page, window, lengths, q_lens):
    rng = np.random.default_rng(H + DK + sum(lengths))
    q, cache, step, scale, args, want = shaped_case(rng, H, 1, DK, C, page, 0.0, window, lengths, q_lens, torch.bfloat16, dist=False, sink=True)
    for plain in (False, True):
        out = torch.empty((q.shape[0], H * C), dtype=torch.bfloat16, device="cuda")
        ops16.force_plain_attention = plain
        try:
            ops16.paged_attention(q, H, 1, DK, cache, step, window, scale, out, **args)
        finally:
            ops16.force_plain_attention = False
        err = np.max(np.abs(out.float().cpu().numpy() - want))
        assert err <= 0.03, f"plain {plain}: {err:.3e}"


def test_attention_refuses_what_does_not_go_together(ops16):
    from hf_cpu_amd.status import EngineError
    rng = np.random.default_rng(0)
    q, cache, step, scale, args, _ = shaped_case(rng, 4, 2, 32, 32, 16, 5.0, 7, [20], [1], torch.bfloat16)
    out = torch.empty((1, 128), dtype=torch.bfloat16, device="cuda")
    vec = dev(np.ones(4))
    for bad in (dict(distance=(vec, vec), weights="sigmoid"), dict(sink_scores=vec), dict(distance=(vec[:3], vec)), dict(distance=(vec, vec), slopes=vec)):
        with pytest.raises(EngineError):
            ops16.paged_attention(q, 4, 2, 32, cache, step, 7, scale, out, **bad)


@pytest.mark.parametrize("reader", [False, True])
@pytest.mark.parametrize("H,G,D,cap,window,lengths", [(8, 2, 64, 15.0, 61, [700, 62, 5, 1]), (16, 4, 128, 50.0, 500, [1300, 501]), (4, 4, 32, 8.0, 0, [900])])
def test_decoded_tokens_in_one_kernel_with_shaped_scores(ops16, reader, H, G, D, cap, window, lengths):
    """Product, store of the new key and value and attention of single tokens as a decode step chains them (one kernel behind the
    product; a layer that reads another's keys stores nothing) against the separate kernels and float64."""
    rng = np.random.default_rng(H + D + reader)
    E, B = 256, len(lengths)
    _, cache, step, scale, args, _ = shaped_case(rng, H, G, D, D, 16, cap, window, lengths, [1] * B, torch.bfloat16)
    slot_map = ints([int(step.group(0).block_table[s, (n - 1) // 16]) * 16 + (n - 1) % 16 for s, n in enumerate(lengths)])
    step._g.slot_map = slot_map
    h = dev(rng.standard_normal((B, E)), torch.bfloat16)
    width = H * D + (0 if reader else 2 * G * D)
    w = dev(rng.standard_normal((width, E)) / math.sqrt(E) * 1.3, torch.bfloat16)
    k0, v0 = cache.k.clone(), cache.v.clone()
    res = []
    args.pop("v_head_dim")
    for fused in (True, False):
        cache.k.copy_(k0), cache.v.copy_(v0)
        ops16.fuse_rows = fused
        try:
            qkv = torch.empty((B, width), dtype=torch.bfloat16, device="cuda")
            ops16.gemm(h, w, qkv, defer=True)
            ops16.rope_store(qkv, step.positions, None, 0, H, 0 if reader else G, D, cache, None if reader else slot_map)
            assert (ops16._lazy_rope is not None) == fused
            out = torch.empty((B, H * D), dtype=torch.bfloat16, device="cuda")
            ops16.paged_attention(qkv, H, G, D, cache, step, window, scale, out, **args)
        finally:
            ops16.fuse_rows = True
        res.append((out.float().cpu().numpy(), cache.k.clone(), cache.v.clone()))
    assert np.max(np.abs(res[0][0] - res[1][0])) <= 0.03
    assert (res[0][1].float() - res[1][1].float()).abs().max() <= 0.05 and (res[0][2].float() - res[1][2].float()).abs().max() <= 0.05
    if reader:
        assert torch.equal(res[0][1], k0) and torch.equal(res[0][2], v0)
    proj = h.double().cpu().numpy() @ w.double().cpu().numpy().T
    kc, vc = res[0][1].double().cpu().numpy(), from_value_layout(res[0][2].float().cpu().numpy(), 16).astype(np.float64)
    table, (r1, r2), grp = step.group(0).block_table.cpu().numpy(), args["distance"], np.arange(H) // (H // G)
    r1, r2 = r1.double().cpu().numpy(), r2.double().cpu().numpy()
    for s, n in enumerate(lengths):
        j = np.arange(max(0, n - window) if window else 0, n)
        rows = table[s, j // 16] * 16 + j % 16
        sc = np.einsum("hd,jhd->hj", proj[s, :H * D].reshape(H, D), kc[rows].reshape(-1, G, D)[:, grp]) * scale
        sc = pf.soft_cap(sc, cap) - r1[:, None] * np.log(1.0 + r2[:, None] * (n - 1 - j)[None])
        a = pf.softmax_weights(sc[:, None], np.ones((1, len(j)), bool))[:, 0]
        want = np.einsum("hj,jhd->hd", a, vc[rows].reshape(-1, G, D)[:, grp]).reshape(-1)
        assert np.max(np.abs(res[0][0][s] - want)) <= 0.04, f"request {s}"


@pytest.mark.parametrize("a_dtype", DTYPES)
@pytest.mark.parametrize("T,H,N,K,pad", [(1, 4, 96, 64, 0), (5, 1, 32, 16, 8), (33, 6, 160, 32, 24), (64, 16, 512, 128, 64), (7, 3, 64, 512, 0)])
def test_products_of_heads_for_few_rows(ops16, a_dtype, T, H, N, K, pad):
    """``head_rows`` alone (rows with something between the heads, results beside something that must stay, with and without a
    gate), against float64 and against the grouped product for many rows."""
    rng = np.random.default_rng(T + N + K)
    a_head, o_head = K + pad, N + pad
    a = dev(rng.standard_normal((T, H * a_head + 16)), a_dtype)[:, :H * a_head]
    w = dev(rng.standard_normal((H, N, K)) / math.sqrt(K), torch.bfloat16)
    gate = dev(rng.standard_normal((T, H * N + 4)) * 2.0)[:, :H * N]
    ar = rounded(a.float().cpu().numpy(), torch.bfloat16).reshape(T, H, a_head)[..., :K]
    want = np.einsum("thk,hnk->thn", ar, w.double().cpu().numpy())
    for g in (None, gate):
        out = torch.full((T, H * o_head), 7.0, dtype=torch.bfloat16, device="cuda")
        ops16.head_rows(a, w, out, a_head, o_head, gate=g)
        got = out.float().cpu().numpy().reshape(T, H, o_head)
        ref = want if g is None else want * pf.sigmoid(gate.double().cpu().numpy().reshape(T, H, N))
        assert np.max(np.abs(got[..., :N] - ref) / (np.abs(ref) + 1.0)) <= 1e-2
        assert np.all(got[..., N:] == 7.0)
    if a_dtype == torch.bfloat16:
        own = a.contiguous()
        out = torch.full((T, H * o_head), 7.0, dtype=torch.bfloat16, device="cuda")
        ops16.head_products(own.view(T * H, a_head), w, out.view(T * H, o_head), H)
        got = out.float().cpu().numpy().reshape(T, H, o_head)
        assert np.max(np.abs(got[..., :N] - want) / (np.abs(want) + 1.0)) <= 1e-2 and np.all(got[..., N:] == 7.0)


@pytest.mark.parametrize("T,H,N,K,lda", [(300, 3, 64, 32, 36), (5, 3, 64, 32, 36), (70, 5, 7, 9, 11), (700, 2, 96, 64, 64)])
def test_grouped_products_of_heads_whose_rows_start_anywhere(ops16, T, H, N, K, lda):
    rng = np.random.default_rng(T + N)
    a, w = dev(rng.standard_normal((T * H, lda)), torch.bfloat16), dev(rng.standard_normal((H, N, K)) / math.sqrt(K), torch.bfloat16)
    out = torch.full((T * H, N + 5), 7.0, dtype=torch.bfloat16, device="cuda")
    ops16.head_products(a, w, out[:, 3:3 + N], H)
    got = out.float().cpu().numpy().reshape(T, H, N + 5)
    want = np.einsum("thk,hnk->thn", a.double().cpu().numpy().reshape(T, H, lda)[..., :K], w.double().cpu().numpy())
    assert np.max(np.abs(got[..., 3:3 + N] - want) / (np.abs(want) + 1.0)) <= 1e-2
    assert np.all(got[..., :3] == 7.0) and np.all(got[..., 3 + N:] == 7.0)


@pytest.mark.parametrize("q_dtype", DTYPES)
@pytest.mark.parametrize("T,H,D,R,C", [(3, 4, 64, 16, 96), (40, 2, 32, 8, 32), (1, 16, 128, 64, 512)])
def test_fold_and_store_of_latents_in_one_launch(ops16, q_dtype, T, H, D, R, C):
    """The few rows of a decode step: the same cache rows and queries as the store and the heads' products one after the other."""
    from hf_cpu_amd.cache.storage import PagedView
    rng = np.random.default_rng(T + D)
    HD, P = R + C, 16
    q = dev(rng.standard_normal((T, H * (D + R))), q_dtype)
    down = dev(rng.standard_normal((T, C + R)) * 2.0)
    w, fold = dev(1.0 + 0.2 * rng.standard_normal(C)), dev(rng.standard_normal((H, C, D)) / math.sqrt(D), torch.bfloat16)
    inv, positions, slots = dev(100.0 ** (-2.0 * np.arange(R // 2) / R)), ints(rng.integers(0, 2000, T)), ints(rng.permutation(64)[:T])
    res = []
    for one in (True, False):
        cache = PagedView(0, torch.zeros((64, HD), dtype=torch.bfloat16, device="cuda"), torch.zeros((64, C), dtype=torch.bfloat16, device="cuda"), P, 0)
        out = torch.zeros((T, H * HD), dtype=torch.bfloat16, device="cuda")
        ops16.latent_store(down, q, w, 1e-6, positions, inv, R, "interleaved", out, cache, slots, H, D, R, C, fold=fold if one else None)
        if not one:
            ops16.head_rows(q, fold, out[:, R:], D + R, HD)
        res.append((out, cache.k, cache.v))
    for a, b in zip(*res):
        assert torch.equal(a, b)
    want = np.einsum("thd,hcd->thc", rounded(q.float().cpu().numpy(), torch.bfloat16).reshape(T, H, D + R)[..., :D], fold.double().cpu().numpy())
    got = res[0][0].float().cpu().numpy().reshape(T, H, HD)[..., R:]
    assert np.max(np.abs(got - want) / (np.abs(want) + 1.0)) <= 1e-2


@pytest.mark.parametrize("T,H,G,D,page", [(600, 4, 2, 64, 16), (513, 6, 3, 40, 8), (20, 4, 2, 32, 16)])
def test_store_of_keys_and_values_without_a_rotation(ops16, T, H, G, D, page):
    """Portions of a prompt long enough for the kernel of many tokens, and short ones: rows as they are, whole runs of a page and
    scattered rows."""
    from hf_cpu_amd.cache.storage import PagedView
    rng = np.random.default_rng(T)
    qkv = dev(rng.standard_normal((T, (H + 2 * G) * D)), torch.bfloat16)
    n_pages = -(-T // page) + 3
    perm = rng.permutation(n_pages)
    rows = np.concatenate([perm[b] * page + np.arange(page) for b in range(n_pages)])[3:3 + T]
    cache = PagedView(0, torch.zeros((n_pages * page, G * D), dtype=torch.bfloat16, device="cuda"),
                      torch.zeros((n_pages * page, G * D), dtype=torch.bfloat16, device="cuda"), page, 0)
    before = qkv.clone()
    ops16.rope_store(qkv, ints(np.arange(T)), None, 0, H, G, D, cache, ints(rows))
    assert torch.equal(qkv, before)
    idx = torch.from_numpy(rows).cuda()
    assert torch.equal(cache.k[idx], qkv[:, H * D:(H + G) * D])
    assert np.array_equal(from_value_layout(cache.v.float().cpu().numpy(), page)[rows], qkv[:, (H + G) * D:].float().cpu().numpy())


# ---- whole models ----------------------------------------------------------------------------------------------------

LENGTHS = [1, 2, 9, 57, 96, 131, 24, 3]


@pytest.fixture(scope="module", params=list(fh.CONFIGS))
def tiny(request, tmp_path_factory, gpu):
    name = request.param
    cfg = fh.CONFIGS[name]
    d = fh.make_model_dir(str(tmp_path_factory.mktemp(name)), cfg, seed=1, stored=fh.STORED[name])
    reqs = fh.random_requests(cfg, LENGTHS, seed=8)
    return name, cfg, d, reqs, fh.plain_logits(d, reqs)


def engine_for(d, dtype, name, max_tokens, max_seqs=4, **kw):
    import hf_cpu_amd
    P = fh.PAGE[name]
    return hf_cpu_amd.load_engine(d, dtype=dtype, page_tokens=P, max_tokens=-(-max_tokens // P) * P, max_seqs=max_seqs, **kw)


def tol_of(name, dtype):
    return TOL_OF.get((name, dtype), TOL[dtype])


def run_against_plain(name, d, want, dtype, steps, what, **kw):
    engine = engine_for(d, dtype, name, helpers.max_live_tokens(steps), **kw)
    got = helpers.run_trace_in_engine(engine, steps)
    worst = helpers.compare(got, want, tol_of(name, dtype), what)
    engine.manager.check()
    assert engine.manager.stats()["requests"] == 0
    return engine, got, worst


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_streams_after_every_layer(gpu, tiny, dtype):
    """The sum of the streams after each layer of one prompt, then of its last tokens decoded one by one."""
    name, cfg, d, reqs, _ = tiny
    toks = reqs["r6"]
    pcfg, w = pf.read_model(d)
    want = []
    pf.forward(pcfg, w, toks, want)
    engine = engine_for(d, dtype, name, 64, graphs=False)
    seen = []
    for l in engine.model.layers:
        def wrapped(ops, step, x, parts, caches, write_cache=True, inner=l.block.forward):
            inner(ops, step, x, parts, caches, write_cache)
            ops.settle()
            seen.append(x.sum(1).cpu().numpy())
        l.block.forward = wrapped
    at = 0
    for n in [19, 1, 1, 2, 1]:
        seen.clear()
        engine.step([("a", toks[at:at + n], [0])])
        for l, got in enumerate(seen):
            ref = want[l][at:at + n]
            err = np.max(np.abs(got - ref)) / np.max(np.abs(want[l]))
            assert err <= (2e-5 if dtype == "float32" else 4e-2), f"layer {l}, tokens from {at}: {err:.3e}"
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
        helpers.compare(got, want, tol_of(name, dtype), "trace_run " + dtype)


def test_greedy_generation_through_the_session(gpu, tiny):
    """Greedy continuation of three prompts through Session.generate (the scheduler, the sampler, graphs): every token
    is the plain implementation's best, or within rounding of it."""
    import hf_cpu_amd.session as S
    name, cfg, d, reqs, _ = tiny
    prompts = [reqs["r3"], reqs["r4"], reqs["r5"]]
    pcfg, w = pf.read_model(d)
    s = S.Session(d, dtype="float32", ctx_max=256, batch=16, page_size=fh.PAGE[name], max_seqs=4)
    gens = s.generate(prompts, temp=0.0, max_tokens=20)
    for g, p in zip(gens, prompts):
        assert len(g.tokens) == 20
        rows = pf.forward(pcfg, w, list(p) + g.tokens)
        for i, t in enumerate(g.tokens):
            row = rows[len(p) - 1 + i]
            assert row[int(np.argmax(row))] - row[t] <= 1e-4 * max(1.0, float(np.max(np.abs(row)))), \
                f"token {i} = {t}, plain picks {int(np.argmax(row))}"


def test_command_line_generates_and_forks(gpu, tiny):
    """bin/hfamd on a folder of this design: greedy tokens are the plain implementation's; two continuations of one prompt
    (the second forks the first's pages and state rows after the prompt) are the same; sampled runs with one seed repeat
    themselves."""
    import os
    import subprocess
    import sys
    name, cfg, d, reqs, _ = tiny
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    prompt = reqs["r3"]

    def run(extra):
        r = subprocess.run([sys.executable, os.path.join(root, "bin", "hfamd"), "--stdin-mode", "none", "--model", d, "--dtype", "float32",
                            "--ctx-max", "128", "--page-size", str(fh.PAGE[name]), "--max-seqs", "4", "--log-level", "error",
                            "--prompt-ids", " ".join(map(str, prompt))] + extra, text=True, capture_output=True, timeout=300)
        assert r.returncode == 0, r.stderr
        toks = {}
        for line in r.stdout.replace("\x1e", "\n").splitlines():
            if line.startswith("@token "):
                f = dict(x.split("=", 1) for x in line.split(" ")[1:] if "=" in x)
                toks.setdefault(f.get("seq", "0"), []).append(int(f["id"]))
        return toks
    greedy = run(["--temp", "0", "--max-tokens", "6"])["0"]
    pcfg, w = pf.read_model(d)
    rows = pf.forward(pcfg, w, prompt + greedy)
    for i, t in enumerate(greedy):
        row = rows[len(prompt) - 1 + i]
        assert row[int(np.argmax(row))] - row[t] <= 1e-4 * max(1.0, float(np.max(np.abs(row))))
    both = run(["--temp", "0", "--max-tokens", "5", "--n", "2"])
    assert both["0"] == greedy[:5] and both["1"] == greedy[:5]
    drawn = run(["--temp", "0.9", "--seed", "11", "--max-tokens", "8", "--n", "2"])
    assert drawn == run(["--temp", "0.9", "--seed", "11", "--max-tokens", "8", "--n", "2"]) and len(drawn["0"]) == 8 and len(drawn["1"]) == 8


def window_model(kind, window):
    """One layer that shows a single key. Token 1 alone has an entry in the table's column before the last, every token the same
    entry in the last column. Queries are a fixed vector times the last column's entry, token 1's key a large multiple of that
    vector: every query that sees token 1 gives it nearly all its weight. The convolution is silent, so a window of W tokens
    shows token 1 to the W queries from it on and to no other. ``reader``: the layer that looks reads another layer's keys, which
    alone would forget them earlier."""
    E = 64
    rng = np.random.default_rng(5)
    if kind == "latent":
        layers = [fh.layer(fh.latent(2, 16, 8, 32, 32, window, scale=1.0), None)]
    elif kind == "attention":
        layers = [fh.layer(fh.attention(2, 1, 32, 32, window, 40.0, scale=1.0), None)]
    else:
        layers = [fh.layer(fh.attention(2, 1, 32, 32, 3, 40.0, scale=1.0), None), fh.layer(fh.attention(2, 1, 32, 32, window, 40.0, scale=1.0, kv_from=0), None)]
    cfg = fh.config(50, E, layers, streams=2, taps=3)
    w = fh.make_weights(cfg, seed=1)
    for l, lc in enumerate(layers):
        p = f"l{l}.mix."
        w[f"l{l}.canon1"][:], w[f"l{l}.norm1"][:] = 0.0, 0.0
        w[f"l{l}.hc1.in"][:], w[f"l{l}.hc1.mix"][:], w[f"l{l}.hc1.out"][:] = [1.0, 0.0], [[1.0, 0.0], [0.0, 1.0]], [0.0, 1.0]
        w[p + "q"][:] = 0.0
        if lc["type"] == "latent_attention":
            w[p + "dkv"][0] = 0.0
            w[p + "dkv"][0, E - 2] = 6.0
            w[p + "dkv"][32:] = 0.0                          # nothing in the rotated part
            w[p + "dkv.norm"][:] = 1.0
            w[p + "uk"][:, 0] = helpers.bf16_round(np.abs(rng.standard_normal(32)) + 1.0)
            w[p + "uv"][:, 0] = helpers.bf16_round(rng.standard_normal(64) * 2.0)
            for hd in range(2):
                w[p + "q"][hd * 24:hd * 24 + 16, E - 1] = helpers.bf16_round(np.abs(rng.standard_normal(16)) * 0.2)
            w[p + "sink"][:] = 0.5
        else:
            u = helpers.bf16_round(rng.standard_normal(32))
            w[p + "q"][:32, E - 1], w[p + "q"][32:, E - 1] = u, u
            if p + "k" in w:
                w[p + "k"][:, E - 2] = 3.0 * u
                w[p + "v"][:, E - 2] = helpers.bf16_round(rng.standard_normal(32) * 2.0)
            w[p + "r1"][:], w[p + "r2"][:] = 0.25, 0.125
    w["embed"][:, E - 2:] = 0.0
    w["embed"][:, E - 1] = 1.0
    w["embed"][1, E - 2] = 4.0
    return cfg, w


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind,window", [("latent", 20), ("latent", 129), ("latent", 700), ("attention", 33), ("attention", 600), ("reader", 48)])
def test_a_key_just_inside_and_just_outside_the_window(gpu, tmp_path, dtype, kind, window):
    """The marked token at a page's first and last place and in between: the last query that sees it and the first that does not,
    inside a prompt's first portion, in a second portion, and among decoded tokens; far windows among hundreds of keys."""
    import hf_cpu_amd
    cfg, w = window_model(kind, window)
    d = fh.make_model_dir(str(tmp_path / "m"), cfg, seed=0, weights=w, stored="BF16")
    rng = np.random.default_rng(9)
    n = window + 240
    base = [int(t) for t in rng.integers(2, cfg["vocab"], n)]
    reqs = {f"at{at}": base[:at] + [1] + base[at + 1:] for at in (2, 15, 16, 97, 150, 215)}
    reqs["none"] = base
    want = fh.plain_logits(d, reqs)
    size = float(np.max(np.abs(want["none"])))
    steps = []
    for r, t in reqs.items():
        if r != "none":
            at = int(r[2:])
            last = at + window - 1
            assert np.max(np.abs(want[r][last] - want["none"][last])) >= 0.1 * size, "the plain logits do not show the key"
            assert np.max(np.abs(want[r][last + 1] - want["none"][last + 1])) <= 1e-9 * size
        cut, head = window + 60, window + 130
        steps.append(helpers._step(len(steps), [(r, t[:cut], range(cut))]))
        steps.append(helpers._step(len(steps), [(r, t[cut:head], range(head - cut))]))
        for i in range(head, n):
            steps.append(helpers._step(len(steps), [(r, t[i:i + 1], [0])], [r] if i == n - 1 else []))
    engine = hf_cpu_amd.load_engine(d, dtype=dtype, page_tokens=16, max_tokens=helpers.max_live_tokens(steps), max_seqs=1)
    got = helpers.run_trace_in_engine(engine, steps)
    helpers.compare(got, want, TOL[dtype], f"window {kind} {window} {dtype}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_long_prompt_decoded_token_by_token(gpu, tmp_path, dtype):
    """Two requests of 700 and 1,300 tokens: the prompt in two portions (the second begins in the middle of a page),
    then 45 tokens decoded together; windows of hundreds of tokens whose keys a decoded token cuts over many waves."""
    import hf_cpu_amd
    cfg = fh.config(300, 128, streams=3, taps=4, layers=[
        fh.layer(fh.latent(4, 32, 16, 32, 64, 500), 128),
        fh.layer(fh.attention(4, 2, 32, 32, 700, 20.0), None),
        fh.layer(fh.attention(4, 2, 32, 32, 100, 12.0, kv_from=1), 96)])
    d = fh.make_model_dir(str(tmp_path / "m"), cfg, seed=4, stored="BF16")
    reqs = fh.random_requests(cfg, [700, 1300], seed=2)
    want = fh.plain_logits(d, reqs)
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
    cfg = fh.config(120, 64, streams=2, taps=3, layers=[fh.layer(fh.latent(4, 16, 16, 32, 64, 25), 64), fh.layer(fh.attention(2, 2, 32, 32, 30, 9.0), None)])
    d = fh.make_model_dir(str(tmp_path / "m"), cfg, seed=2, stored="BF16")
    reqs = fh.random_requests(cfg, [40, 1300], seed=5)
    want = fh.plain_logits(d, reqs)
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


def test_a_checkpoint_may_hold_the_tensors_of_a_sublayer_that_a_layer_lacks(gpu, tmp_path):
    import hf_cpu_amd
    cfg = fh.config(60, 32, streams=2, taps=2, layers=[fh.layer(fh.latent(2, 8, 4, 8, 16, 6), None)])
    w = fh.make_weights(cfg, 0)
    toks = [3, 9, 27, 50, 1, 4, 5, 6, 7, 8]
    rows = []
    for extra in (False, True):
        if extra:
            w.update({"l0.norm2": np.ones(32), "l0.canon2": np.ones((32, 2)), "l0.hc2.in": np.ones(2), "l0.hc2.out": np.ones(2), "l0.hc2.mix": np.ones((2, 2))})
        d = fh.make_model_dir(str(tmp_path / f"m{extra}"), cfg, 0, weights=w, stored="BF16")
        engine = hf_cpu_amd.load_engine(d, dtype="float32", page_tokens=4, max_tokens=64, max_seqs=1)
        rows.append(engine.step([("a", toks, list(range(10)))]).cpu().numpy())
    assert np.array_equal(rows[0], rows[1])


def test_random_weights_and_other_orders_of_layers(gpu, tmp_path):
    """``write_random_model`` makes a folder for this design too, and the engine reads it back: models of one kind of layer only,
    and one with widths that are no multiple of 8."""
    import hf_cpu_amd
    from hf_cpu_amd.config import config_from_dict
    one = fh.config(90, 64, streams=1, taps=2, layers=[fh.layer(fh.latent(2, 16, 8, 32, 32, 12), 16)])
    two = fh.config(90, 64, streams=2, taps=1, layers=[fh.layer(fh.attention(2, 1, 32, 32, 9, 7.0), None), fh.layer(fh.attention(2, 1, 32, 32, 30, 7.0, kv_from=0), 24)])
    odd = fh.config(77, 100, eps=1e-3, streams=5, taps=5, layers=[
        fh.layer(fh.attention(3, 1, 20, 28, 8, 5.0), 12), fh.layer(fh.latent(5, 4, 2, 3, 9, 6), None), fh.layer(fh.attention(3, 1, 20, 28, 15, 5.0, kv_from=0), 20)])
    for k, c in enumerate((one, two, odd)):
        d = str(tmp_path / f"m{k}")
        hf_cpu_amd.write_random_model(d, config_from_dict(c), seed=3, dtype="bfloat16")
        pcfg, w = pf.read_model(d)
        toks = [int(t) for t in np.random.default_rng(0).integers(0, c["vocab"], 45)]
        want = pf.forward(pcfg, w, toks)
        for dtype in ("float32", "bfloat16"):
            engine = hf_cpu_amd.load_engine(d, dtype=dtype, page_tokens=4, max_tokens=64, max_seqs=1)
            got = engine.step([("a", toks[:31], list(range(31)))]).cpu().numpy()
            rows = {("a", i): row for i, row in enumerate(got)}
            for i in range(31, 45):
                rows[("a", i)] = engine.step([("a", toks[i:i + 1], [0])]).cpu().numpy()[0]
            helpers.compare(rows, {"a": want}, TOL[dtype], f"random weights {k} {dtype}")


@pytest.mark.parametrize("seed", range(8))
def test_configurations_drawn_at_random(gpu, tmp_path, seed):
    """Layers of either kind in any order with sizes drawn at random (even seeds: sizes for the matrix cores): a prompt, a
    portion that starts in the middle of a page, then single tokens, in fp32 and in bf16."""
    import hf_cpu_amd
    rng = np.random.default_rng(100 + seed)
    cfg = fh.random_config(rng, big=seed % 2 == 0)
    d = fh.make_model_dir(str(tmp_path / "m"), cfg, seed=seed, stored="BF16" if seed % 2 == 0 else "F32")
    toks = [int(t) for t in rng.integers(0, cfg["vocab"], 110)]
    pcfg, w = pf.read_model(d)
    want = pf.forward(pcfg, w, toks)
    steps = [helpers._step(0, [("a", toks[:55], range(55))]), helpers._step(1, [("a", toks[55:88], range(33))])]
    steps += [helpers._step(2 + i, [("a", toks[88 + i:89 + i], [0])], ["a"] if i == 21 else []) for i in range(22)]
    for dtype in ("float32", "bfloat16"):
        engine = hf_cpu_amd.load_engine(d, dtype=dtype, page_tokens=16, max_tokens=128, max_seqs=2, graphs=dtype == "float32")
        got = helpers.run_trace_in_engine(engine, steps)
        helpers.compare(got, {"a": want}, TOL[dtype] if dtype == "float32" else 8e-2, f"random configuration {seed} {dtype}: {cfg}")
