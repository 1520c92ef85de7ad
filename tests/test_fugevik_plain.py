"""The plain implementation of Fugevik against second derivations, and the package's reader and plan for it (no GPU)."""
import copy
import math

import numpy as np
import pytest

import fugevik_helpers as fh
import plain_fugevik as pf


def small_weights(cfg, seed=0):
    return {k: np.asarray(v, np.float64) for k, v in fh.make_weights(cfg, seed).items()}


# ---- the plain implementation ------------------------------------------------------------------------------------------

def test_convolution_against_the_sum_at_each_token():
    rng = np.random.default_rng(0)
    h, w = rng.standard_normal((9, 5)), rng.standard_normal((5, 4))
    got = pf.input_conv(h, w)
    for t in range(9):
        want = h[t].copy()
        for j in range(4):
            if t - 3 + j >= 0:
                want += w[:, j] * h[t - 3 + j]
        assert np.allclose(got[t], want)
    assert np.allclose(pf.input_conv(h, w[:, :1]), h * (1.0 + w[:, 0]))          # one tap: the token itself


def test_streams_are_mixed_from_the_old_ones_in_the_direction_from_to():
    rng = np.random.default_rng(1)
    x, y = rng.standard_normal((4, 3, 6)), rng.standard_normal((4, 6))
    mix, out = rng.standard_normal((3, 3)), rng.standard_normal(3)
    got = pf.stream_update(x, y, mix, out)
    for b in range(3):
        assert np.allclose(got[:, b], mix[0, b] * x[:, 0] + mix[1, b] * x[:, 1] + mix[2, b] * x[:, 2] + out[b] * y)
    only = np.zeros((3, 3))
    only[0, 2] = 1.0                                                             # from stream 0 to stream 2
    assert np.allclose(pf.stream_update(x, y, only, np.zeros(3))[:, 2], x[:, 0])
    assert np.allclose(pf.stream_input(x, np.array([0.0, 2.0, 0.0])), 2.0 * x[:, 1])


def test_one_stream_with_unit_weights_is_the_plain_residual_sum():
    rng = np.random.default_rng(2)
    x, y = rng.standard_normal((5, 1, 7)), rng.standard_normal((5, 7))
    assert np.allclose(pf.stream_update(x, y, np.ones((1, 1)), np.ones(1))[:, 0], x[:, 0] + y)


def test_rotation_turns_neighbours_and_depends_on_distance_alone():
    rng = np.random.default_rng(3)
    x = rng.standard_normal((1, 8))
    turned = pf.rotate_pairs(x, [5], 6, 100.0)[0]
    for i in range(3):
        a = 5 * 100.0 ** (-2 * i / 6)
        assert np.allclose(turned[2 * i] + 1j * turned[2 * i + 1], (x[0, 2 * i] + 1j * x[0, 2 * i + 1]) * np.exp(1j * a))
    assert np.allclose(turned[6:], x[0, 6:])
    q, k = rng.standard_normal((1, 8)), rng.standard_normal((1, 8))

    def score(i, j):
        return float((pf.rotate_pairs(q, [i], 8, 50.0) * pf.rotate_pairs(k, [j], 8, 50.0)).sum())
    assert math.isclose(score(40, 33), score(1007, 1000), rel_tol=1e-9)


def test_window_sees_itself_and_the_tokens_before_it():
    m = pf.window_mask(6, 3)
    assert [int(np.argmax(r)) for r in m] == [0, 0, 0, 1, 2, 3] and [int(r.sum()) for r in m] == [1, 2, 3, 3, 3, 3]
    assert np.array_equal(pf.window_mask(4, 1), np.eye(4, dtype=bool))
    assert np.array_equal(pf.window_mask(4, 0), np.tril(np.ones((4, 4), bool)))


def test_sink_takes_weight_without_a_value():
    rng = np.random.default_rng(4)
    s = rng.standard_normal((2, 5, 5)) * 3.0
    mask = pf.window_mask(5, 3)
    sink = np.array([0.7, -40.0])
    a = pf.softmax_weights(s, mask, sink)
    b = pf.softmax_weights(s, mask)
    for h in range(2):
        for i in range(5):
            seen = np.exp(s[h, i][mask[i]])
            assert np.allclose(a[h, i][mask[i]], seen / (seen.sum() + math.exp(sink[h])))
    assert np.all(a[0].sum(-1) < 1.0) and np.allclose(a[1], b[1]) and np.all(a[:, ~mask] == 0.0)
    big = pf.softmax_weights(s, mask, np.array([800.0, 800.0]))                  # a sink far above every score: nothing is left
    assert np.all(np.isfinite(big)) and np.max(big) < 1e-200


def test_capped_scores_are_lowered_by_the_distance_after_the_cap():
    r1, r2 = np.array([0.5, 2.0]), np.array([1.0, 0.25])
    d = pf.distance_penalty(4, r1, r2)
    assert np.allclose(d[:, 3, 3], 0.0) and math.isclose(d[0, 3, 0], 0.5 * math.log(4.0)) and math.isclose(d[1, 3, 1], 2.0 * math.log(1.5))
    assert np.allclose(pf.soft_cap(np.array([0.0, 1e-6, 1e9, -1e9]), 30.0), [0.0, 1e-6, 30.0, -30.0])
    # with scores far beyond the cap all keys score the cap, and only the distance orders them: weights ~ (1 + r2 d)^(-r1)
    cfg = fh.config(20, 6, [fh.layer(fh.attention(1, 1, 2, 2, 50, 5.0), None)], streams=1, taps=1)
    w = small_weights(cfg)
    p = "l0.mix."
    h = np.ones((7, 6))
    w[p + "q"][:], w[p + "k"][:] = 100.0, 100.0
    w[p + "r1"], w[p + "r2"] = np.array([0.8]), np.array([0.6])
    v = h @ w[p + "v"].T + np.arange(7)[:, None]
    y, (k_own, v_own) = pf.attention(h, w, p, cfg["layers"][0]["mixer"], {})
    assert np.allclose(v_own[:, 0], h @ w[p + "v"].T)
    dist = np.arange(6, -1, -1)
    wt = (1.0 + 0.6 * dist) ** -0.8
    assert np.allclose(y[6], (wt / wt.sum()) @ (v - np.arange(7)[:, None]) @ w[p + "o"].T)


def test_a_layer_reads_the_keys_and_values_of_its_source():
    cfg = fh.SMALL
    w = small_weights(cfg)
    h = np.random.default_rng(5).standard_normal((9, 42))
    m0, m2 = cfg["layers"][0]["mixer"], dict(cfg["layers"][2]["mixer"])
    _, own = pf.attention(h, w, "l0.mix.", m0, {})
    y, none = pf.attention(2.0 * h, w, "l2.mix.", m2, {0: own})
    assert none is None
    w2 = dict(w)
    w2["l2.mix.k"], w2["l2.mix.v"] = 0.5 * w["l0.mix.k"], 0.5 * w["l0.mix.v"]   # projections that give the source's from twice the input
    m2.pop("kv_from")
    assert np.allclose(y, pf.attention(2.0 * h, w2, "l2.mix.", m2, {})[0])


def test_latent_attention_against_the_form_that_keeps_latents_only():
    rng = np.random.default_rng(6)
    cfg = fh.config(20, 16, [fh.layer(fh.latent(3, 4, 6, 5, 7, 4, base=30.0), None)], streams=1, taps=1)
    w = small_weights(cfg)
    p, m = "l0.mix.", cfg["layers"][0]["mixer"]
    T, H, D, R, P, C = 11, 3, 4, 6, 5, 7
    h, pos = rng.standard_normal((T, 16)), np.arange(T) + 3
    got = pf.latent_attention(h, w, p, m, 1e-6, pos)
    down = h @ w[p + "dkv"].T
    c = pf.rms_norm(down[:, :C], w[p + "dkv.norm"], 1e-6)
    k = np.concatenate([pf.rotate_pairs(down[:, C:], pos, R, 30.0), c], axis=1)
    q = (h @ w[p + "q"].T).reshape(T, H, D + R)
    q = np.concatenate([pf.rotate_pairs(q[..., D:], pos, R, 30.0), np.einsum("thd,hdc->thc", q[..., :D], w[p + "uk"].reshape(H, D, C))], axis=-1)
    out = np.zeros((T, H * P))
    for i in range(T):
        lo = max(0, i - 3)
        for hd in range(H):
            e = np.exp(k[lo:i + 1] @ q[i, hd] * m["scale"])
            mean = e @ c[lo:i + 1] / (e.sum() + math.exp(w[p + "sink"][hd]))
            out[i, hd * P:(hd + 1) * P] = w[p + "uv"].reshape(H, P, C)[hd] @ mean
    assert np.allclose(got, (out * pf.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T)


def test_a_model_whose_sublayers_are_silenced_is_its_embedding_mixed():
    cfg = copy.deepcopy(fh.SMALL)
    w = small_weights(cfg, 3)
    for k in list(w):
        if k.endswith(".out"):
            w[k] = np.zeros_like(w[k])
        elif k.endswith(".mix"):
            w[k] = np.eye(3)
    toks = [5, 9, 136, 0, 77]
    want = pf.rms_norm(3.0 * w["embed"][toks], 1.0 + w["final.norm"], 1e-5) @ w["embed"].T
    assert np.allclose(pf.forward(cfg, w, toks), want)


def test_a_position_does_not_depend_on_what_follows_and_far_tokens_leave_the_windows():
    cfg = fh.SMALL
    w = small_weights(cfg, 1)
    toks = [int(t) for t in np.random.default_rng(7).integers(0, cfg["vocab"], 14)]
    whole = pf.forward(cfg, w, toks)
    assert np.allclose(pf.forward(cfg, w, toks[:9]), whole[:9])
    # one layer with a window of 5 behind convolutions over 3 tokens: a token 5 + 2 places back still shows, one 7 places back does not
    one = fh.config(30, 20, [fh.layer(fh.attention(2, 1, 4, 4, 5, 3.0), None)], streams=2, taps=3)
    w1 = small_weights(one)
    base = [1, 2, 3, 4, 5, 6, 7, 8, 9, 10]
    last = pf.forward(one, w1, base)[-1]
    for at, shows in ((3, True), (2, False)):
        other = list(base)
        other[at] = 25
        assert np.allclose(pf.forward(one, w1, other)[-1], last) != shows, at


# ---- the package's reader and plan ------------------------------------------------------------------------------------

@pytest.mark.parametrize("name", list(fh.CONFIGS))
def test_configuration_reads_every_size_and_constant(name):
    from hf_cpu_amd.config import config_from_dict
    cfg = fh.CONFIGS[name]
    c = config_from_dict(cfg)
    assert (c.architecture, c.vocab, c.width, c.streams, c.taps, c.norm_eps) == \
        ("Fugevik", cfg["vocab"], cfg["width"], cfg["streams"], cfg["canon"]["taps"], cfg["norm"]["eps"])
    for lc, raw in zip(c.layers, cfg["layers"]):
        m = raw["mixer"]
        assert lc.type == raw["type"] and lc.ff == (raw["mlp"] or {}).get("ff", 0)
        assert (lc.mixer.heads, lc.mixer.dim, lc.mixer.vdim, lc.mixer.scale, lc.mixer.window) == (m["heads"], m["dim"], m["vdim"], m["scale"], m["mask"]["size"])
        if lc.type == "latent_attention":
            assert (lc.mixer.rot_dim, lc.mixer.kv_rank, lc.mixer.rot_base, lc.mixer.rot_dims) == (m["rot_dim"], m["kv_rank"], m["rot"]["base"], m["rot"]["dims"])
        else:
            assert (lc.mixer.kv_heads, lc.mixer.softcap, lc.mixer.kv_from) == (m["kv_heads"], m["softcap"], m.get("kv_from"))
    assert c.to_dict() == cfg


@pytest.mark.parametrize("change,word", [
    (lambda c: c["layers"][0].update(type="conv"), "conv"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "kv_heads"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=3), "dims"),
    (lambda c: c["layers"][1]["mixer"].pop("kv_rank"), "kv_rank"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=4), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "kv_from"),
    (lambda c: c["layers"][5]["mixer"].update(kv_from=2), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(vdim=9), "other sizes"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "moe"),
    (lambda c: c["layers"][0]["mixer"].update(softcap=-1.0), "softcap"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c.pop("streams"), "streams"),
    (lambda c: c["canon"].update(taps=9), "taps"),
])
def test_configuration_errors_name_the_key(change, word):
    from hf_cpu_amd.config import config_from_dict
    from hf_cpu_amd.status import EngineError
    cfg = copy.deepcopy(fh.SMALL)
    change(cfg)
    with pytest.raises(EngineError) as e:
        config_from_dict(cfg)
    assert word in str(e.value.msg)


@pytest.mark.parametrize("name", list(fh.CONFIGS))
def test_plan_declares_the_tensors_of_a_checkpoint(name):
    from hf_cpu_amd.config import config_from_dict
    from hf_cpu_amd.model import Model
    cfg = fh.CONFIGS[name]
    model = Model.from_config(config_from_dict(cfg))
    declared = {s.name: s for s in model.param_specs()}
    made = fh.make_weights(cfg, 0)
    assert {n for n, s in declared.items() if not s.optional} == set(made)
    assert all(tuple(declared[n].shape) == np.shape(made[n]) for n in made)
    # a layer without a feed-forward may come with the second sublayer's small tensors, which nothing reads
    bare = [l for l, lc in enumerate(cfg["layers"]) if lc["mlp"] is None]
    assert all(f"l{l}.{n}" in declared for l in bare for n in ("norm2", "canon2", "hc2.in", "hc2.out", "hc2.mix"))
    assert model.graph_safe


def test_readers_share_keys_and_keep_their_own_convolution_inputs():
    from hf_cpu_amd.cache import CacheManager
    from hf_cpu_amd.config import config_from_dict
    from hf_cpu_amd.model import Model
    from hf_cpu_amd.parts.base import FixedState, PagedKV
    model = Model.from_config(config_from_dict(fh.SMALL))
    needs = model.cache_needs()
    slots = model.cache_slots
    assert [e.cache_of for e in model.schedule] == [None, None, 0, None, None, 0, 4]
    paged = [n for n in needs if isinstance(n, PagedKV)]
    assert [(n.k_width, n.v_width, n.window) for n in paged] == [(20, 14, 11), (14, 10, 5), (9, 7, 1), (35, 35, 40)]
    # layer 0's keys are kept as long as the widest of its readers' windows wants them
    assert set(paged[0].readers) == {(23, 0), (3, 0)} and paged[0].first_kept(100) == 100 - 23 + 1
    assert slots[2]["mixer"] == slots[0]["mixer"] == slots[5]["mixer"] and slots[6]["mixer"] == slots[4]["mixer"]
    # every sublayer of every layer has the inputs of its own convolution
    states = [s[k] for s in slots for k in s if k.startswith("input")]
    assert len(states) == len(set(states)) == 13 and all(isinstance(needs[k], FixedState) and needs[k].n_floats == 3 * 42 for k in states)
    ones = Model.from_config(config_from_dict(fh.ONES))
    assert not [n for n in ones.cache_needs() if isinstance(n, FixedState)]      # one tap keeps nothing
    m = CacheManager(needs, 8, 12, 2, 96)
    h = m.admit("a")
    for _ in range(9):
        m.reserve("a", 8)
        m.commit("a", 8)
    held = {(g.k_width, g.window): [b for b, p in enumerate(h.tables[g.index]) if p >= 0] for g in m.groups}
    assert held[(20, 11)] == [6, 7, 8] and held[(14, 5)] == [8] and held[(9, 1)] == [] and held[(35, 40)] == [4, 5, 6, 7, 8]
    m.check()
