"""Shared by the Fugevik tests: small configurations that differ in every size and option, weights that give activations of
order one, model folders, and the plain implementation's logits."""
import json
import math
import os

import numpy as np

import helpers
import plain_fugevik as pf


def latent(heads, dim, rot_dim, vdim, kv_rank, window, base=10000.0, scale=None):
    return dict(type="latent_attention", mixer=dict(
        heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, rot=dict(base=base, dims=rot_dim), mask=dict(size=window),
        scale=scale if scale is not None else 1.4 / math.sqrt(dim + rot_dim)))


def attention(heads, kv_heads, dim, vdim, window, softcap, scale=None, kv_from=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=window), softcap=softcap,
             scale=scale if scale is not None else 1.6 / math.sqrt(dim))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return dict(type="attention", mixer=m)


def layer(mixer, ff):
    return dict(mixer, mlp=None if ff is None else dict(kind="dense", ff=ff))


def config(vocab, width, layers, streams, taps, eps=1e-6):
    return dict(architecture="Fugevik", vocab=vocab, width=width, streams=streams, canon=dict(taps=taps), norm=dict(eps=eps), layers=layers)


# Sizes that no matrix-core kernel takes (a width that is no multiple of 4, heads of 5, 6, 7 and 9), value heads of a size of
# their own, windows of 1, 5, 11 and 40 tokens that divide no page, a layer without a feed-forward, a reader straight after its
# source and one further on whose window is wider than the source's, another query scale and cap for a reader.
SMALL = config(137, 42, streams=3, taps=4, eps=1e-5, layers=[
    layer(attention(6, 2, 10, 7, 11, 4.0), 26),
    layer(latent(3, 6, 4, 5, 10, 5, base=90.0), 31),
    layer(attention(6, 2, 10, 7, 23, 9.0, scale=0.25, kv_from=0), None),
    layer(latent(1, 9, 2, 12, 7, 1), 18),
    layer(attention(5, 5, 7, 7, 40, 2.5), 22),
    layer(attention(6, 2, 10, 7, 3, 6.0, scale=0.6, kv_from=0), 9),
    layer(attention(10, 5, 7, 7, 17, 3.5, kv_from=4), 14),
])
# Sizes that the matrix-core kernels take: heads of 32, 64, 96 and 128, latents of 32 to 160 values, windows of several pages and
# of less than one.
CORES = config(530, 256, streams=4, taps=2, layers=[
    layer(latent(4, 64, 16, 96, 96, 37, base=3000.0), 512),
    layer(attention(8, 2, 64, 64, 61, 15.0), 320),
    layer(attention(8, 2, 64, 64, 33, 25.0, kv_from=1), 256),
    layer(latent(6, 32, 64, 32, 160, 80), None),
    layer(attention(4, 4, 32, 32, 9, 8.0), 384),
    layer(latent(2, 128, 32, 64, 32, 18, base=500.0), 128),
])
# One stream, one tap, one head, one layer that reads another: what is 1 must not be taken for granted.
ONES = config(96, 64, streams=1, taps=1, eps=1e-4, layers=[
    layer(attention(1, 1, 32, 32, 14, 12.0), 40),
    layer(attention(1, 1, 32, 32, 14, 12.0, kv_from=0), 1),
    layer(latent(1, 16, 8, 32, 32, 20, base=20.0), 72),
])
CONFIGS = {"small": SMALL, "cores": CORES, "ones": ONES}
PAGE = {"small": 8, "cores": 16, "ones": 4}
STORED = {"small": "F32", "cores": "BF16", "ones": "BF16"}


def make_weights(cfg, seed):
    """name -> float32 array, every value a bfloat16 value (the engine in bf16 then holds what the plain implementation reads).
    Streams are read and mixed with weights of both signs that keep them of one order; distance terms lower a far key's score
    by one or two, so that it still weighs; sinks take from a tenth to most of a head's weight."""
    rng = np.random.default_rng(seed)
    E, V, S, K = cfg["width"], cfg["vocab"], cfg["streams"], cfg["canon"]["taps"]

    def n(shape, std, mean=0.0):
        return helpers.bf16_round(mean + rng.standard_normal(shape) * std)

    def u(shape, lo, hi):
        return helpers.bf16_round(rng.uniform(lo, hi, shape))
    w = {"embed": n((V, E), 1.0 / math.sqrt(E) * 3.0), "final.norm": n(E, 0.2)}
    for l, lc in enumerate(cfg["layers"]):
        p, m = f"l{l}.", lc["mixer"]
        for q in ("1",) + (("2",) if lc["mlp"] is not None else ()):
            w[p + "norm" + q] = n(E, 0.2)
            w[p + "canon" + q] = n((E, K), 0.35)
            w[p + f"hc{q}.in"], w[p + f"hc{q}.out"] = n(S, 0.6, 0.3), n(S, 0.4, 0.6)
            w[p + f"hc{q}.mix"] = helpers.bf16_round(0.7 * np.eye(S) + rng.standard_normal((S, S)) * 0.45 / math.sqrt(S))
        q, H = p + "mix.", m["heads"]
        if lc["type"] == "latent_attention":
            D, R, P, C = m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            w[q + "q"] = n((H * (D + R), E), 1.2 / math.sqrt(E))
            w[q + "dkv"], w[q + "dkv.norm"] = n((C + R, E), 1.0 / math.sqrt(E)), n(C, 0.2, 1.0)
            w[q + "uk"], w[q + "uv"] = n((H * D, C), 1.2 / math.sqrt(C)), n((H * P, C), 1.0 / math.sqrt(C))
            w[q + "sink"] = n(H, 1.2, 0.5)
            w[q + "g"] = n((H * P, E), 1.2 / math.sqrt(E))
            w[q + "o"] = n((E, H * P), 1.5 / math.sqrt(H * P))
        else:
            G, D, P = m["kv_heads"], m["dim"], m["vdim"]
            w[q + "q"] = n((H * D, E), 1.2 / math.sqrt(E))
            if m.get("kv_from") is None:
                w[q + "k"], w[q + "v"] = n((G * D, E), 1.2 / math.sqrt(E)), n((G * P, E), 1.0 / math.sqrt(E))
            w[q + "r1"], w[q + "r2"] = u(H, 0.1, 0.9), u(H, 0.05, 1.5)
            w[q + "o"] = n((E, H * P), 1.5 / math.sqrt(H * P))
        if lc["mlp"] is not None:
            F = lc["mlp"]["ff"]
            w[p + "mlp.up"], w[p + "mlp.down"] = n((F, E), 1.0 / math.sqrt(E)), n((E, F), 0.8 / math.sqrt(F))
    return w


def make_model_dir(path, cfg, seed, weights=None, stored="F32"):
    """``stored``: F32 (a bf16 engine then keeps the matrices in 32-bit and runs the kernels for mixed operands) or
    BF16 (the kernels of the serving path)."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    helpers.write_safetensors(os.path.join(path, "model.safetensors"), weights if weights is not None else make_weights(cfg, seed), stored)
    return path


def random_requests(cfg, lengths, seed):
    rng = np.random.default_rng(seed)
    return {f"r{i}": [int(t) for t in rng.integers(0, cfg["vocab"], n)] for i, n in enumerate(lengths)}


def plain_logits(model_dir, reqs):
    cfg, w = pf.read_model(model_dir)
    return {r: pf.forward(cfg, w, toks) for r, toks in reqs.items()}


def random_config(rng, big):
    """A configuration drawn at random: two to six layers of either kind in any order, readers among them, with sizes that the
    matrix-core kernels take (``big``) or that none of them takes."""
    def pick(*xs):
        return xs[int(rng.integers(0, len(xs)))]
    width = pick(128, 256, 384) if big else pick(22, 36, 50, 76)
    layers, own = [], []
    for l in range(int(rng.integers(2, 7))):
        window = pick(1, 2, 7, 15, 16, 17, 30, 50, 64, 200)
        if pick(True, False):
            mix = latent(pick(1, 2, 5), pick(32, 64, 80) if big else pick(3, 8, 11), pick(8, 32, 64) if big else pick(2, 4, 6, 10),
                         pick(32, 64, 128) if big else pick(4, 9, 16), pick(32, 64, 160) if big else pick(5, 12, 30), window, base=pick(100.0, 10000.0))
        else:
            cap = pick(2.0, 10.0, 30.0)
            src = pick(*own) if own and pick(True, False) else None
            if src is None:
                G = pick(1, 2, 3)
                D = pick(32, 64, 128) if big else pick(5, 10, 16, 24)
                mix = attention(G * pick(1, 2, 4), G, D, D if big else pick(D, 4, 14), window, cap)
                own.append(l)
            else:
                m = layers[src]["mixer"]
                mix = attention(m["heads"], m["kv_heads"], m["dim"], m["vdim"], window, cap, scale=m["scale"] * 0.7, kv_from=src)
        layers.append(layer(mix, pick(None, pick(32, 64, 96) if big else pick(4, 10, 23))))
    return config(int(rng.integers(50, 400)), width, layers, streams=pick(1, 2, 3, 4, 5, 9), taps=pick(1, 2, 3, 4, 6), eps=pick(1e-5, 1e-6))
