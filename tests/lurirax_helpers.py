"""Shared by the Lurirax tests: small configurations that differ in every size and option, weights that give
activations of order one, model folders, and the plain implementation's logits."""
import json
import math
import os

import numpy as np

import helpers
import plain_lurirax as pl


def rot(dims, base=10000.0, scaling=None):
    r = dict(base=base, dims=dims)
    if scaling is not None:
        r["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return r


def attention(heads, kv_heads, dim, vdim, window, rot_dims, base=10000.0, scaling=None, scale=None):
    return dict(type="attention", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=window), rot=rot(rot_dims, base, scaling),
                                             scale=scale if scale is not None else 1.5 / math.sqrt(dim)))


def left(heads, kv_heads, dim, vdim, chunk, bias_max, rows, scale=None):
    """``rows``: of the table of distance terms (only the tensor tells; kept here for the weights)."""
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=chunk), bias_max=bias_max, bias_rows=rows,
                scale=scale if scale is not None else 1.5 / math.sqrt(dim))


def right(heads, dim, vdim, rot_dims, base=1000.0, decay=None):
    return dict(heads=heads, dim=dim, vdim=vdim, rot=rot(rot_dims, base),
                decay=list(decay) if decay is not None else [1.0 - 0.4 * 0.35 ** h for h in range(heads)])


def parallel(lt, rt, left_scale=0.7, right_scale=1.2):
    return dict(type="parallel", mixer=dict(left=lt, right=rt, left_scale=left_scale, right_scale=right_scale))


def diff(heads, kv_heads, dim, vdim, window, keep_first, factor=0.4, scale=None):
    return dict(type="attention_2", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, diff=factor, mask=dict(size=window, keep_first=keep_first),
                                               scale=scale if scale is not None else 1.5 / math.sqrt(dim)))


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff, shared=None, scale=1.5):
    f = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top, scale=scale))
    if shared is not None:
        f["shared"] = dict(ff=shared)
    return f


def layer(mixer, mlp):
    return dict(mixer, mlp=mlp)


def config(vocab, width, layers, eps=1e-6, embedding_scale=None):
    return dict(architecture="Lurirax", vocab=vocab, width=width, norm=dict(eps=eps), layers=layers,
                embedding=dict(scale=embedding_scale if embedding_scale is not None else math.sqrt(width)))


# Sizes that no matrix-core kernel takes (an odd width, heads of 5, 7, 9, 10 and 12), value heads smaller and larger than the
# keys', a model that begins with differential attention, layers without a feed-forward, a window of one token and windows, chunks
# and kept first tokens on both sides of a page, more kept tokens than a window has, one head and several, as many key/value heads
# as heads and fewer, rotation of a part of a head and of all of it, frequencies rescaled and not, tables of distance terms that
# end inside a chunk and beyond it, one choice among the experts, several and all of them, with a shared expert and without.
SMALL = config(133, 44, eps=1e-5, embedding_scale=3.0, layers=[
    layer(diff(6, 3, 5, 7, 9, 3, 0.3), None),
    layer(attention(3, 1, 10, 6, 7, 6, base=500.0, scaling=(4.0, 1.0, 3.0, 64), scale=0.4), moe(5, 3, 12)),
    layer(parallel(left(4, 2, 6, 9, 11, 9, 8), right(3, 7, 5, 4)), dense(20)),
    layer(attention(2, 2, 12, 12, 1, 12), moe(4, 4, 32, shared=8, scale=0.6)),
    layer(parallel(left(1, 1, 8, 8, 33, 40, 10), right(1, 20, 4, 20, decay=[0.9]), -0.5, 1.0), None),
    layer(diff(2, 1, 9, 4, 13, 17, 0.7), moe(3, 1, 10, shared=6, scale=2.0)),
])
# Sizes that the matrix-core kernels take: heads of 32, 64 and 128 with value heads as large, half and twice as large, states of
# 32 x 64 and 64 x 128, experts of 64 and 96, dense layers of 512 and 320.
CORES = config(520, 256, layers=[
    layer(attention(8, 2, 64, 64, 37, 32, base=40000.0, scaling=(6.0, 1.0, 3.0, 128)), moe(8, 2, 64, shared=128, scale=1.0)),
    layer(parallel(left(8, 2, 64, 64, 29, 24, 16), right(4, 32, 64, 32)), dense(512)),
    layer(diff(4, 2, 32, 64, 21, 40, 0.55), moe(6, 3, 96)),
    layer(attention(4, 4, 128, 64, 70, 128), None),
    layer(parallel(left(6, 2, 32, 64, 64, 100, 32), right(2, 64, 128, 64, base=300.0), 1.0, 0.5), dense(320)),
    layer(diff(2, 1, 64, 64, 50, 5, 0.2), dense(256)),
])
# Ones wherever a one is possible.
ONES = config(61, 32, embedding_scale=1.0, layers=[
    layer(attention(1, 1, 4, 1, 1, 2), moe(1, 1, 1, shared=1, scale=1.0)),
    layer(parallel(left(1, 1, 4, 1, 5, 2, 2), right(1, 2, 1, 2, decay=[1.0]), 1.0, 1.0), dense(1)),
    layer(diff(1, 1, 4, 2, 1, 1, 0.5), moe(2, 1, 4, scale=1.0)),
])
CONFIGS = {"small": SMALL, "cores": CORES, "ones": ONES}
PAGE = {"small": 8, "cores": 16, "ones": 4}
STORED = {"small": "F32", "cores": "BF16", "ones": "BF16"}


def make_weights(cfg, seed):
    """name -> float32 array, every value a bfloat16 value (the engine in bf16 then holds what the plain implementation
    reads). Sinks and distance terms are of order one, so that leaving one out or taking a neighbour's shows; the routers'
    corrections are spread so that a rounding seldom changes a choice, and that the choice without them is another one."""
    rng = np.random.default_rng(seed)
    E, V = cfg["width"], cfg["vocab"]

    def n(shape, std, mean=0.0):
        return helpers.bf16_round(mean + rng.standard_normal(shape) * std)

    def gated(p, F):
        w[p + "gate"], w[p + "up"] = n((F, E), 1.0 / math.sqrt(E)), n((F, E), 1.0 / math.sqrt(E))
        w[p + "down"] = n((E, F), 1.0 / math.sqrt(F))

    w = {"embed": n((V, E), 1.0 / cfg["embedding"]["scale"]), "final.norm": n(E, 0.2, 1.0), "head": n((V, E), 1.0 / math.sqrt(E))}
    for l, lc in enumerate(cfg["layers"]):
        p, m = f"l{l}.", lc["mixer"]
        w[p + "norm1"] = n(E, 0.2, 0.6)
        if lc["mlp"] is not None:
            w[p + "norm2"] = n(E, 0.2, 0.6)
        q = p + "mix."
        if lc["type"] == "parallel":
            lt, rt = m["left"], m["right"]
            H, G, D, P = lt["heads"], lt["kv_heads"], lt["dim"], lt["vdim"]
            a = q + "left."
            for name, rows in (("q", H * D), ("k", G * D), ("v", G * P)):
                w[a + name], w[a + name + ".b"] = n((rows, E), 1.0 / math.sqrt(E)), n(rows, 0.3)
            w[a + "q.norm"], w[a + "k.norm"] = n(D, 0.2, 1.0), n(D, 0.2, 1.0)
            w[a + "rel"], w[a + "sink"] = n((lt["bias_rows"], H), 1.2), n(H, 1.2)
            w[a + "g"], w[a + "o"] = n((H, E), 1.2 / math.sqrt(E)), n((E, H * P), 1.0 / math.sqrt(H * P))
            H, D, P = rt["heads"], rt["dim"], rt["vdim"]
            a = q + "right."
            for name, rows in (("q", H * D), ("k", H * D), ("v", H * P), ("g", H * P)):
                w[a + name] = n((rows, E), 1.0 / math.sqrt(E))
            w[a + "o"] = n((E, H * P), 1.0 / math.sqrt(H * P))
        else:
            H, G, D, P = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            maps = 2 if lc["type"] == "attention_2" else 1
            w[q + "q"], w[q + "k"], w[q + "v"] = (n((rows, E), 1.0 / math.sqrt(E)) for rows in (H * maps * D, G * maps * D, G * P))
            w[q + "o"] = n((E, H * P), 1.0 / math.sqrt(H * P))
            if maps == 1:
                w[q + "sink"] = n(H, 1.2)
            else:
                w[q + "q.norm"], w[q + "k.norm"] = n(D, 0.2, 1.0), n(D, 0.2, 1.0)
                for name in ("lq1", "lk1", "lq2", "lk2"):
                    w[q + name] = n(D, 0.3 / D ** 0.25)
        f = lc["mlp"]
        if f is None:
            continue
        q = p + "mlp."
        if f["kind"] == "dense":
            gated(q, f["ff"])
        else:
            X = f["router"]["experts"]
            w[q + "router"] = n((X, E), 1.0 / math.sqrt(E))
            w[q + "correction"] = helpers.bf16_round(rng.permutation(X) * 0.25)
            for e in range(X):
                gated(f"{q}e{e}.", f["expert"]["ff"])
            if f.get("shared") is not None:
                gated(q + "shared.", f["shared"]["ff"])
                w[q + "shared.sg"] = n((1, E), 1.0 / math.sqrt(E))
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
    cfg, w = pl.read_model(model_dir)
    return {r: pl.forward(cfg, w, toks) for r, toks in reqs.items()}


def random_config(rng, big):
    """A configuration drawn at random: two to six layers of every kind in any order, with sizes that the matrix-core
    kernels take (``big``) or that none of them takes."""
    def pick(*xs):
        return xs[int(rng.integers(0, len(xs)))]
    width = pick(128, 192, 256, 384) if big else pick(24, 40, 58, 72, 100)
    layers = []
    for _ in range(int(rng.integers(2, 7))):
        kind = pick("attention", "parallel", "diff")
        G = pick(1, 2, 3, 4)
        H = G * pick(1, 2, 3)
        D, P = (pick(32, 64, 96, 128), pick(32, 64, 128)) if big else (pick(6, 10, 16, 24), pick(3, 8, 14, 17))
        if kind == "attention":
            mix = attention(H, G, D, P, pick(1, 5, 20, 47, 300), pick(D, D // 2 - (D // 2) % 2), base=pick(1000.0, 40000.0),
                            scaling=pick(None, (6.0, 1.0, 3.0, 128), (2.0, 0.5, 8.0, 40)))
        elif kind == "diff":
            D = min(D, 64)
            mix = diff(H, G, D, P, pick(1, 6, 19, 40, 300), pick(0, 1, 4, 16, 33), pick(0.2, 0.5, 0.8))
        else:
            rows = pick(2, 8, 32, 24)
            lt = left(H, G, D, P, pick(1, 7, 16, 50, 300), rows // 2 + pick(1, 5, 30, 200), rows)
            rh, rd = pick(1, 2, 4), pick(32, 64, 128) if big else pick(4, 8, 18, 24)
            rt = right(rh, rd, pick(32, 64) if big else pick(4, 5, 12, 20), pick(rd, rd // 2 - (rd // 2) % 2), base=pick(100.0, 10000.0))
            mix = parallel(lt, rt, pick(1.0, 0.55, -0.4), pick(1.0, 1.15, 0.3))
        X = pick(2, 5, 8)
        ff = pick(None, dense(pick(32, 64, 96) if big else pick(4, 10, 24)),
                  moe(X, pick(1, 2, X), pick(32, 64, 96) if big else pick(4, 10, 32), shared=pick(None, 32 if big else 6), scale=pick(0.5, 1.0, 2.5)))
        layers.append(layer(mix, ff))
    return config(int(rng.integers(50, 400)), width, layers, eps=pick(1e-5, 1e-6), embedding_scale=pick(1.0, 4.0, math.sqrt(width)))
