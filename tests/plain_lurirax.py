"""The plain implementation of the Lurirax design: whole sequences, float64 numpy, one function a mechanism.

No cache, no batching, no kernels, and no code shared with the package. The engine is compared with this.

The stream starts as ``embed[token] * scale``. A layer norms what its sublayers give and nothing else: ``x <- x + norm1(mixer(x))``,
then ``x <- x + norm2(ff(x))`` where the layer has a feed-forward. Three kinds of mixers:

* ``attention``: rotated queries and keys (frequencies rescaled by their wavelength) that are divided by their root mean square
  after the rotation; a sliding window; a softmax with one more term of a learned score a head and no value.
* ``parallel``: the weighted sum of two mixers on the same input. Left: attention inside chunks with biases, weighted per-head
  norms, a learned number per (distance bucket, head) added to the scores, a sink and one gate a head. Right: retention, a linear
  recurrence with a fixed decay a head, rotated queries and keys, a per-head norm and a silu gate.
* ``attention_2``: differential attention: two maps a head over the same values, the second subtracted with one learned factor;
  a sliding window beside the sequence's first tokens, which stay visible.

The feed-forward is a dense gated unit (tanh gelu) or a mixture of gated experts (silu): sigmoid scores, a correction that enters
the choice alone, and a shared expert behind a gate of its own.
"""
import math

import numpy as np

from plain import read_model          # noqa: F401  (the container reader is the same for every design)


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rotary_frequencies(dims, base, scaling=None):
    """f_i = base^(-2i / dims), i < dims / 2; rescaled by the wavelength l = 2 pi / f: kept where l < original / high, divided by
    ``factor`` where l > original / low, blended in between."""
    out = []
    for i in range(dims // 2):
        f = float(base) ** (-2.0 * i / dims)
        if scaling is not None:
            l = 2.0 * math.pi / f
            if l > scaling["original"] / scaling["low"]:
                f = f / scaling["factor"]
            elif l >= scaling["original"] / scaling["high"]:
                s = (scaling["original"] / l - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return np.array(out)


def rotate(x, positions, freqs):
    """x: [T, heads, n]; dimension i of the first 2 len(freqs) turns with dimension i + len(freqs) by positions * freqs[i]."""
    half = len(freqs)
    a = np.asarray(positions, dtype=np.float64)[:, None, None] * freqs
    u, v, rest = x[..., :half], x[..., half:2 * half], x[..., 2 * half:]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a), rest], axis=-1)


def sees_window(T, size, keep_first=0):
    """[T, T]: i sees j <= i among the last ``size`` positions, itself included, or among the first ``keep_first``."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def sees_chunk(T, size):
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & (i // size == j // size)


def bucket(n, rows, bias_max):
    """The row of a table of ``rows`` rows for the distance n: one a distance below rows / 2, logarithmic from there to ``bias_max``."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + int(math.floor(math.log(n / half) / math.log(bias_max / half) * (rows - half))))


def distance_bias(table, T, bias_max):
    """[heads, T, T]: table[bucket(i - j), head] (0 above the diagonal, where nothing is visible)."""
    by_distance = np.stack([table[bucket(n, table.shape[0], bias_max)] for n in range(T)])          # [T, heads]
    d = np.arange(T)[:, None] - np.arange(T)[None, :]
    return np.where((d >= 0)[..., None], by_distance[np.maximum(d, 0)], 0.0).transpose(2, 0, 1)


def softmax_attention(q, k, v, scale, visible, bias=None, sink=None):
    """q: [T, H, D], k: [T, G, D], v: [T, G', Dv] with G' dividing H -> [T, H, Dv]. ``sink`` [H]: the score of one more term of
    the denominator that has no value."""
    T, H, _ = q.shape
    kk = np.repeat(k, H // k.shape[1], axis=1)
    vv = np.repeat(v, H // v.shape[1], axis=1)
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        s = q[:, h] @ kk[:, h].T * scale
        if bias is not None:
            s = s + bias[h]
        s = np.where(visible, s, -np.inf)
        top = s.max(axis=-1, keepdims=True)
        if sink is not None:
            top = np.maximum(top, sink[h])
        e = np.exp(s - top)
        total = e.sum(axis=-1, keepdims=True)
        if sink is not None:
            total = total + np.exp(sink[h] - top)
        out[:, h] = (e / total) @ vv[:, h]
    return out


def attention(h, w, p, m, eps, positions):
    """``m``: heads, kv_heads, dim, vdim, scale, mask.size, rot = {base, dims, scaling}."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    f = rotary_frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
    q = unit_rms(rotate((h @ w[p + "q"].T).reshape(T, H, m["dim"]), positions, f), eps)
    k = unit_rms(rotate((h @ w[p + "k"].T).reshape(T, G, m["dim"]), positions, f), eps)
    v = (h @ w[p + "v"].T).reshape(T, G, m["vdim"])
    o = softmax_attention(q, k, v, m["scale"], sees_window(T, m["mask"]["size"]), sink=w[p + "sink"])
    return o.reshape(T, -1) @ w[p + "o"].T


def chunk_attention(h, w, p, m, eps):
    """The left side of ``parallel``. ``m``: heads, kv_heads, dim, vdim, scale, bias_max, mask.size."""
    T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = unit_rms((h @ w[p + "q"].T + w[p + "q.b"]).reshape(T, H, D), eps) * w[p + "q.norm"]
    k = unit_rms((h @ w[p + "k"].T + w[p + "k.b"]).reshape(T, G, D), eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].T + w[p + "v.b"]).reshape(T, G, m["vdim"])
    o = softmax_attention(q, k, v, m["scale"], sees_chunk(T, m["mask"]["size"]), bias=distance_bias(w[p + "rel"], T, m["bias_max"]),
                          sink=w[p + "sink"])
    o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, -1) @ w[p + "o"].T


def fixed_decay_recurrence(q, k, v, decay):
    """Per head S_t = decay S_(t-1) + k_t v_t^T, o_t = S_t^T q_t, S_0 = 0. q, k: [T, H, D]; v: [T, H, Dv]."""
    T, H, D = q.shape
    S = np.zeros((H, D, v.shape[2]))
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        S = np.asarray(decay)[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hdv,hd->hv", S, q[t])
    return out


def retention(h, w, p, m, eps, positions):
    """The right side of ``parallel``. ``m``: heads, dim, vdim, decay, rot = {base, dims}."""
    T, H, D = h.shape[0], m["heads"], m["dim"]
    f = rotary_frequencies(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling"))
    q = rotate((h @ w[p + "q"].T).reshape(T, H, D), positions, f)
    k = rotate((h @ w[p + "k"].T).reshape(T, H, D), positions, f) * D ** -0.5
    v = (h @ w[p + "v"].T).reshape(T, H, m["vdim"])
    o = unit_rms(fixed_decay_recurrence(q, k, v, m["decay"]), eps).reshape(T, -1)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel(h, w, p, m, eps, positions):
    return m["left_scale"] * chunk_attention(h, w, p + "left.", m["left"], eps) \
        + m["right_scale"] * retention(h, w, p + "right.", m["right"], eps, positions)


def map_factor(w, p, diff):
    """The factor of the second map: exp(lq1 . lk1) - exp(lq2 . lk2) + diff."""
    return math.exp(float((w[p + "lq1"] * w[p + "lk1"]).sum())) - math.exp(float((w[p + "lq2"] * w[p + "lk2"]).sum())) + diff


def differential_attention(h, w, p, m, eps):
    """``m``: heads, kv_heads, dim, vdim, scale, diff, mask = {size, keep_first}."""
    T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = unit_rms((h @ w[p + "q"].T).reshape(T, H, 2, D), eps) * w[p + "q.norm"]
    k = unit_rms((h @ w[p + "k"].T).reshape(T, G, 2, D), eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].T).reshape(T, G, m["vdim"])
    visible = sees_window(T, m["mask"]["size"], m["mask"].get("keep_first", 0))
    a1, a2 = (softmax_attention(q[:, :, i], k[:, :, i], v, m["scale"], visible) for i in (0, 1))
    o = unit_rms(a1 - map_factor(w, p, m["diff"]) * a2, eps) * (1.0 - m["diff"])
    return o.reshape(T, -1) @ w[p + "o"].T


def gated_unit(h, w, p, act):
    return (act(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h, w, p, router):
    """(ids [T, top], weights [T, top]): the largest sigmoid scores after the correction is added (the lower index among equals);
    their weights are the scores without it, times ``scale``."""
    s = sigmoid(h @ w[p + "router"].T)
    ids = np.argsort(-(s + w[p + "correction"]), axis=-1, kind="stable")[:, :router["top"]]
    return ids, np.take_along_axis(s, ids, axis=-1) * router["scale"]


def feed_forward(h, w, p, f):
    if f["kind"] == "dense":
        return gated_unit(h, w, p, gelu_tanh)
    ids, weights = route(h, w, p, f["router"])
    out = np.zeros((h.shape[0], w[p + "e0.down"].shape[0]))
    for t in range(h.shape[0]):
        for e, c in zip(ids[t], weights[t]):
            out[t] += c * gated_unit(h[t:t + 1], w, f"{p}e{e}.", silu)[0]
    if f.get("shared") is not None:
        out += sigmoid(h @ w[p + "shared.sg"].T) * gated_unit(h, w, p + "shared.", silu)
    return out


def mixer(kind, h, w, p, m, eps, positions):
    if kind == "attention":
        return attention(h, w, p, m, eps, positions)
    if kind == "parallel":
        return parallel(h, w, p, m, eps, positions)
    if kind == "attention_2":
        return differential_attention(h, w, p, m, eps)
    raise ValueError(f"unknown mixer '{kind}'")


def forward(cfg, w, tokens, layers_out=None):
    """Logits [T, vocab] of one whole sequence. ``layers_out``: a list that receives the stream after every layer."""
    w = {k: np.asarray(v, dtype=np.float64) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    positions = np.arange(len(tokens))
    x = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    for i, lc in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + unit_rms(mixer(lc["type"], x, w, p + "mix.", lc["mixer"], eps, positions), eps) * w[p + "norm1"]
        if lc.get("mlp") is not None:
            x = x + unit_rms(feed_forward(x, w, p + "mlp.", lc["mlp"]), eps) * w[p + "norm2"]
        if layers_out is not None:
            layers_out.append(x.copy())
    return unit_rms(x, eps) * w["final.norm"] @ w["head"].T
