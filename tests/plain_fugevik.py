"""The plain implementation of the Fugevik design: whole sequences, float64 numpy, one function a mechanism.

No cache, no batching, no kernels, and no code shared with the package. The engine is compared with this.

The residual is several streams side by side, all of them the embedding at the start. A sublayer (mixer, feed-forward) reads one
weighted sum of the streams, normed and passed through a short causal convolution per channel that is added to its own input;
its result goes back into every stream while the streams are mixed among themselves. Two mixers:

* ``latent_attention``: windowed softmax attention whose keys and values are expanded from one normed latent a token, with one
  rotated key part a token that all heads share; every head's denominator has a learned extra term; a sigmoid gate on the heads.
* ``attention``: windowed softmax attention with grouped heads and no rotation; scores are soft-capped, then lowered by a
  logarithm of the distance. A layer may read the keys and values of an earlier one.

The feed-forward is ``Wdown relu(Wup h)^2``; the logits come from the embedding table.
"""
import numpy as np

from plain import read_model          # noqa: F401  (the container reader is the same for every design)


def rms_norm(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last axis."""
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def relu2(z):
    return np.maximum(z, 0.0) ** 2


def causal_conv(h, w):
    """h: [T, E], w: [E, K] -> [T, E]: sum_j w[:, j] h_(t - K + 1 + j), zeros before the first token."""
    T, K = h.shape[0], w.shape[1]
    padded = np.concatenate([np.zeros((K - 1, h.shape[1])), h])
    return sum(w[:, j] * padded[j:j + T] for j in range(K))


def input_conv(h, w):
    return h + causal_conv(h, w)


def stream_input(x, w_in):
    """x: [T, S, E] -> the weighted sum of the streams [T, E]."""
    return np.einsum("s,tse->te", w_in, x)


def stream_update(x, y, mix, out):
    """x: [T, S, E], y: [T, E]: stream b becomes sum_a mix[a, b] x_a + out[b] y, all from the old streams."""
    return np.einsum("ab,tae->tbe", mix, x) + out[None, :, None] * y[:, None, :]


def rotate_pairs(x, positions, dims, base):
    """x: [T, ..., n >= dims]: dimensions (2i, 2i + 1), i < dims / 2, are turned by p base^(-2i / dims); the rest passes."""
    f = base ** (-2.0 * np.arange(dims // 2, dtype=np.float64) / dims)
    a = np.asarray(positions, dtype=np.float64)[:, None] * f
    shape = (x.shape[0],) + (1,) * (x.ndim - 2) + (dims // 2,)
    cos, sin = np.cos(a).reshape(shape), np.sin(a).reshape(shape)
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out = x.copy()
    out[..., 0:dims:2] = u * cos - v * sin
    out[..., 1:dims:2] = v * cos + u * sin
    return out


def window_mask(T, size):
    """[T, T] of bool: query i sees key j iff 0 <= i - j < size (size 0: every j <= i)."""
    d = np.arange(T)[:, None] - np.arange(T)[None, :]
    return (d >= 0) & ((d < size) if size else True)


def softmax_weights(s, mask, sink=None):
    """s: [H, T, T] -> weights of the visible keys; with ``sink`` ([H]) a head's denominator has one more term exp(sink_h)."""
    s = np.where(mask[None], s, -np.inf)
    top = s.max(axis=-1, keepdims=True)
    if sink is not None:
        top = np.maximum(top, sink[:, None, None])
    e = np.exp(s - top)
    z = e.sum(axis=-1, keepdims=True)
    if sink is not None:
        z = z + np.exp(sink[:, None, None] - top)
    return e / z


def soft_cap(s, cap):
    return cap * np.tanh(s / cap)


def distance_penalty(T, r1, r2):
    """[H, T, T]: r1_h ln(1 + r2_h (i - j)) for j <= i (0 elsewhere)."""
    d = np.maximum(np.arange(T)[:, None] - np.arange(T)[None, :], 0).astype(np.float64)
    return r1[:, None, None] * np.log(1.0 + r2[:, None, None] * d[None])


def latent_attention(h, w, p, m, eps, positions):
    """``m``: heads, dim, rot_dim, vdim, kv_rank, scale, rot = {base, dims}, mask = {size}."""
    T = h.shape[0]
    H, D, R, Dv, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (h @ w[p + "q"].T).reshape(T, H, D + R)
    down = h @ w[p + "dkv"].T
    c = rms_norm(down[:, :C], w[p + "dkv.norm"], eps)
    k_rot = rotate_pairs(down[:, C:], positions, m["rot"]["dims"], m["rot"]["base"])
    q_rot = rotate_pairs(q[..., D:], positions, m["rot"]["dims"], m["rot"]["base"])
    k = (c @ w[p + "uk"].T).reshape(T, H, D)
    v = (c @ w[p + "uv"].T).reshape(T, H, Dv)
    s = (np.einsum("ihd,jhd->hij", q[..., :D], k) + np.einsum("ihr,jr->hij", q_rot, k_rot)) * m["scale"]
    a = softmax_weights(s, window_mask(T, (m.get("mask") or {}).get("size", 0)), w[p + "sink"])
    o = np.einsum("hij,jhd->ihd", a, v).reshape(T, H * Dv)
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def attention(h, w, p, m, kept):
    """``m``: heads, kv_heads, dim, vdim, scale, softcap, mask = {size}, optionally kv_from. ``kept``: (k, v) of the layers that
    ran, by index. Returns (result, own (k, v) or None)."""
    T = h.shape[0]
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).reshape(T, H, D)
    own = None
    if m.get("kv_from") is None:
        own = ((h @ w[p + "k"].T).reshape(T, G, D), (h @ w[p + "v"].T).reshape(T, G, Dv))
    k, v = own if own is not None else kept[m["kv_from"]]
    k, v = np.repeat(k, H // G, axis=1), np.repeat(v, H // G, axis=1)
    s = np.einsum("ihd,jhd->hij", q, k) * m["scale"]
    if m.get("softcap"):
        s = soft_cap(s, m["softcap"])
    s = s - distance_penalty(T, w[p + "r1"], w[p + "r2"])
    a = softmax_weights(s, window_mask(T, (m.get("mask") or {}).get("size", 0)))
    return np.einsum("hij,jhd->ihd", a, v).reshape(T, H * Dv) @ w[p + "o"].T, own


def feed_forward(h, w, p):
    return relu2(h @ w[p + "up"].T) @ w[p + "down"].T


def forward(cfg, w, tokens, layers_out=None):
    """Logits [T, vocab] in float64; ``layers_out`` (a list) receives the sum of the streams after every layer."""
    eps, S = cfg["norm"]["eps"], cfg["streams"]
    T = len(tokens)
    positions = np.arange(T)
    w = {k: np.asarray(v, dtype=np.float64) for k, v in w.items()}
    x = np.repeat(w["embed"][np.asarray(tokens)][:, None, :], S, axis=1)
    kept = {}

    def sublayer(x, p, q, run):
        h = rms_norm(stream_input(x, w[f"{p}hc{q}.in"]), 1.0 + w[f"{p}norm{q}"], eps)
        h = input_conv(h, w[f"{p}canon{q}"])
        return stream_update(x, run(h), w[f"{p}hc{q}.mix"], w[f"{p}hc{q}.out"])

    for l, lc in enumerate(cfg["layers"]):
        p, m = f"l{l}.", lc["mixer"]

        def mixer(h):
            if lc["type"] == "latent_attention":
                return latent_attention(h, w, p + "mix.", m, eps, positions)
            y, own = attention(h, w, p + "mix.", m, kept)
            if own is not None:
                kept[l] = own
            return y
        x = sublayer(x, p, 1, mixer)
        if lc["mlp"] is not None:
            x = sublayer(x, p, 2, lambda h: feed_forward(h, w, p + "mlp."))
        if layers_out is not None:
            layers_out.append(x.sum(axis=1))
    return rms_norm(x.sum(axis=1), 1.0 + w["final.norm"], eps) @ w["embed"].T
