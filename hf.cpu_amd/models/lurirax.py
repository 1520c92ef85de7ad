"""Lurirax as a plan: the stream starts as the scaled embedding; every layer norms what its sublayers give and nothing else
(``postnorm``); the mixer is, layer by layer, windowed attention whose rotated queries and keys are normed after the rotation, with a
learned sink (``attention``); two mixers side by side whose weighted sum is the result (``parallel``: attention in chunks with biases,
per-head norms, a table of distance terms, a sink and a gate a head, beside retention); or differential attention under a window
beside which the first tokens stay in sight (``attention_2``). The feed-forward, where a layer has one, is a dense gated unit with
the tanh gelu or a mixture of gated experts (sigmoid scores, a correction for the choice alone) with a gated shared expert; logits
from a head of its own after the model's norm.

Tensor names: ``embed``, ``head``, ``final.norm``; ``l<i>.norm1``, ``l<i>.norm2``; ``l<i>.mix.*`` (``q``, ``k``, ``v``, ``sink``, ``o`` /
``left.{q,k,v}`` (+ ``.b``), ``left.{q,k}.norm``, ``left.{rel,sink,g,o}``, ``right.{q,k,v,g,o}`` / ``q``, ``k``, ``v``, ``q.norm``, ``k.norm``, ``lq1``,
``lk1``, ``lq2``, ``lk2``, ``o``); ``l<i>.mlp.{gate,up,down}`` or ``l<i>.mlp.router``, ``l<i>.mlp.correction``, ``l<i>.mlp.e<n>.{gate,up,down}``,
``l<i>.mlp.shared.{gate,up,down,sg}``.
"""
from ..config.lurirax import LuriraxConfig
from ..plan import LayerPlan, ModelPlan, PartSpec, ScheduleEntry
from ..registry import register_architecture

EXPERT_ALPHA = 1.0            # an expert's gate half is g sigmoid(g), silu
GATED_NAMES = dict(gate="gate", up="up", down="down")
PROJECTIONS = dict(q="q", k="k", v="v", o="o", q_norm="q.norm", k_norm="k.norm")


def _norm(cfg, name):
    return PartSpec("rmsnorm", dict(size=cfg.width, eps=cfg.norm_eps, prefix=name, weight=""))


def _rotary(rot, head_dim):
    scaling = None if rot.scaling is None else dict(zip(("factor", "low", "high", "original"), rot.scaling))
    return PartSpec("rotary", dict(head_dim=head_dim, rot_dim=rot.dims, theta=rot.base, scaling=scaling))


def _mixer(cfg, lc, prefix):
    E, eps, m = cfg.width, cfg.norm_eps, lc.mixer
    if lc.type == "attention":
        return PartSpec("attention", dict(
            hidden_size=E, n_heads=m.heads, n_kv_heads=m.kv_heads, head_dim=m.dim, v_head_dim=m.vdim, qkv_bias=False, window=m.window,
            scale=m.scale, position=_rotary(m.rot, m.dim), head_norm=eps, head_norm_weight=False, norm_after=True, sink="learned",
            prefix=prefix, names=PROJECTIONS))
    if lc.type == "attention_2":
        return PartSpec("attention", dict(
            hidden_size=E, n_heads=m.heads, n_kv_heads=m.kv_heads, head_dim=m.dim, v_head_dim=m.vdim, qkv_bias=False, window=m.window,
            scale=m.scale, position=PartSpec("none", dict(head_dim=m.dim)), head_norm=eps, keep_first=m.keep_first, maps=2, diff=m.diff,
            prefix=prefix, names=PROJECTIONS))
    lt, rt = m.left, m.right
    left = PartSpec("attention", dict(
        hidden_size=E, n_heads=lt.heads, n_kv_heads=lt.kv_heads, head_dim=lt.dim, v_head_dim=lt.vdim, qkv_bias=True, window=0,
        mask_chunk=lt.chunk, scale=lt.scale, position=PartSpec("none", dict(head_dim=lt.dim)), head_norm=eps, sink="learned",
        rel_bias=dict(rows=lt.bias_rows, reach=lt.bias_max), out_gate="head", prefix=prefix + "left.",
        names=dict(PROJECTIONS, g="g", q_bias="q.b", k_bias="k.b", v_bias="v.b")))
    right = PartSpec("retention", dict(
        hidden_size=E, n_heads=rt.heads, head_dim=rt.dim, v_head_dim=rt.vdim, decay=rt.decay, eps=eps, position=_rotary(rt.rot, rt.dim),
        prefix=prefix + "right.", names=dict(q="q", k="k", v="v", g="g", o="o")))
    return PartSpec("side_by_side", dict(hidden_size=E, left=left, right=right, normed=False, left_scale=m.left_scale,
                                         right_scale=m.right_scale, prefix=prefix))


def _feed_forward(cfg, f, prefix):
    E = cfg.width
    if f.kind == "dense":
        return PartSpec("gated_mlp", dict(hidden_size=E, intermediate_size=f.ff, activation="gelu_tanh", prefix=prefix, names=GATED_NAMES))
    shared = None
    if f.shared_ff:
        shared = PartSpec("gated_mlp", dict(hidden_size=E, intermediate_size=f.shared_ff, prefix=prefix + "shared.", names=GATED_NAMES))
    return PartSpec("moe", dict(
        hidden_size=E, expert_size=f.ff, n_experts=f.experts, top=f.top, scoring="sigmoid", renormalize=False, weight_scale=f.scale,
        weight_on="output", gated=dict(alpha=EXPERT_ALPHA, limit=0.0, shift=0.0), correction=True, shared=shared,
        shared_gate=shared is not None, prefix=prefix,
        names=dict(router="router", correction="correction", shared_gate="shared.sg", gate="e{e}.gate", up="e{e}.up", down="e{e}.down")))


def lurirax_plan(cfg):
    E = cfg.width
    layers, schedule = [], []
    for l, lc in enumerate(cfg.layers):
        prefix = f"l{l}."
        parts = dict(norm1=_norm(cfg, prefix + "norm1"), mixer=_mixer(cfg, lc, prefix + "mix."))
        unused = ()
        if lc.mlp is not None:
            parts.update(norm2=_norm(cfg, prefix + "norm2"), feed_forward=_feed_forward(cfg, lc.mlp, prefix + "mlp."))
        else:                        # a checkpoint may hold the second norm's weight all the same
            unused = (("norm2", (E,)),)
        layers.append(LayerPlan.of(prefix, PartSpec("postnorm", dict(hidden_size=E, prefix=prefix, unused=unused)), **parts))
        schedule.append(ScheduleEntry(l))
    return ModelPlan(
        hidden_size=E, vocab_size=cfg.vocab,
        embedding=PartSpec("lookup", dict(vocab_size=cfg.vocab, hidden_size=E, prefix="", weight="embed", scale=cfg.embedding_scale, copy=True)),
        layers=tuple(layers), schedule=tuple(schedule), final_norm=_norm(cfg, "final.norm"),
        head=PartSpec("linear", dict(vocab_size=cfg.vocab, hidden_size=E, tied=False, prefix="", weight="head")),
    ).check()


register_architecture("Lurirax", LuriraxConfig, lurirax_plan)
