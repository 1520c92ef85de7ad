"""Fugevik as a plan: the residual is several streams side by side (hyper-connections), all of them the embedding at the start; what
a sublayer reads is one weighted sum of them, RMS-normed with a weight stored as its distance from 1 and passed through a short
causal convolution that is added to its own input; the mixer is, layer by layer, attention through latents with a window, a learned
sink and a gate (``latent_attention``) or windowed attention without rotation whose scores are soft-capped and lowered by a logarithm
of the distance (``attention``), which may read an earlier layer's keys and values; the feed-forward, where a layer has one, is dense
with the square of relu; logits from the embedding table after the norm of the streams' sum.

Tensor names: ``embed``, ``final.norm``; ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.canon1``, ``l<i>.canon2``, ``l<i>.hc1.{in,out,mix}``, ``l<i>.hc2.{..}``;
``l<i>.mix.*`` (``q``, ``dkv``, ``dkv.norm``, ``uk``, ``uv``, ``sink``, ``g``, ``o`` / ``q``, ``k``, ``v``, ``r1``, ``r2``, ``o``); ``l<i>.mlp.{up,down}``.
"""
from ..config.fugevik import FugevikConfig
from ..plan import LayerPlan, ModelPlan, PartSpec, ScheduleEntry
from ..registry import register_architecture


def _norm(cfg, name):
    return PartSpec("rmsnorm", dict(size=cfg.width, eps=cfg.norm_eps, prefix=name, weight="", offset=1.0))


def _mixer(cfg, lc, prefix):
    E, m = cfg.width, lc.mixer
    if lc.type == "latent_attention":
        rot = PartSpec("rotary", dict(head_dim=m.rot_dim, rot_dim=m.rot_dims, theta=m.rot_base, pairing="interleaved"))
        return PartSpec("latent_attention", dict(
            hidden_size=E, n_heads=m.heads, head_dim=m.dim, rot_dim=m.rot_dim, v_head_dim=m.vdim, kv_rank=m.kv_rank, q_latent=False,
            scale=m.scale, eps=cfg.norm_eps, position=rot, window=m.window, sink=True, prefix=prefix))
    return PartSpec("attention", dict(
        hidden_size=E, n_heads=m.heads, n_kv_heads=m.kv_heads, head_dim=m.dim, v_head_dim=m.vdim, qkv_bias=False, window=m.window,
        scale=m.scale, position=PartSpec("none", dict(head_dim=m.dim)), own_kv=m.kv_from is None, softcap=m.softcap or None,
        distance=True, prefix=prefix, names=dict(q="q", k="k", v="v", o="o", dist_scale="r1", dist_rate="r2")))


def fugevik_plan(cfg):
    E, S = cfg.width, cfg.streams
    layers, schedule = [], []
    for l, lc in enumerate(cfg.layers):
        prefix = f"l{l}."

        def conv(name):
            return PartSpec("causal_conv", dict(size=E, taps=cfg.taps, prefix=prefix, weight=name))
        parts = dict(norm1=_norm(cfg, prefix + "norm1"), input1=conv("canon1"), mixer=_mixer(cfg, lc, prefix + "mix."))
        names, unused = {"mixer": "hc1."}, ()
        if lc.ff:
            parts.update(norm2=_norm(cfg, prefix + "norm2"), input2=conv("canon2"),
                         feed_forward=PartSpec("mlp", dict(hidden_size=E, intermediate_size=lc.ff, activation="relu2", prefix=prefix + "mlp.",
                                                           names=dict(up="up", down="down"))))
            names["feed_forward"] = "hc2."
        else:                        # a checkpoint may hold the second sublayer's small tensors all the same
            unused = (("norm2", (E,)), ("canon2", (E, cfg.taps)), ("hc2.in", (S,)), ("hc2.out", (S,)), ("hc2.mix", (S, S)))
        block = PartSpec("hyper", dict(hidden_size=E, streams=S, names=names, prefix=prefix, unused=unused))
        layers.append(LayerPlan.of(prefix, block, **parts))
        schedule.append(ScheduleEntry(l, cache_of=lc.mixer.kv_from if lc.type == "attention" else None))
    return ModelPlan(
        hidden_size=E, vocab_size=cfg.vocab, streams=S,
        embedding=PartSpec("lookup", dict(vocab_size=cfg.vocab, hidden_size=E, prefix="", weight="embed")),
        layers=tuple(layers), schedule=tuple(schedule), final_norm=_norm(cfg, "final.norm"),
        head=PartSpec("linear", dict(vocab_size=cfg.vocab, hidden_size=E, tied=True, tied_to="embed", prefix="", weight="head")),
    ).check()


register_architecture("Fugevik", FugevikConfig, fugevik_plan)
