"""The typed configuration of the Lurirax design.

config.json: ``architecture`` (the name), ``vocab``, ``width``, ``embedding.scale``, ``norm.eps`` and ``layers``, a list with one object a
layer: ``type`` (the kind of mixer), ``mixer`` (its sizes and constants) and ``mlp`` (null, or a feed-forward). Mixers:

* ``attention``: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``mask`` = {``size``} (the window in tokens; absent: none), ``rot`` =
  {``base``, ``dims``, optionally ``scaling`` = {``factor``, ``low``, ``high``, ``original``}}
* ``parallel``: ``left`` (attention in chunks: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``mask`` = {``size``} (the chunk; absent: none),
  ``bias_max`` (the distance from which the last row of the table of distance terms holds); optionally ``bias_rows``, the table's rows, which
  a checkpoint's tensor gives otherwise), ``right`` (retention: ``heads``, ``dim``, ``vdim``, ``decay``, one number a head, ``rot``),
  ``left_scale`` and ``right_scale``
* ``attention_2``: differential attention: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``diff``, ``mask`` = {``size``, ``keep_first``} (the
  window and how many first tokens stay in sight beside it)

Feed-forwards: ``kind`` ``dense`` with ``ff``, or ``moe`` with ``expert.ff``, ``router.experts``, ``router.top``, ``router.scale`` and optionally
``shared.ff`` (an expert that every token passes, behind a gate).

Every size and constant of a model comes from there; layers may differ from one another in all of them, and come in any order.
"""
from dataclasses import dataclass
from typing import Optional

from ..status import EFORMAT, ENOTSUP, fail
from .reader import KeyReader


@dataclass(frozen=True)
class LuriraxRotary:
    base: float
    dims: int
    scaling: Optional[tuple]     # (factor, low, high, original)


@dataclass(frozen=True)
class LuriraxAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int          # 0: none
    rot: LuriraxRotary


@dataclass(frozen=True)
class LuriraxLeft:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int           # 0: none
    bias_max: int
    bias_rows: int       # 0: the tensor says


@dataclass(frozen=True)
class LuriraxRight:
    heads: int
    dim: int
    vdim: int
    decay: tuple
    rot: LuriraxRotary


@dataclass(frozen=True)
class LuriraxParallel:
    left: LuriraxLeft
    right: LuriraxRight
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class LuriraxDifferential:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    diff: float
    window: int          # 0: none
    keep_first: int


@dataclass(frozen=True)
class LuriraxMLP:
    kind: str            # dense | moe
    ff: int              # the dense layer's size, or an expert's
    experts: int = 0
    top: int = 0
    scale: float = 1.0
    shared_ff: int = 0   # 0: no shared expert


@dataclass(frozen=True)
class LuriraxLayer:
    type: str
    mixer: object
    mlp: Optional[LuriraxMLP]


MIXERS = ("attention", "parallel", "attention_2")


@dataclass(frozen=True, eq=False)
class LuriraxConfig:
    architecture: str
    vocab: int
    width: int
    embedding_scale: float
    norm_eps: float
    layers: tuple
    raw: dict            # config.json as read (to_dict gives it back)

    @staticmethod
    def _sub(r, key):
        v = r.obj.get(key)
        if not isinstance(v, dict):
            fail(EFORMAT, f"{r.origin}: key '{key}' is missing or not an object")
        return KeyReader(v, f"{r.origin}: {key}")

    @classmethod
    def _rotary(cls, m, limit):
        r = cls._sub(m, "rot")
        dims = r.integer("dims", lo=2, hi=limit)
        if dims % 2:
            fail(EFORMAT, f"{r.origin}: key 'dims' must be even, got {dims}")
        scaling = None
        if r.has("scaling"):
            s = cls._sub(r, "scaling")
            scaling = tuple(s.number(k, lo=0.0) for k in ("factor", "low", "high", "original"))
            if not scaling[2] > scaling[1]:
                fail(EFORMAT, f"{s.origin}: 'high' must exceed 'low'")
        return LuriraxRotary(r.number("base", lo=0.0), dims, scaling)

    @classmethod
    def _mask(cls, m, key, lo=1):
        """A number of the mask; 0 without one."""
        if not m.has("mask"):
            return 0
        mask = cls._sub(m, "mask")
        return mask.integer(key, lo=lo, hi=1 << 30) if key == "size" else mask.integer(key, 0, lo=lo, hi=1 << 30)

    @staticmethod
    def _heads(m):
        heads, kv = m.integer("heads", hi=1024), m.integer("kv_heads")
        if heads % kv:
            fail(EFORMAT, f"{m.origin}: {heads} heads are not a multiple of {kv} kv_heads")
        return heads, kv, m.integer("dim", hi=256), m.integer("vdim", hi=256), m.number("scale", lo=0.0)

    @classmethod
    def _mixer(cls, kind, m):
        if kind == "attention":
            sizes = cls._heads(m)
            return LuriraxAttention(*sizes, cls._mask(m, "size"), cls._rotary(m, sizes[2]))
        if kind == "attention_2":
            return LuriraxDifferential(*cls._heads(m), m.number("diff"), cls._mask(m, "size"), cls._mask(m, "keep_first", 0))
        lt, rt = cls._sub(m, "left"), cls._sub(m, "right")
        left = LuriraxLeft(*cls._heads(lt), cls._mask(lt, "size"), lt.integer("bias_max", lo=2, hi=1 << 30),
                           lt.integer("bias_rows", 0, lo=0, hi=1 << 16))
        dim = rt.integer("dim", hi=256)
        decay = rt.obj.get("decay")
        if not isinstance(decay, list) or any(isinstance(d, bool) or not isinstance(d, (int, float)) for d in decay):
            fail(EFORMAT, f"{rt.origin}: key 'decay' is missing or not a list of numbers")
        right = LuriraxRight(rt.integer("heads"), dim, rt.integer("vdim"), tuple(float(d) for d in decay), cls._rotary(rt, dim))
        if len(right.decay) != right.heads:
            fail(EFORMAT, f"{rt.origin}: {len(right.decay)} decays for {right.heads} heads")
        return LuriraxParallel(left, right, m.number("left_scale"), m.number("right_scale"))

    @classmethod
    def _mlp(cls, f):
        kind = f.string("kind")
        if kind == "dense":
            return LuriraxMLP("dense", f.integer("ff"))
        if kind != "moe":
            fail(ENOTSUP, f"{f.origin}: a feed-forward of kind '{kind}' is not supported (supported: dense, moe)")
        router = cls._sub(f, "router")
        experts, top = router.integer("experts", hi=1024), router.integer("top", hi=64)
        if top > experts:
            fail(EFORMAT, f"{router.origin}: {top} choices among {experts} experts")
        shared = cls._sub(f, "shared").integer("ff") if f.has("shared") else 0
        return LuriraxMLP("moe", cls._sub(f, "expert").integer("ff"), experts, top, router.number("scale", 1.0), shared)

    @classmethod
    def from_dict(cls, obj, origin="config.json"):
        r = KeyReader(obj, origin)
        raw_layers = obj.get("layers")
        if not isinstance(raw_layers, list) or not raw_layers:
            fail(EFORMAT, f"{origin}: key 'layers' is missing or not a list of layers")
        layers = []
        for i, lo in enumerate(raw_layers):
            lr = KeyReader(lo, f"{origin}: layers[{i}]")
            kind = lr.string("type")
            if kind not in MIXERS:
                fail(ENOTSUP, f"{lr.origin}: a mixer of type '{kind}' is not supported (supported: {', '.join(MIXERS)})")
            mixer = cls._mixer(kind, cls._sub(lr, "mixer"))
            layers.append(LuriraxLayer(kind, mixer, cls._mlp(cls._sub(lr, "mlp")) if lr.has("mlp") else None))
        norm, emb = cls._sub(r, "norm"), cls._sub(r, "embedding")
        return cls(architecture=r.string("architecture"), vocab=r.integer("vocab", hi=1 << 24), width=r.integer("width"),
                   embedding_scale=emb.number("scale"), norm_eps=norm.number("eps", lo=0.0), layers=tuple(layers), raw=obj)

    def to_dict(self):
        """The config.json content that reads back as this configuration."""
        return dict(self.raw)
