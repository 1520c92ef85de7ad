"""The typed configuration of the Fugevik design.

config.json: ``architecture`` (the name), ``vocab``, ``width``, ``streams`` (how many streams the residual is), ``canon.taps`` (inputs of the
convolution in front of every sublayer), ``norm.eps`` and ``layers``, a list with one object a layer: ``type`` (the kind of mixer),
``mixer`` (its sizes and constants) and ``mlp`` (null, or ``kind`` ``dense`` with ``ff``). Mixers:

* ``latent_attention``: ``heads``, ``dim`` (unrotated query/key dimensions a head), ``rot_dim`` (rotated ones), ``vdim``, ``kv_rank``, ``scale``,
  ``rot`` = {``base``, ``dims``}, ``mask`` = {``size``} (the window in tokens; absent: none)
* ``attention``: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``softcap`` (absent or 0: none), ``mask`` = {``size``}, optionally ``kv_from``
  (the earlier layer whose keys and values are read)

Every size and constant of a model comes from there; layers may differ from one another in all of them, and come in any order.
"""
from dataclasses import dataclass
from typing import Optional

from ..status import EFORMAT, ENOTSUP, fail
from .reader import KeyReader


@dataclass(frozen=True)
class FugevikLatent:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    rot_base: float
    rot_dims: int
    window: int          # 0: none


@dataclass(frozen=True)
class FugevikAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float       # 0: none
    window: int          # 0: none
    kv_from: Optional[int]


@dataclass(frozen=True)
class FugevikLayer:
    type: str
    mixer: object
    ff: int              # the feed-forward's size, 0: none


MIXERS = ("latent_attention", "attention")


@dataclass(frozen=True, eq=False)
class FugevikConfig:
    architecture: str
    vocab: int
    width: int
    streams: int
    taps: int
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
    def _window(cls, m):
        return cls._sub(m, "mask").integer("size", hi=1 << 30) if m.has("mask") else 0

    @classmethod
    def _mixer(cls, kind, m, index, layers):
        if kind == "latent_attention":
            rot_dim = m.integer("rot_dim", hi=512)
            rot = cls._sub(m, "rot")
            dims = rot.integer("dims", lo=2, hi=rot_dim)
            if dims % 2:
                fail(EFORMAT, f"{rot.origin}: key 'dims' must be even, got {dims}")
            return FugevikLatent(m.integer("heads", hi=1024), m.integer("dim", hi=512), rot_dim, m.integer("vdim", hi=512),
                                 m.integer("kv_rank", hi=4096), m.number("scale"), rot.number("base", lo=0.0), dims, cls._window(m))
        a = FugevikAttention(m.integer("heads", hi=1024), m.integer("kv_heads"), m.integer("dim", hi=256), m.integer("vdim", hi=256),
                             m.number("scale"), m.number("softcap", 0.0) or 0.0, cls._window(m),
                             m.integer("kv_from", lo=0) if m.has("kv_from") else None)
        if a.heads % a.kv_heads:
            fail(EFORMAT, f"{m.origin}: {a.heads} heads are not a multiple of {a.kv_heads} kv_heads")
        if a.softcap < 0.0:
            fail(EFORMAT, f"{m.origin}: key 'softcap' has an implausible value {a.softcap}")
        if a.kv_from is not None:
            src = layers[a.kv_from] if a.kv_from < index else None
            if src is None or src.type != "attention" or src.mixer.kv_from is not None:
                fail(EFORMAT, f"{m.origin}: key 'kv_from' names layer {a.kv_from}, which is no earlier attention layer with keys of its own")
            if (src.mixer.kv_heads, src.mixer.dim, src.mixer.vdim) != (a.kv_heads, a.dim, a.vdim):
                fail(EFORMAT, f"{m.origin}: layer {a.kv_from} has keys and values of other sizes")
        return a

    @classmethod
    def _ff(cls, f):
        kind = f.string("kind")
        if kind != "dense":
            fail(ENOTSUP, f"{f.origin}: a feed-forward of kind '{kind}' is not supported (supported: dense)")
        return f.integer("ff")

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
            mixer = cls._mixer(kind, cls._sub(lr, "mixer"), i, layers)
            layers.append(FugevikLayer(kind, mixer, cls._ff(cls._sub(lr, "mlp")) if lr.has("mlp") else 0))
        return cls(architecture=r.string("architecture"), vocab=r.integer("vocab", hi=1 << 24), width=r.integer("width", hi=12288),
                   streams=r.integer("streams", hi=32), taps=cls._sub(r, "canon").integer("taps", hi=8),
                   norm_eps=cls._sub(r, "norm").number("eps", lo=0.0), layers=tuple(layers), raw=obj)

    def to_dict(self):
        """The config.json content that reads back as this configuration."""
        return dict(self.raw)
