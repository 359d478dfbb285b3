"""Typed configuration of the Figalorn decoder: pre-norm layers listed one by one, each a mixer (the difference of two
softmax attentions over chunks of positions, or a softmax attention over a window whose values are its keys) and an
optional dense feed-forward; a stretch of the layers may run several times over.

config.json names the design under "architecture"; every size and every constant that can differ between models is
a key here, and an unknown layer type or feed-forward kind is an error. A section that a model leaves out switches its
mechanism off: "mask" (the attention then sees every earlier key), "rot", "rot.scaling", "softcap", "mlp", "loop".
"""
from dataclasses import dataclass
from typing import Optional, Tuple

from ..errors import ConfigError
from .base import Reader

# The design names no longest sequence: positions are bounded by what the cache holds.
MAX_POSITIONS = 1 << 20


def _section(raw, key, where):
    v = raw.get(key)
    if not isinstance(v, dict):
        raise ConfigError(f"config.json: {where}{key} must be an object")
    return Reader(v)


def _positive(where, **values):
    for name, v in values.items():
        if v is None or v <= 0:
            raise ConfigError(f"config.json: {where}{name} must be positive")


@dataclass(frozen=True)
class Rotation:
    base: float
    dims: int
    scaling: Optional[Tuple[Tuple[str, float], ...]] = None      # its constants by name, in the order of the mixer's kind

    @staticmethod
    def from_reader(r, where, dim, constants):
        if r.raw.get("rot") is None:
            return None
        rot, where = _section(r.raw, "rot", where + "."), where + ".rot"
        scaling = None
        if rot.raw.get("scaling") is not None:
            sc = _section(rot.raw, "scaling", where + ".")
            scaling = tuple((k, sc.number(k, required=True)) for k in constants)
            _positive(where + ".scaling.", **dict(scaling))
        c = Rotation(rot.number("base", required=True), rot.integer("dims", required=True), scaling)
        _positive(where + ".", base=c.base, dims=c.dims)
        if c.dims % 2 or c.dims > dim:
            raise ConfigError(f"config.json: {where}.dims must be even and at most {dim}")
        return c

    def to_dict(self):
        d = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            d["scaling"] = dict(self.scaling)
        return d


@dataclass(frozen=True)
class _Attention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    size: Optional[int]                     # mask.size; None: every earlier key is seen
    rot: Optional[Rotation]

    SCALING = ()

    @classmethod
    def _common(cls, r, where):
        size = None
        if r.raw.get("mask") is not None:
            size = _section(r.raw, "mask", where + ".").integer("size", required=True)
            _positive(where + ".mask.", size=size)
        sizes = {k: r.integer(k, required=True) for k in ("heads", "kv_heads", "dim")}
        vdim = r.integer("vdim", sizes["dim"])
        scale = r.number("scale", required=True)
        _positive(where + ".", vdim=vdim, scale=scale, **sizes)
        if sizes["heads"] % sizes["kv_heads"]:
            raise ConfigError(f"config.json: {where}: heads must be a multiple of kv_heads")
        return (*sizes.values(), vdim, scale, size, Rotation.from_reader(r, where, sizes["dim"], cls.SCALING))

    def to_dict(self):
        d = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.size is not None:
            d["mask"] = {"size": self.size}
        if self.rot is not None:
            d["rot"] = self.rot.to_dict()
        return d


@dataclass(frozen=True)
class DifferenceConfig(_Attention):
    """Two maps of `dim` a head over the same values, within chunks of `size` positions."""
    diff: float = 0.0

    SCALING = ("factor", "low", "high", "original")

    @classmethod
    def from_reader(cls, r, where):
        return cls(*cls._common(r, where), r.number("diff", required=True))

    def to_dict(self):
        return {**super().to_dict(), "diff": self.diff}


@dataclass(frozen=True)
class KeyValueConfig(_Attention):
    """Values that are the keys as projected, over a window of `size` positions."""
    softcap: Optional[float] = None

    SCALING = ("factor", "original", "fast", "slow")

    @classmethod
    def from_reader(cls, r, where):
        c = cls(*cls._common(r, where), r.number("softcap"))
        if c.vdim != c.dim:
            raise ConfigError(f"config.json: {where}: the values are the keys, so vdim must be dim")
        if c.softcap is not None:
            _positive(where + ".", softcap=c.softcap)
        return c

    def to_dict(self):
        d = super().to_dict()
        if self.softcap is not None:
            d["softcap"] = self.softcap
        return d


MIXERS = {"attention": DifferenceConfig, "attention_2": KeyValueConfig}


@dataclass(frozen=True)
class FigalornLayer:
    type: str
    mixer: object
    ff: Optional[int]                       # of the dense feed-forward; None: the layer has none

    def to_dict(self):
        return {"type": self.type, "mixer": self.mixer.to_dict(),
                "mlp": None if self.ff is None else {"kind": "dense", "ff": self.ff}}


@dataclass(frozen=True)
class Loop:
    """Layers start .. stop - 1 run `times` times in a row with the same weights."""
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class FigalornConfig:
    vocab_size: int
    hidden_size: int
    layers: Tuple[FigalornLayer, ...]
    norm_eps: float
    loop: Optional[Loop] = None
    eos_token_id: Optional[int] = None
    max_position_embeddings: int = MAX_POSITIONS

    @property
    def num_hidden_layers(self):
        return len(self.layers)

    @staticmethod
    def from_dict(raw):
        r = Reader(raw)
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            raise ConfigError("config.json: layers must be a list with at least one layer")
        layers = []
        for i, entry in enumerate(listed):
            where = f"layers[{i}]"
            if not isinstance(entry, dict):
                raise ConfigError(f"config.json: {where} must be an object")
            kind = entry.get("type")
            if kind not in MIXERS:
                raise ConfigError(f"config.json: {where}: unknown layer type {kind!r} (known: {', '.join(sorted(MIXERS))})")
            mixer = MIXERS[kind].from_reader(_section(entry, "mixer", where + "."), where + ".mixer")
            ff = None
            if entry.get("mlp") is not None:
                m = _section(entry, "mlp", where + ".")
                if m.raw.get("kind") != "dense":
                    raise ConfigError(f"config.json: {where}.mlp: unknown feed-forward kind {m.raw.get('kind')!r} (known: 'dense')")
                ff = m.integer("ff", required=True)
                _positive(where + ".mlp.", ff=ff)
            layers.append(FigalornLayer(kind, mixer, ff))
        loop = None
        if raw.get("loop") is not None:
            section = _section(raw, "loop", "")
            loop = Loop(*(section.integer(k, required=True) for k in ("start", "stop", "times")))
            if not 0 <= loop.start < loop.stop <= len(layers) or loop.times < 1:
                raise ConfigError(f"config.json: loop: layers {loop.start} .. {loop.stop - 1} of {len(layers)}, {loop.times} times")
        cfg = FigalornConfig(r.integer("vocab", required=True), r.integer("width", required=True), tuple(layers),
                             _section(raw, "norm", "").number("eps", required=True), loop, r.integer("eos_token_id"))
        _positive("", vocab=cfg.vocab_size, width=cfg.hidden_size)
        return cfg

    def to_dict(self):
        d = {"architecture": "Figalorn", "vocab": self.vocab_size, "width": self.hidden_size,
             "layers": [layer.to_dict() for layer in self.layers], "norm": {"eps": self.norm_eps}}
        if self.loop is not None:
            d["loop"] = {"start": self.loop.start, "stop": self.loop.stop, "times": self.loop.times}
        if self.eos_token_id is not None:
            d["eos_token_id"] = self.eos_token_id
        return d
