"""Typed configuration of the Mutedra decoder: layers normed before and after each part, listed one by one, each a mixer
(a softmax attention over a window and the first keys with a learned bias by distance, or one of two forms of an
attention over one shared latent a token) and an optional dense feed-forward; a stretch of the layers may run
several times over.

config.json names the design under "architecture"; every size and every constant that can differ between models is
a key here (but the number of a bias table's rows, which the stored table gives), and an unknown layer type or
feed-forward kind is an error. A section that a model leaves out switches its mechanism off: "mask" (the attention
then sees every earlier key), "mask.keep_first", "mlp", "loop", "logit_softcap".
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
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    bias_max: float                         # the distance from which on the last bias holds
    window: Optional[int] = None            # mask.size; None: every earlier key is seen
    keep_first: int = 0                     # keys at the sequence's start that every query sees

    @staticmethod
    def from_reader(r, where):
        window, keep = None, 0
        if r.raw.get("mask") is not None:
            mask = _section(r.raw, "mask", where + ".")
            window, keep = mask.integer("size", required=True), mask.integer("keep_first", 0)
            _positive(where + ".mask.", size=window)
            if keep < 0:
                raise ConfigError(f"config.json: {where}.mask.keep_first must not be negative")
        c = AttentionConfig(*(r.integer(k, required=True) for k in ("heads", "kv_heads", "dim", "vdim")),
                            r.number("scale", required=True), r.number("bias_max", required=True), window, keep)
        _positive(where + ".", heads=c.heads, kv_heads=c.kv_heads, dim=c.dim, vdim=c.vdim, scale=c.scale, bias_max=c.bias_max)
        if c.heads % c.kv_heads:
            raise ConfigError(f"config.json: {where}: heads must be a multiple of kv_heads")
        return c

    def to_dict(self):
        d = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale,
             "bias_max": self.bias_max}
        if self.window is not None:
            d["mask"] = {"size": self.window, "keep_first": self.keep_first}
        return d


@dataclass(frozen=True)
class LatentAttentionConfig:
    heads: int
    dim: int
    vdim: int
    kv_rank: int
    q_rank: int
    scale: float

    @staticmethod
    def from_reader(r, where):
        c = LatentAttentionConfig(*(r.integer(k, required=True) for k in ("heads", "dim", "vdim", "kv_rank", "q_rank")),
                                  r.number("scale", required=True))
        _positive(where + ".", **c.to_dict())
        return c

    def to_dict(self):
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "kv_rank": self.kv_rank, "q_rank": self.q_rank,
                "scale": self.scale}


@dataclass(frozen=True)
class RotatedLatentConfig:
    """A latent attention with a rotated part that every head's key shares, a sink and a gate a head."""
    latent: LatentAttentionConfig
    rot_dim: int
    rot_base: float

    @staticmethod
    def from_reader(r, where):
        rot = _section(r.raw, "rot", where + ".")
        c = RotatedLatentConfig(LatentAttentionConfig.from_reader(r, where), r.integer("rot_dim", required=True),
                                rot.number("base", required=True))
        _positive(where + ".", rot_dim=c.rot_dim)
        _positive(where + ".rot.", base=c.rot_base)
        if rot.integer("dims", required=True) != c.rot_dim or c.rot_dim % 2:
            raise ConfigError(f"config.json: {where}.rot.dims must be rot_dim, and even: the whole rotated part turns in pairs")
        return c

    def to_dict(self):
        return {**self.latent.to_dict(), "rot_dim": self.rot_dim, "rot": {"dims": self.rot_dim, "base": self.rot_base}}


MIXERS = {"attention": AttentionConfig, "latent_attention": LatentAttentionConfig, "latent_attention_2": RotatedLatentConfig}


@dataclass(frozen=True)
class MutedraLayer:
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
class MutedraConfig:
    vocab_size: int
    hidden_size: int
    layers: Tuple[MutedraLayer, ...]
    norm_eps: float
    embedding_scale: float = 1.0
    loop: Optional[Loop] = None
    logit_softcap: Optional[float] = None
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
            layers.append(MutedraLayer(kind, mixer, ff))
        loop = None
        if raw.get("loop") is not None:
            l = _section(raw, "loop", "")
            loop = Loop(*(l.integer(k, required=True) for k in ("start", "stop", "times")))
            if not 0 <= loop.start < loop.stop <= len(layers) or loop.times < 1:
                raise ConfigError(f"config.json: loop: layers {loop.start} .. {loop.stop - 1} of {len(layers)}, {loop.times} times")
        scale = 1.0
        if raw.get("embedding") is not None:
            scale = _section(raw, "embedding", "").number("scale", 1.0)
        cfg = MutedraConfig(r.integer("vocab", required=True), r.integer("width", required=True), tuple(layers),
                            _section(raw, "norm", "").number("eps", required=True), scale, loop,
                            r.number("logit_softcap"), r.integer("eos_token_id"))
        _positive("", vocab=cfg.vocab_size, width=cfg.hidden_size)
        if cfg.logit_softcap is not None:
            _positive("", logit_softcap=cfg.logit_softcap)
        return cfg

    def to_dict(self):
        d = {"architecture": "Mutedra", "vocab": self.vocab_size, "width": self.hidden_size,
             "layers": [l.to_dict() for l in self.layers], "norm": {"eps": self.norm_eps},
             "embedding": {"scale": self.embedding_scale}}
        if self.loop is not None:
            d["loop"] = {"start": self.loop.start, "stop": self.loop.stop, "times": self.loop.times}
        if self.logit_softcap is not None:
            d["logit_softcap"] = self.logit_softcap
        if self.eos_token_id is not None:
            d["eos_token_id"] = self.eos_token_id
        return d
