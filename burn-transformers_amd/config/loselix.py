"""Loselix's typed configuration, read from the keys of its own config.json.

    architecture     "Loselix"
    vocab, width     sizes of the token table and of the residual stream
    norm.eps         the epsilon of every RMS norm of the model (layers, whole projections, heads' differences, final)
    loop             null / absent, or {start, stop, times}: layers start .. stop - 1 run ``times`` times in a row
                     with the same tensors, every run with a cache entry of its own; the embedding's output joins
                     the stream before every pass but the first
    layers           a list; each entry has ``type``, ``mixer`` and ``mlp``:
        type "attention"     mixer {heads, kv_heads, dim, vdim, scale, rot, softcap, diff}: two maps a head
        type "attention_2"   mixer {heads, kv_heads, dim, vdim, scale, rot}: a gate per head
        type "attention_3"   mixer {heads, kv_heads, dim, vdim, scale, q_temp {coef, every}}: sigmoid weights, values
                             that are the keys (vdim = dim), a gate per channel
        rot                  null, or {dims, base}
        mlp                  null, or {kind: "dense", ff}
"""

from dataclasses import dataclass
from typing import Optional, Tuple, Union

from .base import ConfigError, MAX_LAYERS, positive_extent, positive_finite, take

FAMILY = "loselix"
MIXERS = ("attention", "attention_2", "attention_3")


def _need(data, field, kind, where):
    full = f"{where}.{field}" if where else field
    if not isinstance(data, dict) or field not in data or data[field] is None:
        raise ConfigError(FAMILY, full, "is required")
    return take({full: data[field]}, FAMILY, full, kind, None)


def _optional(data, field, where):
    """A nested object that may be absent or null."""
    value = data.get(field) if isinstance(data, dict) else None
    if value is not None and not isinstance(value, dict):
        raise ConfigError(FAMILY, f"{where}.{field}" if where else field, "must be an object or null")
    return value


def _object(data, field, where):
    value = _optional(data, field, where)
    if value is None:
        raise ConfigError(FAMILY, f"{where}.{field}" if where else field, "must be an object")
    return value


@dataclass(frozen=True)
class Rotation:
    dims: int
    base: float

    def to_dict(self):
        return {"base": self.base, "dims": self.dims}


@dataclass(frozen=True)
class DifferentialSizes:
    heads: int
    kv_heads: int
    dim: int                                     # of one map's queries and keys
    vdim: int
    scale: float
    rot: Optional[Rotation]
    softcap: float                               # 0: the scores are not capped
    diff: float

    def to_dict(self):
        return {"diff": self.diff, "dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads,
                "rot": self.rot.to_dict() if self.rot else None, "scale": self.scale, "softcap": self.softcap or None,
                "vdim": self.vdim}


@dataclass(frozen=True)
class HeadGatedSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Optional[Rotation]

    def to_dict(self):
        return {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "rot": self.rot.to_dict() if self.rot else None,
                "scale": self.scale, "vdim": self.vdim}


@dataclass(frozen=True)
class SigmoidSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    temp_coef: float
    temp_every: int                              # 0: no temperature

    def to_dict(self):
        return {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "scale": self.scale, "vdim": self.vdim,
                "q_temp": {"coef": self.temp_coef, "every": self.temp_every} if self.temp_every else None}


@dataclass(frozen=True)
class DenseSizes:
    ff: int

    def to_dict(self):
        return {"ff": self.ff, "kind": "dense"}


@dataclass(frozen=True)
class Loop:
    start: int
    stop: int
    times: int

    def to_dict(self):
        return {"start": self.start, "stop": self.stop, "times": self.times}


@dataclass(frozen=True)
class LoselixLayer:
    type: str
    mixer: Union[DifferentialSizes, HeadGatedSizes, SigmoidSizes]
    mlp: Optional[DenseSizes]

    def to_dict(self):
        return {"mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp else None, "type": self.type}


def _rotation(m, at):
    rot = _optional(m, "rot", at)
    if not rot or not rot.get("dims"):
        return None
    return Rotation(_need(rot, "dims", int, f"{at}.rot"), _need(rot, "base", float, f"{at}.rot"))


def _mixer(kind, m, at):
    sizes = [_need(m, key, int, at) for key in ("heads", "kv_heads", "dim", "vdim")] + [_need(m, "scale", float, at)]
    if kind == "attention":
        return DifferentialSizes(*sizes, _rotation(m, at), take(m, FAMILY, f"{at}.softcap", float, 0.0, ("softcap",)),
                                 _need(m, "diff", float, at))
    if kind == "attention_2":
        return HeadGatedSizes(*sizes, _rotation(m, at))
    temperature, where = _optional(m, "q_temp", at), f"{at}.q_temp"
    return SigmoidSizes(*sizes, _need(temperature, "coef", float, where) if temperature else 0.0,
                        _need(temperature, "every", int, where) if temperature else 0)


def _mlp(mlp, at):
    if mlp is None:
        return None
    kind = _need(mlp, "kind", str, at)
    if kind != "dense":
        raise ConfigError(FAMILY, f"{at}.kind", f"unknown feed-forward `{kind}`, expected `dense`")
    return DenseSizes(_need(mlp, "ff", int, at))


@dataclass(frozen=True)
class LoselixConfig:
    vocab: int
    width: int
    norm_eps: float
    loop: Optional[Loop]
    layers: Tuple[LoselixLayer, ...]

    @classmethod
    def from_dict(cls, data):
        if not isinstance(data.get("layers"), (list, tuple)) or not data["layers"]:
            raise ConfigError(FAMILY, "layers", "must be a list with at least one layer")
        if len(data["layers"]) > MAX_LAYERS:
            raise ConfigError(FAMILY, "layers", f"must not exceed {MAX_LAYERS} entries")
        layers = []
        for index, entry in enumerate(data["layers"]):
            where = f"layers[{index}]"
            if not isinstance(entry, dict):
                raise ConfigError(FAMILY, where, "must be an object")
            kind = _need(entry, "type", str, where)
            if kind not in MIXERS:
                raise ConfigError(FAMILY, f"{where}.type", f"unknown mixer `{kind}`, expected one of " + ", ".join(f"`{m}`" for m in MIXERS))
            mixer = _mixer(kind, _object(entry, "mixer", where), f"{where}.mixer")
            layers.append(LoselixLayer(kind, mixer, _mlp(_optional(entry, "mlp", where), f"{where}.mlp")))
        loop = _optional(data, "loop", "")
        if loop:
            loop = Loop(*(_need(loop, key, int, "loop") for key in ("start", "stop", "times")))
        config = cls(vocab=_need(data, "vocab", int, ""), width=_need(data, "width", int, ""),
                     norm_eps=_need(_object(data, "norm", ""), "eps", float, "norm"), loop=loop or None, layers=tuple(layers))
        config.validate()
        return config

    def validate(self):
        positive_extent(FAMILY, "vocab", self.vocab)
        positive_extent(FAMILY, "width", self.width)
        positive_finite(FAMILY, "norm.eps", self.norm_eps)
        if self.loop is not None:
            if not 0 <= self.loop.start < self.loop.stop <= len(self.layers):
                raise ConfigError(FAMILY, "loop.stop", "start < stop must name layers of the model")
            positive_extent(FAMILY, "loop.times", self.loop.times)
        for index, layer in enumerate(self.layers):
            where, m = f"layers[{index}].mixer", layer.mixer
            for key in ("heads", "kv_heads", "dim", "vdim"):
                positive_extent(FAMILY, f"{where}.{key}", getattr(m, key))
            if m.heads % m.kv_heads != 0:
                raise ConfigError(FAMILY, f"{where}.kv_heads", "must divide heads")
            positive_finite(FAMILY, f"{where}.scale", m.scale)
            rot = getattr(m, "rot", None)
            if rot is not None:
                if rot.dims <= 0 or rot.dims % 2 != 0 or rot.dims > m.dim:
                    raise ConfigError(FAMILY, f"{where}.rot.dims", f"must be even and at most {m.dim}")
                positive_finite(FAMILY, f"{where}.rot.base", rot.base)
            if layer.type == "attention":
                if m.softcap != 0.0:
                    positive_finite(FAMILY, f"{where}.softcap", m.softcap)
                if m.diff != m.diff or abs(m.diff) == float("inf"):
                    raise ConfigError(FAMILY, f"{where}.diff", "must be finite")
            if layer.type == "attention_3":
                if m.vdim != m.dim:
                    raise ConfigError(FAMILY, f"{where}.vdim", "must equal dim: the values are the keys")
                if m.temp_every < 0:
                    raise ConfigError(FAMILY, f"{where}.q_temp.every", "must be positive")
                if m.temp_coef != m.temp_coef or abs(m.temp_coef) == float("inf"):
                    raise ConfigError(FAMILY, f"{where}.q_temp.coef", "must be finite")
            if layer.mlp is not None:
                positive_extent(FAMILY, f"layers[{index}].mlp.ff", layer.mlp.ff)

    def runs(self):
        """[(layer, whether the embedding's output joins the stream before it)] in the order the layers run: the
        looped stretch ``times`` times in a row, entered with that sum from the second pass on."""
        count = len(self.layers)
        if self.loop is None:
            return [(i, False) for i in range(count)]
        order = [(i, False) for i in range(self.loop.start)]
        for number in range(self.loop.times):
            order += [(i, number > 0 and i == self.loop.start) for i in range(self.loop.start, self.loop.stop)]
        return order + [(i, False) for i in range(self.loop.stop, count)]

    def to_dict(self):
        return {"architecture": "Loselix", "layers": [layer.to_dict() for layer in self.layers],
                "loop": self.loop.to_dict() if self.loop else None, "norm": {"eps": self.norm_eps}, "vocab": self.vocab,
                "width": self.width}
