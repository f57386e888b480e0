"""Rirovik's typed configuration, read from the keys of its own config.json.

    architecture     "Rirovik"
    vocab, width     sizes of the token table and of the residual stream
    embedding.scale  factor on the token table's rows
    norm.eps         the epsilon of every RMS norm of the model (layers, latents, heads, final)
    layers           a list; each entry has ``type``, ``mixer`` and ``mlp``:
        type "attention"           mixer {heads, kv_heads, dim, vdim, scale, mask}
        type "latent_attention"    mixer {heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, rot, mask, kv_from}, an output
                                   gate per head
        type "latent_attention_2"  the same without the gate
        rot                        {base, dims}; needed where rot_dim is not zero, which dims must equal
        mask                       null / absent: every earlier position is seen; else {size, keep_first}: the latest ``size``
                                   positions and, with keep_first, the first so many of the sequence
        kv_from                    null / absent, or the number of an EARLIER latent layer with a latent of its own, of the
                                   same kv_rank, rot_dim and rotation, whose cached latent this layer attends over
        mlp                        null, or {kind: "moe", expert {ff}, router {experts, top}, shared: null or {ff}}
"""

from dataclasses import dataclass
from typing import Optional, Tuple, Union

from .base import ConfigError, MAX_LAYERS, positive_extent, positive_finite, take

FAMILY = "rirovik"
MIXERS = ("attention", "latent_attention", "latent_attention_2")


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
    value = data.get(field) if isinstance(data, dict) else None
    if not isinstance(value, dict):
        raise ConfigError(FAMILY, f"{where}.{field}" if where else field, "must be an object")
    return value


@dataclass(frozen=True)
class Mask:
    size: int
    keep_first: int

    def to_dict(self):
        return {"keep_first": self.keep_first, "size": self.size} if self.keep_first else {"size": self.size}


@dataclass(frozen=True)
class AttentionSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    mask: Optional[Mask]

    def to_dict(self):
        return {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads, "mask": self.mask.to_dict() if self.mask else None,
                "scale": self.scale, "vdim": self.vdim}


@dataclass(frozen=True)
class LatentSizes:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float                              # 0: nothing is turned (rot_dim is zero)
    mask: Optional[Mask]
    kv_from: Optional[int]

    def to_dict(self):
        data = {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank, "q_rank": self.q_rank, "rot_dim": self.rot_dim,
                "rot": {"base": self.rot_base, "dims": self.rot_dim} if self.rot_dim else None, "scale": self.scale, "vdim": self.vdim,
                "mask": self.mask.to_dict() if self.mask else None}
        if self.kv_from is not None:
            data["kv_from"] = self.kv_from
        return data


@dataclass(frozen=True)
class ExpertSizes:
    experts: int
    ff: int
    top: int
    shared_ff: int                               # 0: no expert that every token uses

    def to_dict(self):
        return {"expert": {"ff": self.ff}, "kind": "moe", "router": {"experts": self.experts, "top": self.top},
                "shared": {"ff": self.shared_ff} if self.shared_ff else None}


@dataclass(frozen=True)
class RirovikLayer:
    type: str
    mixer: Union[AttentionSizes, LatentSizes]
    mlp: Optional[ExpertSizes]

    @property
    def gated(self):
        """Whether a latent attention's heads have an output gate (attention always has one per channel)."""
        return self.type != "latent_attention_2"

    def to_dict(self):
        return {"mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp else None, "type": self.type}


def _mask(m, at):
    mask = _optional(m, "mask", at)
    if not mask:
        return None
    return Mask(_need(mask, "size", int, f"{at}.mask"), take(mask, FAMILY, f"{at}.mask.keep_first", int, 0, ("keep_first",)))


def _mixer(kind, m, at):
    if kind == "attention":
        return AttentionSizes(heads=_need(m, "heads", int, at), kv_heads=_need(m, "kv_heads", int, at), dim=_need(m, "dim", int, at),
                              vdim=_need(m, "vdim", int, at), scale=_need(m, "scale", float, at), mask=_mask(m, at))
    rot_dim = take(m, FAMILY, f"{at}.rot_dim", int, 0, ("rot_dim",))
    base = 0.0
    if rot_dim:
        rot = _object(m, "rot", at)
        base = _need(rot, "base", float, f"{at}.rot")
        if take(rot, FAMILY, f"{at}.rot.dims", int, rot_dim, ("dims",)) != rot_dim:
            raise ConfigError(FAMILY, f"{at}.rot.dims", "must equal rot_dim")
    return LatentSizes(
        heads=_need(m, "heads", int, at), dim=_need(m, "dim", int, at), rot_dim=rot_dim, vdim=_need(m, "vdim", int, at),
        q_rank=_need(m, "q_rank", int, at), kv_rank=_need(m, "kv_rank", int, at), scale=_need(m, "scale", float, at),
        rot_base=base, mask=_mask(m, at), kv_from=take(m, FAMILY, f"{at}.kv_from", int, None, ("kv_from",)))


def _mlp(mlp, at):
    if mlp is None:
        return None
    kind = _need(mlp, "kind", str, at)
    if kind != "moe":
        raise ConfigError(FAMILY, f"{at}.kind", f"unknown feed-forward `{kind}`, expected `moe`")
    expert, router, shared = _object(mlp, "expert", at), _object(mlp, "router", at), _optional(mlp, "shared", at)
    return ExpertSizes(experts=_need(router, "experts", int, f"{at}.router"), ff=_need(expert, "ff", int, f"{at}.expert"),
                       top=_need(router, "top", int, f"{at}.router"),
                       shared_ff=_need(shared, "ff", int, f"{at}.shared") if shared else 0)


@dataclass(frozen=True)
class RirovikConfig:
    vocab: int
    width: int
    embedding_scale: float
    norm_eps: float
    layers: Tuple[RirovikLayer, ...]

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
            layers.append(RirovikLayer(kind, mixer, _mlp(_optional(entry, "mlp", where), f"{where}.mlp")))
        embedding = _optional(data, "embedding", "") or {}
        config = cls(vocab=_need(data, "vocab", int, ""), width=_need(data, "width", int, ""),
                     embedding_scale=take(embedding, FAMILY, "embedding.scale", float, 1.0, ("scale",)),
                     norm_eps=_need(_object(data, "norm", ""), "eps", float, "norm"), layers=tuple(layers))
        config.validate()
        return config

    def validate(self):
        positive_extent(FAMILY, "vocab", self.vocab)
        positive_extent(FAMILY, "width", self.width)
        positive_finite(FAMILY, "norm.eps", self.norm_eps)
        if self.embedding_scale != self.embedding_scale or abs(self.embedding_scale) == float("inf"):
            raise ConfigError(FAMILY, "embedding.scale", "must be finite")
        for index, layer in enumerate(self.layers):
            where, m = f"layers[{index}].mixer", layer.mixer
            keys = ("heads", "kv_heads", "dim", "vdim") if layer.type == "attention" else ("heads", "dim", "vdim", "q_rank", "kv_rank")
            for key in keys:
                positive_extent(FAMILY, f"{where}.{key}", getattr(m, key))
            positive_finite(FAMILY, f"{where}.scale", m.scale)
            if m.mask is not None:
                positive_extent(FAMILY, f"{where}.mask.size", m.mask.size)
                if m.mask.keep_first < 0:
                    raise ConfigError(FAMILY, f"{where}.mask.keep_first", "must not be negative")
            if layer.type == "attention":
                if m.heads % m.kv_heads != 0:
                    raise ConfigError(FAMILY, f"{where}.kv_heads", "must divide heads")
            else:
                self._validate_latent(index, m, where)
            e, where = layer.mlp, f"layers[{index}].mlp"
            if e is not None:
                for key, name in (("experts", "router.experts"), ("ff", "expert.ff"), ("top", "router.top")):
                    positive_extent(FAMILY, f"{where}.{name}", getattr(e, key))
                if e.top > e.experts:
                    raise ConfigError(FAMILY, f"{where}.router.top", "must not exceed the experts")
                if e.shared_ff < 0:
                    raise ConfigError(FAMILY, f"{where}.shared.ff", "must be positive")

    def _validate_latent(self, index, m, where):
        if m.rot_dim < 0 or m.rot_dim % 2 != 0:
            raise ConfigError(FAMILY, f"{where}.rot_dim", "must be even")
        if m.rot_dim:
            positive_finite(FAMILY, f"{where}.rot.base", m.rot_base)
        if m.kv_from is None:
            return
        if not 0 <= m.kv_from < index:
            raise ConfigError(FAMILY, f"{where}.kv_from", "must name an earlier layer")
        source = self.layers[m.kv_from]
        if source.type == "attention" or source.mixer.kv_from is not None:
            raise ConfigError(FAMILY, f"{where}.kv_from", f"layer {m.kv_from} keeps no latent of its own")
        for key, name in (("kv_rank", "kv_rank"), ("rot_dim", "rot_dim"), ("rot_base", "rot.base")):
            if getattr(source.mixer, key) != getattr(m, key):
                raise ConfigError(FAMILY, f"{where}.{name}", f"must equal that of layer {m.kv_from}, whose latent is read")

    def to_dict(self):
        return {"architecture": "Rirovik", "embedding": {"scale": self.embedding_scale},
                "layers": [layer.to_dict() for layer in self.layers], "norm": {"eps": self.norm_eps}, "vocab": self.vocab,
                "width": self.width}
