"""Typed configuration of Vakesun, read from the design's own config.json keys.

A Vakesun file names its design under ``architecture`` (one string), gives ``vocab``, ``width``, ``embedding.scale``,
``norm.eps``, ``residual_mult``, ``token_side.dim`` (the features a token brings to every layer; null or absent: none) and a
list ``layers``; each entry has a ``type`` (the kind of its mixer), the mixer's sizes and constants under ``mixer`` and its
feed-forward under ``mlp`` (null: none).

    mixer (type "attention"):         heads, kv_heads, dim, vdim, scale,
                                      rot {base, dims, scaling {factor, original, fast, slow}?}?
    mixer (type "mlstm"):             heads, dim, vdim, gate_cap
    mixer (type "latent_attention"):  heads, dim, vdim, scale, q_rank?, kv_rank?, mask {size}?, kv_from?
    mlp   (kind "dense"):             ff

``kv_from`` is the index of an earlier layer of that type whose cached latent rows this layer attends over.  Ranks that the
file does not give are the stored tensors' shapes (:func:`complete`).

As with the other architectures an unknown key is an error that names the key (a key this reader does not know would
be a mechanism it does not compute); a key whose value is null counts as left out.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Optional, Tuple

from ..errors import ConfigError
from .fazezen import _int, _num
from .makuzen import DEFAULT_MAX_POSITION, YarnScaling

ARCHITECTURE = "Vakesun"
ATTENTION = "attention"
MLSTM = "mlstm"
LATENT = "latent_attention"
DENSE = "dense"

# keys that describe provenance, read by nobody
_IGNORED = frozenset({"seed", "name", "description", "comment", "dtype", "torch_dtype"})


def _section(raw, where: str, required, optional=()):
    """``raw`` as a dictionary holding exactly the ``required`` keys and any of the ``optional`` ones."""
    if not isinstance(raw, dict):
        raise ConfigError(f"{where} must be an object, found {raw!r}", key=where)
    known = set(required) | set(optional) | _IGNORED
    for k, v in raw.items():
        if k not in known and v is not None:
            raise ConfigError(f"unsupported key {k!r} in {where} (no Vakesun feature declares it)", key=f"{where}.{k}")
    for k in required:
        if raw.get(k) is None:
            raise ConfigError(f"{where} lacks the required key {k!r}", key=f"{where}.{k}")
    return raw


@dataclass(frozen=True)
class YarnTurn:
    """Rotary positions over the first ``dims`` features of a head, feature ``i`` with ``i + dims / 2``."""

    base: float
    dims: int
    scaling: Optional[YarnScaling] = None

    @staticmethod
    def from_dict(raw, where: str, head: int) -> Optional["YarnTurn"]:
        if raw is None:
            return None
        _section(raw, where, ("base", "dims"), ("scaling",))
        dims = _int(raw, "dims", where, least=0)
        if dims % 2 or dims > head:
            raise ConfigError(f"{where}.dims must be even and at most a head's {head} features", key=where + ".dims")
        scaling = None
        if raw.get("scaling") is not None:
            w = where + ".scaling"
            s = _section(raw["scaling"], w, ("factor", "original", "fast", "slow"))
            scaling = YarnScaling(*(_num(s, k, w, True) for k in ("factor", "original", "fast", "slow")))
        base = _num(raw, "base", where, positive=True)
        if scaling is not None and base == 1.0:
            raise ConfigError(f"{where}.base must not be 1: its logarithm divides", key=where + ".base")
        return YarnTurn(base, dims, scaling) if dims else None

    def to_json(self) -> dict:
        return {"base": self.base, "dims": self.dims, "scaling": None if self.scaling is None else self.scaling.to_json()}


@dataclass(frozen=True)
class GroupedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Optional[YarnTurn] = None

    def __post_init__(self):
        if self.heads % self.kv_heads:
            raise ConfigError("heads must be a multiple of kv_heads", heads=self.heads, kv_heads=self.kv_heads)

    @staticmethod
    def from_dict(raw, where: str) -> "GroupedAttentionConfig":
        _section(raw, where, ("heads", "kv_heads", "dim", "vdim", "scale"), ("rot",))
        dim = _int(raw, "dim", where)
        return GroupedAttentionConfig(_int(raw, "heads", where), _int(raw, "kv_heads", where), dim, _int(raw, "vdim", where),
                                      _num(raw, "scale", where), YarnTurn.from_dict(raw.get("rot"), where + ".rot", dim))

    def to_json(self) -> dict:
        return {"dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads,
                "rot": None if self.rot is None else self.rot.to_json(), "scale": self.scale, "vdim": self.vdim}


@dataclass(frozen=True)
class MatrixMemoryConfig:
    heads: int
    dim: int
    vdim: int
    gate_cap: float

    @staticmethod
    def from_dict(raw, where: str) -> "MatrixMemoryConfig":
        _section(raw, where, ("heads", "dim", "vdim", "gate_cap"))
        return MatrixMemoryConfig(*(_int(raw, k, where) for k in ("heads", "dim", "vdim")), _num(raw, "gate_cap", where, True))

    def to_json(self) -> dict:
        return {"dim": self.dim, "gate_cap": self.gate_cap, "heads": self.heads, "vdim": self.vdim}


@dataclass(frozen=True)
class SinkLatentConfig:
    """Latent attention without positions, with a sink a head; ``kv_from``: the layer whose latent rows it reads."""

    heads: int
    dim: int
    vdim: int
    scale: float
    q_rank: int
    kv_rank: int
    window: Optional[int] = None
    kv_from: Optional[int] = None

    @staticmethod
    def from_dict(raw, where: str) -> "SinkLatentConfig":
        _section(raw, where, ("heads", "dim", "vdim", "scale"), ("q_rank", "kv_rank", "mask", "kv_from"))
        for k in ("q_rank", "kv_rank"):
            if raw.get(k) is None:
                raise ConfigError(f"{where}.{k} is not given and no stored tensor tells it", key=f"{where}.{k}")
        window = kv_from = None
        if raw.get("mask") is not None:
            mask = _section(raw["mask"], where + ".mask", (), ("size",))
            window = None if mask.get("size") is None else _int(mask, "size", where + ".mask")
        if raw.get("kv_from") is not None:
            kv_from = _int(raw, "kv_from", where, least=0)
        return SinkLatentConfig(*(_int(raw, k, where) for k in ("heads", "dim", "vdim")), _num(raw, "scale", where),
                                _int(raw, "q_rank", where), _int(raw, "kv_rank", where), window, kv_from)

    def to_json(self) -> dict:
        out = {"dim": self.dim, "heads": self.heads, "kv_rank": self.kv_rank,
               "mask": None if self.window is None else {"size": self.window}, "q_rank": self.q_rank, "scale": self.scale,
               "vdim": self.vdim}
        if self.kv_from is not None:
            out["kv_from"] = self.kv_from
        return out


@dataclass(frozen=True)
class SquaredReluConfig:
    ff: int

    @staticmethod
    def from_dict(raw, where: str) -> Optional["SquaredReluConfig"]:
        if raw is None:
            return None
        _section(raw, where, ("kind", "ff"))
        if raw["kind"] != DENSE:
            raise ConfigError(f"{where}.kind = {raw['kind']!r}: Vakesun's feed-forward is {DENSE!r}", key=where + ".kind")
        return SquaredReluConfig(_int(raw, "ff", where))

    def to_json(self) -> dict:
        return {"ff": self.ff, "kind": DENSE}


_MIXERS = {ATTENTION: GroupedAttentionConfig, MLSTM: MatrixMemoryConfig, LATENT: SinkLatentConfig}


@dataclass(frozen=True)
class VakesunLayer:
    type: str
    mixer: object                    # GroupedAttentionConfig | MatrixMemoryConfig | SinkLatentConfig
    mlp: Optional[SquaredReluConfig]

    def __post_init__(self):
        if not isinstance(self.mixer, _MIXERS.get(self.type, ())):
            raise ConfigError(f"a layer of type {self.type!r} needs that type's mixer", known=sorted(_MIXERS))


@dataclass(frozen=True)
class VakesunConfig:
    vocab: int
    width: int
    layers: Tuple[VakesunLayer, ...]
    embedding_scale: float = 1.0
    norm_eps: float = 1e-6
    residual_mult: float = 1.0
    side_dim: Optional[int] = None
    # not a key of the file (and no part of what makes two configurations equal): what the rotation tables are made for
    max_position: int = field(default=DEFAULT_MAX_POSITION, compare=False)

    def __post_init__(self):
        if self.vocab < 1 or self.width < 1:
            raise ConfigError("vocab and width must be positive", vocab=self.vocab, width=self.width)
        if not self.layers:
            raise ConfigError("a model has at least one layer")
        if not self.norm_eps > 0:
            raise ConfigError("norm.eps must be a positive number", eps=self.norm_eps)
        for i, layer in enumerate(self.layers):
            j = getattr(layer.mixer, "kv_from", None)
            if j is None:
                continue
            where = f"layers[{i}].mixer.kv_from"
            if not 0 <= j < i or self.layers[j].type != LATENT:
                raise ConfigError(f"{where} = {j} is no earlier layer of type {LATENT!r}", key=where)
            src = self.layers[j].mixer
            if src.kv_from is not None:
                raise ConfigError(f"{where} = {j}: that layer makes no latent rows of its own", key=where)
            if src.kv_rank != layer.mixer.kv_rank:
                raise ConfigError(f"{where} = {j}: latent rows of {src.kv_rank} features are read as {layer.mixer.kv_rank}", key=where)

    @staticmethod
    def from_dict(raw: dict) -> "VakesunConfig":
        top = "config.json"
        _section(raw, top, ("architecture", "vocab", "width", "layers", "norm"),
                 ("architectures", "embedding", "residual_mult", "token_side"))
        if raw["architecture"] != ARCHITECTURE:
            raise ConfigError(f"architecture is {raw['architecture']!r}, this reader takes {ARCHITECTURE!r}")
        norm = _section(raw["norm"], "norm", ("eps",))
        scale, mult, side = 1.0, 1.0, None
        if raw.get("embedding") is not None:
            scale = _num(_section(raw["embedding"], "embedding", ("scale",)), "scale", "embedding")
        if raw.get("residual_mult") is not None:
            mult = _num(raw, "residual_mult", top)
        if raw.get("token_side") is not None:
            side = _int(_section(raw["token_side"], "token_side", ("dim",)), "dim", "token_side")
        if not isinstance(raw["layers"], list):
            raise ConfigError("layers must be a list", key="layers")
        layers = []
        for i, entry in enumerate(raw["layers"]):
            where = f"layers[{i}]"
            _section(entry, where, ("type", "mixer"), ("mlp",))
            if entry["type"] not in _MIXERS:
                raise ConfigError(f"{where}.type = {entry['type']!r}: Vakesun has {sorted(_MIXERS)}", key=where + ".type")
            mixer = _MIXERS[entry["type"]].from_dict(entry["mixer"], where + ".mixer")
            layers.append(VakesunLayer(entry["type"], mixer, SquaredReluConfig.from_dict(entry.get("mlp"), where + ".mlp")))
        return VakesunConfig(vocab=_int(raw, "vocab", top), width=_int(raw, "width", top), layers=tuple(layers),
                             embedding_scale=scale, norm_eps=_num(norm, "eps", "norm", True), residual_mult=mult, side_dim=side)

    def to_json(self) -> dict:
        return {"architecture": ARCHITECTURE, "embedding": {"scale": self.embedding_scale},
                "layers": [{"mixer": L.mixer.to_json(), "mlp": None if L.mlp is None else L.mlp.to_json(), "type": L.type}
                           for L in self.layers],
                "norm": {"eps": self.norm_eps}, "residual_mult": self.residual_mult,
                "token_side": None if self.side_dim is None else {"dim": self.side_dim}, "vocab": self.vocab, "width": self.width}


def complete(raw: dict, shape_of) -> dict:
    """The file's keys with the latent mixers' ranks filled in from the stored tensors, where the file does not give them."""
    layers = raw.get("layers")
    if not isinstance(layers, list):
        return raw
    out = copy.deepcopy(raw)
    for i, entry in enumerate(out["layers"]):
        mixer = entry.get("mixer") if isinstance(entry, dict) and entry.get("type") == LATENT else None
        if not isinstance(mixer, dict):
            continue
        for key, tensor, axis in (("q_rank", "dq", 0), ("kv_rank", "uk", 1)):
            if mixer.get(key) is None:
                shape = shape_of(f"l{i}.mix.{tensor}")
                if shape is not None and len(shape) == 2:
                    mixer[key] = int(shape[axis])
    return out
