"""Typed configuration of Bilolix, read from the design's own config.json keys.

A Bilolix file names its design under ``architecture`` (one string), gives ``vocab``, ``width``, ``norm.eps``, a list
``layers`` and, optionally, ``loop`` (``start``, ``stop``, ``times``: the layers ``start .. stop - 1`` run ``times`` times in
a row with the same weights, each pass with a cache of its own and a vector of its own added to the stream before it).
Each entry of ``layers`` has a ``type`` (the kind of its mixer), the mixer's sizes and constants under ``mixer`` and its
feed-forward under ``mlp`` (null: none).

    mixer (type "attention"):      heads, kv_heads, dim, vdim, scale, diff, rot {base, dims}?, mask {size}?
    mixer (type "gla"):            heads, dim, vdim, tau, rank?
    mixer (type "channel_delta"):  heads, kv_heads, dim, vdim, conv, rank?, gate_rank?
    mlp (kind "dense"):            ff
    mlp (kind "moe"):              router {experts, top}, expert {ff}

Some sizes have no key of their own in files that other tools write: the widths of the bottlenecks through which decays
(``rank``) and a gate (``gate_rank``) are made are the row counts of the stored tensors ``l<i>.mix.a1`` and
``l<i>.mix.g1``; :func:`complete` reads them from there before the keys are parsed.  Files written from here carry them.

As with the other architectures an unknown key is an error that names the key (a key this reader does not know would
be a mechanism it does not compute); a key whose value is null counts as left out.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Optional, Tuple

from ..errors import ConfigError
from .fazezen import DEFAULT_MAX_POSITION, _int, _num
from .togalorn import LoopConfig

ARCHITECTURE = "Bilolix"
ATTENTION = "attention"
GLA = "gla"
CHANNEL_DELTA = "channel_delta"
DENSE = "dense"
MOE = "moe"

# keys that describe provenance, read by nobody
_IGNORED = frozenset({"seed", "name", "description", "comment", "dtype", "torch_dtype"})


def _section(raw, where: str, required, optional=()):
    """``raw`` as a dictionary holding exactly the ``required`` keys and any of the ``optional`` ones."""
    if not isinstance(raw, dict):
        raise ConfigError(f"{where} must be an object, found {raw!r}", key=where)
    known = set(required) | set(optional) | _IGNORED
    for k, v in raw.items():
        if k not in known and v is not None:
            raise ConfigError(f"unsupported key {k!r} in {where} (no Bilolix feature declares it)", key=f"{where}.{k}")
    for k in required:
        if raw.get(k) is None:
            raise ConfigError(f"{where} lacks the required key {k!r}", key=f"{where}.{k}")
    return raw


def _shared_heads(heads: int, kv_heads: int) -> None:
    if heads % kv_heads:
        raise ConfigError("heads must be a multiple of kv_heads", heads=heads, kv_heads=kv_heads)


def _rank(raw, key: str, where: str) -> int:
    if raw.get(key) is None:
        raise ConfigError(f"{where}.{key} is not given and no stored tensor tells it", key=f"{where}.{key}")
    return _int(raw, key, where)


@dataclass(frozen=True)
class PairTurn:
    """Rotary positions over the first ``dims`` features of a map, neighbouring features a pair."""

    base: float
    dims: int


@dataclass(frozen=True)
class MapAttentionConfig:
    """Softmax attention as the difference of two maps over one value row: ``o1 - lam o2``, ``diff`` the constant in ``lam``."""

    heads: int
    kv_heads: int
    dim: int              # features of one map's query and key
    vdim: int
    scale: float
    diff: float
    rot: Optional[PairTurn] = None
    window: Optional[int] = None

    def __post_init__(self):
        _shared_heads(self.heads, self.kv_heads)

    @staticmethod
    def from_dict(raw, where: str) -> "MapAttentionConfig":
        _section(raw, where, ("heads", "kv_heads", "dim", "vdim", "scale", "diff"), ("rot", "mask"))
        dim, rot, window = _int(raw, "dim", where), None, None
        if raw.get("rot") is not None:
            r = _section(raw["rot"], where + ".rot", ("base", "dims"))
            dims = _int(r, "dims", where + ".rot", least=0)
            if dims % 2 or dims > dim:
                raise ConfigError(f"{where}.rot.dims must be even and at most a map's {dim} features", key=where + ".rot.dims")
            rot = PairTurn(_num(r, "base", where + ".rot", positive=True), dims) if dims else None
        if raw.get("mask") is not None:
            mask = _section(raw["mask"], where + ".mask", (), ("size",))
            window = None if mask.get("size") is None else _int(mask, "size", where + ".mask")
        return MapAttentionConfig(_int(raw, "heads", where), _int(raw, "kv_heads", where), dim, _int(raw, "vdim", where),
                                  _num(raw, "scale", where), _num(raw, "diff", where), rot, window)

    def to_json(self) -> dict:
        return {"diff": self.diff, "dim": self.dim, "heads": self.heads, "kv_heads": self.kv_heads,
                "mask": None if self.window is None else {"size": self.window},
                "rot": None if self.rot is None else {"base": self.rot.base, "dims": self.rot.dims}, "scale": self.scale,
                "vdim": self.vdim}


@dataclass(frozen=True)
class FadingConfig:
    """Linear attention with a decay per key channel."""

    heads: int
    dim: int
    vdim: int
    tau: float
    rank: int             # features between the two products that make the decays

    @staticmethod
    def from_dict(raw, where: str) -> "FadingConfig":
        _section(raw, where, ("heads", "dim", "vdim", "tau"), ("rank",))
        return FadingConfig(_int(raw, "heads", where), _int(raw, "dim", where), _int(raw, "vdim", where),
                            _num(raw, "tau", where, positive=True), _rank(raw, "rank", where))

    def to_json(self) -> dict:
        return {"dim": self.dim, "heads": self.heads, "rank": self.rank, "tau": self.tau, "vdim": self.vdim}


@dataclass(frozen=True)
class ChannelDeltaConfig:
    """The gated delta rule with a decay per key channel and a gate through a bottleneck."""

    heads: int
    kv_heads: int         # heads of q and k
    dim: int
    vdim: int
    conv: int             # taps of the convolutions over q, k and v
    rank: int             # features between the two products that make the decays
    gate_rank: int        # and between those that make the gate

    def __post_init__(self):
        _shared_heads(self.heads, self.kv_heads)

    @staticmethod
    def from_dict(raw, where: str) -> "ChannelDeltaConfig":
        sizes = ("heads", "kv_heads", "dim", "vdim", "conv")
        _section(raw, where, sizes, ("rank", "gate_rank"))
        return ChannelDeltaConfig(*(_int(raw, k, where) for k in sizes), _rank(raw, "rank", where),
                                  _rank(raw, "gate_rank", where))

    def to_json(self) -> dict:
        return {"conv": self.conv, "dim": self.dim, "gate_rank": self.gate_rank, "heads": self.heads,
                "kv_heads": self.kv_heads, "rank": self.rank, "vdim": self.vdim}


@dataclass(frozen=True)
class GeluFFConfig:
    ff: int

    def to_json(self) -> dict:
        return {"ff": self.ff, "kind": DENSE}


@dataclass(frozen=True)
class SoftmaxMoEConfig:
    experts: int
    top: int
    ff: int

    def __post_init__(self):
        if self.top > self.experts:
            raise ConfigError("top exceeds the number of experts", top=self.top, experts=self.experts)

    def to_json(self) -> dict:
        return {"expert": {"ff": self.ff}, "kind": MOE, "router": {"experts": self.experts, "top": self.top}}


def _mlp(raw, where: str):
    if raw is None:
        return None
    if not isinstance(raw, dict) or raw.get("kind") not in (DENSE, MOE):
        raise ConfigError(f"{where}.kind must be {DENSE!r} or {MOE!r}", key=where + ".kind")
    if raw["kind"] == DENSE:
        _section(raw, where, ("kind", "ff"))
        return GeluFFConfig(_int(raw, "ff", where))
    _section(raw, where, ("kind", "router", "expert"))
    r = _section(raw["router"], where + ".router", ("experts", "top"))
    e = _section(raw["expert"], where + ".expert", ("ff",))
    return SoftmaxMoEConfig(_int(r, "experts", where + ".router"), _int(r, "top", where + ".router"),
                            _int(e, "ff", where + ".expert"))


_MIXERS = {ATTENTION: MapAttentionConfig, GLA: FadingConfig, CHANNEL_DELTA: ChannelDeltaConfig}


@dataclass(frozen=True)
class BilolixLayer:
    type: str
    mixer: object                    # MapAttentionConfig | FadingConfig | ChannelDeltaConfig
    mlp: Optional[object]            # GeluFFConfig | SoftmaxMoEConfig | None

    def __post_init__(self):
        if not isinstance(self.mixer, _MIXERS.get(self.type, ())):
            raise ConfigError(f"a layer of type {self.type!r} needs that type's mixer", known=sorted(_MIXERS))


@dataclass(frozen=True)
class BilolixConfig:
    vocab: int
    width: int
    layers: Tuple[BilolixLayer, ...]
    norm_eps: float = 1e-6
    loop: Optional[LoopConfig] = None
    # not a key of the file (and no part of what makes two configurations equal): what the rotation tables are made for
    max_position: int = field(default=DEFAULT_MAX_POSITION, compare=False)

    def __post_init__(self):
        if self.vocab < 1 or self.width < 1:
            raise ConfigError("vocab and width must be positive", vocab=self.vocab, width=self.width)
        if not self.layers:
            raise ConfigError("a model has at least one layer")
        if not self.norm_eps > 0:
            raise ConfigError("norm.eps must be a positive number", eps=self.norm_eps)
        if self.loop is not None:
            lp = self.loop
            if not (0 <= lp.start < lp.stop <= len(self.layers)) or lp.times < 1:
                raise ConfigError("loop must name a run of layers and a positive number of passes", start=lp.start,
                                  stop=lp.stop, times=lp.times, layers=len(self.layers))

    @staticmethod
    def from_dict(raw: dict) -> "BilolixConfig":
        top = "config.json"
        _section(raw, top, ("architecture", "vocab", "width", "layers", "norm"), ("architectures", "loop"))
        if raw["architecture"] != ARCHITECTURE:
            raise ConfigError(f"architecture is {raw['architecture']!r}, this reader takes {ARCHITECTURE!r}")
        norm = _section(raw["norm"], "norm", ("eps",))
        loop = None
        if raw.get("loop") is not None:
            lp = _section(raw["loop"], "loop", ("start", "stop", "times"))
            loop = LoopConfig(_int(lp, "start", "loop", least=0), _int(lp, "stop", "loop"), _int(lp, "times", "loop"))
        if not isinstance(raw["layers"], list):
            raise ConfigError("layers must be a list", key="layers")
        layers = []
        for i, entry in enumerate(raw["layers"]):
            where = f"layers[{i}]"
            _section(entry, where, ("type", "mixer"), ("mlp",))
            if entry["type"] not in _MIXERS:
                raise ConfigError(f"{where}.type = {entry['type']!r}: Bilolix has {sorted(_MIXERS)}", key=where + ".type")
            mixer = _MIXERS[entry["type"]].from_dict(entry["mixer"], where + ".mixer")
            layers.append(BilolixLayer(entry["type"], mixer, _mlp(entry.get("mlp"), where + ".mlp")))
        return BilolixConfig(vocab=_int(raw, "vocab", top), width=_int(raw, "width", top), layers=tuple(layers),
                             norm_eps=_num(norm, "eps", "norm", True), loop=loop)

    def to_json(self) -> dict:
        return {"architecture": ARCHITECTURE,
                "layers": [{"mixer": L.mixer.to_json(), "mlp": None if L.mlp is None else L.mlp.to_json(), "type": L.type}
                           for L in self.layers],
                "loop": None if self.loop is None else self.loop.to_json(), "norm": {"eps": self.norm_eps},
                "vocab": self.vocab, "width": self.width}


# the sizes that only stored tensors tell: layer type -> (key, tensor whose row count it is)
_FROM_TENSORS = {GLA: (("rank", "a1"),), CHANNEL_DELTA: (("rank", "a1"), ("gate_rank", "g1"))}


def complete(raw: dict, shape_of) -> dict:
    """The file's keys with the bottlenecks' widths filled in from the stored tensors, where the file does not give them."""
    layers = raw.get("layers")
    if not isinstance(layers, list):
        return raw
    out = copy.deepcopy(raw)
    for i, entry in enumerate(out["layers"]):
        mixer = entry.get("mixer") if isinstance(entry, dict) else None
        if not isinstance(mixer, dict) or not isinstance(entry.get("type"), str):
            continue
        for key, tensor in _FROM_TENSORS.get(entry["type"], ()):
            if mixer.get(key) is None:
                shape = shape_of(f"l{i}.mix.{tensor}")
                if shape is not None and len(shape) == 2:
                    mixer[key] = int(shape[0])
    return out
