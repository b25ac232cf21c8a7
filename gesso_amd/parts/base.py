"""What every part is: a spec, the tensors it needs, and a forward over flattened tokens.

A part never learns which model holds it.  It is built from its spec (every size and
constant a field) and a :class:`Runtime` (device, dtype, kernels); it names the tensors it
needs by local names (``q_proj.weight``); the block's name table maps those to the names
in the weight file.

Interfaces (duck-typed; the classes below are convenient bases):

* norm            ``tensor_specs(spec)``, ``bind(tensors)``, ``add_norm(stream, rows=None, out=None) -> normed``;
                  optional hint ``row_weight``: a float32 vector ``w`` with ``norm(x) = inv_rms(x) * (x * w)``, which
                  lets whatever writes the stream before the norm leave the rows pre-weighted (None: no such form);
                  optional ``seam()``: the norm in the form that the kernel between two sub-layers takes
                  (``ops.SeamNorm``), for blocks that norm a sub-layer's output as well
* position        ``tensor_specs(spec)`` (usually none), ``bind``, attributes
                  ``cos``, ``sin`` (``(max_position, rotary_dim/2)`` float32), ``rotary_dim`` and ``layout``
                  (``"half"``: pairs ``(i, i + rotary_dim/2)``, ``"interleaved"``: ``(2i, 2i + 1)``);
                  or ``rotary_dim == 0`` for none
* mixer           ``tensor_specs(spec)``, ``cache_need(spec) -> PagedKV | SlotState | None`` or a tuple of these
                  (a mixer made of several, each with a cache of its own: ``cache`` is then a tuple of views),
                  ``bind(tensors)``, ``forward(x, ctx, cache) -> (T, hidden)``
* feed-forward    ``tensor_specs(spec)``, ``bind(tensors)``, ``forward(x, ctx) -> (T, hidden)``
* side input      the same, with ``out_seam()``: the norm its output passes before it is added (a form the seam kernel takes)
* block           ``tensor_specs(spec)``, ``cache_need(spec)``, ``bind``,
                  ``forward(stream, ctx, cache)`` on a :class:`ResidualStream`; optional hint ``first_norm``: the
                  norm that reads the stream first when the block runs (None: unknown)

``Part`` below carries the optional hints with their defaults, so a part derived from it need not mention them.
"""
from __future__ import annotations

from dataclasses import dataclass, replace
from typing import Dict, Optional, Tuple

MATRIX = "matrix"     # operand of a matrix product: keeps the stored width (bfloat16 stays bfloat16)
VECTOR = "vector"     # norm weights, taps, biases: held in float32 (an exact widening)
TABLE = "table"       # embedding table; a matrix that is also gathered from
INDEX = "index"       # a table of integers (which experts a token id uses): held as int32


@dataclass(frozen=True)
class TensorSpec:
    shape: Tuple[int, ...]
    role: str = MATRIX
    init: str = "normal"          # "normal": N(0, std); "one_plus_normal": 1 + N(0, std);
                                  # "distinct": integers below ``high``, those of a row all different
    high: int = 0


@dataclass(frozen=True)
class PagedKV:
    """Per-token state kept in pages: per token and key head a key row of ``head_dim`` and a value row of
    ``value_dim`` numbers (None: as wide as the key; 0: no value rows at all, for a mixer that caches one row per
    token and derives both from it).

    ``window``: only the last ``window`` tokens are ever read again (None = all of them).
    ``chunk``: positions are cut into runs of ``chunk`` from 0 on and a token reads only its own run, so the runs
    before the newest token's are never read again (None = no such cut).
    ``keep_first``: the first positions of a sequence that stay readable when a window has passed them: the pages
    that hold them are never given back while the request lives.
    """

    n_kv_heads: int
    head_dim: int
    window: Optional[int] = None
    value_dim: Optional[int] = None
    chunk: Optional[int] = None
    keep_first: int = 0

    def pages_kept(self, page_size: int) -> int:
        """How many pages at a sequence's start hold positions that stay readable whatever has passed."""
        return -(-int(self.keep_first) // page_size) if self.window is not None and self.chunk is None else 0

    def reaching(self, other: "PagedKV") -> "PagedKV":
        """What a cache must keep so that ``other``'s reader, too, finds every row it may see: the rows' shape is this
        cache's (``other`` must agree), the reach the wider of the two."""
        if (self.n_kv_heads, self.head_dim, self.value_width) != (other.n_kv_heads, other.head_dim, other.value_width):
            raise ValueError(f"a reader of rows {other} cannot share a cache of {self}")
        if self.chunk != other.chunk:
            raise ValueError("readers of one cache cut their positions into the same runs, or none does")
        window = None if self.window is None or other.window is None else max(self.window, other.window)
        keep = max(self.keep_first, other.keep_first) if window is not None else 0
        return replace(self, window=window, keep_first=keep)

    def first_needed(self, length: int) -> int:
        """The oldest position that the token after ``length`` cached ones can read."""
        first = 0
        if self.window is not None:
            first = max(first, length - self.window + 1)
        if self.chunk is not None:
            first = max(first, length - length % self.chunk)
        return first

    @property
    def value_width(self) -> int:
        return self.head_dim if self.value_dim is None else int(self.value_dim)


@dataclass(frozen=True)
class SlotState:
    """Per-request state of fixed size.  ``tensors``: ``(name, shape, dtype name)`` or ``(name, shape, dtype name,
    initial value)`` each; ``dtype name`` is ``"float32"`` or ``"bfloat16"``; a slot handed to a request is filled
    with the initial value (0 unless given)."""

    tensors: Tuple[tuple, ...]

    def entries(self):
        """``(name, shape, dtype name, initial value)`` of every tensor."""
        out = []
        for t in self.tensors:
            if len(t) not in (3, 4):
                raise ValueError(f"a state tensor is (name, shape, dtype[, initial value]), not {t!r}")
            name, shape, dtype = t[:3]
            out.append((name, tuple(int(n) for n in shape), dtype, float(t[3]) if len(t) == 4 else 0.0))
        return out


class Part:
    """Base of parts: keeps spec and runtime; subclasses fill the rest."""

    graph_safe = False      # True: forward makes no host round trip, so a decode step through it may be recorded
    row_weight = None       # norms: see the module's text
    first_norm = None       # blocks: see the module's text

    def __init__(self, spec, rt):
        self.spec = spec
        self.rt = rt

    @staticmethod
    def tensor_specs(spec) -> Dict[str, TensorSpec]:
        return {}

    def bind(self, tensors: Dict[str, "object"]) -> None:
        if tensors:
            raise ValueError(f"{type(self).__name__} takes no tensors, got {sorted(tensors)}")


def sub_tensors(tensors: Dict[str, object], prefix: str) -> Dict[str, object]:
    """The entries of ``tensors`` under ``prefix.``, with the prefix removed."""
    p = prefix + "."
    return {k[len(p):]: v for k, v in tensors.items() if k.startswith(p)}
