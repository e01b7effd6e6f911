"""Architecture-neutral descriptions of a decoder: what an architecture's
configuration is turned into before any tensor exists.

A model is a list of layers, each a :class:`LayerSpec` that names its mixer,
feed-forward, norms and arrangement by *kind* (a key of the part registries in
``cie_amd.parts``) together with every size and constant the part needs, and an
*order*: the list of :class:`LayerCall` that says which layer runs when and on
which cache.  Nothing here knows a model family; a configuration class (for
instance ``Qwen2Config``) produces these from its own ``config.json`` keys.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any


class ConfigError(ValueError):
    """A ``config.json`` that no registered architecture can run: an unknown name, a key
    that is missing, a value outside what the parts take."""


@dataclass(frozen=True)
class PartSpec:
    """``kind`` selects the part class; ``params`` are its constructor arguments."""

    kind: str
    params: tuple[tuple[str, Any], ...] = ()

    @classmethod
    def of(cls, kind: str, **params: Any) -> "PartSpec":
        return cls(kind, tuple(sorted(params.items())))

    def as_dict(self) -> dict[str, Any]:
        return dict(self.params)


@dataclass(frozen=True)
class LayerSpec:
    """One decoder layer: which parts, how arranged, and under which tensor names.

    ``names`` maps the block's part roles (``norm1``, ``mixer``, ``norm2``,
    ``feed_forward``) to the sub-prefix of the checkpoint's tensor names.
    ``options`` are the arrangement's own constants (a factor on the branches, the layer's depth), which
    the block class reads.  ``norm1_out`` and ``norm2_out`` are the norms on the sublayers' outputs of an arrangement
    that has norms on both sides of a sublayer.  ``side`` is a branch of its own that follows the layer's other ones
    (a part of the role "side").
    """

    mixer: PartSpec
    feed_forward: PartSpec
    norm1: PartSpec
    norm2: PartSpec
    block: str = "pre_norm"
    names: tuple[tuple[str, str], ...] = ()
    options: tuple[tuple[str, Any], ...] = ()
    norm1_out: PartSpec | None = None
    norm2_out: PartSpec | None = None
    side: PartSpec | None = None

    def option(self, name: str, default: Any = None) -> Any:
        return dict(self.options).get(name, default)

    def name_of(self, role: str) -> str:
        return dict(self.names).get(role, role)


@dataclass(frozen=True)
class LayerCall:
    """One entry of the run order.

    ``layer``  index into ``ModelSpec.layers`` (a layer may be named twice).
    ``cache``  index of the cache unit the mixer reads; two calls may name the
               same unit, then the later one reads what the earlier one wrote.
    ``writes`` whether this call appends its own keys/values (or state) to the
               unit before reading it.
    ``adds_embedding`` the embedding's rows (scaled, as they entered the stream) join the
               stream once more right in front of this call.
    ``entry``  the model's entry step (``ModelSpec.entry``) runs right in front of this
               call, as the entry of that number; ``None``: it does not.
    """

    layer: int
    cache: int
    writes: bool = True
    adds_embedding: bool = False
    entry: int | None = None


@dataclass(frozen=True)
class ModelSpec:
    architecture: str
    vocab_size: int
    hidden_size: int
    layers: tuple[LayerSpec, ...]
    order: tuple[LayerCall, ...]
    final_norm: PartSpec
    tie_word_embeddings: bool
    max_position: int
    eos_token_id: int | None = None
    embedding_name: str = "model.embed_tokens.weight"
    final_norm_name: str = "model.norm"
    head_name: str = "lm_head.weight"
    layer_prefix: str = "model.layers.{index}."
    embedding_scale: float = 1.0          # the embedding's rows are multiplied by this on their way into the stream
    logit_softcap: float | None = None    # logits <- cap * tanh(logits / cap)
    logit_scale: float = 1.0              # logits <- scale * logits, in front of the cap
    # what remakes the stream in front of the calls that have an ``entry`` (a part of the role "entry"), and the prefix of
    # its tensors' names
    entry: PartSpec | None = None
    entry_name: str = "entry"
    # a norm of the embedding's rows, with which the stream begins
    embedding_norm: PartSpec | None = None
    embedding_norm_name: str = "embed.norm"
    # a second table looked up by token, of that many columns, which the layers' ``side`` parts read; 0: none
    side_table_columns: int = 0
    side_table_name: str = "side.embed"
    extra: dict[str, Any] = field(default_factory=dict, compare=False)

    def __post_init__(self) -> None:
        units: dict[int, int] = {}
        for call in self.order:
            if not 0 <= call.layer < len(self.layers):
                raise ValueError(f"run order names layer {call.layer}, model has {len(self.layers)}")
            if call.cache < 0:
                raise ValueError("cache unit indices are non-negative")
            if call.entry is not None and (self.entry is None or call.entry < 0):
                raise ValueError(f"layer {call.layer} is run behind entry {call.entry}, and the model has no such step")
            if call.writes:
                units.setdefault(call.cache, call.layer)
        for call in self.order:
            if call.cache not in units:
                raise ValueError(f"cache unit {call.cache} is read by layer {call.layer} but never written")

    @property
    def cache_units(self) -> int:
        return max((call.cache for call in self.order), default=-1) + 1
