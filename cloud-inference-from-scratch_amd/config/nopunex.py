"""Configuration of the Nopunex decoder, read from its ``config.json``.

The file lists the layers one by one: ``layers[i] = {"type", "mixer", "mlp"}``.  Every layer has a layer norm (weight and
bias) in front of each sublayer and one on its output (``x += norm1b(mixer(norm1(x)))``, ``x += norm2b(mlp(norm2(x)))``: a
``sandwich_norm`` block without a scale per channel).  ``type`` is

* ``delta``: the gated delta rule (``heads``, ``kv_heads``, ``dim``, ``vdim``, ``conv`` taps);
* ``latent_attention``: keys and values expanded from a latent of ``kv_rank`` numbers, queries from one of ``q_rank``
  (where the file does not say, the checkpoint does), per head ``dim`` plain and ``rot_dim`` turned numbers, values of
  ``vdim``, a rotation by halves with stretched frequencies (``rot.scaling``), a window of ``mask.size`` tokens and a
  learned sink per head;
* ``attention``: grouped-query attention with two maps a head whose difference counts (``diff``), a rotation by halves of
  the first ``rot.dims`` numbers of every map, chunks of ``mask.size`` positions and a gate on every number of the output.

``mlp`` is ``{"kind": "dense", "ff"}`` (a gated unit with silu) or ``null``.  ``loop = {start, stop, times}`` lets layers
``start .. stop - 1`` run ``times`` times over with the same weights, each pass on cache units of its own, and every pass
begins with ``x <- W [x; x0] + s_t`` (``x0`` the embedding's rows, ``s_t`` a vector of the pass).  Beside these: ``vocab``,
``width``, ``norm.eps``, ``logit_scale``.  Every size and constant that the file gives is read from it; what the design
fixes (which mixer has which steps, the activations) is handed to the parts as parameters here.

Tensors are named ``embed``, ``loop.in``, ``loop.step``, ``l<i>.norm1``, ``l<i>.norm1.b``, ``l<i>.mix.*``, ``l<i>.norm1b``,
..., ``l<i>.mlp.*``, ``final.norm`` and ``head``.
"""

from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any

from .givizen import _need, _positive, _positive_int
from .nokipel import _count
from .senuvik import _rotation
from .specs import ConfigError, LayerCall, LayerSpec, ModelSpec, PartSpec

MIXER_TYPES = ("delta", "latent_attention", "attention")
NAMES = (("norm1", "norm1"), ("mixer", "mix"), ("norm1_out", "norm1b"),
         ("norm2", "norm2"), ("feed_forward", "mlp"), ("norm2_out", "norm2b"))


def _reach(sizes: dict, where: str) -> int | None:
    """The size of a mixer's mask; none: every earlier token is seen."""
    if sizes.get("mask") is None:
        return None
    _need(sizes["mask"], ("size",), where + ".mask")
    return _positive_int(sizes["mask"], "size", where + ".mask")


@dataclass(frozen=True)
class NopunexConfig:
    raw: dict = field(compare=False)

    architecture = "Nopunex"

    @classmethod
    def from_hf_config(cls, raw: dict[str, Any]) -> "NopunexConfig":
        _need(raw, ("layers", "norm", "vocab", "width"), "config")
        if not isinstance(raw["layers"], list) or not raw["layers"]:
            raise ConfigError("config: layers must be a list with at least one layer")
        _need(raw["norm"], ("eps",), "config.norm")
        _positive(raw["norm"], "eps", "config.norm")
        for key in ("vocab", "width"):
            _positive_int(raw, key, "config")
        config = cls(copy.deepcopy(raw))
        spec = config.model_spec()
        from ..parts.model import DecoderModel  # (the parts are built once here: what one refuses is a ConfigError)

        try:
            model = DecoderModel(spec)
            model.expected_tensors()
            model.cache_needs()
        except (KeyError, TypeError, ValueError) as error:
            if isinstance(error, ConfigError):
                raise
            raise ConfigError(f"config: {error}") from error
        return config

    def to_hf_config(self) -> dict[str, Any]:
        out = copy.deepcopy(self.raw)
        out["architecture"] = self.architecture
        return out

    @property
    def hidden_size(self) -> int:
        return int(self.raw["width"])

    @property
    def vocab_size(self) -> int:
        return int(self.raw["vocab"])

    @property
    def eps(self) -> float:
        return float(self.raw["norm"]["eps"])

    def loop(self) -> tuple[int, int, int]:
        """(start, stop, times): how often the run of layers from start to in front of stop is gone through.  No loop: (0, 0, 1)."""
        loop = self.raw.get("loop")
        if loop is None:
            return 0, 0, 1
        _need(loop, ("start", "stop", "times"), "config.loop")
        start, stop = _count(loop, "start", "config.loop"), _count(loop, "stop", "config.loop")
        times = _positive_int(loop, "times", "config.loop")
        if not start < stop <= len(self.raw["layers"]):
            raise ConfigError(f"config.loop: layers {start} .. {stop} are no run of the {len(self.raw['layers'])} layers")
        return start, stop, times

    # -- mixers
    def _delta(self, sizes: dict, where: str) -> PartSpec:
        _need(sizes, ("heads", "dim", "vdim", "conv"), where)
        heads = _positive_int(sizes, "heads", where)
        return PartSpec.of("delta_rule", hidden_size=self.hidden_size, num_heads=heads,
                           num_kv_heads=_positive_int(sizes, "kv_heads", where) if "kv_heads" in sizes else heads,
                           head_dim=_positive_int(sizes, "dim", where), value_dim=_positive_int(sizes, "vdim", where),
                           taps=_positive_int(sizes, "conv", where), eps=self.eps)

    def _latent(self, sizes: dict, where: str) -> PartSpec:
        _need(sizes, ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale"), where)
        rot_dim = _count(sizes, "rot_dim", where)
        return PartSpec.of(
            "windowed_latent_attention", hidden_size=self.hidden_size, num_heads=_positive_int(sizes, "heads", where),
            head_dim=_positive_int(sizes, "dim", where), rot_dim=rot_dim, value_dim=_positive_int(sizes, "vdim", where),
            kv_rank=_positive_int(sizes, "kv_rank", where), scale=float(sizes["scale"]), eps=self.eps,
            q_rank=_positive_int(sizes, "q_rank", where) if sizes.get("q_rank") is not None else 0,
            window=_reach(sizes, where), sink=True, position=_rotation(sizes.get("rot"), rot_dim, "rotary_half", where + ".rot"))

    def _attention(self, sizes: dict, where: str) -> PartSpec:
        _need(sizes, ("heads", "dim", "vdim", "scale", "diff"), where)
        heads, dim = _positive_int(sizes, "heads", where), _positive_int(sizes, "dim", where)
        return PartSpec.of(
            "scored_attention", hidden_size=self.hidden_size, num_heads=heads,
            num_kv_heads=_positive_int(sizes, "kv_heads", where) if "kv_heads" in sizes else heads, head_dim=dim,
            value_dim=_positive_int(sizes, "vdim", where), scale=float(sizes["scale"]), eps=self.eps,
            chunk=_reach(sizes, where), output_gate=True, differential=float(sizes["diff"]),
            position=_rotation(sizes.get("rot"), dim, "rotary_half", where + ".rot"))

    def _mixer(self, kind: str, sizes: Any, where: str) -> PartSpec:
        if kind not in MIXER_TYPES:
            raise ConfigError(f"{where}: unknown layer type {kind!r}; known: {MIXER_TYPES}")
        if not isinstance(sizes, dict):
            raise ConfigError(f"{where}: must be a table")
        return {"delta": self._delta, "latent_attention": self._latent, "attention": self._attention}[kind](sizes, where)

    def _feed_forward(self, mlp: Any, where: str) -> PartSpec:
        if mlp is None:
            return PartSpec.of("none", hidden_size=self.hidden_size)
        _need(mlp, ("kind",), where)
        if mlp["kind"] != "dense":
            raise ConfigError(f"{where}: unknown kind {mlp['kind']!r}; known: ('dense',)")
        _need(mlp, ("ff",), where)
        return PartSpec.of("gated_mlp", hidden_size=self.hidden_size, intermediate_size=_positive_int(mlp, "ff", where),
                           names=("gate", "up", "down"))

    def model_spec(self) -> ModelSpec:
        norm = PartSpec.of("layer_norm", size=self.hidden_size, eps=self.eps)
        layers = []
        for index, layer in enumerate(self.raw["layers"]):
            where = f"layers[{index}]"
            _need(layer, ("type", "mixer"), where)
            try:
                layers.append(LayerSpec(
                    mixer=self._mixer(layer["type"], layer["mixer"], where + ".mixer"),
                    feed_forward=self._feed_forward(layer.get("mlp"), where + ".mlp"),
                    norm1=norm, norm2=norm, norm1_out=norm, norm2_out=norm, block="sandwich_norm", names=NAMES,
                    options=(("layer_scale", False),),
                ))
            except (TypeError, ValueError) as error:
                if isinstance(error, ConfigError):
                    raise
                raise ConfigError(f"{where}: {error}") from error
        start, stop, times = self.loop()
        # the run order: every run of a layer has a cache unit of its own, and every pass begins with the entry step
        runs: list[tuple[int, int | None]] = [(i, None) for i in range(start)]
        for turn in range(times if stop > start else 0):
            runs += [(i, turn if i == start else None) for i in range(start, stop)]
        runs += [(i, None) for i in range(stop, len(layers))]
        order = tuple(LayerCall(layer=i, cache=unit, writes=True, entry=turn) for unit, (i, turn) in enumerate(runs))
        return ModelSpec(
            architecture=self.architecture, vocab_size=self.vocab_size, hidden_size=self.hidden_size,
            layers=tuple(layers), order=order, final_norm=norm, tie_word_embeddings=False, max_position=1 << 30,
            eos_token_id=self.raw.get("eos_token_id"), embedding_name="embed", final_norm_name="final.norm",
            head_name="head", layer_prefix="l{index}.", logit_scale=float(self.raw.get("logit_scale", 1.0)),
            entry=PartSpec.of("join_embedding", hidden_size=self.hidden_size, times=times) if stop > start else None,
            entry_name="loop",
        )
