"""Configuration of the Nogapel decoder, read from its ``config.json``.

The file lists the layers one by one: ``layers[i] = {"type", "mixer", "mlp"}``.  The stream begins with an RMS norm of the
embedding's rows.  In a layer both sublayers read one RMS norm of the stream (``x += mixer(norm1(x)) + mlp(norm1(x))``: a
``parallel`` block), and behind them the layer adds a branch made from the stream and from its own columns of a second
embedding table (``token_side.dim`` columns a layer).  ``type`` is

* ``attention``: grouped-query attention under a window of ``mask.size`` tokens whose projected queries, keys and values
  each pass a causal convolution of ``conv`` taps, with an RMS norm of every query and key head, a rotation of the first
  ``rot.dims`` numbers in pairs of neighbours (``rot.scaling = {factor, low, high, original}``: frequencies divided by
  wavelength), and, with ``v_mix``, values mixed with those of the first such layer;
* ``latent_attention``: keys and values expanded from a latent of ``kv_rank`` numbers, queries from one of ``q_rank`` (where
  the file does not say, the checkpoint does), per head ``dim`` plain and ``rot_dim`` turned numbers, values of ``vdim``, and a
  learned sink per head, over all earlier tokens.

``mlp`` is ``{"kind": "dense", "ff"}`` (one product, the square of relu, one product) or ``null``.  Beside these: ``vocab``,
``width``, ``norm.eps``.  Every size and constant that the file gives is read from it; what the design fixes (which mixer has
which steps, the activations) is handed to the parts as parameters here.

Tensors are named ``embed``, ``embed.norm``, ``side.embed``, ``l<i>.norm1``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``l<i>.side.*``,
``final.norm`` and ``head``.
"""

from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any

from .givizen import _need, _positive, _positive_int
from .nokipel import _count
from .nopunex import _reach
from .specs import ConfigError, LayerCall, LayerSpec, ModelSpec, PartSpec

MIXER_TYPES = ("attention", "latent_attention")
NAMES = (("norm1", "norm1"), ("mixer", "mix"), ("feed_forward", "mlp"), ("side", "side"))


def _banded_rotation(rot: Any, dim: int, where: str) -> PartSpec | None:
    """A rotation of neighbouring pairs: ``rot = {dims, base, scaling}`` with ``scaling = {factor, low, high, original}``."""
    if rot is None:
        return None
    _need(rot, ("dims", "base"), where)
    dims = _count(rot, "dims", where)
    if dims == 0:
        return None
    if dims % 2 or dims > dim:
        raise ConfigError(f"{where}: dims must be even and at most the head size {dim}, got {dims}")
    bands = None
    if rot.get("scaling") is not None:
        keys = ("factor", "low", "high", "original")
        _need(rot["scaling"], keys, where + ".scaling")
        bands = tuple(float(_positive(rot["scaling"], key, where + ".scaling")) for key in keys)
    return PartSpec.of("rotary_pairs", head_dim=dim, theta=_positive(rot, "base", where), max_position=None, rotary_dim=dims,
                       bands=bands)


@dataclass(frozen=True)
class NogapelConfig:
    raw: dict = field(compare=False)

    architecture = "Nogapel"

    @classmethod
    def from_hf_config(cls, raw: dict[str, Any]) -> "NogapelConfig":
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

    @property
    def side_dim(self) -> int:
        """Columns of the second table that a layer has for itself; 0: the model has no such table."""
        side = self.raw.get("token_side")
        if side is None:
            return 0
        _need(side, ("dim",), "config.token_side")
        return _positive_int(side, "dim", "config.token_side")

    # -- mixers
    def _attention(self, sizes: dict, where: str, first_values: dict) -> PartSpec:
        _need(sizes, ("heads", "dim", "vdim", "scale"), where)
        heads, dim = _positive_int(sizes, "heads", where), _positive_int(sizes, "dim", where)
        kv_heads = _positive_int(sizes, "kv_heads", where) if "kv_heads" in sizes else heads
        vdim = _positive_int(sizes, "vdim", where)
        value_mix = None
        if sizes.get("v_mix"):
            # the first layer that mixes values is the one whose values the later ones mix in
            value_mix = "mixed" if first_values else "first"
            width = first_values.setdefault("width", kv_heads * vdim)
            if width != kv_heads * vdim:
                raise ConfigError(f"{where}: {kv_heads} value heads of {vdim} cannot be mixed with the first such layer's {width} numbers")
        return PartSpec.of(
            "scored_attention", hidden_size=self.hidden_size, num_heads=heads, num_kv_heads=kv_heads, head_dim=dim,
            value_dim=vdim, scale=float(sizes["scale"]), eps=self.eps, window=_reach(sizes, where), qk_norm="weight",
            conv_taps=_positive_int(sizes, "conv", where) if sizes.get("conv") is not None else None, value_mix=value_mix,
            position=_banded_rotation(sizes.get("rot"), dim, where + ".rot"))

    def _latent(self, sizes: dict, where: str) -> PartSpec:
        _need(sizes, ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale"), where)
        rot_dim = _count(sizes, "rot_dim", where)
        return PartSpec.of(
            "windowed_latent_attention", hidden_size=self.hidden_size, num_heads=_positive_int(sizes, "heads", where),
            head_dim=_positive_int(sizes, "dim", where), rot_dim=rot_dim, value_dim=_positive_int(sizes, "vdim", where),
            kv_rank=_positive_int(sizes, "kv_rank", where), scale=float(sizes["scale"]), eps=self.eps,
            q_rank=_positive_int(sizes, "q_rank", where) if sizes.get("q_rank") is not None else 0,
            window=_reach(sizes, where), sink=True, position=_banded_rotation(sizes.get("rot"), rot_dim, where + ".rot"))

    def _mixer(self, kind: str, sizes: Any, where: str, first_values: dict) -> PartSpec:
        if kind not in MIXER_TYPES:
            raise ConfigError(f"{where}: unknown layer type {kind!r}; known: {MIXER_TYPES}")
        if not isinstance(sizes, dict):
            raise ConfigError(f"{where}: must be a table")
        return self._attention(sizes, where, first_values) if kind == "attention" else self._latent(sizes, where)

    def _feed_forward(self, mlp: Any, where: str) -> PartSpec:
        if mlp is None:
            return PartSpec.of("none", hidden_size=self.hidden_size)
        _need(mlp, ("kind",), where)
        if mlp["kind"] != "dense":
            raise ConfigError(f"{where}: unknown kind {mlp['kind']!r}; known: ('dense',)")
        _need(mlp, ("ff",), where)
        return PartSpec.of("dense_mlp", hidden_size=self.hidden_size, intermediate_size=_positive_int(mlp, "ff", where))

    def model_spec(self) -> ModelSpec:
        norm = PartSpec.of("rms_norm_groups", size=self.hidden_size, eps=self.eps)
        layers: list[LayerSpec] = []
        first_values: dict = {}
        for index, layer in enumerate(self.raw["layers"]):
            where = f"layers[{index}]"
            _need(layer, ("type", "mixer"), where)
            side = PartSpec.of("token_side", hidden_size=self.hidden_size, dim=self.side_dim, index=index,
                               eps=self.eps) if self.side_dim else None
            try:
                layers.append(LayerSpec(
                    mixer=self._mixer(layer["type"], layer["mixer"], where + ".mixer", first_values),
                    feed_forward=self._feed_forward(layer.get("mlp"), where + ".mlp"),
                    norm1=norm, norm2=norm, block="parallel", names=NAMES, side=side,
                ))
            except (TypeError, ValueError) as error:
                if isinstance(error, ConfigError):
                    raise
                raise ConfigError(f"{where}: {error}") from error
        order = tuple(LayerCall(layer=i, cache=i, writes=True) for i in range(len(layers)))
        return ModelSpec(
            architecture=self.architecture, vocab_size=self.vocab_size, hidden_size=self.hidden_size,
            layers=tuple(layers), order=order, final_norm=norm, tie_word_embeddings=False, max_position=1 << 30,
            eos_token_id=self.raw.get("eos_token_id"), embedding_name="embed", final_norm_name="final.norm",
            head_name="head", layer_prefix="l{index}.", embedding_norm=norm, embedding_norm_name="embed.norm",
            side_table_columns=self.side_dim * len(layers), side_table_name="side.embed",
        )
