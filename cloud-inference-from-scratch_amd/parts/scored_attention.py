"""Grouped-query softmax attention over a window of the paged cache, without rotation, whose scores are shaped by
the position in other ways.  Every step is a parameter of the part and may be left out:

* a per-head RMS norm of queries and keys (``qk_norm``: ``"weight"`` with one weight vector for all query heads
  and one for all key heads, ``"unit"`` without weights, ``None``), or (``"whole"``) one RMS norm over all query
  heads of a token together and one over all its key heads, with a weight for every number of the projection;
* a factor on the queries that grows with the logarithm of the position (``q_temperature = (coef, every)``:
  ``1 + coef * ln(floor((p + 1) / every) + 1)``);
* ``score = q . k * scale``, then a smooth cap (``softcap``: ``c * tanh(score / c)``), then a bias on the distance
  itself (``slope_base = b``: head h of H loses ``2^(-b (h + 1) / H) * (i - j)``);
* a window (``window``: the token itself and the ``window - 1`` before it; with ``keep_first`` the first that many
  tokens of the sequence stay visible from behind the window too, at their own positions), or chunks (``chunk``: the token sees the
  keys of its own chunk of that many positions up to itself; the first chunk begins at position 0);
* biases on the projections of queries, keys and values (``qkv_bias``);
* a rotation of the first numbers of every query and key head by the position (``position``: a position part such
  as ``rotary_pairs``, applied after the heads' norm);
* a sink (``sink``: one learned number per head whose exponential stands in the softmax's denominator, and
  nowhere else);
* a gate on every head's output (``head_gate``: ``sigmoid(W_g x)_h``, read from the layer's own input), or on every
  number of the heads' outputs (``output_gate``: ``sigmoid(W_g x)`` has heads x vdim numbers);
* two maps a head (``differential = d``): queries and keys are projected as pairs of ``head_dim`` numbers, each map is a
  softmax of its own over the same values, and with ``lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + d`` (learned vectors of
  ``head_dim`` numbers) a head's output is ``a1 - lambda a2``, divided by its root mean square, times ``1 - d``;
* a causal convolution over the tokens of every channel of the projected queries, keys and values (``conv_taps``, in
  front of the heads' norm), whose last inputs are a state of the request beside its pages;
* values that are a mean of the layer's own and of those that an earlier layer of the same step made of the same token
  (``value_mix``: ``"first"`` is that earlier layer, ``"mixed"`` one that mixes, by a learned weight; what is cached is the
  mean);
* key and value heads of different sizes;
* no keys and values of its own (``own_kv=False``): the layer has no tensors for them and reads the cache unit that
  another layer of the same head sizes writes, with its own queries, mask and everything else.

One product makes queries, keys, values and gate logits; one kernel norms and scales the heads, lays the queries
out and writes the cache (``ops.heads_prepare``); the attention kernel shapes the scores, and applies sink and
gate in its epilogue (and there joins the two maps of a head): bfloat16 with head sizes up to 128 on the matrix cores
(``ops.scored_attention_mfma``, the heads zero-padded to 64 or 128 numbers, a map of a pair to 32, 64 or 128: no score
and no output changes), anything else, and float32, in the generic form.  Norm statistics, the logarithm, scores, softmax, value sums and the gate are float32.
"""

from __future__ import annotations

import math
import warnings
from typing import Optional

import torch

from ..cache.manager import FixedState, PagedKV
from ..config.specs import PartSpec
from ..kernels import ops
from ..weights.tensors import TensorSpec
from .base import Part, build_part, register_part
from .linear import linear
from .position import positions_bound

_SAID_GENERIC: set = set()
PROMPT_ROW_TILES = 2  # tiles of 16 (token, head) rows that a workgroup of the matrix-core form takes of a prompt's portion


def _round8(n: int) -> int:
    return -(-n // 8) * 8


class ScoredAttention(Part):
    graph_safe = True

    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int, value_dim: int,
                 scale: float, eps: float, window: Optional[int] = None, qk_norm: Optional[str] = None,
                 q_temperature: Optional[tuple] = None, softcap: Optional[float] = None,
                 slope_base: Optional[float] = None, sink: bool = False, head_gate: bool = False,
                 chunk: Optional[int] = None, qkv_bias: bool = False, position: Optional[PartSpec] = None,
                 keep_first: int = 0, own_kv: bool = True, output_gate: bool = False,
                 differential: Optional[float] = None, conv_taps: Optional[int] = None,
                 value_mix: Optional[str] = None) -> None:
        for name, value in (("hidden_size", hidden_size), ("num_heads", num_heads), ("num_kv_heads", num_kv_heads),
                            ("head_dim", head_dim), ("value_dim", value_dim)):
            if isinstance(value, bool) or not isinstance(value, int) or value < 1:
                raise ValueError(f"{name} must be a positive integer, got {value!r}")
        if num_heads % num_kv_heads:
            raise ValueError(f"{num_heads} query heads are no multiple of {num_kv_heads} key heads")
        if max(head_dim, value_dim) > 256:
            raise ValueError(f"heads of up to 256 numbers, got {head_dim} and {value_dim}")
        if window is not None and window < 1:
            raise ValueError("window must be positive")
        if chunk is not None and (isinstance(chunk, bool) or not isinstance(chunk, int) or chunk < 1 or window is not None):
            raise ValueError(f"chunks hold a positive number of tokens and stand in a window's place, got {chunk!r}")
        if isinstance(keep_first, bool) or not isinstance(keep_first, int) or keep_first < 0:
            raise ValueError(f"keep_first is a count of tokens, got {keep_first!r}")
        if window is None:
            keep_first = 0  # (every key is seen anyway)
        if qk_norm not in ops.NORM_MODES:
            raise ValueError(f"qk_norm must be one of {list(ops.NORM_MODES)}, got {qk_norm!r}")
        if not eps > 0:
            raise ValueError("eps must be positive")
        if softcap is not None and not softcap > 0:
            raise ValueError("softcap must be positive")
        if q_temperature is not None:
            coef, every = q_temperature
            if isinstance(every, bool) or int(every) != every or every < 1:
                raise ValueError(f"the temperature's period must be a positive integer, got {every!r}")
            q_temperature = (float(coef), int(every))
        self.hidden_size, self.num_heads, self.num_kv_heads = hidden_size, num_heads, num_kv_heads
        self.head_dim, self.value_dim = head_dim, value_dim
        self.scale, self.eps, self.window = float(scale), float(eps), window
        self.qk_norm, self.q_temperature, self.softcap = qk_norm, q_temperature, softcap
        self.slope_base, self.sink, self.head_gate = slope_base, bool(sink), bool(head_gate)
        self.chunk, self.qkv_bias = chunk, bool(qkv_bias)
        self.keep_first, self.own_kv = keep_first, bool(own_kv)
        self.output_gate = bool(output_gate)
        self.differential = float(differential) if differential is not None else None
        self.maps = 1 if differential is None else 2
        if self.output_gate and self.head_gate:
            raise ValueError("one gate: a number a head or a number for every number of it")
        if self.maps == 2 and (self.sink or qk_norm is not None or not self.own_kv):
            raise ValueError("two maps a head come with neither a sink nor a norm on the heads, and with keys of their own")
        if conv_taps is not None and (isinstance(conv_taps, bool) or not isinstance(conv_taps, int)
                                      or not 1 <= conv_taps <= ops.MAX_CONV_TAPS):
            raise ValueError(f"a convolution of 1 to {ops.MAX_CONV_TAPS} taps, got {conv_taps!r}")
        if value_mix not in (None, "first", "mixed"):
            raise ValueError(f"value_mix is 'first' or 'mixed' or None, got {value_mix!r}")
        self.conv_taps, self.value_mix = conv_taps, value_mix
        if self.by_channel and (self.maps == 2 or qk_norm == "whole" or not self.own_kv):
            raise ValueError("a convolution and mixed values come with one map a head, a norm of single heads and keys of their own")
        self.position = build_part("position", position) if position is not None else None
        if self.position is not None and self.position.rotates and self.position.rotary_dim > head_dim:
            raise ValueError(f"{self.position.rotary_dim} turning numbers in heads of {head_dim}")
        # the head sizes the kernels and the cache see: those of the matrix-core form where it has them
        if self.maps == 2:
            fitting = [pair for pair in ops.DIFFERENTIAL_MFMA_DIMS if pair[0] >= head_dim and pair[1] >= value_dim]
            self.mfma_dims = min(fitting, key=lambda pair: (pair[0], pair[1])) if fitting else None
            self.most_row_tiles = ops.DIFFERENTIAL_MFMA_DIMS[self.mfma_dims] if fitting else 0
        else:
            sizes = tuple(next((s for s in (64, 128) if s >= n), None) for n in (head_dim, value_dim))
            self.mfma_dims = sizes if sizes in ops.SCORED_MFMA_DIMS else None
            self.most_row_tiles = 4
        self.kernel_dim, self.kernel_vdim = self.mfma_dims or (_round8(head_dim), _round8(value_dim))

    @property
    def by_channel(self) -> bool:
        """Whether the projections pass the kernel that convolves them and mixes values."""
        return self.conv_taps is not None or self.value_mix is not None

    @property
    def joins_products(self) -> bool:
        return not self.qkv_bias

    @property
    def channels(self) -> int:
        return (self.num_heads + self.num_kv_heads) * self.head_dim + self.num_kv_heads * self.value_dim

    def cache_need(self):
        # (a chunk's keys all lie inside a window of the chunk's length: pages behind it go back to the pool)
        width = self.maps * self.kernel_dim
        pages = PagedKV(self.num_kv_heads, width, self.window if self.chunk is None else self.chunk,
                        value_dim=self.kernel_vdim if self.kernel_vdim != width else None,
                        keep_first=self.keep_first)
        if self.conv_taps is None or self.conv_taps == 1:
            return pages
        return (pages, FixedState((self.conv_taps - 1, self.channels)))

    def expected_tensors(self, prefix: str) -> dict[str, TensorSpec]:
        h, g, d, v, width = self.num_heads, self.num_kv_heads, self.head_dim, self.value_dim, self.hidden_size
        out = {prefix + "q": TensorSpec((h * self.maps * d, width))}
        if self.own_kv:
            out[prefix + "k"] = TensorSpec((g * self.maps * d, width))
            out[prefix + "v"] = TensorSpec((g * v, width))
        out[prefix + "o"] = TensorSpec((width, h * v))
        if self.qkv_bias:
            out[prefix + "q.b"] = TensorSpec((h * self.maps * d,))
            if self.own_kv:
                out[prefix + "k.b"] = TensorSpec((g * self.maps * d,))
                out[prefix + "v.b"] = TensorSpec((g * v,))
        if self.qk_norm in ("weight", "whole"):
            whole = self.qk_norm == "whole"
            out[prefix + "q.norm"] = TensorSpec((h * d if whole else d,), init="norm", keeps_float32=True)
            if self.own_kv:
                out[prefix + "k.norm"] = TensorSpec((g * d if whole else d,), init="norm", keeps_float32=True)
        if self.conv_taps is not None:
            for name, rows in (("q", h * d), ("k", g * d), ("v", g * v)):
                out[f"{prefix}{name}.conv"] = TensorSpec((rows, self.conv_taps))
        if self.value_mix is not None:  # (the first of the layers has nothing to mix with: its weight is not read)
            out[prefix + "vmix"] = TensorSpec((), keeps_float32=True, optional=self.value_mix == "first")
        if self.sink:
            out[prefix + "sink"] = TensorSpec((h,), keeps_float32=True)
        if self.head_gate or self.output_gate:
            out[prefix + "g"] = TensorSpec((h if self.head_gate else h * v, width))
        if self.maps == 2:
            for name in ("lq1", "lk1", "lq2", "lk2"):
                out[prefix + name] = TensorSpec((d,), keeps_float32=True)
        return out

    def bind(self, tensors, prefix, dtype, device) -> None:
        super().bind(tensors, prefix, dtype, device)
        h, g, d, v = self.num_heads, self.num_kv_heads, self.head_dim, self.value_dim
        blocks = [tensors[prefix + "q"]]
        if self.own_kv:
            blocks += [tensors[prefix + "k"], tensors[prefix + "v"]]
        d *= self.maps
        self.offsets = (0, h * d, h * d + g * d) if self.own_kv else (0, 0, 0)
        self.gate_offset = None
        if self.head_gate or self.output_gate:
            # gate logits ride in the same product, on columns that start at a multiple of 8 (and the row is
            # padded to one), so that the rows of the result stay 16-byte aligned
            pad = lambda rows: blocks[0].new_zeros((rows, self.hidden_size))
            used = h * d + (g * d + g * v if self.own_kv else 0)
            if used % 8:
                blocks.append(pad(8 - used % 8))
            self.gate_offset = _round8(used)
            blocks.append(tensors[prefix + "g"])
            gates = blocks[-1].shape[0]
            if gates % 8:
                blocks.append(pad(8 - gates % 8))
        self.w_in = torch.cat(blocks, dim=0).contiguous()
        self.b_in = None
        if self.qkv_bias:
            names = ("q.b", "k.b", "v.b") if self.own_kv else ("q.b",)
            bias = torch.cat([tensors[prefix + name] for name in names], dim=0)
            self.b_in = torch.cat([bias, bias.new_zeros(self.w_in.shape[0] - bias.shape[0])]).contiguous()
        self.q_weight = self.k_weight = None
        if self.qk_norm in ("weight", "whole"):
            self.q_weight = tensors[prefix + "q.norm"].float().contiguous()
            if self.own_kv:
                self.k_weight = tensors[prefix + "k.norm"].float().contiguous()
        self.taps_w, self.mix_weight = None, 0.0
        if self.conv_taps is not None:
            self.taps_w = torch.cat([tensors[f"{prefix}{name}.conv"] for name in ("q", "k", "v")], dim=0).t().contiguous()
        if self.value_mix == "mixed":
            self.mix_weight = float(tensors[prefix + "vmix"].float().item())
        self.pair = None  # what joins the two maps of a head: lambda, the factor behind the norm, its eps
        if self.maps == 2:
            dot = lambda n: float((tensors[f"{prefix}lq{n}"].float() * tensors[f"{prefix}lk{n}"].float()).sum())
            self.pair = (math.exp(dot(1)) - math.exp(dot(2)) + self.differential, 1.0 - self.differential, self.eps)
        self.sinks = tensors[prefix + "sink"].float().contiguous() if self.sink else None
        self.slopes = None
        if self.slope_base is not None:
            self.slopes = torch.tensor([2.0 ** (-self.slope_base * (i + 1) / h) for i in range(h)],
                                       dtype=torch.float32, device=device)
        w_o = tensors[prefix + "o"]
        if self.kernel_vdim != v:  # the attention's rows hold padded heads: zero columns under the padding
            wide = w_o.new_zeros((self.hidden_size, h, self.kernel_vdim))
            wide[:, :, :v] = w_o.reshape(self.hidden_size, h, v)
            w_o = wide.reshape(self.hidden_size, h * self.kernel_vdim)
        self.w_o = w_o.contiguous()

    def warm_up(self, rows: int) -> None:
        if self.w_in is None:
            return
        blank = lambda width: torch.zeros((rows, width), dtype=self.w_in.dtype, device=self.w_in.device)
        linear(blank(self.hidden_size), self.w_in, self.b_in)
        linear(blank(self.num_heads * self.kernel_vdim), self.w_o)

    def product_in(self) -> torch.Tensor:
        return self.w_in

    def product_out(self) -> torch.Tensor:
        return self.w_o

    def drop_products(self) -> None:
        self.w_in = self.w_o = None

    def forward(self, x: torch.Tensor, batch, view, writes: bool = True) -> torch.Tensor:
        return linear(self.mix(linear(x, self.w_in, self.b_in), batch, view, writes), self.w_o)

    def mix(self, proj: torch.Tensor, batch, view, writes: bool = True, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """What lies between the layer's first product and its last; the heads' outputs go to ``out`` if it is given."""
        if writes and not self.own_kv:
            raise ValueError("a layer without keys and values of its own reads the cache unit that another layer writes")
        rotary = None
        if self.position is not None and self.position.rotates:
            if batch.max_context > self.position.max_position:
                raise ValueError(f"position {batch.max_context - 1} is beyond the rotary table of {self.position.max_position}")
            cos, sin = self.position.tables(proj.device, positions_bound(batch))
            rotary = (cos, sin, self.position.rotary_dim, getattr(self.position, "pairing", "halves") == "neighbours")
        gate = proj[:, self.gate_offset:] if self.gate_offset is not None else None
        if self.by_channel:
            q, view = self._convolve(proj, batch, view, writes, rotary)
            return self.attend(q, gate, batch, view, out)
        q = ops.heads_prepare(proj, self.offsets, self.num_heads, self.num_kv_heads, self.head_dim, self.value_dim,
                              self.kernel_dim, self.kernel_vdim, self.qk_norm, self.q_weight, self.k_weight, self.eps,
                              self.q_temperature, batch.positions, batch.seq_of_token, batch.seq_slot,
                              view.block_table, view.k_pool, view.v_pool, batch.tokens, write_kv=writes, rotary=rotary,
                              maps=self.maps)
        return self.attend(q, gate, batch, view, out)

    def _convolve(self, proj: torch.Tensor, batch, view, writes: bool, rotary: Optional[tuple]):
        if not writes:
            raise ValueError("a layer whose projections are convolved moves its state on whenever it runs")
        pages, past = (view[0], view[1].state) if isinstance(view, (tuple, list)) else (view, None)
        first_out = first_in = None
        if self.value_mix == "first":
            first_out = torch.empty((batch.tokens, self.num_kv_heads * self.value_dim), dtype=proj.dtype, device=proj.device)
            batch.carried["first_values"] = first_out
        elif self.value_mix == "mixed":
            first_in = batch.carried.get("first_values")
            if first_in is None:
                raise ValueError("a layer mixes its values with an earlier layer's, and none has left any")
        q = ops.heads_conv_prepare(proj, self.offsets, self.num_heads, self.num_kv_heads, self.head_dim, self.value_dim,
                                   self.kernel_dim, self.kernel_vdim, self.taps_w, past, batch.q_start_loc, batch.sequences,
                                   batch.max_q_len <= 1, self.qk_norm, self.q_weight, self.k_weight, self.eps,
                                   self.q_temperature, batch.positions, batch.seq_of_token, batch.seq_slot, pages.block_table,
                                   pages.k_pool, pages.v_pool, rotary=rotary, first_out=first_out, first_in=first_in,
                                   mix=self.mix_weight)
        return q, pages

    def attend(self, q: torch.Tensor, gate, batch, view, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        shape = dict(window=self.window, scale=self.scale, softcap=self.softcap, slopes=self.slopes,
                     sinks=self.sinks, gate=gate, chunk=self.chunk, keep_first=self.keep_first, gate_wide=self.output_gate,
                     real_vdim=self.value_dim, differential=self.pair, out=out)
        return scored_attend(q, batch, view, self.num_heads, self.num_kv_heads, self.kernel_dim, self.kernel_vdim,
                             self.most_row_tiles if self.mfma_dims else 0, shape)


def scored_attend(q: torch.Tensor, batch, view, h: int, g: int, dim: int, vdim: int, most_row_tiles: int,
                  shape: dict) -> torch.Tensor:
    """Pick the attention kernel for this step's rows: ``h`` query heads on ``g`` key heads of ``dim`` and ``vdim``
    numbers as the kernels see them.  ``most_row_tiles``: the most tiles of 16 rows a workgroup of the matrix-core form
    takes at these sizes (0: it does not take them).  ``shape``: what both kernels are told about the scores."""
    window, chunk, keep_first = shape["window"], shape.get("chunk"), shape.get("keep_first", 0)
    maps = 1 if shape.get("differential") is None else 2
    group = h // g
    page_size = view.page_size
    # rows of a tile: a token's heads of one key head (of each map), and as many tokens as fill the tile
    least = maps * (1 if group <= 16 else 2 if group <= 32 else 4)
    if (q.dtype == torch.bfloat16 and group <= 64 and least <= most_row_tiles and page_size >= 4
            and not page_size & (page_size - 1)):
        # the most keys a token sees in this step (a captured step: in any of its replays)
        bound = batch.static_plan.max_keys if batch.static_plan is not None else batch.max_context
        reach = window if chunk is None else chunk  # the most keys a token sees, if bounded
        if reach is not None and keep_first:
            reach += -(-keep_first // 32) * 32 + 32  # (the kept first keys are walked in whole blocks of 32)
        bound = bound if reach is None else min(bound, reach)

        def shares(tiles: int, span: int) -> dict:
            """Few tiles over many keys: the keys in shares of at least 128, about two workgroups a compute unit."""
            reach = bound + span + 32                        # a tile's range starts at a multiple of 32
            wanted = min(2 * ops.compute_units() // max(tiles * g, 1), reach // 128)
            if wanted < 2:
                return {}
            per = -(-(-(-reach // wanted)) // 128) * 128
            return dict(n_splits=-(-reach // per), keys_per_split=per)

        if batch.static_plan is not None and batch.static_plan.decode_rows in (None, batch.sequences):
            # a captured step of single tokens: tile i is sequence i, nothing comes from the host
            return ops.scored_attention_mfma(q, view.k_pool, view.v_pool, view.block_table, None, None,
                                             batch.sequences, batch.seq_slot, batch.seq_start, batch.seq_q_len,
                                             batch.q_start_loc, batch.tokens, h, g, dim, vdim, 1, least, **shape,
                                             **shares(batch.sequences, 1))
        row_tiles = min(most_row_tiles, max(least, PROMPT_ROW_TILES if batch.max_q_len * group > 16 else maps))
        while row_tiles > least and -(-batch.tokens * group * maps // (16 * row_tiles)) * g < ops.compute_units():
            row_tiles //= 2  # (fewer rows a tile where the tiles would not fill the compute units)
        per_tile = (16 * row_tiles) // (group * maps)
        tile_seq, tile_q0, n_tiles = batch.tiles(per_tile, decode=None)
        return ops.scored_attention_mfma(q, view.k_pool, view.v_pool, view.block_table, tile_seq, tile_q0, n_tiles,
                                         batch.seq_slot, batch.seq_start, batch.seq_q_len, batch.q_start_loc,
                                         batch.tokens, h, g, dim, vdim, per_tile, row_tiles, **shape,
                                         **shares(n_tiles, per_tile))
    if q.dtype == torch.bfloat16 and (dim, vdim, group, page_size) not in _SAID_GENERIC:
        _SAID_GENERIC.add((dim, vdim, group, page_size))
        warnings.warn(f"bfloat16 attention with heads of {dim} and {vdim} numbers, {group} query heads per key head and pages "
                      f"of {page_size} takes the generic kernel (the matrix-core form takes heads of up to 128 numbers, pairs "
                      f"of maps of up to 128 with values of up to 256, latents as ops.LATENT_MFMA_DIMS lists them, a token's "
                      f"heads on up to 64 rows and pages of a power of two >= 4)",
                      RuntimeWarning, stacklevel=2)
    return ops.scored_attention_generic(q, view.k_pool, view.v_pool, view.block_table, batch.positions,
                                        batch.seq_of_token, batch.seq_slot, batch.tokens, h, g, dim, vdim, **shape)


register_part("mixer", "scored_attention", ScoredAttention)
