"""Softmax attention whose keys and values are expanded from one small latent vector per token.

Per token the layer projects ``heads`` queries, each ``[plain (P) | turned (R)]``, and one vector
``[latent (C) | turned key part (R)]``.  The latent is RMS-normed (with a weight); head h's plain key is
``W_uk[h] c`` and its value ``W_uv[h] c``; the turned key part is shared by all heads; queries' and the key's turned
parts rotate with the position.  The score of query t and key j is ``(q_plain . k_plain + q_turned . k_turned) * scale``
over all ``j <= t``, softmax; the heads' outputs are multiplied by ``sigmoid(W_g x)`` and projected by ``W_o``.

Only the normed latent and the turned key part are cached, and the expansions are never applied to the cache:
since ``q_plain . (W_uk[h] c) = (W_uk[h]^T q_plain) . c``, a query is folded into the latent space once, and since
``sum_j p_j W_uv[h] c_j = W_uv[h] sum_j p_j c_j`` the value expansion is applied once to the head's weighted sum of
latents.  To the paged attention kernels this is one key head of ``R + C`` numbers (padded to a head size they take)
shared by all query heads, whose value is the cache entry itself: the layer reuses them as they are, in both
precisions.  The per-head folding and unfolding are block-diagonal products (``ops.block_linear``).
"""

from __future__ import annotations

from typing import Optional

import torch

from ..cache.manager import PagedKV
from ..config.specs import PartSpec
from ..kernels import ops
from ..weights.tensors import TensorSpec
from .attention import attend
from .base import Part, build_part, register_part
from .linear import linear
from .position import positions_bound
from .scored_attention import scored_attend


class LatentAttention(Part):
    graph_safe = True  # (a captured step's rotation tables reach the bound the step was captured for)

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, rot_dim: int, value_dim: int, kv_rank: int,
                 scale: float, eps: float, position: PartSpec) -> None:
        for name, value in (("hidden_size", hidden_size), ("num_heads", num_heads), ("head_dim", head_dim),
                            ("value_dim", value_dim), ("kv_rank", kv_rank)):
            if value < 1:
                raise ValueError(f"{name} must be positive, got {value}")
        if rot_dim < 0 or rot_dim % 2:
            raise ValueError(f"the turned part of a head must be even, got {rot_dim}")
        if not scale > 0 or not eps > 0:
            raise ValueError("scale and eps must be positive")
        self.hidden_size = hidden_size
        self.num_heads = num_heads
        self.head_dim = head_dim
        self.rot_dim = rot_dim
        self.value_dim = value_dim
        self.kv_rank = kv_rank
        self.scale = float(scale)
        self.eps = float(eps)
        self.position = build_part("position", position)
        entry = rot_dim + kv_rank
        # the cache entry is as wide as a head of the attention kernels: the next size their matrix-core forms take
        self.entry_dim = next((size for size in ops.MFMA_HEAD_DIMS if size >= entry), None)
        if self.entry_dim is None:
            raise ValueError(f"a cache entry of {entry} numbers is more than the attention kernels' {ops.MFMA_HEAD_DIMS[-1]}")

    def cache_need(self) -> PagedKV:
        return PagedKV(1, self.entry_dim, None)

    def expected_tensors(self, prefix: str) -> dict[str, TensorSpec]:
        h, p, r, v, c, hidden = self.num_heads, self.head_dim, self.rot_dim, self.value_dim, self.kv_rank, self.hidden_size
        return {
            prefix + "q": TensorSpec((h * (p + r), hidden)),
            prefix + "dkv": TensorSpec((c + r, hidden)),
            prefix + "dkv.norm": TensorSpec((c,), init="norm", keeps_float32=True),
            prefix + "uk": TensorSpec((h * p, c)),
            prefix + "uv": TensorSpec((h * v, c)),
            prefix + "g": TensorSpec((h * v, hidden)),
            prefix + "o": TensorSpec((hidden, h * v)),
        }

    def bind(self, tensors, prefix, dtype, device) -> None:
        super().bind(tensors, prefix, dtype, device)
        h, p, r, v, c = self.num_heads, self.head_dim, self.rot_dim, self.value_dim, self.kv_rank
        self.w_in = torch.cat([tensors[prefix + "q"], tensors[prefix + "dkv"], tensors[prefix + "g"]], dim=0).contiguous()
        self.latent_weight = tensors[prefix + "dkv.norm"].contiguous()
        # fold: [heads, C, P] so that (q_plain of head h) @ fold[h].T lies in the latent space
        self.w_fold = tensors[prefix + "uk"].reshape(h, p, c).transpose(1, 2).contiguous()
        # unfold: [heads, V, entry] reads the latent part of a head's weighted sum of cache entries
        unfold = torch.zeros((h, v, self.entry_dim), dtype=dtype, device=device)
        unfold[:, :, r: r + c] = tensors[prefix + "uv"].reshape(h, v, c)
        self.w_unfold = unfold.contiguous()
        self.w_o = tensors[prefix + "o"].contiguous()

    def forward(self, x: torch.Tensor, batch, view, writes: bool = True) -> torch.Tensor:
        h, p, r, c, width = self.num_heads, self.head_dim, self.rot_dim, self.kv_rank, self.entry_dim
        if batch.max_context > self.position.max_position and self.position.rotates:
            raise ValueError(f"position {batch.max_context - 1} is beyond the rotary table of {self.position.max_position}")
        queries = h * (p + r)
        proj = linear(x, self.w_in)
        rows = ops.latent_rows(proj[:, : queries + c + r], self.latent_weight, h, p, r, c, width, self.eps)
        ops.block_linear(proj, self.w_fold, a_block=p + r, out=rows, out_offset=r, c_block=width)
        turns = bool(r) and self.position.rotates
        cos, sin = self.position.tables(x.device, positions_bound(batch))
        ops.rope_kv_write(rows, cos, sin, batch.positions, batch.seq_of_token, batch.seq_slot, view.block_table,
                          view.k_pool, view.v_pool, h, 1, width, rotate=turns, write_kv=writes,
                          rotary_dim=r if turns else None)
        context = attend(rows, batch, view, h, 1, width, None, self.scale)
        gated = ops.block_linear(context, self.w_unfold, gate=proj, gate_offset=queries + c + r)
        return linear(gated, self.w_o)


register_part("mixer", "latent_attention", LatentAttention)


class WindowedLatentAttention(Part):
    """The same attention with what its scores may be shaped by: queries that come from a latent of their own
    (``q_rank``: ``q = W_uq norm(W_dq x)``; ``None``: ``q = W_q x``), a window (the token and the ``window - 1`` before
    it), a sink per head in the softmax's denominator, and no gate on the output.  A token's cache entry is
    ``[turned key part | normed latent | zeros]`` and its value the normed latent alone, so that the attention kernels
    that shape their scores (``scored_attend``) see one key head for all query heads, whose value is narrower than its
    key.  ``q_rank=0`` reads the rank off the checkpoint."""

    graph_safe = True
    joins_products = True

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, rot_dim: int, value_dim: int, kv_rank: int,
                 scale: float, eps: float, position: Optional[PartSpec] = None, q_rank: Optional[int] = None,
                 window: Optional[int] = None, sink: bool = False) -> None:
        for name, value in (("hidden_size", hidden_size), ("num_heads", num_heads), ("head_dim", head_dim),
                            ("value_dim", value_dim), ("kv_rank", kv_rank)):
            if isinstance(value, bool) or not isinstance(value, int) or value < 1:
                raise ValueError(f"{name} must be a positive integer, got {value!r}")
        if rot_dim < 0 or not eps > 0 or (q_rank is not None and q_rank < 0):
            raise ValueError(f"a turned part of {rot_dim} numbers, a query latent of {q_rank}, eps {eps}: not negative, eps positive")
        if window is not None and window < 1:
            raise ValueError("window must be positive")
        self.hidden_size, self.num_heads, self.head_dim, self.rot_dim = hidden_size, num_heads, head_dim, rot_dim
        self.value_dim, self.kv_rank, self.scale, self.eps = value_dim, kv_rank, float(scale), float(eps)
        self.q_rank, self.window, self.sink = q_rank, window, bool(sink)
        self.position = build_part("position", position) if position is not None else None
        if self.position is not None and self.position.rotates and self.position.rotary_dim > rot_dim:
            raise ValueError(f"{self.position.rotary_dim} turning numbers in a turned part of {rot_dim}")
        entry = rot_dim + kv_rank
        fitting = [pair for pair in ops.LATENT_MFMA_DIMS if pair[0] >= entry and pair[1] >= kv_rank]
        self.mfma_dims = min(fitting) if fitting else None
        round8 = lambda n: -(-n // 8) * 8
        self.entry_dim, self.latent_dim = self.mfma_dims or (round8(entry), round8(kv_rank))
        if self.latent_dim > ops.MAX_GENERIC_VALUE:
            raise ValueError(f"a latent of {kv_rank} numbers is more than the attention kernels' {ops.MAX_GENERIC_VALUE}")

    def cache_need(self) -> PagedKV:
        return PagedKV(1, self.entry_dim, self.window,
                       value_dim=self.latent_dim if self.latent_dim != self.entry_dim else None)

    def expected_tensors(self, prefix: str) -> dict[str, TensorSpec]:
        h, p, r, v, c, hidden = self.num_heads, self.head_dim, self.rot_dim, self.value_dim, self.kv_rank, self.hidden_size
        if self.q_rank is None:
            out = {prefix + "q": TensorSpec((h * (p + r), hidden))}
        else:
            rank, drawn = self.q_rank or None, self.q_rank or max(8, hidden // 4 // 8 * 8)
            out = {prefix + "dq": TensorSpec((rank, hidden), drawn=(drawn, hidden)),
                   prefix + "dq.norm": TensorSpec((rank,), init="norm", keeps_float32=True, drawn=(drawn,)),
                   prefix + "uq": TensorSpec((h * (p + r), rank), drawn=(h * (p + r), drawn))}
        out.update({
            prefix + "dkv": TensorSpec((c + r, hidden)),
            prefix + "dkv.norm": TensorSpec((c,), init="norm", keeps_float32=True),
            prefix + "uk": TensorSpec((h * p, c)),
            prefix + "uv": TensorSpec((h * v, c)),
            prefix + "o": TensorSpec((hidden, h * v)),
        })
        if self.sink:
            out[prefix + "sink"] = TensorSpec((h,), keeps_float32=True)
        return out

    def bind(self, tensors, prefix, dtype, device) -> None:
        super().bind(tensors, prefix, dtype, device)
        h, p, r, v, c = self.num_heads, self.head_dim, self.rot_dim, self.value_dim, self.kv_rank
        pad = lambda t: t if t.shape[0] % 8 == 0 else torch.cat([t, t.new_zeros((8 - t.shape[0] % 8, t.shape[1]))], dim=0)
        self.dq_weight = self.w_uq = None
        self.q_latent = 0
        if self.q_rank is None:
            first = tensors[prefix + "q"]
        else:
            first = tensors[prefix + "dq"]
            self.q_latent = first.shape[0]
            self.dq_weight = tensors[prefix + "dq.norm"].float().contiguous()
            self.w_uq = tensors[prefix + "uq"].contiguous()
            if self.w_uq.shape[1] != self.q_latent or self.dq_weight.shape[0] != self.q_latent:
                raise ValueError(f"{prefix}dq, dq.norm and uq disagree on the query latent's size")
        # (the parts of a row of the product's result start at multiples of 16 bytes)
        first = pad(first)
        self.c_offset = first.shape[0]
        self.w_in = torch.cat([first, pad(tensors[prefix + "dkv"])], dim=0).contiguous()
        self.dkv_weight = tensors[prefix + "dkv.norm"].float().contiguous()
        # fold: [heads, C, P] so that (q_plain of head h) @ fold[h].T lies in the latent space
        self.w_fold = tensors[prefix + "uk"].reshape(h, p, c).transpose(1, 2).contiguous()
        # unfold: [heads, V, latent_dim] reads a head's weighted sum of latents
        unfold = torch.zeros((h, v, self.latent_dim), dtype=dtype, device=device)
        unfold[:, :, :c] = tensors[prefix + "uv"].reshape(h, v, c)
        self.w_unfold = unfold.contiguous()
        self.w_o = tensors[prefix + "o"].contiguous()
        self.sinks = tensors[prefix + "sink"].float().contiguous() if self.sink else None

    def warm_up(self, rows: int) -> None:
        blank = lambda width: torch.zeros((rows, width), dtype=self.dtype, device=self.device)
        if self.w_uq is not None:
            linear(blank(self.q_latent), self.w_uq)
        if self.w_in is not None:
            linear(blank(self.hidden_size), self.w_in)
            linear(blank(self.num_heads * self.value_dim), self.w_o)

    def product_in(self) -> torch.Tensor:
        return self.w_in

    def product_out(self) -> torch.Tensor:
        return self.w_o

    def drop_products(self) -> None:
        self.w_in = self.w_o = None

    def forward(self, x: torch.Tensor, batch, view, writes: bool = True) -> torch.Tensor:
        return linear(self.mix(linear(x, self.w_in), batch, view, writes), self.w_o)

    def mix(self, proj: torch.Tensor, batch, view, writes: bool = True, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """What lies between the layer's first product and its last; the heads' outputs go to ``out`` if it is given."""
        h, p, r, c = self.num_heads, self.head_dim, self.rot_dim, self.kv_rank
        rotary = None
        if self.position is not None and self.position.rotates:
            if batch.max_context > self.position.max_position:
                raise ValueError(f"position {batch.max_context - 1} is beyond the rotary table of {self.position.max_position}")
            cos, sin = self.position.tables(proj.device, positions_bound(batch))
            rotary = (cos, sin, self.position.rotary_dim, getattr(self.position, "pairing", "halves") == "neighbours")
        q_latent = ops.latent_down(proj, 0, self.q_latent, self.c_offset, self.dq_weight, self.dkv_weight, c, r, rotary,
                                   batch.positions, batch.seq_of_token, batch.seq_slot, view.block_table, view.k_pool,
                                   view.v_pool, self.eps, write_kv=writes)
        q = proj[:, : h * (p + r)] if q_latent is None else linear(q_latent, self.w_uq)
        rows = ops.latent_queries(q, h, p, r, c, self.entry_dim, rotary, batch.positions)
        ops.block_linear(q, self.w_fold, a_block=p + r, out=rows, out_offset=r, c_block=self.entry_dim)
        shape = dict(window=self.window, scale=self.scale, sinks=self.sinks)
        context = scored_attend(rows, batch, view, h, 1, self.entry_dim, self.latent_dim,
                                ops.LATENT_MFMA_DIMS[self.mfma_dims] if self.mfma_dims else 0, shape)
        return ops.block_linear(context, self.w_unfold, out=out)


register_part("mixer", "windowed_latent_attention", WindowedLatentAttention)
