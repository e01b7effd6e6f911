"""The gated delta rule: a memory of fixed size per head that is corrected, not only added to.

Queries, keys (``kv_heads`` heads of ``dim``, each serving ``heads / kv_heads`` neighbouring heads) and values (``heads``
of ``vdim``) are projected and pass a causal convolution over each channel's last ``taps`` inputs and silu; queries and
keys come to length one per head, queries times ``q_scale``.  A head's memory S becomes ``g S + k u^T`` with the
correction ``u = beta (v - g S^T k)``, so that with a step size of one the memory answers k with v; the query reads the
new memory.  Step size (a sigmoid of ``b``) and decay (``A_log``, ``dt_bias`` and a softplus of ``a``) are one number per
head and token.  The read-out is RMS-normed per head under one weight for all heads, gated by silu of ``g`` and
projected.  Products run in the engine's type; everything else, and the state (the
memory [heads, vdim, dim] and the convolutions' last inputs per head), is float32.  A request's state lies in its slot and
moves on with its tokens, so a prompt may be cut anywhere.  Kernels: ``csrc/delta_rule.hip``.
"""

from __future__ import annotations

from typing import Optional

import torch

from ..cache.manager import FixedState
from ..kernels import ops
from ..weights.tensors import TensorSpec
from .base import Part, register_part
from .linear import linear


class DeltaRule(Part):
    graph_safe = True

    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int, value_dim: int, taps: int,
                 eps: float, q_scale: Optional[float] = None) -> None:
        for name, value in (("hidden_size", hidden_size), ("num_heads", num_heads), ("num_kv_heads", num_kv_heads),
                            ("head_dim", head_dim), ("value_dim", value_dim), ("taps", taps)):
            if isinstance(value, bool) or not isinstance(value, int) or value < 1:
                raise ValueError(f"{name} must be a positive integer, got {value!r}")
        if num_heads % num_kv_heads:
            raise ValueError(f"{num_heads} heads are no multiple of {num_kv_heads} key heads")
        if taps > ops.DELTA_MAX_TAPS or not eps > 0:
            raise ValueError(f"up to {ops.DELTA_MAX_TAPS} taps and a positive eps, got {taps}, {eps}")
        ops.plan_delta_walk(head_dim, value_dim)  # (refuses memories the kernel has no room for)
        if num_heads * (value_dim + 1) > ops.MAX_NORM_WIDTH:
            raise ValueError(f"{num_heads} heads of {value_dim}: the read-out's norm takes rows of up to {ops.MAX_NORM_WIDTH} numbers")
        self.hidden_size, self.num_heads, self.num_kv_heads = hidden_size, num_heads, num_kv_heads
        self.head_dim, self.value_dim, self.taps, self.eps = head_dim, value_dim, taps, float(eps)
        self.q_scale = head_dim ** -0.5 if q_scale is None else float(q_scale)

    def cache_need(self) -> tuple:
        return (FixedState((self.num_heads, self.value_dim, self.head_dim)),
                FixedState((self.num_heads, max(self.taps - 1, 1), 2 * self.head_dim + self.value_dim)))

    def expected_tensors(self, prefix: str) -> dict[str, TensorSpec]:
        h, width = self.num_heads, self.hidden_size
        qk, v = self.num_kv_heads * self.head_dim, h * self.value_dim
        small = dict(keeps_float32=True)
        return {
            prefix + "q": TensorSpec((qk, width)), prefix + "q.conv": TensorSpec((qk, self.taps)),
            prefix + "k": TensorSpec((qk, width)), prefix + "k.conv": TensorSpec((qk, self.taps)),
            prefix + "v": TensorSpec((v, width)), prefix + "v.conv": TensorSpec((v, self.taps)),
            prefix + "b": TensorSpec((h, width)), prefix + "a": TensorSpec((h, width)),
            prefix + "A_log": TensorSpec((h,), **small), prefix + "dt_bias": TensorSpec((h,), **small),
            prefix + "norm": TensorSpec((self.value_dim,), init="norm", **small),
            prefix + "g": TensorSpec((v, width)), prefix + "o": TensorSpec((width, v)),
        }

    def bind(self, tensors, prefix, dtype, device) -> None:
        super().bind(tensors, prefix, dtype, device)
        parts = [tensors[prefix + name] for name in ("q", "k", "v", "g", "b", "a")]
        self.offsets = tuple(sum(p.shape[0] for p in parts[:i]) for i in range(len(parts)))
        used = sum(p.shape[0] for p in parts)
        if used % 8:  # (the rows of the product's result stay 16-byte aligned)
            parts.append(parts[0].new_zeros((8 - used % 8, self.hidden_size)))
        self.w_in = torch.cat(parts, dim=0).contiguous()
        self.taps_w = torch.cat([tensors[prefix + name + ".conv"] for name in ("q", "k", "v")], dim=0).contiguous()
        self.a_log = tensors[prefix + "A_log"].float().contiguous()
        self.dt_bias = tensors[prefix + "dt_bias"].float().contiguous()
        self.norm_weight = tensors[prefix + "norm"].float().contiguous()
        self.w_o = tensors[prefix + "o"].contiguous()

    def warm_up(self, rows: int) -> None:
        blank = lambda width: torch.zeros((rows, width), dtype=self.w_in.dtype, device=self.w_in.device)
        linear(blank(self.hidden_size), self.w_in)
        linear(blank(self.num_heads * self.value_dim), self.w_o)

    def forward(self, x: torch.Tensor, batch, view, writes: bool = True) -> torch.Tensor:
        if not writes:
            raise ValueError("a recurrent mixer moves its state on whenever it runs")
        out = ops.delta_rule(linear(x, self.w_in), self.offsets, self.taps_w, self.a_log, self.dt_bias, self.q_scale,
                             self.norm_weight, self.eps, view[0].state, view[1].state, batch.seq_of_token, batch.seq_slot,
                             batch.q_start_loc, batch.sequences, self.num_heads, self.num_kv_heads, self.head_dim,
                             self.value_dim)
        return linear(out, self.w_o)


register_part("mixer", "delta_rule", DeltaRule)
