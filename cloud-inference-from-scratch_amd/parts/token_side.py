"""What a layer adds from an embedding of the tokens that is its own.

``TokenSide``: behind the layer's other branches the stream x meets the layer's part e of the token's row of a second
table, ``y = W_proj (gelu_tanh(W_gate x) * e)``, and y joins the stream under an RMS norm of its own with a weight:
``x += y / sqrt(mean(y^2) + eps) * w``.  Layer i's part are the columns ``i * dim .. (i + 1) * dim - 1``.  The table is the
model's (``ModelSpec.side_table_columns``); the step's batch carries it together with the tokens as the embedding took
them.  The stream, the norm and the gate are float32; the two products run in the engine's type.  In bfloat16 few rows take a
kernel for everything up to ``gelu_tanh(W_gate x) * e``, many rows one kernel for all of it, the add of the layer's other
branches and the next layer's norm included (``csrc/token_side.hip``).
"""

from __future__ import annotations

from typing import Any, Optional

import torch

from ..kernels import ops
from ..weights.tensors import TensorSpec
from .base import Part, register_part
from .linear import Added, RowSumsq, WeightedPair, linear

# Rows from which one kernel does all of it, a workgroup to sixteen rows, and up to which the gate's product, the gate and
# the lookup are one kernel (all of the branch for a table part of 256, us, one kernel / few rows / in parts: width 2,048 at
# 16 rows 33 / 18 / 19, at 64 35 / 19 / 34, at 256 35 / 26 / 29, at 512 35 / 34 / 34, at 2,048 41 / 72 / 51; width 3,584 at 512
# rows 60 / 51 / 45, at 1,024 60 / 75 / 54, at 2,048 62 / 117 / 71)
WHOLE_FROM_ROWS = 512
FEW_ROWS = 511


class TokenSide(Part):
    graph_safe = True

    def __init__(self, hidden_size: int, dim: int, index: int, eps: float, names: tuple[str, str, str] = ("gate", "proj", "norm")) -> None:
        if hidden_size < 1 or dim < 1 or index < 0 or not eps > 0:
            raise ValueError(f"sizes and eps must be positive, got {hidden_size}, {dim}, {eps} at part {index}")
        if hidden_size > ops.MAX_NORM_WIDTH:
            raise ValueError(f"the norm kernels take rows of up to {ops.MAX_NORM_WIDTH} numbers, not {hidden_size}")
        self.hidden_size, self.dim, self.column, self.eps = hidden_size, dim, index * dim, float(eps)
        self.names = tuple(names)

    def expected_tensors(self, prefix: str) -> dict[str, TensorSpec]:
        gate, proj, norm = self.names
        return {prefix + gate: TensorSpec((self.dim, self.hidden_size)),
                prefix + proj: TensorSpec((self.hidden_size, self.dim)),
                prefix + norm: TensorSpec((self.hidden_size,), init="norm", keeps_float32=True)}

    def bind(self, tensors, prefix, dtype, device) -> None:
        super().bind(tensors, prefix, dtype, device)
        gate, proj, norm = self.names
        self.w_gate, self.w_proj = tensors[prefix + gate].contiguous(), tensors[prefix + proj].contiguous()
        self.weight = tensors[prefix + norm].float().contiguous()
        # the weights once more, as the kernels of this branch alone read them
        self.gate_pieces = self.proj_pieces = None
        if dtype == torch.bfloat16 and self.hidden_size % 8 == 0:
            self.gate_pieces = ops.weight_pieces(self.w_gate)
            if ops.plan_token_side(self.hidden_size, self.dim):
                self.proj_pieces = ops.weight_pieces(self.w_proj)

    def warm_up(self, rows: int) -> None:
        blank = lambda width: torch.zeros((rows, width), dtype=self.dtype, device=self.device)
        linear(blank(self.hidden_size), self.w_gate, out_dtype=torch.float32)
        linear(blank(self.dim), self.w_proj)

    def forward(self, residual: torch.Tensor, pending: Any, batch, dtype: torch.dtype,
                then: Any = None) -> Optional[torch.Tensor]:
        """``residual`` (float32, in place) takes what is pending and then this part's own branch; ``then``: an RMS norm of
        one group under which the new stream's rows come back."""
        if then is not None and then.eps != self.eps:  # (the kernels have one eps for both norms)
            self.forward(residual, pending, batch, dtype)
            return then.forward(residual, None, dtype)
        table, ids = batch.carried["side_table"], batch.carried["token_ids"]
        first = second = None
        if isinstance(pending, WeightedPair) and pending.scales == (1.0, 1.0):
            first, second = pending.first, pending.second
        elif isinstance(pending, WeightedPair):
            first = pending.combined()
        elif pending is not None and not isinstance(pending, (Added, RowSumsq)):
            first = pending
        tokens = residual.shape[0]
        if self.proj_pieces is not None and tokens >= WHOLE_FROM_ROWS and second is None:
            return ops.token_side(residual, first, self.gate_pieces, self.proj_pieces, self.dim, table, self.column, ids,
                                  self.weight, self.eps, next_weight=None if then is None else then.weight_f32)
        few = self.gate_pieces is not None and tokens <= FEW_ROWS
        rows = ops.stream_rows(residual, first, second, dtype, want_rows=dtype != torch.float32 and not few)
        if few:
            gated = ops.token_gate(residual, self.gate_pieces, self.dim, table, self.column, ids)
        else:
            z = linear(residual if rows is None else rows, self.w_gate, out_dtype=torch.float32)
            gated = ops.gated_token_rows(z, table, self.column, ids)
        y = linear(gated, self.w_proj)
        made = ops.branch_norm_add(residual, y, self.weight, self.eps, dtype, want_rows=False,
                                   next_weight=None if then is None else then.weight_f32)
        return None if then is None else made[1]


register_part("side", "token_side", TokenSide)
