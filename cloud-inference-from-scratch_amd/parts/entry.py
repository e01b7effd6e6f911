"""What remakes the stream in front of a call of the run order.

``JoinEmbedding``: a stream row and the embedding's row as it entered the stream, side by side, go through one product,
and a vector that belongs to the entry's number n joins the result: the first step of a run of layers that repeats.
The two halves of a row lie in one tensor of the activation type: the embedding kernel fills the right half once a step,
the kernel that ends the layer in front of an entry leaves the stream in the left one, and one product with float32
results makes the new stream.  The vector is handed on to the norm behind it, which adds it in its own kernel.
"""

from __future__ import annotations

import torch

from ..weights.tensors import TensorSpec
from .base import Part, register_part
from .linear import linear


class JoinEmbedding(Part):
    graph_safe = True

    def __init__(self, hidden_size: int, times: int, names: tuple[str, str] = ("in", "step")) -> None:
        if hidden_size < 1 or times < 1:
            raise ValueError(f"sizes must be positive, got {hidden_size} and {times} entries")
        self.hidden_size, self.times = hidden_size, times
        self.names = tuple(names)

    def expected_tensors(self, prefix: str) -> dict[str, TensorSpec]:
        return {prefix + self.names[0]: TensorSpec((self.hidden_size, 2 * self.hidden_size)),
                prefix + self.names[1]: TensorSpec((self.times, self.hidden_size), keeps_float32=True)}

    def bind(self, tensors, prefix, dtype, device) -> None:
        super().bind(tensors, prefix, dtype, device)
        self.weight = tensors[prefix + self.names[0]].contiguous()
        self.steps = tensors[prefix + self.names[1]].float().contiguous()

    def joint(self, tokens: int) -> torch.Tensor:
        return torch.empty((tokens, 2 * self.hidden_size), dtype=self.weight.dtype, device=self.weight.device)

    def warm_up(self, rows: int) -> None:
        self.forward(self.joint(rows).zero_(), 0)

    def forward(self, joint: torch.Tensor, number: int) -> tuple[torch.Tensor, torch.Tensor]:
        return linear(joint, self.weight, out_dtype=torch.float32), self.steps[number]


register_part("entry", "join_embedding", JoinEmbedding)
