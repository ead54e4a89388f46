"""What may happen to the residual stream between two layer runs."""
from __future__ import annotations

from typing import Any, Dict, List

import torch

from .. import ops
from .base import BuildContext, Junction, ResidualStream, TensorSpec, join, register


@register("junction", "embedding_rejoin")
class EmbeddingRejoin(Junction):
    """The stream starts over from one linear map of itself and of the embedding output:
    ``x <- Wx x + We x0``, the two square maps stored side by side as one tensor ``(W, 2 W)``, x's
    columns in front.

    Parameters: ``hidden_size``.  The tensor is the prefix itself.  ``We x0`` is the same wherever a
    step runs the part: it is made once, and every use is one product of the stream's rows (in the
    activation dtype, the result float32) whose sum with it is left for the norm behind it to form
    on its way."""

    graph_safe = True

    @classmethod
    def tensor_specs(cls, params: Dict[str, Any], prefix: str) -> List[TensorSpec]:
        W = params["hidden_size"]
        return [TensorSpec(prefix, (W, 2 * W))]

    def __init__(self, params: Dict[str, Any], prefix: str, ctx: BuildContext):
        super().__init__(params, prefix, ctx)
        W = int(params["hidden_size"])
        w = ctx.take(prefix)
        self.w_stream, self.w_embedding = (t.contiguous() for t in (w[:, :W], w[:, W:]))

    def begin(self, stream: ResidualStream) -> torch.Tensor:
        return ops.linear_f32(stream.rows(), self.w_embedding)

    def forward(self, stream: ResidualStream, kept: torch.Tensor) -> None:
        y = ops.linear(stream.rows(), self.w_stream, torch.float32, partials=True)
        if y.dim() == 3:
            stream.x = ops.weighted_sum(y, 1.0, kept, 1.0)
        else:
            stream.x = y
            stream.add(kept)
