"""The embedding's output brought back into the residual: x <- W [x; x0], W [hidden, 2 hidden], x0 the residual as the
embedding left it, x first.  For models some of whose layers run several times in a row: every pass then starts from where
the last one ended and from the tokens themselves.

Each row of [x; x0] lies in one buffer in the activations' type: x0 is written there once a step, x by the kernel that
also does the update still pending (``pulse_residual_norms``), and the product leaves its float32 result in the residual.
A vector that the run adds (``RunSpec.offset``) is handed on to the kernel that reads the residual next.
"""
from __future__ import annotations

from typing import Any, Dict, List, Optional, Tuple

import torch

from ..ops import kernels
from ..weights.store import TensorSpec
from .base import BuildContext, Part, ResidualStream, StepContext, SumUpdate
from .linear import Linear


class OriginRejoin(Part):
    """Parameters: ``hidden_size``, ``name`` (the tensor's)."""

    records_cleanly = True

    @classmethod
    def weight_specs(cls, params: Dict[str, Any]) -> Dict[str, TensorSpec]:
        hidden = params["hidden_size"]
        return {params["name"]: TensorSpec((hidden, 2 * hidden), fan_in=2 * hidden)}

    def __init__(self, params: Dict[str, Any], build: BuildContext):
        self.hidden = int(params["hidden_size"])
        self.linear = Linear(build.loader.get(params["name"]), build.mode)
        self.act_dtype = build.act_dtype

    @staticmethod
    def rows(ctx: StepContext, tokens: int, hidden: int, dtype: torch.dtype) -> torch.Tensor:
        """[x | x0] of the step's tokens (one buffer for all tensors of a model: x0 is the same)."""
        return ctx.workspace.buffer("rejoin.rows", tokens, 2 * hidden, dtype)

    @classmethod
    def keep_origin(cls, h: torch.Tensor, ctx: StepContext, dtype: torch.dtype) -> None:
        """The residual as the embedding leaves it, kept for the step."""
        tokens, hidden = h.shape
        kernels.residual_norms(h, [], outs=[(cls.rows(ctx, tokens, hidden, dtype)[:, hidden:], None, 0.0)])

    def forward(self, stream: ResidualStream, ctx: StepContext, row: Optional[torch.Tensor] = None) -> None:
        """``row`` [hidden]: a vector added to every row of the result."""
        tokens = stream.h.shape[0]
        both = self.rows(ctx, tokens, self.hidden, self.act_dtype)
        update = stream.take_sum()
        kernels.residual_norms(stream.h, update.terms, experts=update.experts_args(), row=update.row,
                               outs=[(both[:, :self.hidden], None, 0.0)])
        stream.stats = stream.copy = None
        self.linear.forward(both, stream.h)
        if row is not None:
            stream.push(SumUpdate([], row=row))
