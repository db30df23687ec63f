"""Parts that stand between two runs of the order and make the residual stream anew.

``reinjection``: ``x <- W [x; x0]`` with ``x0`` the embedding's output, which is what a stack of
layers that runs several times in a row does at the start of every pass.  The product's
operands are of the activation type, its sums float32 like the stream.
"""

from __future__ import annotations

import torch
from pydantic import BaseModel, Field, StrictInt

from ..kernels import ops
from .base import JUNCTIONS, Junction, ParamDecl


class ReinjectionParams(BaseModel):
    size: StrictInt = Field(gt=0)


@JUNCTIONS.register("reinjection")
class Reinjection(Junction):
    Params = ReinjectionParams
    graph_safe = True

    def param_decls(self):
        return {"weight": ParamDecl((self.p.size, 2 * self.p.size))}

    def finalize(self):
        self.t_weight = None
        if self.build.tiled_weights and self.weight.is_cuda and self.weight.dtype == torch.bfloat16 and self.p.size % 4 == 0:
            self.t_weight = ops.tile_weight(self.weight)

    def start(self, h0):
        # rows [x | x0]: the right half holds for the whole step, the left one is written at every pass
        rows = torch.empty((h0.shape[0], 2 * self.p.size), dtype=self.build.dtype, device=h0.device)
        ops.cast_cols(h0, rows[:, self.p.size :])
        return rows

    def stream_rows(self, kept):
        return kept[:, : self.p.size]

    def forward(self, kept):
        return ops.linear(kept, self.weight, out_dtype=torch.float32, tiled=self.t_weight)
