"""A gated recurrence per channel whose gates read the token alone (a minimal gated recurrent
unit): with ``z = sigmoid(W_z x + b_z)``, ``u = W_x x + b_x`` and the candidate ``u + 1/2`` where
``u >= 0`` and ``sigmoid(u)`` elsewhere,

    S_t = (1 - z_t) * S_(t-1) + z_t * candidate_t,   result = W_out (S_t * silu(W_gate x_t)).

Per request the mixer keeps the state (float32, zero at the start); it has no paged cache.
Since the gates do not read the state, long prompts are cut into chunks that are walked side
by side.  Gates, candidates and the state are float32.
"""

from __future__ import annotations

import torch
from pydantic import BaseModel, Field, StrictInt

from ..kernels import ops
from .base import MIXERS, Mixer, ParamDecl, StateNeed
from .state_space import plan_scan_chunks, scan_arrays


class MinGRUParams(BaseModel):
    hidden_size: StrictInt = Field(gt=0)
    width: StrictInt = Field(gt=0)


@MIXERS.register("mingru")
class MinGRU(Mixer):
    Params = MinGRUParams
    graph_safe = True

    def param_decls(self):
        d, n = self.p.hidden_size, self.p.width
        decls = {f"{name}.weight": ParamDecl((n, d)) for name in ("z", "x", "gate")}
        decls.update({"z.bias": ParamDecl((n,)), "x.bias": ParamDecl((n,)), "out.weight": ParamDecl((d, n))})
        return decls

    def allocate(self, dtypes):
        d, n = self.p.hidden_size, self.p.width
        dev = self.build.device
        if len({dtypes[f"{name}.weight"] for name in ("z", "x", "gate")}) != 1 or dtypes["z.bias"] != dtypes["x.bias"]:
            raise ValueError("the gates' weights (and biases) are stored with different element types")
        # one product, its rows in the scan's order
        self.w_in = torch.empty((3 * n, d), dtype=dtypes["z.weight"], device=dev)
        out = {f"{name}.weight": self.w_in[i * n : (i + 1) * n] for i, name in enumerate(("z", "x", "gate"))}
        for name, shape in (("z.bias", (n,)), ("x.bias", (n,)), ("out.weight", (d, n))):
            t = torch.empty(shape, dtype=dtypes[name], device=dev)
            setattr(self, "w_" + name.replace(".", "_"), t)
            out[name] = t
        return out

    def finalize(self):
        self.t_in = self.t_out = None
        if self.build.tiled_weights and self.w_in.is_cuda:
            tile = lambda w: ops.tile_weight(w) if w.dtype == torch.bfloat16 and w.shape[1] % 8 == 0 else None  # noqa: E731
            self.t_in, self.t_out = tile(self.w_in), tile(self.w_out_weight)

    def state_need(self):
        return {"state": StateNeed((self.p.width,))}

    def prepare(self, ctx, run):
        plan_scan_chunks(ctx)  # (the state-space scan's cut, shared by the step's layers)

    def forward(self, x, ctx, run):
        a = ops.linear(x, self.w_in, out_dtype=torch.float32, tiled=self.t_in)
        y = ops.gated_scan(a, self.w_z_bias, self.w_x_bias, run.state["state"], ctx.seg_q_start, ctx.seg_q_len,
                           ctx.token_slot, x.dtype, **scan_arrays(ctx))
        return ops.linear(y, self.w_out_weight, out_dtype=torch.float32, tiled=self.t_out)
