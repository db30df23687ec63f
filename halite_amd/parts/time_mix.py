"""Time mixing: a recurrence with a matrix state per head whose projections read the token's
row mixed with the row before it.  With ``x'`` the previous token's row (zeros for a request's
first token), each of ``r, k, v, gate, decay`` reads its own mix ``x + (x' - x) * mu``, and per
head, with the state ``S`` (key channel x value channel, zero when a request starts),

    o_t = (S_(t-1) + diag(bonus) k_t v_t^T)^T r_t,   S_t = diag(w_t) S_(t-1) + k_t v_t^T,
    w_t = exp(-exp(decay.bias + W_up tanh(W_down mix_decay))).

Every head's ``o`` is divided by its root mean square, multiplied by a weight and by
``silu(W_gate mix_gate)``, and projected out.  Per request the mixer keeps the state (float32)
and the last token's row; it has no paged cache.  Decays, state, sums over the state, norm and
gate are float32.
"""

from __future__ import annotations

import torch
from pydantic import BaseModel, Field, StrictInt

from ..kernels import ops
from .base import MIXERS, Mixer, ParamDecl, StateNeed
from .state_space import plan_scan_chunks, scan_arrays


class TimeMixParams(BaseModel):
    hidden_size: StrictInt = Field(gt=0)
    n_heads: StrictInt = Field(gt=0)
    head_dim: StrictInt = Field(gt=0, le=256)
    decay_rank: StrictInt = Field(gt=0, le=1024)
    eps: float = Field(gt=0)


@MIXERS.register("time_mix")
class TimeMix(Mixer):
    Params = TimeMixParams
    graph_safe = True

    # the projections of one size, in the order of their weights, mixes and results; the decay's
    # inner projection reads the last mix
    _PROJECTIONS = ("r", "k", "v", "gate")

    def __init__(self, params, build):
        super().__init__(params, build)
        self.inner = params.n_heads * params.head_dim

    def param_decls(self):
        p = self.p
        d, n = p.hidden_size, self.inner
        decls = {f"mu.{name}": ParamDecl((d,)) for name in (*self._PROJECTIONS, "decay")}
        decls.update({f"{name}.weight": ParamDecl((n, d)) for name in self._PROJECTIONS})
        decls["decay_down.weight"] = ParamDecl((p.decay_rank, d))
        decls["decay_up.weight"] = ParamDecl((n, p.decay_rank))
        decls["decay.bias"] = ParamDecl((n,))
        decls["bonus"] = ParamDecl((p.n_heads, p.head_dim))
        decls["norm.weight"] = ParamDecl((n,), init="ones")
        decls["out.weight"] = ParamDecl((d, n))
        return decls

    def allocate(self, dtypes):
        p = self.p
        dev = self.build.device
        decls = self.param_decls()
        mus = [f"mu.{name}" for name in (*self._PROJECTIONS, "decay")]
        small = ["decay_up.weight", "decay.bias", "bonus", "norm.weight"]
        for names, what in ((mus, "shifts"), ([f"{n}.weight" for n in self._PROJECTIONS], "projections"),
                            (small, "decay, bonus and norm")):
            if len({dtypes[n] for n in names}) != 1:
                raise ValueError(f"the {what} of a time-mixing mixer are stored with different element types")
        self.w_mu = torch.empty((len(mus), p.hidden_size), dtype=dtypes[mus[0]], device=dev)
        self.w_in = torch.empty((len(self._PROJECTIONS), self.inner, p.hidden_size), dtype=dtypes["r.weight"], device=dev)
        out = {name: self.w_mu[i] for i, name in enumerate(mus)}
        out.update({f"{name}.weight": self.w_in[i] for i, name in enumerate(self._PROJECTIONS)})
        for name in decls:
            if name not in out:
                t = torch.empty(decls[name].shape, dtype=dtypes[name], device=dev)
                setattr(self, "w_" + name.replace(".", "_"), t)
                out[name] = t
        return out

    def finalize(self):
        self.t_down = self.t_out = None
        if self.build.tiled_weights and self.w_in.is_cuda:
            tile = lambda w: ops.tile_weight(w) if w.dtype == torch.bfloat16 and w.shape[1] % 8 == 0 else None  # noqa: E731
            self.t_down, self.t_out = tile(self.w_decay_down_weight), tile(self.w_out_weight)

    def state_need(self):
        p = self.p
        return {"state": StateNeed((p.n_heads, p.head_dim, p.head_dim)), "last": StateNeed((p.hidden_size,))}

    def prepare(self, ctx, run):
        plan_scan_chunks(ctx)  # (the state-space scan's cut, shared by the step's layers)

    def forward(self, x, ctx, run):
        p = self.p
        n, t = self.inner, x.shape[0]
        # few tokens: the four products of one size are one launch, on the mixes side by side
        together = x.dtype == torch.bfloat16 and self.w_in.dtype == torch.bfloat16 and t <= ops.SKINNY_ROWS
        mixed, mixed_decay = ops.token_shift(x, self.w_mu, run.state["last"], ctx, together)
        x1 = ops.linear(mixed_decay, self.w_decay_down_weight, out_dtype=torch.float32, tiled=self.t_down)
        if together:
            rows = torch.empty((t, 4 * n), dtype=torch.float32, device=x.device)
            ops.grouped_gemm(mixed, self.w_in, rows, n_rows=t, x_group_cols=p.hidden_size, y_group_cols=n)
            r, k, v, gate = (rows[:, i * n : (i + 1) * n] for i in range(4))
        else:
            r, k, v, gate = (ops.linear(mixed[i], self.w_in[i], out_dtype=torch.float32) for i in range(4))
        state = run.state["state"]
        if t == ctx.n_segs and p.head_dim in ops.WKV_STEP_DIMS:
            y = ops.wkv_step(r, k, v, gate, x1, self.w_decay_up_weight, self.w_decay_bias, self.w_bonus,
                             self.w_norm_weight, p.eps, state, ctx.token_slot, x.dtype)
        else:
            decay = torch.empty_strided((t, n), (r.stride(0), 1), dtype=torch.float32, device=x.device)
            ops.wkv_decay(x1, self.w_decay_up_weight, self.w_decay_bias, decay)
            o = ops.wkv_scan(r, k, v, decay, self.w_bonus, state, ctx.seg_q_start, ctx.seg_q_len, ctx.token_slot,
                             **scan_arrays(ctx))
            y = ops.head_norm_gate(o, gate, self.w_norm_weight, p.eps, p.n_heads, x.dtype, silu=True)
        return ops.linear(y, self.w_out_weight, out_dtype=torch.float32, tiled=self.t_out)
