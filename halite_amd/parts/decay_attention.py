"""A linear attention with one constant decay per head ("lightning" attention, retention): per
head a state ``S`` of ``qk_dim x v_dim`` numbers, zero when a request starts, that every token
decays and writes to, ``S_t = decay_h S_(t-1) + k_t v_t^T``, and reads from, ``o_t = S_t^T q_t``.
Its pieces, each a parameter:

* ``activation``: what the projections ``q = act(W_q x)``, ``k = act(W_k x)``, ``v = act(W_v x)`` go
  through (SiLU, or nothing).
* ``position``: a rotary encoding of the leading entries of every query and key head.
* ``key_scale``: a number that the keys are multiplied by (after the rotation).
* the result is divided by its root mean square, over the whole row of all heads or
  (``norm_per_head``) each head on its own; with ``norm_weight`` it is multiplied by a weight of the
  row's size.
* ``gate``: it is multiplied by ``sigmoid(W_g x)`` or by ``silu(W_g x)`` element by element, and
  projected out.

Per request the mixer keeps the state (float32); it has no paged cache.  The recurrence is
the state-space scan's with constant decays and unit step sizes (keys in the place of its
``B``, queries of its ``C``, one group a head), so prompts are cut into chunks in the same way; for
states of up to 128 x 256 a chunk's part is computed as products on the matrix cores (float32),
larger ones are walked.  A step of single tokens whose heads are normed each on its own is one
kernel from the projections to the gated rows.  Rotation, decays, state, sums over the
state, norm and gate are float32.
"""

from __future__ import annotations

from typing import Literal

import torch
from pydantic import BaseModel, Field, StrictBool, StrictInt, model_validator

from ..kernels import ops
from .base import MIXERS, Mixer, ParamDecl, RotaryPositionEncoding, StateNeed
from .state_space import SCAN_CHUNK, plan_scan_chunks, scan_arrays


class DecayAttentionParams(BaseModel):
    hidden_size: StrictInt = Field(gt=0)
    n_heads: StrictInt = Field(gt=0)
    qk_dim: StrictInt = Field(gt=0, le=256)
    v_dim: StrictInt = Field(gt=0)
    decay: list[float]
    """One number in (0, 1] a head."""
    eps: float = Field(gt=0)
    activation: Literal["silu"] | None = "silu"
    position: str | None = None
    key_scale: float = 1.0
    norm_per_head: StrictBool = False
    norm_weight: StrictBool = True
    gate: Literal["sigmoid", "silu"] = "sigmoid"

    @model_validator(mode="after")
    def _check(self):
        if len(self.decay) != self.n_heads:
            raise ValueError(f"{len(self.decay)} decays for {self.n_heads} heads")
        if any(not 0.0 < d <= 1.0 for d in self.decay):
            raise ValueError("a head's decay lies in (0, 1]")
        if self.activation is not None and (self.position is not None or self.key_scale != 1.0):
            raise ValueError("queries and keys that are turned or scaled come without an activation")
        return self


@MIXERS.register("decay_attention")
class DecayAttention(Mixer):
    Params = DecayAttentionParams
    graph_safe = True

    def __init__(self, params, build):
        super().__init__(params, build)
        p = params
        self.inner = p.n_heads * p.v_dim
        self.n_qk = p.n_heads * p.qk_dim
        self.position = None
        if p.position is not None:
            if p.position not in build.positions:
                raise ValueError(f"linear attention names position encoding {p.position!r}, which the model does not define")
            self.position = build.positions[p.position]
            if not isinstance(self.position, RotaryPositionEncoding):
                raise ValueError(f"position encoding {p.position!r} is not a RotaryPositionEncoding")
            if self.position.rotary_dim > p.qk_dim:
                raise ValueError("the position encoding rotates more elements than a head has")

    def param_decls(self):
        p = self.p
        d = p.hidden_size
        decls = {
            "v.weight": ParamDecl((self.inner, d)), "k.weight": ParamDecl((self.n_qk, d)),
            "q.weight": ParamDecl((self.n_qk, d)), "gate.weight": ParamDecl((self.inner, d)),
        }
        if p.norm_weight:
            decls["norm.weight"] = ParamDecl((self.inner,), init="ones")
        decls["out.weight"] = ParamDecl((d, self.inner))
        return decls

    def allocate(self, dtypes):
        p = self.p
        dev = self.build.device
        names = ("v", "k", "q", "gate")
        if len({dtypes[f"{n}.weight"] for n in names}) != 1:
            raise ValueError("q, k, v and gate weights are stored with different element types")
        rows = {"v": self.inner, "k": self.n_qk, "q": self.n_qk, "gate": self.inner}
        # one product, its rows in the scan's order: values, keys, queries; then the gate
        self.w_in = torch.empty((sum(rows.values()), p.hidden_size), dtype=dtypes["q.weight"], device=dev)
        out, at = {}, 0
        for n in names:
            out[f"{n}.weight"] = self.w_in[at : at + rows[n]]
            at += rows[n]
        self.w_norm = None
        if p.norm_weight:
            self.w_norm = torch.empty((self.inner,), dtype=dtypes["norm.weight"], device=dev)
            out["norm.weight"] = self.w_norm
        self.w_out = torch.empty((p.hidden_size, self.inner), dtype=dtypes["out.weight"], device=dev)
        out["out.weight"] = self.w_out
        return out

    def finalize(self):
        p = self.p
        decay = torch.tensor(p.decay, dtype=torch.float64)
        self.decay, self.powers = decay.float().to(self.build.device), ops.decay_powers(decay).to(self.build.device)
        self.t_in = self.t_out = None
        if self.build.tiled_weights and self.w_in.is_cuda and self.w_in.dtype == torch.bfloat16:
            if p.hidden_size % 8 == 0:
                self.t_in = ops.tile_weight(self.w_in)
            if self.inner % 8 == 0 and self.w_out.dtype == torch.bfloat16:
                self.t_out = ops.tile_weight(self.w_out)

    def state_need(self):
        p = self.p
        return {"state": StateNeed((p.n_heads, p.qk_dim, p.v_dim))}

    def prepare(self, ctx, run):
        plan_scan_chunks(ctx)  # (the state-space scan's cut, shared by the step's layers)

    def forward(self, x, ctx, run):
        p = self.p
        n_act = self.inner + 2 * self.n_qk
        a = ops.linear(x, self.w_in, out_dtype=torch.float32, tiled=self.t_in)
        gate, silu = a[:, n_act:], p.gate == "silu"
        turn = {}
        if self.position is not None:
            cos, sin = self.position.tables(ctx.max_position + 1)
            turn = dict(positions=ctx.positions, cos=cos, sin=sin, interleaved=self.position.interleaved)
        state = run.state["state"]
        values, keys, queries = a[:, : self.inner], a[:, self.inner : self.inner + self.n_qk], a[:, self.inner + self.n_qk : n_act]
        recur = dict(k_scale=p.key_scale, in_silu=p.activation == "silu", **turn)
        finish = dict(eps=p.eps, out_dtype=x.dtype, weight=self.w_norm, silu=silu)
        if p.norm_per_head and x.shape[0] == ctx.n_segs and ops.decay_step_fits(p.qk_dim, p.v_dim):
            # single tokens: one kernel
            gated = ops.decay_step(values, keys, queries, gate, self.decay, state, ctx.token_slot, **finish, **recur)
            return ops.linear(gated, self.w_out, out_dtype=torch.float32, tiled=self.t_out)
        cut = scan_arrays(ctx)
        if cut["chunks"] is not None and SCAN_CHUNK <= ops.DECAY_CHUNK and ops.decay_chunks_fit(p.qk_dim, p.v_dim):
            # long segments: chunks as products
            segs = (ctx.seg_q_start, ctx.seg_q_len, ctx.token_slot)
            if p.norm_per_head and p.activation is None:
                gated = ops.decay_chunks(values, keys, queries, gate, self.powers, state, *segs, **cut, **finish, **recur)
            else:
                y = ops.decay_chunks(values, keys, queries, None, self.powers, state, *segs, **cut, **recur)
                gated = ops.head_norm_gate(y, gate, self.w_norm, p.eps, p.n_heads if p.norm_per_head else 1, x.dtype, silu=silu)
            return ops.linear(gated, self.w_out, out_dtype=torch.float32, tiled=self.t_out)
        if turn or p.key_scale != 1.0:
            ops.rotate_heads_(a[:, self.inner : n_act], 2 * p.n_heads, p.qk_dim, n_scaled=p.n_heads, scale=p.key_scale, **turn)
        # (SiLU of values, keys and queries where the scan reads them: float32 in either mode)
        y = ops.ssd_scan(a[:, :n_act], None, None, None, None, state, ctx.seg_q_start, ctx.seg_q_len, ctx.token_slot,
                         p.n_heads, fixed_decay=self.decay, in_silu=p.activation == "silu", **cut)
        gated = ops.head_norm_gate(y, gate, self.w_norm, p.eps, p.n_heads if p.norm_per_head else 1, x.dtype, silu=silu)
        return ops.linear(gated, self.w_out, out_dtype=torch.float32, tiled=self.t_out)
