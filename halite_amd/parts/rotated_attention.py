"""Softmax self-attention over the paged cache with grouped heads and these pieces, each a
parameter:

* ``position``: a rotary encoding of the leading entries of every query and key head.
* ``value_position``: a rotary encoding of all entries of every value head: the value of the
  token at ``j`` is cached turned by ``j``, and a head's weighted sum for the query at ``i`` is
  turned back by ``i``, so a value arrives turned by its distance.
* ``window``: a query sees itself and the ``window - 1`` tokens before it; ``keep_first``: and the
  first so many tokens of its request, for ever, at their true positions.
* every head's result is multiplied by ``sigmoid(W_gate x)`` of that head, one number a head.

The key and value heads may differ in size; pages hold heads of the larger size (in steps
of 16), the rest zero.  Rotations, scores, softmax and gates are float32; the result is float32
(the accumulators of the output projection).
"""

from __future__ import annotations

import torch
from pydantic import BaseModel, Field, StrictInt, model_validator

from ..kernels import attention as attention_kernels
from ..kernels import ops
from .base import MIXERS, Mixer, PagedKVNeed, ParamDecl, RotaryPositionEncoding


class RotatedAttentionParams(BaseModel):
    hidden_size: StrictInt = Field(gt=0)
    n_heads: StrictInt = Field(gt=0)
    n_kv_heads: StrictInt = Field(gt=0)
    qk_dim: StrictInt = Field(gt=0)
    v_dim: StrictInt = Field(gt=0)
    scale: float
    position: str | None = None
    value_position: str | None = None
    window: StrictInt | None = Field(default=None, gt=0)
    keep_first: StrictInt = Field(default=0, ge=0)

    @model_validator(mode="after")
    def _check(self):
        if self.n_heads % self.n_kv_heads:
            raise ValueError(f"{self.n_heads} heads are not a multiple of {self.n_kv_heads} kv heads")
        return self


@MIXERS.register("rotated_attention")
class RotatedAttention(Mixer):
    Params = RotatedAttentionParams
    graph_safe = True

    def __init__(self, params, build):
        super().__init__(params, build)
        p = params
        self.head_dim = -(-max(p.qk_dim, p.v_dim) // 16) * 16
        self.n_q, self.n_k, self.n_v = p.n_heads * p.qk_dim, p.n_kv_heads * p.qk_dim, p.n_kv_heads * p.v_dim
        self.position = self._encoding(p.position, p.qk_dim, whole=False)
        self.value_position = self._encoding(p.value_position, p.v_dim, whole=True)
        if None not in (self.position, self.value_position) and self.position.interleaved != self.value_position.interleaved:
            raise ValueError("keys and values are turned in pairs of one layout")
        # (without a window every key stays visible anyway)
        self.keep = p.keep_first if p.window is not None else 0

    def _encoding(self, name, dim: int, whole: bool):
        if name is None:
            return None
        if name not in self.build.positions:
            raise ValueError(f"attention names position encoding {name!r}, which the model does not define")
        position = self.build.positions[name]
        if not isinstance(position, RotaryPositionEncoding):
            raise ValueError(f"position encoding {name!r} is not a RotaryPositionEncoding")
        if position.rotary_dim > dim or (whole and position.rotary_dim != dim):
            raise ValueError(f"position encoding {name!r} turns {position.rotary_dim} entries of a head of {dim}")
        return position

    def attention_sizes(self):
        return self.p.n_heads, self.p.n_kv_heads, self.p.qk_dim

    def param_decls(self):
        p = self.p
        d = p.hidden_size
        return {"q.weight": ParamDecl((self.n_q, d)), "k.weight": ParamDecl((self.n_k, d)),
                "v.weight": ParamDecl((self.n_v, d)), "gate.weight": ParamDecl((p.n_heads, d)),
                "out.weight": ParamDecl((d, p.n_heads * p.v_dim))}

    def allocate(self, dtypes):
        p = self.p
        dev = self.build.device
        names = ("q", "k", "v", "gate")
        if len({dtypes[f"{n}.weight"] for n in names}) != 1:
            raise ValueError("q, k, v and gate weights are stored with different element types")
        rows = {"q": self.n_q, "k": self.n_k, "v": self.n_v, "gate": p.n_heads}
        # one product for q, k, v and the gate
        self.w_in = torch.empty((sum(rows.values()), p.hidden_size), dtype=dtypes["q.weight"], device=dev)
        out, at = {}, 0
        for n in names:
            out[f"{n}.weight"] = self.w_in[at : at + rows[n]]
            at += rows[n]
        self.w_out = torch.empty((p.hidden_size, p.n_heads * p.v_dim), dtype=dtypes["out.weight"], device=dev)
        out["out.weight"] = self.w_out
        return out

    def finalize(self):
        p = self.p
        self.t_in = self.t_out = None
        if self.build.tiled_weights and self.w_in.is_cuda and self.w_in.dtype == torch.bfloat16:
            if p.hidden_size % 8 == 0:
                self.t_in = ops.tile_weight(self.w_in)
            if (p.n_heads * p.v_dim) % 8 == 0 and self.w_out.dtype == torch.bfloat16:
                self.t_out = ops.tile_weight(self.w_out)
        self.rule = ops.ScoreRule(keep=self.keep) if self.keep else None

    def cache_need(self):
        # (the attention kernels walk the kept keys in whole units)
        return PagedKVNeed(self.p.n_kv_heads, self.head_dim, self.p.window, keep=attention_kernels.kept_units(self.keep))

    def prepare(self, ctx, run):
        group = ctx.cache.groups[run.kv.group_id]
        if attention_kernels.mfma_supported(self.build.dtype, self.head_dim, group.page_size):
            ctx.plan_attention(group.group_id, self.p.n_heads, self.p.n_kv_heads, self.p.window or 0, self.head_dim,
                               keep=self.keep)

    def forward(self, x, ctx, run):
        p = self.p
        kv = run.kv
        group = ctx.group(kv.group_id)
        D = self.head_dim
        a = ops.linear(x, self.w_in, out_dtype=torch.float32, tiled=self.t_in)
        n_qk = self.n_q + self.n_k
        q, k, v, gate = a[:, : self.n_q], a[:, self.n_q : n_qk], a[:, n_qk : n_qk + self.n_v], a[:, n_qk + self.n_v :]
        pages = dict(token_seg=ctx.token_seg, block_table=group.block_table, k_pages=kv.k, v_pages=kv.v,
                     page_size=group.page_size, tiled=kv.tiled)
        tables, back = {}, {}
        if self.position is not None:
            tables["cos"], tables["sin"] = self.position.tables(ctx.max_position + 1)
            tables["interleaved"] = self.position.interleaved
        if self.value_position is not None:
            tables["cos_v"], tables["sin_v"] = self.value_position.tables(ctx.max_position + 1)
            tables["interleaved"] = self.value_position.interleaved
            back = dict(positions=ctx.positions, cos=tables["cos_v"], sin=tables["sin_v"], interleaved=tables["interleaved"])
        packed = ops.turn_pack(q, k, v, ctx.positions, p.n_heads, p.n_kv_heads, p.qk_dim, p.v_dim, D, x.dtype,
                               **tables, **(pages if run.appends else {}))
        out = ctx.attention(packed, packed.shape[1], kv, group, p.n_heads, p.scale, p.window or 0, rule=self.rule)
        heads = ops.head_gate_cols(out, D, gate, p.v_dim, p.n_heads, **back)
        return ops.linear(heads, self.w_out, out_dtype=torch.float32, tiled=self.t_out)
