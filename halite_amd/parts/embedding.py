"""Token embedding and output head (src/halite/transformers/embedding.py:7-51;
src/halite/transformers/feedforward.py:72-114)."""

from __future__ import annotations

import torch
from pydantic import BaseModel, Field, StrictBool, StrictInt, model_validator

from ..kernels import ops
from .base import EMBEDDINGS, HEADS, Embedding, Head, ParamDecl, StateNeed


class TokenPairs(BaseModel):
    """A table of ``buckets + 1`` rows that is indexed by the token before and the token: row
    ``(before * mul_prev + token * mul_cur) mod buckets``; a request's first token has the last row."""

    buckets: StrictInt = Field(gt=0, lt=2**31 - 1)
    mul_prev: StrictInt = Field(ge=0, lt=2**31)
    mul_cur: StrictInt = Field(ge=0, lt=2**31)


class EmbeddingParams(BaseModel):
    vocab_size: StrictInt = Field(gt=0)
    size: StrictInt = Field(gt=0)
    scale: float = 1.0
    """Every row is multiplied by this on its way into the stream (in float32)."""
    norm_eps: float | None = Field(default=None, gt=0)
    """With a value: a tensor ``norm.weight`` of the rows' size, and every row enters the
    stream as ``x / sqrt(mean(x^2) + norm_eps) * weight`` (float32)."""
    side_size: StrictInt | None = Field(default=None, gt=0)
    """With a value: a second table ``side.weight`` ``[vocab_size, side_size]`` of which parts of
    the layers read column ranges by token (``BuildContext.embedding.side_weight``)."""
    pairs: TokenPairs | None = None
    """With a value: a table ``pairs.weight`` ``[buckets + 1, size]`` whose row for the token and the one
    before it is added to the scaled row (float32); a request's last token is state that it
    keeps between steps."""

    @model_validator(mode="after")
    def _check(self):
        if self.pairs is not None and self.norm_eps is not None:
            raise ValueError("rows with a table of pairs are not normed")
        return self


@EMBEDDINGS.register("embedding")
class TokenEmbedding(Embedding):
    """Row lookup (embedding.py:36-44) into the float32 residual stream, times ``scale``
    (1 in the reference's models)."""

    Params = EmbeddingParams
    graph_safe = True

    def param_decls(self):
        decls = {"weight": ParamDecl((self.p.vocab_size, self.p.size))}
        if self.p.norm_eps is not None:
            decls["norm.weight"] = ParamDecl((self.p.size,), init="ones")
        if self.p.side_size is not None:
            decls["side.weight"] = ParamDecl((self.p.vocab_size, self.p.side_size))
        if self.p.pairs is not None:
            decls["pairs.weight"] = ParamDecl((self.p.pairs.buckets + 1, self.p.size))
        return decls

    def allocate(self, dtypes):
        if self.p.pairs is not None and dtypes["pairs.weight"] != dtypes["weight"]:
            raise ValueError("the embedding and its table of pairs are stored with different element types")
        return super().allocate(dtypes)

    @property
    def reads_step(self):
        return self.p.pairs is not None

    def state_need(self):
        if self.p.pairs is None:
            return {}
        return {"last_id": StateNeed((1,), torch.int32)}

    def forward(self, tokens, out=None, ctx=None, run=None):
        if self.p.pairs is not None:
            b = self.p.pairs
            return ops.pair_embedding(tokens, self.weight, self.pairs_weight, self.p.scale, b.mul_prev, b.mul_cur, ctx,
                                      run.state["last_id"], out=out)
        if self.p.norm_eps is None:
            return ops.embedding(tokens, self.weight, out=out, scale=self.p.scale)
        x = ops.rmsnorm_exact(ops.embedding(tokens, self.weight, scale=self.p.scale), self.norm_weight, self.p.norm_eps,
                              torch.float32)
        if out is None:
            return x
        out.copy_(x)
        return out


class LinearHeadParams(BaseModel):
    vocab_size: StrictInt = Field(gt=0)
    size: StrictInt = Field(gt=0)
    tied: StrictBool = False
    logit_scale: float = 1.0
    """The float32 logits are multiplied by this."""
    logit_softcap: float | None = Field(default=None, gt=0)
    """With a value: the scaled logits ``z`` become ``logit_softcap * tanh(z / logit_softcap)``."""


@HEADS.register("linear_head")
class LinearHead(Head):
    """Bias-free projection to the vocabulary with float32 logits
    (src/halite/transformers/infer/postprocessor.py:45-57).  When ``tied`` the
    weight is the embedding's table itself
    (src/halite/transformers/transformer.py:59-61), bound by the model builder."""

    Params = LinearHeadParams
    graph_safe = True

    def param_decls(self):
        if self.p.tied:
            return {}
        return {"weight": ParamDecl((self.p.vocab_size, self.p.size))}

    def bind(self, embedding):
        if self.p.tied:
            self.weight = embedding.weight

    def finalize(self):
        self.t_weight = None
        if self.build.tiled_weights and self.weight.dtype == torch.bfloat16 and self.weight.is_cuda:
            self.t_weight = ops.tile_weight(self.weight)

    def forward(self, x):
        z = ops.scale_(ops.linear(x, self.weight, out_dtype=torch.float32, tiled=self.t_weight), self.p.logit_scale)
        return z if self.p.logit_softcap is None else ops.soft_cap_(z, self.p.logit_softcap)
