"""Typed configuration of the Nodupel decoder, read from its own ``config.json`` keys.

Every size and every constant that can differ between two models of the design is a key
of the file and has no default here; a key that the file leaves out switches its mechanism
off (no table of token pairs, no loop, no window or no kept first tokens, no stretched
frequencies, no rotation, a residual multiplier of one, logits without a cap).  The rank of
a time-mixing mixer's decay projection is not a key of the file: it is the first dimension of
the layer's ``mix.right.w1`` tensor and is filled in from the folder's tensors
(``complete_from_tensors``); a configuration that is used without a folder (random weights)
states it as ``decay_rank``.
"""

from __future__ import annotations

from typing import Annotated, Literal, Union

from pydantic import BaseModel, ConfigDict, Field, model_validator

from .zabunex import Size, _Keys


class NodupelNorm(_Keys):
    eps: float = Field(gt=0)


class NodupelBigram(_Keys):
    buckets: Size = Field(gt=0, lt=2**31 - 1)
    mul_prev: Size = Field(ge=0, lt=2**31)
    mul_cur: Size = Field(ge=0, lt=2**31)


class NodupelEmbedding(_Keys):
    scale: float
    bigram: NodupelBigram | None = None


class NodupelMask(_Keys):
    size: Size = Field(gt=0)
    keep_first: Size = Field(default=0, ge=0)


class NodupelRotScaling(_Keys):
    factor: float = Field(gt=0)


class NodupelRot(_Keys):
    base: float = Field(gt=0)
    dims: Size = Field(gt=0)
    scaling: NodupelRotScaling | None = None


class NodupelAttention(_Keys):
    heads: Size = Field(gt=0)
    kv_heads: Size = Field(gt=0)
    dim: Size = Field(gt=0)
    vdim: Size = Field(gt=0)
    scale: float
    rot: NodupelRot | None = None
    mask: NodupelMask | None = None

    @model_validator(mode="after")
    def _check(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} heads are not a multiple of {self.kv_heads} kv_heads")
        if self.rot is not None and (self.rot.dims % 2 or self.rot.dims > self.dim):
            raise ValueError(f"rot.dims {self.rot.dims} must be even and at most dim {self.dim}")
        if self.rot is not None and self.vdim % 2:
            raise ValueError(f"values of {self.vdim} entries are turned in pairs")
        return self


class NodupelTimeMix(_Keys):
    heads: Size = Field(gt=0)
    dim: Size = Field(gt=0)
    decay_rank: Size | None = Field(default=None, gt=0)


class NodupelParallelMixer(_Keys):
    left: NodupelAttention
    right: NodupelTimeMix


class NodupelMinGRUMixer(_Keys):
    width: Size = Field(gt=0)


class NodupelDense(_Keys):
    kind: Literal["dense"]
    ff: Size = Field(gt=0)


class NodupelParallelLayer(_Keys):
    type: Literal["parallel"]
    mixer: NodupelParallelMixer
    mlp: NodupelDense | None = None


class NodupelMinGRULayer(_Keys):
    type: Literal["mingru"]
    mixer: NodupelMinGRUMixer
    mlp: NodupelDense | None = None


NodupelLayer = Annotated[Union[NodupelParallelLayer, NodupelMinGRULayer], Field(discriminator="type")]


class NodupelLoop(_Keys):
    start: Size = Field(ge=0)
    stop: Size = Field(gt=0)
    times: Size = Field(gt=0)


class NodupelConfig(BaseModel):
    """``config.json`` of a Nodupel folder."""

    model_config = ConfigDict(extra="ignore")

    architecture: Literal["Nodupel"]
    vocab: Size = Field(gt=0)
    width: Size = Field(gt=0)
    norm: NodupelNorm
    embedding: NodupelEmbedding
    layers: list[NodupelLayer] = Field(min_length=1)
    loop: NodupelLoop | None = None
    """Layers ``start`` to ``stop - 1`` run ``times`` times in a row (absent: every layer once)."""
    residual_mult: float | None = None
    """What a part's result is multiplied by on its way into the stream (absent: one)."""
    logit_softcap: float | None = Field(default=None, gt=0)
    max_positions: Size | None = Field(default=None, gt=0)
    """Not a key of the design (a request may be as long as the cache allows)."""
    stop_token_ids: tuple[int, ...] = ()

    @model_validator(mode="after")
    def _check(self):
        loop = self.loop
        if loop is not None and not loop.start < loop.stop <= len(self.layers):
            raise ValueError(f"loop from {loop.start} to {loop.stop} of {len(self.layers)} layers")
        return self

    @property
    def architectures(self) -> list[str]:
        return [self.architecture]

    def to_json_dict(self) -> dict:
        d = self.model_dump(exclude_none=True)
        if not self.stop_token_ids:
            d.pop("stop_token_ids")
        for layer in d["layers"]:
            if layer["type"] == "parallel":
                layer["mixer"]["right"].pop("decay_rank", None)  # the tensor's shape says it
            layer.setdefault("mlp", None)
        return d
