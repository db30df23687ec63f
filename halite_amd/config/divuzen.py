"""Typed configuration of the Divuzen decoder, read from its own ``config.json`` keys.

Every size and every constant that can differ between two models of the design is a key
of the file and has no default here; a key that the file leaves out switches its mechanism
off (no rotation, no limit on a dense feed-forward's products, no groups of experts, no shared
expert, no feed-forward; a scale that is left out multiplies nothing).
"""

from __future__ import annotations

from typing import Annotated, Literal, Union

from pydantic import BaseModel, ConfigDict, Field, model_validator

from .zabunex import Size, _Keys


class DivuzenNorm(_Keys):
    eps: float = Field(gt=0)


class DivuzenRot(_Keys):
    base: float = Field(gt=0)
    dims: Size = Field(gt=0)


def _check_rotation(rot: DivuzenRot | None, dim: int) -> None:
    if rot is not None and (rot.dims % 2 or rot.dims > dim):
        raise ValueError(f"rot.dims {rot.dims} must be even and at most dim {dim}")


class DivuzenAttentionMixer(_Keys):
    heads: Size = Field(gt=0)
    kv_heads: Size = Field(gt=0)
    dim: Size = Field(gt=0)
    vdim: Size = Field(gt=0)
    scale: float = Field(gt=0)
    rot: DivuzenRot | None = None
    kv_from: Size | None = Field(default=None, ge=0)
    """An earlier attention layer whose keys and values this one attends to (it has none of its own)."""

    @model_validator(mode="after")
    def _check(self):
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} heads are not a multiple of {self.kv_heads} kv_heads")
        _check_rotation(self.rot, self.dim)
        return self


class DivuzenRetentionMixer(_Keys):
    heads: Size = Field(gt=0)
    dim: Size = Field(gt=0)
    vdim: Size = Field(gt=0)
    decay: list[float]
    rot: DivuzenRot | None = None

    @model_validator(mode="after")
    def _check(self):
        if len(self.decay) != self.heads:
            raise ValueError(f"{len(self.decay)} decays for {self.heads} heads")
        _check_rotation(self.rot, self.dim)
        return self


class DivuzenDense(_Keys):
    kind: Literal["dense"]
    ff: Size = Field(gt=0)
    limit: float | None = Field(default=None, gt=0)


class DivuzenExpert(_Keys):
    ff: Size = Field(gt=0)


class DivuzenGroups(_Keys):
    count: Size = Field(gt=0)
    keep: Size = Field(gt=0)


class DivuzenRouter(_Keys):
    experts: Size = Field(gt=0)
    top: Size = Field(gt=0)
    scale: float = 1.0
    groups: DivuzenGroups | None = None

    @model_validator(mode="after")
    def _check(self):
        open_ = self.experts
        g = self.groups
        if g is not None:
            if self.experts % g.count or g.keep > g.count:
                raise ValueError(f"{self.experts} experts in {g.count} equal groups of which {g.keep} are kept")
            open_ = self.experts // g.count * g.keep
        if self.top > open_:
            raise ValueError(f"top {self.top} of {open_} experts")
        return self


class DivuzenMoE(_Keys):
    kind: Literal["moe"]
    expert: DivuzenExpert
    router: DivuzenRouter
    shared: DivuzenExpert | None = None


DivuzenMLP = Annotated[Union[DivuzenDense, DivuzenMoE], Field(discriminator="kind")]


class DivuzenAttentionLayer(_Keys):
    type: Literal["attention"]
    mixer: DivuzenAttentionMixer
    mlp: DivuzenMLP | None = None


class DivuzenRetentionLayer(_Keys):
    type: Literal["retention"]
    mixer: DivuzenRetentionMixer
    mlp: DivuzenMLP | None = None


DivuzenLayer = Annotated[Union[DivuzenAttentionLayer, DivuzenRetentionLayer], Field(discriminator="type")]


class DivuzenConfig(BaseModel):
    """``config.json`` of a Divuzen folder."""

    model_config = ConfigDict(extra="ignore")

    architecture: Literal["Divuzen"]
    vocab: Size = Field(gt=0)
    width: Size = Field(gt=0)
    norm: DivuzenNorm
    layers: list[DivuzenLayer] = Field(min_length=1)
    logit_scale: float = 1.0
    max_positions: Size | None = Field(default=None, gt=0)
    """Not a key of the design (a request may be as long as the cache allows)."""
    stop_token_ids: tuple[int, ...] = ()

    @model_validator(mode="after")
    def _check(self):
        for i, layer in enumerate(self.layers):
            source = getattr(layer.mixer, "kv_from", None)
            if source is None:
                continue
            if not (source < i and isinstance(self.layers[source], DivuzenAttentionLayer)
                    and self.layers[source].mixer.kv_from is None):
                raise ValueError(f"layer {i}: kv_from {source} is no earlier attention with keys and values of its own")
            a, b = layer.mixer, self.layers[source].mixer
            if (a.kv_heads, a.dim, a.vdim, a.rot) != (b.kv_heads, b.dim, b.vdim, b.rot):
                raise ValueError(f"layer {i}: the keys and values of layer {source} have other sizes or another rotation")
        return self

    @property
    def architectures(self) -> list[str]:
        return [self.architecture]

    def to_json_dict(self) -> dict:
        d = self.model_dump(exclude_none=True)
        if not self.stop_token_ids:
            d.pop("stop_token_ids")
        for layer in d["layers"]:
            layer.setdefault("mlp", None)
        return d
