"""The model: embedding, the layers in the order of the run list, final norm, head.

Built from a ``ModelSpec`` alone; which parts a layer has, in which arrangement, and
in which order the layers run are all data.  The flat-batch forward pass follows
src/halite/transformers/infer/transformer.py:82-114: embed, run every block on the
step's tokens, normalise the wanted rows, project them to float32 logits.
"""

from __future__ import annotations

from dataclasses import dataclass

import torch

from ..config.spec import ModelSpec
from ..kernels import ops
from .base import (
    ARRANGEMENTS,
    EMBEDDINGS,
    HEADS,
    JUNCTIONS,
    NORMS,
    POSITIONS,
    BuildContext,
    ConfigError,
    ParamDecl,
    Part,
    RunBinding,
)


EMBEDDING_RUN = -1  # the index of the embedding's state rows among the runs'


@dataclass
class ParamSlot:
    path: str  # e.g. layers.3.mixer.q.weight
    part: Part
    name: str  # the part's own name for it, e.g. q.weight
    decl: ParamDecl


class Decoder:
    def __init__(self, spec: ModelSpec, dtype: torch.dtype, device: torch.device | str,
                 tiled_weights: bool = False):
        # the kinds of parts register themselves when their modules are imported
        from . import (attention, block, capped_attention, connection, decay_attention, embedding, feedforward,  # noqa: F401
                       general_delta, junction, latent_attention, mingru, mixer_sum, moe, norm, normed_attention, rope,
                       rotated_attention, sigmoid_attention, state_space, time_mix, token_gated)

        self.spec = spec
        self.dtype = dtype
        self.device = torch.device(device)
        build = BuildContext(dtype=dtype, device=self.device, hidden_size=spec.hidden_size,
                             tiled_weights=tiled_weights and dtype == torch.bfloat16)
        for name, pspec in spec.positions.items():
            build.positions[name] = POSITIONS.build(pspec, build)
        self.build = build
        self.positions = build.positions
        self.embedding = EMBEDDINGS.build(spec.embedding, build)
        build.embedding = self.embedding
        self.layers = {}
        for name, lspec in spec.layers.items():
            if lspec.arrangement not in ARRANGEMENTS:
                known = ", ".join(sorted(ARRANGEMENTS))
                raise ConfigError(f"unknown arrangement {lspec.arrangement!r}; known: {known}")
            self.layers[name] = ARRANGEMENTS[lspec.arrangement].build(lspec.arrangement, lspec.parts, build)
        self.junctions = {name: JUNCTIONS.build(pspec, build) for name, pspec in spec.junctions.items()}
        self.final_norm = NORMS.build(spec.final_norm, build)
        self.head = HEADS.build(spec.head, build)
        self.runs = [
            RunBinding(index=i, appends=run.cache_from is None) for i, run in enumerate(spec.order)
        ]
        # what an embedding with per-request state is bound to (before the first run)
        self.embedding_run = RunBinding(index=EMBEDDING_RUN)
        # an arrangement may keep the residual stream in several copies ([copies, T, width]);
        # then every block of the model does, and the last one says how they become one again
        copies = {getattr(self.layers[run.layer], "stream_copies", None) for run in spec.order}
        if len(copies) != 1:
            raise ConfigError(f"the model's blocks keep the residual stream in different ways: {sorted(map(str, copies))} copies")
        self.stream_copies = copies.pop()

    # -- declarations -------------------------------------------------------------
    def named_parts(self) -> dict[str, Part]:
        out = {"embedding": self.embedding}
        for lname, block in self.layers.items():
            for pname, part in block.parts().items():
                out[f"layers.{lname}.{pname}"] = part
        for jname, part in self.junctions.items():
            out[f"junctions.{jname}"] = part
        out["final_norm"] = self.final_norm
        out["head"] = self.head
        return out

    def param_slots(self) -> list[ParamSlot]:
        """Every tensor of the model in a fixed order (the order that the random
        weights are drawn in)."""
        slots = []
        for prefix, part in self.named_parts().items():
            for name, decl in part.param_decls().items():
                slots.append(ParamSlot(f"{prefix}.{name}", part, name, decl))
        return slots

    def mixer_of_run(self, index: int):
        return self.layers[self.spec.order[index].layer].mixer

    def finalize(self):
        self.head.bind(self.embedding)
        for part in self.named_parts().values():
            part.finalize()

    def param_bytes(self) -> int:
        n = 0
        for slot in self.param_slots():
            size = 1
            for d in slot.decl.shape:
                size *= d
            n += size * (4 if slot.decl.integer else self.dtype.itemsize)
        return n

    # -- the forward pass of one step -----------------------------------------------
    def forward(self, ctx) -> torch.Tensor:
        """float32 logits ``[len(ctx.logit_rows), vocab]``; keys and values of all
        the step's tokens are in the cache afterwards."""
        reads = dict(ctx=ctx, run=self.embedding_run) if self.embedding.reads_step else {}
        if self.stream_copies is None:
            h = h0 = self.embedding.forward(ctx.tokens, **reads)
        else:  # every copy starts as the embedding's output
            h = torch.empty((self.stream_copies, ctx.tokens.numel(), self.spec.hidden_size), dtype=torch.float32,
                            device=self.device)
            h0 = self.embedding.forward(ctx.tokens, out=h[0], **reads)
            for copy in h[1:]:  # (an embedding that reads the step moves its state on: it runs once)
                copy.copy_(h0) if reads else self.embedding.forward(ctx.tokens, out=copy)
        kept = {name: junction.start(h0) for name, junction in self.junctions.items()}
        pending = None
        blocks = [self.layers[self.spec.order[run.index].layer] for run in self.runs]
        for i, run in enumerate(self.runs):
            name = self.spec.order[run.index].junction
            if name is not None:
                h = self._through_junction(self.junctions[name], kept[name], h, pending, blocks[max(i - 1, 0)], ctx)
                pending = None
            # what the next block's first norm lets this block's last product do for it
            # (both are optional abilities of an arrangement: `takes_next_norm` of the one that
            # runs now, `first_norm_for` of the one that runs next)
            ahead = blocks[i + 1] if i + 1 < len(blocks) and self.spec.order[i + 1].junction is None else None
            next_norm = None
            if getattr(blocks[i], "takes_next_norm", False) and hasattr(ahead, "first_norm_for"):
                next_norm = ahead.first_norm_for(h)
            if next_norm is not None:
                pending = blocks[i].forward(h, pending, ctx, run, next_norm=next_norm)
            else:
                pending = blocks[i].forward(h, pending, ctx, run)
        if ctx.n_logit_rows == 0:
            return torch.empty((0, self.spec.vocab_size), dtype=torch.float32, device=self.device)
        if self.stream_copies is not None:
            x = blocks[-1].leave_normed(h, pending, ctx.logit_rows, self.final_norm) if hasattr(blocks[-1], "leave_normed") else None
            if x is None:
                x = self.final_norm.forward(blocks[-1].leave(h, pending, ctx.logit_rows))
        else:
            x = self.final_norm.forward(h, delta=pending, rows=ctx.logit_rows)
        return self.head.forward(x)

    def _through_junction(self, junction, kept, h, pending, block, ctx):
        """The stream that the next run starts from; ``block`` ran last and left ``pending``."""
        rows = junction.stream_rows(kept)
        ctx.rounded_rows = None
        if self.stream_copies is None:
            if pending is not None:
                ops.residual_add(h, pending)
            ops.cast_cols(h, rows)
            return junction.forward(kept)
        block.leave(h, pending, None, out=rows)
        x = junction.forward(kept)
        return x.unsqueeze(0) if self.stream_copies == 1 else x.unsqueeze(0).repeat(self.stream_copies, 1, 1)
