"""Nodupel: a pre-norm decoder whose layers are listed one by one in ``config.json``; a stretch of
them may run several times in a row with the same weights, every pass starting from a
projection of the stream beside the embedding's output.  The embedding adds a row of a second
table that is chosen by the token and the one before it.  A layer's mixer is either two mixers
side by side, each normed before the sum (a softmax attention with a sliding window and kept
first tokens whose values are rotated, and a time-mixing recurrence with a decay per key
channel), or a gated recurrence per channel whose gates read the token alone.  The feed-forward
is a gated dense layer with gelu; the logits are capped.
"""

from __future__ import annotations

from ..config.nodupel import NodupelConfig, NodupelParallelLayer
from ..config.registry import Architecture, ConfigError, register_architecture
from ..config.spec import LayerRun, LayerSpec, ModelSpec, PartSpec

# The design has no longest request; the position tables are made for this many positions
# unless the folder states ``max_positions``.
DEFAULT_MAX_POSITIONS = 1 << 18
# Constants that the design fixes.
MEMBER_SCALE = 0.5  # of the two normed results of a parallel mixer
LOOP_JUNCTION = "loop"


def _rope(base: float, dims: int, head: int, factor: float | None, max_positions: int) -> tuple[str, PartSpec]:
    name = f"rope_{dims}_of_{head}_base_{base!r}" + (f"_by_{factor!r}" if factor is not None else "")
    return name, PartSpec(kind="rope", head_dim=head, rotary_dim=dims, theta=base, max_positions=max_positions,
                          scaling=None if factor is None else dict(kind="linear", factor=factor), angles="float64")


def run_order(cfg: NodupelConfig) -> list[LayerRun]:
    """Every layer once, and those of the loop once a pass; a pass begins with the junction."""
    n, loop = len(cfg.layers), cfg.loop
    if loop is None:
        return [LayerRun(layer=f"l{i}") for i in range(n)]
    order = [LayerRun(layer=f"l{i}") for i in range(loop.start)]
    for _ in range(loop.times):
        order += [LayerRun(layer=f"l{i}", junction=LOOP_JUNCTION if i == loop.start else None)
                  for i in range(loop.start, loop.stop)]
    return order + [LayerRun(layer=f"l{i}") for i in range(loop.stop, n)]


def nodupel_spec(cfg: NodupelConfig) -> ModelSpec:
    max_positions = cfg.max_positions or DEFAULT_MAX_POSITIONS
    eps = cfg.norm.eps
    norm = PartSpec(kind="rmsnorm", size=cfg.width, eps=eps, round_before_weight=False)
    link = PartSpec(kind="hyper_connection", streams=1, learned=False,
                    mult=1.0 if cfg.residual_mult is None else cfg.residual_mult)
    positions, layers = {}, {}
    for i, layer in enumerate(cfg.layers):
        m = layer.mixer
        if isinstance(layer, NodupelParallelLayer):
            a, b = m.left, m.right
            if b.decay_rank is None:
                raise ConfigError(
                    f"layer {i}: the rank of the decay projection is the first dimension of the tensor 'l{i}.mix.right.w1'; "
                    "a configuration that is used without the folder's tensors states it as 'decay_rank'"
                )
            position = value_position = None
            if a.rot is not None:
                factor = a.rot.scaling.factor if a.rot.scaling is not None else None
                position, spec = _rope(a.rot.base, a.rot.dims, a.dim, factor, max_positions)
                positions.setdefault(position, spec)
                # (values turn with the unstretched frequencies, over the whole head)
                value_position, spec = _rope(a.rot.base, a.vdim, a.vdim, None, max_positions)
                positions.setdefault(value_position, spec)
            left = dict(kind="rotated_attention", hidden_size=cfg.width, n_heads=a.heads, n_kv_heads=a.kv_heads,
                        qk_dim=a.dim, v_dim=a.vdim, scale=a.scale, position=position, value_position=value_position,
                        window=a.mask.size if a.mask is not None else None,
                        keep_first=a.mask.keep_first if a.mask is not None else 0)
            right = dict(kind="time_mix", hidden_size=cfg.width, n_heads=b.heads, head_dim=b.dim,
                         decay_rank=b.decay_rank, eps=eps)
            mixer = PartSpec(kind="sum", names=["left", "right"], mixers=[left, right],
                             scales=[MEMBER_SCALE, MEMBER_SCALE], norm_eps=eps, size=cfg.width)
        else:
            mixer = PartSpec(kind="mingru", hidden_size=cfg.width, width=m.width)
        parts = dict(mixer_norm=norm, mixer=mixer, mixer_link=link)
        if layer.mlp is not None:
            parts["ff_norm"], parts["ff_link"] = norm, link
            parts["ff"] = PartSpec(kind="gated", hidden_size=cfg.width, intermediate_size=layer.mlp.ff,
                                   activation="gelu_tanh", float32_result=True)
        layers[f"l{i}"] = LayerSpec(arrangement="hyper_pre_norm", parts=parts)
    pairs = cfg.embedding.bigram
    return ModelSpec(
        architecture="Nodupel",
        vocab_size=cfg.vocab,
        hidden_size=cfg.width,
        max_positions=max_positions,
        embedding=PartSpec(kind="embedding", vocab_size=cfg.vocab, size=cfg.width, scale=cfg.embedding.scale,
                           pairs=None if pairs is None else pairs.model_dump()),
        positions=positions,
        layers=layers,
        order=run_order(cfg),
        junctions={} if cfg.loop is None else {LOOP_JUNCTION: PartSpec(kind="reinjection", size=cfg.width)},
        final_norm=norm,
        head=PartSpec(kind="linear_head", vocab_size=cfg.vocab, size=cfg.width, tied=False, logit_softcap=cfg.logit_softcap),
    )


_PARALLEL_TENSORS = (
    ("left.q", "left.q.weight"), ("left.k", "left.k.weight"), ("left.v", "left.v.weight"), ("left.g", "left.gate.weight"),
    ("left.o", "left.out.weight"), ("left.out", "left_norm.weight"),
    ("right.mu.r", "right.mu.r"), ("right.mu.k", "right.mu.k"), ("right.mu.v", "right.mu.v"),
    ("right.mu.g", "right.mu.gate"), ("right.mu.w", "right.mu.decay"),
    ("right.r", "right.r.weight"), ("right.k", "right.k.weight"), ("right.v", "right.v.weight"),
    ("right.g", "right.gate.weight"), ("right.w1", "right.decay_down.weight"), ("right.w2", "right.decay_up.weight"),
    ("right.w0", "right.decay.bias"), ("right.u", "right.bonus"), ("right.norm", "right.norm.weight"),
    ("right.o", "right.out.weight"), ("right.out", "right_norm.weight"),
)
_MINGRU_TENSORS = (("z", "z.weight"), ("z.b", "z.bias"), ("x", "x.weight"), ("x.b", "x.bias"), ("g", "gate.weight"),
                   ("o", "out.weight"))


def nodupel_weight_map(cfg: NodupelConfig) -> dict[str, str | None]:
    """Tensor name in the folder -> parameter of a part, layer by layer."""
    table = {"embed": "embedding.weight", "final.norm": "final_norm.weight", "head": "head.weight"}
    if cfg.embedding.bigram is not None:
        table["bigram"] = "embedding.pairs.weight"
    if cfg.loop is not None:
        table["loop.in"] = f"junctions.{LOOP_JUNCTION}.weight"
    for i, layer in enumerate(cfg.layers):
        src, dst = f"l{i}.", f"layers.l{i}."
        table[src + "norm1"] = dst + "mixer_norm.weight"
        for theirs, ours in _PARALLEL_TENSORS if isinstance(layer, NodupelParallelLayer) else _MINGRU_TENSORS:
            table[f"{src}mix.{theirs}"] = f"{dst}mixer.{ours}"
        if layer.mlp is None:
            table[src + "norm2"] = None  # stored without a reader, perhaps
            continue
        table[src + "norm2"] = dst + "ff_norm.weight"
        table[src + "mlp.gate"] = dst + "ff.linear_gate.weight"
        table[src + "mlp.up"] = dst + "ff.linear_proj.weight"
        table[src + "mlp.down"] = dst + "ff.linear_out.weight"
    return table


def nodupel_complete(cfg: NodupelConfig, shape_of) -> NodupelConfig:
    """Fills in what the folder's tensors say and the file does not: the rank of every
    time-mixing mixer's decay projection."""
    layers = []
    for i, layer in enumerate(cfg.layers):
        if isinstance(layer, NodupelParallelLayer):
            shape = shape_of(f"l{i}.mix.right.w1")
            if shape is not None and len(shape) == 2:
                right = layer.mixer.right.model_copy(update={"decay_rank": int(shape[0])})
                layer = layer.model_copy(update={"mixer": layer.mixer.model_copy(update={"right": right})})
        layers.append(layer)
    return cfg.model_copy(update={"layers": layers})


NODUPEL = register_architecture(
    Architecture(
        name="Nodupel",
        config_cls=NodupelConfig,
        to_spec=nodupel_spec,
        weight_map=nodupel_weight_map,
        complete_from_tensors=nodupel_complete,
    )
)
