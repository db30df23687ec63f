"""Divuzen: a decoder whose layers norm what a part reads and what it returns
(``x += norm_b(part(norm_a(x)))``, the norms' weights stored as their distance from one), listed
one by one in ``config.json``.  A layer's mixer is one of two: a softmax attention with a
weighted norm per head on q and k, rotation of neighbouring entries and a learned sink per
head, which may attend to the keys and values of an earlier layer instead of its own; or a
retention, a linear attention with rotated queries and keys and one constant decay per head,
every head normed on its own and gated by SiLU.  The feed-forward is a clamped gated dense
layer or a mixture of SiLU-gated experts, chosen by sigmoid scores with a correction among
the best groups of neighbours, with a shared expert behind a sigmoid gate of its own.  The
logits are made with the embedding table.
"""

from __future__ import annotations

from ..config.divuzen import DivuzenAttentionLayer, DivuzenConfig, DivuzenDense
from ..config.registry import Architecture, register_architecture
from ..config.spec import LayerRun, LayerSpec, ModelSpec, PartSpec

# The design has no longest request; the position tables are made for this many positions
# unless the folder states ``max_positions``.
DEFAULT_MAX_POSITIONS = 1 << 18
# Constants that the design fixes.
NORM_WEIGHT_OFFSET = 1.0  # a norm multiplies by this plus its stored weight
DENSE_ALPHA, DENSE_UP_SHIFT = 1.702, 1.0  # the dense gate: g sigmoid(DENSE_ALPHA g) (u + DENSE_UP_SHIFT)
ROUTER_NORM_EPS = 1e-20  # added to the sum of the chosen scores before it divides them


def _rope(rot, head: int, interleaved: bool, max_positions: int, positions: dict) -> str | None:
    """The name of the position encoding for ``rot`` (added to ``positions``), or None."""
    if rot is None:
        return None
    name = f"rope_{rot.dims}_of_{head}_base_{rot.base!r}_{'pairs' if interleaved else 'halves'}"
    positions.setdefault(name, PartSpec(kind="rope", head_dim=head, rotary_dim=rot.dims, theta=rot.base, interleaved=interleaved,
                                        max_positions=max_positions, angles="float64"))
    return name


def divuzen_spec(cfg: DivuzenConfig) -> ModelSpec:
    max_positions = cfg.max_positions or DEFAULT_MAX_POSITIONS
    eps = cfg.norm.eps
    norm = PartSpec(kind="rmsnorm", size=cfg.width, eps=eps, round_before_weight=False, weight_offset=NORM_WEIGHT_OFFSET)
    link = PartSpec(kind="hyper_connection", streams=1, learned=False)
    positions, layers, order = {}, {}, []
    for i, layer in enumerate(cfg.layers):
        m = layer.mixer
        if isinstance(layer, DivuzenAttentionLayer):
            mixer = PartSpec(
                kind="capped_attention", hidden_size=cfg.width, n_heads=m.heads, n_kv_heads=m.kv_heads, qk_dim=m.dim,
                v_dim=m.vdim, scale=m.scale, eps=eps, position=_rope(m.rot, m.dim, True, max_positions, positions),
                head_gate=False, learned_sink=True, own_kv=m.kv_from is None,
            )
        else:
            mixer = PartSpec(
                kind="decay_attention", hidden_size=cfg.width, n_heads=m.heads, qk_dim=m.dim, v_dim=m.vdim,
                decay=list(m.decay), eps=eps, position=_rope(m.rot, m.dim, False, max_positions, positions),
                activation=None, key_scale=m.dim**-0.5, norm_per_head=True, norm_weight=False, gate="silu",
            )
        parts = dict(mixer_norm=norm, mixer=mixer, mixer_out_norm=norm, mixer_link=link)
        f = layer.mlp
        if f is not None:
            if isinstance(f, DivuzenDense):
                parts["ff"] = PartSpec(kind="gated", hidden_size=cfg.width, intermediate_size=f.ff, activation="clamped",
                                       limit=f.limit, alpha=DENSE_ALPHA, up_shift=DENSE_UP_SHIFT, float32_result=True)
            else:
                gate = dict(limit=None, alpha=1.0, up_shift=0.0)  # silu(gate) * up
                r = f.router
                parts["ff"] = PartSpec(
                    kind="moe", hidden_size=cfg.width, n_experts=r.experts, top_k=r.top,
                    expert=dict(intermediate_size=f.expert.ff, **gate),
                    shared=dict(intermediate_size=f.shared.ff, **gate) if f.shared is not None else None,
                    shared_gate=f.shared is not None, score="sigmoid", normalize=True, norm_eps=ROUTER_NORM_EPS,
                    correction=True, weight_scale=r.scale,
                    groups=dict(count=r.groups.count, keep=r.groups.keep) if r.groups is not None else None,
                    float32_result=True,
                )
            parts.update(ff_norm=norm, ff_out_norm=norm, ff_link=link)
        layers[f"l{i}"] = LayerSpec(arrangement="hyper_pre_norm", parts=parts)
        order.append(LayerRun(layer=f"l{i}", cache_from=getattr(m, "kv_from", None)))
    return ModelSpec(
        architecture="Divuzen",
        vocab_size=cfg.vocab,
        hidden_size=cfg.width,
        max_positions=max_positions,
        embedding=PartSpec(kind="embedding", vocab_size=cfg.vocab, size=cfg.width),
        positions=positions,
        layers=layers,
        order=order,
        final_norm=norm,
        head=PartSpec(kind="linear_head", vocab_size=cfg.vocab, size=cfg.width, tied=True, logit_scale=cfg.logit_scale),
    )


_QUERY_TENSORS = (("q", "q.weight"), ("q.norm", "q_norm.weight"), ("sink", "sink"), ("o", "out.weight"))
_KEY_TENSORS = (("k", "k.weight"), ("v", "v.weight"), ("k.norm", "k_norm.weight"))
_RETENTION_TENSORS = (("q", "q.weight"), ("k", "k.weight"), ("v", "v.weight"), ("g", "gate.weight"), ("o", "out.weight"))
_DENSE_TENSORS = (("gate", "linear_gate.weight"), ("up", "linear_proj.weight"), ("down", "linear_out.weight"))
_EXPERT_TENSORS = (("gate", "gate.weight"), ("up", "up.weight"), ("down", "down.weight"))


def divuzen_weight_map(cfg: DivuzenConfig) -> dict[str, str | None]:
    """Tensor name in the folder -> parameter of a part, layer by layer."""
    table = {"embed": "embedding.weight", "final.norm": "final_norm.weight"}
    for i, layer in enumerate(cfg.layers):
        src, dst = f"l{i}.", f"layers.l{i}."
        table[src + "norm1"], table[src + "norm1b"] = dst + "mixer_norm.weight", dst + "mixer_out_norm.weight"
        if isinstance(layer, DivuzenAttentionLayer):
            names = _QUERY_TENSORS + (_KEY_TENSORS if layer.mixer.kv_from is None else ())
        else:
            names = _RETENTION_TENSORS
        for theirs, ours in names:
            table[f"{src}mix.{theirs}"] = f"{dst}mixer.{ours}"
        f = layer.mlp
        if f is None:
            table[src + "norm2"] = table[src + "norm2b"] = None  # stored without a reader, perhaps
            continue
        table[src + "norm2"], table[src + "norm2b"] = dst + "ff_norm.weight", dst + "ff_out_norm.weight"
        if isinstance(f, DivuzenDense):
            for theirs, ours in _DENSE_TENSORS:
                table[f"{src}mlp.{theirs}"] = f"{dst}ff.{ours}"
            continue
        table[src + "mlp.router"], table[src + "mlp.correction"] = dst + "ff.router.weight", dst + "ff.correction"
        groups = [(f"e{e}", f"experts.{e}") for e in range(f.router.experts)]
        if f.shared is not None:
            groups.append(("shared", "shared"))
            table[src + "mlp.shared.sg"] = dst + "ff.shared_gate.weight"
        for theirs_of, ours_of in groups:
            for theirs, ours in _EXPERT_TENSORS:
                table[f"{src}mlp.{theirs_of}.{theirs}"] = f"{dst}ff.{ours_of}.{ours}"
    return table


DIVUZEN = register_architecture(
    Architecture(
        name="Divuzen",
        config_cls=DivuzenConfig,
        to_spec=divuzen_spec,
        weight_map=divuzen_weight_map,
    )
)
