"""A plain, slow implementation of the Divuzen decoder: one function per mechanism, written
from the design's equations in float64 (or any torch dtype), sharing no code with the
framework.  Tests compare the framework with it.

Notation: ``h`` is a part's input ``[T, width]`` for the ``T`` tokens of one request, in
order; weights are ``[out, in]`` and applied as ``h @ W.T``.  A model is a dict ``cfg`` with
the keys of ``config.json`` and a dict ``w`` of tensors by their names in the folder.
"""

from __future__ import annotations

import json
import math
import os

import torch


def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    """``x / sqrt(mean(x^2) + eps)`` over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def model_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """The norm of the stream and of the parts' results: its weight is stored around zero."""
    return rms_unit(x, eps) * (1.0 + weight)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def rotate(x: torch.Tensor, positions: torch.Tensor, rot: dict | None, interleaved: bool) -> torch.Tensor:
    """Turns the first ``rot.dims`` entries of the last dimension of ``x`` [T, heads, D] by the
    token's position: pairs ``(2i, 2i + 1)`` if ``interleaved``, else ``(i, i + dims/2)``."""
    if not rot:
        return x
    dims = rot["dims"]
    i = torch.arange(dims // 2, dtype=torch.float64)
    angle = positions.to(torch.float64)[:, None] * rot["base"] ** (-2.0 * i / dims)
    cos, sin = torch.cos(angle).to(x.dtype)[:, None], torch.sin(angle).to(x.dtype)[:, None]
    first, second = (slice(0, dims, 2), slice(1, dims, 2)) if interleaved else (slice(0, dims // 2), slice(dims // 2, dims))
    out = x.clone()
    out[..., first] = x[..., first] * cos - x[..., second] * sin
    out[..., second] = x[..., second] * cos + x[..., first] * sin
    return out


def sink_softmax(scores: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """Weights ``[T, keys]`` of one head: ``exp(s) / (sum exp(s) + exp(sink))``."""
    top = torch.maximum(scores.max(-1, keepdim=True).values, sink)
    e = torch.exp(scores - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def sink_attention(h, w, pre, m, eps, kv=None):
    """Grouped heads, a weighted norm per head on q and k, rotation of neighbouring entries, a
    learned term without key and value in every head's softmax.  ``kv``: another layer's keys (after norm and
    rotation) and values in the place of own ones.  Returns the result and the keys and values attended to."""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    q = rms_unit((h @ w[pre + "q"].T).view(T, H, D), eps) * w[pre + "q.norm"]
    q = rotate(q, pos, m.get("rot"), True)
    if kv is None:
        k = rms_unit((h @ w[pre + "k"].T).view(T, G, D), eps) * w[pre + "k.norm"]
        kv = rotate(k, pos, m.get("rot"), True), (h @ w[pre + "v"].T).view(T, G, V)
    k, v = kv
    later = torch.ones(T, T, dtype=torch.bool).triu(1)
    out = h.new_zeros((T, H, V))
    for head in range(H):
        g = head // (H // G)
        s = (q[:, head] @ k[:, g].T * m["scale"]).masked_fill(later, -math.inf)
        out[:, head] = sink_softmax(s, w[pre + "sink"][head]) @ v[:, g]
    return out.reshape(T, H * V) @ w[pre + "o"].T, kv


def decayed_state_walk(q, k, v, decay, S):
    """``q``, ``k`` [T, H, D], ``v`` [T, H, V], ``decay`` [H], ``S`` [H, D, V] the state before
    the first token: ``S <- decay S + k v^T`` then the read ``S^T q``, token by token.
    Returns the reads [T, H, V] and the state after the last token."""
    out = v.new_zeros(v.shape)
    for t in range(q.shape[0]):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out, S


def retention(h, w, pre, m, eps):
    """A recurrence with a matrix state per head and one constant decay per head, on rotated
    queries and keys; every head normed on its own, gated by SiLU."""
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    q = rotate((h @ w[pre + "q"].T).view(T, H, D), pos, m.get("rot"), False)
    k = rotate((h @ w[pre + "k"].T).view(T, H, D), pos, m.get("rot"), False) * D**-0.5
    v = (h @ w[pre + "v"].T).view(T, H, V)
    out, _ = decayed_state_walk(q, k, v, torch.tensor(m["decay"], dtype=h.dtype), h.new_zeros((H, D, V)))
    y = rms_unit(out, eps).reshape(T, H * V) * silu(h @ w[pre + "g"].T)
    return y @ w[pre + "o"].T


def clamped_dense(h, w, pre, f):
    """A gated feed-forward whose two products are held to a limit."""
    g = torch.clamp(h @ w[pre + "gate"].T, max=f["limit"])
    u = torch.clamp(h @ w[pre + "up"].T, -f["limit"], f["limit"])
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w[pre + "down"].T


def gated_expert(h, w, pre):
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def choose_experts(scores, correction, router, margins_out=None):
    """The indices ``[T, top]`` of the experts that every token uses: by ``scores + correction``,
    among the best ``groups.keep`` groups (a group counts with the sum of its two best).
    ``margins_out`` receives, per token, how far the closest of these choices is from turning over."""
    choice = scores + correction
    T, n = choice.shape
    margin = torch.full((T,), math.inf, dtype=choice.dtype)
    groups = router.get("groups")
    if groups:
        per = n // groups["count"]
        best = torch.sort(choice.view(T, groups["count"], per), -1, descending=True).values[..., :2].sum(-1)
        order = torch.argsort(best, dim=-1, descending=True, stable=True)
        ranked = best.gather(1, order)
        if groups["keep"] < groups["count"]:
            margin = torch.minimum(margin, ranked[:, groups["keep"] - 1] - ranked[:, groups["keep"]])
        open_ = torch.zeros_like(best, dtype=torch.bool).scatter(1, order[:, : groups["keep"]], True)
        choice = choice.masked_fill(~open_.repeat_interleave(per, 1), -math.inf)
    top = router["top"]
    order = torch.argsort(choice, dim=-1, descending=True, stable=True)
    ranked = choice.gather(1, order)
    if top < n:
        margin = torch.minimum(margin, ranked[:, top - 1] - ranked[:, top])
    if margins_out is not None:
        margins_out.append(margin)
    return order[:, :top]


def routed_experts(h, w, pre, f, margins_out=None):
    """Sigmoid scores; the chosen experts' scores (without the correction) over their sum, times
    ``router.scale``; and an expert for every token times a sigmoid of its own."""
    r = f["router"]
    s = torch.sigmoid(h @ w[pre + "router"].T)
    chosen = choose_experts(s, w[pre + "correction"], r, margins_out)
    weights = s.gather(1, chosen)
    weights = weights / (weights.sum(-1, keepdim=True) + 1e-20) * r["scale"]
    out = torch.zeros_like(h)
    for e in range(r["experts"]):
        for j in range(r["top"]):
            rows = (chosen[:, j] == e).nonzero()[:, 0]
            if rows.numel():
                out[rows] += weights[rows, j : j + 1] * gated_expert(h[rows], w, f"{pre}e{e}.")
    if f.get("shared"):
        out = out + torch.sigmoid(h @ w[pre + "shared.sg"].T) * gated_expert(h, w, pre + "shared.")
    return out


def forward(cfg: dict, w: dict, tokens, dtype=torch.float64, layers_out: list | None = None, round_inputs=None,
            margins_out: list | None = None, disturb: float = 0.0, seed: int = 0) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one request's tokens; ``layers_out`` collects the stream
    after every layer.  ``round_inputs``: an element type that every part's input is rounded
    to on the way (how far the logits move then says how sensitive a position is to arithmetic
    in that type); ``disturb``: a relative error that every entry of every part's input is moved by,
    drawn from ``seed``.  ``margins_out`` receives every router's margins (see ``choose_experts``)."""
    gen = torch.Generator().manual_seed(seed)

    def rounded(t):
        if round_inputs is not None:
            t = t.to(round_inputs).to(dtype)
        if disturb:
            t = t * (1.0 + disturb * torch.randn(t.shape, generator=gen, dtype=dtype))
        return t

    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    left = {}  # keys and values of the layers that have projections of their own
    for i, layer in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", layer["mixer"]
        h = rounded(model_norm(x, w[pre + "norm1"], eps))
        if layer["type"] == "attention":
            source = m.get("kv_from")
            y, left[i] = sink_attention(h, w, pre + "mix.", m, eps, None if source is None else left[source])
        elif layer["type"] == "retention":
            y = retention(h, w, pre + "mix.", m, eps)
        else:
            raise ValueError(layer["type"])
        x = x + model_norm(y, w[pre + "norm1b"], eps)
        f = layer.get("mlp")
        if f:
            h = rounded(model_norm(x, w[pre + "norm2"], eps))
            if f["kind"] == "dense":
                y = clamped_dense(h, w, pre + "mlp.", f)
            else:
                y = routed_experts(h, w, pre + "mlp.", f, margins_out)
            x = x + model_norm(y, w[pre + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return model_norm(x, w["final.norm"], eps) @ w["embed"].T * cfg["logit_scale"]


def load_folder(folder: str):
    """``(cfg, w)`` of a model folder, read with the safetensors package."""
    from safetensors.torch import load_file

    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    return cfg, load_file(os.path.join(folder, "model.safetensors"))


def tokens_with_clear_routing(cfg, w, tokens, margin=0.03, seed=0, tries=600):
    """``tokens`` with as few replaced as it takes for no router of the model to make a choice (of a
    group or of an expert) closer than ``margin``: arithmetic in 16 bits moves a score by about a
    hundredth, and a choice that turns over makes another model of it.  The first token with such a
    call is drawn anew until there is none (earlier tokens stay as they are: the model is causal)."""
    gen = torch.Generator().manual_seed(seed)
    ids = list(tokens)
    for _ in range(tries):
        margins = []
        forward(cfg, w, ids, margins_out=margins)
        if not margins:
            return ids
        close = (torch.stack(margins).min(0).values < margin).nonzero()
        if close.numel() == 0:
            return ids
        ids[int(close[0])] = int(torch.randint(0, cfg["vocab"], (1,), generator=gen))
    raise RuntimeError("no sequence without a close call of a router")


# ---- configurations, tensors and folders for the tests ------------------------------------------
def rot(base, dims):
    return {"base": base, "dims": dims}


def attention_layer(heads, kv_heads, dim, vdim, scale, rot=None, kv_from=None, mlp=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    for key, value in (("rot", rot), ("kv_from", kv_from)):
        if value is not None:
            mixer[key] = value
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def retention_layer(heads, dim, vdim, decay, rot=None, mlp=None):
    mixer = {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}
    if rot is not None:
        mixer["rot"] = rot
    return {"type": "retention", "mixer": mixer, "mlp": mlp}


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, top, ff, scale=1.0, groups=None, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale}}
    if groups is not None:
        out["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def model_cfg(width, vocab, layers, eps=1e-5, logit_scale=1.0):
    return {"architecture": "Divuzen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale,
            "layers": layers}


def tensor_shapes(cfg) -> dict:
    """Name -> shape of every tensor of a folder."""
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "final.norm": (W,)}
    for i, layer in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", layer["mixer"]
        mix = pre + "mix."
        out[pre + "norm1"], out[pre + "norm1b"] = (W,), (W,)
        if layer["type"] == "attention":
            out[mix + "q"], out[mix + "q.norm"] = (m["heads"] * m["dim"], W), (m["dim"],)
            out[mix + "sink"], out[mix + "o"] = (m["heads"],), (W, m["heads"] * m["vdim"])
            if m.get("kv_from") is None:
                out[mix + "k"], out[mix + "k.norm"] = (m["kv_heads"] * m["dim"], W), (m["dim"],)
                out[mix + "v"] = (m["kv_heads"] * m["vdim"], W)
        else:
            nk, nv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            out[mix + "q"], out[mix + "k"], out[mix + "v"], out[mix + "g"], out[mix + "o"] = (nk, W), (nk, W), (nv, W), (nv, W), (W, nv)
        f = layer.get("mlp")
        if f is None:
            continue
        out[pre + "norm2"], out[pre + "norm2b"] = (W,), (W,)
        if f["kind"] == "dense":
            parts = [("", f["ff"])]
        else:
            n = f["router"]["experts"]
            out[pre + "mlp.router"], out[pre + "mlp.correction"] = (n, W), (n,)
            parts = [(f"e{e}.", f["expert"]["ff"]) for e in range(n)]
            if f.get("shared"):
                parts.append(("shared.", f["shared"]["ff"]))
                out[pre + "mlp.shared.sg"] = (1, W)
        for name, ff in parts:
            out[f"{pre}mlp.{name}gate"], out[f"{pre}mlp.{name}up"], out[f"{pre}mlp.{name}down"] = (ff, W), (ff, W), (W, ff)
    return out


def random_weights(cfg, seed, std=0.12, stored=torch.bfloat16):
    """Matrices N(0, std); the model's norms around zero, those of q and k around one; sinks of a
    size that counts and corrections that make choice scores of either sign; rounded to ``stored`` so
    that engine and plain model hold the same numbers."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        parts = name.split(".")
        last = parts[-1]
        r = lambda scale=1.0: scale * torch.randn(shape, generator=gen)  # noqa: E731
        if name == "embed":
            t = r(0.7)
        elif last in ("norm1", "norm1b", "norm2", "norm2b") or name == "final.norm":
            t = r(0.2)
        elif last == "norm":
            t = 1.0 + r(0.2)
        elif last == "sink":
            t = 1.0 + r(1.5)
        elif last == "correction":
            t = r(0.3) - 0.5
        elif last == "router":
            t = r(4 * std)
        elif last in ("gate", "up", "down"):
            t = r(1.5 * std)
        else:
            t = r(std)
        out[name] = t.to(stored).float()
    return out


def write_model_folder(folder, cfg, weights, dtype=torch.bfloat16):
    from safetensors.torch import save_file

    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(dtype).contiguous() for k, v in weights.items()}, os.path.join(folder, "model.safetensors"))
    return folder


# both mixers and both feed-forwards; grouped key/value heads; a retention head whose values are
# longer than its keys; an attention that borrows its keys from the layer before, with a scale of its own;
# groups of two experts; a limit that holds many products
DIV_A = model_cfg(64, 331, [
    retention_layer(2, 16, 24, [0.9, 0.995], rot=rot(1000.0, 8), mlp=dense(48, 0.8)),
    attention_layer(4, 2, 16, 16, 0.3, rot=rot(500.0, 8), mlp=moe(8, 2, 32, scale=1.7, groups=(4, 2), shared=24)),
    attention_layer(4, 2, 16, 16, 0.2, rot=rot(500.0, 8), kv_from=1, mlp=dense(48, 1.5)),
    retention_layer(2, 16, 24, [0.97, 1.0], rot=rot(1000.0, 16), mlp=moe(8, 3, 32, scale=0.8, groups=(2, 1))),
], logit_scale=0.3)
# an attention first, without rotation and feed-forward, two layers that borrow from it and one in
# between with keys of its own that another borrows; values larger and smaller than keys; a whole head rotated;
# every expert chosen, and one of three, without groups; a retention without rotation
DIV_B = model_cfg(48, 257, [
    attention_layer(6, 3, 8, 24, 0.5),
    retention_layer(3, 8, 16, [0.5, 0.97, 1.0], mlp=moe(5, 5, 24, scale=2.5, shared=16)),
    attention_layer(6, 3, 8, 24, 0.3, kv_from=0, mlp=moe(3, 1, 36)),
    attention_layer(2, 2, 24, 8, 0.25, rot=rot(200.0, 24), mlp=dense(40, 3.0)),
    attention_layer(6, 3, 8, 24, 0.4, kv_from=0),
    attention_layer(2, 2, 24, 8, 0.3, rot=rot(200.0, 24), kv_from=3, mlp=moe(6, 2, 20, scale=1.2, groups=(3, 2))),
])
# sizes that are multiples of nothing; one key/value head; retention states that no fused step takes
# (value heads of 10) and one head without decay; groups of one expert; a group of six
DIV_C = model_cfg(42, 203, [
    attention_layer(5, 1, 12, 20, 0.2, rot=rot(77.0, 6), mlp=moe(6, 3, 20, scale=1.3, groups=(6, 4), shared=28)),
    retention_layer(3, 14, 10, [0.8, 0.99, 1.0], rot=rot(90.0, 6), mlp=dense(30, 0.5)),
    attention_layer(5, 1, 12, 20, 0.25, rot=rot(77.0, 6), kv_from=0),
    retention_layer(1, 20, 12, [1.0], rot=rot(50.0, 20), mlp=moe(12, 2, 20, groups=(2, 1), shared=10)),
], eps=1e-6, logit_scale=2.0)
