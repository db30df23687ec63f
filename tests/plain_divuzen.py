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
