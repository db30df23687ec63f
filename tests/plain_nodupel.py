"""A plain, slow implementation of the Nodupel decoder: one function per mechanism, written
from the design's equations in float64 (or any torch dtype), sharing no code with the
framework.  Tests compare the framework with it.

Notation: ``h`` is a mixer's or feed-forward's input ``[T, width]`` for the ``T`` tokens of
one request, in order; weights are ``[out, in]`` and applied as ``h @ W.T``.  A model is a
dict ``cfg`` with the keys of ``config.json`` and a dict ``w`` of tensors by their names in
the folder.
"""

from __future__ import annotations

import json
import math
import os

import torch


def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    """``x / sqrt(mean(x^2) + eps)`` over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z**3)))


def bigram_rows(tokens, buckets: int, mul_prev: int, mul_cur: int) -> list[int]:
    """Row of the table of pairs for every token of a request: a hash of the token before and
    the token; the first token has a row of its own, behind the hashed ones."""
    rows = []
    for t, token in enumerate(tokens):
        rows.append(buckets if t == 0 else (int(tokens[t - 1]) * mul_prev + int(token) * mul_cur) % buckets)
    return rows


def embed(cfg, w, tokens):
    e = cfg["embedding"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * e["scale"]
    if e.get("bigram"):
        b = e["bigram"]
        x = x + w["bigram"][torch.as_tensor(bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"]))]
    return x


def turn(x: torch.Tensor, positions, dims: int, base: float, factor: float = 1.0, backwards: bool = False):
    """``x`` [T, heads, n]: the pairs ``(i, i + dims/2)`` of the first ``dims`` entries of every
    head turned by ``position * base^(-2i/dims) / factor`` (the other way with ``backwards``)."""
    x = x.clone()
    for i in range(dims // 2):
        angle = torch.as_tensor(positions, dtype=torch.float64) * (base ** (-2.0 * i / dims) / factor)
        if backwards:
            angle = -angle
        c, s = torch.cos(angle).to(x.dtype)[:, None], torch.sin(angle).to(x.dtype)[:, None]
        u, v = x[:, :, i].clone(), x[:, :, i + dims // 2].clone()
        x[:, :, i] = u * c - v * s
        x[:, :, i + dims // 2] = v * c + u * s
    return x


def sees(i: int, j: int, mask: dict | None) -> bool:
    """Whether the query at position ``i`` sees the key at ``j``: a sliding window, and the
    first few tokens of the request for ever."""
    if j > i:
        return False
    return mask is None or i - j < mask["size"] or j < mask.get("keep_first", 0)


def visible(T: int, mask: dict | None) -> torch.Tensor:
    return torch.tensor([[sees(i, j, mask) for j in range(T)] for i in range(T)], dtype=torch.bool)


def kept_window_attention(h, w, pre, m):
    """Grouped heads, rotated queries, keys and values, a sliding window with kept first tokens,
    softmax, the heads' results turned back, a gate per head."""
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    rot = m["rot"]
    factor = (rot.get("scaling") or {}).get("factor", 1.0)
    at = list(range(T))
    q = turn((h @ w[pre + "q"].T).view(T, H, D), at, rot["dims"], rot["base"], factor)
    k = turn((h @ w[pre + "k"].T).view(T, G, D), at, rot["dims"], rot["base"], factor)
    v = turn((h @ w[pre + "v"].T).view(T, G, V), at, V, rot["base"])
    seen = visible(T, m.get("mask"))
    out = h.new_zeros((T, H, V))
    for head in range(H):
        g = head // (H // G)
        s = (q[:, head] @ k[:, g].T) * m["scale"]
        s = s.masked_fill(~seen, float("-inf"))
        out[:, head] = torch.softmax(s, -1) @ v[:, g]
    out = turn(out, at, V, rot["base"], backwards=True)
    out = out * torch.sigmoid(h @ w[pre + "g"].T)[:, :, None]
    return out.reshape(T, H * V) @ w[pre + "o"].T


def shifted(h, mu, before):
    """``h_t + (h_(t-1) - h_t) * mu``; ``before`` stands for the row before the first."""
    previous = torch.cat([before[None], h[:-1]], 0)
    return h + (previous - h) * mu


def wkv_recurrence(r, k, v, decay, u, S):
    """One head: ``r``, ``k``, ``decay`` [T, D], ``v`` [T, D], the bonus ``u`` [D]; ``S`` [D, D]
    (key channel x value channel) is the state before the first token.  A token reads the old
    state and its own pair weighted by the bonus, then the state decays and takes the pair."""
    S = S.clone()
    o = torch.zeros_like(v)
    for t in range(r.shape[0]):
        pair = torch.outer(k[t], v[t])
        o[t] = (S + u[:, None] * pair).T @ r[t]
        S = decay[t][:, None] * S + pair
    return o, S


def wkv_decay(mixed, w, pre):
    """Decay per key channel, ``exp(-exp(.))`` of a projection through a small inner size."""
    return torch.exp(-torch.exp(torch.tanh(mixed @ w[pre + "w1"].T) @ w[pre + "w2"].T + w[pre + "w0"]))


def time_mixing(h, w, pre, m, eps, before=None, state=None):
    """The recurrent mixer with its shifted inputs, per-head norm, gate and output projection.
    Returns the result, the last token's ``h`` and the states [H, D, D] after it."""
    T = h.shape[0]
    H, D = m["heads"], m["dim"]
    before = h.new_zeros(h.shape[1]) if before is None else before
    mixed = {s: shifted(h, w[f"{pre}mu.{s}"], before) for s in "rkvgw"}
    r, k, v = ((mixed[s] @ w[pre + s].T).view(T, H, D) for s in "rkv")
    gate = silu(mixed["g"] @ w[pre + "g"].T)
    decay = wkv_decay(mixed["w"], w, pre).view(T, H, D)
    S = h.new_zeros((H, D, D)) if state is None else state
    o, left = h.new_zeros((T, H, D)), []
    for head in range(H):
        o[:, head], s = wkv_recurrence(r[:, head], k[:, head], v[:, head], decay[:, head], w[pre + "u"][head], S[head])
        left.append(s)
    o = rms_unit(o, eps).reshape(T, H * D) * w[pre + "norm"] * gate
    return o @ w[pre + "o"].T, h[-1], torch.stack(left)


def parallel_mixer(h, w, pre, m, eps):
    """Half the sum of the two mixers' results, each normed over the model's width."""
    a = kept_window_attention(h, w, pre + "left.", m["left"])
    b, _, _ = time_mixing(h, w, pre + "right.", m["right"], eps)
    return 0.5 * (rms_unit(a, eps) * w[pre + "left.out"] + rms_unit(b, eps) * w[pre + "right.out"])


def mingru_gates(h, w, pre):
    z = torch.sigmoid(h @ w[pre + "z"].T + w[pre + "z.b"])
    u = h @ w[pre + "x"].T + w[pre + "x.b"]
    return z, torch.where(u >= 0, u + 0.5, torch.sigmoid(u))


def mingru(h, w, pre, state=None):
    """A gated recurrence per channel whose gates read the token alone; the result and the
    state [channels] after the last token."""
    z, candidate = mingru_gates(h, w, pre)
    S = h.new_zeros(z.shape[1]) if state is None else state
    rows = []
    for t in range(h.shape[0]):
        S = (1.0 - z[t]) * S + z[t] * candidate[t]
        rows.append(S)
    return (torch.stack(rows) * silu(h @ w[pre + "g"].T)) @ w[pre + "o"].T, S


def feed_forward(h, w, pre):
    return (gelu_tanh(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def run_order(cfg) -> list[tuple[int, bool]]:
    """(layer, whether a pass of the loop begins right before it), in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    order = [(i, False) for i in range(loop["start"])]
    for _ in range(loop["times"]):
        order += [(i, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return order + [(i, False) for i in range(loop["stop"], n)]


def soft_cap(logits, cap):
    return logits if cap is None else cap * torch.tanh(logits / cap)


def forward(cfg: dict, w: dict, tokens, dtype=torch.float64, layers_out: list | None = None, round_inputs=None):
    """Logits ``[T, vocab]`` of one request's tokens.  ``layers_out`` receives the stream
    after every layer run.  ``round_inputs``: an element type that every part's normed input is
    rounded to on the way (how far the logits move then says how sensitive a position is to
    arithmetic in that type)."""
    w = {n: (t.to(dtype) if t.is_floating_point() else t) for n, t in w.items()}
    eps = cfg["norm"]["eps"]
    m = cfg.get("residual_mult", 1.0)
    rounded = (lambda t: t.to(round_inputs).to(dtype)) if round_inputs is not None else (lambda t: t)  # noqa: E731
    x = embed(cfg, w, tokens)
    x0 = x.clone()
    for i, begins in run_order(cfg):
        if begins:
            x = rounded(torch.cat([x, x0], -1)) @ w["loop.in"].T
        pre, layer = f"l{i}.", cfg["layers"][i]
        h = rounded(rms_unit(x, eps) * w[pre + "norm1"])
        if layer["type"] == "parallel":
            y = parallel_mixer(h, w, pre + "mix.", layer["mixer"], eps)
        elif layer["type"] == "mingru":
            y, _ = mingru(h, w, pre + "mix.")
        else:
            raise ValueError(layer["type"])
        x = x + m * y
        if layer.get("mlp") is not None:
            x = x + m * feed_forward(rounded(rms_unit(x, eps) * w[pre + "norm2"]), w, pre + "mlp.")
        if layers_out is not None:
            layers_out.append(x.clone())
    return soft_cap((rms_unit(x, eps) * w["final.norm"]) @ w["head"].T, cfg.get("logit_softcap"))


# ---- configurations, tensors and folders for the tests ------------------------------------------


def parallel_layer(heads, kv_heads, dim, vdim, scale, rot, right_heads, right_dim, mask=None, mlp=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot}
    if mask is not None:
        left["mask"] = mask
    return {"type": "parallel", "mixer": {"left": left, "right": {"heads": right_heads, "dim": right_dim}}, "mlp": mlp}


def mingru_layer(width, mlp=None):
    return {"type": "mingru", "mixer": {"width": width}, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def rotation(base, dims, factor=None):
    rot = {"base": base, "dims": dims}
    if factor is not None:
        rot["scaling"] = {"factor": factor}
    return rot


def window(size, keep_first=None):
    return {"size": size} if keep_first is None else {"size": size, "keep_first": keep_first}


def model_cfg(width, vocab, layers, scale=1.0, bigram=None, loop=None, residual_mult=None, softcap=None, eps=1e-5):
    cfg = {"architecture": "Nodupel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers,
           "embedding": {"scale": scale}}
    if bigram is not None:
        cfg["embedding"]["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))
    if loop is not None:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    if residual_mult is not None:
        cfg["residual_mult"] = residual_mult
    if softcap is not None:
        cfg["logit_softcap"] = softcap
    return cfg


def tensor_shapes(cfg, ranks) -> dict:
    """Name -> shape of every tensor of a folder; ``ranks``: layer -> rank of its decay projection."""
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "final.norm": (W,), "head": (cfg["vocab"], W)}
    if cfg["embedding"].get("bigram"):
        out["bigram"] = (cfg["embedding"]["bigram"]["buckets"] + 1, W)
    if cfg.get("loop"):
        out["loop.in"] = (W, 2 * W)
    for i, layer in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", layer["mixer"]
        out[pre + "norm1"] = (W,)
        if layer["type"] == "parallel":
            a, b = m["left"], m["right"]
            n = b["heads"] * b["dim"]
            out[pre + "mix.left.q"] = (a["heads"] * a["dim"], W)
            out[pre + "mix.left.k"] = (a["kv_heads"] * a["dim"], W)
            out[pre + "mix.left.v"] = (a["kv_heads"] * a["vdim"], W)
            out[pre + "mix.left.g"] = (a["heads"], W)
            out[pre + "mix.left.o"] = (W, a["heads"] * a["vdim"])
            for s in "rkvgw":
                out[f"{pre}mix.right.mu.{s}"] = (W,)
            for s in "rkvg":
                out[f"{pre}mix.right.{s}"] = (n, W)
            out[pre + "mix.right.w1"], out[pre + "mix.right.w2"] = (ranks[i], W), (n, ranks[i])
            out[pre + "mix.right.w0"], out[pre + "mix.right.u"] = (n,), (b["heads"], b["dim"])
            out[pre + "mix.right.norm"], out[pre + "mix.right.o"] = (n,), (W, n)
            out[pre + "mix.left.out"] = out[pre + "mix.right.out"] = (W,)
        else:
            for s in ("z", "x"):
                out[f"{pre}mix.{s}"], out[f"{pre}mix.{s}.b"] = (m["width"], W), (m["width"],)
            out[pre + "mix.g"], out[pre + "mix.o"] = (m["width"], W), (W, m["width"])
        if layer.get("mlp") is not None:
            ff = layer["mlp"]["ff"]
            out[pre + "norm2"] = (W,)
            out[pre + "mlp.gate"], out[pre + "mlp.up"], out[pre + "mlp.down"] = (ff, W), (ff, W), (W, ff)
    return out


def random_weights(cfg, ranks, seed, std=0.12, stored=torch.bfloat16):
    """Matrices N(0, std); norm weights around one; shifts in (0, 1); biases, bonus and decays of
    a size that counts; rounded to ``stored`` so that engine and plain model hold the same numbers."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, ranks).items():
        parts = name.split(".")
        last = parts[-1]
        r = lambda scale=1.0: scale * torch.randn(shape, generator=gen)  # noqa: E731
        if name == "embed":
            t = r(0.7) / max(1.0, cfg["embedding"]["scale"])
        elif name == "bigram":
            t = r(0.5)
        elif name == "loop.in":
            t = r(0.8 / math.sqrt(shape[1]))
        elif last in ("norm1", "norm2", "norm", "out"):
            t = 1.0 + r(0.2)
        elif "mu" in parts:
            t = torch.rand(shape, generator=gen)
        elif last == "w0":
            t = -1.0 + r(1.5)
        elif last in ("b", "u"):
            t = r(0.8)
        elif last == "w2":
            t = r(0.6)
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


# a loop over two of three layers, both kinds of mixer, kept first tokens, a table of pairs
NOD_A = model_cfg(64, 331, [
    parallel_layer(4, 2, 16, 16, 0.3, rotation(5000.0, 16, 2.5), 2, 16, window(24, 5), dense(96)),
    mingru_layer(40, dense(72)),
    parallel_layer(4, 1, 16, 32, 0.35, rotation(900.0, 8, 1.5), 4, 8, window(40, 21), dense(80)),
], scale=3.0, bigram=(37, 5, 11), loop=(1, 3, 2), residual_mult=0.6, softcap=8.0)
NOD_A_RANKS = {0: 8, 2: 6}
# the loop begins at the first layer and runs three times; no table of pairs, no multiplier, no cap; no
# window; a window shorter than what is kept; value heads larger and smaller than the keys'; a layer
# without feed-forward; one head of 48 channels
NOD_B = model_cfg(48, 257, [
    mingru_layer(56),
    parallel_layer(6, 3, 8, 24, 0.5, rotation(10.0, 4), 1, 48, None, dense(40)),
    parallel_layer(2, 2, 24, 8, 0.25, rotation(300.0, 24), 2, 24, window(7, 20), dense(52)),
], loop=(0, 2, 3))
NOD_B_RANKS = {1: 5, 2: 3}
# sizes that are multiples of nothing; a window without kept tokens; a loop of one pass; a hash that
# passes the token before over
NOD_C = model_cfg(42, 203, [
    parallel_layer(5, 1, 12, 20, 0.2, rotation(77.0, 6, 3.0), 2, 20, window(33), dense(50)),
    mingru_layer(30, dense(38)),
    parallel_layer(3, 3, 10, 6, 0.4, rotation(20.0, 10), 3, 10, window(17, 1), None),
], scale=0.5, bigram=(7, 0, 3), loop=(1, 2, 1), residual_mult=1.3, softcap=30.0, eps=1e-6)
NOD_C_RANKS = {0: 6, 2: 2}
