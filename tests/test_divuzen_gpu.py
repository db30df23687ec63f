"""Divuzen on the GPU against the plain implementation in ``plain_divuzen``: every new or changed
kernel alone, every mechanism alone in a model of one or two layers, then whole models of three
configurations under the ways of cutting (whole, decoded tail, portions down to two tokens,
mixed batches over a pool of exactly the trace's peak, filled with NaN, whose pages and slots
serve again), tokens made loud far back, at the first positions and on both sides of a page's and
of a chunk's border (in prompts and decoded), for an attention's own keys, for borrowed ones and for
the retention's state, long decoding beside requests that come and go, the stream after every
layer, and greedy generation through the engine's entry point and the programs."""

import math

import pytest
import torch

import plain_divuzen as P
import replay
from halite_amd.config import ModelConfig, ServerConfig
from halite_amd.engine import InferenceEngine
from halite_amd.engine.runner import ModelRunner
from halite_amd.kernels import ops

pytestmark = pytest.mark.gpu
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}
TOL = {"float32": 5e-5, "bfloat16": 2.5e-2}  # of the largest logit
CONFIGS = {"A": P.DIV_A, "B": P.DIV_B, "C": P.DIV_C}
LENGTHS = {"A": [5, 70, 33, 1, 150], "B": [90, 2, 41, 160], "C": [64, 17, 200, 3]}
F = torch.float64


def tokens(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def plain_logits(cfg, weights, ids):
    return P.forward(cfg, weights, ids).float()


def make_runner(folder, dtype, pool_tokens, page_size=16, graphs=False):
    server = ServerConfig(kv_cache_num_tokens=pool_tokens, page_size=page_size, max_seqs_per_forward=4,
                          use_cudagraph=graphs)
    runner = ModelRunner.from_pretrained(folder, server, ModelConfig(dtype=dtype))
    for g in runner.cache.groups:  # a page that is read before it is written, or after its time, shows
        g.storage.fill_(float("nan"))
    return runner


def sensitivity(cfg, weights, requests, ref):
    """Per request and position: how far the plain model's logits move (of the largest logit)
    when every part's input is rounded to bfloat16."""
    out = {}
    for rid, ids in requests.items():
        moved = P.forward(cfg, weights, ids, round_inputs=torch.bfloat16).float()
        out[rid] = (moved - ref[rid]).abs().amax(-1) / max(1.0, float(ref[rid].abs().max()))
    return out


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    out = {}
    for name, cfg in CONFIGS.items():
        weights = P.random_weights(cfg, seed=15 + ord(name))
        requests = {f"r{i}": P.tokens_with_clear_routing(cfg, weights, tokens(cfg, n, 700 + i)) for i, n in enumerate(LENGTHS[name])}
        ref = {rid: plain_logits(cfg, weights, ids) for rid, ids in requests.items()}
        sens = sensitivity(cfg, weights, requests, ref)
        for dtype in DT:
            folder = str(tmp_path_factory.mktemp(f"div{name}_{dtype}"))
            P.write_model_folder(folder, cfg, weights, DT[dtype])
            out[(name, dtype)] = (folder, requests, ref, weights, sens)
    return out


def check(rows, ref, dtype, sens):
    """float32: every row within the tolerance.  bfloat16: the norms on the parts' results make a
    position whose result nearly cancels as sensitive to the roundings before it as the result is
    small; the plain model with rounded inputs says which positions those are.  So every row
    is finite and within five times the tolerance plus three times its position's sensitivity,
    and all but a few (4%, at least two) within the tolerance plus that."""
    if dtype == "float32":
        return replay.compare(rows, ref, TOL[dtype])
    n = over = 0
    for rid, by_pos in rows.items():
        scale = max(1.0, float(ref[rid].abs().max()))
        for p, row in by_pos.items():
            err = float((row - ref[rid][p]).abs().max()) / scale
            room = 3.0 * float(sens[rid][p])
            assert err <= 5 * TOL[dtype] + room, f"request {rid} position {p}: error {err:.3e} (sensitivity {float(sens[rid][p]):.3e})"
            n, over = n + 1, over + (err > TOL[dtype] + room)
    assert over <= max(2, 0.04 * n), f"{over} of {n} rows beyond the tolerance"


def rand(*shape, seed=0, scale=1.0):
    return scale * torch.randn(*shape, generator=torch.Generator().manual_seed(seed))


def i32(x, gpu):
    return torch.tensor(x, dtype=torch.int32, device=gpu)


def close(got, want, tol):
    got = got.double().cpu()
    assert not bool(torch.isnan(got).any())
    err = float((got - want).abs().max())
    assert err <= tol * max(1e-6, float(want.abs().max())), f"{err:.3e} of {float(want.abs().max()):.3e}"


def table(rot, n, gpu):
    a = torch.arange(n, dtype=F)[:, None] * rot["base"] ** (-2.0 * torch.arange(rot["dims"] // 2, dtype=F) / rot["dims"])[None, :]
    return dict(cos=a.cos().float().to(gpu), sin=a.sin().float().to(gpu))


# -- kernels alone --------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("interleaved", [False, True])
@pytest.mark.parametrize("shape", [(4, 2, 16, 16, 16, 8), (5, 1, 12, 20, 32, 12), (3, 3, 70, 24, 80, 34)])
def test_heads_normed_weighted_and_turned(gpu, dtype, interleaved, shape):
    """q and k normed, weighted and turned in the kernel that packs them; queries alone, as a layer
    that borrows its keys takes them, are the same rows without the keys' columns."""
    H, K, dq, dv, D, dims = shape
    t = 19
    q, k, v = rand(t, H * dq, seed=1, scale=2.0), rand(t, K * dq, seed=2, scale=0.3), rand(t, K * dv, seed=3)
    wq, wk = (1 + 0.3 * rand(dq, seed=5)).to(DT[dtype]), (1 + 0.3 * rand(dq, seed=6)).to(DT[dtype])
    rot = P.rot(40.0, dims)
    pos = torch.randint(0, 90, (t,), generator=torch.Generator().manual_seed(7))
    turn = dict(positions=i32(pos.tolist(), gpu), interleaved=interleaved, **table(rot, 90, gpu))
    packed = ops.head_norm_pack(q.to(gpu), k.to(gpu), v.to(gpu), 1e-5, H, K, dq, dv, D, DT[dtype], w_q=wq.to(gpu), w_k=wk.to(gpu),
                                norm_v=False, **turn)
    got = packed.float().cpu().view(t, H + 2 * K, D)
    tol = 1e-5 if dtype == "float32" else 1e-2
    turned = lambda x, heads, w: P.rotate(P.rms_unit(x.to(F).view(t, heads, dq), 1e-5) * w.to(F), pos, rot, interleaved)  # noqa: E731
    for part, want, d in ((got[:, :H], turned(q, H, wq), dq), (got[:, H : H + K], turned(k, K, wk), dq),
                          (got[:, H + K :], v.to(F).view(t, K, dv), dv)):
        close(part[..., :d], want, tol)
        assert float(part[..., d:].abs().max() if D > d else 0.0) == 0.0
    alone = ops.head_norm_pack(q.to(gpu), None, None, 1e-5, H, 0, dq, dv, D, DT[dtype], w_q=wq.to(gpu), w_k=wq.to(gpu), norm_v=False, **turn)
    assert torch.equal(alone, packed[:, : H * D].contiguous())


@pytest.mark.parametrize("interleaved", [False, True])
@pytest.mark.parametrize("dims", [0, 6, 20])
def test_heads_turned_in_place(gpu, interleaved, dims):
    """Keys and queries side by side in a column range of wider rows; the keys alone are scaled."""
    H, D, t = 3, 20, 17
    a = rand(t, 5 + 2 * H * D + 3, seed=1)
    pos = torch.randint(0, 50, (t,), generator=torch.Generator().manual_seed(2))
    ag = a.to(gpu)
    turn = dict(positions=i32(pos.tolist(), gpu), interleaved=interleaved, **table(P.rot(30.0, dims), 50, gpu)) if dims else {}
    ops.rotate_heads_(ag[:, 5 : 5 + 2 * H * D], 2 * H, D, n_scaled=H, scale=0.3, **turn)
    got = ag.cpu()
    want = P.rotate(a[:, 5 : 5 + 2 * H * D].to(F).view(t, 2 * H, D), pos, P.rot(30.0, dims) if dims else None, interleaved)
    want = torch.cat([want[:, :H] * 0.3, want[:, H:]], 1).reshape(t, 2 * H * D)
    close(got[:, 5 : 5 + 2 * H * D], want, 1e-6)
    assert torch.equal(got[:, :5], a[:, :5]) and torch.equal(got[:, 5 + 2 * H * D :], a[:, 5 + 2 * H * D :])


def retention_rows(H, N, Pv, t, seed):
    """Float32 rows [v | k | q | gate] of a recurrence with H heads."""
    return rand(t, 2 * H * Pv + 2 * H * N, seed=seed, scale=0.7)


def parts_of(a, H, N, Pv):
    cuts = [H * Pv, H * N, H * N, H * Pv]
    return torch.split(a, cuts, dim=1)


def plain_retention(a, H, N, Pv, decay, S, pos, rot, interleaved, k_scale, in_silu):
    """The reads of the recurrence and the state after it, from float64 rows."""
    act = P.silu if in_silu else (lambda x: x)
    v, k, q, gate = parts_of(a.to(F), H, N, Pv)
    t = a.shape[0]
    v = act(v).view(t, H, Pv)
    k = P.rotate(act(k).view(t, H, N), pos, rot, interleaved) * k_scale
    q = P.rotate(act(q).view(t, H, N), pos, rot, interleaved)
    out, S = P.decayed_state_walk(q, k, v, decay, S)
    return out, S, gate


DECAYS = torch.tensor([0.9, 1.0, 0.999, 0.5, 0.03], dtype=F)
STATES = [(4, 16, 16), (1, 48, 8), (3, 8, 24), (2, 20, 72), (2, 64, 64), (1, 130, 4), (2, 32, 260), (1, 256, 128)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("shape", STATES)
@pytest.mark.parametrize("variant", ["retention", "weighted", "bare"])
def test_a_step_of_single_tokens_in_one_kernel(gpu, dtype, shape, variant):
    """Three requests in slots that are not in order, a token each, four steps in a row on states that
    are not zero: turned, walked, normed and gated.  The rows of other slots hold NaN."""
    H, N, Pv = shape
    rot = None if variant == "bare" else P.rot(25.0, N if variant == "weighted" else max(2, N // 4 * 2))
    interleaved, in_silu, silu = variant == "weighted", variant == "bare", variant != "bare"
    decay = DECAYS[:H]
    slots, at = [4, 0, 2], [7, 0, 30]
    state = torch.full((6, H, N, Pv), float("nan"), device=gpu)
    S = {s: 0.5 * rand(H, N, Pv, seed=40 + s).to(F) for s in slots}
    for s in slots:
        state[s] = S[s].float().to(gpu)
    w = (1 + 0.2 * rand(H * Pv, seed=3)).to(DT[dtype]) if variant == "weighted" else None
    for step in range(4):
        a = retention_rows(H, N, Pv, 3, seed=50 + step)
        pos = torch.tensor([p + step for p in at])
        v, k, q, gate = parts_of(a.to(gpu), H, N, Pv)
        turn = dict(positions=i32(pos.tolist(), gpu), interleaved=interleaved, **table(rot, 64, gpu)) if rot else {}
        y = ops.decay_step(v, k, q, gate, decay.float().to(gpu), state, i32(slots, gpu), 1e-5, DT[dtype], k_scale=0.3,
                           in_silu=in_silu, weight=None if w is None else w.to(gpu), silu=silu, **turn)
        for i, s in enumerate(slots):
            out, S[s], g = plain_retention(a[i : i + 1], H, N, Pv, decay, S[s], pos[i : i + 1], rot, interleaved, 0.3, in_silu)
            want = P.rms_unit(out, 1e-5).reshape(1, H * Pv) * (1.0 if w is None else w.to(F)) * (P.silu(g) if silu else torch.sigmoid(g))
            close(y[i : i + 1], want, 2e-5 if dtype == "float32" else 1e-2)
    for s in slots:
        close(state[s], S[s], 1e-5)
    assert all(bool(torch.isnan(state[s]).all()) for s in (1, 3, 5))


CHUNKED = [(4, 16, 16), (3, 8, 24), (2, 20, 70), (2, 64, 64), (1, 128, 5), (1, 33, 130), (2, 100, 256), (1, 4, 3)]


@pytest.mark.parametrize("shape", CHUNKED)
@pytest.mark.parametrize("variant,dtype", [("retention", "float32"), ("retention", "bfloat16"), ("weighted", "float32"),
                                           ("weighted", "bfloat16"), ("raw", "float32")])
def test_chunks_as_products(gpu, dtype, shape, variant):
    """Long segments beside short ones, down to a single token, each cut into chunks that start at
    the segment's own start, from states that are not zero and positions that are not zero."""
    H, N, Pv = shape
    rot = None if variant == "raw" else P.rot(25.0, N // 2 * 2 if variant == "weighted" else max(2, N // 4 * 2))
    interleaved, in_silu, silu = variant == "weighted", variant == "raw", variant == "retention"
    decay = DECAYS[:H]
    slots, cuts, at = [3, 0, 5, 1], [150, 1, 64, 67], [9, 40, 0, 3]
    state = torch.full((6, H, N, Pv), float("nan"), device=gpu)
    S = {s: 0.5 * rand(H, N, Pv, seed=60 + s).to(F) for s in slots}
    for s in slots:
        state[s] = S[s].float().to(gpu)
    w = (1 + 0.2 * rand(H * Pv, seed=3)).to(DT[dtype]) if variant == "weighted" else None
    starts = [sum(cuts[:i]) for i in range(4)]
    a = retention_rows(H, N, Pv, sum(cuts), seed=70)
    pos = torch.cat([torch.arange(n) + p for n, p in zip(cuts, at)])
    per = [-(-n // 64) for n in cuts]
    chunks = [[starts[s] + c * 64, min(64, cuts[s] - c * 64), s, 0] for s in range(4) for c in range(per[s])]
    seg_chunks = [[sum(per[:s]), per[s]] for s in range(4)]
    slot_of = [s for s, n in zip(slots, cuts) for _ in range(n)]
    v, k, q, gate = parts_of(a.to(gpu), H, N, Pv)
    turn = dict(positions=i32(pos.tolist(), gpu), interleaved=interleaved, **table(rot, 200, gpu)) if rot else {}
    y = ops.decay_chunks(v, k, q, None if variant == "raw" else gate, ops.decay_powers(decay).to(gpu), state, i32(starts, gpu),
                         i32(cuts, gpu), i32(slot_of, gpu), i32(chunks, gpu), i32(seg_chunks, gpu), 1e-5, DT[dtype], k_scale=0.3,
                         in_silu=in_silu, weight=None if w is None else w.to(gpu), silu=silu, **turn)
    for s in range(4):
        part = slice(starts[s], starts[s] + cuts[s])
        out, end, g = plain_retention(a[part], H, N, Pv, decay, S[slots[s]], pos[part], rot, interleaved, 0.3, in_silu)
        want = out.reshape(cuts[s], H * Pv)
        if variant != "raw":
            want = P.rms_unit(out, 1e-5).reshape(cuts[s], H * Pv) * (1.0 if w is None else w.to(F)) * (P.silu(g) if silu else torch.sigmoid(g))
        close(y[part], want, 5e-5 if dtype == "float32" else 1e-2)
        close(state[slots[s]], end, 2e-5)
    assert bool(torch.isnan(state[2]).all()) and bool(torch.isnan(state[4]).all())


ROUTERS = [(6, 3, 0, 0), (6, 3, 3, 2), (6, 2, 6, 4), (64, 8, 8, 3), (17, 5, 1, 1), (100, 7, 10, 4), (96, 4, 48, 5), (256, 8, 8, 4),
           (250, 6, 125, 30), (384, 9, 8, 4), (1024, 12, 128, 40), (1000, 3, 0, 0)]


@pytest.mark.parametrize("sizes", ROUTERS)
@pytest.mark.parametrize("stored", ["float32", "bfloat16"])
def test_the_choice_among_groups(gpu, sizes, stored):
    """Sigmoid scores with a correction of either sign (all choice scores of some tokens negative),
    the best groups, the best experts of those, weights without the correction, from a column range
    of wider rows; the kernel that routes and sorts makes the same choice."""
    E, top, groups, keep = sizes
    t = 13
    z = rand(t, E + 2, seed=1, scale=2.0)
    corr = (0.4 * rand(E, seed=2) - 0.5).to(DT[stored])
    router = dict(experts=E, top=top)
    if groups:
        router["groups"] = dict(count=groups, keep=keep)
    scores = torch.sigmoid(z[:, :E].to(F))
    margins = []
    want = P.choose_experts(scores, corr.to(F), router, margins)
    clear = margins[0] > 1e-6
    assert int(clear.sum()) >= t - 1
    how = dict(normalize=True, norm_eps=1e-20, scale=1.7, correction=corr.to(gpu), groups=groups, keep=keep)
    idx, wgt = ops.moe_route(z.to(gpu)[:, :E], top, **how)
    assert torch.equal(idx.cpu().long()[clear], want[clear])
    s = scores.gather(1, want)
    close(wgt[clear.to(gpu)], (s / s.sum(-1, keepdim=True) * 1.7)[clear], 1e-5)
    if E <= ops.ROUTE_SORT_MAX_EXPERTS:
        idx2, wgt2, offsets, tiles, order = ops.moe_route_sort(z.to(gpu)[:, :E], top, E, **how)
        assert torch.equal(idx2, idx) and torch.equal(wgt2, wgt)
    else:
        offsets, tiles, order = ops.moe_sort(idx, E)
    o, pairs, flat = offsets.cpu().tolist(), order.cpu().tolist(), idx.cpu().flatten().tolist()
    assert o[0] == 0 and o[E] == t * top and sorted(pairs) == list(range(t * top))
    assert all(flat[pairs[i]] == e for e in range(E) for i in range(o[e], o[e + 1]))
    assert tiles.cpu().tolist() == [sum(-(-(o[j + 1] - o[j]) // ops.GROUP_TILE_ROWS) for j in range(e)) for e in range(E + 1)]


def test_equal_scores_go_to_the_lower_index(gpu):
    z = torch.zeros(3, 12)
    for E in (12,):
        idx, wgt = ops.moe_route(z.to(gpu), 3, normalize=True)
        assert idx.cpu().tolist() == [[0, 1, 2]] * 3 and float((wgt.cpu() - 1 / 3).abs().max()) < 1e-6
        idx, _ = ops.moe_route(z.to(gpu), 3, groups=4, keep=2)
        assert idx.cpu().tolist() == [[0, 1, 2]] * 3
    wide = torch.zeros(2, 300)
    idx, _ = ops.moe_route(wide.to(gpu), 70, groups=3, keep=1)
    assert idx.cpu().tolist() == [list(range(70))] * 2


@pytest.mark.parametrize("limit", [0.7, math.inf])
def test_the_clamped_gate(gpu, limit):
    """As a pass of its own over a product's rows (float32 and bf16, row lengths that are and are not
    multiples of four) and as the small-batch product's epilogue."""
    clamp = ops.Clamp(limit, 1.702, 1.0)

    def plain(g, u):
        g, u = g.clamp(max=limit), u.clamp(-limit, limit)
        return g * torch.sigmoid(1.702 * g) * (u + 1.0)

    for f in (20, 21):
        gu = rand(9, 2 * f, seed=f, scale=2.0)
        close(ops.gate_mul(gu.to(gpu), "clamped", clamp), plain(gu[:, :f].to(F), gu[:, f:].to(F)), 1e-6)
        low = gu.to(torch.bfloat16)
        close(ops.gate_mul(low.to(gpu), "clamped", clamp), plain(low[:, :f].to(F), low[:, f:].to(F)), 1e-2)
    x, wg, wu = (rand(*s, seed=i, scale=0.3).to(torch.bfloat16) for i, s in enumerate(((11, 72), (40, 72), (40, 72))))
    want = plain(x.to(F) @ wg.to(F).T, x.to(F) @ wu.to(F).T)
    tiled = [ops.tile_weight(t.to(gpu)) for t in (wg, wu)]
    close(ops.gemm_bf16_skinny(x.to(gpu), tiled[0], w_up=tiled[1], tiled_shape=(40, 72), activation="clamped", clamp=clamp), want, 1e-2)


@pytest.mark.parametrize("width", [64, 42, 2048])
def test_a_normed_result_written_and_the_next_row_read(gpu, width):
    """``x += norm(y)`` with a weight stored around zero, and the next part's normed row, in one pass."""
    t = 7
    x, y, w1, w2 = rand(t, width, seed=1), rand(t, width, seed=2, scale=5.0), 0.3 * rand(width, seed=3), 0.3 * rand(width, seed=4)
    want = x.to(F) + P.model_norm(y.to(F), w1.to(F), 1e-5)
    xg = x.to(gpu)
    got = ops.stream_step(xg, y=ops.NormedTerms([(y.to(gpu), (1.0 + w1).to(gpu), 1.0)], 1e-5), read=True, norm_weight=w2.to(gpu),
                          offset=1.0, eps=1e-5, dtype=torch.float32)
    close(xg, want, 1e-6)
    close(got, P.model_norm(want, w2.to(F), 1e-5), 2e-6)


@pytest.mark.parametrize("width", [64, 42, 1032])
@pytest.mark.parametrize("shared", [False, True])
def test_the_experts_sum_in_the_pass_that_norms_it(gpu, width, shared):
    """The weighted sum of a token's experts (and the gated shared one) made by the stream's step, of all
    rows and of chosen ones."""
    t, top = 9, 3
    x, rows, wgt = rand(t, width, seed=1), rand(t * top, width, seed=2, scale=3.0), rand(t, top, seed=3).abs()
    extra, gates, w1, w2 = rand(t, width, seed=4), rand(t, 5, seed=5), 0.3 * rand(width, seed=6), 0.3 * rand(width, seed=7)
    y = (wgt.to(F)[:, :, None] * rows.to(F).view(t, top, width)).sum(1)
    if shared:
        y = y + torch.sigmoid(gates[:, 4:].to(F)) * extra.to(F)
    want = x.to(F) + P.model_norm(y, w1.to(F), 1e-5)
    term = ops.ExpertSum(rows.to(gpu), wgt.to(gpu), extra.to(gpu) if shared else None, gates.to(gpu)[:, 4:] if shared else None)
    close(term.materialize(), y, 1e-6)
    how = dict(read=True, norm_weight=w2.to(gpu), offset=1.0, eps=1e-5, dtype=torch.float32)
    terms = ops.NormedTerms([(term, (1.0 + w1).to(gpu), 1.0)], 1e-5)
    some = [4, 0, 7]
    chosen = ops.stream_step(x.to(gpu), y=terms, rows=i32(some, gpu), **how)
    close(chosen, P.model_norm(want, w2.to(F), 1e-5)[some], 2e-6)
    xg = x.to(gpu)
    close(ops.stream_step(xg, y=terms, **how), P.model_norm(want, w2.to(F), 1e-5), 2e-6)
    close(xg, want, 1e-6)


# -- every mechanism alone ----------------------------------------------------------------------

SMALL_LAYERS = {
    "attention": [P.attention_layer(4, 2, 8, 12, 0.4, rot=P.rot(500.0, 4))],
    "attention_whole_head": [P.attention_layer(3, 3, 8, 8, 0.4, rot=P.rot(20.0, 8))],
    "borrowed": [P.attention_layer(4, 2, 8, 12, 0.4, rot=P.rot(500.0, 4)),
                 P.attention_layer(4, 2, 8, 12, 0.6, rot=P.rot(500.0, 4), kv_from=0)],
    "retention": [P.retention_layer(3, 8, 12, [0.8, 0.99, 1.0], rot=P.rot(30.0, 4))],
    "retention_unturned": [P.retention_layer(2, 6, 5, [0.8, 0.99])],
    "retention_wide": [P.retention_layer(1, 136, 20, [0.98], rot=P.rot(100.0, 64))],
    "dense": [P.retention_layer(1, 8, 8, [0.9], mlp=P.dense(20, 0.4))],
    "experts": [P.retention_layer(1, 8, 8, [0.9], mlp=P.moe(8, 2, 12, scale=2.2, groups=(4, 2), shared=10))],
    "experts_plain": [P.retention_layer(1, 8, 8, [0.9], mlp=P.moe(7, 3, 12))],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(SMALL_LAYERS))
def test_small_models(name, dtype, tmp_path):
    """A model of one layer for each mechanism (of two for borrowed keys): a prompt whole against
    token by token, portions and mixed batches."""
    cfg = P.model_cfg(32, 97, SMALL_LAYERS[name], logit_scale=0.5)
    w = P.random_weights(cfg, seed=31)
    requests = {"a": P.tokens_with_clear_routing(cfg, w, tokens(cfg, 140, 1)), "b": P.tokens_with_clear_routing(cfg, w, tokens(cfg, 21, 2))}
    ref = {rid: plain_logits(cfg, w, ids) for rid, ids in requests.items()}
    sens = sensitivity(cfg, w, requests, ref)
    folder = P.write_model_folder(str(tmp_path), cfg, w, DT[dtype])
    for make in (replay.whole, lambda q: replay.tail_one_by_one(q, tail=50), replay.portions, replay.mixed):
        trace = make(requests)
        runner = make_runner(folder, dtype, replay.peak_tokens(trace, 16))
        rows = replay.collect(trace, replay.run_trace(runner, trace), cfg["vocab"])
        check(rows, ref, dtype, sens)
        assert runner.cache.idle()


# -- whole models -----------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("schedule", ["whole", "tail", "portions", "twos", "mixed", "mixed2"])
def test_schedules(folders, name, dtype, schedule):
    folder, requests, ref, _, sens = folders[(name, dtype)]
    cfg = CONFIGS[name]
    make = {"whole": replay.whole, "tail": lambda q: replay.tail_one_by_one(q, tail=40), "portions": replay.portions,
            "twos": lambda q: replay.portions(q, sizes=(2, 2, 130, 3, 2)),
            "mixed": replay.mixed, "mixed2": lambda q: replay.mixed(q, seed=7, decode_tail=30)}[schedule]
    trace = make(requests)
    runner = make_runner(folder, dtype, replay.peak_tokens(trace, 16))
    rows = replay.collect(trace, replay.run_trace(runner, trace), cfg["vocab"])
    check(rows, ref, dtype, sens)
    assert runner.cache.idle()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("page_size", [8, 32, 64])
@pytest.mark.parametrize("name", ["A", "C"])
def test_other_page_sizes(folders, name, page_size, dtype):
    folder, requests, ref, _, sens = folders[(name, dtype)]
    trace = replay.mixed(requests, seed=3)
    runner = make_runner(folder, dtype, replay.peak_tokens(trace, page_size), page_size=page_size)
    rows = replay.collect(trace, replay.run_trace(runner, trace), CONFIGS[name]["vocab"])
    check(rows, ref, dtype, sens)
    assert runner.cache.idle()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_batch_of_unequal_requests_against_each_alone(folders, dtype):
    """All requests' prompts in one step (the long ones in chunks, a single token among them)."""
    folder, requests, ref, _, sens = folders[("A", dtype)]
    runner = make_runner(folder, dtype, 512)
    ids = {rid: r for rid, r in requests.items() if rid != "r2"}
    trace = [{"step": 0, "entries": [{"id": rid, "tokens": t, "want": list(range(len(t)))} for rid, t in ids.items()], "end": list(ids)}]
    rows = replay.collect(trace, replay.run_trace(runner, trace), P.DIV_A["vocab"])
    check(rows, ref, dtype, sens)


@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_the_stream_after_every_layer(folders, name):
    from halite_amd.parts import block

    folder, requests, _, weights, _ = folders[(name, "float32")]
    cfg = CONFIGS[name]
    ids = requests["r1"]
    want = []
    P.forward(cfg, weights, ids, layers_out=want)
    runner = make_runner(folder, "float32", 256)
    seen, inner = [], block.HyperPreNormBlock.forward

    def forward(self, h, pending, ctx, run):
        out = inner(self, h, pending, ctx, run)
        seen.append(h[0] + out[0].materialize())  # (the block's last result is pending)
        return out

    block.HyperPreNormBlock.forward = forward
    try:
        replay.run_trace(runner, replay.whole({"r1": ids}))
    finally:
        block.HyperPreNormBlock.forward = inner
    assert len(seen) == len(want) == len(cfg["layers"])
    for got, w in zip(seen, want):
        assert float((got.cpu() - w.float()).abs().max()) < 5e-5 * max(1.0, float(w.abs().max()))


# -- tokens made loud -----------------------------------------------------------------------------

LOUD, ASK = 7, 11


def mark_embedding(w):
    """Channel 0 of the embedding is nonzero for LOUD alone and channel 1 for ASK alone (a norm
    keeps zeros), so a projection that reads one of them tells that token from all others."""
    w["embed"][:, :2] = 0.0
    w["embed"][LOUD, 0] = 3.0
    w["embed"][ASK, 1] = 3.0
    w["l0.norm1"][:2] = 0.0


def make_loud(w, name, heads, dim, row0, col, gain, quiet):
    """Row ``row0`` of every head of a projection reads one channel of the embedding alone; the rest is quiet."""
    w[name] *= quiet
    w[name][:, :2] = 0.0
    for head in range(heads):
        w[name][head * dim + row0] = 0.0
        w[name][head * dim + row0, col] = gain


def loud_attention_model(kv_heads=1):
    """Key channel 12 (which is not turned) is large for LOUD and zero for every other token, query
    channel 12 large for ASK and zero otherwise: behind the norms per head ASK's score on LOUD is
    nearly ``scale * dim`` where all other scores are small."""
    cfg = P.model_cfg(64, 61, [P.attention_layer(2, kv_heads, 16, 24, 1.2, rot=P.rot(1000.0, 8))])
    w = P.random_weights(cfg, seed=77)
    mark_embedding(w)
    make_loud(w, "l0.mix.k", kv_heads, 16, 12, 0, 4.0, 0.2)
    make_loud(w, "l0.mix.q", 2, 16, 12, 1, 4.0, 0.2)
    w["l0.mix.o"] *= 3.0
    return cfg, {k: v.to(torch.bfloat16).float() for k, v in w.items()}


def loud_borrowing_model():
    """The second layer asks for the first one's loud key (both norms keep the marked channels: the
    first layer's result does not touch them); the first layer itself asks for nothing."""
    cfg = P.model_cfg(64, 61, [P.attention_layer(2, 1, 16, 24, 1.2, rot=P.rot(1000.0, 8)),
                               P.attention_layer(2, 1, 16, 24, 1.2, rot=P.rot(1000.0, 8), kv_from=0)])
    w = P.random_weights(cfg, seed=78)
    mark_embedding(w)
    make_loud(w, "l0.mix.k", 1, 16, 12, 0, 4.0, 0.2)
    w["l0.mix.q"] *= 0.2
    w["l0.mix.o"][:2] = 0.0
    w["l1.norm1"][:2] = 0.0
    make_loud(w, "l1.mix.q", 2, 16, 12, 1, 4.0, 0.2)
    w["l1.mix.o"] *= 3.0
    return cfg, {k: v.to(torch.bfloat16).float() for k, v in w.items()}


def loud_retention_model():
    """A retention that forgets next to nothing, whose key channel 10 (which is not turned) is large for
    LOUD and zero for every other token and whose query channel 10 is large for ASK alone: what ASK
    reads is mostly LOUD's value, however long ago it was written."""
    cfg = P.model_cfg(64, 61, [P.retention_layer(2, 16, 24, [0.9998, 1.0], rot=P.rot(1000.0, 8))])
    w = P.random_weights(cfg, seed=79)
    mark_embedding(w)
    make_loud(w, "l0.mix.k", 2, 16, 10, 0, 4.0, 0.1)
    make_loud(w, "l0.mix.q", 2, 16, 10, 1, 4.0, 0.1)
    w["l0.mix.o"] *= 3.0
    return cfg, {k: v.to(torch.bfloat16).float() for k, v in w.items()}


LOUD_MODELS = {"attention": loud_attention_model, "attention_two_kv": lambda: loud_attention_model(kv_heads=2),
               "borrowed": loud_borrowing_model, "retention": loud_retention_model}


def loud_sequence(cfg, n, loud_at, ask_at, seed):
    ids = [t if t not in (LOUD, ASK) else 1 for t in tokens(cfg, n, seed)]
    for p in loud_at:
        ids[p] = LOUD
    for p in ask_at:
        ids[p] = ASK
    return ids


def quiet(ids):
    return [1 if t == LOUD else t for t in ids]


def replay_all(cfg, w, requests, dtype, tmp_path, tail=80, page_size=16):
    ref = {rid: plain_logits(cfg, w, ids) for rid, ids in requests.items()}
    sens = sensitivity(cfg, w, requests, ref) if dtype == "bfloat16" else None
    folder = P.write_model_folder(str(tmp_path), cfg, w, DT[dtype])
    for make in (replay.whole, lambda q: replay.tail_one_by_one(q, tail=tail), replay.portions,
                 lambda q: replay.portions(q, sizes=(15, 1, 32, 2, 1, 1, 16, 64, 129)), replay.mixed):
        trace = make(requests)
        runner = make_runner(folder, dtype, replay.peak_tokens(trace, page_size), page_size=page_size)
        rows = replay.collect(trace, replay.run_trace(runner, trace), cfg["vocab"])
        check(rows, ref, dtype, sens)
        assert runner.cache.idle()
    return ref


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("model", list(LOUD_MODELS))
def test_a_loud_token_far_back_and_at_the_first_positions(model, dtype, tmp_path):
    """LOUD at position 3 (and at 0) among hundreds of tokens across many pages and chunks; ASK right
    behind it, far behind it, and at the last position."""
    cfg, w = LOUD_MODELS[model]()
    requests = {"far": loud_sequence(cfg, 400, [3], [4, 200, 255, 256, 399], 2),
                "first": loud_sequence(cfg, 300, [0], [1, 150, 299], 3)}
    ref = replay_all(cfg, w, requests, dtype, tmp_path)
    for rid in requests:
        silent = plain_logits(cfg, w, quiet(requests[rid]))
        assert float((ref[rid][-1] - silent[-1]).abs().max()) > 0.1 * float(ref[rid].abs().max())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("model,edge", [("attention", 16), ("borrowed", 16), ("attention", 32), ("borrowed", 64), ("retention", 64)])
def test_loud_tokens_on_both_sides_of_an_edge(model, edge, dtype, tmp_path):
    """LOUD in the last place of a page (of a chunk of the retention) and in the first of the next one,
    ASK in the places around them and a few further on; the schedules put these places into
    prompts and into decoded tokens."""
    cfg, w = LOUD_MODELS[model]()
    n = 4 * edge + 9
    requests = {"last": loud_sequence(cfg, n, [2 * edge - 1], [2 * edge, 2 * edge + 1, 3 * edge - 1, 3 * edge, n - 1], 4),
                "first": loud_sequence(cfg, n, [2 * edge], [2 * edge + 1, 3 * edge - 1, 3 * edge, n - 1], 5)}
    ref = replay_all(cfg, w, requests, dtype, tmp_path, tail=2 * edge + 12, page_size=min(edge, 64))
    for rid in requests:
        silent = plain_logits(cfg, w, quiet(requests[rid]))
        assert float((ref[rid][n - 1] - silent[n - 1]).abs().max()) > 0.1 * float(ref[rid].abs().max())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_sink_that_takes_most_of_a_row(dtype, tmp_path):
    """Sinks of 3, -2 and 0.5: a request's first tokens lose most of their weight to the first head's."""
    cfg = P.model_cfg(32, 97, [P.attention_layer(3, 1, 8, 12, 0.5, rot=P.rot(500.0, 4))])
    w = P.random_weights(cfg, seed=33)
    w["l0.mix.sink"][:] = torch.tensor([3.0, -2.0, 0.5])
    requests = {"a": tokens(cfg, 70, 1), "b": tokens(cfg, 2, 2)}
    ref = replay_all(cfg, w, requests, dtype, tmp_path, tail=68)
    other = plain_logits(cfg, dict(w, **{"l0.mix.sink": torch.full((3,), -60.0)}), requests["a"])
    assert float((ref["a"][0] - other[0]).abs().max()) > 0.05 * float(ref["a"].abs().max())


# -- long decoding, slots and pages that serve again ------------------------------------------------


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("graphs", [False, True])
def test_long_decoding_beside_requests_that_come_and_go(folders, dtype, graphs):
    """A short prompt and 200 tokens decoded one by one (the state and the positions run on) beside
    short requests that take the freed slot and pages one after the other."""
    folder, _, _, weights, _ = folders[("A", dtype)]
    cfg = P.DIV_A
    ids, other = (P.tokens_with_clear_routing(cfg, weights, tokens(cfg, n, seed)) for n, seed in ((215, 41), (30, 42)))
    ref = {"long": plain_logits(cfg, weights, ids)}
    short = plain_logits(cfg, weights, other)
    sens = sensitivity(cfg, weights, {"long": ids, "other": other}, {"long": ref["long"], "other": short})
    trace = [{"step": 0, "entries": [{"id": "long", "tokens": ids[:15], "want": list(range(15))}], "end": []}]
    for i in range(15, 215):
        entries = [{"id": "long", "tokens": [ids[i]], "want": [0]}]
        j, rid = (i - 15) % 40, f"other{(i - 15) // 40}"
        if j < 30:
            entries.append({"id": rid, "tokens": [other[j]], "want": [0]})
            ref[rid], sens[rid] = short, sens["other"]
        trace.append({"step": len(trace), "entries": entries,
                      "end": (["long"] if i == 214 else []) + ([rid] if j == 29 else [])})
    runner = make_runner(folder, dtype, replay.peak_tokens(trace, 16), graphs=graphs)
    rows = replay.collect(trace, replay.run_trace(runner, trace), cfg["vocab"])
    check(rows, ref, dtype, sens)
    assert runner.cache.idle()
    if graphs:
        assert runner.graphs_allowed and runner.graph_replays > 100


# -- through the engine's entry point ----------------------------------------------------------------


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_greedy_generation_through_the_engine(folders, name, dtype):
    folder, _, _, weights, _ = folders[(name, dtype)]
    cfg = CONFIGS[name]
    prompts = [P.tokens_with_clear_routing(cfg, weights, tokens(cfg, n, 500 + n)) for n in (5, 17, 33, 2, 48, 9)]
    engine = InferenceEngine.from_pretrained(
        folder, ServerConfig(kv_cache_num_tokens=1024, page_size=16, max_seqs_per_forward=3, chunked_prefill_size=20,
                             max_tokens_per_forward=24),
        ModelConfig(dtype=dtype),
    )
    params = {"max_new_tokens": 12, "temperature": 0.0}
    results = engine.infer_batch([(i, p, params) for i, p in enumerate(prompts)])
    checked = 0
    for r, prompt in zip(results, prompts):
        ids = list(prompt)
        for step, tok in enumerate(r.output_ids[0]):
            margins = []
            logits = P.forward(cfg, weights, ids, margins_out=margins).float()[-1]
            if dtype == "bfloat16" and margins and float(torch.stack(margins).min()) < 0.03:
                break  # a router's close call among the generated tokens: 16 bits may take the other expert from here on
            best = int(torch.argmax(logits))
            if tok != best:  # 16 bits may turn a near tie; anything else is a fault
                gap = float(logits[best] - logits[tok])
                limit = (1e-4 if dtype == "float32" else 2 * TOL[dtype]) * max(1.0, float(logits.abs().max()))
                assert gap < limit, f"request {r.id} token {step}: {tok} for {best}, gap {gap}"
            ids.append(tok)
        assert len(r.output_ids[0]) == 12
        checked += len(ids) - len(prompt)
    # (in 16 bits the comparison of a request ends at a router's close call)
    assert checked >= (36 if dtype == "float32" else 12)


# -- the programs: generation from the command line, the random-weights mode, trace replay -----


def test_command_line_and_replay_program(folders, tmp_path):
    import json
    import os
    import subprocess
    import sys

    import numpy as np

    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    folder, _, _, weights, _ = folders[("A", "float32")]
    cfg = P.DIV_A
    cmd = [sys.executable, os.path.join(root, "bin", "halite_generate"), "--model", folder, "--prompt-ids", "5,17,3,90,9",
           "sampling.temperature=0", "sampling.max_new_tokens=5", "model.dtype=float32", "server.kv_cache_num_tokens=256"]
    proc = subprocess.run(cmd, cwd=root, capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    rec = json.loads(proc.stdout.strip().split("\n")[-1])
    ids = [5, 17, 3, 90, 9]
    for tok in rec["output_ids"][0]:
        assert tok == int(torch.argmax(plain_logits(cfg, weights, ids)[-1]))
        ids.append(tok)
    assert len(ids) == 10
    cfgfile, out = tmp_path / "c.json", tmp_path / "rand"
    cfgfile.write_text(json.dumps(P.DIV_C))
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "halite_make_random_model"), "--config", str(cfgfile),
                           "--out", str(out), "--seed", "3", "--dtype", "bfloat16", "--std", "0.1"], capture_output=True, text=True)
    assert proc.returncode == 0, proc.stderr[-2000:]
    # the replay program on that folder: a prompt in two portions and a decoded token, beside a
    # second request; two slots, so the third request takes the one that was freed
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": [1, 2, 3, 4, 5], "want": [4]}, {"id": "b", "tokens": [7], "want": [0]}], "end": ["b"]},
        {"step": 1, "entries": [{"id": "a", "tokens": [6, 7], "want": []}, {"id": "c", "tokens": [9, 8], "want": [1]}], "end": ["c"]},
        {"step": 2, "entries": [{"id": "a", "tokens": [8], "want": [0]}], "end": ["a"]},
    ]
    logits = tmp_path / "logits"
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(out), "--dtype", "float32",
                           "--out", str(logits), "--max-tokens", "128", "--slots", "2"],
                          input="\n".join(json.dumps(s) for s in steps) + "\n", cwd=root, capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.split("\n") if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    from safetensors.torch import load_file

    stored = {k: v.float() for k, v in load_file(str(out / "model.safetensors")).items()}
    got = [torch.from_numpy(np.fromfile(logits / f"{i}.f32", dtype="<f4").reshape(-1, P.DIV_C["vocab"])) for i in range(3)]
    want = plain_logits(P.DIV_C, stored, [1, 2, 3, 4, 5, 6, 7, 8])
    scale = max(1.0, float(want.abs().max()))
    for row, ref in ((got[0][0], want[4]), (got[2][0], want[7]), (got[0][1], plain_logits(P.DIV_C, stored, [7])[0]),
                     (got[1][0], plain_logits(P.DIV_C, stored, [9, 8])[1])):
        assert float((row - ref).abs().max()) < 5e-5 * scale
