"""Nodupel without a GPU: the configuration and what is read from tensors' shapes, the run
order and its junctions, the table of tensor names and the loader, the random-weights mode,
pages that stay behind a window, and the plain implementation's own pins."""

import json
import math
import os

import pytest
import torch

import plain_nodupel as P
from halite_amd.cache.manager import CacheManager
from halite_amd.config import parse_config, read_config
from halite_amd.config.registry import ConfigError
from halite_amd.config.spec import LayerRun, ModelSpec
from halite_amd.parts import Decoder
from halite_amd.parts.base import PagedKVNeed
from halite_amd.weights import load_weights, write_random_model
from halite_amd.weights.loader import WeightError

CONFIGS = {"A": (P.NOD_A, P.NOD_A_RANKS), "B": (P.NOD_B, P.NOD_B_RANKS), "C": (P.NOD_C, P.NOD_C_RANKS)}
F = torch.float64


def rand(*shape, seed=0, scale=1.0):
    return scale * torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F)


def stated(cfg, ranks):
    out = json.loads(json.dumps(cfg))
    for i, n in ranks.items():
        out["layers"][i]["mixer"]["right"]["decay_rank"] = n
    return out


def test_the_decay_rank_comes_from_the_tensor(tmp_path):
    cfg, ranks = CONFIGS["A"]
    arch, parsed = parse_config(cfg)
    assert arch.name == "Nodupel"
    with pytest.raises(ConfigError, match="decay_rank"):
        arch.to_spec(parsed)
    folder = P.write_model_folder(str(tmp_path), cfg, P.random_weights(cfg, ranks, 1))
    arch, parsed = read_config(folder)
    spec = arch.to_spec(parsed)
    assert spec.layers["l0"].parts["mixer"].params()["mixers"][1]["decay_rank"] == 8
    written = parsed.to_json_dict()
    assert "decay_rank" not in json.dumps(written) and written["layers"][0]["mixer"]["left"]["mask"] == {"size": 24, "keep_first": 5}
    assert written["loop"] == cfg["loop"] and written["embedding"] == cfg["embedding"]
    assert parse_config(stated(cfg, ranks))[0].to_spec(parse_config(stated(cfg, ranks))[1]) == spec
    assert ModelSpec(**json.loads(spec.model_dump_json())) == spec  # plain data


def test_the_run_order_and_its_junctions():
    order = {}
    for name, (cfg, ranks) in CONFIGS.items():
        arch, parsed = parse_config(stated(cfg, ranks))
        spec = arch.to_spec(parsed)
        order[name] = [(r.layer, r.junction) for r in spec.order]
        assert all(r.cache_from is None for r in spec.order)  # every pass keeps a cache and state of its own
        assert [(int(l[1:]), j is not None) for l, j in order[name]] == P.run_order(cfg)
    assert order["A"] == [("l0", None), ("l1", "loop"), ("l2", None), ("l1", "loop"), ("l2", None)]
    assert order["B"][0] == ("l0", "loop") and len(order["B"]) == 7
    once = stated(P.NOD_A, P.NOD_A_RANKS)
    once.pop("loop")
    arch, parsed = parse_config(once)
    spec = arch.to_spec(parsed)
    assert [r.layer for r in spec.order] == ["l0", "l1", "l2"] and spec.junctions == {}
    assert "loop.in" not in arch.weight_map(parsed)
    with pytest.raises(ValueError, match="junction"):
        ModelSpec(**{**spec.model_dump(), "order": [LayerRun(layer="l0", junction="nowhere")]})


def test_keys_that_are_left_out_switch_their_mechanism_off():
    arch, parsed = parse_config(stated(P.NOD_B, P.NOD_B_RANKS))
    spec = arch.to_spec(parsed)
    assert spec.embedding.params()["pairs"] is None and spec.head.params()["logit_softcap"] is None
    assert spec.layers["l0"].parts["mixer_link"].params()["mult"] == 1.0 and "ff" not in spec.layers["l0"].parts
    left = spec.layers["l1"].parts["mixer"].params()["mixers"][0]
    assert left["window"] is None and left["keep_first"] == 0
    assert spec.positions[left["position"]].params()["scaling"] is None
    names = arch.weight_map(parsed)
    assert "bigram" not in names and names["loop.in"] == "junctions.loop.weight" and names["l0.norm2"] is None
    # the keys turn with stretched frequencies, the values with unstretched ones over the whole head
    arch, parsed = parse_config(stated(P.NOD_A, P.NOD_A_RANKS))
    spec = arch.to_spec(parsed)
    left = spec.layers["l2"].parts["mixer"].params()["mixers"][0]
    keys, values = spec.positions[left["position"]].params(), spec.positions[left["value_position"]].params()
    assert keys["rotary_dim"] == 8 and keys["scaling"]["factor"] == 1.5 and keys["angles"] == "float64"
    assert values["rotary_dim"] == 32 and values["scaling"] is None and values["theta"] == keys["theta"] == 900.0


@pytest.mark.parametrize("bad", [
    lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=3),
    lambda c: c["layers"][0]["mixer"]["left"].pop("scale"),
    lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=7),
    lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=18),
    lambda c: c["layers"][0]["mixer"]["left"].update(vdim=15),
    lambda c: c["layers"][0]["mixer"]["left"].update(mask={"size": 0}),
    lambda c: c["layers"][0]["mixer"].pop("right"),
    lambda c: c["layers"][1]["mixer"].update(width=0),
    lambda c: c["layers"][0].update(type="recurrent"),
    lambda c: c["layers"][0]["mlp"].update(kind="moe"),
    lambda c: c["loop"].update(stop=4),
    lambda c: c["loop"].update(start=3),
    lambda c: c["loop"].update(times=0),
    lambda c: c["embedding"].pop("scale"),
    lambda c: c["embedding"]["bigram"].update(buckets=0),
    lambda c: c.update(logit_softcap=0.0),
    lambda c: c.update(layers=[]),
    lambda c: c.pop("norm"),
    lambda c: c.update(width=64.5),
])
def test_configurations_that_are_refused(bad):
    cfg = json.loads(json.dumps(P.NOD_A))
    bad(cfg)
    with pytest.raises(ConfigError):
        parse_config(cfg)


@pytest.mark.parametrize("name", list(CONFIGS))
def test_the_model_as_data_and_its_tensors(name, tmp_path):
    cfg, ranks = CONFIGS[name]
    weights = P.random_weights(cfg, ranks, 2)
    folder = P.write_model_folder(str(tmp_path), cfg, weights)
    arch, parsed = read_config(folder)
    spec = arch.to_spec(parsed)
    assert [l.arrangement for l in spec.layers.values()] == ["hyper_pre_norm"] * len(cfg["layers"])
    model = Decoder(spec, torch.float32, "cpu")
    load_weights(model, arch.weight_map(parsed), folder)
    assert torch.equal(model.embedding.weight, weights["embed"]) and torch.equal(model.head.weight, weights["head"])
    if "bigram" in cfg["embedding"]:
        assert torch.equal(model.embedding.pairs_weight, weights["bigram"])
        assert model.embedding.state_need()["last_id"].dtype == torch.int32 and model.embedding.reads_step
    else:
        assert model.embedding.state_need() == {} and not model.embedding.reads_step
    if "loop" in cfg:
        assert torch.equal(model.junctions["loop"].weight, weights["loop.in"])
    for i, layer in enumerate(cfg["layers"]):
        block = model.layers[f"l{i}"]
        m, mixer = layer["mixer"], block.mixer
        assert (block.ff is None) == (layer["mlp"] is None)
        if layer["type"] == "mingru":
            n = m["width"]
            for j, t in enumerate(("z", "x", "g")):
                assert torch.equal(mixer.w_in[j * n : (j + 1) * n], weights[f"l{i}.mix.{t}"])
            assert torch.equal(mixer.w_x_bias, weights[f"l{i}.mix.x.b"]) and mixer.state_need()["state"].shape == (n,)
            assert mixer.cache_need() is None
            continue
        (_, left, _), (_, right, _) = mixer.members
        a, b = m["left"], m["right"]
        nq, nk, nv = a["heads"] * a["dim"], a["kv_heads"] * a["dim"], a["kv_heads"] * a["vdim"]
        assert torch.equal(left.w_in[nq : nq + nk], weights[f"l{i}.mix.left.k"])
        assert torch.equal(left.w_in[nq + nk + nv :], weights[f"l{i}.mix.left.g"])
        need = mixer.cache_need()
        mask = a.get("mask") or {}
        assert need.window == mask.get("size") and need.keep == -(-mask.get("keep_first", 0) // 64) * 64
        assert need.n_kv_heads == a["kv_heads"] and need.head_dim >= max(a["dim"], a["vdim"]) and need.head_dim % 16 == 0
        for j, t in enumerate("rkvg"):
            assert torch.equal(right.w_in[j], weights[f"l{i}.mix.right.{t}"])
            assert torch.equal(right.w_mu[j], weights[f"l{i}.mix.right.mu.{t}"])
        assert torch.equal(right.w_mu[4], weights[f"l{i}.mix.right.mu.w"]) and torch.equal(right.w_bonus, weights[f"l{i}.mix.right.u"])
        assert torch.equal(mixer.norms[0], weights[f"l{i}.mix.left.out"]) and torch.equal(mixer.norms[1], weights[f"l{i}.mix.right.out"])
        assert mixer.state_need()["right.state"].shape == (b["heads"], b["dim"], b["dim"])
        assert mixer.state_need()["right.last"].shape == (cfg["width"],)
    from safetensors.torch import save_file

    broken = dict(weights)
    broken.pop("l1.norm1")
    broken["l0.mix.extra"] = torch.zeros(3)
    save_file({k: v.to(torch.bfloat16) for k, v in broken.items()}, os.path.join(folder, "model.safetensors"))
    with pytest.raises(WeightError) as e:
        load_weights(Decoder(spec, torch.float32, "cpu"), arch.weight_map(parsed), folder)
    assert "l1.norm1" in e.value.missing and "l0.mix.extra" in e.value.unexpected


def test_a_folder_of_random_weights(tmp_path):
    """The random-weights mode writes the design's own tensor names and keys, and the folder
    reads back to the same model as data."""
    arch, parsed = parse_config(stated(P.NOD_A, P.NOD_A_RANKS))
    folder = write_random_model(str(tmp_path / "m"), parsed, 3, "bfloat16", 0.1, arch)
    from safetensors import safe_open

    with safe_open(os.path.join(folder, "model.safetensors"), "pt") as f:
        shapes = {k: tuple(f.get_slice(k).get_shape()) for k in f.keys()}
    assert shapes == {k: tuple(v) for k, v in P.tensor_shapes(P.NOD_A, P.NOD_A_RANKS).items()}
    arch2, back = read_config(folder)
    assert arch2.to_spec(back) == arch.to_spec(parsed)


# -- pages that stay behind a window -------------------------------------------------------------------


def test_pages_of_kept_tokens_stay_behind_the_window():
    need = PagedKVNeed(1, 16, window=20, keep=13)
    cache = CacheManager({0: need}, page_size=8, num_pages=12, n_slots=2, allocate=False)
    (g,) = cache.groups
    assert g.kept_pages == 2
    slot = cache.admit()
    pos = 0
    for n in (5, 20, 1, 1, 30, 2, 7, 1, 1, 1, 9):
        cache.reserve([(slot, pos + n)])
        pos += n
        cache.advance(slot, pos)
        cache.check()
        table = g.tables[slot]
        passed = max(pos - 20 + 1, 0) // 8  # pages wholly before the next token's window
        assert [i for i, p in enumerate(table) if p >= 0] == [i for i in range(len(table)) if i < 2 or i >= passed]
        assert g.pool.capacity - g.pool.available <= g.pages_per_token_span(pos) + -(-n // 8)
    other = cache.admit()  # the pages that came back serve another request
    cache.reserve([(other, 30)])
    cache.advance(other, 30)
    cache.check()
    assert not set(p for p in g.tables[slot] if p >= 0) & set(p for p in g.tables[other] if p >= 0)
    cache.free(slot), cache.free(other)
    assert cache.idle()
    assert g.tokens_held_at_most(1000) == (3 + 1 + 2) * 8
    # without a window nothing passes and nothing has to be kept
    assert CacheManager({0: PagedKVNeed(1, 16, keep=13)}, page_size=8, num_pages=4, n_slots=1, allocate=False).groups[0].kept_pages == 0


# -- the plain implementation's own pins -----------------------------------------------------------------


def test_plain_rotation_turns_and_turns_back():
    x = rand(7, 3, 10, seed=1)
    at = [0, 1, 5, 9, 100, 1000, 31]
    y = P.turn(x, at, 6, 50.0, 2.0)
    assert float((y[0] - x[0]).abs().max()) == 0.0 and float((y[..., 6:] - x[..., 6:]).abs().max()) == 0.0
    assert float((P.turn(y, at, 6, 50.0, 2.0, backwards=True) - x).abs().max()) < 1e-12
    # as complex numbers, pair by pair; and a product depends on the distance alone
    z = torch.complex(x[..., :3], x[..., 3:6])
    angle = torch.tensor(at, dtype=F)[:, None] * torch.tensor([50.0 ** (-2 * i / 6) / 2.0 for i in range(3)], dtype=F)
    z = z * torch.polar(torch.ones_like(angle), angle)[:, None, :]
    assert float((y[..., :6] - torch.cat([z.real, z.imag], -1)).abs().max()) < 1e-12
    a, b = x[:1], x[1:2]
    near = (P.turn(a, [12], 10, 50.0) * P.turn(b, [9], 10, 50.0)).sum()
    far = (P.turn(a, [512], 10, 50.0) * P.turn(b, [509], 10, 50.0)).sum()
    assert abs(float(near - far)) < 1e-10


def test_plain_mask():
    m = {"size": 4, "keep_first": 2}
    assert [j for j in range(12) if P.sees(10, j, m)] == [0, 1, 7, 8, 9, 10]
    assert [j for j in range(12) if P.sees(3, j, m)] == [0, 1, 2, 3]
    assert [j for j in range(12) if P.sees(5, j, {"size": 4})] == [2, 3, 4, 5]
    assert [j for j in range(12) if P.sees(5, j, None)] == list(range(6))


def test_plain_attention_by_distance():
    """One key/value head: values arrive turned by their distance, so the whole attention does not
    change when the positions are shifted; checked against the sum written out for one query."""
    T, W = 14, 12
    m = {"heads": 2, "kv_heads": 1, "dim": 6, "vdim": 4, "scale": 0.6, "rot": {"base": 30.0, "dims": 4, "scaling": {"factor": 2.0}},
         "mask": {"size": 5, "keep_first": 2}}
    w = {"q": rand(12, W, seed=1), "k": rand(6, W, seed=2), "v": rand(4, W, seed=3), "g": rand(2, W, seed=4), "o": rand(W, 8, seed=5)}
    h = rand(T, W, seed=6)
    got = P.kept_window_attention(h, w, "", m)
    i, heads = 11, []
    for head in range(2):
        q = (h[i] @ w["q"].T)[head * 6 : head * 6 + 6]
        s, v = [], []
        for j in (0, 1, 7, 8, 9, 10, 11):
            k = P.turn((h[j] @ w["k"].T).view(1, 1, 6), [j - i], 4, 30.0, 2.0)[0, 0]  # only the distance counts
            s.append(float(q @ k) * 0.6)
            v.append(P.turn((h[j] @ w["v"].T).view(1, 1, 4), [j - i], 4, 30.0)[0, 0])
        p = torch.softmax(torch.tensor(s, dtype=F), 0)
        heads.append(sum(pj * vj for pj, vj in zip(p, v)) * torch.sigmoid(h[i] @ w["g"].T)[head])
    assert float((got[i] - torch.cat(heads) @ w["o"].T).abs().max()) < 1e-12


def test_plain_time_mixing_in_two_halves_and_as_sums():
    T, D = 18, 6
    r, k, v = rand(T, D, seed=1), rand(T, D, seed=2), rand(T, D, seed=3)
    decay, u = torch.sigmoid(rand(T, D, seed=4)), rand(D, seed=5)
    S0 = rand(D, D, seed=6)
    o, S = P.wkv_recurrence(r, k, v, decay, u, S0)
    o1, S1 = P.wkv_recurrence(r[:7], k[:7], v[:7], decay[:7], u, S0)
    o2, S2 = P.wkv_recurrence(r[7:], k[7:], v[7:], decay[7:], u, S1)
    assert float((torch.cat([o1, o2]) - o).abs().max()) < 1e-12 and float((S2 - S).abs().max()) < 1e-12
    # as a sum over the earlier tokens with the decays between, and the bonus for the token itself
    o0, _ = P.wkv_recurrence(r, k, v, decay, u, torch.zeros(D, D, dtype=F))
    t = 11
    want = sum((r[t] * torch.prod(decay[j + 1 : t], 0) * k[j]).sum() * v[j] for j in range(t)) + (r[t] * u * k[t]).sum() * v[t]
    assert float((o0[t] - want).abs().max()) < 1e-12
    # the whole mixer with its shifted inputs, cut in two
    cfg, ranks = CONFIGS["A"]
    w = {n: x.to(F) for n, x in P.random_weights(cfg, ranks, 4).items()}
    h, m = rand(15, cfg["width"], seed=1), cfg["layers"][0]["mixer"]["right"]
    y, last, S = P.time_mixing(h, w, "l0.mix.right.", m, 1e-5)
    y1, last1, S1 = P.time_mixing(h[:4], w, "l0.mix.right.", m, 1e-5)
    y2, last2, S2 = P.time_mixing(h[4:], w, "l0.mix.right.", m, 1e-5, before=last1, state=S1)
    assert float((torch.cat([y1, y2]) - y).abs().max()) < 1e-12 and float((S2 - S).abs().max()) < 1e-12
    assert torch.equal(last, h[-1]) and torch.equal(last2, last)
    d = P.wkv_decay(h, w, "l0.mix.right.")
    assert 0.0 <= float(d.min()) and float(d.max()) <= 1.0 and float(d.max() - d.min()) > 0.3


def test_plain_gated_recurrence_and_small_pieces():
    cfg, ranks = CONFIGS["A"]
    w = {n: x.to(F) for n, x in P.random_weights(cfg, ranks, 4).items()}
    h = rand(12, cfg["width"], seed=2)
    y, S = P.mingru(h, w, "l1.mix.")
    y1, S1 = P.mingru(h[:5], w, "l1.mix.")
    y2, S2 = P.mingru(h[5:], w, "l1.mix.", state=S1)
    assert float((torch.cat([y1, y2]) - y).abs().max()) < 1e-12 and float((S2 - S).abs().max()) < 1e-12
    z, c = P.mingru_gates(h, w, "l1.mix.")
    want = sum(torch.prod(1 - z[j + 1 :], 0) * z[j] * c[j] for j in range(12))
    assert float((S - want).abs().max()) < 1e-12 and float(c.min()) > 0.0  # both branches are positive
    x = rand(9, 7, seed=9)
    assert float((P.gelu_tanh(x) - torch.nn.functional.gelu(x, approximate="tanh")).abs().max()) < 1e-12
    assert P.bigram_rows([3, 1, 1, 4], 10, 7, 2) == [10, (21 + 2) % 10, (7 + 2) % 10, (7 + 8) % 10]
    assert float(P.soft_cap(torch.tensor([1e6, -1e6], dtype=F), 5.0).abs().max()) <= 5.0
    assert math.isclose(float(P.soft_cap(torch.tensor(0.01, dtype=F), 5.0)), 0.01, rel_tol=1e-5)
