"""Divuzen without a GPU: the configuration, keys that switch a mechanism off when they are left
out, the table of tensor names and the loader, the model as data (which layer reads whose cache),
the random-weights mode, and the plain implementation's own pins."""

import json
import math
import os

import pytest
import torch

import plain_divuzen as P
from halite_amd.config import parse_config, read_config
from halite_amd.config.registry import ConfigError
from halite_amd.parts import Decoder
from halite_amd.weights import load_weights, write_random_model
from halite_amd.weights.loader import WeightError

CONFIGS = {"A": P.DIV_A, "B": P.DIV_B, "C": P.DIV_C}
F = torch.float64


def rand(*shape, seed=0, scale=1.0):
    return scale * torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=F)


def test_the_model_as_data():
    arch, parsed = parse_config(P.DIV_A)
    assert arch.name == "Divuzen"
    spec = arch.to_spec(parsed)
    assert {l.arrangement for l in spec.layers.values()} == {"hyper_pre_norm"}
    kinds = [l.parts["mixer"].kind for l in spec.layers.values()]
    assert kinds == ["decay_attention", "capped_attention", "capped_attention", "decay_attention"]
    assert [run.cache_from for run in spec.order] == [None, None, 1, None]
    own, borrowing = (spec.layers[n].parts["mixer"].params() for n in ("l1", "l2"))
    assert own["own_kv"] and not borrowing["own_kv"] and own["learned_sink"] and not own["head_gate"]
    assert own["position"] == borrowing["position"] and (own["scale"], borrowing["scale"]) == (0.3, 0.2)
    assert spec.positions[own["position"]].params()["interleaved"] is True
    retention = spec.layers["l0"].parts["mixer"].params()
    assert spec.positions[retention["position"]].params()["interleaved"] is False
    assert len(spec.positions) == 3  # one table a distinct rotation
    assert retention["key_scale"] == 0.25 and retention["activation"] is None and retention["gate"] == "silu"
    assert retention["norm_per_head"] and not retention["norm_weight"]
    ff = spec.layers["l0"].parts["ff"].params()
    assert (ff["activation"], ff["limit"], ff["alpha"], ff["up_shift"]) == ("clamped", 0.8, 1.702, 1.0)
    experts = spec.layers["l1"].parts["ff"].params()
    assert experts["score"] == "sigmoid" and experts["correction"] and experts["weight_scale"] == 1.7
    assert experts["groups"] == {"count": 4, "keep": 2} and experts["norm_eps"] == 1e-20 and experts["shared_gate"]
    assert experts["expert"]["limit"] is None and experts["expert"]["up_shift"] == 0.0
    for part in ("mixer_norm", "mixer_out_norm", "ff_norm", "ff_out_norm"):
        assert spec.layers["l3"].parts[part].params()["weight_offset"] == 1.0
    assert spec.head.params()["tied"] is True and spec.head.params()["logit_scale"] == 0.3


def test_keys_that_are_left_out_switch_their_mechanism_off():
    cfg = json.loads(json.dumps(P.DIV_B))
    del cfg["logit_scale"], cfg["layers"][3]["mlp"]["limit"], cfg["layers"][2]["mlp"]["router"]["scale"]
    arch, parsed = parse_config(cfg)
    spec = arch.to_spec(parsed)
    assert spec.layers["l0"].parts["mixer"].params()["position"] is None and "ff" not in spec.layers["l0"].parts
    assert "ff_out_norm" not in spec.layers["l0"].parts and spec.layers["l1"].parts["mixer"].params()["position"] is None
    assert spec.head.params()["logit_scale"] == 1.0 and spec.layers["l3"].parts["ff"].params()["limit"] is None
    assert spec.layers["l2"].parts["ff"].params()["weight_scale"] == 1.0
    assert spec.layers["l1"].parts["ff"].params()["groups"] is None and spec.layers["l2"].parts["ff"].params()["shared"] is None
    assert [run.cache_from for run in spec.order] == [None, None, 0, None, 0, 3]
    names = arch.weight_map(parsed)
    assert "l2.mix.k" not in names and "l2.mix.v" not in names and "l2.mix.k.norm" not in names and "l2.mix.q.norm" in names
    assert names["l0.norm2"] is None and names["l0.norm2b"] is None and "l2.mlp.shared.sg" not in names
    written = parsed.to_json_dict()
    assert written["layers"][0]["mlp"] is None and written["layers"][2]["mixer"]["kv_from"] == 0


@pytest.mark.parametrize("bad", [
    lambda c: c["layers"][1]["mixer"].update(kv_heads=3),
    lambda c: c["layers"][1]["mixer"].pop("scale"),
    lambda c: c["layers"][1]["mixer"]["rot"].update(dims=7),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=18),
    lambda c: c["layers"][0]["mixer"].update(decay=[0.5]),
    lambda c: c["layers"][2]["mixer"].update(kv_from=0),  # no attention
    lambda c: c["layers"][2]["mixer"].update(kv_from=2),
    lambda c: c["layers"][2]["mixer"].update(kv_from=3),
    lambda c: c["layers"][2]["mixer"].update(dim=8),  # other sizes than the layer it borrows from
    lambda c: c["layers"][2]["mixer"]["rot"].update(base=7.0),
    lambda c: c["layers"][1]["mlp"]["router"].update(top=9),
    lambda c: c["layers"][1]["mlp"]["router"].update(top=5),  # more than the kept groups hold
    lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(count=3),
    lambda c: c["layers"][1]["mlp"]["router"]["groups"].update(keep=5),
    lambda c: c["layers"][0].update(type="recurrent"),
    lambda c: c["layers"][0]["mlp"].update(kind="wide"),
    lambda c: c["layers"][0]["mlp"].update(limit=0.0),
    lambda c: c.update(layers=[]),
    lambda c: c.pop("norm"),
    lambda c: c.update(width=64.5),
])
def test_configurations_that_are_refused(bad):
    cfg = json.loads(json.dumps(P.DIV_A))
    bad(cfg)
    with pytest.raises(ConfigError):
        parse_config(cfg)


def test_a_layer_does_not_borrow_from_one_that_borrows():
    cfg = json.loads(json.dumps(P.DIV_B))
    cfg["layers"][4]["mixer"]["kv_from"] = 2
    with pytest.raises(ConfigError):
        parse_config(cfg)


def test_decays_outside_of_zero_to_one_are_refused():
    cfg = json.loads(json.dumps(P.DIV_A))
    cfg["layers"][0]["mixer"]["decay"] = [0.9, 1.5]
    arch, parsed = parse_config(cfg)
    with pytest.raises(ConfigError):
        Decoder(arch.to_spec(parsed), torch.float32, "cpu")


@pytest.mark.parametrize("name", list(CONFIGS))
def test_the_loader_and_the_tensors(name, tmp_path):
    cfg = CONFIGS[name]
    weights = P.random_weights(cfg, 2)
    folder = P.write_model_folder(str(tmp_path), cfg, weights)
    arch, parsed = read_config(folder)
    model = Decoder(arch.to_spec(parsed), torch.float32, "cpu")
    assert model.stream_copies == 1
    load_weights(model, arch.weight_map(parsed), folder)
    assert torch.equal(model.embedding.weight, weights["embed"]) and model.head.weight is model.embedding.weight
    assert torch.equal(model.final_norm.multiplier, 1.0 + weights["final.norm"])
    for i, layer in enumerate(cfg["layers"]):
        block = model.layers[f"l{i}"]
        m, mixer = layer["mixer"], block.mixer
        assert (block.ff is None) == (layer["mlp"] is None) == (block.ff_out_norm is None)
        assert torch.equal(block.mixer_norm.weight, weights[f"l{i}.norm1"])
        assert torch.equal(block.mixer_out_norm.multiplier, 1.0 + weights[f"l{i}.norm1b"])
        if layer["type"] == "attention":
            nq, nk = m["heads"] * m["dim"], m["kv_heads"] * m["dim"]
            assert torch.equal(mixer.w_in[:nq], weights[f"l{i}.mix.q"])
            assert torch.equal(mixer.rule.sink_values, weights[f"l{i}.mix.sink"]) and mixer.rule.sink and mixer.rule.softcap == 0.0
            if m.get("kv_from") is None:
                assert torch.equal(mixer.w_in[nq : nq + nk], weights[f"l{i}.mix.k"]) and torch.equal(mixer.w_in[nq + nk :], weights[f"l{i}.mix.v"])
                assert torch.equal(mixer.w_k_norm, weights[f"l{i}.mix.k.norm"])
            else:
                assert mixer.w_in.shape[0] == nq
            need = mixer.cache_need()
            assert need.n_kv_heads == m["kv_heads"] and need.head_dim >= max(m["dim"], m["vdim"]) and need.window is None
            assert mixer.state_need() == {}
        else:
            nk, nv = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            assert torch.equal(mixer.w_in[:nv], weights[f"l{i}.mix.v"]) and torch.equal(mixer.w_in[nv + nk : nv + 2 * nk], weights[f"l{i}.mix.q"])
            assert torch.equal(mixer.w_in[nv + 2 * nk :], weights[f"l{i}.mix.g"])
            assert mixer.state_need()["state"].shape == (m["heads"], m["dim"], m["vdim"]) and mixer.cache_need() is None
            assert torch.equal(mixer.decay, torch.tensor(m["decay"]).float()) and mixer.p.key_scale == m["dim"] ** -0.5
            for n in (0, 1, 37, 64):
                assert torch.allclose(mixer.powers[:, n].double(), torch.tensor(m["decay"], dtype=F) ** n, rtol=1e-7)
        f = layer["mlp"]
        if f is not None:
            assert torch.equal(block.ff_out_norm.multiplier, 1.0 + weights[f"l{i}.norm2b"])
            if f["kind"] == "dense":
                assert torch.equal(block.ff.w_gate_up[: f["ff"]], weights[f"l{i}.mlp.gate"]) and block.ff.p.clamp.limit == f["limit"]
                continue
            e = f["router"]["experts"]
            assert torch.equal(block.ff.w_router[:e], weights[f"l{i}.mlp.router"])
            assert torch.equal(block.ff.w_correction, weights[f"l{i}.mlp.correction"])
            assert torch.equal(block.ff.w_gate[e - 1], weights[f"l{i}.mlp.e{e - 1}.gate"])
            if f.get("shared"):
                assert torch.equal(block.ff.w_router[e:], weights[f"l{i}.mlp.shared.sg"])
                assert torch.equal(block.ff.ws_down, weights[f"l{i}.mlp.shared.down"])
    # a tensor that is missing and one that nobody knows are both named
    from safetensors.torch import save_file

    broken = dict(weights)
    broken.pop("l0.norm1b")
    broken["l0.mix.extra"] = torch.zeros(3)
    save_file({k: v.to(torch.bfloat16) for k, v in broken.items()}, os.path.join(folder, "model.safetensors"))
    with pytest.raises(WeightError) as e:
        load_weights(Decoder(arch.to_spec(parsed), torch.float32, "cpu"), arch.weight_map(parsed), folder)
    assert "l0.norm1b" in str(e.value) and "l0.mix.extra" in str(e.value)


def test_a_borrowing_layer_appends_nothing():
    arch, parsed = parse_config(P.DIV_B)
    model = Decoder(arch.to_spec(parsed), torch.float32, "cpu")
    appends = [run.appends for run in model.runs]
    assert appends == [True, True, False, True, False, False]
    assert [model.mixer_of_run(i).p.own_kv for i in (0, 2, 3, 4, 5)] == [True, False, True, False, False]


def test_the_random_weights_mode(tmp_path):
    arch, parsed = parse_config(P.DIV_B)
    folder = write_random_model(str(tmp_path / "m"), parsed, seed=4, dtype="bfloat16", std=0.1)
    arch2, again = read_config(folder)
    assert arch2.to_spec(again) == arch.to_spec(parsed)
    from safetensors.torch import load_file

    assert set(load_file(os.path.join(folder, "model.safetensors"))) == set(P.tensor_shapes(P.DIV_B))
    assert json.load(open(os.path.join(folder, "config.json")))["layers"][0]["mlp"] is None


# -- the plain implementation's own pins -----------------------------------------------------------


def test_the_recurrence_as_sums_and_in_halves():
    T, H, D, V = 13, 2, 5, 7
    q, k, v = rand(T, H, D, seed=1), rand(T, H, D, seed=2), rand(T, H, V, seed=3)
    decay = torch.tensor([0.8, 1.0], dtype=F)
    out, S = P.decayed_state_walk(q, k, v, decay, torch.zeros(H, D, V, dtype=F))
    for t in (0, 6, 12):
        for h in range(H):
            want = sum(decay[h] ** (t - j) * (q[t, h] @ k[j, h]) * v[j, h] for j in range(t + 1))
            assert float((out[t, h] - want).abs().max()) < 1e-12
    first, mid = P.decayed_state_walk(q[:6], k[:6], v[:6], decay, torch.zeros(H, D, V, dtype=F))
    second, end = P.decayed_state_walk(q[6:], k[6:], v[6:], decay, mid)
    assert float((torch.cat([first, second]) - out).abs().max()) < 1e-12 and float((end - S).abs().max()) < 1e-12


def test_the_rotations_are_rotations():
    """Lengths stay, entries behind the turned ones stay, and the product of two turned vectors
    depends on the distance of their positions alone."""
    x, pos = rand(9, 3, 12, seed=1), torch.arange(9)
    r = P.rot(100.0, 8)
    for interleaved in (False, True):
        y = P.rotate(x, pos, r, interleaved)
        assert float((y[..., 8:] - x[..., 8:]).abs().max()) == 0.0 and float((y[0] - x[0]).abs().max()) < 1e-15
        assert float((y.norm(dim=-1) - x.norm(dim=-1)).abs().max()) < 1e-12
        a, b = (P.rotate(x[i : i + 1].expand(9, 3, 12), pos, r, interleaved) for i in (0, 1))
        assert float(((a[5] * b[3]).sum(-1) - (a[8] * b[6]).sum(-1)).abs().max()) < 1e-12
    # halves pair entry i with i + dims/2, neighbours 2i with 2i + 1: one is the other with the entries reordered
    order = [0, 4, 1, 5, 2, 6, 3, 7, 8, 9, 10, 11]
    assert float((P.rotate(x[..., order], pos, r, True) - P.rotate(x, pos, r, False)[..., order]).abs().max()) < 1e-12
    # the second pair turns by base^(-2/dims) a position
    e = torch.zeros(5, 1, 8, dtype=F)
    e[:, 0, 2] = 1.0
    turned = P.rotate(e, torch.arange(5), r, True)
    assert abs(float(turned[3, 0, 3]) - math.sin(3 * 100.0 ** (-2.0 / 8))) < 1e-12


def test_the_sink_is_one_more_term_of_the_denominator():
    s, sink = rand(4, 6, seed=2), torch.tensor(0.7, dtype=F)
    w = P.sink_softmax(s, sink)
    want = torch.exp(s) / (torch.exp(s).sum(-1, keepdim=True) + math.exp(0.7))
    assert float((w - want).abs().max()) < 1e-12
    assert float((P.sink_softmax(s, torch.tensor(-800.0, dtype=F)) - torch.softmax(s, -1)).abs().max()) < 1e-12
    assert float(P.sink_softmax(s, torch.tensor(800.0, dtype=F)).max()) < 1e-200


def test_a_layer_that_borrows_reads_the_other_layers_keys_and_values():
    cfg = P.model_cfg(16, 11, [P.attention_layer(2, 1, 4, 6, 0.7, rot=P.rot(50.0, 4)),
                               P.attention_layer(2, 1, 4, 6, 0.5, rot=P.rot(50.0, 4), kv_from=0)])
    w = {k: v.to(F) for k, v in P.random_weights(cfg, 3, stored=torch.float32).items()}
    a, b = rand(6, 16, seed=2), rand(6, 16, seed=5)
    y, kv = P.sink_attention(a, w, "l0.mix.", cfg["layers"][0]["mixer"], 1e-5)
    borrowed, same = P.sink_attention(b, w, "l1.mix.", cfg["layers"][1]["mixer"], 1e-5, kv)
    assert same is kv
    joined = dict(w, **{f"l1.mix.{n}": w[f"l0.mix.{n}"] for n in ("k", "v", "k.norm")})
    own, _ = P.sink_attention(b, joined, "l1.mix.", cfg["layers"][1]["mixer"], 1e-5)
    assert float((own - borrowed).abs().max()) > 1e-3  # keys of b's rows are others
    own, _ = P.sink_attention(a, joined, "l1.mix.", cfg["layers"][1]["mixer"], 1e-5)
    again, _ = P.sink_attention(a, w, "l1.mix.", cfg["layers"][1]["mixer"], 1e-5, kv)
    assert float((own - again).abs().max()) < 1e-12  # the same rows: the same keys


def test_the_choice_of_experts_by_hand():
    scores = torch.tensor([[0.9, 0.1, 0.6, 0.5, 0.7, 0.65]], dtype=F)
    none = torch.zeros(6, dtype=F)
    pick = lambda c, **r: sorted(P.choose_experts(scores, c, dict(r, experts=6))[0].tolist())  # noqa: E731
    assert pick(none, top=2) == [0, 4]
    # three groups of two: sums 1.0, 1.1, 1.35: the best single expert's group is left out
    assert pick(none, top=2, groups={"count": 3, "keep": 2}) == [4, 5] and pick(none, top=3, groups={"count": 3, "keep": 2}) == [2, 4, 5]
    # two groups of three: the two largest of each count, 1.5 and 1.35
    assert pick(none, top=2, groups={"count": 2, "keep": 1}) == [0, 2]
    # corrections of either sign move the choice; negative choice scores still beat a closed group
    low = torch.tensor([-2.0, -2.0, -2.0, -2.0, -3.0, -3.0], dtype=F)
    assert pick(low, top=3, groups={"count": 3, "keep": 2}) == [0, 2, 3]
    margins = []
    P.choose_experts(scores, none, {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 2}}, margins)
    assert abs(float(margins[0]) - 0.05) < 1e-12  # 0.65 against 0.6; the groups are 0.1 apart
    margins = []
    P.choose_experts(scores, none, {"experts": 6, "top": 4, "groups": {"count": 3, "keep": 2}}, margins)
    assert abs(float(margins[0]) - 0.1) < 1e-12


def test_the_experts_weights_and_the_clamped_gate():
    cfg = P.model_cfg(12, 9, [P.retention_layer(1, 4, 4, [0.9], mlp=P.moe(4, 2, 6, scale=1.5, shared=5))])
    w = {k: v.to(F) for k, v in P.random_weights(cfg, 7, stored=torch.float32).items()}
    h = rand(5, 12, seed=1)
    f = cfg["layers"][0]["mlp"]
    out = P.routed_experts(h, w, "l0.mlp.", f)
    s = torch.sigmoid(h @ w["l0.mlp.router"].T)
    for t in range(5):
        a, b = torch.topk(s[t] + w["l0.mlp.correction"], 2).indices.tolist()
        want = torch.sigmoid(h[t] @ w["l0.mlp.shared.sg"][0]) * P.gated_expert(h[t : t + 1], w, "l0.mlp.shared.")[0]
        for e in (a, b):
            want = want + 1.5 * s[t, e] / (s[t, a] + s[t, b]) * P.gated_expert(h[t : t + 1], w, f"l0.mlp.e{e}.")[0]
        assert float((out[t] - want).abs().max()) < 1e-12
    one = {"g.gate": torch.tensor([[4.0], [-9.0], [1.0]], dtype=F), "g.up": torch.tensor([[9.0], [-9.0], [0.5]], dtype=F),
           "g.down": torch.eye(3, dtype=F)}
    y = P.clamped_dense(torch.ones(1, 1, dtype=F), one, "g.", {"limit": 2.0})[0]
    sig = lambda z: 1.0 / (1.0 + math.exp(-z))  # noqa: E731
    want = [2.0 * sig(3.404) * 3.0, -9.0 * sig(-9.0 * 1.702) * -1.0, sig(1.702) * 1.5]  # the gate is not held below
    assert float((y - torch.tensor(want, dtype=F)).abs().max()) < 1e-12


@pytest.mark.parametrize("name", list(CONFIGS))
def test_every_mechanism_changes_the_logits(name):
    """Leaving out a sink, a correction, the groups, a limit, a rotation or a norm's distance from one moves the
    plain model's logits by far more than the tests' tolerance, so a fault in any of them shows."""
    cfg = CONFIGS[name]
    w = P.random_weights(cfg, 5)
    ids = torch.randint(0, cfg["vocab"], (40,), generator=torch.Generator().manual_seed(1)).tolist()
    ref = P.forward(cfg, w, ids)
    changed = {}
    for key, new in (("sink", -60.0), ("correction", 0.0), ("norm1b", 0.0), ("norm2b", 0.0), ("norm1", 0.0), ("q.norm", 1.0)):
        names = [n for n in w if n.endswith("." + key)]
        changed[key] = (cfg, dict(w, **{n: torch.full_like(w[n], new) for n in names}))
    for key in ("groups", "limit", "rot"):
        other = json.loads(json.dumps(cfg))
        for layer in other["layers"]:
            f = layer["mlp"] or {}
            if key == "groups":
                f.get("router", {}).pop("groups", None)
            elif key == "limit" and "limit" in f:
                f["limit"] = 1e9
            elif key == "rot":
                layer["mixer"].pop("rot", None)
        changed[key] = (other, w)
    for key, (c, ww) in changed.items():
        moved = float((P.forward(c, ww, ids) - ref).abs().max()) / float(ref.abs().max())
        assert moved > 0.02, (key, moved)
