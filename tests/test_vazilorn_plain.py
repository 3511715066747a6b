"""Vazilorn on the CPU: the configuration reader and its refusals, the plan (which parts with which constants), tensor names
and shapes, cache needs, and the plain implementation's own invariants (the norm's element-wise form, frequencies stretched by
bands at and between their edges, rotation by distance, window edges, the sink's share, the router's groups by their two best
among negative choices, the shared expert, prefixes)."""
import json
import math

import pytest
import torch

import alice_llm_amd as alice
from alice_llm_amd.engine.model import CausalLM
from alice_llm_amd.parts import FEED_FORWARDS, MIXERS, NORMS, POSITIONS, Precision
from helpers import VAZILORN, random_tokens, vazilorn_tensors
from plain import vazilorn_plain as P


def rnd(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64) * scale


# ------------------------------------------------------------------ configuration and plan

def test_architecture_is_found_by_its_key_and_round_trips():
    for make in VAZILORN.values():
        cfg = alice.config_from_dict(make())
        assert type(cfg).__name__ == "VazilornConfig"
        assert alice.config_from_dict(json.loads(json.dumps(cfg.to_dict()))) == cfg
    assert "Vazilorn" in alice.registered_architectures()
    plan = alice.config_from_dict(VAZILORN["vz-a"]()).plan()
    assert [(e.layer, e.cache_from) for e in plan.schedule] == [(i, None) for i in range(4)]
    assert [l.mixer.kind for l in plan.layers] == ["attention"] * 4 and all(l.block == "sandwich" for l in plan.layers)
    assert [None if l.feed_forward is None else l.feed_forward.kind for l in plan.layers] == ["gated_mlp", "expert_mlp", None, "expert_mlp"]
    assert all(set(l.norms) == ({"pre_mixer", "post_mixer"} | ({"pre_ff", "post_ff"} if l.feed_forward else set())) for l in plan.layers)
    assert all(n.kind == "dynamic_tanh" for l in plan.layers for n in l.norms.values()) and plan.final_norm.kind == "dynamic_tanh"
    a = plan.layers[0].mixer.args
    assert (a["num_heads"], a["num_kv_heads"], a["head_dim"], a["value_head_dim"], a["scale"], a["window"]) == (4, 2, 16, 24, 0.5, 9)
    assert a["sink"] is True and a["qk_norm"] == "head" and a["qk_norm_eps"] == 1e-6 and plan.layers[3].mixer.args["window"] == 30
    assert len(plan.positions) == 1
    rot = next(iter(plan.positions.values())).args
    assert rot["interleaved"] is True and rot["rotary_dim"] == 8 and rot["dim"] == 16 and rot["theta"] == 100.0
    assert rot["scaling"] == {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 16.0}
    ex = plan.layers[1].feed_forward.args
    assert (ex["experts"], ex["top"], ex["intermediate_size"], ex["groups"], ex["weight_scale"]) == (6, 2, 24, (2, 1), 1.7)
    assert ex["shared"] == {"intermediate_size": 40, "activation": "silu"} and ex["scoring"] == "sigmoid" and ex["group_best"] == 2
    assert ex["shared_gate"] is False and ex["activation"] == "silu" and plan.layers[0].feed_forward.args["activation"] == "gelu_tanh"
    assert len(alice.config_from_dict(VAZILORN["vz-c"]()).plan().positions) == 3


def test_defaults_and_absent_keys():
    plan = alice.config_from_dict(VAZILORN["vz-b"]()).plan()
    ex = plan.layers[0].feed_forward.args
    assert ex["groups"] is None and ex["shared"] is None and ex["weight_scale"] == 0.8 and plan.layers[0].mixer.args["qk_norm_eps"] == 1e-4
    assert all(p.args["scaling"] is None for p in plan.positions.values())
    raw = VAZILORN["vz-b"]()
    del raw["norm"], raw["layers"][0]["mixer"]["vdim"], raw["layers"][0]["mixer"]["rot"]["dims"], raw["layers"][0]["mixer"]["kv_heads"]
    del raw["layers"][0]["mlp"]["router"]["scale"], raw["layers"][0]["mixer"]["mask"], raw["layers"][1]["mixer"]["rot"], raw["layers"][1]["mlp"]
    cfg = alice.config_from_dict(raw)
    m = cfg.layers[0]["mixer"]
    assert cfg.norm_eps == 1e-6 and m["vdim"] == 20 and m["rot"]["dims"] == 20 and m["kv_heads"] == 3
    plan = cfg.plan()
    assert plan.layers[0].mixer.args["window"] is None and plan.layers[1].mixer.args["position"] is None and plan.layers[1].feed_forward is None
    assert plan.layers[0].feed_forward.args["weight_scale"] == 1.0 and len(plan.positions) == 1


@pytest.mark.parametrize("change,match", [
    (lambda r: r["layers"][0]["mixer"].update(kv_heads=3), "kv_heads"),
    (lambda r: r["layers"][0]["mixer"].update(mask={"size": 0}), "mask.size"),
    (lambda r: r["layers"][0]["mixer"]["rot"].update(dims=7), "rot"),
    (lambda r: r["layers"][0]["mixer"]["rot"].update(dims=18), "rot"),
    (lambda r: r["layers"][0]["mixer"]["rot"]["scaling"].update(low=5.0), "scaling"),
    (lambda r: r["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0.0), "scaling"),
    (lambda r: r["layers"][0]["mixer"]["rot"]["scaling"].pop("original"), "original"),
    (lambda r: r["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda r: r["layers"][1]["mlp"]["router"].update(top=7), "top"),
    (lambda r: r["layers"][1]["mlp"]["router"].update(scale=0.0), "scale"),
    (lambda r: r["layers"][1]["mlp"]["router"].update(groups={"count": 4, "keep": 1}), "groups"),
    (lambda r: r["layers"][1]["mlp"]["router"].update(groups={"count": 6, "keep": 1}), "groups"),
    (lambda r: r["layers"][1]["mlp"]["shared"].update(ff=0), "ff"),
    (lambda r: r["layers"][2].update(type="conv"), "no mixer"),
    (lambda r: r["layers"][0]["mlp"].update(kind="sparse"), "no feed-forward"),
    (lambda r: r["norm"].update(eps=0.0), "eps"),
])
def test_refusals(change, match):
    raw = json.loads(json.dumps(VAZILORN["vz-a"]()))             # (no part of it shared between layers)
    change(raw)
    with pytest.raises(alice.ConfigError, match=match):
        alice.config_from_dict(raw)


def test_refusals_of_the_parts():
    p = Precision.of("float32")
    ff = FEED_FORWARDS.get("expert_mlp")
    with pytest.raises(ValueError, match="scoring"):
        ff(p, hidden_size=8, intermediate_size=8, experts=2, top=1, weight_scale=2.0)
    with pytest.raises(ValueError, match="group_best"):
        ff(p, hidden_size=8, intermediate_size=8, experts=4, top=1, scoring="sigmoid", group_best=3)
    with pytest.raises(ValueError, match="qk_norm"):
        MIXERS.get("attention")(p, {"none": object()}, hidden_size=8, num_heads=2, num_kv_heads=2, head_dim=4, scale=1.0, qk_norm="row")
    turned = POSITIONS.get("rope_pairs")(p, "cpu", dim=4, theta=10.0, max_positions=8, value_dim=4)
    with pytest.raises(ValueError, match="values"):
        MIXERS.get("attention")(p, {"t": turned}, hidden_size=8, num_heads=2, num_kv_heads=2, head_dim=4, scale=1.0, qk_norm="head", position="t")
    with pytest.raises(ValueError, match="bands"):
        POSITIONS.get("rope_pairs")(p, "cpu", dim=4, theta=10.0, max_positions=8, scaling={"factor": 2.0, "low": 4.0, "high": 1.0, "original": 8})


def test_tensor_names_shapes_and_cache_needs():
    cfg = alice.config_from_dict(VAZILORN["vz-a"]())
    lm = CausalLM(cfg.plan(), Precision.of("float32"), "cpu")
    specs = {k: tuple(v.shape) for k, v in lm.param_specs().items()}
    want = {"embed": (97, 64), "head": (97, 64), "final.norm": (64,), "final.norm.b": (64,), "final.norm.alpha": (), "l0.norm1": (64,),
            "l0.norm1.b": (64,), "l0.norm1.alpha": (), "l0.norm1b": (64,), "l0.norm1b.alpha": (), "l0.norm2b.b": (64,), "l2.norm1b.b": (64,),
            "l0.mix.q": (64, 64), "l0.mix.k": (32, 64), "l0.mix.v": (48, 64), "l0.mix.q.norm": (16,), "l0.mix.k.norm": (16,), "l0.mix.sink": (4,),
            "l0.mix.o": (64, 96), "l0.mlp.gate": (96, 64), "l0.mlp.up": (96, 64), "l0.mlp.down": (64, 96), "l1.mlp.router": (6, 64),
            "l1.mlp.correction": (6,), "l1.mlp.e5.gate": (24, 64), "l1.mlp.e0.up": (24, 64), "l1.mlp.e0.down": (64, 24),
            "l1.mlp.shared.gate": (40, 64), "l1.mlp.shared.up": (40, 64), "l1.mlp.shared.down": (64, 40), "l3.mlp.e4.down": (64, 16)}
    for name, shape in want.items():
        assert specs.get(name) == shape, (name, specs.get(name))
    for absent in ("l2.norm2", "l2.norm2b", "l2.mlp.up", "l1.mlp.e6.up", "l1.mlp.router.b", "l1.mlp.shared.sg", "l3.mlp.shared.up", "l0.mix.q.b"):
        assert absent not in specs, absent
    needs = lm.cache_needs()
    assert [(n.kv.num_kv_heads, n.kv.head_dim, n.kv.v_dim, n.kv.window) for n in needs] == [(2, 16, 24, 9)] * 3 + [(2, 16, 24, 30)]
    assert not any(n.state for n in needs) and lm.graph_safe() and lm.prompt_graph_safe()
    for name, make in VAZILORN.items():
        cfg, tensors = vazilorn_tensors(make(), 1)
        assert set(tensors) == set(CausalLM(cfg.plan(), Precision.of("bfloat16"), "cpu").param_specs()), name


def test_random_folder_holds_every_tensor_and_runs(tmp_path):
    """The random-weights mode: names, shapes (a number without dimensions too), norm weights around one, logits of order one."""
    raw = VAZILORN["vz-a"]()
    alice.write_random_model(str(tmp_path), dict(raw), seed=3)
    plain = P.PlainVazilorn.from_folder(str(tmp_path))
    specs = CausalLM(alice.config_from_dict(raw).plan(), Precision.of("float32"), "cpu").param_specs()
    assert {k: tuple(v.shape) for k, v in plain.tensors.items()} == {k: tuple(v.shape) for k, v in specs.items()}
    assert abs(float(plain.tensors["l0.norm1"].mean()) - 1.0) < 0.1 and 0.2 < float(plain.tensors["l0.norm1.alpha"]) < 0.8
    assert abs(float(plain.tensors["l0.mix.q.norm"].mean()) - 1.0) < 0.2 and float(plain.tensors["embed"].std()) > 0.8
    logits = plain.forward(random_tokens(97, 12, 1))
    assert bool(torch.isfinite(logits).all()) and float(logits.std()) > 0.01


# ------------------------------------------------------------------ the plain implementation's own invariants

def test_dynamic_tanh_acts_on_every_element_by_itself():
    x, w, b = rnd(3, 20, seed=1, scale=3.0), rnd(20, seed=2), rnd(20, seed=3)
    y = P.dynamic_tanh(x, 0.4, w, b)
    assert abs(float(y[1, 7]) - (math.tanh(0.4 * float(x[1, 7])) * float(w[7]) + float(b[7]))) < 1e-12
    x2 = x.clone()
    x2[:, 3] = 50.0
    assert torch.equal(P.dynamic_tanh(x2, 0.4, w, b)[:, 4:], y[:, 4:])
    norm = NORMS.get("dynamic_tanh")(Precision.of("float32"), dim=20)
    assert set(norm.param_specs()) == {"weight", "bias", "alpha"}
    norm.assign("alpha", torch.tensor(0.4, dtype=torch.bfloat16))
    assert norm.alpha == float(torch.tensor(0.4, dtype=torch.bfloat16))


def test_frequencies_stretched_by_bands():
    f = P.banded_frequencies(16, 100.0, None)
    assert torch.allclose(f, 100.0 ** (-torch.arange(8, dtype=torch.float64) / 8))
    sc = {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 64}
    g = P.banded_frequencies(16, 100.0, sc)
    turns = 64 * f / (2 * math.pi)
    assert bool((turns > 4).any()) and bool((turns < 1).any()) and bool(((turns > 1) & (turns < 4)).any())
    for fi, gi, t in zip(f.tolist(), g.tolist(), turns.tolist()):
        want = fi if t > 4 else fi / 4 if t < 1 else fi / 4 + (fi - fi / 4) * (t - 1) / 3
        assert abs(gi - want) < 1e-14
    for name in VAZILORN:                                        # the product's tables hold the same angles
        for spec in alice.config_from_dict(VAZILORN[name]()).plan().positions.values():
            a = dict(spec.args, max_positions=50)
            part = POSITIONS.get("rope_pairs")(Precision.of("float32"), "cpu", **a)
            ang = torch.arange(50).double()[:, None] * P.banded_frequencies(a["rotary_dim"], a["theta"], a["scaling"])[None]
            assert float((part.cos - torch.cos(ang)).abs().max()) < 1e-6 and float((part.sin - torch.sin(ang)).abs().max()) < 1e-6


def test_turning_depends_on_the_distance_only_and_leaves_the_rest():
    f = P.banded_frequencies(6, 50.0, {"factor": 2.0, "low": 1.0, "high": 2.0, "original": 30})
    q, k = rnd(1, 1, 10, seed=1).expand(9, 1, 10), rnd(1, 1, 10, seed=2).expand(9, 1, 10)
    pos = torch.arange(9)
    qt = P.turn_pairs(q, pos, f)
    assert torch.equal(qt[..., 6:], q[..., 6:]) and not torch.allclose(qt[3], q[3])
    s = qt[:, 0] @ P.turn_pairs(k, pos, f)[:, 0].T
    for lag in range(-8, 9):
        d = torch.diagonal(s, lag)
        assert float((d - d[0]).abs().max()) < 1e-12


def test_window_edges():
    m = P.window_mask(torch.arange(12), 12, 5)
    assert m[7].nonzero()[:, 0].tolist() == [3, 4, 5, 6, 7] and m[2].nonzero()[:, 0].tolist() == [0, 1, 2]
    assert m[0].tolist() == [True] + [False] * 11
    assert bool(P.window_mask(torch.arange(3), 3, 1).equal(torch.eye(3, dtype=torch.bool)))


def test_sink_takes_its_share_once():
    s = torch.tensor([[1.0, 2.0, 0.5]], dtype=torch.float64)
    w = P.sink_softmax(s, torch.tensor([[True, True, False]]), torch.tensor(1.5, dtype=torch.float64))
    den = math.exp(1.0) + math.exp(2.0) + math.exp(1.5)
    assert torch.allclose(w, torch.tensor([[math.exp(1.0) / den, math.exp(2.0) / den, 0.0]], dtype=torch.float64))
    big = P.sink_softmax(s + 700.0, torch.ones(1, 3, dtype=torch.bool), torch.tensor(-700.0, dtype=torch.float64))
    assert abs(float(big.sum()) - 1.0) < 1e-12


def test_router_scores_groups_and_weights():
    z = torch.tensor([[2.0, -1.0, 1.4, 1.3, -3.0, 0.2]], dtype=torch.float64)
    s = torch.sigmoid(z)[0]
    none = torch.zeros(6, dtype=torch.float64)
    w = P.route(z, none, {"experts": 6, "top": 2, "scale": 2.5})[0]
    assert torch.nonzero(w)[:, 0].tolist() == [0, 2] and abs(float(w.sum()) - 2.5) < 1e-12 and abs(float(w[0] / w[2] - s[0] / s[2])) < 1e-12
    # three groups of two: (0, 1) holds the largest choice, (2, 3) the largest sum of two
    w = P.route(z, none, {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 1}})[0]
    assert torch.nonzero(w)[:, 0].tolist() == [2, 3]
    # the correction moves the choice, not the weights; all choices are negative and masked ones still lose
    corr = torch.tensor([-9.0, -2.0, -2.0, -3.0, -1.5, -2.0], dtype=torch.float64)
    w = P.route(z, corr, {"experts": 6, "top": 2})[0]
    assert torch.nonzero(w)[:, 0].tolist() == [2, 5]
    chosen = torch.nonzero(w)[:, 0]
    assert torch.allclose(w[chosen], s[chosen] / s[chosen].sum())
    w = P.route(z, none - 5.0, {"experts": 6, "top": 3, "groups": {"count": 3, "keep": 2}})[0]
    assert torch.nonzero(w)[:, 0].tolist() == [0, 2, 3]
    # groups of one expert: its own choice is the group's
    w = P.route(z, none, {"experts": 6, "top": 2, "groups": {"count": 6, "keep": 3}})[0]
    assert torch.nonzero(w)[:, 0].tolist() == [0, 2]


def test_shared_expert_is_added_as_it_is():
    W, F = 8, 6
    mlp = {"kind": "moe", "expert": {"ff": F}, "router": {"experts": 1, "top": 1, "scale": 3.0}, "shared": {"ff": F}}
    p = {f"{n}.{m}": rnd(*((W, F) if m == "down" else (F, W)), seed=i * 3 + j) for i, n in enumerate(("e0", "shared"))
         for j, m in enumerate(("gate", "up", "down"))}
    p["router"], p["correction"] = rnd(1, W, seed=7), torch.zeros(1, dtype=torch.float64)
    h = rnd(3, W, seed=9)
    part = lambda n: P.gated_ff(h, p[n + ".gate"], p[n + ".up"], p[n + ".down"], P.silu)
    assert torch.allclose(P.routed_ff(h, p, mlp), 3.0 * part("e0") + part("shared"))


def test_prefixes_and_what_the_weights_touch():
    """A prefix's logits do not depend on what follows; a token out of every window's reach changes nothing; the sinks matter."""
    raw = VAZILORN["vz-a"]()
    _, t = vazilorn_tensors(raw, 3)
    t = {k: v.double() for k, v in t.items()}
    toks = random_tokens(raw["vocab"], 70, 4)
    full = P.forward(raw, t, toks)
    for n in (1, 2, 17):
        assert torch.allclose(P.forward(raw, t, toks[:n]), full[:n], atol=1e-9)
    reach = sum(l["mixer"]["mask"]["size"] - 1 for l in raw["layers"])
    other = [(toks[0] + 1) % 97] + toks[1:]
    moved = (P.forward(raw, t, other) - full).abs().amax(-1)
    assert float(moved[reach + 1:].max()) < 1e-12 and float(moved[:20].min()) > 1e-9
    t2 = dict(t)
    t2["l3.mix.sink"] = t["l3.mix.sink"] + 1.0
    assert float((P.forward(raw, t2, toks) - full).abs().max()) > 1e-2
