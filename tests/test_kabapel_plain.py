"""Kabapel on the CPU: the configuration reader and its refusals, the plan (which parts with which constants, which run
reads whose cache), tensor names and shapes, cache needs, and the plain implementation's own invariants (a recurrence
cut in two, its chunk form, stretched frequencies, the latent attention with the per-head maps on the query's side, the
router's choice among negative scores, identity and shared experts, rows read from another layer)."""
import json
import math

import pytest
import torch

import alice_llm_amd as alice
from alice_llm_amd.engine.model import CausalLM
from alice_llm_amd.parts import FEED_FORWARDS, MIXERS, Precision
from helpers import KABAPEL, kabapel_tensors, random_tokens
from plain import kabapel_plain as P


def rnd(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64) * scale


# ------------------------------------------------------------------ configuration and plan

def test_architecture_is_found_by_its_key_and_round_trips():
    for make in KABAPEL.values():
        cfg = alice.config_from_dict(make())
        assert type(cfg).__name__ == "KabapelConfig"
        assert alice.config_from_dict(json.loads(json.dumps(cfg.to_dict()))) == cfg
    assert "Kabapel" in alice.registered_architectures()
    plan = alice.config_from_dict(KABAPEL["kb-a"]()).plan()
    assert [(e.layer, e.cache_from) for e in plan.schedule] == [(0, None), (1, None), (2, None), (3, 1)]
    assert [l.mixer.kind for l in plan.layers] == ["lightning", "latent_attention", "lightning", "latent_attention"]
    assert [None if l.feed_forward is None else l.feed_forward.kind for l in plan.layers] == ["dense_mlp", "expert_mlp", None, "expert_mlp"]
    assert all(set(l.norms) == ({"pre_mixer", "pre_ff"} if l.feed_forward else {"pre_mixer"}) for l in plan.layers)
    assert all(n.kind == "layernorm" and n.args["eps"] == 1e-6 for l in plan.layers for n in l.norms.values())
    assert plan.final_norm.kind == "layernorm" and plan.embedding.args["scale"] == 3.0
    own, other = plan.layers[1].mixer.args, plan.layers[3].mixer.args
    assert own["own_rows"] and not other["own_rows"] and own["position"] == other["position"] and len(plan.positions) == 1
    assert (own["kv_rank"], own["scale"], other["scale"], other["num_heads"]) == (40, 0.3, 0.25, 3)
    rot = next(iter(plan.positions.values())).args
    assert rot["interleaved"] is False and rot["rotary_dim"] == 8 and rot["dim"] == 8 and rot["scaling"]["factor"] == 4.0
    assert plan.layers[0].mixer.args["decay"] == (0.4, 0.8, 0.97, 0.999)
    ex = plan.layers[1].feed_forward.args
    assert (ex["experts"], ex["top"], ex["intermediate_size"], ex["limit"], ex["identity"], ex["groups"]) == (6, 2, 24, 1.1, 2, (2, 1))
    assert ex["shared"] == {"intermediate_size": 40, "activation": "swish_limited", "limit": 0.8} and ex["scoring"] == "all"


def test_defaults_and_absent_keys():
    plan = alice.config_from_dict(KABAPEL["kb-b"]()).plan()
    ex = plan.layers[0].feed_forward.args
    assert ex["groups"] is None and ex["shared"] is None and ex["identity"] == 0
    assert next(iter(plan.positions.values())).args["scaling"] is None
    raw = KABAPEL["kb-b"]()
    del raw["norm"], raw["embedding"], raw["layers"][0]["mixer"]["vdim"], raw["layers"][0]["mixer"]["rot"]["dims"]
    raw["layers"][1]["mlp"].pop("kind")
    cfg = alice.config_from_dict(raw)
    assert cfg.norm_eps == 1e-6 and cfg.embedding_scale == 1.0 and cfg.layers[0]["mixer"]["vdim"] == 20
    assert cfg.layers[0]["mixer"]["rot"]["dims"] == 6 and cfg.layers[1]["mlp"]["kind"] == "dense"
    free = alice.config_from_dict(KABAPEL["kb-d"]()).plan()
    assert free.layers[2].mixer.args["position"] is None and len(free.positions) == 1


@pytest.mark.parametrize("change,match", [
    (lambda r: r["layers"][0]["mixer"].update(decay=[0.5]), "decay"),
    (lambda r: r["layers"][0]["mixer"].update(decay=0.5), "decay"),
    (lambda r: r["layers"][0]["mixer"].pop("decay"), "decay"),
    (lambda r: r["layers"][3]["mixer"].update(kv_from=0), "kv_from"),
    (lambda r: r["layers"][3]["mixer"].update(kv_from=3), "kv_from"),
    (lambda r: r["layers"][3]["mixer"].update(kv_rank=32), "kv_from"),
    (lambda r: r["layers"][3]["mixer"]["rot"].update(base=99.0), "kv_from"),
    (lambda r: r["layers"][1]["mixer"].update(rot_dim=7), "rot"),
    (lambda r: r["layers"][1]["mixer"]["rot"].update(dims=4), "rot"),
    (lambda r: r["layers"][1]["mixer"].pop("rot"), "rot"),
    (lambda r: r["layers"][1]["mixer"]["rot"]["scaling"].update(slow=0.0), "scaling"),
    (lambda r: r["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda r: r["layers"][1]["mlp"]["router"].update(top=9), "top"),
    (lambda r: r["layers"][1]["mlp"]["router"].update(groups={"count": 3, "keep": 1}), "groups"),
    (lambda r: r["layers"][1]["mlp"]["router"].update(groups={"count": 8, "keep": 1}), "groups"),
    (lambda r: r["layers"][1]["mlp"]["expert"].update(limit=0.0), "limit"),
    (lambda r: r["layers"][1]["mlp"]["shared"].pop("limit"), "limit"),
    (lambda r: r["layers"][2].update(type="conv"), "no mixer"),
    (lambda r: r["layers"][0]["mlp"].update(kind="sparse"), "no feed-forward"),
])
def test_refusals(change, match):
    raw = json.loads(json.dumps(KABAPEL["kb-a"]()))             # (no part of it shared between layers)
    change(raw)
    with pytest.raises(alice.ConfigError, match=match):
        alice.config_from_dict(raw)


def test_refusals_of_the_parts():
    p = Precision.of("float32")
    ff = FEED_FORWARDS.get("expert_mlp")
    with pytest.raises(ValueError, match="limit"):
        ff(p, hidden_size=8, intermediate_size=8, experts=2, top=1, activation="swish_limited")
    with pytest.raises(ValueError, match="scoring"):
        ff(p, hidden_size=8, intermediate_size=8, experts=2, top=1, identity=1)
    with pytest.raises(ValueError, match="groups"):
        ff(p, hidden_size=8, intermediate_size=8, experts=4, top=3, scoring="all", groups=(2, 1))
    with pytest.raises(ValueError, match="decays"):
        MIXERS.get("lightning")(p, {}, hidden_size=8, num_heads=2, head_dim=4, decay=[0.5])
    with pytest.raises(ValueError, match="another's rows"):
        MIXERS.get("latent_attention")(p, {}, hidden_size=8, num_heads=2, head_dim=4, rot_dim=0, value_head_dim=4, q_rank=4, kv_rank=8,
                                       scale=1.0, norm_eps=1e-6, own_rows=False)


def test_tensor_names_shapes_and_cache_needs():
    cfg = alice.config_from_dict(KABAPEL["kb-a"]())
    lm = CausalLM(cfg.plan(), Precision.of("float32"), "cpu")
    specs = {k: tuple(v.shape) for k, v in lm.param_specs().items()}
    want = {"embed": (97, 64), "head": (97, 64), "final.norm": (64,), "final.norm.b": (64,), "l0.norm1": (64,), "l0.norm1.b": (64,),
            "l0.norm2.b": (64,), "l0.mix.q": (64, 64), "l0.mix.k": (64, 64), "l0.mix.v": (96, 64), "l0.mix.g": (96, 64), "l0.mix.o": (64, 96),
            "l0.mix.norm": (96,), "l0.mlp.up": (96, 64), "l0.mlp.down": (64, 96), "l1.mix.q": (96, 64), "l1.mix.dkv": (48, 64),
            "l1.mix.dkv.norm": (40,), "l1.mix.uk": (64, 40), "l1.mix.uv": (96, 40), "l1.mix.o": (64, 96), "l1.mlp.router": (8, 64),
            "l1.mlp.correction": (8,), "l1.mlp.e5.gate": (24, 64), "l1.mlp.e0.up": (24, 64), "l1.mlp.e0.down": (64, 24),
            "l1.mlp.shared.gate": (40, 64), "l1.mlp.shared.up": (40, 64), "l1.mlp.shared.down": (64, 40), "l1.mlp.shared.sg": (1, 64),
            "l3.mix.q": (96, 64), "l3.mix.uk": (72, 40), "l3.mix.uv": (48, 40), "l3.mix.o": (64, 48)}
    for name, shape in want.items():
        assert specs.get(name) == shape, (name, specs.get(name))
    for absent in ("l2.norm2", "l2.mlp.up", "l3.mix.dkv", "l3.mix.dkv.norm", "l1.mlp.e6.up", "l1.mlp.router.b", "l0.mlp.gate", "l1.mix.dq", "l1.mix.uq"):
        assert absent not in specs, absent
    needs = lm.cache_needs()
    assert needs[3] is None and (needs[1].kv.num_kv_heads, needs[1].kv.head_dim, needs[1].kv.v_dim, needs[1].kv.window) == (1, 48, 0, None)
    assert [s.shape for s in needs[0].state] == [(4, 16, 24)] and needs[0].kv is None and not needs[1].state
    assert lm.graph_safe() and lm.prompt_graph_safe()


def test_every_tensor_is_wanted_once_by_the_loader(tmp_path):
    """Random folders are written and listed by the same names on every configuration."""
    for name, make in KABAPEL.items():
        cfg, tensors = kabapel_tensors(make(), 1)
        assert set(tensors) == set(CausalLM(cfg.plan(), Precision.of("bfloat16"), "cpu").param_specs()), name


def test_halves_are_put_in_pair_order_with_the_same_scores():
    """The rows of the rotated parts are reordered at load: q . k over them is what it was, for both kinds of rows."""
    p = Precision.of("float32")
    cfg = alice.config_from_dict(KABAPEL["kb-a"]())
    lm = CausalLM(cfg.plan(), p, "cpu")
    mix = lm.layers[1].mixer
    w = rnd(4 * 24, 64, seed=1).float()
    moved = mix._pair_order(w, 4, 16).view(4, 24, 64)
    assert torch.equal(moved[:, :16], w.view(4, 24, 64)[:, :16])
    assert torch.equal(moved[:, 16::2], w.view(4, 24, 64)[:, 16:20]) and torch.equal(moved[:, 17::2], w.view(4, 24, 64)[:, 20:])


# ------------------------------------------------------------------ the plain implementation's own invariants

def test_layer_norm_takes_mean_and_scale_off():
    x = rnd(5, 64, seed=1, scale=3.0) + 7.0
    w, b = rnd(64, seed=2), rnd(64, seed=3)
    y = P.layer_norm(x, w, b, 1e-12)
    ref = torch.nn.functional.layer_norm(x, (64,), w, b, 1e-12)
    assert torch.allclose(y, ref, atol=1e-12)
    assert torch.allclose(P.layer_norm(x + 100.0, w, b, 1e-9), P.layer_norm(x, w, b, 1e-9), atol=1e-9)


def test_stretched_frequencies():
    f, m = P.stretched_frequencies(16, 100.0, None)
    assert m == 1.0 and torch.allclose(f, 100.0 ** (-torch.arange(8, dtype=torch.float64) / 8))
    g, m = P.stretched_frequencies(16, 100.0, {"factor": 4.0, "original": 16, "fast": 8.0, "slow": 1.0})
    assert m == 0.1 * math.log(4.0) + 1.0 and float(g[0]) == 1.0 and abs(float(g[-1] / f[-1]) - 0.25) < 1e-12
    assert all(0.25 - 1e-12 <= float(r) <= 1.0 + 1e-12 for r in g / f) and bool((g[1:] < g[:-1]).all())


def test_turning_depends_on_the_distance_only():
    rot = {"base": 50.0, "dims": 8}
    q, k = rnd(1, 1, 8, seed=1).expand(9, 1, 8), rnd(1, 1, 8, seed=2).expand(9, 1, 8)
    pos = torch.arange(9)
    s = (P.turn_halves(q, pos, rot)[:, 0] @ P.turn_halves(k, pos, rot)[:, 0].T)
    for lag in range(-8, 9):
        d = torch.diagonal(s, lag)
        assert float((d - d[0]).abs().max()) < 1e-12


def test_recurrence_cut_in_two_and_in_chunk_form():
    T, H, d, dv, cut = 50, 3, 5, 4, 17
    q, k, v = rnd(T, H, d, seed=1), rnd(T, H, d, seed=2), rnd(T, H, dv, seed=3)
    g = torch.tensor([0.3, 0.97, 1.0], dtype=torch.float64)
    o, S = P.constant_decay_scan(q, k, v, g)
    o1, S1 = P.constant_decay_scan(q[:cut], k[:cut], v[:cut], g)
    o2, S2 = P.constant_decay_scan(q[cut:], k[cut:], v[cut:], g, S1)
    assert torch.allclose(torch.cat([o1, o2]), o, atol=1e-12) and torch.allclose(S2, S, atol=1e-12)
    lag = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    for h in range(H):
        D = torch.where(lag >= 0, g[h] ** lag.clamp(min=0).double(), torch.zeros((), dtype=torch.float64))
        assert torch.allclose(((q[:, h] @ k[:, h].T) * D) @ v[:, h], o[:, h], atol=1e-10)


def test_the_maps_may_stand_on_the_querys_side():
    """Scores and outputs from the latent rows alone, with Uk^T on the query and Uv behind the sum."""
    m = KABAPEL["kb-a"]()["layers"][1]["mixer"]
    H, d, r, dv, R, W, T = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], 64, 20
    p = {"q": rnd(H * (d + r), W, seed=1, scale=0.2), "dkv": rnd(R + r, W, seed=2, scale=0.2), "dkv.norm": rnd(R, seed=3).abs(),
         "uk": rnd(H * d, R, seed=4, scale=0.3), "uv": rnd(H * dv, R, seed=5, scale=0.3), "o": rnd(W, H * dv, seed=6)}
    h, pos = rnd(T, W, seed=7), torch.arange(T)
    c, kr = P.latent_rows(h, p, m, 1e-6, pos)
    ref = P.latent_mixer(h, p, m, pos, (c, kr))
    q = (h @ p["q"].T).view(T, H, d + r)
    qr = P.turn_halves(q[..., d:], pos, m["rot"])
    out = []
    for j in range(H):
        uk, uv = p["uk"].view(H, d, R)[j], p["uv"].view(H, dv, R)[j]
        s = ((q[:, j, :d] @ uk) @ c.T + qr[:, j] @ kr.T) * m["scale"]
        w = torch.softmax(s.masked_fill(torch.ones(T, T).triu(1).bool(), -math.inf), dim=-1)
        out.append((w @ c) @ uv.T)
    assert torch.allclose(torch.stack(out, 1).reshape(T, H * dv) @ p["o"].T, ref, atol=1e-10)


def test_router_choice_groups_and_weights():
    z = torch.tensor([[2.0, 1.0, 0.0, 3.0, 0.5, 0.2]], dtype=torch.float64)
    p = torch.softmax(z, -1)[0]
    none = torch.zeros(6, dtype=torch.float64)
    w = P.route(z, none, {"experts": 6, "top": 2})[0]
    assert torch.nonzero(w)[:, 0].tolist() == [0, 3] and abs(float(w.sum()) - 1.0) < 1e-12
    assert abs(float(w[3] / w[0]) - math.e) < 1e-9
    # the correction moves the choice, not the weights; all choices are negative and masked ones still lose
    corr = torch.tensor([-9.0, -2.0, -2.0, -3.0, -2.0, -2.0], dtype=torch.float64)
    w = P.route(z, corr, {"experts": 6, "top": 2})[0]
    assert torch.nonzero(w)[:, 0].tolist() == [1, 4] and abs(float(w[1] / w[4]) - float(p[1] / p[4])) < 1e-9
    # three groups of two: the best choice of each is in (0, 1), (2, 3), (4, 5)
    w = P.route(z, none, {"experts": 6, "top": 2, "groups": {"count": 3, "keep": 1}})[0]
    assert torch.nonzero(w)[:, 0].tolist() == [2, 3]
    w = P.route(z, none - 5.0, {"experts": 6, "top": 3, "groups": {"count": 3, "keep": 2}})[0]
    assert torch.nonzero(w)[:, 0].tolist() == [0, 1, 3]


def test_identity_and_shared_experts():
    W, F = 8, 6
    mlp = {"kind": "moe", "expert": {"ff": F, "limit": 1.0}, "router": {"experts": 1, "top": 1, "identity": 1}, "shared": {"ff": F, "limit": 0.5}}
    p = {f"{n}.{m}": rnd(*((W, F) if m == "down" else (F, W)), seed=i * 3 + j) for i, n in enumerate(("e0", "shared"))
         for j, m in enumerate(("gate", "up", "down"))}
    p["router"], p["shared.sg"] = torch.zeros(2, W, dtype=torch.float64), torch.zeros(1, W, dtype=torch.float64)
    p["correction"] = torch.tensor([-3.0, -1.0], dtype=torch.float64)          # the identity expert wins
    h = rnd(3, W, seed=9)
    sh = 0.5 * P.limited_gated_ff(h, p["shared.gate"], p["shared.up"], p["shared.down"], 0.5)
    assert torch.allclose(P.routed_ff(h, p, mlp), h + sh)
    p["correction"] = torch.tensor([-1.0, -3.0], dtype=torch.float64)
    assert torch.allclose(P.routed_ff(h, p, mlp), P.limited_gated_ff(h, p["e0.gate"], p["e0.up"], p["e0.down"], 1.0) + sh)
    big = P.limited_gated_ff(torch.full((1, 1), 50.0, dtype=torch.float64), torch.ones(1, 1).double(), torch.ones(1, 1).double(), torch.ones(1, 1).double(), 2.0)
    assert abs(float(big) - 2.0 / (1.0 + math.exp(-1.702 * 2.0)) * 3.0) < 1e-12


def test_rows_of_another_layer_and_prefixes():
    """A prefix's logits do not depend on what follows; the shared rows are the owner's, not the reader's own input."""
    for name in ("kb-a", "kb-d"):
        raw = KABAPEL[name]()
        _, t = kabapel_tensors(raw, 3)
        t = {k: v.double() for k, v in t.items()}
        toks = random_tokens(raw["vocab"], 40, 4)
        full = P.forward(raw, t, toks)
        for n in (1, 2, 17):
            assert torch.allclose(P.forward(raw, t, toks[:n]), full[:n], atol=1e-9)
        t2 = dict(t)
        owner = 1 if name == "kb-a" else 0
        t2[f"l{owner}.mix.dkv"] = t[f"l{owner}.mix.dkv"] * -1.0
        assert float((P.forward(raw, t2, toks) - full).abs().max()) > 1e-3
