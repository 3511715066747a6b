"""Seeded random Kabapel configurations and schedules against the plain implementation: every size and option drawn
(layer order, head counts and sizes, decays, ranks, rotated parts with or without stretched frequencies or none at all,
experts, groups, identity and shared experts, layers without a feed-forward, layers on another's rows), a prompt whole,
the same prompt in random pieces, and two unequal requests together that then go on by single tokens.  Most cases run in
32-bit, where every logit is held to the plain model's; every fourth runs in bfloat16 with dense feed-forwards in the
routed ones' places (a token whose scores nearly tie takes another expert under bfloat16's rounding, and layers with
state carry that on; the fixed configurations cover routed layers in bfloat16)."""
import random

import pytest
import torch

from helpers import kabapel_tensors, model_from_tensors, random_tokens
from plain.kabapel_plain import PlainKabapel
from test_gpu_vifirax import assert_close

pytestmark = pytest.mark.gpu


def _moe(rng):
    experts, identity = rng.randint(1, 16), rng.choice([0, 0, 1, 4, 8])
    n = experts + identity
    router = {"experts": experts, "top": rng.randint(1, min(4, n))}
    if identity:
        router["identity"] = identity
    if rng.random() < 0.6:
        count = rng.choice([g for g in range(1, n + 1) if n % g == 0])
        least = -(-router["top"] // (n // count))
        router["groups"] = {"count": count, "keep": rng.randint(least, count)}
    mlp = {"kind": "moe", "expert": {"ff": rng.choice([8, 16, 17, 24, 64]), "limit": rng.uniform(0.5, 4.0)}, "router": router}
    if rng.random() < 0.6:
        mlp["shared"] = {"ff": rng.choice([8, 24, 33, 64]), "limit": rng.uniform(0.5, 4.0)}
    return mlp


def draw_config(rng: random.Random, routed: bool = True) -> dict:
    width = rng.choice([40, 48, 64, 96, 136, 200, 256])
    layers, owners = [], []
    for i in range(rng.randint(2, 7)):
        if rng.random() < 0.5:
            heads = rng.choice([1, 2, 3, 4, 6])
            m = {"heads": heads, "dim": rng.choice([4, 8, 16, 24, 64, 96, 128, 192]), "vdim": rng.choice([6, 8, 16, 40, 64, 128]),
                 "decay": [rng.choice([1.0, 0.999, 0.5, rng.uniform(0.2, 1.0)]) for _ in range(heads)]}
            kind = "lightning"
        else:
            kind = "latent_attention"
            m = {"heads": rng.choice([1, 2, 3, 4, 6, 8, 20]), "dim": rng.choice([8, 16, 24, 40, 64]), "vdim": rng.choice([8, 16, 24, 40, 64, 96]),
                 "scale": rng.uniform(0.1, 0.35)}
            if owners and rng.random() < 0.5:
                j = rng.choice(owners)
                m.update({k: layers[j]["mixer"][k] for k in ("kv_rank", "rot_dim", "rot") if k in layers[j]["mixer"]}, kv_from=j)
            else:
                m.update(kv_rank=rng.choice([8, 20, 32, 40, 64, 128, 264]), rot_dim=rng.choice([0, 2, 6, 8, 16, 32, 64]))
                if m["rot_dim"]:
                    m["rot"] = {"base": rng.choice([50.0, 1e4, 2.5e5]), "dims": m["rot_dim"]}
                    if rng.random() < 0.7:
                        m["rot"]["scaling"] = {"factor": rng.choice([2.0, 8.0, 32.0]), "original": rng.choice([8, 64, 2048]),
                                               "fast": rng.choice([4.0, 32.0]), "slow": rng.choice([0.5, 1.0, 2.0])}
                owners.append(i)
        r = rng.random()
        if r < 0.2:
            mlp = None
        elif r < 0.5 or not routed:
            mlp = {"kind": "dense", "ff": rng.choice([17, 32, 96, 160])}
        else:
            mlp = _moe(rng)
        layers.append({"type": kind, "mixer": m, "mlp": mlp})
    return {"architecture": "Kabapel", "vocab": rng.randint(50, 700), "width": width, "norm": {"eps": rng.choice([1e-6, 1e-5])},
            "embedding": {"scale": rng.choice([1.0, 2.5, 12.0])}, "layers": layers}


@pytest.mark.parametrize("seed", range(14))
def test_random_configuration(seed):
    rng = random.Random(2000 + seed)
    dtype = "bfloat16" if seed % 4 == 3 else "float32"
    raw = draw_config(rng, routed=dtype == "float32")
    cfg, tensors = kabapel_tensors(raw, seed)
    plain = PlainKabapel(raw, {k: v.double() for k, v in tensors.items()})
    model = model_from_tensors(cfg, {k: v.to("cuda") for k, v in tensors.items()}, dtype)
    V = raw["vocab"]
    eng = model.engine(max_tokens=1024, max_seqs=3)
    n = rng.randint(1, 200)
    toks = random_tokens(V, n, seed)
    ref = plain.forward(toks)
    s = eng.open(1)
    assert_close(eng.step(s, [toks], "all"), ref, dtype, ("whole", raw))
    eng.close(s)
    s, got, at = eng.open(1), [], 0
    while at < n:
        c = min(n - at, rng.choice([1, 2, 3, 17, 64, 70]))
        got.append(eng.step(s, [toks[at:at + c]], "all"))
        at += c
    eng.close(s)
    assert_close(torch.cat(got), ref, dtype, ("pieces", raw))
    lens, dec = [rng.randint(1, 90), rng.randint(1, 90)], [rng.randint(1, 12), rng.randint(1, 12)]
    seqs = [random_tokens(V, L + d, 50 + seed + i) for i, (L, d) in enumerate(zip(lens, dec))]
    refs = [plain.forward(t) for t in seqs]
    slots = eng.open(2)
    out = eng.step(slots, [t[:L] for t, L in zip(seqs, lens)], "last")
    rows = [[out[0]], [out[1]]]
    live = [0, 1]
    for step in range(max(dec)):
        live = [b for b in live if step < dec[b]]
        out = eng.step([slots[b] for b in live], [[seqs[b][lens[b] + step]] for b in live], "last")
        for r, b in enumerate(live):
            rows[b].append(out[r])
        for b in list(live):
            if step + 1 == dec[b]:
                eng.close([slots[b]])
    for b in range(2):
        assert_close(torch.stack(rows[b]), refs[b][lens[b] - 1:], dtype, ("together", b, raw))
    eng.cache.check_consistent()
