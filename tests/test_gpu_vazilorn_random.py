"""Seeded random Vazilorn configurations and schedules against the plain implementation: every size and option drawn (head
counts and sizes, values of another size than keys, windows from one position on, the turned part of a head with and without
stretched frequencies, experts, groups, a shared expert, layers without a feed-forward), a prompt whole, the same prompt in random
pieces, and two unequal requests together that then go on by single tokens.  Most cases run in 32-bit, where every logit is held
to the plain model's; every fourth runs in bfloat16 with dense feed-forwards in the routed ones' places (a token whose scores
nearly tie takes another expert under bfloat16's rounding; the fixed configurations cover routed layers in bfloat16)."""
import random

import pytest
import torch

from helpers import model_from_tensors, random_tokens, vazilorn_tensors
from plain.vazilorn_plain import PlainVazilorn
from test_gpu_vifirax import assert_close

pytestmark = pytest.mark.gpu


def _moe(rng):
    n = rng.choice([1, 2, 3, 4, 6, 8, 9, 12, 16, 20])
    router = {"experts": n, "top": rng.randint(1, min(4, n)), "scale": rng.choice([1.0, 2.5, rng.uniform(0.3, 3.0)])}
    if rng.random() < 0.6:
        count = rng.choice([g for g in range(1, n + 1) if n % g == 0])
        least = -(-router["top"] // (n // count))
        router["groups"] = {"count": count, "keep": rng.randint(least, count)}
    mlp = {"kind": "moe", "expert": {"ff": rng.choice([8, 16, 17, 24, 32, 64])}, "router": router}
    if rng.random() < 0.6:
        mlp["shared"] = {"ff": rng.choice([8, 24, 33, 64])}
    return mlp


def draw_config(rng: random.Random, routed: bool = True) -> dict:
    width = rng.choice([40, 48, 50, 64, 96, 136, 192, 256])
    layers = []
    for _ in range(rng.randint(1, 5)):
        kv = rng.choice([1, 1, 2, 3])
        dim = rng.choice([6, 8, 20, 24, 48, 64, 64, 80, 128, 128, 256])
        m = {"heads": kv * rng.choice([1, 2, 3, 4, 6]), "kv_heads": kv, "dim": dim, "vdim": dim if rng.random() < 0.6 else rng.choice([5, 8, 24, 64, 96, 128]),
             "scale": rng.uniform(0.5, 1.5) * dim ** -0.5, "mask": {"size": rng.choice([1, 2, 5, 16, 31, 33, 63, 64, 65, 100, 129, 500])},
             "rot": {"base": rng.choice([50.0, 1e4, 2.5e5]), "dims": rng.choice([dim, dim, dim // 4 * 2, 2])}}
        if rng.random() < 0.7:
            low = rng.choice([0.5, 1.0, 2.0])
            m["rot"]["scaling"] = {"factor": rng.choice([2.0, 8.0, 32.0]), "low": low, "high": low * rng.choice([1.5, 4.0]), "original": rng.choice([8, 64, 2048])}
        r = rng.random()
        if r < 0.15:
            mlp = None
        elif r < 0.4 or not routed:
            mlp = {"kind": "dense", "ff": rng.choice([17, 32, 96, 160])}
        else:
            mlp = _moe(rng)
        layers.append({"type": "attention", "mixer": m, "mlp": mlp})
    return {"architecture": "Vazilorn", "vocab": rng.randint(50, 700), "width": width, "norm": {"eps": rng.choice([1e-6, 1e-5, 1e-3])}, "layers": layers}


@pytest.mark.parametrize("seed", range(16))
def test_random_configuration(seed):
    rng = random.Random(3000 + seed)
    dtype = "bfloat16" if seed % 4 == 3 else "float32"
    raw = draw_config(rng, routed=dtype == "float32")
    cfg, tensors = vazilorn_tensors(raw, seed)
    plain = PlainVazilorn(raw, {k: v.double() for k, v in tensors.items()})
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
