"""Kabapel on the GPU against the plain implementation, in 32-bit and in bfloat16: every mechanism alone (the layer norm on
the fused add, linear attention with constant decays by walk and by chunks, the gate behind it, the scored router, the
routed feed-forward with groups, identity experts and a shared one, the latent attention without a query latent, on its
own rows and on another layer's), then the model through the engine: whole prompts, the stream after every layer, a
prefix and then single tokens, prompts in pieces down to two tokens, unequal batches against each request alone on slots
and pages that are used again, long decoding from the first token, captured against eager steps, keys far away and at
page borders, and greedy generation, the command line and trace replay through the package's own entry points."""
import json
import os
import subprocess
import sys

import pytest
import torch

import alice_llm_amd as alice
from alice_llm_amd.hip import ops
from alice_llm_amd.parts import FEED_FORWARDS, NORMS, FragmentActs, Precision, ResidualStream
from helpers import KABAPEL, kabapel_folder, kabapel_pair, kabapel_tensors, max_err, model_from_tensors, random_tokens
from plain import kabapel_plain as P
from test_gpu_vifirax import _STEPS, _TOTAL, _Ctx, _walk, assert_close, rnd, row_errors

pytestmark = pytest.mark.gpu
DEV = "cuda"
DTYPES = ["float32", "bfloat16"]
CASES = [(n, d) for n in KABAPEL for d in DTYPES]
_PAIRS = {}


def pair(name, dtype):
    if (name, dtype) not in _PAIRS:
        _PAIRS[(name, dtype)] = kabapel_pair(name, dtype, seed=len(name) + 3)
    return _PAIRS[(name, dtype)]


# ------------------------------------------------------------------ mechanisms alone

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W,parts", [(1, 64, 1), (3, 100, 0), (7, 37, 2), (5, 1000, 1), (400, 256, 1), (330, 2052, 4), (321, 4100, 1), (2, 8200, 3)])
def test_layer_norm_on_the_fused_add(dtype, T, W, parts):
    """Every kernel of the fused add (a row a block in registers or from memory, a row a wave, two waves a row): a pending
    branch of several partial sums, rows with a mean far from zero, then the same rows picked by index."""
    p = Precision.of(dtype)
    eps = 3e-5
    norm = NORMS.get("layernorm")(p, dim=W, eps=eps, tensor_name="", bias_name="b")
    w, b = (1.0 + rnd(W, seed=1, scale=0.3)).to(torch.bfloat16), rnd(W, seed=2).to(torch.bfloat16)
    assert set(norm.param_specs()) == {"", "b"}
    norm.assign("", w.to(DEV))
    norm.assign("b", b.to(DEV))
    x = rnd(T, W, seed=3) + 4.0
    br = rnd(max(1, parts), T, W, seed=4)
    stream = ResidualStream(x.clone().to(DEV), p)
    ref_x = x.double()
    if parts:
        stream.push(br.to(DEV) if parts > 1 else br[0].to(DEV))
        ref_x = ref_x + br.double().sum(0)
    ref = P.layer_norm(ref_x, w.double(), b.double(), eps)
    tol = 3e-5 if dtype == "float32" else 5e-3 * float(ref.abs().max())
    out = stream.normed(norm)
    assert out.dtype == p.act and max_err(out, ref) < tol and max_err(stream.x, ref_x) < 1e-4
    rows = torch.tensor([T - 1, 0, T // 2], dtype=torch.int32, device=DEV)
    assert max_err(stream.rows_normed(norm, rows), ref[rows.cpu().long()]) < tol
    if dtype == "bfloat16" and W % 32 == 0:
        f = stream.normed(norm, fragments=True)
        assert isinstance(f, FragmentActs)
        back = f.data.view(-1, W // 32, 4, 16, 8).permute(0, 3, 1, 2, 4).reshape(-1, W)[:T]
        assert max_err(back, out) == 0.0


def test_layer_norm_takes_a_mean_off_that_is_large_against_the_spread():
    p = Precision.of("float32")
    norm = NORMS.get("layernorm")(p, dim=512, eps=1e-6)
    norm.assign("weight", torch.ones(512, device=DEV))
    norm.assign("bias", torch.zeros(512, device=DEV))
    for T in (3, 400):
        x = rnd(T, 512, seed=T, scale=0.01) + 300.0
        ref = P.layer_norm(x.double(), torch.ones(512).double(), torch.zeros(512).double(), 1e-6)
        assert max_err(ResidualStream(x.to(DEV), p).normed(norm), ref) < 2e-2        # (the rows themselves are rounded at 3e-5 of 0.01)


def _lin_ctx(lens, slots):
    ctx = _Ctx(lens, slots)
    ctx.max_new = max(lens)
    return ctx


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunked", [None, False, True])
@pytest.mark.parametrize("decay,d,dv", [([0.4, 0.999], 16, 24), ([0.97, 0.5, 1.0], 20, 28), ([0.9], 128, 128), ([0.99, 0.2], 64, 7), ([0.8, 1.0], 256, 20),
                                        ([0.95], 1, 1), ([0.6, 0.7], 200, 80), ([0.0, 0.9375], 132, 64)])
def test_lightning_over_pieces_and_slots(dtype, chunked, decay, d, dv):
    """Against the plain scan, by tokens and by chunks, the state carried from step to step in the slots' rows: pieces down
    to one and two tokens and beyond a chunk, a sequence that sits a step out, a slot that is cleared and used again; with
    and without silu on the way in."""
    H, act = len(decay), Precision.of(dtype).act
    width = 2 * H * d + H * dv + 3
    cols = (3, 3 + H * d, 3 + 2 * H * d)
    powers = (torch.tensor(decay, dtype=torch.float64)[:, None] ** torch.arange(ops.LIGHTNING_CHUNK + 1).double()).float().to(DEV)
    for silu in (True, False):
        data, refs = {}, {}
        for i, n in _TOTAL.items():
            x = (rnd(n, width, seed=20 + i) * 0.7).to(act)
            data[i] = x
            a = P.silu(x.double()) if silu else x.double()
            part = lambda c, k: a[:, c:c + H * k].view(n, H, k)
            refs[i] = P.constant_decay_scan(part(cols[0], d), part(cols[1], d), part(cols[2], dv), torch.tensor(decay, dtype=torch.float64))
        S = torch.full((6, H, d, dv), 3.0, device=DEV)
        S[[2, 0, 5]] = 0.0
        for step, (lens, ids, slots, spans) in enumerate(_walk(_TOTAL)):
            if step == 5:
                S[0] = 0.0
            rows = torch.cat([data[i][a:e] for i, (a, e) in zip(ids, spans)]).to(DEV).contiguous()
            out = torch.empty(rows.shape[0], H * dv, device=DEV)
            ops.lightning(rows, cols, powers, out, _lin_ctx(lens, slots), S, heads=H, head_dim=d, value_head_dim=dv, silu=silu, chunked=chunked)
            at = 0
            for i, (a, e) in zip(ids, spans):
                ref = refs[i][0].reshape(-1, H * dv)
                assert max_err(out[at:at + e - a], ref[a:e]) < 1e-5 * max(1.0, float(ref.abs().max())), (silu, step, i)
                at += e - a
        for i, slot in ((0, 2), (2, 5), (3, 0)):
            assert max_err(S[slot], refs[i][1]) < 1e-5 * max(1.0, float(refs[i][1].abs().max())), i
        assert float((S[[1, 3, 4]] - 3.0).abs().max()) == 0.0                        # rows of other slots are untouched


@pytest.mark.parametrize("T", [63, 64, 65, 128, 200, 700])
def test_lightning_keeps_a_far_token_by_a_decay_of_one_and_loses_it_by_one_half(T):
    """One key and value at the start, zeros after it but for the queries: the head whose decay is one reads the value at
    every distance, the other reads it halved at every step; across chunk borders, by chunks and by tokens."""
    H, d, dv = 2, 16, 16
    powers = (torch.tensor([1.0, 0.5], dtype=torch.float64)[:, None] ** torch.arange(ops.LIGHTNING_CHUNK + 1).double()).float().to(DEV)
    rows = torch.zeros(T, H * (2 * d + dv))
    val = torch.arange(1, dv + 1).float()
    rows[:, 0] = rows[:, d] = 1.0                                # q of both heads
    rows[0, 2 * d] = rows[0, 3 * d] = 1.0                        # k
    rows[0, 4 * d:4 * d + dv] = rows[0, 4 * d + dv:] = val
    for chunked in (True, False):
        S = torch.zeros(2, H, d, dv, device=DEV)
        out = torch.empty(T, H * dv, device=DEV)
        ops.lightning(rows.to(DEV), (0, 2 * d, 4 * d), powers, out, _lin_ctx([T], [1]), S, heads=H, head_dim=d, value_head_dim=dv, silu=False, chunked=chunked)
        assert max_err(out[:, :dv], val.expand(T, dv)) < 1e-6
        want = (val.double()[None] * 0.5 ** torch.arange(T).double()[:, None])
        assert float(((out[:, dv:].cpu().double() - want).abs() / want.clamp_min(1e-37)).max()) < 1e-5 or T > 120
        assert max_err(out[:, dv:], want) < 1e-6
        assert max_err(S[1, 0, 0], val) < 1e-6 and float(S[0].abs().max()) == 0.0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,width", [(5, 64), (33, 60), (2, 1024), (300, 96), (1, 4100)])
def test_norm_of_all_heads_with_a_gate_in_the_activation_dtype(dtype, T, width):
    act = Precision.of(dtype).act
    x, gate, eps = rnd(T, width, seed=1, scale=3.0), rnd(T, width + 5, seed=2, scale=2.0).to(act), 1e-5
    w = rnd(width, seed=3).abs() + 0.5
    ref = P.unit_rms(x.double(), eps) * w.double() * torch.sigmoid(gate.double()[:, 2:2 + width])
    out = torch.empty(T, width, dtype=act, device=DEV)
    ops.norm_gate(x.to(DEV), w.to(DEV), out, parts=1, eps=eps, weight_shared=False, gate=gate.to(DEV), gate_col=2, gate_act="sigmoid")
    assert max_err(out, ref) < (1e-5 if dtype == "float32" else 2e-2) * max(1.0, float(ref.abs().max()))


@pytest.mark.parametrize("T,E,Z,top,groups,corr", [(9, 6, 2, 2, (2, 1), -1.5), (70, 16, 0, 3, None, 0.2), (3, 5, 0, 5, None, -1.0), (4, 2, 7, 3, (3, 2), -2.0),
                                                   (2, 200, 56, 8, (8, 3), -1.25), (1, 1, 0, 1, None, -1.0), (5, 12, 4, 1, (16, 4), 0.0), (6, 300, 700, 5, (100, 2), -1.0)])
def test_router_with_scores_over_all_outputs(T, E, Z, top, groups, corr):
    n = E + Z
    z = rnd(T, n + 3, seed=1, scale=2.0)
    c = corr + 0.05 * rnd(n, seed=2)
    router = {"experts": E, "top": top}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    ref = P.route(z[:, :n].double(), c.double(), router)
    w, side = torch.empty(T, E, device=DEV), torch.empty(T, 2, device=DEV)
    for shared in (False, True):
        ops.route_scored(z.to(DEV), c.to(DEV), w, side, identity=Z, top=top, groups=groups[0] if groups else 1, keep=groups[1] if groups else 1,
                         has_shared=shared)
        assert max_err(w, ref[:, :E]) < 1e-6 and max_err(side[:, 0], ref[:, E:].sum(-1)) < 1e-6
        assert max_err(side[:, 1], torch.sigmoid(z[:, n].double()) if shared else torch.zeros(T)) < 1e-6
    # equal choices: the lower index first
    if n > 3 and top == 1 and not groups:
        z[:, :n] = 0.0
        ops.route_scored(z.to(DEV), torch.zeros(n, device=DEV), w, side, identity=Z, top=top)
        assert float((w[:, 0] - 1.0).abs().max()) < 1e-6
    for bad in ({"top": n + 1}, {"groups": n + 1}, {"groups": n, "keep": max(1, top - 1)}):
        if bad.get("keep", 0) >= top:
            continue
        with pytest.raises(ops.HipLibraryError):
            ops.route_scored(z.to(DEV), c.to(DEV), w, side, **dict({"identity": Z, "top": top}, **bad))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W,F,E,top,Z,groups,shared", [
    (5, 64, 24, 6, 2, 2, (2, 1), (40, 0.8)), (70, 72, 18, 5, 5, 0, None, None), (1, 128, 64, 14, 3, 2, (4, 2), (96, 1.2)),
    (130, 128, 64, 14, 3, 2, (4, 2), (96, 1.2)), (33, 48, 7, 3, 1, 0, None, (24, 1.0)), (300, 256, 96, 16, 3, 0, (4, 3), None), (9, 40, 32, 2, 3, 7, (3, 2), (8, 2.0)),
    (1000, 72, 64, 3, 3, 1, None, (64, 0.5)), (257, 136, 160, 33, 4, 3, (6, 2), (32, 4.0)), (16, 256, 128, 12, 2, 4, (2, 1), (128, 1.0)),
    (2, 512, 256, 32, 4, 0, None, (64, 7.0)), (64, 96, 64, 40, 2, 8, (4, 1), None)])
def test_routed_feed_forward_with_everything(dtype, T, W, F, E, top, Z, groups, shared):
    p = Precision.of(dtype)
    limit = 1.3
    args = dict(hidden_size=W, intermediate_size=F, experts=E, top=top, activation="swish_limited", limit=limit, scoring="all", identity=Z, groups=groups,
                shared=None if shared is None else {"intermediate_size": shared[0], "activation": "swish_limited", "limit": shared[1]})
    ff = FEED_FORWARDS.get("expert_mlp")(p, **args)
    ws = {}
    for i, (n, s) in enumerate(ff.param_specs().items()):
        if n == "correction":
            t = -1.5 + 0.1 * rnd(*s.shape, seed=i)
        else:
            t = rnd(*s.shape, seed=i, scale=(2.5 if n in ("router", "shared.sg") else 1.5 if not n.endswith("down") else 1.0) / s.shape[1] ** 0.5)
        ws[n] = t.to(torch.bfloat16).to(DEV)
        ff.assign(n, ws[n])
    ff.finalize()
    x = rnd(T, W, seed=99).to(torch.bfloat16)                    # the router sees the same numbers on both paths
    mlp = {"router": {"experts": E, "top": top}, "expert": {"limit": limit}}
    if groups:
        mlp["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared:
        mlp["shared"] = {"limit": shared[1]}
    pd = {k: v.double().cpu() for k, v in ws.items()}
    ref = P.routed_ff(x.double(), pd, mlp)
    # a token whose choice hangs on a rounding is left out
    choice = torch.softmax(x.double() @ pd["router"].T, -1) + pd["correction"]
    srt = choice.sort(dim=-1, descending=True).values
    gap = (srt[:, :-1] - srt[:, 1:]).amin(-1) if srt.shape[1] > 1 else torch.ones(T)
    keep = gap > 1e-5
    assert int(keep.sum()) >= T // 2
    from alice_llm_amd.parts import experts
    kept = experts.GROUPED_FROM_TOKENS, experts.FEW_CHOICES
    try:
        # the grouped products wherever they apply; every expert's matrices; the chosen ones' only; the part's own choice
        for experts.GROUPED_FROM_TOKENS, experts.FEW_CHOICES in ((1, 0.0), (10 ** 9, 0.0), (10 ** 9, 1e9), kept):
            out = ff.forward(x.to(p.act).to(DEV), None)
            out = out.sum(0) if out.dim() == 3 else out
            assert max_err(out[keep.to(DEV)], ref[keep]) < (3e-5 if dtype == "float32" else 3e-2) * max(1.0, float(ref.abs().max())), experts.GROUPED_FROM_TOKENS
    finally:
        experts.GROUPED_FROM_TOKENS, experts.FEW_CHOICES = kept


# ------------------------------------------------------------------ far keys through the cache

def _marked_latent(kind):
    """A model of latent layers in which one marker token's key stands out for one asking token, on every head of the layer
    that reads the rows (its own, or the first layer's), and the marker's value is large."""
    rot = {"base": 1e4, "dims": 16, "scaling": {"factor": 2.0, "original": 64, "fast": 4.0, "slow": 1.0}}
    W, H, d, R, r, dv = (96, 3, 24, 40, 16, 24) if kind == "plain" else (128, 4, 32, 64, 16, 64)
    lat = {"heads": H, "dim": d, "rot_dim": r, "vdim": dv, "kv_rank": R, "scale": 0.2, "rot": rot}
    layers = [{"type": "latent_attention", "mixer": dict(lat), "mlp": None}, {"type": "latent_attention", "mixer": dict(lat, heads=2 * H, kv_from=0), "mlp": None}]
    raw = {"architecture": "Kabapel", "vocab": 60, "width": W, "norm": {"eps": 1e-6}, "embedding": {"scale": 2.0}, "layers": layers}
    cfg, t = kabapel_tensors(raw, 5)
    t = {k: v.double() for k, v in t.items()}
    t["l0.mix.o"] *= 0.05                                        # the first layer leaves the stream nearly as it is
    x = t["embed"] * 2.0
    h = P.layer_norm(x, t["l0.norm1"], t["l0.norm1.b"], 1e-6)
    c = P.unit_rms(h @ t["l0.mix.dkv"][:R].T, 1e-6) * t["l0.mix.dkv.norm"]
    mark, ask = 7, 9
    h1 = P.layer_norm(x, t["l1.norm1"], t["l1.norm1.b"], 1e-6)
    q = (h1[ask] @ t["l1.mix.q"].T).view(2 * H, d + r)[:, :d]
    uk = t["l1.mix.uk"].view(2 * H, d, R)
    for j in range(2 * H):                                       # Uk c(mark) gains a part along the asking query
        uk[j] += 60.0 * torch.outer(q[j] / q[j].norm() ** 2, c[mark] / c[mark].norm() ** 2) / 0.2
    t["l1.mix.uk"] = uk.reshape(2 * H * d, R)
    t = {k: v.to(torch.bfloat16) for k, v in t.items()}
    return raw, cfg, t, mark, ask


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["plain", "tiles"])
def test_far_key_at_the_start_and_at_page_borders(dtype, kind):
    """One key among hundreds that a late query must find, at the first positions, just before and behind page borders and
    next to the query, in a prompt, in a piece and in decoding; a cache that loses it or reads the neighbouring row gives
    logits far from the plain model's."""
    raw, cfg, t, mark, ask = _marked_latent(kind)
    plain = P.PlainKabapel(raw, {k: v.double() for k, v in t.items()})
    model = model_from_tensors(cfg, {k: v.to(DEV) for k, v in t.items()}, dtype)
    eng = model.engine(max_tokens=1024)
    n = 330
    base = [x for x in random_tokens(60, 3 * n, 3) if x not in (mark, ask)][:n]
    for at in (0, 1, 63, 64, 65, 127, 128, 255, 256, n - 2):
        toks = list(base)
        toks[at], toks[-1] = mark, ask
        ref = plain.forward(toks)[-1:]
        without = list(toks)
        without[at] = base[at - 1] if at else base[5]
        assert float(row_errors(ref, plain.forward(without)[-1:])) > 0.3          # the oracle's own check: the marker matters
        s = eng.open(1)
        got = [eng.step(s, [toks], "last")]
        eng.close(s)
        for cut in (n - 1, n - 2, 200):
            s = eng.open(1)
            eng.step(s, [toks[:cut]], "none")
            got.append(eng.step(s, [toks[cut:]], "last"))
            eng.close(s)
        for g in got:
            assert float(row_errors(g, ref)) < (1e-4 if dtype == "float32" else 0.06), at
    eng.cache.check_consistent()


@pytest.fixture
def spelled():
    """Every prompt step whose sizes allow it spells the latent layers' keys and values out; yields the part's module."""
    from alice_llm_amd.parts import latent
    kept = latent.SPELL_SECONDS
    latent.SPELL_SECONDS = -1e9
    yield latent
    latent.SPELL_SECONDS = kept


@pytest.mark.parametrize("name", ["kb-a", "kb-c", "kb-d", "kb-f", "pf-a", "pf-c"])
def test_keys_and_values_spelled_out_for_prompts(name, spelled, monkeypatch):
    """The other way of a prompt step's latent attention, against the plain model: whole prompts, pieces down to two tokens on
    cached rows, unequal batches, with and without a window (Pefitar's), and the same step the usual way."""
    from helpers import pefitar_pair
    model, plain = pefitar_pair(name, "bfloat16", seed=4) if name.startswith("pf") else pair(name, "bfloat16")
    V = (plain.c if name.startswith("pf") else plain.config)["vocab"]
    calls = []
    old = ops.latent_attention_spelled
    monkeypatch.setattr(ops, "latent_attention_spelled", lambda *a, **k: (calls.append(1), old(*a, **k))[1])
    latents = sum(1 for l in model.lm.layers if getattr(l.mixer, "spell", None) is not None)
    assert latents >= 1
    eng = model.engine(max_tokens=1024)
    for n in (2, 64, 65, 200):
        toks = random_tokens(V, n, n)
        s = eng.open(1)
        got = eng.step(s, [toks], "all")
        eng.close(s)
        assert_close(got, plain.forward(toks), "bfloat16", n)
    assert len(calls) >= 4 * latents
    toks = random_tokens(V, 190, 9)
    ref = plain.forward(toks)
    s, got, at = eng.open(1), [], 0
    for c in (63, 2, 2, 60, 1, 62):
        got.append(eng.step(s, [toks[at:at + c]], "all"))
        at += c
    eng.close(s)
    assert_close(torch.cat(got), ref, "bfloat16")
    lens = [1, 130, 64, 7]
    seqs = [random_tokens(V, n, 70 + n) for n in lens]
    slots = eng.open(4)[::-1]
    first = eng.step(slots, [t[:(n + 1) // 2] for t, n in zip(seqs, lens)], "all")
    rest = eng.step(slots[1:], [t[(n + 1) // 2:] for t, n in list(zip(seqs, lens))[1:]], "all")
    a = b = 0
    for i, n in enumerate(lens):
        h = (n + 1) // 2
        rows = [first[a:a + h]] + ([rest[b:b + n - h]] if i else [])
        a, b = a + h, b + (n - h if i else 0)
        assert_close(torch.cat(rows), plain.forward(seqs[i]), "bfloat16", i)
    eng.close(slots)
    spelled.SPELL_SECONDS = 1e9
    done = len(calls)
    s = eng.open(1)
    other = eng.step(s, [toks], "all")
    eng.close(s)
    assert len(calls) == done
    assert_close(other, ref, "bfloat16")
    eng.cache.check_consistent()


def test_spelling_out_pays_for_long_prompts_and_long_contexts_only():
    raw = dict(KABAPEL["kb-c"]())
    cfg, t = kabapel_tensors(raw, 1)
    mix = model_from_tensors(cfg, {k: v.to(DEV) for k, v in t.items()}, "bfloat16").lm.layers[1].mixer

    class Step:
        is_decode, captured = False, False

        def __init__(self, start, new):
            self.start_lens, self.new_lens = start, new

    assert not mix._spelled_pays(Step([0], [64])) and not mix._spelled_pays(Step([30, 0], [2, 90]))
    assert mix._spelled_pays(Step([0], [60000])) and mix._spelled_pays(Step([4000], [2]))
    one = Step([0], [60000])
    one.captured = True
    assert not mix._spelled_pays(one)
    assert model_from_tensors(cfg, {k: v.to(DEV) for k, v in t.items()}, "float32").lm.layers[1].mixer.spell is None


def test_far_key_spelled_out(spelled):
    test_far_key_at_the_start_and_at_page_borders(kind="tiles", dtype="bfloat16")


# ------------------------------------------------------------------ the model through the engine

@pytest.mark.parametrize("name,dtype", CASES)
def test_whole_prompts(name, dtype):
    model, plain = pair(name, dtype)
    eng = model.engine(max_tokens=512)
    V = plain.config["vocab"]
    for n, seed in ((1, 1), (2, 2), (9, 3), (64, 4), (65, 5), (200, 6)):
        toks = random_tokens(V, n, seed)
        s = eng.open(1)
        got = eng.step(s, [toks], "all")
        eng.close(s)
        assert_close(got, plain.forward(toks), dtype, n)
    eng.cache.check_consistent()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["kb-a", "kb-d"])
def test_residual_stream_after_every_layer(name, dtype):
    model, plain = pair(name, dtype)
    toks = random_tokens(plain.config["vocab"], 21, 8)
    _, runs = plain.forward(toks, return_layers=True)
    seen = []
    blocks = [l.block for l in model.lm.layers]
    olds = [b.forward for b in blocks]
    try:
        for b, old in zip(blocks, olds):
            def fwd(stream, ctx, cache, old=old):
                old(stream, ctx, cache)
                stream.flush()
                seen.append(stream.x.clone())
            b.forward = fwd
        eng = model.engine(max_tokens=64, use_graphs=False)
        s = eng.open(1)
        eng.step(s, [toks], "none")
        eng.close(s)
    finally:
        for b, old in zip(blocks, olds):
            b.forward = old
    assert len(seen) == runs.shape[0] == len(plain.config["layers"])
    for i, x in enumerate(seen):
        if dtype == "float32":
            assert max_err(x, runs[i]) < 2e-5 * float(runs[i].abs().max()), i
        else:
            e = row_errors(x, runs[i])
            assert float(e.mean()) < 0.03 and float(e.max()) < 0.3, (i, float(e.mean()), float(e.max()))


@pytest.mark.parametrize("name,dtype", CASES)
def test_prefix_then_single_tokens_past_pages(name, dtype):
    model, plain = pair(name, dtype)
    eng = model.engine(max_tokens=256)
    toks = random_tokens(plain.config["vocab"], 190, 7)
    s = eng.open(1)
    got = [eng.step(s, [toks[:50]], "all")]                     # decoding crosses positions 64 and 128
    for t in toks[50:]:
        got.append(eng.step(s, [[t]], "last"))
    eng.close(s)
    assert_close(torch.cat(got), plain.forward(toks), dtype)


@pytest.mark.parametrize("name,dtype", CASES)
def test_prompt_in_pieces(name, dtype):
    model, plain = pair(name, dtype)
    eng = model.engine(max_tokens=256)
    toks = random_tokens(plain.config["vocab"], 180, 9)
    ref = plain.forward(toks)
    for cuts in ([2, 3, 7, 64, 1, 73, 30], [63, 2, 2, 113], [128, 52], [1, 1, 2, 176], [2] * 20 + [70, 70], [16, 15, 17, 132]):
        assert sum(cuts) == 180
        s = eng.open(1)
        got, at = [], 0
        for c in cuts:
            got.append(eng.step(s, [toks[at:at + c]], "all"))
            at += c
        eng.close(s)
        assert_close(torch.cat(got), ref, dtype, cuts)
    eng.cache.check_consistent()


@pytest.mark.parametrize("name,dtype", CASES)
def test_unequal_batch_against_each_alone_on_reused_slots(name, dtype):
    model, plain = pair(name, dtype)
    V = plain.config["vocab"]
    eng = model.engine(max_tokens=640, max_seqs=4)
    for rnd_ in range(2):                                       # the second round runs on slots and pages used before
        lens = [1, 66, 23, 130] if rnd_ == 0 else [70, 2, 129, 5]
        n_dec = [12, 30, 5, 20]
        seqs = [random_tokens(V, L + d, 20 + 10 * rnd_ + i) for i, (L, d) in enumerate(zip(lens, n_dec))]
        refs = [plain.forward(t) for t in seqs]
        slots = eng.open(4)
        if rnd_ == 1:
            slots = slots[::-1]
        got = [[] for _ in seqs]
        out = eng.step(slots, [t[:L] for t, L in zip(seqs, lens)], "last")
        for b in range(4):
            got[b].append(out[b])
        live = list(range(4))
        for step in range(max(n_dec)):
            live = [b for b in live if step < n_dec[b]]
            out = eng.step([slots[b] for b in live], [[seqs[b][lens[b] + step]] for b in live], "last")
            for r, b in enumerate(live):
                got[b].append(out[r])
            for b in list(live):
                if step + 1 == n_dec[b]:
                    eng.close([slots[b]])                       # shorter requests end earlier and give their slot back
        for b in range(4):
            assert_close(torch.stack(got[b]), refs[b][lens[b] - 1:], dtype, (rnd_, b))
        eng.cache.check_consistent()
    assert eng.cache.slots.n_free() == 4


@pytest.mark.parametrize("name,dtype", [("kb-a", "float32"), ("kb-b", "bfloat16"), ("kb-c", "float32"), ("kb-d", "bfloat16"), ("kb-e", "float32"), ("kb-f", "bfloat16")])
def test_long_decoding_from_the_first_token(name, dtype):
    model, plain = pair(name, dtype)
    toks = random_tokens(plain.config["vocab"], 330, 11)
    eng = model.engine(max_tokens=384)
    s = eng.open(1)
    got = torch.cat([eng.step(s, [[t]], "last") for t in toks])
    eng.close(s)
    assert_close(got, plain.forward(toks), dtype)


@pytest.mark.parametrize("name", list(KABAPEL))
def test_captured_steps_equal_eager_ones(name):
    model, plain = pair(name, "bfloat16")
    toks = [random_tokens(plain.config["vocab"], 40 + 9 * i, 30 + i) for i in range(3)]
    outs = []
    for graphs in (False, True):
        eng = model.engine(max_tokens=512, use_graphs=graphs)
        assert eng.use_graphs == graphs and (not graphs or eng.capture_prompts)
        slots = eng.open(3)
        rows = [eng.step(slots, [t[:20] for t in toks], "last")]
        for j in range(20, 40):
            rows.append(eng.step(slots, [[t[j]] for t in toks], "last"))
        # short pieces of several tokens: recorded at their second sighting
        pieces = []
        for rep in range(4):
            eng.close(slots)
            slots = eng.open(3)
            pieces.append(eng.step(slots, [t[:7] for t in toks], "last"))
        eng.close(slots)
        outs.append((torch.cat(rows), pieces))
    assert max_err(outs[0][0], outs[1][0]) < 1e-4 * max(1.0, float(outs[0][0].abs().max()))
    # a recorded step of short pieces is padded to 32 tokens and may take the chunks where the eager one goes by tokens: the
    # same numbers up to bfloat16's rounding behind them, and the recorded ones equal each other
    for a, b in zip(outs[0][1], outs[1][1]):
        assert float(row_errors(a, b).max()) < 0.05
    assert max_err(outs[1][1][2], outs[1][1][3]) == 0.0


@pytest.mark.parametrize("name,dtype", CASES)
def test_greedy_generation_through_the_entry_point(name, dtype):
    model, plain = pair(name, dtype)
    V = plain.config["vocab"]
    prompts = [random_tokens(V, n, 40 + n) for n in (3, 17, 70)]
    res = model.generate(prompts, max_new_tokens=[10, 6, 12], stop_token_ids=[])
    for p, r, cap in zip(prompts, res, (10, 6, 12)):
        assert len(r.tokens) == cap
        seq = list(p)
        for tok in r.tokens:
            lg = plain.forward(seq)[-1]
            if dtype == "float32":
                assert float(lg.max() - lg[tok]) < 1e-4 * max(1.0, float(lg.abs().max())), "the chosen token is not the plain model's maximum"
            else:
                assert float(lg.max() - lg[tok]) < 0.3 * float(lg.std()) + 0.05
            seq.append(tok)
    model.release_engine()


# ------------------------------------------------------------------ a folder on disk: loader, command line, trace replay
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay_of_a_folder(dtype, tmp_path):
    """bin/trace_run on a model folder: prompts of unequal lengths as one batch, single tokens together, a request that ends
    early, one that starts later on the slot given back; rows asked for by index."""
    folder = kabapel_folder("kb-a", 5)
    plain = P.PlainKabapel.from_folder(folder)
    a, b, c = (random_tokens(97, n, 60 + n) for n in (70, 9, 40))
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:66], "want": [0, 64, 65]}, {"id": "b", "tokens": b[:7], "want": [6]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[66:67], "want": [0]}, {"id": "b", "tokens": b[7:8], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[67:68], "want": []}, {"id": "b", "tokens": b[8:9], "want": [0]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": a[68:69], "want": [0]}], "end": []},
             {"step": 4, "entries": [{"id": "c", "tokens": c[:38], "want": [37]}], "end": []},
             {"step": 5, "entries": [{"id": "c", "tokens": c[38:], "want": [0, 1]}], "end": ["c"]},
             {"step": 6, "entries": [{"id": "a", "tokens": a[69:], "want": [0]}], "end": ["a"]}]
    out = tmp_path / "out"
    proc = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(out),
                           "--max-tokens", "140"], input="".join(json.dumps(s) + "\n" for s in steps),
                          capture_output=True, text=True, timeout=300, cwd=ROOT)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.split("\n") if l.startswith("done")] == [f"done {i}" for i in range(7)]
    ra, rb, rc = plain.forward(a), plain.forward(b), plain.forward(c)
    want = {0: torch.stack([ra[0], ra[64], ra[65], rb[6]]), 1: torch.stack([ra[66], rb[7]]), 2: rb[8][None], 3: ra[68][None],
            4: rc[37][None], 5: torch.stack([rc[38], rc[39]]), 6: ra[69][None]}
    got_all, want_all = [], []
    for i, w in want.items():
        got = torch.frombuffer(bytearray((out / f"{i}.f32").read_bytes()), dtype=torch.float32).view(-1, 97)
        assert got.shape == w.shape, i
        got_all.append(got)
        want_all.append(w)
    assert_close(torch.cat(got_all), torch.cat(want_all), dtype)


def test_command_line_generates_from_a_folder():
    folder = kabapel_folder("kb-c", 6)
    plain = P.PlainKabapel.from_folder(folder)
    proc = subprocess.run([sys.executable, "-m", "alice_llm_amd.generate", "--model", folder, "--dtype", "float32",
                           "--prompt-ids", "5,9,11,60", "--prompt-ids", "3", "--max-tokens", "5"],
                          capture_output=True, text=True, timeout=300, cwd=ROOT)
    assert proc.returncode == 0, proc.stderr[-2000:]
    for prompt in ([5, 9, 11, 60], [3]):
        ids = plain.greedy(prompt, 5)
        assert ",".join(str(i) for i in ids) in proc.stdout, (ids, proc.stdout[-500:])
