"""Vazilorn on the GPU against the plain implementation, in 32-bit and in bfloat16: every mechanism alone (the tanh norms on
the residual add, norm a head with rotation and cache write into row-major pages and into pages in fragment order, attention
with a window and a sink by every kernel that serves it, the sigmoid router with groups by their two best, the routed
feed-forward by each of its ways), then the model through the engine: whole prompts, the stream after every layer, a prefix and
then single tokens, prompts in pieces down to two tokens, unequal batches against each request alone on slots and pages that
are used again, long decoding from the first token, captured against eager steps, keys at window and page borders and just
outside, and greedy generation, the command line and trace replay through the package's own entry points."""
import json
import os
import subprocess
import sys

import pytest
import torch

import alice_llm_amd as alice
from alice_llm_amd.hip import ops
from alice_llm_amd.parts import FEED_FORWARDS, NORMS, POSITIONS, FragmentActs, Precision, ResidualStream
from helpers import VAZILORN, max_err, model_from_tensors, random_tokens, vazilorn_folder, vazilorn_pair, vazilorn_tensors
from plain import vazilorn_plain as P
from test_gpu_vifirax import _paged, _Step, assert_close, rnd, row_errors

pytestmark = pytest.mark.gpu
DEV = "cuda"
DTYPES = ["float32", "bfloat16"]
CASES = [(n, d) for n in VAZILORN for d in DTYPES]
_PAIRS = {}


def pair(name, dtype):
    if (name, dtype) not in _PAIRS:
        _PAIRS[(name, dtype)] = vazilorn_pair(name, dtype, seed=len(name) + 3)
    return _PAIRS[(name, dtype)]


def i32(v):
    return torch.tensor(v, dtype=torch.int32, device=DEV)


# ------------------------------------------------------------------ mechanisms alone

def _tanh_norm(p, W, alpha, seed):
    norm = NORMS.get("dynamic_tanh")(p, dim=W, tensor_name="", bias_name="b", alpha_name="alpha")
    w, b, a = (1.0 + rnd(W, seed=seed, scale=0.3)).to(torch.bfloat16), rnd(W, seed=seed + 1).to(torch.bfloat16), torch.tensor(alpha).to(torch.bfloat16)
    assert set(norm.param_specs()) == {"", "b", "alpha"}
    for n, t in (("", w), ("b", b), ("alpha", a)):
        norm.assign(n, t.to(DEV))
    return norm, lambda x: P.dynamic_tanh(x.double(), float(a), w.double(), b.double())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W,parts", [(1, 64, 1), (3, 100, 0), (7, 37, 2), (5, 1000, 1), (400, 256, 1), (330, 2052, 4), (1025, 96, 1), (1024, 33, 3),
                                       (2, 8200, 3), (2050, 160, 5)])
def test_tanh_norms_on_the_residual_add(dtype, T, W, parts):
    """A pending branch of several partial sums with a norm behind it, the norm ahead of the next part, then rows picked by
    index; a norm on one side alone; both norms between a norm of another kind."""
    p = Precision.of(dtype)
    post, post_ref = _tanh_norm(p, W, 0.7, 1)
    pre, pre_ref = _tanh_norm(p, W, 0.25, 5)
    x, br = rnd(T, W, seed=3, scale=2.0), rnd(max(1, parts), T, W, seed=4)
    stream = ResidualStream(x.clone().to(DEV), p)
    ref_x = x.double()
    if parts:
        stream.push(br.to(DEV) if parts > 1 else br[0].to(DEV), post)
        ref_x = ref_x + post_ref(br.double().sum(0))
    ref = pre_ref(ref_x)
    tol = 3e-6 if dtype == "float32" else 5e-3 * float(ref.abs().max())
    xtol = 3e-6 * float(ref_x.abs().max()) if dtype == "float32" else 1e-4          # (the quick tanh)
    out = stream.normed(pre)
    assert out.dtype == p.act and max_err(out, ref) < tol * 2 and max_err(stream.x, ref_x) < xtol
    rows = i32([T - 1, 0, T // 2])
    assert max_err(stream.rows_normed(pre, rows), ref[rows.cpu().long()]) < tol * 2
    if dtype == "bfloat16" and W % 32 == 0:
        unpack = lambda f, n: f.data.view(-1, W // 32, 4, 16, 8).permute(0, 3, 1, 2, 4).reshape(-1, W)[:n]
        if FragmentActs.possible(p, T, W):
            assert max_err(unpack(stream.normed(pre, fragments=True), T), out) == 0.0
        f = stream.rows_normed(pre, rows, fragments=True)
        assert isinstance(f, FragmentActs) and max_err(unpack(f, 3), stream.rows_normed(pre, rows)) == 0.0
    # a branch without a norm behind it, and a norm behind it alone
    stream.push(br[0].to(DEV), None)
    ref_x = ref_x + br[0].double()
    assert max_err(stream.normed(pre), pre_ref(ref_x)) < tol * 2
    stream.push(br[0].to(DEV), post)
    stream.flush()
    ref_x = ref_x + post_ref(br[0])
    assert max_err(stream.x, ref_x) < xtol * 2
    stream.push(br[0].to(DEV), post)
    other = NORMS.get("rmsnorm")(p, dim=W, eps=1e-5)
    other.assign("weight", torch.ones(W, device=DEV))
    ref_x = ref_x + post_ref(br[0])
    assert max_err(stream.normed(other), P.unit_rms(ref_x, 1e-5)) < (1e-5 if dtype == "float32" else 3e-2)
    with pytest.raises(ops.HipLibraryError):
        ops.add_dyntanh(stream.x, None, post.pointwise(), None, None, full_precision=True)


def _fragment_places(kp, vp, page, tp):
    """The key [heads, d] and value [heads, d] that a page in fragment order holds at place tp, by plain indexing."""
    d = kp.shape[-1]
    e = torch.arange(d)
    koff = (((tp // 16) * (d // 32) + e // 32) * 64 + ((e % 32) // 8) * 16 + tp % 16) * 8 + e % 8
    w = tp % 16
    voff = (((tp // 32) * (d // 16) + e // 16) * 64 + (w // 4) * 16 + e % 16) * 8 + (((tp % 32) // 16) * 4 + w % 4)
    flat = lambda t: t[page].reshape(t.shape[1], -1).cpu()
    return flat(kp)[:, koff], flat(vp)[:, voff]


@pytest.mark.parametrize("dtype,layout,H,G,d,dv,R,interleaved,bias", [
    ("float32", 0, 3, 3, 20, 12, 20, True, False), ("bfloat16", 0, 4, 2, 16, 24, 8, True, True), ("float32", 0, 2, 1, 7, 5, 4, True, False),
    ("bfloat16", 0, 5, 1, 136, 40, 64, False, False), ("float32", 0, 1, 1, 256, 256, 256, False, True), ("float32", 0, 6, 2, 64, 64, 0, True, False),
    ("bfloat16", 1, 6, 2, 64, 64, 64, True, False), ("bfloat16", 1, 4, 4, 128, 128, 32, True, False), ("bfloat16", 1, 2, 1, 256, 256, 96, True, True),
    ("bfloat16", 1, 3, 1, 64, 64, 0, True, False), ("bfloat16", 1, 10, 5, 64, 64, 24, True, True), ("float32", 0, 4, 2, 128, 96, 64, True, True),
    ("bfloat16", 0, 2, 1, 256, 44, 256, True, False), ("bfloat16", 1, 2, 2, 128, 128, 128, False, False)])
@pytest.mark.parametrize("spare", [4, 8])                    # further columns of a row: the wide loads want rows of whole 32-byte units
@pytest.mark.parametrize("starts,lens", [([60, 3], [10, 70]), ([0, 17, 5], [700, 380, 1]), ([0], [64]), ([31, 0, 100, 9], [1, 1, 1, 1])])
def test_norm_a_head_rotation_and_cache_write(dtype, layout, H, G, d, dv, R, interleaved, bias, starts, lens, spare):
    """Every head divided by its own root mean square and weighted, turned, and put with its value into scattered pages, for
    sequences of one step that start at other positions than 0; nothing beside their own places is touched."""
    act, page, eps, T = Precision.of(dtype).act, 64, 1e-3, sum(lens)
    width = H * d + G * (d + dv)
    rows, bv, wn = rnd(T, width + spare, seed=1), rnd(width, seed=2, scale=0.5), 1.0 + rnd(2, d, seed=3, scale=0.3)
    pos = torch.cat([torch.arange(s, s + n) for s, n in zip(starts, lens)])
    seq = torch.cat([torch.full((n,), i) for i, n in enumerate(lens)])
    per = int(pos.max()) // page + 1
    n_pages = per * len(lens) + 3
    bt = (torch.randperm(n_pages - 1, generator=torch.Generator().manual_seed(5)) + 1)[:per * len(lens)].view(len(lens), per).to(torch.int32)
    x = rows.double()[:, :width] + (bv.double() if bias else 0.0)
    q = P.unit_rms(x[:, :H * d].view(T, H, d), eps) * wn[0].double()
    k = P.unit_rms(x[:, H * d:(H + G) * d].view(T, G, d), eps) * wn[1].double()
    v = x[:, (H + G) * d:].view(T, G, dv)
    cos = sin = None
    if R:
        sc = {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 64}
        part = POSITIONS.get("rope_pairs")(Precision.of(dtype), DEV, dim=d, theta=300.0, max_positions=int(pos.max()) + 1, rotary_dim=R,
                                           interleaved=interleaved, scaling=sc)
        cos, sin = part.cos, part.sin
        f, half = P.banded_frequencies(R, 300.0, sc), R // 2
        order = torch.arange(R) if interleaved else torch.stack([torch.arange(half), torch.arange(half) + half], 1).flatten()

        def turn(a):
            b = a.clone()
            b[..., order] = P.turn_pairs(a[..., order].contiguous(), pos, f)
            return b
        q, k = turn(q), turn(k)
    kp, vp = torch.full((n_pages, G, page, d), 9.0, dtype=act, device=DEV), torch.full((n_pages, G, page, dv), 9.0, dtype=act, device=DEV)
    q_out = torch.full((T, H * d), 9.0, dtype=act, device=DEV)
    common = dict(num_heads=H, num_kv_heads=G, head_dim=d, value_head_dim=dv, max_position=int(pos.max()), cos=cos, sin=sin, rotary_dim=R,
                  interleaved=interleaved, norm_weight=wn.to(DEV), norm_eps=eps, norm_heads=True)
    b_dev = bv.to(DEV) if bias else None
    ops.qkv_prepare(rows.to(DEV), b_dev, q_out, kp, vp, i32(pos.tolist()), i32(seq.tolist()), bt.to(DEV), kv_layout=layout, **common)
    tol = 3e-6 if dtype == "float32" else 2 ** -8
    big = lambda t: max(1.0, float(t.abs().max()))
    assert max_err(q_out.view(T, H, d), q) < tol * big(q)
    for t in range(T):
        page_id, tp = int(bt[seq[t], pos[t] // page]), int(pos[t] % page)
        if layout:
            if t % 7 and t < T - 8:                             # (a sample of the longer pieces, and the end)
                continue
            gk, gv = _fragment_places(kp, vp, page_id, tp)
        else:
            gk, gv = kp[page_id, :, tp], vp[page_id, :, tp]
        assert max_err(gk, k[t]) < tol * big(k) and max_err(gv, v[t]) < tol * big(v), t
    written = int((vp == 9.0).sum())
    assert written == (n_pages * page - T) * G * dv
    assert int((kp == 9.0).sum()) == (n_pages * page - T) * G * d
    # queries alone, from rows that hold no k and v
    q2 = torch.empty_like(q_out)
    ops.qkv_prepare(rows[:, :H * d + spare // 2].contiguous().to(DEV), b_dev, q2, None, None, i32(pos.tolist()), None, None, **common)
    assert max_err(q2, q_out) < tol * big(q)
    if layout:
        with pytest.raises(ops.HipLibraryError):
            ops.qkv_prepare(rows.to(DEV), b_dev, q_out, kp, vp, i32(pos.tolist()), i32(seq.tolist()), bt.to(DEV), kv_layout=layout,
                            **dict(common, norm_heads=False, norm_weight=torch.ones((H + G) * d, device=DEV)))


def _attend(q, k, v, scale, window, sink, pos):
    """q [n, H, d] at positions pos over keys [T, G, d] and values, with a window and a sink a head."""
    H, G = q.shape[1], k.shape[1]
    mask = P.window_mask(pos, k.shape[0], window)
    return torch.stack([P.sink_softmax((q[:, h] @ k[:, h // (H // G)].T) * scale, mask, sink[h]) @ v[:, h // (H // G)] for h in range(H)], 1)


def _fragment_pools(k, v, seed):
    """Keys and values [T, G, d] of one sequence in scattered pages in fragment order."""
    T, G, d = k.shape
    n = -(-T // 64)
    bt = (torch.randperm(n + 3, generator=torch.Generator().manual_seed(seed))[:n] + 1).to(torch.int32)[None].to(DEV)
    kp, vp = torch.zeros(n + 5, G, 64, d, dtype=torch.bfloat16, device=DEV), torch.zeros(n + 5, G, 64, d, dtype=torch.bfloat16, device=DEV)
    qkv = torch.cat([torch.zeros(T, d, dtype=torch.bfloat16), k.reshape(T, -1), v.reshape(T, -1)], 1).contiguous().to(DEV)
    ops.rope_cache_write(qkv, torch.empty(T, d, dtype=torch.bfloat16, device=DEV), kp, vp, None, None, torch.arange(T, dtype=torch.int32, device=DEV),
                         torch.zeros(T, dtype=torch.int32, device=DEV), bt, num_heads=1, num_kv_heads=G, head_dim=d, rotary_dim=0, max_position=T - 1,
                         kv_layout=ops.KV_FRAGMENT)
    return kp, vp, bt


@pytest.mark.parametrize("H,G,d", [(6, 2, 64), (4, 4, 128), (2, 1, 256), (8, 1, 128), (16, 1, 64)])
@pytest.mark.parametrize("window", [None, 1, 50, 64, 200])
def test_sink_in_the_matrix_core_attention(H, G, d, window):
    """Prompts by every form of the kernel and single tokens at several splits, with sinks from far below the scores to far
    above them; a sink that is left out, or counted once a part, is far outside the tolerance."""
    T, scale, bf = 300, 1.5 * d ** -0.5, torch.bfloat16
    q, k, v = rnd(T, H, d, seed=1).to(bf), rnd(T, G, d, seed=2).to(bf), rnd(T, G, d, seed=3).to(bf)
    sink = torch.linspace(-3.0, 6.0, H) if H > 1 else torch.tensor([2.0])
    pos = torch.arange(T)
    ref = _attend(q.double(), k.double(), v.double(), scale, window, sink.double(), pos)
    assert float((ref - _attend(q.double(), k.double(), v.double(), scale, window, sink.double() - 30.0, pos)).abs().max()) > 0.2
    kp, vp, bt = _fragment_pools(k, v, 4)
    common = dict(num_heads=H, scale=scale, softcap=None, window=window, sink=sink.to(DEV))
    for new in (T, 37, 2):
        qs = q[T - new:].reshape(new, H * d).contiguous().to(DEV)
        for variant in (ops.PREFILL_TILES, ops.PREFILL_SPLIT, ops.PREFILL_SHARED4, ops.PREFILL_SHARED8, ops.PREFILL_SHARED4X2, ops.PREFILL_AUTO):
            out = torch.full_like(qs, float("nan"))
            ops.attention_prefill(qs, kp, vp, out, i32([0, new]), i32([T]), bt, n_seqs=1, max_new=new, max_context=T, variant=variant, **common)
            assert max_err(out.view(new, H, d), ref[T - new:]) < 3e-2, (new, variant)      # (outputs up to 4.5: half a bfloat16 step is 0.016)
    places = [0, 1, 31, 63, 64, 199, 255, 299]
    qs = q[places].reshape(len(places), H * d).contiguous().to(DEV)
    lens, tables = i32([p + 1 for p in places]), bt.expand(len(places), -1).contiguous()
    w = rnd(96, H * d, seed=5, scale=0.1).to(bf)
    for splits in (None, 1, 2, 5, 16):
        out = torch.full_like(qs, float("nan"))
        ops.attention_decode(qs, kp, vp, out, lens, tables, max_context=T, splits=splits, **common)
        assert max_err(out.view(-1, H, d), ref[places]) < 3e-2, splits
        if splits in (2, 5):
            slices = ops.linear_parts_slices(len(places), 96, H, d, splits)
            assert slices > 0
            parts, _ = ops.attention_decode(qs, kp, vp, None, lens, tables, max_context=T, splits=splits, **common)
            y = torch.empty(slices, len(places), 96, device=DEV)
            ops.linear_parts(parts, splits, ops.to_frag16(w.to(DEV)), y, num_heads=H, head_dim=d)
            want = ref[places].reshape(len(places), -1) @ w.double().T
            assert max_err(y.sum(0), want) < 4e-2 * (H * d / 64) ** 0.5 * 0.3
    with pytest.raises(ops.HipLibraryError):
        ops.attention_decode(qs, kp, vp, out, lens, tables, max_context=T, **dict(common, sink=sink[:H - 1].to(DEV) if H > 1 else torch.zeros(2, device=DEV)))


@pytest.mark.parametrize("kind", ["fragment", "row16", "row32"])
@pytest.mark.parametrize("window", [1, 2, 31, 32, 33, 63, 64, 65, 100])
def test_keys_just_inside_and_just_outside_a_window(kind, window):
    """One key that a query scores far above all others, at the last place inside its window and at the first outside, for
    queries at page and tile borders, in a prompt, in pieces and as single tokens."""
    T, H, G, d = 200, 4, 2, 64
    act = torch.float32 if kind == "row32" else torch.bfloat16
    q, k, v = rnd(T, H, d, seed=1), rnd(T, G, d, seed=2), rnd(T, G, d, seed=3)
    scale, sink = 0.2, torch.tensor([0.5, -1.0, 2.0, 1.0])
    for at in (63, 64, 65, 127, 128, 140, 199):
        for back in (0, window - 1, window, window + 1):
            if at - back < 0:
                continue
            kk = k.clone()
            for h in range(H):                                  # (both heads of a group look for their own part of the key)
                kk[at - back, h // 2] += 1.2 * q[at, h]
            kk = kk.to(act)
            ref = _attend(q.to(act).double()[at:at + 1], kk.double(), v.to(act).double(), scale, window, sink.double(), torch.tensor([at]))
            gone = kk.clone()
            gone[at - back] = 0
            moved = float((ref - _attend(q.to(act).double()[at:at + 1], gone.double(), v.to(act).double(), scale, window, sink.double(), torch.tensor([at]))).abs().max())
            assert moved > 0.3 if back < window else moved == 0.0
            tol = 1e-4 if kind == "row32" else 3e-2
            if kind == "fragment":
                kp, vp, bt = _fragment_pools(kk, v.to(act), 4)
                common = dict(num_heads=H, scale=scale, softcap=None, window=window, sink=sink.to(DEV))
                one = q[at].reshape(1, -1).to(act).contiguous().to(DEV)
                for splits in (1, 3):
                    out = torch.empty_like(one)
                    ops.attention_decode(one, kp, vp, out, i32([at + 1]), bt, max_context=at + 1, splits=splits, **common)
                    assert max_err(out.view(1, H, d), ref) < tol, (at, back, splits)
                for new in (2, at + 1):
                    qs = q[at + 1 - new:at + 1].reshape(new, -1).to(act).contiguous().to(DEV)
                    out = torch.empty_like(qs)
                    ops.attention_prefill(qs, kp, vp, out, i32([0, new]), i32([at + 1]), bt, n_seqs=1, max_new=new, max_context=at + 1, **common)
                    assert max_err(out.view(new, H, d)[-1:], ref) < tol, (at, back, new)
                continue
            kp, vp, bt = _paged(kk, v.to(act), 64, 4)
            common = dict(num_heads=H, scale=scale, window=window, sink=sink.to(DEV))
            one = q[at].reshape(1, -1).to(act).contiguous().to(DEV)
            out = torch.empty_like(one)
            ops.attention_split(one, kp, vp, out, i32([at]), i32([0]), bt, max_position=at, max_keys=min(at + 1, window), **common)
            assert max_err(out.view(1, H, d), ref) < tol, (at, back, "split")
            ops.attention_masked(one, kp, vp, out, i32([at]), i32([0]), bt, max_position=at, full_precision=kind == "row32", **common)
            assert max_err(out.view(1, H, d), ref) < tol, (at, back, "masked")
            if kind == "row16":
                ctx = _Step([(at - 1, at + 1)], T)
                qs = q[at - 1:at + 1].reshape(2, -1).to(act).contiguous().to(DEV)
                out = torch.empty_like(qs)
                ops.attention_tiled(qs, kp, vp, out, ctx, bt, **common)
                assert max_err(out.view(2, H, d)[-1:], ref) < tol, (at, back, "tiled")


@pytest.mark.parametrize("T,E,top,groups,corr,scale", [(9, 6, 2, (2, 1), -0.6, 1.0), (70, 16, 3, None, 0.2, 2.5), (3, 5, 5, None, -1.0, 0.7), (4, 9, 3, (3, 2), -2.0, 1.3),
                                                       (2, 256, 8, (8, 3), -0.5, 2.5), (1, 1, 1, None, -1.0, 3.0), (5, 16, 1, (16, 4), 0.0, 1.0), (6, 1000, 5, (100, 2), -1.0, 2.0),
                                                       (33, 12, 4, (4, 3), -0.3, 1.0)])
def test_router_with_sigmoid_scores(T, E, top, groups, corr, scale):
    z = rnd(T, E + 3, seed=1, scale=2.0)
    c = corr + 0.2 * rnd(E, seed=2)
    router = {"experts": E, "top": top, "scale": scale}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    ref = P.route(z[:, :E].double(), c.double(), router)
    w, side = torch.empty(T, E, device=DEV), torch.empty(T, 2, device=DEV)
    args = dict(identity=0, top=top, groups=groups[0] if groups else 1, keep=groups[1] if groups else 1, sigmoid=True, group_best=2, weight_scale=scale)
    for shared, gate in ((False, False), (True, False), (True, True)):
        ops.route_scored(z.to(DEV), c.to(DEV), w, side, has_shared=shared, shared_gate=gate, **args)
        assert max_err(w, ref) < 2e-6 and float(side[:, 0].abs().max()) == 0.0
        want = torch.zeros(T) if not shared else torch.sigmoid(z[:, E].double()) if gate else torch.ones(T)
        assert max_err(side[:, 1], want) < 1e-6


def test_a_group_counts_by_its_two_best_choices():
    """The best single choice lies in a group whose second best is poor; equal choices take the lower index; groups of one
    expert count by it alone; choices of either sign."""
    z = torch.tensor([[3.0, -4.0, 1.5, 1.4, -1.0, 0.0], [0.0, 0.0, 0.0, 0.0, 0.0, 0.0]])
    for corr in (0.0, -0.9, -5.0):
        c = torch.full((6,), corr)
        w, side = torch.empty(2, 6, device=DEV), torch.empty(2, 2, device=DEV)
        picked = lambda r: torch.nonzero(w[r].cpu())[:, 0].tolist()
        ops.route_scored(z.to(DEV), c.to(DEV), w, side, identity=0, top=2, groups=3, keep=1, sigmoid=True, group_best=2)
        assert picked(0) == [2, 3] and picked(1) == [0, 1]
        ops.route_scored(z.to(DEV), c.to(DEV), w, side, identity=0, top=2, groups=3, keep=1, sigmoid=True, group_best=1)
        assert picked(0) == [0, 1]
        ops.route_scored(z.to(DEV), c.to(DEV), w, side, identity=0, top=2, groups=6, keep=2, sigmoid=True, group_best=2)
        assert picked(0) == [0, 2] and picked(1) == [0, 1]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W,F,E,top,groups,shared,scale", [
    (5, 64, 24, 6, 2, (2, 1), 40, 1.7), (70, 72, 18, 5, 5, None, None, 0.6), (1, 128, 64, 16, 3, (4, 2), 96, 2.5), (130, 128, 64, 16, 3, (4, 2), 96, 2.5),
    (33, 48, 7, 3, 1, None, 24, 1.0), (300, 256, 96, 16, 3, (4, 3), None, 1.4), (1000, 72, 64, 3, 3, None, 64, 2.0), (257, 136, 160, 36, 4, (6, 2), 32, 1.0),
    (16, 256, 128, 12, 2, (2, 1), 128, 3.0), (2, 512, 256, 32, 4, None, 64, 2.5), (64, 96, 64, 40, 2, (4, 1), None, 1.0)])
def test_routed_feed_forward_by_each_of_its_ways(dtype, T, W, F, E, top, groups, shared, scale):
    p = Precision.of(dtype)
    args = dict(hidden_size=W, intermediate_size=F, experts=E, top=top, activation="silu", scoring="sigmoid", group_best=2, weight_scale=scale,
                groups=groups, shared=None if shared is None else {"intermediate_size": shared, "activation": "silu"}, shared_gate=False)
    ff = FEED_FORWARDS.get("expert_mlp")(p, **args)
    ws = {}
    for i, (n, s) in enumerate(ff.param_specs().items()):
        if n == "correction":
            t = -0.6 + 0.1 * rnd(*s.shape, seed=i)
        else:
            t = rnd(*s.shape, seed=i, scale=(2.5 if n == "router" else 1.5 if not n.endswith("down") else 1.0) / s.shape[1] ** 0.5)
        ws[n] = t.to(torch.bfloat16).to(DEV)
        ff.assign(n, ws[n])
    ff.finalize()
    x = rnd(T, W, seed=99).to(torch.bfloat16)                    # the router sees the same numbers on both paths
    mlp = {"router": {"experts": E, "top": top, "scale": scale}}
    if groups:
        mlp["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared:
        mlp["shared"] = {"ff": shared}
    pd = {k: v.double().cpu() for k, v in ws.items()}
    ref = P.routed_ff(x.double(), pd, mlp)
    # a token whose choice hangs on a rounding is left out
    choice = torch.sigmoid(x.double() @ pd["router"].T) + pd["correction"]
    srt = choice.sort(dim=-1, descending=True).values
    gap = (srt[:, :-1] - srt[:, 1:]).amin(-1)
    keep = gap > 1e-6
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


# ------------------------------------------------------------------ one key among hundreds, through the cache

def _marked(kind):
    """A model of one layer in which a marker token's key stands out for one asking token: both gain, on every head, the same
    direction of the dimensions that are not turned, and all other tokens' keys are small there."""
    W, H, G, d, dv, R, window = {"fragment": (128, 4, 2, 64, 64, 32, 150), "tiles": (96, 4, 2, 48, 24, 16, 150), "wide": (96, 3, 1, 256, 256, 64, 64),
                                 "group": (96, 18, 1, 64, 64, 16, 130)}[kind]
    raw = {"architecture": "Vazilorn", "vocab": 60, "width": W, "norm": {"eps": 1e-6}, "layers": [
        {"type": "attention", "mixer": {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": 16.0 / d, "mask": {"size": window},
                                        "rot": {"base": 1e4, "dims": R}}, "mlp": None}]}
    cfg, t = vazilorn_tensors(raw, 5)
    t = {k: v.double() for k, v in t.items()}
    h = P.dynamic_tanh(t["embed"], t["l0.norm1.alpha"], t["l0.norm1"], t["l0.norm1.b"])
    mark, ask = 7, 9
    u = torch.zeros(d, dtype=torch.float64)
    u[R:] = rnd(d - R, seed=8).double()
    u = u / u.norm() * d ** 0.5
    solve = torch.linalg.pinv(h)                                 # a row that is one at one token and zero at the others
    t["l0.mix.k"] += 4.0 * torch.outer(u.repeat(G), solve[:, mark])
    t["l0.mix.q"] += 4.0 * torch.outer(u.repeat(H), solve[:, ask])
    t["l0.mix.sink"], t["l0.mix.o"] = torch.linspace(-2.0, 3.0, H).double(), t["l0.mix.o"] * 4.0
    t = {k: v.to(torch.bfloat16) for k, v in t.items()}
    return raw, cfg, t, mark, ask, window


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["fragment", "tiles", "wide", "group"])
def test_far_key_at_the_start_at_page_borders_and_at_the_windows_edge(dtype, kind):
    """One key among hundreds that a late query must find, or must no longer see: at the first positions, just before and
    behind page borders, next to the query, at the window's last place and the first outside; in a prompt, in a piece and
    decoded."""
    raw, cfg, t, mark, ask, window = _marked(kind)
    plain = P.PlainVazilorn(raw, {k: v.double() for k, v in t.items()})
    model = model_from_tensors(cfg, {k: v.to(DEV) for k, v in t.items()}, dtype)
    eng = model.engine(max_tokens=1024)
    for n in (window, 330):
        base = [x for x in random_tokens(60, 3 * n, 3) if x not in (mark, ask)][:n]
        places = {0, 1, 63, 64, 65, n - window - 2, n - window - 1, n - window, n - window + 1, n - 2, 255, 256}
        for at in sorted(p for p in places if 0 <= p < n - 1):
            toks = list(base)
            toks[at], toks[-1] = mark, ask
            ref = plain.forward(toks)[-1:]
            without = list(toks)
            without[at] = base[at - 1] if at else base[5]
            moved = float(row_errors(ref, plain.forward(without)[-1:]))
            assert moved > 0.2 if at >= n - window else moved < 1e-9      # the oracle's own check: whether the marker matters
            s = eng.open(1)
            got = [eng.step(s, [toks], "last")]
            eng.close(s)
            for cut in (n - 1, n - 2, n // 2):
                s = eng.open(1)
                eng.step(s, [toks[:cut]], "none")
                got.append(eng.step(s, [toks[cut:]], "last"))
                eng.close(s)
            for g in got:
                assert float(row_errors(g, ref)) < (1e-4 if dtype == "float32" else 0.06), (n, at)
    eng.cache.check_consistent()


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
@pytest.mark.parametrize("name", ["vz-a", "vz-d"])
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


@pytest.mark.parametrize("name,dtype", [("vz-a", "float32"), ("vz-b", "bfloat16"), ("vz-c", "float32"), ("vz-d", "bfloat16"), ("vz-e", "float32"), ("vz-f", "bfloat16")])
def test_long_decoding_from_the_first_token(name, dtype):
    model, plain = pair(name, dtype)
    toks = random_tokens(plain.config["vocab"], 330, 11)
    eng = model.engine(max_tokens=384)
    s = eng.open(1)
    got = torch.cat([eng.step(s, [[t]], "last") for t in toks])
    eng.close(s)
    assert_close(got, plain.forward(toks), dtype)


@pytest.mark.parametrize("name", list(VAZILORN))
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
    # a recorded step of short pieces is padded to a multiple of 16 tokens and may take another form of the prompt attention: the
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
    folder = vazilorn_folder("vz-a", 5)
    plain = P.PlainVazilorn.from_folder(folder)
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
    folder = vazilorn_folder("vz-c", 6)
    plain = P.PlainVazilorn.from_folder(folder)
    proc = subprocess.run([sys.executable, "-m", "alice_llm_amd.generate", "--model", folder, "--dtype", "float32",
                           "--prompt-ids", "5,9,11,60", "--prompt-ids", "3", "--max-tokens", "5"],
                          capture_output=True, text=True, timeout=300, cwd=ROOT)
    assert proc.returncode == 0, proc.stderr[-2000:]
    for prompt in ([5, 9, 11, 60], [3]):
        ids = plain.greedy(prompt, 5)
        assert ",".join(str(i) for i in ids) in proc.stdout, (ids, proc.stdout[-500:])
