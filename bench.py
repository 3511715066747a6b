"""Decode and prefill throughput of the Gemma 2 shapes with random weights on one MI355X.

    python bench.py --gpus 1 --steps K --warmup W

A step is one decode step of a batch of 8 sequences that were prefilled with 2,048-token prompts;
by default the timed steps run the context from 2,048 out to 4,096.  The printed line also holds the
prefill of one 2,048-token prompt (and of prompts of 8,192, 512 and 128 tokens), the decode step's memory roofline (at the
mean context of the timed steps), and decode throughput at batch 1 and 64 over the same range, each with
its roofline.  Beside the published peaks the line gives what this GPU itself reaches (`peak_measured`: a
device-to-device copy and a large bfloat16 matrix product of the vendor library) and, under `shapes`, shorter runs
of the other configurations: the 2B shape at contexts from 8,000, 16 unequal prompts at the 9B shape, and 8 prompts
of 6,000 tokens, past the window, at the 27B shape.

    python bench.py --telulorn w2048,w4096
        instead of the above: the Telulorn design beside Novotar and Gemma 2 at equal layer sizes, in a line of its own
    python bench.py --pefitar w2048,w4096
        instead of the above: the Pefitar design beside Telulorn and Gemma 2 at equal layer sizes, in a line of its own
    python bench.py --vifirax w2048,w4096
        instead of the above: the Vifirax design beside Telulorn and Gemma 2 at equal layer sizes, in a line of its own
    python bench.py --kabapel w2048,w4096
        instead of the above: the Kabapel design beside Vifirax and Pefitar at equal layer sizes, in a line of its own
    python bench.py --vazilorn w2048,w4096
        instead of the above: the Vazilorn design beside Kabapel and Gemma 2 at equal layer sizes, in a line of its own
    python bench.py --novotar w2048,w4096
        instead of the above: prefill and decode throughput of the Novotar design at layer sizes of real models
        (random weights, a few layers), beside Gemma 2 at equal sizes; prints a line of its own

Other runs of the same program:
    python bench.py --preset 9b --batch 16 --prompt-lens uniform:64:2048 --steps 256 --points "" --shapes ""
        16 prompts of unequal, seeded lengths in ragged steps, then 256 decode steps
    python bench.py --preset 27b --batch 8 --prompt 6000 --context 8192 --steps 128 --points "" --shapes ""
        8 prompts of 6,000 tokens, past the window of 4,096, then 128 decode steps
"""
import argparse
import json
import os
import sys
import time

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

PEAK_HBM_GBS = 8000.0                       # MI355X HBM3E
PEAK_FLOPS = {"bf16": 2.5e15, "fp32": 157.3e12}


def decode_bytes(cfg, weight_bytes, contexts, elem):
    """Bytes a decode step has to read: every weight once, and the keys and values of the live requests
    (a sliding layer reads at most its window of them)."""
    kv = 0
    for ctx in contexts:
        for i in range(cfg.num_hidden_layers):
            w = cfg.layer_window(i)
            keys = ctx if w is None else min(ctx, w)
            kv += 2 * keys * cfg.kv_dim * elem
    return weight_bytes + kv


def prefill_flops(cfg, T, n_logit_rows=1):
    H, Q, KV, I = cfg.hidden_size, cfg.q_dim, cfg.kv_dim, cfg.intermediate_size
    per_layer = 2 * T * (H * (Q + 2 * KV) + Q * H + 3 * H * I)
    attn = 0
    for i in range(cfg.num_hidden_layers):
        w = cfg.layer_window(i)
        pairs = T * (T + 1) // 2 if not w or w >= T else w * (w + 1) // 2 + (T - w) * w
        attn += 4 * cfg.num_attention_heads * cfg.head_dim * pairs
    return cfg.num_hidden_layers * per_layer + attn + 2 * n_logit_rows * H * cfg.vocab_size


def prompt_lengths(spec, batch, prompt, seed=0):
    """--prompt-lens: 'uniform:LO:HI' draws each sequence's prompt length from [LO, HI] (seeded); a list
    'a,b,c' gives them; nothing gives --prompt to every sequence."""
    import random
    if not spec:
        return [prompt] * batch
    if spec.startswith("uniform:"):
        lo, hi = (int(x) for x in spec.split(":")[1:3])
        rng = random.Random(seed)
        return [rng.randint(lo, hi) for _ in range(batch)]
    lens = [int(x) for x in spec.split(",")]
    if len(lens) != batch:
        raise SystemExit(f"--prompt-lens lists {len(lens)} lengths for a batch of {batch}")
    return lens


def measured_peaks():
    """What this GPU reaches by itself, beside the published peaks: a device-to-device copy of 2 GB (bytes read
    plus bytes written over its time) and an 8,192-cubed bfloat16 matrix product of the vendor library, each the
    median of five by HIP events.  Neither is on the product path."""
    import torch
    out = {}

    def median_ms(fn, n=5):
        fn()
        ts = []
        for _ in range(n):
            a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            a.record()
            fn()
            b.record()
            torch.cuda.synchronize()
            ts.append(a.elapsed_time(b))
        return sorted(ts)[n // 2]

    src = torch.empty(1 << 30, dtype=torch.int16, device="cuda")
    dst = torch.empty_like(src)
    ms = median_ms(lambda: dst.copy_(src))
    out["copy_gbs"] = round(2 * src.numel() * 2 / (ms / 1e3) / 1e9, 1)
    del src, dst
    a = torch.randn(8192, 8192, device="cuda", dtype=torch.bfloat16)
    b = torch.randn(8192, 8192, device="cuda", dtype=torch.bfloat16)
    ms = median_ms(lambda: torch.matmul(a, b))
    out["bf16_matmul_tflops"] = round(2 * 8192 ** 3 / (ms / 1e3) / 1e12, 1)
    del a, b
    torch.cuda.empty_cache()
    return out


class Run:
    """One model shape with random weights and the measurements on it."""

    def __init__(self, preset, layers, dtype, ids_through_host=False, raw=None):
        import torch
        import alice_llm_amd as alice
        self.torch, self.alice = torch, alice
        if raw is None:
            raw = alice.preset(preset)
            self.full_layers = raw["num_hidden_layers"]
            if layers:
                raw["num_hidden_layers"] = layers
        else:
            self.full_layers = None
        self.cfg = alice.config_from_dict(raw)
        self.dtype = dtype
        self.elem = 2 if dtype == "bfloat16" else 4
        self.short = "bf16" if dtype == "bfloat16" else "fp32"
        self.ids_through_host = ids_through_host
        t0 = time.time()
        self.model = alice.Model.random(self.cfg, seed=0, dtype=dtype, fast=True)
        self.weight_bytes = self.model.lm.weight_bytes()
        print(f"[bench] {preset}: model built in {time.time() - t0:.1f} s, weights {self.weight_bytes / 1e9:.2f} GB",
              file=sys.stderr, flush=True)
        self.gen = torch.Generator().manual_seed(0)
        self.gpu_ms = None

    def prompts(self, lens):
        return [self.torch.randint(0, self.model.lm.plan.vocab_size, (n,), generator=self.gen).tolist() for n in lens]

    def decode(self, lens, steps, warmup, context=0):
        """Prefill prompts of these lengths (in the generation loop's ragged steps), then time `steps` decode steps
        (greedy, tokens fed back).  Returns the time and every sequence's context at the first and after the
        last timed step."""
        torch, alice, cfg = self.torch, self.alice, self.cfg
        from alice_llm_amd.hip import ops
        batch = len(lens)
        room = [max(n + warmup + steps, context) for n in lens]
        if max(n + warmup + steps for n in lens) > self.model.lm.plan.max_positions:
            raise SystemExit(f"prompt + warmup + steps reach beyond the model's {self.model.lm.plan.max_positions} positions")
        eng = self.model.engine(seq_lens=room, max_seqs=batch)
        slots = eng.open(batch)
        ps = self.prompts(lens)
        # the prompts run as the generation loop runs them: ragged steps of at most its token budget each
        ids = ops.argmax(alice.run_prompt_steps(eng, slots, ps)).tolist()
        # Decode steps as the library's own generation loop runs them: the chosen ids go from the sampling kernel
        # to the next step on the device, and the host queues step n + 1 before it reads step n's ids (through a
        # pinned buffer and an event), so it is one step ahead and no further.
        pending = []

        def one(ids):
            if self.ids_through_host:
                return ops.argmax(eng.step(slots, [[t_] for t_ in ids], "last")).tolist()
            out = ops.argmax(eng.step(slots, ids, "last"))
            host = torch.empty(out.shape, dtype=out.dtype, pin_memory=True)
            host.copy_(out, non_blocking=True)
            ev = torch.cuda.Event()
            ev.record()
            pending.append((ev, host))
            if len(pending) > 1:
                ev0, host0 = pending.pop(0)
                ev0.synchronize()
                host0.tolist()                                   # where a loop would look for stop tokens
            return out

        if not self.ids_through_host:
            ids = torch.tensor(ids, dtype=torch.int32, device="cuda")
        for _ in range(warmup):
            ids = one(ids)
        ctx0 = [eng.length(s) for s in slots]
        torch.cuda.synchronize()
        pending.clear()
        t = time.perf_counter()
        for _ in range(steps):
            ids = one(ids)
        torch.cuda.synchronize()
        dt = time.perf_counter() - t
        ctx1 = [eng.length(s) for s in slots]
        # The GPU's own time for a step: the last captured step replayed back to back with nothing of the host
        # between the replays (it writes the same cache places again and again).  What the timed steps took
        # beyond that is the host's: bookkeeping, the copy of the step's integers, reading the chosen tokens.
        self.gpu_ms = None
        captured = [g for g in eng._graphs.values() if g.graph is not None]
        if captured:
            a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            a.record()
            for _ in range(20):
                captured[-1].graph.replay()
            b.record()
            torch.cuda.synchronize()
            self.gpu_ms = a.elapsed_time(b) / 20
        eng.close(slots)
        del eng
        torch.cuda.empty_cache()
        return dt, ctx0, ctx1

    def roofline(self, dt, steps, ctx0, ctx1):
        mids = [(a + b) // 2 for a, b in zip(ctx0, ctx1)]
        achieved = decode_bytes(self.cfg, self.weight_bytes, mids, self.elem) / (dt / steps) / 1e9
        return {"bound": "hbm", "achieved": round(achieved, 1), "peak": PEAK_HBM_GBS, "unit": "GB/s",
                "frac": round(achieved / PEAK_HBM_GBS, 4)}

    def prefill(self, T, repeats=5):
        """One prompt of T tokens through one step: the median of `repeats` timings by HIP events (after one
        untimed pass), the wall clock's minimum beside it."""
        torch = self.torch
        eng = self.model.engine(seq_lens=[T], max_seqs=1)
        p = self.prompts([T])
        gpu, wall = [], []
        for it in range(repeats + 1):
            s = eng.open(1)
            torch.cuda.synchronize()
            a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            t = time.perf_counter()
            a.record()
            eng.step(s, p, "last")
            b.record()
            torch.cuda.synchronize()
            if it:
                wall.append((time.perf_counter() - t) * 1e3)
                gpu.append(a.elapsed_time(b))
            eng.close(s)
        ms = sorted(gpu)[len(gpu) // 2]
        fl = prefill_flops(self.cfg, T)
        # frac: the step's flops over the matrix cores' peak; hbm_frac: the weights, which every step reads once,
        # over the memory's peak (what bounds a prompt of a few hundred tokens)
        out = {"value": round(T / (ms / 1e3), 1), "tokens": T, "ms": round(ms, 3),
               "frac": round(fl / (ms / 1e3) / PEAK_FLOPS[self.short], 4),
               "hbm_frac": round(self.weight_bytes / (ms / 1e3) / 1e9 / PEAK_HBM_GBS, 4),
               "timing": f"median of {repeats} by HIP events", "wall_ms_min": round(min(wall), 3)}
        del eng
        torch.cuda.empty_cache()
        return out

    def prefill_batch(self, lens, repeats=3):
        """Several prompts as one ragged step; the median of `repeats` timings by HIP events, in ms."""
        torch = self.torch
        eng = self.model.engine(seq_lens=list(lens), max_seqs=len(lens))
        ps = self.prompts(lens)
        gpu = []
        for it in range(repeats + 1):
            s = eng.open(len(lens))
            torch.cuda.synchronize()
            a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
            a.record()
            eng.step(s, ps, "last")
            b.record()
            torch.cuda.synchronize()
            if it:
                gpu.append(a.elapsed_time(b))
            eng.close(s)
        del eng
        torch.cuda.empty_cache()
        return sorted(gpu)[len(gpu) // 2]

    def step_bytes(self, contexts):
        """Bytes a decode step moves whatever the architecture: every weight once (of a routed feed-forward that reads the
        chosen experts only, those), each run's keys and values within its window, and each run's fixed-size state read
        and written."""
        total = self.weight_bytes
        for l in self.model.lm.layers:                # experts that no token of the step chooses are not read (uniform choices)
            unread = getattr(l.feed_forward, "unread_bytes", None)
            total -= unread(len(contexts)) if unread else 0
        for need in self.model.lm.cache_needs():
            if need is None:
                continue
            if need.kv is not None:
                for c in contexts:
                    keys = c if need.kv.window is None else min(c, need.kv.window)
                    total += keys * need.kv.num_kv_heads * (need.kv.head_dim + need.kv.v_dim) * self.elem
            for st in need.state:
                n = 1
                for x in st.shape:
                    n *= x
                total += 2 * n * 4 * len(contexts)
        return total

    def close(self):
        del self.model
        self.torch.cuda.empty_cache()


# ---------------------------------------------------------------------------------- Novotar beside Gemma 2
NOVOTAR_SIZES = {
    # width, feed-forward, attention heads / kv heads / head size, matrix-memory heads / key size / value size
    "w2048": dict(width=2048, ff=8192, heads=16, kv=4, dim=128, mheads=8, mdim=128, mvdim=256),
    "w4096": dict(width=4096, ff=14336, heads=32, kv=8, dim=128, mheads=16, mdim=128, mvdim=256),
}


def novotar_pair_configs(size, vocab=32768, window=1024):
    """A Novotar configuration of four layers, the middle two run twice (six layer runs), and a Gemma 2 configuration
    of six layers with the same width, feed-forward, heads, head size, window and vocabulary."""
    z = NOVOTAR_SIZES[size]
    layer = {"type": "parallel",
             "mixer": {"left": {"heads": z["heads"], "kv_heads": z["kv"], "dim": z["dim"], "vdim": z["dim"],
                                "scale": z["dim"] ** -0.5, "mask": {"size": window}},
                       "right": {"heads": z["mheads"], "dim": z["mdim"], "vdim": z["mvdim"], "gate_cap": 15.0}},
             "mlp": {"kind": "dense", "ff": z["ff"], "limit": 7.0}}
    nov = {"architecture": "Novotar", "vocab": vocab, "width": z["width"], "embedding": {"scale": 1.0}, "norm": {"eps": 1e-6},
           "layers": [layer] * 4, "loop": {"start": 1, "stop": 3, "times": 2}, "token_side": {"dim": 64}}
    gem = {"architectures": ["Gemma2ForCausalLM"], "model_type": "gemma2", "vocab_size": vocab, "hidden_size": z["width"],
           "num_hidden_layers": 6, "num_attention_heads": z["heads"], "num_key_value_heads": z["kv"], "head_dim": z["dim"],
           "intermediate_size": z["ff"], "max_position_embeddings": 65536, "sliding_window": window,
           "layer_types": ["sliding_attention"] * 6, "query_pre_attn_scalar": z["dim"],
           "attn_logit_softcapping": None, "final_logit_softcapping": None, "tie_word_embeddings": False}
    return nov, gem


def telulorn_configs(size, vocab=32768, window=1024):
    """A Telulorn configuration of four layers (side-by-side mixer, attention, side-by-side mixer, attention), the middle
    two run twice (six layer runs), at the sizes of novotar_pair_configs: the same width, feed-forward, attention
    heads and window (as the chunk of the one mixer and the window of the other, which keeps 64 first positions);
    the recurrence with the matrix memory's heads and head sizes."""
    z = NOVOTAR_SIZES[size]
    heads = {"heads": z["heads"], "kv_heads": z["kv"], "dim": z["dim"], "vdim": z["dim"], "scale": z["dim"] ** -0.5}
    mlp = {"kind": "dense", "ff": z["ff"]}
    par = {"type": "parallel", "mlp": mlp,
           "mixer": {"left": dict(heads, mask={"size": window}), "left_scale": 1.0, "right_scale": 0.9,
                     "right": {"heads": z["mheads"], "dim": z["mdim"], "vdim": z["mvdim"], "tau": 8.0, "rank": 64}}}
    att = {"type": "attention", "mlp": mlp,
           "mixer": dict(heads, mask={"size": window, "keep_first": 64}, rot={"base": 10000.0, "dims": z["dim"] // 2})}
    return {"architecture": "Telulorn", "vocab": vocab, "width": z["width"], "norm": {"eps": 1e-6},
            "layers": [par, att, par, att], "loop": {"start": 1, "stop": 3, "times": 2}}


def pefitar_configs(size, vocab=32768, window=1024):
    """A Pefitar configuration of four layers (latent attention, gated attention, latent attention, gated attention), the
    middle two run twice (six layer runs), at the sizes of novotar_pair_configs: the same width, feed-forward, heads and
    window.  The latent layers keep 128 plain and 64 rotated dimensions a head, values of 128, a key/value latent of 512
    and a query latent of three eighths of the width; the gated attention layers see every earlier key."""
    z = NOVOTAR_SIZES[size]
    mlp = {"kind": "dense", "ff": z["ff"]}
    lat = {"type": "latent_attention", "mlp": mlp,
           "mixer": {"heads": z["heads"], "dim": z["dim"], "rot_dim": 64, "vdim": z["dim"], "q_rank": 3 * z["width"] // 8,
                     "kv_rank": 512, "scale": (z["dim"] + 64) ** -0.5, "mask": {"size": window},
                     "rot": {"base": 10000.0, "dims": 64}}}
    att = {"type": "attention", "mlp": mlp,
           "mixer": {"heads": z["heads"], "kv_heads": z["kv"], "dim": z["dim"], "vdim": z["dim"], "scale": z["dim"] ** -0.5,
                     "rot": {"base": 10000.0, "dims": z["dim"] // 2}}}
    return {"architecture": "Pefitar", "vocab": vocab, "width": z["width"], "norm": {"eps": 1e-6}, "residual_mult": 0.7,
            "logit_softcap": 30.0, "layers": [lat, att, lat, att], "loop": {"start": 1, "stop": 3, "times": 2}}


def vifirax_configs(size, vocab=32768):
    """A Vifirax configuration of six layers (attention, state space, delta rule, attention on the first layer's keys, state
    space, delta rule) at the sizes of novotar_pair_configs: the same width and attention heads; every earlier key
    visible; the state-space layers with an inner width of twice the model's in heads of 64 and a state of 128; the
    delta-rule layers with the attention's heads and head size; feed-forwards in turn dense (the same size) and routed
    (16 experts of a quarter of that size, 2 a token: half the dense layer's work a token, four times its weights)."""
    z = NOVOTAR_SIZES[size]
    dense = {"kind": "dense", "ff": z["ff"]}
    moe = {"kind": "moe", "expert": {"ff": z["ff"] // 4}, "router": {"experts": 16, "top": 2}}
    att = {"heads": z["heads"], "kv_heads": z["kv"], "dim": z["dim"], "vdim": z["dim"], "scale": z["dim"] ** -0.5,
           "rot": {"base": 10000.0, "dims": z["dim"] // 2, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
    ssm = {"heads": 2 * z["width"] // 64, "vdim": 64, "state": 128, "groups": 1, "norm_groups": 1, "conv": 4}
    dlt = {"heads": z["heads"], "kv_heads": z["heads"], "dim": z["dim"], "vdim": z["dim"], "conv": 4, "decay_rank": z["dim"],
           "gate_rank": z["dim"]}
    layers = [{"type": "attention", "mixer": att, "mlp": dense}, {"type": "mamba2", "mixer": ssm, "mlp": moe},
              {"type": "channel_delta", "mixer": dlt, "mlp": dense}, {"type": "attention", "mixer": dict(att, kv_from=0), "mlp": moe},
              {"type": "mamba2", "mixer": ssm, "mlp": dense}, {"type": "channel_delta", "mixer": dlt, "mlp": moe}]
    return {"architecture": "Vifirax", "vocab": vocab, "width": z["width"], "norm": {"eps": 1e-6}, "logit_scale": 0.5, "layers": layers}


def kabapel_configs(size, vocab=32768):
    """A Kabapel configuration of six layers (linear attention, latent attention, linear attention twice, latent attention on
    the second layer's rows, linear attention) at the sizes of novotar_pair_configs: the same width; the linear-attention
    layers with the attention's heads and head size; the latent layers with 128 plain and 64 rotated dimensions a head,
    values of 128 and a latent of 512, every earlier key visible; the first and the last feed-forward dense (the same
    size, two matrices), the others routed (16 experts of a quarter of that size and 4 identity experts in two groups,
    2 a token from one of them, and a shared expert of a quarter)."""
    z = NOVOTAR_SIZES[size]
    dense = {"kind": "dense", "ff": z["ff"]}
    moe = {"kind": "moe", "expert": {"ff": z["ff"] // 4, "limit": 7.0}, "shared": {"ff": z["ff"] // 4, "limit": 7.0},
           "router": {"experts": 16, "identity": 4, "top": 2, "groups": {"count": 2, "keep": 1}}}
    H = z["heads"]
    lin = {"heads": H, "dim": z["dim"], "vdim": z["dim"], "decay": [1.0 - 2.0 ** (-1.0 - 8.0 * i / H) for i in range(H)]}
    lat = {"heads": H, "dim": z["dim"], "rot_dim": 64, "vdim": z["dim"], "kv_rank": 512, "scale": (z["dim"] + 64) ** -0.5,
           "rot": {"base": 500000.0, "dims": 64, "scaling": {"factor": 8.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
    layer = lambda kind, m, ff: {"type": kind, "mixer": m, "mlp": ff}
    return {"architecture": "Kabapel", "vocab": vocab, "width": z["width"], "norm": {"eps": 1e-6}, "embedding": {"scale": 12.0},
            "layers": [layer("lightning", lin, dense), layer("latent_attention", lat, moe), layer("lightning", lin, moe),
                       layer("lightning", lin, moe), layer("latent_attention", dict(lat, kv_from=1), moe), layer("lightning", lin, dense)]}


def vazilorn_configs(size, vocab=32768, window=1024):
    """A Vazilorn configuration of six layers at the sizes of novotar_pair_configs: the same width, attention heads and window;
    the first and the last feed-forward dense (the same size), the others routed (16 experts of a quarter of that size in two
    groups, 2 a token from one of them, and a shared expert of a quarter), as in kabapel_configs."""
    z = NOVOTAR_SIZES[size]
    dense = {"kind": "dense", "ff": z["ff"]}
    moe = {"kind": "moe", "expert": {"ff": z["ff"] // 4}, "shared": {"ff": z["ff"] // 4},
           "router": {"experts": 16, "top": 2, "scale": 2.5, "groups": {"count": 2, "keep": 1}}}
    att = {"heads": z["heads"], "kv_heads": z["kv"], "dim": z["dim"], "vdim": z["dim"], "scale": z["dim"] ** -0.5, "mask": {"size": window},
           "rot": {"base": 500000.0, "dims": z["dim"], "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}
    return {"architecture": "Vazilorn", "vocab": vocab, "width": z["width"], "norm": {"eps": 1e-6},
            "layers": [{"type": "attention", "mixer": att, "mlp": dense if i in (0, 5) else moe} for i in range(6)]}


def novotar_bench(sizes, dtype, steps, warmup, with_telulorn=False, with_pefitar=False, with_vifirax=False, with_kabapel=False,
                  with_vazilorn=False):
    out = {}
    for size in sizes:
        if size not in NOVOTAR_SIZES:
            raise SystemExit(f"unknown size '{size}'; known: {sorted(NOVOTAR_SIZES)}")
        res = {}
        models = list(zip(("novotar", "gemma2"), novotar_pair_configs(size)))
        if with_telulorn:
            models.insert(0, ("telulorn", telulorn_configs(size)))
        if with_pefitar:
            models = [("pefitar", pefitar_configs(size)), ("telulorn", telulorn_configs(size)), models[-1]]
        if with_vifirax:
            models = [("vifirax", vifirax_configs(size)), ("telulorn", telulorn_configs(size)), models[-1]]
        if with_kabapel:
            models = [("kabapel", kabapel_configs(size)), ("vifirax", vifirax_configs(size)), ("pefitar", pefitar_configs(size))]
        if with_vazilorn:
            models = [("vazilorn", vazilorn_configs(size)), ("kabapel", kabapel_configs(size)), models[-1]]
        for name, raw in models:
            run = Run(None, None, dtype, raw=raw)
            r = {"weights_gb": round(run.weight_bytes / 1e9, 3), "layer_runs": len(run.model.lm.plan.schedule)}
            for T in (2048, 8192):
                ms = run.prefill_batch([T])
                r[f"prefill_{T}"] = {"ms": round(ms, 3), "tok_s": round(T / ms * 1e3, 1)}
            ms = run.prefill_batch([2048] * 8)
            r["prefill_8x2048"] = {"ms": round(ms, 3), "tok_s": round(8 * 2048 / ms * 1e3, 1)}
            for b in (1, 8, 64):
                dt, c0, c1 = run.decode([2048] * b, steps, warmup)
                gbs = run.step_bytes([(x + y) // 2 for x, y in zip(c0, c1)]) / (dt / steps) / 1e9
                r[f"decode_b{b}"] = {"ms_per_step": round(dt / steps * 1e3, 4), "tok_s": round(b * steps / dt, 1),
                                     "gpu_ms_per_step": round(run.gpu_ms, 4) if run.gpu_ms else None,
                                     "roofline_gbs": round(gbs, 1), "roofline_frac": round(gbs / PEAK_HBM_GBS, 4)}
            print(f"[bench] {size} {name}: {r}", file=sys.stderr, flush=True)
            res[name] = r
            run.close()
        out[size] = res
    return out


SHAPES = {
    "2b-ctx8k": dict(preset="2b", batches=(8, 64), prompt=8000, lens="", steps=20),
    "9b-unequal": dict(preset="9b", batches=(16,), prompt=0, lens="uniform:64:2048", steps=64),
    "27b-6000": dict(preset="27b", batches=(8,), prompt=6000, lens="", steps=32),
}


def shape_run(name, dtype):
    """A shorter run of another configuration, every figure with its configuration beside it."""
    spec = SHAPES[name]
    run = Run(spec["preset"], None, dtype)
    cfg = run.cfg
    out = {"model": f"gemma2-{spec['preset']}", "layers": cfg.num_hidden_layers, "weights_gb": round(run.weight_bytes / 1e9, 2),
           "steps": spec["steps"], "warmup": 3}
    for b in spec["batches"]:
        lens = prompt_lengths(spec["lens"], b, spec["prompt"])
        dt, c0, c1 = run.decode(lens, spec["steps"], 3)
        roof = run.roofline(dt, spec["steps"], c0, c1)
        out[f"decode_b{b}"] = {"tok_s": round(b * spec["steps"] / dt, 1), "ms_per_step": round(dt / spec["steps"] * 1e3, 4),
                               "prompt_len_min": min(lens), "prompt_len_max": max(lens),
                               "context_start": int(round(sum(c0) / len(c0))), "context_end": int(round(sum(c1) / len(c1))),
                               "roofline_gbs": roof["achieved"], "roofline_frac": roof["frac"]}
        print(f"[bench] {name} decode_b{b}: {out[f'decode_b{b}']}", file=sys.stderr, flush=True)
    if spec["preset"] != "2b":
        pf = run.prefill(2048, repeats=3)
        out["prefill_2048"] = {"tok_s": pf["value"], "ms": pf["ms"], "frac": pf["frac"]}
    run.close()
    return out


def main() -> int:
    ap = argparse.ArgumentParser(description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=2048)
    ap.add_argument("--warmup", type=int, default=8)
    ap.add_argument("--preset", default="2b")
    ap.add_argument("--layers", type=int, default=None, help="fewer layers than the preset (both numbers are reported)")
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--prompt", type=int, default=2048)
    ap.add_argument("--prompt-lens", default="", help="unequal prompts: 'uniform:LO:HI' (seeded) or a list 'a,b,c'")
    ap.add_argument("--context", type=int, default=4096)
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--points", default="1,64", help="other batch sizes to measure decode at ('' for none)")
    ap.add_argument("--point-steps", type=int, default=None, help="steps for the other batch sizes (default: --steps)")
    ap.add_argument("--no-prefill", action="store_true")
    ap.add_argument("--ids-through-host", action="store_true",
                    help="read every step's chosen ids on the host before the next step is queued (the loop with an observer)")
    ap.add_argument("--prefill-tokens", default="2048,8192,512,128", help="prompt lengths whose prefill is timed (the first is the headline's)")
    ap.add_argument("--shapes", default=",".join(SHAPES),
                    help="shorter runs of other configurations, reported under 'shapes' ('' for none)")
    ap.add_argument("--novotar", default="", help="sizes (w2048,w4096): measure the Novotar design beside Gemma 2 at equal "
                    "sizes instead of the default workload, and print a line of its own")
    ap.add_argument("--telulorn", default="", help="sizes (w2048,w4096): measure the Telulorn design beside Novotar and Gemma 2 at "
                    "equal sizes instead of the default workload, and print a line of its own")
    ap.add_argument("--pefitar", default="", help="sizes (w2048,w4096): measure the Pefitar design beside Telulorn and Gemma 2 at "
                    "equal layer sizes, in a line of its own")
    ap.add_argument("--vifirax", default="", help="sizes (w2048,w4096): measure the Vifirax design beside Telulorn and Gemma 2 at "
                    "equal layer sizes, in a line of its own")
    ap.add_argument("--kabapel", default="", help="sizes (w2048,w4096): measure the Kabapel design beside Vifirax and Pefitar at "
                    "equal layer sizes, in a line of its own")
    ap.add_argument("--vazilorn", default="", help="sizes (w2048,w4096): measure the Vazilorn design beside Kabapel and Gemma 2 at "
                    "equal layer sizes, in a line of its own")
    ap.add_argument("--no-peaks", action="store_true", help="skip the measurement of this GPU's own copy and matrix-product rates")
    args = ap.parse_args()
    if args.gpus != 1:
        print(f"bench.py: this library runs on one GPU; --gpus {args.gpus} is not supported", flush=True)
        return 2

    import torch
    torch.cuda.set_device(0)
    if args.vazilorn:
        steps = min(args.steps, 64)
        res = novotar_bench([x for x in args.vazilorn.split(",") if x], args.dtype, steps, min(args.warmup, 5), with_vazilorn=True)
        print(json.dumps({"metric": "Vazilorn beside Kabapel and Gemma 2 at equal layer sizes: prefill and decode, random weights",
                          "unit": "tokens/s", "n_gpus": 1, "steps": steps, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
                          "data": "synthetic (uniform random token ids, random weights)", "sizes": res}), flush=True)
        return 0
    if args.kabapel:
        steps = min(args.steps, 64)
        res = novotar_bench([x for x in args.kabapel.split(",") if x], args.dtype, steps, min(args.warmup, 5), with_kabapel=True)
        print(json.dumps({"metric": "Kabapel beside Vifirax and Pefitar at equal layer sizes: prefill and decode, random weights",
                          "unit": "tokens/s", "n_gpus": 1, "steps": steps, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
                          "data": "synthetic (uniform random token ids, random weights)", "sizes": res}), flush=True)
        return 0
    if args.vifirax:
        steps = min(args.steps, 64)
        res = novotar_bench([x for x in args.vifirax.split(",") if x], args.dtype, steps, min(args.warmup, 5), with_vifirax=True)
        print(json.dumps({"metric": "Vifirax beside Telulorn and Gemma 2 at equal layer sizes: prefill and decode, random weights",
                          "unit": "tokens/s", "n_gpus": 1, "steps": steps, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
                          "data": "synthetic (uniform random token ids, random weights)", "sizes": res}), flush=True)
        return 0
    if args.pefitar:
        steps = min(args.steps, 64)
        res = novotar_bench([x for x in args.pefitar.split(",") if x], args.dtype, steps, min(args.warmup, 5), with_pefitar=True)
        print(json.dumps({"metric": "Pefitar beside Telulorn and Gemma 2 at equal layer sizes: prefill and decode, random weights",
                          "unit": "tokens/s", "n_gpus": 1, "steps": steps, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
                          "data": "synthetic (uniform random token ids, random weights)", "sizes": res}), flush=True)
        return 0
    if args.telulorn:
        steps = min(args.steps, 64)
        res = novotar_bench([x for x in args.telulorn.split(",") if x], args.dtype, steps, min(args.warmup, 5), with_telulorn=True)
        print(json.dumps({"metric": "Telulorn beside Novotar and Gemma 2 at equal layer sizes: prefill and decode, random weights",
                          "unit": "tokens/s", "n_gpus": 1, "steps": steps, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
                          "data": "synthetic (uniform random token ids, random weights)", "sizes": res}), flush=True)
        return 0
    if args.novotar:
        steps = min(args.steps, 64)
        res = novotar_bench([x for x in args.novotar.split(",") if x], args.dtype, steps, min(args.warmup, 5))
        print(json.dumps({"metric": "Novotar beside Gemma 2 at equal layer sizes: prefill and decode, random weights",
                          "unit": "tokens/s", "n_gpus": 1, "steps": steps, "dtype": "bf16" if args.dtype == "bfloat16" else "fp32",
                          "data": "synthetic (uniform random token ids, random weights)", "sizes": res}), flush=True)
        return 0
    run = Run(args.preset, args.layers, args.dtype, args.ids_through_host)
    cfg, short = run.cfg, run.short

    # ---- prefill of one prompt (2,048 tokens for the headline; other lengths beside it)
    prefills = {}
    if not args.no_prefill:
        for T in [int(x) for x in args.prefill_tokens.split(",") if x]:
            if T > cfg.max_position_embeddings:
                continue
            prefills[T] = run.prefill(T)
            print(f"[bench] prefill {prefills[T]}", file=sys.stderr, flush=True)
    prefill_keys = list(prefills)

    # ---- the headline: decode at the default batch
    lens = prompt_lengths(args.prompt_lens, args.batch, args.prompt)
    context = 0 if args.prompt_lens else args.context
    dt, ctx0, ctx1 = run.decode(lens, args.steps, args.warmup, context)
    ms_step = dt / args.steps * 1e3
    gpu_ms_step = run.gpu_ms
    value = args.batch * args.steps / dt
    points, point_rooflines = {}, {}
    for b in [int(x) for x in args.points.split(",") if x]:
        psteps = args.point_steps or args.steps
        pdt, p0, p1 = run.decode(prompt_lengths(args.prompt_lens, b, args.prompt), psteps, args.warmup, context)
        points[f"decode_b{b}"] = round(b * psteps / pdt, 1)
        point_rooflines[f"decode_b{b}"] = dict(run.roofline(pdt, psteps, p0, p1), ms_per_step=round(pdt / psteps * 1e3, 4))
        print(f"[bench] decode_b{b}: {points[f'decode_b{b}']} tok/s, {point_rooflines[f'decode_b{b}']}", file=sys.stderr, flush=True)
    roof = run.roofline(dt, args.steps, ctx0, ctx1)
    weight_bytes, full_layers = run.weight_bytes, run.full_layers
    prefill_fl = {T: prefill_flops(cfg, T) for T in prefills}
    run.close()

    shapes = {}
    for name in [s for s in args.shapes.split(",") if s]:
        if name not in SHAPES:
            raise SystemExit(f"--shapes: unknown '{name}'; known: {sorted(SHAPES)}")
        t0 = time.time()
        shapes[name] = shape_run(name, args.dtype)
        print(f"[bench] shape {name} took {time.time() - t0:.1f} s", file=sys.stderr, flush=True)

    # this GPU's own rates last, so that their heat is not in the figures above; the fractions of them are added here
    peaks = {} if args.no_peaks else measured_peaks()
    if peaks:
        print(f"[bench] measured on this GPU: {peaks}", file=sys.stderr, flush=True)
        for r in [roof] + list(point_rooflines.values()):
            r["frac_of_measured_copy"] = round(r["achieved"] / peaks["copy_gbs"], 4)
        if short == "bf16":
            for T, pf in prefills.items():
                pf["frac_of_measured_matmul"] = round(prefill_fl[T] / (pf["ms"] / 1e3) / 1e12 / peaks["bf16_matmul_tflops"], 4)

    mean = lambda xs: int(round(sum(xs) / len(xs)))
    line = {
        "metric": (f"decode tok/s @ batch {args.batch}, Gemma-2-{args.preset.upper()} {short} "
                   f"(points: batch {'/'.join(str(int(x)) for x in args.points.split(',') if x) or '-'}; "
                   f"prefill tok/s @ {prefill_keys[0] if prefill_keys else 0:,} tok)"),
        "value": round(value, 1), "unit": "tokens/s", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": round(ms_step, 4), "gpu_ms_per_step": round(gpu_ms_step, 4) if gpu_ms_step else None, "higher_is_better": True, "scaling": "weak", "vs_baseline": None,
        "dtype": short, "data": "synthetic (uniform random token ids, random weights N(0, 0.02))",
        "config": {"model": f"gemma2-{args.preset}", "global_batch": args.batch, "seq_len": max(args.context, max(ctx1)),
                   "prompt_len": mean(lens), "prompt_lens": args.prompt_lens or "equal",
                   "prompt_len_min": min(lens), "prompt_len_max": max(lens),
                   "context_start": mean(ctx0), "context_end": mean(ctx1), "parallelism": "single-gpu",
                   "layers": cfg.num_hidden_layers, "layers_of_model": full_layers, "hidden": cfg.hidden_size,
                   "heads": cfg.num_attention_heads, "kv_heads": cfg.num_key_value_heads, "head_dim": cfg.head_dim,
                   "intermediate": cfg.intermediate_size, "vocab": cfg.vocab_size, "sliding_window": cfg.sliding_window,
                   "weights_gb": round(weight_bytes / 1e9, 3)},
        "prefill": prefills[prefill_keys[0]] if prefill_keys else None,
        "roofline": roof,
        "points": points,
        "point_rooflines": point_rooflines,
    }
    for T in prefill_keys[1:]:
        line[f"prefill_{T}"] = prefills[T]
    if peaks:
        line["peak_measured"] = peaks
    if shapes:
        line["shapes"] = shapes
    print(json.dumps(line), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
