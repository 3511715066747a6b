"""Plain, slow Kabapel for whole sequences: the oracle of the tests.

One function per mechanism, written from the design's equations; whole sequences, dense masks, token-by-token
recurrences, no cache, float64 by default, and no code shared with the package under test: it reads config.json
keys and safetensors tensor names itself.

The design in this file's notation (T tokens, width W, weights stored [out, in], y = x A^T):

  x        = a E[token]                                   (a: embedding.scale)
  layer    : x <- x + mix(L_1(x));  x <- x + ff(L_2(x))   (ff may be absent)
  L(x)     = (x - m) / sqrt(mean((x - m)^2) + eps) * w + b,  m = mean(x)
  logits   = Hd L_f(x)                                    (Hd: a matrix of its own)

  mixer "lightning":  q, k, v = silu of three projections, H heads of d, d and dv; per head S_t = g S_(t-1) + k_t v_t^T
             with the head's constant g, o_t = S_t^T q_t; all heads together divided by their root mean square, times a
             weight, times sigmoid(G x); output matrix.
  mixer "latent_attention":  q = Q x, per head [d plain | r turned]; D x = [c' (R) | kr' (r)], c = c' / rms(c') * w,
             kr = kr' turned, shared by the heads; keys [Uk_h c | kr], values Uv_h c; scores q.k * scale over j <= i,
             softmax, output matrix.  The r dimensions are turned in the pairs (i, i + r/2) by p * f_i, cos and sin
             times m, with stretched frequencies.  With `kv_from` c and kr are the ones another layer made.
  ff "dense":  D (max(U h, 0)^2)
  ff "moe":  p = softmax(R h) over all E + Z outputs; choice = p + correction; of `count` equal runs of neighbours the
             `keep` with the largest choice in them stay; of those the `top` largest choices serve the token with
             weights p / (sum of the chosen p + 1e-20).  The first E outputs are small feed-forwards
             D (g sigmoid(1.702 g) (u + 1)), g = min(G h, limit), u = clamp(U h, -limit, limit); the last Z give h back.
             A shared one of the same form with sizes of its own is added, times sigmoid(s . h).
"""
from __future__ import annotations

import json
import math
import os
import struct

import torch

DT = torch.float64
SUM_EPS = 1e-20


# --------------------------------------------------------------------------- small formulas

def layer_norm(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor, eps: float) -> torch.Tensor:
    m = x.mean(dim=-1, keepdim=True)
    c = x - m
    return c / torch.sqrt((c * c).mean(dim=-1, keepdim=True) + eps) * w + b


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def limited_gated_ff(h, gate, up, down, limit: float):
    g = torch.clamp(h @ gate.T, max=limit)
    u = torch.clamp(h @ up.T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def squared_relu_ff(h, up, down):
    return torch.clamp(h @ up.T, min=0.0) ** 2 @ down.T


# --------------------------------------------------------------------------- rotation

def stretched_frequencies(dims: int, base: float, scaling):
    """(f [dims/2], m): f_i = base^(-2i/dims); with scaling (factor s, original length N, fast, slow):
    D(t) = dims ln(N / (2 pi t)) / (2 ln base), lo = max(floor D(fast), 0), hi = min(ceil D(slow), dims - 1),
    r_i = clamp((i - lo) / max(hi - lo, 0.001), 0, 1), f_i <- f_i / s * r_i + f_i (1 - r_i), m = 0.1 ln s + 1."""
    i = torch.arange(dims // 2, dtype=DT)
    f = base ** (-2.0 * i / dims)
    if not scaling:
        return f, 1.0
    s, N = float(scaling["factor"]), float(scaling["original"])

    def where(turns):
        return dims * math.log(N / (2 * math.pi * turns)) / (2 * math.log(base))

    lo = max(math.floor(where(float(scaling["fast"]))), 0)
    hi = min(math.ceil(where(float(scaling["slow"]))), dims - 1)
    r = torch.clamp((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / s * r + f * (1 - r), 0.1 * math.log(s) + 1.0


def turn_halves(x: torch.Tensor, positions: torch.Tensor, rot: dict) -> torch.Tensor:
    """x: [T, heads, r], turned as a whole in the pairs (i, i + r/2)."""
    r = x.shape[-1]
    if r == 0:
        return x
    f, m = stretched_frequencies(r, float(rot["base"]), rot.get("scaling"))
    ang = positions.to(DT)[:, None] * f[None, :]
    c, s = (torch.cos(ang) * m)[:, None, :], (torch.sin(ang) * m)[:, None, :]
    u, v = x[..., :r // 2], x[..., r // 2:]
    return torch.cat([u * c - v * s, v * c + u * s], dim=-1)


# --------------------------------------------------------------------------- mixers

def constant_decay_scan(q, k, v, decay, S0=None):
    """q, k: [T, H, d]; v: [T, H, dv]; decay: [H]: S <- decay S + k v^T; o = S^T q.  Returns o [T, H, dv] and S."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype) if S0 is None else S0.clone()
    o = torch.empty_like(v)
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(dim=1)
    return o, S


def lightning_mixer(h, p, m, eps, S0=None, return_state=False):
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, v = (silu(h @ p[n].T) for n in ("q", "k", "v"))
    decay = torch.as_tensor(m["decay"], dtype=h.dtype)
    o, S = constant_decay_scan(q.view(T, H, d), k.view(T, H, d), v.view(T, H, dv), decay, S0)
    o = unit_rms(o.reshape(T, H * dv), eps) * p["norm"] * torch.sigmoid(h @ p["g"].T)
    y = o @ p["o"].T
    return (y, S) if return_state else y


def latent_rows(h, p, m, eps, positions):
    """What a layer makes and caches: the latent c [T, R] and the turned shared key part kr [T, r]."""
    R, r = m["kv_rank"], m["rot_dim"]
    rows = h @ p["dkv"].T
    c = unit_rms(rows[:, :R], eps) * p["dkv.norm"]
    return c, turn_halves(rows[:, R:].view(rows.shape[0], 1, r), positions, m.get("rot"))[:, 0]


def latent_mixer(h, p, m, positions, latents):
    """latents: (c, kr) of the whole sequence, this layer's own or another's."""
    T, H, d, r, dv = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    q = (h @ p["q"].T).view(T, H, d + r)
    qr = turn_halves(q[..., d:], positions, m.get("rot"))
    c, kr = latents
    n = c.shape[0]
    seen = torch.arange(n)[None, :] <= positions[:, None]        # the keys stand at positions 0 .. n - 1
    uk, uv = p["uk"].view(H, d, -1), p["uv"].view(H, dv, -1)
    out = torch.empty(T, H, dv, dtype=h.dtype)
    for j in range(H):
        s = (q[:, j, :d] @ (c @ uk[j].T).T + qr[:, j] @ kr.T) * m["scale"]
        out[:, j] = torch.softmax(s.masked_fill(~seen, -math.inf), dim=-1) @ (c @ uv[j].T)
    return out.reshape(T, H * dv) @ p["o"].T


# --------------------------------------------------------------------------- routed feed-forward

def route(z, correction, router):
    """z: [T, n] router outputs; returns dense weights [T, n], zero where an output does not serve the token."""
    T, n = z.shape
    p = torch.softmax(z, dim=-1)
    choice = p + correction
    groups = router.get("groups")
    if groups:
        count, keep = groups["count"], groups["keep"]
        best = choice.view(T, count, n // count).max(dim=-1).values
        stay = torch.zeros(T, count, dtype=torch.bool).scatter_(1, torch.topk(best, keep, dim=-1).indices, True)
        choice = choice.masked_fill(~stay.repeat_interleave(n // count, dim=1), -math.inf)
    idx = torch.topk(choice, router["top"], dim=-1).indices
    chosen = p.gather(1, idx)
    return torch.zeros_like(p).scatter_(1, idx, chosen / (chosen.sum(dim=-1, keepdim=True) + SUM_EPS))


def routed_ff(h, p, mlp):
    router = mlp["router"]
    E, limit = router["experts"], float(mlp["expert"]["limit"])
    w = route(h @ p["router"].T, p["correction"], router)
    out = w[:, E:].sum(dim=-1, keepdim=True) * h                 # the outputs beyond E give the input back
    for e in range(E):
        rows = torch.nonzero(w[:, e])[:, 0]
        if rows.numel():
            y = limited_gated_ff(h[rows], p[f"e{e}.gate"], p[f"e{e}.up"], p[f"e{e}.down"], limit)
            out[rows] += w[rows, e:e + 1] * y
    sh = mlp.get("shared")
    if sh is not None:
        y = limited_gated_ff(h, p["shared.gate"], p["shared.up"], p["shared.down"], float(sh["limit"]))
        out = out + torch.sigmoid(h @ p["shared.sg"].T) * y
    return out


def feed_forward(h, p, mlp):
    if mlp.get("kind", "dense") == "dense":
        return squared_relu_ff(h, p["up"], p["down"])
    return routed_ff(h, p, mlp)


# --------------------------------------------------------------------------- the model

def sub(p: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in p.items() if k.startswith(prefix)}


def forward(config: dict, tensors: dict, tokens, return_layers: bool = False):
    """Logits [T, vocab] of a whole sequence (and, if asked, the stream after every layer [layers, T, W])."""
    eps = config["norm"]["eps"]
    tok = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(tok.numel())
    x = tensors["embed"][tok] * config["embedding"]["scale"]
    made, after = {}, []
    for i, layer in enumerate(config["layers"]):
        p, m = sub(tensors, f"l{i}."), layer["mixer"]
        pm = sub(p, "mix.")
        h = layer_norm(x, p["norm1"], p["norm1.b"], eps)
        if layer["type"] == "lightning":
            y = lightning_mixer(h, pm, m, eps)
        elif layer["type"] == "latent_attention":
            src = m.get("kv_from")
            if src is None:
                made[i] = latent_rows(h, pm, m, eps, positions)
            y = latent_mixer(h, pm, m, positions, made[i if src is None else src])
        else:
            raise ValueError(layer["type"])
        x = x + y
        if layer.get("mlp") is not None:
            x = x + feed_forward(layer_norm(x, p["norm2"], p["norm2.b"], eps), sub(p, "mlp."), layer["mlp"])
        after.append(x)
    logits = layer_norm(x, tensors["final.norm"], tensors["final.norm.b"], eps) @ tensors["head"].T
    return (logits, torch.stack(after)) if return_layers else logits


# --------------------------------------------------------------------------- files

_DTYPES = {"F32": torch.float32, "BF16": torch.bfloat16, "I32": torch.int32, "F64": torch.float64}


def read_safetensors(path: str) -> dict:
    with open(path, "rb") as f:
        (n,) = struct.unpack("<Q", f.read(8))
        header = json.loads(f.read(n))
        data = f.read()
    out = {}
    for name, info in header.items():
        if name == "__metadata__":
            continue
        a, b = info["data_offsets"]
        t = torch.frombuffer(bytearray(data[a:b]), dtype=_DTYPES[info["dtype"]]).reshape(info["shape"])
        out[name] = t.to(DT) if t.is_floating_point() else t
    return out


class PlainKabapel:
    def __init__(self, config: dict, tensors: dict):
        self.config, self.tensors = config, tensors

    @classmethod
    def from_folder(cls, folder: str) -> "PlainKabapel":
        with open(os.path.join(folder, "config.json")) as f:
            config = json.load(f)
        return cls(config, read_safetensors(os.path.join(folder, "model.safetensors")))

    def forward(self, tokens, return_layers: bool = False):
        return forward(self.config, self.tensors, tokens, return_layers)

    def greedy(self, prompt, n: int):
        seq, out = list(prompt), []
        for _ in range(n):
            out.append(int(torch.argmax(self.forward(seq)[-1])))
            seq.append(out[-1])
        return out
