"""Plain, slow Vazilorn for whole sequences: the oracle of the tests.

One function per mechanism, written from the design's equations; whole sequences, dense masks, no cache, float64 by
default, and no code shared with the package under test: it reads config.json keys and safetensors tensor names itself.

The design in this file's notation (T tokens, width W, weights stored [out, in], y = x A^T):

  x        = E[token]
  layer    : x <- x + D_1b(mix(D_1(x)));  x <- x + D_2b(ff(D_2(x)))    (ff may be absent)
  D(x)     = tanh(a x) * w + b, element by element (a: one number)
  logits   = Hd D_f(x)                                                  (Hd: a matrix of its own)

  mixer "attention":  q = Q h (H heads of d), k = K h (G heads of d), v = V h (G heads of dv); every q and k head divided
             by its root mean square and multiplied by a weight of d that the heads share; then the first R dimensions
             turned in the pairs (2i, 2i + 1) by p * f_i; scores s = q.k * scale over the keys 0 <= i - j < size;
             weights exp(s_j) / (exp(sink_h) + sum_j exp(s_j)); output matrix.
             f_i = base^(-2i/R); with scaling (factor, low, high, original) and turns t = original f / (2 pi):
             f where t > high, f / factor where t < low, between them m f + (1 - m) f / factor, m = (t - low) / (high - low).
  ff "dense":  Dn (gelu_tanh(Gt h) * (U h))
  ff "moe":  s = sigmoid(R h); choice = s + correction; of `count` equal runs of neighbours the `keep` whose two largest
             choices sum highest stay; of those the `top` largest choices serve the token with weights
             scale * s / (sum of the chosen s + 1e-20).  Each is Dn (silu(Gt h) * (U h)); a shared one is added as it is.
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

def dynamic_tanh(x: torch.Tensor, alpha, w: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    return torch.tanh(alpha * x) * w + b


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def gated_ff(h, gate, up, down, act):
    return (act(h @ gate.T) * (h @ up.T)) @ down.T


# --------------------------------------------------------------------------- rotation

def banded_frequencies(dims: int, base: float, scaling) -> torch.Tensor:
    """f [dims/2], stretched band by band by how often a frequency turns within `original` positions."""
    f = base ** (-2.0 * torch.arange(dims // 2, dtype=DT) / dims)
    if not scaling:
        return f
    factor, low, high, original = (float(scaling[k]) for k in ("factor", "low", "high", "original"))
    out = f.clone()
    for i, fi in enumerate(f.tolist()):
        length = 2.0 * math.pi / fi
        if length < original / high:
            continue
        if length > original / low:
            out[i] = fi / factor
        else:
            m = (original / length - low) / (high - low)
            out[i] = (1.0 - m) * fi / factor + m * fi
    return out


def turn_pairs(x: torch.Tensor, positions: torch.Tensor, f: torch.Tensor) -> torch.Tensor:
    """x: [T, heads, d]; dimensions 2i and 2i + 1 are a pair for i < len(f); the rest pass."""
    n = 2 * f.numel()
    ang = positions.to(f.dtype)[:, None] * f[None, :]
    c, s = torch.cos(ang).to(x.dtype)[:, None, :], torch.sin(ang).to(x.dtype)[:, None, :]
    out = x.clone()
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out[..., 0:n:2] = u * c - v * s
    out[..., 1:n:2] = v * c + u * s
    return out


# --------------------------------------------------------------------------- attention

def window_mask(positions: torch.Tensor, n_keys: int, size) -> torch.Tensor:
    """[T, n_keys]: which of the keys at positions 0 .. n_keys - 1 each query sees."""
    back = positions[:, None] - torch.arange(n_keys)[None, :]
    return (back >= 0) if size is None else (back >= 0) & (back < size)


def sink_softmax(scores: torch.Tensor, mask: torch.Tensor, sink) -> torch.Tensor:
    s = scores.masked_fill(~mask, -math.inf)
    top = torch.maximum(s.max(dim=-1, keepdim=True).values, torch.as_tensor(sink, dtype=s.dtype))
    e = torch.exp(s - top)
    return e / (torch.exp(sink - top) + e.sum(dim=-1, keepdim=True))


def attention_mixer(h, p, m, eps, positions):
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = unit_rms((h @ p["q"].T).view(T, H, d), eps) * p["q.norm"]
    k = unit_rms((h @ p["k"].T).view(T, G, d), eps) * p["k.norm"]
    v = (h @ p["v"].T).view(T, G, dv)
    rot = m.get("rot")
    if rot:
        f = banded_frequencies(rot["dims"], float(rot["base"]), rot.get("scaling"))
        q, k = turn_pairs(q, positions, f), turn_pairs(k, positions, f)
    mask = window_mask(positions, T, (m.get("mask") or {}).get("size"))
    out = torch.empty(T, H, dv, dtype=h.dtype)
    for j in range(H):
        g = j // (H // G)
        out[:, j] = sink_softmax((q[:, j] @ k[:, g].T) * m["scale"], mask, p["sink"][j]) @ v[:, g]
    return out.reshape(T, H * dv) @ p["o"].T


# --------------------------------------------------------------------------- routed feed-forward

def route(z, correction, router):
    """z: [T, E] router outputs; returns dense weights [T, E], zero where an expert does not serve the token."""
    T, E = z.shape
    s = torch.sigmoid(z)
    choice = s + correction
    groups = router.get("groups")
    if groups:
        count, keep = groups["count"], groups["keep"]
        parts = choice.view(T, count, E // count)
        two = torch.topk(parts, min(2, E // count), dim=-1).values.sum(dim=-1)
        stay = torch.zeros(T, count, dtype=torch.bool).scatter_(1, torch.topk(two, keep, dim=-1).indices, True)
        choice = choice.masked_fill(~stay.repeat_interleave(E // count, dim=1), -math.inf)
    idx = torch.topk(choice, router["top"], dim=-1).indices
    chosen = s.gather(1, idx)
    w = chosen / (chosen.sum(dim=-1, keepdim=True) + SUM_EPS) * router.get("scale", 1.0)
    return torch.zeros_like(s).scatter_(1, idx, w)


def routed_ff(h, p, mlp):
    w = route(h @ p["router"].T, p["correction"], mlp["router"])
    out = torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        rows = torch.nonzero(w[:, e])[:, 0]
        if rows.numel():
            out[rows] += w[rows, e:e + 1] * gated_ff(h[rows], p[f"e{e}.gate"], p[f"e{e}.up"], p[f"e{e}.down"], silu)
    if mlp.get("shared") is not None:
        out = out + gated_ff(h, p["shared.gate"], p["shared.up"], p["shared.down"], silu)
    return out


def feed_forward(h, p, mlp):
    if mlp.get("kind", "dense") == "dense":
        return gated_ff(h, p["gate"], p["up"], p["down"], gelu_tanh)
    return routed_ff(h, p, mlp)


# --------------------------------------------------------------------------- the model

def sub(p: dict, prefix: str) -> dict:
    return {k[len(prefix):]: v for k, v in p.items() if k.startswith(prefix)}


def named_norm(x, p: dict, name: str):
    return dynamic_tanh(x, p[name + ".alpha"], p[name], p[name + ".b"])


def forward(config: dict, tensors: dict, tokens, return_layers: bool = False):
    """Logits [T, vocab] of a whole sequence (and, if asked, the stream after every layer [layers, T, W])."""
    eps = config["norm"]["eps"]
    tok = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(tok.numel())
    x = tensors["embed"][tok]
    after = []
    for i, layer in enumerate(config["layers"]):
        p = sub(tensors, f"l{i}.")
        if layer["type"] != "attention":
            raise ValueError(layer["type"])
        y = attention_mixer(named_norm(x, p, "norm1"), sub(p, "mix."), layer["mixer"], eps, positions)
        x = x + named_norm(y, p, "norm1b")
        if layer.get("mlp") is not None:
            y = feed_forward(named_norm(x, p, "norm2"), sub(p, "mlp."), layer["mlp"])
            x = x + named_norm(y, p, "norm2b")
        after.append(x)
    logits = named_norm(x, tensors, "final.norm") @ tensors["head"].T
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


class PlainVazilorn:
    def __init__(self, config: dict, tensors: dict):
        self.config, self.tensors = config, tensors

    @classmethod
    def from_folder(cls, folder: str) -> "PlainVazilorn":
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
