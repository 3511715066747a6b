"""The lightning-attention mixer: linear attention whose state per head is a matrix with one constant decay.

With the mixer's input h: q = silu(W_q h) and k = silu(W_k h) (heads x d), v = silu(W_v h) (heads x dv), and per head with
its decay g
    S_t = g S_(t-1) + k_t v_t^T,    o_t = S_t^T q_t.
The heads' o together are divided by their root mean square (eps inside the root), multiplied by a weight and by
sigmoid(W_g h), and go through the output matrix.  S starts at zero, lives in 32-bit in the cache's state rows, one per
slot, and is carried from step to step; the powers of the decays are made on the host in 64-bit and kept in 32-bit; the
recurrence, its read-outs and the norm are 32-bit on both paths.

Head count, head sizes, the decays (one number a head) and the norm's eps are constructor arguments.  One fused matrix
gives [q | k | v | g].  Steps of many tokens run its rows as two products, the first with silu in its epilogue; steps of
few tokens run one product and the recurrence's kernel applies silu on the way in.
"""
from __future__ import annotations

from typing import Dict, Optional, Sequence

import torch

from ..hip import ops
from .base import MIXERS, CacheNeed, ParamSpec, Part, Precision, StateNeed
from .linear import Linear

_DEFAULT_NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "norm": "norm"}
TWO_PRODUCTS_FROM_TOKENS = 65        # below, a second launch costs more than silu in the recurrence's kernel


@MIXERS.register("lightning")
class LightningAttention(Part):
    graph_safe = True
    graph_safe_prompts = True        # the kernels find each sequence's rows and state row on the device

    def __init__(self, precision: Precision, positions: dict, *, hidden_size: int, num_heads: int, head_dim: int,
                 decay: Sequence[float], value_head_dim: Optional[int] = None, norm_eps: float = 1e-6,
                 tensor_names: Optional[Dict[str, str]] = None):
        self.precision = precision
        self.W, self.nH, self.d = hidden_size, num_heads, head_dim
        self.dv = head_dim if value_head_dim is None else int(value_head_dim)
        if min(self.nH, self.d, self.dv) < 1 or self.d > ops.LIGHTNING_MAX_KEY_DIM:
            raise ValueError(f"lightning: heads {self.nH}, head sizes {self.d} and {self.dv}: at least 1, keys at most "
                             f"{ops.LIGHTNING_MAX_KEY_DIM}")
        if len(decay) != self.nH:
            raise ValueError(f"lightning: {len(decay)} decays for {self.nH} heads")
        self.eps = float(norm_eps)
        self.decay = torch.tensor([float(g) for g in decay], dtype=torch.float64)
        self.names = dict(_DEFAULT_NAMES, **(tensor_names or {}))
        self.qk, self.vw = self.nH * self.d, self.nH * self.dv
        self.cols = (0, self.qk, 2 * self.qk)                                  # q, k, v
        self.g_col = 2 * self.qk + self.vw
        self.proj = Linear(hidden_size, self.g_col + self.vw, precision)
        self.qkv_part: Optional[Linear] = None
        self.g_part: Optional[Linear] = None
        self.o = Linear(self.vw, hidden_size, precision)
        self.norm_w: Optional[torch.Tensor] = None
        self.powers: Optional[torch.Tensor] = None
        self._parts: Dict[str, torch.Tensor] = {}

    def param_specs(self) -> Dict[str, ParamSpec]:
        n = self.names
        return {n["q"]: ParamSpec((self.qk, self.W)), n["k"]: ParamSpec((self.qk, self.W)),
                n["v"]: ParamSpec((self.vw, self.W)), n["g"]: ParamSpec((self.vw, self.W)),
                n["o"]: ParamSpec((self.W, self.vw)), n["norm"]: ParamSpec((self.vw,), init_std=0.1)}

    def cache_need(self) -> CacheNeed:
        return CacheNeed(state=(StateNeed("S", (self.nH, self.d, self.dv)),))

    def assign(self, name: str, tensor: torch.Tensor) -> None:
        n = self.names
        if name == n["o"]:
            self.o.load(tensor)
        elif name == n["norm"]:
            self.norm_w = tensor.float().contiguous()
        elif name in (n["q"], n["k"], n["v"], n["g"]):
            self._parts[name] = tensor
        else:
            raise KeyError(name)

    def finalize(self) -> None:
        mats = [self.precision.matrix(self._parts.pop(self.names[c])) for c in ("q", "k", "v", "g")]
        if len({m.dtype for m in mats}) > 1:
            mats = [m.float() for m in mats]
        self.proj.load(torch.cat(mats, dim=0))
        self.qkv_part = self.proj.rows(0, self.g_col, epilogue=ops.EPI_SOFTCAP, epi_param=ops.UNARY_SILU)
        self.g_part = self.proj.rows(self.g_col, self.g_col + self.vw)
        n = torch.arange(ops.LIGHTNING_CHUNK + 1, dtype=torch.float64)
        self.powers = (self.decay[:, None] ** n[None, :]).to(torch.float32).to(self.norm_w.device).contiguous()

    def weight_bytes(self) -> int:
        return self.proj.nbytes() + self.o.nbytes()

    @property
    def accepts_fragment_activations(self) -> bool:
        return self.proj.accepts_fragment_input

    def forward(self, x, ctx, cache) -> torch.Tensor:
        T, act, dev = x.shape[0], self.precision.act, self.powers.device
        two = T >= TWO_PRODUCTS_FROM_TOKENS and self.qkv_part is not None and self.g_part is not None
        if two:
            rows, gate, g_col = self.qkv_part(x, act), self.g_part(x, act), 0
        else:
            rows = gate = self.proj(x, act)
            g_col = self.g_col
        o = torch.empty((T, self.vw), dtype=torch.float32, device=dev)
        ops.lightning(rows, self.cols, self.powers, o, ctx, cache.state["S"], heads=self.nH, head_dim=self.d,
                      value_head_dim=self.dv, silu=not two)
        out = torch.empty((T, self.vw), dtype=act, device=dev)
        ops.norm_gate(o, self.norm_w, out, parts=1, eps=self.eps, weight_shared=False, gate=gate, gate_col=g_col, gate_act="sigmoid")
        return self.o(out, torch.float32, allow_partials=True)
