"""Vazilorn: typed configuration from config.json, and its plan.

A decoder whose layers are written out one by one in config.json (`layers`: per layer its `type`, the sizes of its
`mixer` and its `mlp`, which may be null), with a norm ahead of every sublayer and one behind it:
x += D_1b(mixer(D_1(x))); x += D_2b(ff(D_2(x))).  The norm is a dynamic tanh, tanh(a x) * w + b, which computes nothing over
the row.  The output head has a matrix of its own.  One mixer type:

  "attention"  grouped-query attention without biases; every q and k head divided by its root mean square and multiplied by
               a weight of the head's size that the heads share, then rotated over its first `rot.dims` dimensions in
               neighbouring pairs (2i, 2i + 1), with frequencies stretched by bands (`rot.scaling`: factor, low, high,
               original); scores times `scale`; a window of the last `mask.size` positions; a learned sink number a head
               in the softmax's denominator.

The feed-forward is gated: dense with the tanh form of GELU, or routed with silu: `router.experts` small ones scored by a
sigmoid each, a stored correction for the choice, `router.groups` (count, keep) counted by the sum of their two largest
choices, the `router.top` best, their scores divided by the sum and times `router.scale`; and a shared one (`shared`) that
serves every token.

Everything here is data for the builder: which registered part, with which constants, under which tensor names.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Mapping, Tuple

from .novotar import _obj
from .plan import ConfigError, LayerPlan, ModelPlan, PartSpec, ScheduleEntry, read_key, require
from .vifirax import _plain

DEFAULT_MAX_POSITIONS = 65536        # the design has no position limit of its own; tables are sized by this
MIXER_TYPES = ("attention",)
SCALING_KEYS = ("factor", "low", "high", "original")


def _read_rot(m: Mapping[str, Any], where: str, dim: int):
    rot = _obj(m, "rot", where, optional=True)
    if rot is None:
        return None
    sc = _obj(rot, "scaling", where + "rot: ", optional=True)
    return {"base": read_key(rot, "base", float), "dims": read_key(rot, "dims", int, dim),
            "scaling": None if sc is None else {k: read_key(sc, k, float) for k in SCALING_KEYS}}


def _read_mlp(l: Mapping[str, Any], where: str):
    mlp = _obj(l, "mlp", where, optional=True)
    if mlp is None:
        return None
    where += "mlp: "
    kind = read_key(mlp, "kind", str, "dense")
    require(kind in ("dense", "moe"), f"{where}kind '{kind}' has no feed-forward here (known: 'dense', 'moe')")
    if kind == "dense":
        return {"kind": kind, "ff": read_key(mlp, "ff", int)}
    router, shared = _obj(mlp, "router", where), _obj(mlp, "shared", where, optional=True)
    groups = _obj(router, "groups", where + "router: ", optional=True)
    return {"kind": kind, "expert": {"ff": read_key(_obj(mlp, "expert", where), "ff", int)},
            "shared": None if shared is None else {"ff": read_key(shared, "ff", int)},
            "router": {"experts": read_key(router, "experts", int), "top": read_key(router, "top", int),
                       "scale": read_key(router, "scale", float, 1.0),
                       "groups": None if groups is None else {"count": read_key(groups, "count", int),
                                                              "keep": read_key(groups, "keep", int)}}}


@dataclass(frozen=True)
class VazilornConfig:
    vocab: int
    width: int
    layers: Tuple[Mapping[str, Any], ...]          # as config.json gives them, validated
    norm_eps: float = 1e-6
    max_positions: int = DEFAULT_MAX_POSITIONS
    torch_dtype: str = "bfloat16"

    architecture = "Vazilorn"

    # ------------------------------------------------------------------ reading
    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "VazilornConfig":
        raw_layers = d.get("layers")
        if not isinstance(raw_layers, (list, tuple)) or not raw_layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        norm = _obj(d, "norm", "", optional=True) or {}
        cfg = cls(vocab=read_key(d, "vocab", int), width=read_key(d, "width", int),
                  layers=tuple(cls._read_layer(i, l) for i, l in enumerate(raw_layers)),
                  norm_eps=read_key(norm, "eps", float, 1e-6),
                  max_positions=read_key(d, "max_positions", int, DEFAULT_MAX_POSITIONS),
                  torch_dtype=read_key(d, "torch_dtype", str, "bfloat16"))
        cfg.validate()
        return cfg

    @staticmethod
    def _read_layer(i: int, l: Any) -> Dict[str, Any]:
        where = f"layers[{i}]: "
        if not isinstance(l, Mapping):
            raise ConfigError(f"config.json: {where}must be an object")
        kind = read_key(l, "type", str)
        require(kind in MIXER_TYPES, f"{where}type '{kind}' has no mixer here (known: {', '.join(MIXER_TYPES)})")
        m = _obj(l, "mixer", where)
        mw = where + "mixer: "
        heads, dim = read_key(m, "heads", int), read_key(m, "dim", int)
        mask = _obj(m, "mask", mw, optional=True)
        return {"type": kind, "mlp": _read_mlp(l, where),
                "mixer": {"heads": heads, "kv_heads": read_key(m, "kv_heads", int, heads), "dim": dim,
                          "vdim": read_key(m, "vdim", int, dim), "scale": read_key(m, "scale", float), "rot": _read_rot(m, mw, dim),
                          "mask": None if mask is None else {"size": read_key(mask, "size", int)}}}

    def validate(self) -> None:
        require(self.vocab >= 1 and self.width >= 1, "vocab and width must be at least 1")
        require(self.norm_eps > 0, "norm.eps must be positive")
        require(self.max_positions >= 1, "max_positions must be at least 1")
        for i, l in enumerate(self.layers):
            m, where = l["mixer"], f"layers[{i}].mixer"
            require(min(m["heads"], m["kv_heads"], m["dim"], m["vdim"]) >= 1, f"{where}: heads, kv_heads, dim and vdim must be at least 1")
            require(m["heads"] % m["kv_heads"] == 0, f"{where}.kv_heads must divide heads")
            require(m["mask"] is None or m["mask"]["size"] >= 1, f"{where}.mask.size must be at least 1")
            rot = m["rot"]
            require(rot is None or (rot["base"] > 0 and 0 <= rot["dims"] <= m["dim"] and rot["dims"] % 2 == 0),
                    f"{where}.rot: base must be positive, dims even and at most dim")
            sc = rot["scaling"] if rot else None
            require(sc is None or (min(sc.values()) > 0 and sc["low"] < sc["high"]),
                    f"{where}.rot.scaling: factor, low, high and original must be positive, and low below high")
            self._validate_mlp(l["mlp"], f"layers[{i}].mlp")
        require(self.torch_dtype in ("bfloat16", "float32"),
                f"torch_dtype must be 'bfloat16' or 'float32', found '{self.torch_dtype}'")

    @staticmethod
    def _validate_mlp(mlp, where: str) -> None:
        if mlp is None:
            return
        if mlp["kind"] == "dense":
            require(mlp["ff"] >= 1, f"{where}.ff must be at least 1")
            return
        r, g = mlp["router"], mlp["router"]["groups"]
        require(1 <= r["top"] <= r["experts"] and r["scale"] > 0, f"{where}.router: 1 <= top <= experts, and scale positive")
        require(mlp["expert"]["ff"] >= 1 and (mlp["shared"] is None or mlp["shared"]["ff"] >= 1),
                f"{where}: expert.ff and shared.ff must be at least 1")
        if g is not None:
            require(g["count"] >= 1 and r["experts"] % g["count"] == 0, f"{where}.router.groups.count must divide experts")
            require(1 <= g["keep"] <= g["count"] and g["keep"] * (r["experts"] // g["count"]) >= r["top"],
                    f"{where}.router.groups: 1 <= keep <= count, and the kept groups must hold at least `top` experts")

    def to_dict(self) -> dict:
        strip = lambda d: {k: strip(v) if isinstance(v, Mapping) else v for k, v in d.items() if v is not None}
        layers = [{"type": l["type"], "mixer": strip(_plain(l["mixer"])), "mlp": None if l["mlp"] is None else strip(_plain(l["mlp"]))}
                  for l in self.layers]
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "layers": layers, "max_positions": self.max_positions, "torch_dtype": self.torch_dtype}

    # ------------------------------------------------------------------ the plan
    def _attention(self, m) -> PartSpec:
        names = {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm", "sink": "sink"}
        return PartSpec("attention", {
            "hidden_size": self.width, "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "head_dim": m["dim"],
            "value_head_dim": m["vdim"], "scale": m["scale"], "softcap": None, "window": None if m["mask"] is None else m["mask"]["size"],
            "position": _rot_key(m), "sink": True, "qk_norm": "head", "qk_norm_eps": self.norm_eps, "tensor_names": names}, "mix")

    def _ff(self, mlp) -> PartSpec:
        if mlp["kind"] == "dense":
            return PartSpec("gated_mlp", {"hidden_size": self.width, "intermediate_size": mlp["ff"], "activation": "gelu_tanh",
                                          "tensor_names": {"gate": "gate", "up": "up", "down": "down"}}, "mlp")
        r, sh = mlp["router"], mlp["shared"]
        return PartSpec("expert_mlp", {
            "hidden_size": self.width, "intermediate_size": mlp["expert"]["ff"], "experts": r["experts"], "top": r["top"],
            "activation": "silu", "scoring": "sigmoid", "group_best": 2, "weight_scale": r["scale"],
            "groups": None if r["groups"] is None else (r["groups"]["count"], r["groups"]["keep"]),
            "shared": None if sh is None else {"intermediate_size": sh["ff"], "activation": "silu"}, "shared_gate": False}, "mlp")

    def plan(self) -> ModelPlan:
        W = self.width
        norm = lambda name: PartSpec("dynamic_tanh", {"dim": W, "tensor_name": "", "bias_name": "b", "alpha_name": "alpha"}, name)
        layers, positions = [], {}
        for i, l in enumerate(self.layers):
            m = l["mixer"]
            if _rot_key(m) is not None:
                positions[_rot_key(m)] = PartSpec("rope_pairs", {
                    "dim": m["dim"], "theta": m["rot"]["base"], "rotary_dim": m["rot"]["dims"], "value_dim": None,
                    "max_positions": self.max_positions, "interleaved": True, "scaling": m["rot"]["scaling"]})
            norms = {"pre_mixer": norm("norm1"), "post_mixer": norm("norm1b")}
            if l["mlp"] is not None:
                norms.update(pre_ff=norm("norm2"), post_ff=norm("norm2b"))
            layers.append(LayerPlan(block="sandwich", mixer=self._attention(m), feed_forward=None if l["mlp"] is None else self._ff(l["mlp"]),
                                    norms=norms, prefix=f"l{i}."))
        return ModelPlan(
            vocab_size=self.vocab, hidden_size=W, max_positions=self.max_positions,
            # (nothing in this design brings the stream to a size of its own: random rows of order one)
            embedding=PartSpec("embedding", {"vocab_size": self.vocab, "dim": W, "scale": 1.0, "tensor_name": "", "init_std": 1.0}, "embed"),
            positions=positions, layers=tuple(layers), schedule=tuple(ScheduleEntry(i) for i in range(len(layers))),
            final_norm=norm("final.norm"),
            head=PartSpec("lm_head", {"vocab_size": self.vocab, "dim": W, "softcap": None, "tensor_name": ""}, "head"),
            stop_token_ids=())


def _rot_key(m):
    """One table set per distinct (head size, rotated width, base, scaling); None without a rotation."""
    rot = m["rot"]
    if rot is None or not rot["dims"]:
        return None
    sc = rot["scaling"]
    tail = "" if sc is None else "_" + "_".join(repr(sc[k]) for k in SCALING_KEYS)
    return f"pairs_{m['dim']}_{rot['dims']}_{rot['base']!r}{tail}"
