"""Kabapel: typed configuration from config.json, and its plan.

A pre-norm decoder whose layers are written out one by one in config.json (`layers`: per layer its `type`, the sizes of
its `mixer` and its `mlp`, which may be null): x += mixer(N_1(x)); x += ff(N_2(x)), N a layer norm with weight and bias.
The embedding is multiplied by `embedding.scale`; the output head has a matrix of its own.  Two mixer types:

  "lightning"         linear attention: q, k and v through silu, per head a matrix state with a constant decay (`decay`, a
                      number a head); the heads together are normed, weighted and gated by a sigmoid.
  "latent_attention"  queries straight from the mixer's input, a head's query [`dim` plain | `rot_dim` rotated]; keys and
                      values of all heads made from one normed latent of `kv_rank` numbers a token, beside `rot_dim` rotated
                      key dimensions that all heads share; rotation in halves (i, i + rot_dim/2) with frequencies
                      stretched by `rot.scaling` (factor, original, fast, slow) and cos and sin multiplied by
                      0.1 ln(factor) + 1; every earlier key visible.  The cache holds the latent and the rotated part only.
                      With `kv_from: j` the layer reads the rows that layer j cached, through maps of its own.

The feed-forward is dense, down(max(up h, 0)^2), or routed: `router.experts` small ones with the bounded gated form
(`expert.limit`) and `router.identity` that give their input back; softmax scores over all of them, a stored correction
for the choice, `router.groups` (count, keep), the `router.top` best; and a shared one (`shared`) with a sigmoid gate.

Everything here is data for the builder: which registered part, with which constants, under which tensor names.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Mapping, Tuple

from .novotar import _obj
from .plan import ConfigError, LayerPlan, ModelPlan, PartSpec, ScheduleEntry, read_key, require
from .vifirax import _plain, _read_rot, _rot_name

DEFAULT_MAX_POSITIONS = 65536        # the design has no position limit of its own; tables are sized by this
MIXER_TYPES = ("lightning", "latent_attention")


def _read_gated(d: Mapping[str, Any], key: str, where: str, optional: bool = False):
    m = _obj(d, key, where, optional=optional)
    return None if m is None else {"ff": read_key(m, "ff", int), "limit": read_key(m, "limit", float)}


def _read_mlp(l: Mapping[str, Any], where: str):
    mlp = _obj(l, "mlp", where, optional=True)
    if mlp is None:
        return None
    where += "mlp: "
    kind = read_key(mlp, "kind", str, "dense")
    require(kind in ("dense", "moe"), f"{where}kind '{kind}' has no feed-forward here (known: 'dense', 'moe')")
    if kind == "dense":
        return {"kind": kind, "ff": read_key(mlp, "ff", int)}
    router = _obj(mlp, "router", where)
    groups = _obj(router, "groups", where + "router: ", optional=True)
    return {"kind": kind, "expert": _read_gated(mlp, "expert", where), "shared": _read_gated(mlp, "shared", where, optional=True),
            "router": {"experts": read_key(router, "experts", int), "top": read_key(router, "top", int),
                       "identity": read_key(router, "identity", int, 0),
                       "groups": None if groups is None else {"count": read_key(groups, "count", int),
                                                              "keep": read_key(groups, "keep", int)}}}


@dataclass(frozen=True)
class KabapelConfig:
    vocab: int
    width: int
    layers: Tuple[Mapping[str, Any], ...]          # as config.json gives them, validated
    norm_eps: float = 1e-6
    embedding_scale: float = 1.0
    max_positions: int = DEFAULT_MAX_POSITIONS
    torch_dtype: str = "bfloat16"

    architecture = "Kabapel"

    # ------------------------------------------------------------------ reading
    @classmethod
    def from_dict(cls, d: Mapping[str, Any]) -> "KabapelConfig":
        raw_layers = d.get("layers")
        if not isinstance(raw_layers, (list, tuple)) or not raw_layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        norm = _obj(d, "norm", "", optional=True) or {}
        embedding = _obj(d, "embedding", "", optional=True) or {}
        cfg = cls(vocab=read_key(d, "vocab", int), width=read_key(d, "width", int),
                  layers=tuple(cls._read_layer(i, l) for i, l in enumerate(raw_layers)),
                  norm_eps=read_key(norm, "eps", float, 1e-6), embedding_scale=read_key(embedding, "scale", float, 1.0),
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
        out: Dict[str, Any] = {"heads": heads, "dim": dim, "vdim": read_key(m, "vdim", int, dim)}
        if kind == "lightning":
            decay = m.get("decay")
            ok = isinstance(decay, (list, tuple)) and all(isinstance(g, (int, float)) and not isinstance(g, bool) for g in decay)
            require(ok, f"{mw}decay must be a list of numbers, one a head")
            out["decay"] = [float(g) for g in decay]
        else:
            out.update({"rot_dim": read_key(m, "rot_dim", int), "kv_rank": read_key(m, "kv_rank", int),
                        "scale": read_key(m, "scale", float), "kv_from": read_key(m, "kv_from", int, None, allow_none=True)})
            out["rot"] = _read_rot(m, mw, out["rot_dim"])
        return {"type": kind, "mixer": out, "mlp": _read_mlp(l, where)}

    def validate(self) -> None:
        require(self.vocab >= 1 and self.width >= 1, "vocab and width must be at least 1")
        require(self.norm_eps > 0, "norm.eps must be positive")
        require(self.max_positions >= 1, "max_positions must be at least 1")
        for i, l in enumerate(self.layers):
            m, where = l["mixer"], f"layers[{i}].mixer"
            require(min(m["heads"], m["dim"], m["vdim"]) >= 1, f"{where}: heads, dim and vdim must be at least 1")
            if l["type"] == "lightning":
                require(len(m["decay"]) == m["heads"], f"{where}.decay must hold one number a head")
            else:
                rot = m["rot"]
                require(m["kv_rank"] >= 1, f"{where}.kv_rank must be at least 1")
                require(m["rot_dim"] >= 0 and m["rot_dim"] % 2 == 0, f"{where}.rot_dim must be even and not negative")
                require(m["rot_dim"] == 0 or rot is not None, f"{where}: rotated dimensions need 'rot'")
                require(rot is None or (rot["base"] > 0 and rot["dims"] == m["rot_dim"]),
                        f"{where}.rot: base must be positive and dims equal to rot_dim (the rotated part turns as a whole)")
                sc = rot["scaling"] if rot else None
                require(sc is None or min(sc.values()) > 0, f"{where}.rot.scaling: factor, original, fast and slow must be positive")
                j = m["kv_from"]
                if j is not None:
                    require(0 <= j < i and self.layers[j]["type"] == "latent_attention" and self.layers[j]["mixer"]["kv_from"] is None,
                            f"{where}.kv_from must name an earlier latent_attention layer with rows of its own")
                    o = self.layers[j]["mixer"]
                    require((o["kv_rank"], o["rot_dim"], o["rot"]) == (m["kv_rank"], m["rot_dim"], rot),
                            f"{where}.kv_from: layer {j} has another kv_rank, rot_dim or rotation")
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
        r = mlp["router"]
        n = r["experts"] + r["identity"]
        require(r["experts"] >= 1 and r["identity"] >= 0 and 1 <= r["top"] <= n,
                f"{where}.router: experts at least 1, identity not negative, 1 <= top <= experts + identity")
        for part in ("expert", "shared"):
            require(mlp[part] is None or (mlp[part]["ff"] >= 1 and mlp[part]["limit"] > 0),
                    f"{where}.{part}: ff must be at least 1 and limit positive")
        g = r["groups"]
        if g is not None:
            require(g["count"] >= 1 and n % g["count"] == 0, f"{where}.router.groups.count must divide experts + identity")
            require(1 <= g["keep"] <= g["count"] and g["keep"] * (n // g["count"]) >= r["top"],
                    f"{where}.router.groups: 1 <= keep <= count, and the kept groups must hold at least `top` experts")

    def to_dict(self) -> dict:
        strip = lambda d: {k: strip(v) if isinstance(v, Mapping) else v for k, v in d.items() if v is not None}
        layers = [{"type": l["type"], "mixer": strip(_plain(l["mixer"])), "mlp": None if l["mlp"] is None else strip(_plain(l["mlp"]))}
                  for l in self.layers]
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "embedding": {"scale": self.embedding_scale}, "layers": layers, "max_positions": self.max_positions,
                "torch_dtype": self.torch_dtype}

    # ------------------------------------------------------------------ the plan
    def _lightning(self, m) -> PartSpec:
        return PartSpec("lightning", {"hidden_size": self.width, "num_heads": m["heads"], "head_dim": m["dim"],
                                      "value_head_dim": m["vdim"], "decay": tuple(m["decay"]), "norm_eps": self.norm_eps}, "mix")

    def _latent(self, m) -> PartSpec:
        return PartSpec("latent_attention", {
            "hidden_size": self.width, "num_heads": m["heads"], "head_dim": m["dim"], "rot_dim": m["rot_dim"],
            "value_head_dim": m["vdim"], "kv_rank": m["kv_rank"], "scale": m["scale"], "norm_eps": self.norm_eps,
            "position": _rot_key(m) if m["rot_dim"] else None, "own_rows": m["kv_from"] is None,
            "tensor_names": {"q": "q", "dkv": "dkv", "dkv_norm": "dkv.norm", "uk": "uk", "uv": "uv", "o": "o"}}, "mix")

    def _ff(self, mlp) -> PartSpec:
        if mlp["kind"] == "dense":
            return PartSpec("dense_mlp", {"hidden_size": self.width, "intermediate_size": mlp["ff"], "activation": "relu_squared",
                                          "tensor_names": {"up": "up", "down": "down"}}, "mlp")
        r, sh = mlp["router"], mlp["shared"]
        return PartSpec("expert_mlp", {
            "hidden_size": self.width, "intermediate_size": mlp["expert"]["ff"], "experts": r["experts"], "top": r["top"],
            "activation": "swish_limited", "limit": mlp["expert"]["limit"], "scoring": "all", "identity": r["identity"],
            "groups": None if r["groups"] is None else (r["groups"]["count"], r["groups"]["keep"]),
            "shared": None if sh is None else {"intermediate_size": sh["ff"], "activation": "swish_limited", "limit": sh["limit"]}},
            "mlp")

    def plan(self) -> ModelPlan:
        W = self.width
        norm = lambda name: PartSpec("layernorm", {"dim": W, "eps": self.norm_eps, "tensor_name": "", "bias_name": "b"}, name)
        layers, positions, schedule = [], {}, []
        for i, l in enumerate(self.layers):
            m, cache_from = l["mixer"], None
            if l["type"] == "lightning":
                mixer = self._lightning(m)
            else:
                mixer, cache_from = self._latent(m), m["kv_from"]
                if m["rot_dim"]:
                    positions[_rot_key(m)] = PartSpec("rope_pairs", {
                        "dim": m["rot_dim"], "theta": m["rot"]["base"], "rotary_dim": m["rot_dim"], "value_dim": None,
                        "max_positions": self.max_positions, "interleaved": False, "scaling": m["rot"]["scaling"]})
            norms = {"pre_mixer": norm("norm1")}
            if l["mlp"] is not None:
                norms["pre_ff"] = norm("norm2")
            layers.append(LayerPlan(block="prenorm", mixer=mixer, feed_forward=None if l["mlp"] is None else self._ff(l["mlp"]),
                                    norms=norms, prefix=f"l{i}."))
            schedule.append(ScheduleEntry(i, cache_from=cache_from))
        return ModelPlan(
            vocab_size=self.vocab, hidden_size=W, max_positions=self.max_positions,
            embedding=PartSpec("embedding", {"vocab_size": self.vocab, "dim": W, "scale": self.embedding_scale, "tensor_name": ""}, "embed"),
            positions=positions, layers=tuple(layers), schedule=tuple(schedule), final_norm=norm("final.norm"),
            head=PartSpec("lm_head", {"vocab_size": self.vocab, "dim": W, "softcap": None, "tensor_name": ""}, "head"),
            stop_token_ids=())


def _rot_key(m) -> str:
    """One table set per distinct (rotated width, base, scaling)."""
    return _rot_name({"dim": m["rot_dim"], "rot": m["rot"]})
