"""A routed feed-forward: a token is served by `top` of `experts` small gated feed-forwards.

Router logits z = R h + r in 32-bit; the `top` best-scoring experts serve the token (of equal logits the lower index
wins) and are mixed by a softmax restricted to those `top` logits: y = sum_e w_e down_e(act(gate_e h) * (up_e h)).  Tensors: "router", "router.b", and "e<i>.gate", "e<i>.up", "e<i>.down" for every expert.

The experts' gate and up matrices are stacked into one matrix at load, and their down matrices side by side into
another.  The 32-bit path, sizes that suit no tile and steps in between: one gated product gives every expert's
middle activations, each is multiplied by its expert's weight of that token (zero where the token does not use the
expert), and one down projection over all of them is the weighted sum.  Steps of many tokens in bfloat16: the (token,
expert) pairs are put in expert order on the device and each pair meets its own expert's matrices only (grouped
products over the same stacked matrices).  Steps of few tokens in bfloat16, of which many experts serve none: the chosen
experts' matrices are read, the others' are not.  Every kernel's launch depends on sizes only, never on which experts the
tokens chose.

Variants, by constructor arguments:
  `scoring="all"`   the scores are a softmax over all router outputs; a stored correction (tensor "correction", one number an
                    output) is added for the choice only; the weights are the chosen scores divided by their sum (+ 1e-20).
                    The outputs may form `groups` = (count, keep): equal runs of neighbours of which only the `keep` with the
                    largest choice in them can serve the token.  No router bias.
  `scoring="sigmoid"`  the same with the sigmoid of each router output as its score.
  `group_best=2`    a group counts by the sum of the two largest choices in it instead of the largest one.
  `weight_scale`    a constant factor of the chosen experts' weights.
  `identity=Z`      the last Z router outputs (behind the experts) are experts without matrices that give the token's own
                    input back (with scoring "all").
  `shared`          a further feed-forward of the same gated form, with sizes and constants of its own ("shared.gate" and so
                    on), that serves every token, times sigmoid(s . h) ("shared.sg"; with scoring "all" or "sigmoid"), or, with
                    `shared_gate=False`, as it is.
  `activation="swish_limited"` with `limit`: the experts' bounded gated form.
The shared expert's gate, where it has one, is one more row of the router's matrix, and its output and the identity experts' are added in
the kernel that adds up a token's experts.
"""
from __future__ import annotations

from typing import Dict, Mapping, Optional, Tuple

import torch

from ..hip import ops
from .base import FEED_FORWARDS, ParamSpec, Part, Precision
from .feedforward import GatedMLP
from .linear import Linear

_GATED = {"gelu_tanh": 0.0, "silu": ops.GATED_SILU, "swish_limited": None}
# Which of the ways (bfloat16, sizes that suit the tiles), measured with choices spread evenly over 8 to 128 experts.  Steps of at
# most 64 tokens read the chosen experts only where there are at most FEW_CHOICES (token, expert) pairs to a router output
# (beyond, most tokens meet most experts).  Else steps of GROUPED_FROM_TOKENS and more take the grouped products, and smaller
# ones one pass over all experts' matrices.
GROUPED_FROM_TOKENS = 64
FEW_CHOICES = 24.0
MIDDLE_ELEMENTS = 1 << 28      # the most middle activations (tokens x experts x their width) that a step holds at a time


@FEED_FORWARDS.register("expert_mlp")
class ExpertMLP(Part):
    graph_safe = True

    def __init__(self, precision: Precision, *, hidden_size: int, intermediate_size: int, experts: int, top: int,
                 activation: str = "silu", limit: Optional[float] = None, router_bias: bool = True, scoring: str = "chosen",
                 identity: int = 0, groups: Optional[Tuple[int, int]] = None, shared: Optional[Mapping] = None,
                 group_best: int = 1, weight_scale: float = 1.0, shared_gate: bool = True):
        if activation not in _GATED:
            raise ValueError(f"expert_mlp has no kernel for activation '{activation}'; available: {sorted(_GATED)}")
        if (activation == "swish_limited") != (limit is not None) or (limit is not None and not limit > 0):
            raise ValueError("expert_mlp: 'swish_limited' takes a positive limit, and only it does")
        if scoring not in ("chosen", "all", "sigmoid"):
            raise ValueError(f"expert_mlp: scoring '{scoring}' is not known; available: 'chosen', 'all', 'sigmoid'")
        if scoring == "chosen" and (identity or groups or shared or weight_scale != 1.0):
            raise ValueError("expert_mlp: identity experts, groups, a shared expert and a factor of the weights come with scoring 'all' or 'sigmoid'")
        if group_best not in (1, 2) or not weight_scale > 0:
            raise ValueError(f"expert_mlp: group_best is 1 or 2 and weight_scale positive, found {group_best} and {weight_scale}")
        outputs = int(experts) + int(identity)
        if experts < 1 or identity < 0 or not 1 <= top <= outputs <= ops.ROUTER_MAX_EXPERTS:
            raise ValueError(f"expert_mlp: 1 <= top <= experts <= {ops.ROUTER_MAX_EXPERTS}, found top {top} of {outputs}")
        count, keep = groups or (1, 1)
        if count < 1 or outputs % count or not 1 <= keep <= count or keep * (outputs // count) < top:
            raise ValueError(f"expert_mlp: {count} groups must divide {outputs} outputs, and the {keep} kept ones hold at least {top}")
        self.precision = precision
        self.H, self.F, self.E, self.top = hidden_size, int(intermediate_size), int(experts), int(top)
        self.identity, self.groups, self.scored = int(identity), (int(count), int(keep)), scoring != "chosen"
        self.sigmoid, self.group_best, self.weight_scale = scoring == "sigmoid", int(group_best), float(weight_scale)
        self.outputs = outputs
        self.router_bias = bool(router_bias) and not self.scored
        self.shared = None if shared is None else GatedMLP(precision, hidden_size=hidden_size, tensor_names={
            "gate": "gate", "up": "up", "down": "down"}, **shared)
        self.shared_gate = bool(shared_gate) and self.shared is not None
        self.router = Linear(hidden_size, outputs + self.shared_gate, precision)               # the last row: the shared expert's gate
        self.gate_up = Linear(hidden_size, self.E * self.F, precision, epilogue=ops.EPI_GEGLU,
                              epi_param=float(limit) if limit is not None else _GATED[activation])
        self.down = Linear(self.E * self.F, hidden_size, precision)
        self.bias: Optional[torch.Tensor] = None           # added to the logits; with scoring "all" to the scores, for the choice
        self._parts: Dict[str, torch.Tensor] = {}

    def param_specs(self) -> Dict[str, ParamSpec]:
        specs: Dict[str, ParamSpec] = {}
        for e in range(self.E):
            specs[f"e{e}.gate"] = ParamSpec((self.F, self.H))
            specs[f"e{e}.up"] = ParamSpec((self.F, self.H))
            specs[f"e{e}.down"] = ParamSpec((self.H, self.F))
        specs["router"] = ParamSpec((self.outputs, self.H), init_std=0.1)
        if self.router_bias:
            specs["router.b"] = ParamSpec((self.outputs,), init_std=0.1)
        if self.scored:
            specs["correction"] = ParamSpec((self.outputs,), init_std=0.02 if self.sigmoid else 0.1)
        if self.shared is not None:
            specs.update({f"shared.{n}": spec for n, spec in self.shared.param_specs().items()})
            if self.shared_gate:
                specs["shared.sg"] = ParamSpec((1, self.H), init_std=0.1)
        return specs

    def assign(self, name: str, tensor: torch.Tensor) -> None:
        if (name == "router.b" and self.router_bias) or (name == "correction" and self.scored):
            self.bias = tensor.float().contiguous()
        elif self.shared is not None and name.startswith("shared.") and name != "shared.sg":
            self.shared.assign(name[len("shared."):], tensor)
        elif name in self.param_specs():
            self._parts[name] = tensor
        else:
            raise KeyError(name)

    def finalize(self) -> None:
        router = self.precision.matrix(self._parts.pop("router"))
        if self.shared is not None:
            self.shared.finalize()
        if self.shared_gate:
            sg = self.precision.matrix(self._parts.pop("shared.sg"))
            if sg.dtype != router.dtype:
                router, sg = router.float(), sg.float()
            router = torch.cat([router, sg], dim=0)
        self.router.load(router)
        take = lambda what: [self.precision.matrix(self._parts.pop(f"e{e}.{what}")) for e in range(self.E)]
        gate, up, down = take("gate"), take("up"), take("down")
        if len({m.dtype for m in gate + up}) > 1:
            gate, up = [m.float() for m in gate], [m.float() for m in up]
        if len({m.dtype for m in down}) > 1:
            down = [m.float() for m in down]
        self.gate_up.load(torch.cat(gate + up, dim=0))       # [all gates; all ups]: the gated product's stacked matrix
        self.down.load(torch.cat(down, dim=1).contiguous())  # [W, E F]: the experts' columns side by side

    def weight_bytes(self) -> int:
        return self.router.nbytes() + self.gate_up.nbytes() + self.down.nbytes() + (self.shared.weight_bytes() if self.shared else 0)

    @property
    def accepts_fragment_activations(self) -> bool:
        return False

    def forward(self, x, ctx) -> torch.Tensor:
        T, dev = x.shape[0], self.down.weight.device
        logits = self.router(x, torch.float32)
        weights = torch.empty((T, self.E), dtype=torch.float32, device=dev)
        side = shared = None
        if self.scored:
            side = torch.empty((T, 2), dtype=torch.float32, device=dev)
            ops.route_scored(logits, self.bias, weights, side, identity=self.identity, top=self.top, groups=self.groups[0],
                             keep=self.groups[1], has_shared=self.shared is not None, shared_gate=self.shared_gate, sigmoid=self.sigmoid,
                             group_best=self.group_best, weight_scale=self.weight_scale)
        else:
            ops.route_topk(logits, self.bias, weights, self.top)
        side_used = side if self.identity or self.shared is not None else None
        if self._few(T, x, ctx):
            sh = self.shared
            return ops.expert_few(x, weights, side_used, self.gate_up.weight, self.down.weight, expert_width=self.F,
                                  epi_param=self.gate_up.epi_param, **({} if sh is None else {
                                      "shared_gate_up": sh.gate_up.weight, "shared_down": sh.down.weight, "shared_width": sh.I,
                                      "shared_epi_param": sh.gate_up.epi_param}))
        if self.shared is not None:
            shared = self.shared.forward(x, ctx)
        if (T >= GROUPED_FROM_TOKENS and self.gate_up.layout == ops.LAYOUT_FRAG16 and self.down.layout == ops.LAYOUT_FRAG16
                and ops.expert_products_supported(x.dtype, self.H, self.F)):
            # enough tokens that the experts' products pay: each (token, expert) pair meets its own expert only
            out = torch.empty((T, self.H), dtype=torch.float32, device=dev)
            ops.expert_products(x, weights, self.gate_up.weight, self.down.weight, out, expert_width=self.F, top=min(self.top, self.E),
                                epi_param=self.gate_up.epi_param, side=side_used, shared=shared)
            return out
        rows = max(1, MIDDLE_ELEMENTS // (self.E * self.F))
        if T <= rows:
            out = self._experts(x, weights, True)
        else:
            out = torch.empty((T, self.H), dtype=torch.float32, device=dev)  # a long step: the tokens in runs, so that the middle stays small
            for a in range(0, T, rows):
                out[a:a + rows] = self._experts(x[a:a + rows], weights[a:a + rows], False)
        if side_used is None:
            return out
        y = torch.empty((T, self.H), dtype=torch.float32, device=dev)
        ops.expert_combine(out, x, side, shared, y)
        return y

    def _few(self, T: int, x, ctx) -> bool:
        """Whether this step reads the chosen experts only.  The choice is made from the step's size as captured steps round
        it (single tokens: the batch's bucket; short prompts: a multiple of 16), so that both kinds of step add alike."""
        n = (getattr(ctx, "rounded_seqs", 0) if getattr(ctx, "is_decode", False) else 0) or -(-T // 16) * 16
        tiles = [self.gate_up, self.down] + ([] if self.shared is None else [self.shared.gate_up, self.shared.down])
        return (T <= n and self._few_pays(n)
                and all(p.layout == ops.LAYOUT_FRAG16 for p in tiles) and (self.shared is None or self.shared.I % 32 == 0)
                and ops.expert_products_supported(x.dtype, self.H, self.F))

    def _few_pays(self, n: int) -> bool:
        return n <= ops.EXPERT_FEW_MAX_TOKENS and n * self.top <= FEW_CHOICES * self.outputs

    def unread_bytes(self, tokens: int) -> int:
        """Bytes of expert matrices that a step of so many single tokens is expected to leave unread, for tokens that choose
        evenly among the router's outputs."""
        b = 1
        while b < tokens:
            b *= 2
        if not (self._few_pays(b) and self.gate_up.layout == ops.LAYOUT_FRAG16):
            return 0
        none = (1.0 - self.top / self.outputs) ** tokens
        return int(none * (self.gate_up.nbytes() + self.down.nbytes()))

    def _experts(self, x, weights, allow_partials: bool) -> torch.Tensor:
        mid = self.gate_up(x, torch.float32)                 # every expert's middle activations, not yet rounded
        scaled = torch.empty(mid.shape, dtype=self.precision.act, device=mid.device)
        ops.scale_columns(mid, weights, scaled)
        return self.down(scaled, torch.float32, allow_partials=allow_partials)
