"""A feed-forward of many small experts of which every token uses a few.

    z = W_router h (float32);  s = sigmoid(z);  the `top` experts with the largest s are chosen (lowest index among equals)
    out = sum over the chosen e of expert_e(s_e * h): the score multiplies the expert's INPUT and is not renormalised
    expert(x):  g = min(Wg x, limit),  u = clamp(Wu x, -limit, limit),  Wd (g * sigmoid(alpha * g) * (u + 1))

Nothing of a step goes through the host: the router's product, one launch that chooses and sorts the (token, expert)
pairs by expert in runs padded to tiles of 16 rows, one launch pair for all experts' products (on the matrix cores in
bfloat16), and, with more than one expert a token, the sum of a token's pairs in a fixed order.  A token's result does
not depend on what else the step holds.

Experts' tensors are `e<i>.gate`, `e<i>.up` [ff, E] and `e<i>.down` [E, ff]; they are stacked at load time.
Parameters: experts, top, intermediate_size, limit, alpha (1.702), names ({"router", "expert", "gate", "up", "down"}).

A second family of routers is served by the same launches, each choice a parameter of its own:
    score        "sigmoid" (above), or "softmax": s = softmax(z) over all of the router's outputs
    correction   True: the choice goes by s + the tensor "correction" (one number per output), the weights by s alone
    identity     n: the router has n more outputs behind the experts; one that is chosen gives the token's input itself
                 (times its weight) and has no tensors
    weight_on    "input" (above), or "output": out = sum over the chosen of s_e * expert_e(h)
    limit        None: no clamps, and the plain gate: expert(x) = Wd (silu(Wg x) * (Wu x))
    shared       None, or {"intermediate_size": f}: an expert of the plain gated form (tensors "shared.gate", "shared.up",
                 "shared.down") that every token uses, added times sigmoid(w . h), w the tensor "shared.sg" [1, E]; with
                 {"gate": False} it is added as it is and has no such tensor
    unit         "gated" (above), or "squared_relu": expert(x) = Wd max(Wu x, 0)^2, the shared expert likewise; no gate matrices
    bias         True: the tensor "router_bias" (one number per output) is added to the router's logits
With score "chosen" the choice goes by the logits and the weights are the softmax over the chosen logits alone (which is also the
softmax over all outputs, divided by the sum of the chosen ones); otherwise the weights of the chosen are never renormalised.  Router logits, scores, the choice and all sums are float32.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..errors import ConfigError
from .base import BuildEnv, Part, TensorSpec, register_feed_forward
from .feed_forward import DenseAct, SwiGLU
from .linear import linear, pack_rows
from .stream import ExpertPairs

DEFAULT_NAMES = {"router": "router", "expert": "e{i}", "gate": "gate", "up": "up", "down": "down", "correction": "correction",
                 "shared": "shared", "shared_gate": "shared.sg", "router_bias": "router.b"}
MAX_EXPERTS = 1024
MAX_CHOSEN = 64            # of the softmax over the chosen logits
TILED_FROM = 65            # tokens of a step from which experts without gates run on the dense product's tiles


def tile_rows(n_pairs: int, n_experts: int) -> int:
    """How many rows every expert's run is padded to where it runs on the dense product's tiles: large tiles where the runs fill
    them."""
    each = n_pairs / n_experts
    return 256 if each >= 1536 else 128 if each >= 112 else 64


class RoutedExperts(Part):
    graph_safe = True
    plan_safe = True

    def __init__(self, params: Dict, env: BuildEnv):
        self.env = env
        self.n_experts, self.top = int(params["experts"]), int(params["top"])
        self.ff = int(params["intermediate_size"])
        self.limit = None if params.get("limit") is None else float(params["limit"])
        self.alpha = float(params.get("alpha", 1.702))
        self.identity = int(params.get("identity") or 0)
        self.n_outputs = self.n_experts + self.identity
        if self.identity < 0 or not 0 < self.top <= self.n_outputs <= MAX_EXPERTS or self.n_experts <= 0:
            raise ConfigError(f"routed experts: top {self.top} of {self.n_experts} experts and {self.identity} outputs behind them "
                              f"not supported (at most {MAX_EXPERTS} outputs)")
        if self.ff <= 0 or (self.limit is not None and not self.limit > 0):
            raise ConfigError("routed experts: sizes and the limit must be positive")
        self.score = {"sigmoid": 0, "softmax": 1, "chosen": 2}.get(str(params.get("score", "sigmoid")))
        if self.score is None:
            raise ConfigError(f"routed experts: score {params.get('score')!r} not supported (sigmoid, softmax, chosen)")
        if self.score == 2 and self.top > MAX_CHOSEN:
            raise ConfigError(f"routed experts: the softmax over the chosen takes at most {MAX_CHOSEN} of them, not {self.top}")
        self.has_bias = bool(params.get("bias"))
        self.has_correction = bool(params.get("correction"))
        if self.has_correction and self.score != 1:
            raise ConfigError("routed experts: a correction of the choice goes with the softmax")
        self.weight_on = str(params.get("weight_on", "input"))
        if self.weight_on not in ("input", "output"):
            raise ConfigError(f"routed experts: weight_on {self.weight_on!r} not supported (input, output)")
        if self.identity and self.weight_on != "output":
            raise ConfigError("routed experts: outputs behind the experts go with weights on the experts' outputs")
        self.names = dict(DEFAULT_NAMES, **(params.get("names") or {}))
        self.hidden = env.hidden_size
        self.unit = str(params.get("unit", "gated"))
        if self.unit not in ("gated", "squared_relu"):
            raise ConfigError(f"routed experts: unit {self.unit!r} not supported (gated, squared_relu)")
        if self.unit != "gated" and self.limit is not None:
            raise ConfigError("routed experts: limits belong to gated experts")
        shared = params.get("shared")
        self.shared, self.shared_gate = None, bool(shared is not None and shared.get("gate", True))
        if shared is not None:
            if self.weight_on != "output":
                raise ConfigError("routed experts: a shared expert goes with weights on the experts' outputs")
            base = self.names["shared"]
            names = {"gate": f"{base}.gate", "up": f"{base}.up", "down": f"{base}.down"}
            size = int(shared["intermediate_size"])
            if self.unit == "gated":
                self.shared = SwiGLU({"intermediate_size": size, "names": names}, env)
            else:
                self.shared = DenseAct({"intermediate_size": size, "activation": self.unit, "names": names}, env)
        self.plain = (self.score == 0 and self.weight_on == "input" and not self.identity and self.shared is None
                      and not self.has_bias and self.unit == "gated")
        # the sum over a token's experts may be left to whoever reads it, where it is nothing but that
        self.leaves_pairs = self.weight_on == "output" and not self.identity and self.shared is None
        self.leaves_shared_pairs = self.weight_on == "output" and not self.identity and not self.shared_gate
        self.kinds = ("gate", "up") if self.unit == "gated" else ("up",)

    def _name(self, i: int, what: str) -> str:
        return f"{self.names['expert'].format(i=i)}.{self.names[what]}"

    def tensor_specs(self) -> Dict[str, TensorSpec]:
        out = {self.names["router"]: TensorSpec((self.n_outputs, self.hidden))}
        if self.has_correction:
            out[self.names["correction"]] = TensorSpec((self.n_outputs,), role="gain", init="normal")
        if self.has_bias:
            out[self.names["router_bias"]] = TensorSpec((self.n_outputs,), role="gain", init="normal")
        if self.shared is not None:
            out.update(self.shared.tensor_specs())
        if self.shared_gate:
            out[self.names["shared_gate"]] = TensorSpec((1, self.hidden))
        for i in range(self.n_experts):
            for what in self.kinds:
                out[self._name(i, what)] = TensorSpec((self.ff, self.hidden))
            out[self._name(i, "down")] = TensorSpec((self.hidden, self.ff))
        return out

    def load(self, tensors: Dict[str, torch.Tensor]) -> None:
        lib, allowed = self.env.lib, not getattr(self.env, "generic_only", False)
        r = tensors[self.names["router"]]
        pieces = [(r, 0, None, None)]
        if self.shared_gate:                 # the shared expert's gate is one more row of the router's product
            pieces.append((tensors[self.names["shared_gate"]].reshape(1, self.hidden), r.shape[0], None, None))
        if self.shared is not None:
            self.shared.load({name: tensors[name] for name in self.shared.tensor_specs()})
        rows = r.shape[0] + len(pieces) - 1
        self.w_router = pack_rows(lib, pieces, rows, r.shape[1], r.dtype, r.device, allowed)
        self.correction = tensors[self.names["correction"]].contiguous() if self.has_correction else None
        self.bias = tensors[self.names["router_bias"]].contiguous() if self.has_bias else None
        # all experts' matrices in one tensor each; for the matrix cores (bfloat16, sizes that are multiples of 32) every
        # expert's matrix fragment-major, so that a wave's load is 1 KB in a row
        self.frag = bool(allowed and r.dtype == torch.bfloat16 and self.hidden % 32 == 0 and self.ff % 32 == 0)

        def stack(what: str) -> torch.Tensor:
            first = tensors[self._name(0, what)]
            out = torch.empty((self.n_experts,) + tuple(first.shape), dtype=first.dtype, device=first.device)
            for i in range(self.n_experts):
                lib.place_rows(tensors[self._name(i, what)].contiguous(), out[i], frag=self.frag)
            return out

        # without gates a step of many tokens runs on the dense product's tiles
        self.tiled = bool(self.frag and self.unit == "squared_relu" and self.weight_on == "output" and self.hidden % 64 == 0 and self.ff % 64 == 0)
        self.act = torch.tensor([float("nan"), 1.0], dtype=torch.float32, device=r.device) if self.tiled else None     # (see DenseAct)
        self.w_gate = stack("gate") if self.unit == "gated" else None
        self.w_up, self.w_down = stack("up"), stack("down")

    def forward(self, h: torch.Tensor, ctx=None, stream: Optional[torch.Tensor] = None, next_norm=None, pairs: bool = False):
        """-> float32 [T, E], or, with pairs=True (where `leaves_pairs` or `leaves_shared_pairs`), the `ExpertPairs` of the step."""
        lib, t, dev = self.env.lib, h.shape[0], h.device
        z = linear(lib, h, self.w_router, torch.float32)
        n_pairs = t * self.top
        tiled = self.tiled and t >= TILED_FROM
        unit = tile_rows(n_pairs, self.n_experts) if tiled else 16
        max_rows = lib.routed_rows(t, self.top, self.n_experts, unit)
        sel = torch.empty(n_pairs, dtype=torch.int32, device=dev)
        weight = torch.empty(n_pairs, dtype=torch.float32, device=dev)
        row_pair = torch.empty(max_rows, dtype=torch.int32, device=dev)
        tile_expert = torch.empty(2 * (max_rows // unit), dtype=torch.int32, device=dev)      # experts, then positions in their runs
        if self.plain:
            lib.route_top(z, self.n_experts, self.top, sel, weight, row_pair, tile_expert)
        else:
            lib.route_choose(z, self.n_outputs, self.n_experts, self.top, self.score, self.correction, sel, weight, row_pair,
                             tile_expert, bias=self.bias, unit=unit)
        out = torch.empty((n_pairs, self.hidden), dtype=torch.float32, device=dev)
        if tiled:
            y = torch.empty((max_rows, self.ff), dtype=h.dtype, device=dev)
            lib.routed_experts_tiled(h, self.top, row_pair, tile_expert, unit, self.w_up, self.w_down, self.act, y, out)
        else:
            y = torch.empty((max_rows, self.ff + self.hidden), dtype=h.dtype, device=dev)     # scratch: gated units, scaled inputs
            lib.routed_experts(h, weight if self.weight_on == "input" else None, self.top, row_pair, tile_expert, self.w_gate,
                               self.w_up, self.w_down, y, out, self.limit or 0.0, self.alpha, w_frag=self.frag)
        if pairs:
            if not (self.leaves_pairs or self.leaves_shared_pairs):
                raise ConfigError("routed experts: only a plain weighted sum of the experts' outputs can be left to its reader")
            return ExpertPairs(out, weight, None if self.shared is None else self.shared.forward(h, ctx))
        if self.weight_on == "output":
            total = torch.empty((t, self.hidden), dtype=torch.float32, device=dev)
            both = None if self.shared is None else self.shared.forward(h, ctx)
            lib.experts_combine(out, sel, weight, self.top, self.n_experts, h, both, z if self.shared_gate else None,
                                self.n_outputs, total)
            return total
        if self.top == 1:
            return out
        total = torch.empty((t, self.hidden), dtype=torch.float32, device=dev)
        lib.pairs_sum(out, self.top, total)
        return total


register_feed_forward("routed_experts", RoutedExperts)
