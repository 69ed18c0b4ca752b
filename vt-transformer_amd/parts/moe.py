"""A feed-forward made of many small ones ("experts", gated or not), of which a
router chooses a few for every token.

    z = W_router x                                  in float32 (the router's matrix is kept in float32)
    s = sigmoid(z)   or   softmax(z)                `score`
    the `top` experts with the largest s are chosen (the lower index among equals); their weights are their scores,
    divided by their sum if `renormalize`
    weight_on "input":   out = sum_e expert_e(s_e * x)
    weight_on "output":  out = sum_e s_e * expert_e(x)
    expert_e(x) = W_down,e ( f(W_gate,e x) * (W_up,e x) ),   f = SiLU or the tanh form of GELU; no biases
    expert_e(x) = W_down,e ( max(W_up,e x, 0)^2 )            activation "squared_relu": experts without a gate

Further forms, each a constructor parameter that can be left out:

    correction      the choice is made by s + b, b a vector of the model; the weights stay s
    groups          the router's outputs are `count` runs of neighbours; only those of the `keep` runs whose largest
                    choice score is largest can be chosen
    renorm_eps      added to the sum that the weights are divided by;   router_scale: a factor on the weights
    identity        the last so many of the router's outputs have no expert: choosing one adds its weight times x itself
    shared_expert   a feed-forward of any kind that every token runs, added to the experts' sum

The experts' matrices are stacked when they are loaded ([E, 2 F, W] with an expert's gate rows in front of its up rows,
or [E, F, W] without gates, and [E, W, F]), so a kernel finds an expert by its index.  Nothing of a step's routing reaches the host: the launches
depend on the number of tokens alone.
"""
from __future__ import annotations

import math
from typing import Callable, Dict, Optional

import torch

from ..config.base import PartSpec
from ..kernels import ops
from .base import FEED_FORWARDS, NormedInput, Part, Runtime, SublayerPieces, TensorDecl


@FEED_FORWARDS.register("expert_mixture")
class ExpertMixture(Part):
    hands_pieces = True     # forward(..., pieces=True): the choices' results, not added up

    def __init__(self, *, rt: Runtime, width: int, prefix: str, num_experts: int, top: int, intermediate_size: int,
                 score: str = "sigmoid", renormalize: bool = False, weight_on: str = "input", activation: str = "silu",
                 names: Optional[Dict[str, str]] = None, correction: bool = False, groups: Optional[Dict[str, int]] = None,
                 renorm_eps: float = 0.0, router_scale: float = 1.0, identity: int = 0, shared_expert: Optional[PartSpec] = None):
        """num_experts experts of intermediate_size, `top` of the router's outputs per token; score, renormalize,
        weight_on, correction, groups {count, keep}, renorm_eps, router_scale, identity: module docstring; activation:
        "silu", "gelu_tanh" or "squared_relu" (no gate; the weight is then on the output); shared_expert: a feed-forward whose parameter `prefix` comes behind this part's; names:
        tensor names behind the prefix for the router, the correction and, with {} standing for an expert's index, for an
        expert's gate, up and down matrices."""
        self.rt, self.width = rt, int(width)
        self.ne, self.top, self.inter = int(num_experts), int(top), int(intermediate_size)
        self.identity = int(identity)
        self.n_out = self.ne + self.identity        # the router's outputs
        if not 1 <= self.top <= self.n_out or self.ne < 1 or self.identity < 0 or self.inter <= 0:
            raise ValueError(f"{self.top} of {self.ne} experts of {self.inter} and {self.identity} outputs without one")
        self.groups, self.keep = (int(groups["count"]), int(groups["keep"])) if groups else (1, 1)
        if self.groups < 1 or self.n_out % self.groups or not 1 <= self.keep <= self.groups:
            raise ValueError(f"{self.keep} of {self.groups} equal groups of {self.n_out} router outputs")
        if self.top > self.keep * (self.n_out // self.groups):
            raise ValueError(f"{self.top} choices from {self.keep} groups of {self.n_out // self.groups} router outputs")
        if self.identity and weight_on != "output":
            raise ValueError("outputs without an expert hand the input through times their weight: the weight is on the output")
        self.correction, self.renorm_eps, self.router_scale = bool(correction), float(renorm_eps), float(router_scale)
        if score not in ("sigmoid", "softmax"):
            raise ValueError(f"score '{score}' is not known ('sigmoid' and 'softmax' are)")
        if weight_on not in ("input", "output"):
            raise ValueError(f"weight_on '{weight_on}' is not known ('input' and 'output' are)")
        self.gated = activation != "squared_relu"
        if not self.gated and weight_on != "output":
            raise ValueError("experts without a gate take their weight on the output")
        if activation in ("silu", "squared_relu"):
            self.alpha, self.cubic = 1.0, 0.0
        elif activation == "gelu_tanh":
            self.alpha, self.cubic = 2.0 * math.sqrt(2.0 / math.pi), 0.044715      # (1 + tanh z) / 2 = sigmoid(2 z)
        else:
            raise ValueError(f"activation '{activation}' is not supported ('silu', 'gelu_tanh' and 'squared_relu' are)")
        self.score, self.renormalize, self.weight_on = score, bool(renormalize), weight_on
        n = {"router": "router", "correction": "correction", "gate": "e{}.gate", "up": "e{}.up", "down": "e{}.down"}
        n.update(names or {})
        self.names = {k: prefix + v for k, v in n.items()}
        self.router = self.w_gu = self.w_down = self.bias = None
        self.shared = None
        if shared_expert is not None:
            params = dict(shared_expert.params)
            self.shared = FEED_FORWARDS.build(PartSpec(shared_expert.kind, params), rt=rt, width=width,
                                              prefix=prefix + params.pop("prefix", ""))
        # pairs (token, choice) from which the experts' products run on the matrix cores, sorted by expert (16-bit types
        # with sizes in multiples of 8: few pairs 16 rows of a matrix to a block, many in tiles of 128 x 128)
        self.grouped_from = 1

    @property
    def replayable(self) -> bool:
        return self.shared is None or bool(getattr(self.shared, "replayable", False))

    def tensors(self) -> Dict[str, TensorDecl]:
        nm = self.names
        t = {nm["router"]: TensorDecl((self.n_out, self.width), "matrix32")}
        if self.correction:
            t[nm["correction"]] = TensorDecl((self.n_out,), "bias")
        for e in range(self.ne):
            if self.gated:
                t[nm["gate"].format(e)] = TensorDecl((self.inter, self.width), "matrix")
            t[nm["up"].format(e)] = TensorDecl((self.inter, self.width), "matrix")
            t[nm["down"].format(e)] = TensorDecl((self.width, self.inter), "matrix")
        if self.shared is not None:
            t.update(self.shared.tensors())
        return t

    def load(self, get: Callable[[str], torch.Tensor], rt: Runtime) -> None:
        nm = self.names
        self.router = rt.place(get(nm["router"]), "matrix32")
        if self.correction:
            self.bias = rt.place(get(nm["correction"]), "bias")
        if self.shared is not None:
            self.shared.load(get, rt)
        # (w_gu: the first products' matrices, gate rows and up rows, or up rows alone)
        first = 2 * self.inter if self.gated else self.inter
        self.w_gu = torch.empty((self.ne, first, self.width), dtype=rt.dtype, device=rt.device)
        self.w_down = torch.empty((self.ne, self.width, self.inter), dtype=rt.dtype, device=rt.device)
        for e in range(self.ne):
            if self.gated:
                self.w_gu[e, :self.inter].copy_(rt.place(get(nm["gate"].format(e)), "matrix"))
            self.w_gu[e, first - self.inter:].copy_(rt.place(get(nm["up"].format(e)), "matrix"))
            self.w_down[e].copy_(rt.place(get(nm["down"].format(e)), "matrix"))

    def forward(self, x, ctx=None, pieces: bool = False):
        """pieces: the result may be returned as SublayerPieces."""
        rt = self.rt
        if isinstance(x, NormedInput):
            x = x.materialize()
        n = x.shape[0]
        ids = rt.buffer("moe.ids", (n, self.top), torch.int32)
        wts = rt.buffer("moe.weights", (n, self.top), torch.float32)
        id_wts = rt.buffer("moe.identity", (n,), torch.float32) if self.identity else None
        ops.moe_route(x, self.router, ids, wts, self.score, self.renormalize, self.renorm_eps, self.router_scale, self.bias,
                      self.groups, self.keep, self.identity, id_wts)
        act = rt.buffer("moe.act", (n * self.top, self.inter), rt.dtype)
        # a plain mixture whose sum is wanted adds up its choices itself; everything else is added up behind the products
        whole = not (pieces or self.identity or self.shared is not None)
        on_input, on_output = self.weight_on == "input", self.weight_on == "output"
        if n * self.top >= self.grouped_from and ops.moe_grouped_ok(x, self.ne, self.width, self.inter):
            plan = rt.buffer("moe.plan", (ops.moe_plan_size(n * self.top, self.ne),), torch.int32)
            ops.moe_sort(ids, plan, self.ne)
            if self.gated:
                ops.moe_gate_up_grouped(x, self.w_gu, plan, wts, act, self.top, on_input, self.alpha, self.cubic)
            else:
                ops.moe_up_grouped(x, self.w_gu, plan, act, self.top)
            scratch = rt.buffer("moe.choices", (n * self.top, self.width), torch.float32) if self.top > 1 or not whole else None
            out = rt.buffer("moe.out", (n, self.width), torch.float32) if whole else None
            choices = ops.moe_down_grouped(act, self.w_down, plan, wts, out, scratch, on_output)
        else:
            if self.gated:
                ops.moe_gate_up(x, self.w_gu, ids, wts, act, on_input, self.alpha, self.cubic)
            else:
                ops.moe_up(x, self.w_gu, ids, act)
            # (this kernel adds up a token's choices: one row per token is left)
            choices = ops.moe_down(act, self.w_down, ids, wts, rt.buffer("moe.out", (n, self.width), torch.float32), on_output)
            ids = None
        if whole:
            return choices
        shared = self.shared.forward(x, ctx) if self.shared is not None else None
        out = SublayerPieces(rt, n, self.width, y=shared, choices=choices, ids=ids if self.identity else None,
                             id_weights=id_wts, x=x)
        return out if pieces else out.materialize()
