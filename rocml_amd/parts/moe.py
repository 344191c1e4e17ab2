"""A feed-forward of many small gated feed-forwards (experts) of which each token uses a few.

The router's logits are a product with 32-bit sums, the scores (softmax over all experts), the
choice (the best experts, optionally only of the best groups of neighbouring experts) and the
weights (chosen scores over their sum) are 32-bit.  The step's (token, choice) pairs are sorted by
expert on the device, all experts' first two products and their activation run as one launch over
the sorted rows, the down products as a second, and the weighted sum of a token's experts is
32-bit, in the order of the choices.  Nothing is read back to the host, so a step can be recorded.

Other ways to score: ``sigmoid`` of every logit by itself, a learned correction that counts for the choice only,
groups scored by the sum of their two best.  A shared expert (a gated feed-forward of a size of its own that
every token uses) is added at the end, times ``sigmoid(W_sg h)``, one number per token, or as it is.  Behind the experts the
router may know identity experts, whose output is the token's input: they have no place in the sorted order, and the weighted
sum takes the input's row for them.  Where the shared expert's first product has no fused activation, it rides in the router's.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from .. import ops
from ..config.spec import RoutedExpertsSpec
from ..errors import ConfigError
from .base import BuildContext, FeedForward, ParamSpec
from .registry import register_feed_forward
from .residual import stream


class RoutedExperts(FeedForward):
    adds_only = True
    prompt_graph_safe = True
    kernel_families = ("moe",)

    def __init__(self, spec: RoutedExpertsSpec, ctx: BuildContext):
        if spec.activation not in ops.GATE_ACTIVATIONS:
            raise ConfigError(f"the experts' activation {spec.activation!r} is not supported; known: {sorted(ops.GATE_ACTIVATIONS)}")
        self.identity = int(getattr(spec, "identity", 0))
        self.routed = spec.n_experts + self.identity          # what the router chooses from
        if self.identity < 0 or spec.n_experts < 1:
            raise ConfigError(f"{spec.n_experts} experts and {self.identity} identity experts: at least one and none below zero")
        if not 1 <= spec.top <= min(self.routed, 64):
            raise ConfigError(f"a token uses {spec.top} of {self.routed} experts; at least 1 and at most 64")
        if self.routed > 512:
            raise ConfigError(f"{self.routed} experts exceed the 512 the routing kernel takes")
        self.limit, self.shared_limit = getattr(spec, "limit", None), getattr(spec, "shared_limit", None)
        self.up_offset = float(getattr(spec, "up_offset", 0.0))
        if any(v is not None and not v > 0 for v in (self.limit, self.shared_limit)):
            raise ConfigError(f"the limits of the experts' activation must be positive, got {self.limit} and {self.shared_limit}")
        self.weight_scale = float(getattr(spec, "weight_scale", 1.0))
        if spec.groups is not None and self.identity:
            raise ConfigError("groups of experts go without identity experts")
        if spec.groups is not None:
            count, keep = spec.groups
            if count <= 0 or spec.n_experts % count != 0 or not 1 <= keep <= count or spec.top > keep * (spec.n_experts // count):
                raise ConfigError(f"{spec.n_experts} experts in {count} groups of which {keep} are kept do not allow "
                                  f"{spec.top} choices")
        self.weighting = getattr(spec, "weighting", "softmax_all")
        if self.weighting not in ("softmax_all", "softmax_chosen", "sigmoid"):
            raise ConfigError(f"unknown weighting of the chosen experts {self.weighting!r}; known: softmax_all, softmax_chosen, sigmoid")
        self.correction = bool(getattr(spec, "correction", False))
        self.group_score = getattr(spec, "group_score", "max")
        if self.group_score not in ("max", "top2_sum"):
            raise ConfigError(f"unknown score of a group of experts {self.group_score!r}; known: max, top2_sum")
        self.shared = getattr(spec, "shared_intermediate", None)
        self.shared_gate = bool(getattr(spec, "shared_gate", False))
        if self.shared is None and self.shared_gate:
            raise ConfigError("a gate on the shared expert needs a shared expert")
        # the shared expert's activation as the epilogue of its first product: the bare silu only
        self.shared_fused = (self.shared is not None and spec.activation == "silu" and self.shared_limit is None and self.up_offset == 0.0
                             and ctx.dtype == torch.bfloat16 and spec.hidden % 8 == 0)
        # otherwise its first product and the router's are one
        self.shared_rides = self.shared is not None and not self.shared_fused and not self.shared_gate
        if self.weighting == "softmax_chosen" and spec.groups is not None:
            raise ConfigError("the softmax over the chosen logits alone goes without groups of experts")
        self.router_bias = bool(getattr(spec, "router_bias", False))
        self.spec = spec
        self.dtype = ctx.dtype
        self.w_router: Optional[torch.Tensor] = None
        self.b_router: Optional[torch.Tensor] = None
        self.c_router: Optional[torch.Tensor] = None
        self.w_shared_gate_up: Optional[torch.Tensor] = None

    def param_specs(self) -> Dict[str, ParamSpec]:
        s = self.spec
        specs = {"router.weight": ParamSpec((self.routed, s.hidden))}
        if self.router_bias:
            specs["router.bias"] = ParamSpec((self.routed,), role="gain", init="normal")
        for e in range(s.n_experts):
            specs[f"experts.{e}.gate_proj.weight"] = ParamSpec((s.intermediate, s.hidden))
            specs[f"experts.{e}.up_proj.weight"] = ParamSpec((s.intermediate, s.hidden))
            specs[f"experts.{e}.down_proj.weight"] = ParamSpec((s.hidden, s.intermediate))
        if self.correction:
            specs["correction"] = ParamSpec((self.routed,), role="gain", init="normal")
        if self.shared is not None:
            specs["shared.gate_proj.weight"] = ParamSpec((self.shared, s.hidden))
            specs["shared.up_proj.weight"] = ParamSpec((self.shared, s.hidden))
            specs["shared.down_proj.weight"] = ParamSpec((s.hidden, self.shared))
            if self.shared_gate:
                specs["shared.gate.weight"] = ParamSpec((1, s.hidden))
        return specs

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        n = self.spec.n_experts
        self.w_router = tensors["router.weight"]
        if self.router_bias:
            self.b_router = tensors["router.bias"]
        # one tensor per kind, expert after expert: a launch reaches every expert's matrix by a stride
        self.w_gate = torch.stack([tensors[f"experts.{e}.gate_proj.weight"] for e in range(n)]).contiguous()
        self.w_up = torch.stack([tensors[f"experts.{e}.up_proj.weight"] for e in range(n)]).contiguous()
        self.w_down = torch.stack([tensors[f"experts.{e}.down_proj.weight"] for e in range(n)]).contiguous()
        if self.correction:
            self.c_router = tensors["correction"]
        if self.shared is not None:
            # rows in (gate_j, up_j) pairs, as the dense gated feed-forward keeps them
            gate, up = tensors["shared.gate_proj.weight"], tensors["shared.up_proj.weight"]
            self.w_shared_gate_up = torch.stack([gate, up], dim=1).reshape(2 * gate.shape[0], gate.shape[1]).contiguous()
            self.w_shared_down = tensors["shared.down_proj.weight"]
            if self.shared_gate:
                # the gate's logit rides in the router's product, as one more row
                self.w_router = torch.cat([self.w_router, tensors["shared.gate.weight"]], dim=0).contiguous()
            if self.shared_rides:
                self.w_router = torch.cat([self.w_shared_gate_up, self.w_router], dim=0).contiguous()
                self.w_shared_gate_up = self.w_router[:2 * gate.shape[0]]

    def matrix_elements(self) -> int:
        """What a token is multiplied with: the router and the experts it uses."""
        s = self.spec
        shared = 0 if self.shared is None else 3 * s.hidden * self.shared + (s.hidden if self.shared_gate else 0)
        return self.routed * s.hidden + s.top * 3 * s.hidden * s.intermediate + shared

    def activation_bytes(self, n_tokens: int) -> int:
        s = self.spec
        size = 2 if self.dtype == torch.bfloat16 else 4
        shared = 0 if self.shared is None else self.shared * (size + 8) + s.hidden * 4
        return n_tokens * ((self.routed + 1) * 8 + s.top * (s.intermediate * size + s.hidden * 4 + 16) + shared)

    def forward(self, step, xn, x_accum) -> None:
        s = self.spec
        n = step.n_tokens
        ws = step.workspace
        gate_logit = None
        if self.shared_gate:
            # router and shared gate in one product; the choice kernel reads rows of n_experts numbers
            both = ws.get("moe.logits_gate", (n, self.routed + 1), torch.float32)
            ops.gemm(xn, self.w_router, both, workspace=ws.scratch())
            logits, gate_logit = both[:, :self.routed], both[:, self.routed:]
        elif self.shared_rides:
            # the shared expert's gate and up values and the router's logits in one product
            both = ws.get("moe.shared_logits", (n, 2 * self.shared + self.routed), torch.float32)
            ops.gemm(xn, self.w_router, both, workspace=ws.scratch())
            shared_gate_up, logits = both[:, :2 * self.shared], both[:, 2 * self.shared:]
        else:
            logits = ws.get("moe.logits", (n, self.routed), torch.float32)
            ops.gemm(xn, self.w_router, logits, workspace=ws.scratch())
        chosen = ws.get("moe.chosen", (n, s.top), torch.int32)
        weight = ws.get("moe.weight", (n, s.top), torch.float32)
        # The softmax over the chosen logits alone is the softmax over all of them divided by the chosen ones' sum
        # (the largest logit is among the chosen, so no term underflows that the other form keeps): the same kernel
        # with nothing under the sum.
        ops.moe_route(logits, s.top, s.groups, 0.0 if self.weighting == "softmax_chosen" else s.sum_eps, chosen, weight,
                      bias=self.b_router, sigmoid=self.weighting == "sigmoid", correction=self.c_router,
                      group_top2=self.group_score == "top2_sum", weight_scale=self.weight_scale)
        pairs = n * s.top
        plan = ops.moe_plan(chosen, s.n_experts, ws.get("moe.plan", (ops.moe_plan_words(pairs, s.n_experts),), torch.int32))
        h = ws.get("moe.h", (pairs, s.intermediate), self.dtype)
        ops.moe_gemm(xn, self.w_gate, h, plan, s.top, gather=True, w2=self.w_up, activation=s.activation, limit=self.limit,
                     up_offset=self.up_offset)
        y = ws.get("moe.y", (pairs, s.hidden), torch.float32)
        ops.moe_gemm(h, self.w_down, y, plan, s.top, gather=False)
        accumulate = not stream(step).overwrite
        if accumulate:
            ws.flush_pending()        # the stream must be whole before this kernel adds to it
        ops.moe_combine(y, plan, weight, x_accum, accumulate=accumulate, own=xn if self.identity else None)
        if self.shared is not None:
            hs = ws.get("moe.shared_h", (n, self.shared), self.dtype)
            if self.shared_fused:
                ops.gemm(xn, self.w_shared_gate_up, hs, workspace=ws.scratch(), epilogue="swiglu")
            else:
                if not self.shared_rides:
                    shared_gate_up = ws.get("moe.shared_gate_up", (n, 2 * self.shared), torch.float32)
                    ops.gemm(xn, self.w_shared_gate_up, shared_gate_up, workspace=ws.scratch())
                ops.swiglu(shared_gate_up, hs, interleaved=True, activation=s.activation, limit=self.shared_limit, up_offset=self.up_offset)
            if gate_logit is None:
                # (K pieces of this product are left to the kernel that reads the target next)
                splits = ops.gemm(hs, self.w_shared_down, x_accum, accumulate=True, workspace=ws.scratch(), defer=True)
                if splits:
                    ws.set_pending(x_accum, splits)
            else:
                ys = ws.get("moe.shared_y", (n, s.hidden), torch.float32)
                ops.gemm(hs, self.w_shared_down, ys, workspace=ws.scratch())
                ops.row_gate_add(x_accum, ys, gate_logit)


register_feed_forward("routed_experts", RoutedExperts)
