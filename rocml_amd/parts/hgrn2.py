"""Linear attention in which the forget gate also decides what is written (HGRN2).

One product gives ``[q | gate logits | v]`` with 32-bit sums.  Per head and key channel, in 32-bit,
``f = l + (1 - l) sigmoid(x + b)`` with a learned lower bound ``l``; ``S <- diag(f) S + (1 - f) v^T`` and
``o = S^T silu(q)`` with the new state (there is no key and no scale).  ``silu`` and the gate are formed by the
recurrence's kernel on its way to the state.  Every head's output is normed with one gain for all heads, rounded to the
compute type and projected back.  The cache holds ``S`` per sequence, zero at its start (stored column by column,
``[heads, v_head_dim, head_dim]``).  A prompt step and a step of one token run the same kernel, the same arithmetic per
token.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from .. import ops
from ..config.spec import Hgrn2Spec
from ..errors import ConfigError
from .base import BuildContext, Mixer, ParamSpec, StateRequest
from .registry import register_mixer
from .residual import stream

MAX_HEAD_DIM = 256      # key channels of a head that the recurrence kernel keeps in registers (16 per lane of a row of 16)


class Hgrn2(Mixer):
    adds_only = True
    prompt_graph_safe = True
    kernel_families = ("recurrent",)

    def __init__(self, spec: Hgrn2Spec, ctx: BuildContext):
        if spec.head_dim > MAX_HEAD_DIM:
            raise ConfigError(f"a key size of {spec.head_dim} exceeds the {MAX_HEAD_DIM} the recurrence kernel keeps in registers")
        self.spec = spec
        self.dtype = ctx.dtype
        self.qk_dim = spec.n_heads * spec.head_dim
        self.v_dim = spec.n_heads * spec.v_head_dim
        self.f_col, self.v_col = self.qk_dim, 2 * self.qk_dim
        self.proj_dim = self.v_col + self.v_dim
        self.w_in: Optional[torch.Tensor] = None
        self.w_out: Optional[torch.Tensor] = None

    def param_specs(self) -> Dict[str, ParamSpec]:
        s = self.spec
        return {"q_proj.weight": ParamSpec((self.qk_dim, s.hidden)),
                "f_proj.weight": ParamSpec((self.qk_dim, s.hidden)),
                "f_proj.bias": ParamSpec((self.qk_dim,), role="gain", init="normal"),
                "lower": ParamSpec((self.qk_dim,), role="gain", init="normal"),
                "v_proj.weight": ParamSpec((self.v_dim, s.hidden)),
                "norm.weight": ParamSpec((s.v_head_dim,), role="gain", init="gain"),
                "o_proj.weight": ParamSpec((s.hidden, self.v_dim))}

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        self.w_in = torch.cat([tensors[f"{p}_proj.weight"] for p in ("q", "f", "v")], dim=0).contiguous()
        self.w_out = tensors["o_proj.weight"]
        self.f_bias, self.lower = tensors["f_proj.bias"], tensors["lower"]
        self.norm_gain = tensors["norm.weight"].repeat(self.spec.n_heads).contiguous()      # one gain per column, as the kernel reads it

    def cache_request(self) -> StateRequest:
        s = self.spec
        return StateRequest((s.n_heads, s.v_head_dim, s.head_dim))

    def flops(self, new_counts, starts) -> int:
        # the products with the weights; per token and head the state's update and its read
        s = self.spec
        return 2 * sum(new_counts) * (self.matrix_elements() + 2 * s.n_heads * s.head_dim * s.v_head_dim)

    def activation_bytes(self, n_tokens: int) -> int:
        size = 2 if self.dtype == torch.bfloat16 else 4
        return n_tokens * ((self.proj_dim + self.v_dim) * 4 + self.v_dim * size)

    def input_weight(self) -> Optional[torch.Tensor]:
        return self.w_in

    def adopt_input_weight(self, view: torch.Tensor) -> None:
        self.w_in = view

    def forward(self, step, xn, x_accum, cache, owns_cache: bool, projected=None) -> None:
        if not owns_cache:
            raise ConfigError("a recurrent layer cannot run on another layer's state")
        s = self.spec
        n = step.n_tokens
        ws = step.workspace
        if projected is not None:        # the projection is columns c0 .. of a product shared with other mixers
            proj, c0 = projected
        else:
            proj, c0 = ws.get("hgrn2.proj", (n, self.proj_dim), torch.float32), 0
            ops.gemm(xn, self.w_in, proj, workspace=ws.scratch())
        o = ws.get("hgrn2.o", (n, self.v_dim), torch.float32)
        ops.decay_scan(proj, c0, proj, c0 + self.f_col, proj, c0 + self.v_col, cache.state, step.cu_seqlens, step.seq_slots, o,
                       s.n_heads, s.head_dim, s.v_head_dim, gate_lower=self.lower, gate_bias=self.f_bias)
        normed = ws.get("hgrn2.normed", (n, self.v_dim), self.dtype)
        ops.head_norm_gate(o, None, 0, self.norm_gain, normed, s.n_heads, s.eps, gate=None)
        stream(step).add_product(normed, self.w_out, x_accum)


register_mixer("hgrn2", Hgrn2)
