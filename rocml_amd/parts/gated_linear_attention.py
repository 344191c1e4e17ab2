"""Gated linear attention: linear attention with a decay per token and key channel.

One product gives ``[q | k | v | gate | low]`` with 32-bit sums, ``low`` being the first of the decay's two small matrices.
A kernel of its own multiplies ``low`` (as it is, in 32-bit) with the second one, adds the bias and forms
``alpha = sigmoid(z)^(1 / tau)``.  Per head, in 32-bit, ``S <- diag(alpha) S + k v^T`` and ``o = S^T q head_dim^(-1/2)`` with the
new state.  Every head's output is normed with one gain for all heads, multiplied by ``silu(gate)``, rounded to the compute
type and projected back.  The cache holds ``S`` per sequence, zero at its start (stored column by column,
``[heads, v_head_dim, head_dim]``).  A prompt step and a step of one token run the same kernels, the same arithmetic per token.
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from .. import ops
from ..config.spec import GatedLinearAttentionSpec
from ..errors import ConfigError
from .base import BuildContext, Mixer, ParamSpec, StateRequest
from .registry import register_mixer
from .residual import stream

MAX_HEAD_DIM = 256      # key channels of a head that the recurrence kernel keeps in registers (16 per lane of a row of 16)


class GatedLinearAttention(Mixer):
    adds_only = True
    prompt_graph_safe = True
    kernel_families = ("recurrent",)

    def __init__(self, spec: GatedLinearAttentionSpec, ctx: BuildContext):
        if spec.head_dim > MAX_HEAD_DIM:
            raise ConfigError(f"a key size of {spec.head_dim} exceeds the {MAX_HEAD_DIM} the recurrence kernel keeps in registers")
        if spec.decay_rank <= 0 or not spec.tau > 0:
            raise ConfigError(f"the decay's inner width and root must be positive, got {spec.decay_rank} and {spec.tau}")
        self.spec = spec
        self.dtype = ctx.dtype
        self.qk_dim = spec.n_heads * spec.head_dim
        self.v_dim = spec.n_heads * spec.v_head_dim
        self.k_col, self.v_col = self.qk_dim, 2 * self.qk_dim
        self.g_col = self.v_col + self.v_dim
        self.low_col = self.g_col + self.v_dim
        self.proj_dim = self.low_col + spec.decay_rank
        self.w_in: Optional[torch.Tensor] = None
        self.w_out: Optional[torch.Tensor] = None

    def param_specs(self) -> Dict[str, ParamSpec]:
        s = self.spec
        return {"q_proj.weight": ParamSpec((self.qk_dim, s.hidden)),
                "k_proj.weight": ParamSpec((self.qk_dim, s.hidden)),
                "v_proj.weight": ParamSpec((self.v_dim, s.hidden)),
                "g_proj.weight": ParamSpec((self.v_dim, s.hidden)),
                "a1.weight": ParamSpec((s.decay_rank, s.hidden)),
                "a2.weight": ParamSpec((self.qk_dim, s.decay_rank)),
                "a2.bias": ParamSpec((self.qk_dim,), role="gain", init="normal"),
                "norm.weight": ParamSpec((s.v_head_dim,), role="gain", init="gain"),
                "o_proj.weight": ParamSpec((s.hidden, self.v_dim))}

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        self.w_in = torch.cat([tensors[p] for p in ("q_proj.weight", "k_proj.weight", "v_proj.weight", "g_proj.weight", "a1.weight")],
                              dim=0).contiguous()
        self.w_out = tensors["o_proj.weight"]
        self.a2 = tensors["a2.weight"].t().contiguous()         # [rank, channels], as the decay's kernel reads it
        self.a2_bias = tensors["a2.bias"]
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
        return n_tokens * ((self.proj_dim + self.qk_dim + self.v_dim) * 4 + self.v_dim * size)

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
            proj, c0 = ws.get("gla.proj", (n, self.proj_dim), torch.float32), 0
            ops.gemm(xn, self.w_in, proj, workspace=ws.scratch())
        decay = ws.get("gla.decay", (n, self.qk_dim), torch.float32)
        ops.low_rank_decay(proj, c0 + self.low_col, self.a2, self.a2_bias, s.tau, decay)
        o = ws.get("gla.o", (n, self.v_dim), torch.float32)
        ops.decay_scan(proj, c0, proj, c0 + self.k_col, proj, c0 + self.v_col, cache.state, step.cu_seqlens, step.seq_slots, o,
                       s.n_heads, s.head_dim, s.v_head_dim, decay=decay, out_scale=float(s.head_dim) ** -0.5)
        gated = ws.get("gla.gated", (n, self.v_dim), self.dtype)
        ops.head_norm_gate(o, proj, c0 + self.g_col, self.norm_gain, gated, s.n_heads, s.eps, gate="silu")
        stream(step).add_product(gated, self.w_out, x_accum)


register_mixer("gated_linear_attention", GatedLinearAttention)
