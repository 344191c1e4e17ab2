"""What a layer's mixer reads, plus a short causal convolution over it: ``h_t + sum_j w[:, j] h_(t - taps + 1 + j)`` per
channel, zeros before a sequence's start.  ``h`` is the layer's first norm in the compute type; the sums are 32-bit and the
result is rounded to the compute type.  A sequence keeps its last ``taps - 1`` rows of ``h`` (in the compute type, which
holds them exactly).  A prompt step and a step of one token run the same kernel."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from .. import ops
from ..errors import ConfigError
from .base import BuildContext, ParamSpec, Part, StateRequest


class InputConv(Part):
    prompt_graph_safe = True

    def __init__(self, hidden: int, taps: int, ctx: BuildContext):
        if not 1 <= taps <= ops.ADDED_CONV_MAX_TAPS:
            raise ConfigError(f"the convolution on a mixer's input has {taps} taps; 1 to {ops.ADDED_CONV_MAX_TAPS} are supported")
        self.hidden, self.taps, self.dtype = int(hidden), int(taps), ctx.dtype
        self.w: Optional[torch.Tensor] = None

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {"weight": ParamSpec((self.hidden, self.taps), role="gain", init="normal")}

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        self.w = tensors["weight"].t().contiguous()          # [taps, hidden], as the kernels read it

    def cache_request(self) -> Optional[StateRequest]:
        return StateRequest((self.taps - 1, self.hidden), dtype=self.dtype) if self.taps > 1 else None

    def activation_bytes(self, n_tokens: int) -> int:
        return n_tokens * self.hidden * (2 if self.dtype == torch.bfloat16 else 4)

    def forward(self, step, h: torch.Tensor, view) -> torch.Tensor:
        out = step.workspace.get("block.conv", tuple(h.shape), self.dtype)
        ops.added_conv(h, self.w, None if view is None else view.state, step.cu_seqlens, step.seq_slots, step.new_counts, out)
        return out
