"""Differential attention: every head has two softmax maps over the same values, of which the second counts against the first.

One product gives ``[q | k | v]`` with 32-bit sums; the rows of the q matrix are put in the order (key/value head, map, head of
the group) when the weights are bound, so that a map's query heads of one key head are neighbours and a layer looks to the
kernels like grouped attention with twice the heads, in which two key heads share one value head.  q and k are rotated and k and v appended by the same
kernel as any attention's; the cache holds ``2 n_kv_heads`` key heads and ``n_kv_heads`` value heads.  The attention kernel runs both
maps of a head side by side and forms ``a1 - lam a2``, its norm and the factor ``1 - diff`` in 32-bit before anything is
rounded; in a step of one token per sequence it also rotates and appends, straight from the projection.  The 32-bit path and head sizes the matrix-core
kernels refuse run each map through the plain kernel and combine behind it.  ``lam`` is one number per layer, formed in 64-bit
from the layer's four small vectors when they are bound.
"""
from __future__ import annotations

import math
from typing import Dict, Optional

import torch

from .. import ops
from ..config.spec import DifferentialAttentionSpec
from ..errors import ConfigError
from .base import BuildContext, KVCacheRequest, Mixer, ParamSpec
from .registry import build_position, register_mixer
from .residual import stream

MAX_HEAD_DIM = 512      # what the rotation kernel takes


class DifferentialAttention(Mixer):
    adds_only = True
    kernel_families = ("diff_attention",)

    def __init__(self, spec: DifferentialAttentionSpec, ctx: BuildContext):
        if spec.n_heads % spec.n_kv_heads != 0:
            raise ConfigError(f"{spec.n_heads} query heads are not a multiple of {spec.n_kv_heads} key/value heads")
        if spec.window is not None and spec.window <= 0:
            raise ConfigError(f"window must be positive, got {spec.window}")
        if not spec.scale > 0:
            raise ConfigError(f"the scale of the scores must be positive, got {spec.scale}")
        if max(spec.head_dim, spec.v_head_dim) > MAX_HEAD_DIM:
            raise ConfigError(f"head sizes {spec.head_dim} and {spec.v_head_dim} exceed the {MAX_HEAD_DIM} the kernels take")
        self.spec = spec
        self.dtype = ctx.dtype
        self.n_cus = ops.cu_count(ctx.device)
        self.q_dim = spec.n_heads * 2 * spec.head_dim
        self.k_dim = spec.n_kv_heads * 2 * spec.head_dim
        self.v_dim = spec.n_kv_heads * spec.v_head_dim
        self.o_dim = spec.n_heads * spec.v_head_dim
        self.position = build_position(spec.position, ctx) if spec.position is not None else None
        if self.position is not None and getattr(self.position, "pairing", "halves") != "halves":
            raise ConfigError("the rotation of an attention with two maps pairs a head's halves")
        self.graph_safe = self.position is None or getattr(self.position, "graph_safe", True)
        self.prompt_graph_safe = self.graph_safe and (self.position is None or getattr(self.position, "prompt_graph_safe", False))
        self.w_qkv: Optional[torch.Tensor] = None
        self.w_o: Optional[torch.Tensor] = None
        self.map_weight = 0.0

    def param_specs(self) -> Dict[str, ParamSpec]:
        s = self.spec
        specs = {"q_proj.weight": ParamSpec((self.q_dim, s.hidden)),
                 "k_proj.weight": ParamSpec((self.k_dim, s.hidden)),
                 "v_proj.weight": ParamSpec((self.v_dim, s.hidden)),
                 "o_proj.weight": ParamSpec((s.hidden, self.o_dim))}
        for p in ("lq1", "lk1", "lq2", "lk2"):
            specs[p] = ParamSpec((s.head_dim,), role="gain", init="normal")
        return specs

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        s = self.spec
        group = s.n_heads // s.n_kv_heads
        # rows (head, map, dim) -> (key/value head, map, head of the group, dim)
        q = tensors["q_proj.weight"].view(s.n_kv_heads, group, 2, s.head_dim, s.hidden).transpose(1, 2).reshape(self.q_dim, s.hidden)
        self.w_qkv = torch.cat([q, tensors["k_proj.weight"], tensors["v_proj.weight"]], dim=0).contiguous()
        self.w_o = tensors["o_proj.weight"]

        def dot(a: str, b: str) -> float:
            return float((tensors[a].to(device="cpu", dtype=torch.float64) * tensors[b].to(device="cpu", dtype=torch.float64)).sum())
        self.map_weight = math.exp(dot("lq1", "lk1")) - math.exp(dot("lq2", "lk2")) + s.diff

    def flops(self, new_counts, starts) -> int:
        # the products with the weights, and per query, key it sees and map 2 (head size + value size) a head
        keys = 0
        w = self.spec.window
        for n, s0 in zip(new_counts, starts):
            keys += n * s0 + n * (n + 1) // 2 if w is None else sum(min(s0 + i + 1, w) for i in range(n))
        return 2 * sum(new_counts) * self.matrix_elements() + 4 * self.spec.n_heads * (self.spec.head_dim + self.spec.v_head_dim) * keys

    def activation_bytes(self, n_tokens: int) -> int:
        size = 2 if self.dtype == torch.bfloat16 else 4
        rot = 0 if self.position is None else 2 * n_tokens * (self.position.rot_dim // 2) * 4
        maps = 2 * self.o_dim * 4       # (only where the plain path runs)
        return n_tokens * ((self.q_dim + self.k_dim + self.v_dim) * 4 + (self.q_dim + self.o_dim) * size + maps) + rot

    def cache_request(self) -> KVCacheRequest:
        s = self.spec
        return KVCacheRequest(2 * s.n_kv_heads, s.head_dim, s.window, v_head_dim=s.v_head_dim, n_v_heads=s.n_kv_heads)

    def input_weight(self) -> Optional[torch.Tensor]:
        return None

    def _decode_splits(self, step, cache) -> int:
        """Splits of the key range in a decode step: by the step's shape only, so that a recorded step can be replayed, and at
        most one per page that a window can touch."""
        most = min(cache.block_table.shape[1], 64)
        if self.spec.window is not None:
            most = min(most, (self.spec.window + ops.FUSED_DECODE_PAGE - 2) // ops.FUSED_DECODE_PAGE + 1)
        return ops.decode_splits(step.n_tokens * self.spec.n_kv_heads, self.n_cus, max(most, 1))

    def forward(self, step, xn, x_accum, cache, owns_cache: bool) -> None:
        if not owns_cache:
            raise ConfigError("an attention with two maps cannot run on another layer's cache")
        s = self.spec
        n = step.n_tokens
        ws = step.workspace
        page = cache.k.shape[2]
        rows = self.q_dim + self.k_dim + self.v_dim
        single = step.max_new == 1 and ops.diff_attention_decode_fits(self.dtype, s.n_heads, s.n_kv_heads, s.head_dim, s.v_head_dim, page)
        scratch = ws.scratch()
        qkv = ws.get("diff.qkv", (n, rows), torch.float32)
        splits = ops.gemm(xn, self.w_qkv, qkv, workspace=scratch, defer=True, max_splits=ops.FUSED_DECODE_SPLITS if single else 0)
        if splits:      # the product's K pieces; the next kernel adds them
            qkv = scratch[:splits * n * rows * 4].view(torch.float32).view(splits, n, rows)
        cos = sin = None
        rot = 0
        if self.position is not None:
            cos, sin = self.position.tables(step)
            rot = self.position.rot_dim
        o = ws.get("diff.o", (n, self.o_dim), self.dtype)
        if single:
            # the attention's own partial results go behind the projection's
            used = (splits * n * rows * 4 + 255) // 256 * 256 if splits else 0
            ops.diff_attention_decode(qkv, o, cache.k, cache.v, cache.block_table, step.token_pos, s.n_heads, s.n_kv_heads, s.head_dim,
                                      s.v_head_dim, s.scale, self.map_weight, 1.0 - s.diff, s.eps, cos, sin, window=s.window,
                                      n_splits=self._decode_splits(step, cache), workspace=scratch[used:], max_len=step.max_len)
        else:
            q = ws.get("diff.q", (n, self.q_dim), self.dtype)
            ops.qk_norm_rope_append(qkv, 2 * s.n_heads, 2 * s.n_kv_heads, s.head_dim, None, None, 1.0, cos, sin, rot, q, cache.k, cache.v,
                                    cache.block_table, step.token_seq, step.token_pos, n_splits=max(splits, 1), v_head_dim=s.v_head_dim,
                                    n_v_heads=s.n_kv_heads)
            maps = None
            if not ops.diff_attention_sizes_ok(self.dtype, s.head_dim, s.v_head_dim, page):
                maps = ws.get("diff.maps", (n, 2 * self.o_dim), torch.float32)
            ops.diff_attention(q, o, cache.k, cache.v, cache.block_table, step.token_seq, step.token_pos, s.n_heads, s.n_kv_heads, s.head_dim,
                               s.v_head_dim, s.scale, self.map_weight, 1.0 - s.diff, s.eps, step.cu_seqlens, step.new_counts, window=s.window,
                               maps=maps, max_len=step.max_len)
        stream(step).add_product(o, self.w_o, x_accum)


register_mixer("differential_attention", DifferentialAttention)
