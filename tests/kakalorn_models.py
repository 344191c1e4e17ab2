"""Small Kakalorn configurations and random weights for the tests.

The weights are drawn here and not by the library's own initialiser, with spreads that keep activations of
order one and make every mechanism count: attention scales above 1/sqrt(dim) so that single keys stand out, sinks
from far below the scores to above them, norm gains clearly away from one, convolution taps of order one half, forget
gates whose lower bounds run from zero to almost one and whose biases reach from forgetting at once to keeping.
"""
from __future__ import annotations

import json
import os
from typing import Dict

import torch


def attention(heads, kv_heads, dim, scale, window, keep_first, rot, mlp):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale,
                      "mask": {"size": window, "keep_first": keep_first}, "rot": {"base": rot[0], "dims": rot[1]}}}


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base, scaling, mlp, kv_from=None):
    rot = {"base": base, "dims": rot_dim}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale, "rot": rot}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def hgrn2(heads, dim, vdim, mlp):
    return {"type": "hgrn2", "mixer": {"heads": heads, "dim": dim, "vdim": vdim}, "mlp": mlp}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def config(vocab, width, taps, layers, eps=1e-5) -> Dict:
    return {"architecture": "Kakalorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "canon": {"taps": taps}, "layers": layers}


YARN_A = (4.0, 64, 8.0, 1.0)
# A: every size differs from its neighbours and few are multiples of 8: rotations of a part of the head and of all of it,
# windows of 7 and 70 (across a page of the cache) beside 3 and 1 kept positions, two latent layers with rows of their own
# and two that read them with other head counts, sizes and query ranks, a recurrence with values wider and one with values
# narrower than its keys, layers without a feed-forward.
CFG_A = config(211, 72, 3, [
    latent(3, 12, 8, 20, 28, 40, 0.35, 3000.0, YARN_A, dense(88)),
    attention(6, 2, 24, 0.35, 7, 3, (5000.0, 12), dense(52)),
    latent(5, 16, 8, 8, 20, 40, 0.4, 3000.0, YARN_A, None, kv_from=0),
    hgrn2(3, 20, 36, dense(40)),
    attention(4, 4, 10, 0.5, 70, 1, (300.0, 10), None),
    latent(2, 10, 12, 14, 36, 24, 0.4, 800.0, None, dense(96)),
    hgrn2(2, 33, 9, dense(72)),
    latent(4, 6, 12, 22, 44, 24, 0.3, 800.0, None, dense(64), kv_from=5),
], eps=3e-6)

YARN_B = (8.0, 128, 16.0, 2.0)
# B: sizes the matrix-core kernels know, widths that are multiples of 8: heads of 64 and 128 whose decode steps take the
# kernel that reads the projection (one rotated in part), a head of 32 that does not; windows of 64, 65 and 130 (a page, a
# page and one, two pages and two) with 4, 70 (more than a page) and 64 (a page) kept positions; latent rows of 96 numbers
# whose prompts of 256 tokens and more are expanded; a layer that reads the rows of the first.
CFG_B = config(300, 128, 4, [
    latent(4, 32, 32, 64, 48, 64, 0.2, 100000.0, YARN_B, dense(256)),
    attention(4, 1, 64, 0.2, 65, 4, (10000.0, 64), dense(192)),
    hgrn2(2, 64, 32, dense(192)),
    attention(2, 2, 128, 0.14, 130, 70, (200000.0, 64), dense(256)),
    latent(6, 64, 32, 32, 96, 64, 0.15, 100000.0, YARN_B, dense(128), kv_from=0),
    hgrn2(4, 16, 64, None),
    attention(8, 4, 32, 0.3, 64, 64, (10000.0, 32), dense(136)),
])

# C: the values that make mechanisms vanish or coincide: one head everywhere, a window of one without and with a kept
# position, more kept positions than the window is long, a convolution of one tap, a rotation of a single pair, a ramp of the
# scaled frequencies of no width, a factor of one, a state of one number, a window longer than every request.
CFG_C = config(131, 36, 1, [
    attention(1, 1, 10, 0.5, 1, 0, (10000.0, 2), dense(20)),
    latent(1, 1, 2, 1, 1, 1, 0.8, 50.0, (1.0, 1000, 1.0, 1.0), dense(12)),
    hgrn2(1, 1, 1, dense(8)),
    attention(2, 1, 12, 0.4, 1, 1, (100.0, 12), None),
    attention(2, 2, 6, 0.6, 5, 20, (100.0, 6), dense(16)),
    latent(2, 8, 2, 6, 10, 14, 0.5, 50.0, (1.0, 1000, 1.0, 1.0), None),
    hgrn2(4, 6, 12, dense(24)),
    attention(1, 1, 16, 0.4, 1000, 2, (300.0, 16), dense(36)),
], eps=1e-3)

# D: a width that is no multiple of 4 (no kernel takes its rows as 16-byte pieces), the longest convolution, the layer that
# shares rows right behind their owner, twice.
CFG_D = config(97, 70, 8, [
    hgrn2(2, 10, 14, dense(50)),
    latent(2, 12, 6, 10, 18, 22, 0.35, 1000.0, (3.0, 50, 4.0, 1.0), dense(34)),
    latent(3, 9, 6, 5, 14, 22, 0.35, 1000.0, (3.0, 50, 4.0, 1.0), dense(30), kv_from=1),
    latent(1, 20, 6, 30, 26, 22, 0.3, 1000.0, (3.0, 50, 4.0, 1.0), None, kv_from=1),
    attention(5, 1, 14, 0.4, 9, 2, (100.0, 8), dense(42)),
])

# E: many query heads on one key/value head (more than the single-token matrix-core kernels take), a head of 192 and one of
# 256, latent rows wider than the smaller matrix-core kernels, two taps.
CFG_E = config(160, 64, 2, [
    attention(20, 1, 64, 0.2, 33, 5, (10000.0, 64), dense(64)),
    latent(2, 96, 32, 128, 40, 304, 0.12, 20000.0, (2.0, 512, 32.0, 1.0), dense(96)),
    attention(2, 1, 192, 0.11, 40, 9, (10000.0, 96), None),
    hgrn2(1, 128, 130, dense(72)),
    attention(3, 3, 256, 0.1, 100, 3, (5000.0, 256), dense(80)),
])

CONFIGS = {"A": (CFG_A, 51), "B": (CFG_B, 52), "C": (CFG_C, 53), "D": (CFG_D, 54), "E": (CFG_E, 55)}


def tensor_shapes(cfg: Dict) -> Dict[str, tuple]:
    w = cfg["width"]
    shapes = {"embed": (cfg["vocab"], w), "head": (cfg["vocab"], w), "final.norm": (w,)}
    for i, lay in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lay["mixer"]
        q = p + "mix."
        shapes.update({p + n: (w,) for n in ("norm1", "norm2", "norm1b", "norm2b")})
        shapes[p + "canon1"] = (w, cfg["canon"]["taps"])
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        if lay["type"] == "attention":
            G = m["kv_heads"]
            shapes.update({q + "q": (H * d, w), q + "q.b": (H * d,), q + "k": (G * d, w), q + "k.b": (G * d,), q + "q.norm": (d,),
                           q + "k.norm": (d,), q + "sink": (H,), q + "o": (w, H * dv)})
        elif lay["type"] == "hgrn2":
            shapes.update({q + "q": (H * d, w), q + "f": (H * d, w), q + "f.b": (H * d,), q + "lower": (H * d,), q + "v": (H * dv, w),
                           q + "norm": (dv,), q + "o": (w, H * dv)})
        else:
            r, qr, kr = m["rot_dim"], m["q_rank"], m["kv_rank"]
            shapes.update({q + "dq": (qr, w), q + "dq.norm": (qr,), q + "uq": (H * (d + r), qr), q + "uk": (H * d, kr), q + "uv": (H * dv, kr),
                           q + "g": (H, w), q + "o": (w, H * dv)})
            if m.get("kv_from") is None:
                shapes.update({q + "dkv": (kr + r, w), q + "dkv.norm": (kr,)})
        if lay.get("mlp") is not None:
            ff = lay["mlp"]["ff"]
            shapes.update({p + "mlp.up": (ff, w), p + "mlp.down": (w, ff)})
    return shapes


def random_tensors(cfg: Dict, seed: int) -> Dict[str, torch.Tensor]:
    """Values that bfloat16 holds exactly (so both compute types read the same weights)."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        def n(std=1.0, mean=0.0):
            return mean + std * torch.randn(shape, generator=gen)
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1", "norm2", "norm1b", "norm2b", "norm"):
            t = n(0.3, 1.0)
        elif name == "embed":
            t = n(1.0)
        elif last == "sink":
            t = n(2.5)                                   # from far below the scores to above them
        elif last == "canon1":
            t = n(0.5)
        elif last == "lower":
            t = torch.rand(shape, generator=gen) * 0.95
        elif name.endswith("f.b"):
            t = n(2.0, 1.0)                              # gates from forgetting at once to keeping for long
        elif last == "b":
            t = n(0.6)
        else:
            t = n(1.3 / shape[-1] ** 0.5)
        out[name] = t.to(torch.bfloat16).to(torch.float32)
    return out


def write_model(path: str, cfg: Dict, tensors: Dict[str, torch.Tensor], dtype=torch.bfloat16) -> str:
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(dtype).contiguous() for k, v in tensors.items()}, os.path.join(path, "model.safetensors"))
    return path


def as_double(tensors: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
    return {k: v.double() for k, v in tensors.items()}
