"""Small Nazulorn configurations and random weights for the tests.

The weights are drawn here and not by the library's own initialiser, with spreads that keep activations of
order one and make every mechanism count: links between the copies of the stream away from the identity and unequal
among the copies, attention scales above 1/sqrt(dim) so that single keys stand out, a second map whose weight is far from
``diff``, decays from forgetting at once to keeping for long, corrections that change which experts are chosen, limits that cut
off a good part of the gate and up values.
"""
from __future__ import annotations

import json
import os
from typing import Dict

import torch


def rot(base, dims, scaling=None):
    r = {"base": base, "dims": dims}
    if scaling is not None:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return r


def attention(heads, kv_heads, dim, vdim, scale, window, diff, rotation, mlp):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff, "rot": rotation}
    if window is not None:
        m["mask"] = {"size": window}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def gla(heads, dim, vdim, tau, rank, mlp):
    # (the rank stands in the tensors' shapes alone; the key is taken out before the configuration is written)
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "_rank": rank}, "mlp": mlp}


def moe(experts, identity, top, ff, limit, scale, shared=None):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "identity": identity, "top": top, "scale": scale},
            "shared": None if shared is None else {"ff": shared[0], "limit": shared[1]}}


def config(vocab, width, streams, embed_scale, residual_mult, logit_scale, layers, eps=1e-5) -> Dict:
    return {"architecture": "Nazulorn", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps},
            "embedding": {"scale": embed_scale}, "residual_mult": residual_mult, "logit_scale": logit_scale, "layers": layers}


YARN_A = (4.0, 64, 8.0, 1.0)
# A: every size differs from its neighbours and few are multiples of 8: windows of 7 and 70 (across a page of the cache),
# rotations of a part of the head and of all of it, values wider and narrower than the keys, layers without a feed-forward,
# without a shared expert and without identity experts, other limits for the shared expert.
CFG_A = config(211, 76, 2, 1.5, 0.7, 0.25, [
    attention(6, 2, 20, 27, 0.35, 7, 0.3, rot(3000.0, 12, YARN_A), moe(5, 3, 2, 28, 0.8, 1.3, (44, 1.7))),
    gla(3, 20, 36, 8.0, 5, None),
    gla(2, 33, 9, 3.0, 12, moe(7, 0, 3, 20, 1.2, 0.6, None)),
    attention(4, 4, 14, 10, 0.45, 70, 0.75, rot(500.0, 14), moe(3, 2, 4, 36, 0.5, 2.2, (30, 0.6))),
    attention(3, 1, 18, 24, 0.4, 33, 0.1, rot(1e4, 2, (8.0, 40, 4.0, 1.0)), None),
], eps=3e-6)

YARN_B = (8.0, 128, 16.0, 2.0)
# B: sizes the matrix-core kernels know, widths that are multiples of 8: windows of 64, 65 and 130 (a page, a page and one, two
# pages and two), heads of 64/128, 32/64 and 40/72, groups of 1, 4 and 8 query heads, four copies of the stream.
CFG_B = config(300, 128, 4, 0.8, 0.35, 1.5, [
    attention(4, 1, 64, 128, 0.2, 65, 0.7, rot(100000.0, 64, YARN_B), moe(8, 2, 3, 64, 1.5, 1.7, (96, 2.5))),
    gla(2, 64, 32, 12.0, 24, moe(6, 1, 2, 48, 2.0, 1.2, (64, 1.0))),
    attention(2, 2, 32, 64, 0.3, 130, 0.4, rot(10000.0, 16), moe(4, 4, 4, 40, 0.9, 0.8, None)),
    gla(4, 16, 64, 5.0, 8, None),
    attention(8, 1, 40, 72, 0.25, 64, 0.2, rot(20000.0, 40), moe(10, 0, 1, 56, 1.1, 1.0, (40, 0.7))),
])

# C: the values that make mechanisms vanish or coincide: one copy of the stream, one head everywhere, a window of one, no mask at
# all, no rotation, a rotation of a single pair, a ramp of the scaled frequencies of no width, a factor of one, a diff of zero, a state of one
# number, a root of one, one expert and one identity, as many chosen as there are, no limits, factors of one.
CFG_C = config(131, 36, 1, 1.0, 1.0, 1.0, [
    attention(1, 1, 10, 12, 0.5, 1, 0.5, rot(10000.0, 2), moe(1, 1, 1, 20, None, 1.0, (12, None))),
    attention(1, 1, 2, 6, 0.8, None, 0.0, rot(50.0, 2, (1.0, 1000, 1.0, 1.0)), moe(2, 0, 2, 12, 1.0, None, None)),
    gla(1, 1, 1, 1.0, 1, moe(1, 0, 1, 8, 3.0, 1.0, None)),
    attention(2, 1, 12, 5, 0.4, 1000, 0.6, None, None),
    gla(4, 6, 12, 2.0, 3, moe(2, 3, 5, 16, None, 0.5, (24, 0.5))),
], eps=1e-3)

# D: a width that is no multiple of 4 (no kernel takes its rows as 16-byte pieces), more copies of the stream than the kernels that keep
# them in vectors take, more query heads on a key/value head than the single-token kernel takes.
CFG_D = config(97, 70, 6, 2.0, 0.5, 0.5, [
    attention(18, 2, 24, 40, 0.3, 20, 0.45, rot(1000.0, 16, (3.0, 50, 4.0, 1.0)), moe(4, 1, 2, 34, 1.0, 1.5, (50, 0.8))),
    gla(2, 10, 14, 6.0, 7, moe(3, 1, 1, 22, 0.7, 1.1, None)),
    attention(5, 5, 8, 12, 0.5, 9, 0.9, rot(100.0, 8), moe(6, 2, 5, 18, 1.4, 0.9, (26, 2.0))),
])

# E: large heads: 128/256, 96/136 and 144/160 (larger than the matrix-core kernels take), wide recurrences, three copies.
CFG_E = config(160, 64, 3, 1.2, 0.6, 0.8, [
    attention(2, 1, 128, 256, 0.11, 100, 0.5, rot(20000.0, 128, (2.0, 512, 32.0, 1.0)), moe(5, 1, 2, 64, 1.0, 1.4, (48, 1.2))),
    gla(1, 128, 130, 10.0, 16, None),
    attention(3, 3, 96, 136, 0.12, 40, 0.65, rot(5000.0, 48), moe(3, 1, 2, 40, 0.6, 2.0, None)),
    attention(2, 2, 144, 160, 0.1, 50, 0.35, rot(10000.0, 144), moe(2, 1, 1, 24, 2.0, 0.7, (32, 0.9))),
    gla(2, 200, 24, 4.0, 70, moe(9, 3, 6, 16, 1.3, 1.0, (16, 1.0))),
])

# (C's seed: no choice between its one expert and the identity is close for the tests' requests, which attention would spread)
CONFIGS = {"A": (CFG_A, 61), "B": (CFG_B, 62), "C": (CFG_C, 98), "D": (CFG_D, 64), "E": (CFG_E, 65)}


def written(cfg: Dict) -> Dict:
    """The configuration as config.json holds it."""
    layers = [dict(l, mixer={k: v for k, v in l["mixer"].items() if k != "_rank"}) for l in cfg["layers"]]
    return dict(cfg, layers=layers)


def tensor_shapes(cfg: Dict) -> Dict[str, tuple]:
    w, s = cfg["width"], cfg["streams"]
    shapes = {"embed": (cfg["vocab"], w), "head": (cfg["vocab"], w), "final.norm": (w,)}
    for i, lay in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lay["mixer"]
        q = p + "mix."
        for k in ("1", "2"):
            shapes.update({p + "norm" + k: (w,), p + f"hc{k}.in": (s,), p + f"hc{k}.out": (s,), p + f"hc{k}.mix": (s, s)})
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        if lay["type"] == "attention":
            G = m["kv_heads"]
            shapes.update({q + "q": (H * 2 * d, w), q + "k": (G * 2 * d, w), q + "v": (G * dv, w), q + "o": (w, H * dv)})
            shapes.update({q + n: (d,) for n in ("lq1", "lk1", "lq2", "lk2")})
        else:
            r = m["_rank"]
            shapes.update({q + "q": (H * d, w), q + "k": (H * d, w), q + "v": (H * dv, w), q + "g": (H * dv, w), q + "o": (w, H * dv),
                           q + "norm": (dv,), q + "a1": (r, w), q + "a2": (H * d, r), q + "a2.b": (H * d,)})
        mlp = lay.get("mlp")
        if mlp is not None:
            r = mlp["router"]
            n = r["experts"] + r["identity"]
            shapes.update({p + "mlp.router": (n, w), p + "mlp.correction": (n,)})
            groups = [(f"e{e}", mlp["expert"]["ff"]) for e in range(r["experts"])]
            if mlp.get("shared") is not None:
                groups.append(("shared", mlp["shared"]["ff"]))
            for name, ff in groups:
                shapes.update({p + f"mlp.{name}.gate": (ff, w), p + f"mlp.{name}.up": (ff, w), p + f"mlp.{name}.down": (w, ff)})
    return shapes


def random_tensors(cfg: Dict, seed: int) -> Dict[str, torch.Tensor]:
    """Values that bfloat16 holds exactly (so both compute types read the same weights)."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        def n(std=1.0, mean=0.0):
            return mean + std * torch.randn(shape, generator=gen)
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1", "norm2", "norm"):
            t = n(0.3, 1.0)
        elif name == "embed":
            t = n(1.0)
        elif last == "in":
            t = n(0.4, 1.0 / shape[0])
        elif last == "out":
            t = n(0.4, 1.0)
        elif last == "mix":
            t = torch.eye(shape[0]) + n(0.15)
        elif last in ("lq1", "lk1", "lq2", "lk2"):
            t = n(0.7 / shape[0] ** 0.25)                # products of order one half
        elif last == "correction":
            t = n(0.15)
        elif last == "b":
            t = n(2.0, 1.0)                              # decays from forgetting at once to keeping for long
        else:
            t = n(1.3 / shape[-1] ** 0.5)
        out[name] = t.to(torch.bfloat16).to(torch.float32)
    return out


def write_model(path: str, cfg: Dict, tensors: Dict[str, torch.Tensor], dtype=torch.bfloat16) -> str:
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(written(cfg), f)
    save_file({k: v.to(dtype).contiguous() for k, v in tensors.items()}, os.path.join(path, "model.safetensors"))
    return path


def as_double(tensors: Dict[str, torch.Tensor]) -> Dict[str, torch.Tensor]:
    return {k: v.double() for k, v in tensors.items()}
