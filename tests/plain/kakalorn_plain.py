"""A plain, slow Kakalorn decoder in torch on the CPU, one function per mechanism.

It is the oracle of the tests: written from the design's equations, sharing no code with the
library (it reads the configuration dictionary and the checkpoint's tensor names directly, and
keeps no cache: every call runs whole sequences, the recurrence token by token).

Notation: ``h`` a sublayer's input ``[T, width]``, positions ``0 .. T-1``, ``W x`` for a matrix
stored ``[out, in]``.  The arithmetic type is the type of the tensors handed in (the tests use
64-bit floats so that the oracle's own rounding does not count).
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return rms(x, eps) * w


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def added_conv(h: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """``h [T, C]``, ``w [C, taps]``: ``h_t + sum_j w[:, j] h_(t - taps + 1 + j)``, zeros before the start."""
    taps = w.shape[1]
    y = h.clone()
    for j in range(taps):
        back = taps - 1 - j
        if back < h.shape[0]:
            y[back:] += w[:, j] * h[:h.shape[0] - back]
    return y


def frequencies(rot: Dict) -> Tuple[List[float], float]:
    """Angles per position of the rotated pairs, and the factor on every cosine and sine: ``base^(-2i/n)`` and 1; with
    ``scaling`` slowed down between the pairs that turn ``fast`` and ``slow`` times over the ``original`` length."""
    n, base = rot["dims"], float(rot["base"])
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    sc = rot.get("scaling")
    if sc is None:
        return f, 1.0

    def turning(t: float) -> float:
        return n * math.log(sc["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))
    lo = max(math.floor(turning(sc["fast"])), 0)
    hi = min(math.ceil(turning(sc["slow"])), n - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = (i - lo) / max(hi - lo, 0.001)
        ramp = 0.0 if ramp < 0.0 else 1.0 if ramp > 1.0 else ramp
        out.append(fi / sc["factor"] * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x: torch.Tensor, rot: Dict, pairs: str) -> torch.Tensor:
    """``x [T, heads, d]``: the first ``dims`` numbers of every head turn in pairs, ``(i, i + dims/2)`` (``pairs`` "halves")
    or ``(2i, 2i + 1)`` ("neighbours"); the rest stays."""
    n = rot["dims"]
    f, factor = frequencies(rot)
    angle = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * torch.tensor(f, dtype=torch.float64)[None, :]
    c, s = (torch.cos(angle) * factor).to(x.dtype)[:, None, :], (torch.sin(angle) * factor).to(x.dtype)[:, None, :]
    y = x.clone()
    first, second = (slice(0, n // 2), slice(n // 2, n)) if pairs == "halves" else (slice(0, n, 2), slice(1, n, 2))
    u, v = x[..., first], x[..., second]
    y[..., first] = u * c - v * s
    y[..., second] = v * c + u * s
    return y


def window_seen(n: int, size: int, keep_first: int) -> torch.Tensor:
    """seen[i, j]: j is not after i, and it is one of the last ``size`` positions or one of the first ``keep_first``."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def softmax_seen(scores: torch.Tensor, seen: torch.Tensor, sink: Optional[torch.Tensor] = None) -> torch.Tensor:
    """Weights over the seen keys; ``sink`` (a number): one more term ``exp(sink)`` in the denominator."""
    s = scores.masked_fill(~seen, float("-inf"))
    top = s.max(dim=-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, sink)
    e = torch.exp(s - top)
    total = e.sum(dim=-1, keepdim=True)
    if sink is not None:
        total = total + torch.exp(sink - top)
    return e / total


def window_attention(h: torch.Tensor, p: Dict[str, torch.Tensor], m: Dict, eps: float) -> torch.Tensor:
    """Grouped softmax attention whose values are its keys as projected; biased projections, normed and rotated q and k,
    a window with kept first positions, a learned sink per head."""
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = (h @ p["q"].T + p["q.b"]).view(T, H, d)
    k = (h @ p["k"].T + p["k.b"]).view(T, G, d)
    v = k
    q = rotate(norm(q, p["q.norm"], eps), m["rot"], "halves")
    k = rotate(norm(k, p["k.norm"], eps), m["rot"], "halves")
    seen = window_seen(T, m["mask"]["size"], m["mask"]["keep_first"])
    out = []
    for a in range(H):
        g = a // (H // G)
        out.append(softmax_seen((q[:, a] @ k[:, g].T) * m["scale"], seen, p["sink"][a]) @ v[:, g])
    return torch.cat(out, dim=1) @ p["o"].T


def gated_recurrence(q: torch.Tensor, f: torch.Tensor, v: torch.Tensor) -> torch.Tensor:
    """``q, f [T, H, d]``, ``v [T, H, dv]``: ``S_t = diag(f_t) S_(t-1) + (1 - f_t) v_t^T``, ``o_t = S_t^T q_t``."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        S = f[t][:, :, None] * S + (1.0 - f[t])[:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(dim=1)
    return out


def forget_gate(z: torch.Tensor, lower: torch.Tensor) -> torch.Tensor:
    return lower + (1.0 - lower) * torch.sigmoid(z)


def hgrn2(h: torch.Tensor, p: Dict[str, torch.Tensor], m: Dict, eps: float) -> torch.Tensor:
    """Linear attention whose forget gate decides what is written too."""
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = silu(h @ p["q"].T).view(T, H, d)
    f = forget_gate(h @ p["f"].T + p["f.b"], p["lower"]).view(T, H, d)
    v = (h @ p["v"].T).view(T, H, dv)
    return norm(gated_recurrence(q, f, v), p["norm"], eps).reshape(T, H * dv) @ p["o"].T


def latent_rows(h: torch.Tensor, p: Dict[str, torch.Tensor], m: Dict, eps: float) -> Tuple[torch.Tensor, torch.Tensor]:
    """What a layer keeps per position: the normed latent, and the rotated key part that all heads share."""
    z = h @ p["dkv"].T
    c, r = z[:, :m["kv_rank"]], z[:, m["kv_rank"]:]
    return norm(c, p["dkv.norm"], eps), rotate(r[:, None, :], m["rot"], "neighbours")[:, 0]


def latent_attention(h: torch.Tensor, p: Dict[str, torch.Tensor], m: Dict, eps: float,
                     rows: Tuple[torch.Tensor, torch.Tensor]) -> torch.Tensor:
    """Softmax attention over keys and values expanded from ``rows`` (its own or another layer's); a gate per head."""
    T, H, d, r, dv = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, kr = rows
    q = (norm(h @ p["dq"].T, p["dq.norm"], eps) @ p["uq"].T).view(T, H, d + r)
    qn, qr = q[..., :d], rotate(q[..., d:], m["rot"], "neighbours")
    k = (c @ p["uk"].T).view(T, H, d)
    v = (c @ p["uv"].T).view(T, H, dv)
    seen = window_seen(T, T, 0)
    gate = torch.sigmoid(h @ p["g"].T)
    out = []
    for a in range(H):
        w = softmax_seen((qn[:, a] @ k[:, a].T + qr[:, a] @ kr.T) * m["scale"], seen)
        out.append((w @ v[:, a]) * gate[:, a:a + 1])
    return torch.cat(out, dim=1) @ p["o"].T


def dense(h: torch.Tensor, p: Dict[str, torch.Tensor]) -> torch.Tensor:
    z = torch.relu(h @ p["up"].T)
    return (z * z) @ p["down"].T


def _under(tensors: Dict[str, torch.Tensor], prefix: str) -> Dict[str, torch.Tensor]:
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def forward(cfg: Dict, tensors: Dict[str, torch.Tensor], tokens, streams: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one sequence; ``streams`` collects the residual stream after every layer."""
    eps = cfg["norm"]["eps"]
    x = tensors["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    kept: Dict[int, Tuple[torch.Tensor, torch.Tensor]] = {}
    for i, lay in enumerate(cfg["layers"]):
        t = _under(tensors, f"l{i}.")
        p, m = _under(t, "mix."), lay["mixer"]
        h = added_conv(norm(x, t["norm1"], eps), t["canon1"])
        if lay["type"] == "attention":
            y = window_attention(h, p, m, eps)
        elif lay["type"] == "hgrn2":
            y = hgrn2(h, p, m, eps)
        else:
            src = m.get("kv_from")
            if src is None:
                kept[i] = latent_rows(h, p, m, eps)
            y = latent_attention(h, p, m, eps, kept[i if src is None else src])
        x = x + norm(y, t["norm1b"], eps)
        if lay.get("mlp") is not None:
            x = x + norm(dense(norm(x, t["norm2"], eps), _under(t, "mlp.")), t["norm2b"], eps)
        if streams is not None:
            streams.append(x)
    return norm(x, tensors["final.norm"], eps) @ tensors["head"].T


def greedy(cfg: Dict, tensors: Dict[str, torch.Tensor], prompt, n: int) -> List[int]:
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(forward(cfg, tensors, seq)[-1].argmax()))
    return seq[len(prompt):]
