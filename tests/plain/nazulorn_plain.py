"""A plain, slow Nazulorn decoder in torch on the CPU, one function per mechanism.

It is the oracle of the tests: written from the design's equations, sharing no code with the
library (it reads the configuration dictionary and the checkpoint's tensor names directly, and
keeps no cache: every call runs whole sequences, the recurrence token by token).

Notation: ``h`` a sublayer's input ``[T, width]``, positions ``0 .. T-1``, ``W x`` for a matrix
stored ``[out, in]``.  The arithmetic type is the type of the tensors handed in (the tests use
64-bit floats so that the oracle's own rounding does not count).
"""
from __future__ import annotations

import math
from typing import Callable, Dict, List, Optional, Tuple

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return rms(x, eps) * w


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


# ---- the streams ---------------------------------------------------------------------------
def streams_input(streams: List[torch.Tensor], w_in: torch.Tensor) -> torch.Tensor:
    """What a sublayer reads: one weight per stream."""
    u = torch.zeros_like(streams[0])
    for s, x in enumerate(streams):
        u = u + w_in[s] * x
    return u


def streams_update(streams: List[torch.Tensor], y: torch.Tensor, w_mix: torch.Tensor, w_out: torch.Tensor, m: float) -> List[torch.Tensor]:
    """Every stream anew from all the old ones (``w_mix[from, to]``) and ``m w_out[to]`` times the sublayer's output."""
    new = []
    for t in range(len(streams)):
        x = m * w_out[t] * y
        for s, old in enumerate(streams):
            x = x + w_mix[s, t] * old
        new.append(x)
    return new


# ---- rotation ------------------------------------------------------------------------------
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


def rotate(x: torch.Tensor, rot: Optional[Dict]) -> torch.Tensor:
    """``x [T, heads, d]``: the first ``dims`` numbers of every head turn in pairs ``(i, i + dims/2)``; the rest stays."""
    if rot is None:
        return x
    n = rot["dims"]
    f, factor = frequencies(rot)
    angle = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * torch.tensor(f, dtype=torch.float64)[None, :]
    c, s = (torch.cos(angle) * factor).to(x.dtype)[:, None, :], (torch.sin(angle) * factor).to(x.dtype)[:, None, :]
    y = x.clone()
    u, v = x[..., :n // 2], x[..., n // 2:n]
    y[..., :n // 2] = u * c - v * s
    y[..., n // 2:n] = v * c + u * s
    return y


# ---- attention with two maps ---------------------------------------------------------------
def window_seen(n: int, size: int) -> torch.Tensor:
    """seen[i, j]: j is not after i and one of the last ``size`` positions."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    return (j <= i) & (i - j < size)


def softmax_seen(scores: torch.Tensor, seen: torch.Tensor) -> torch.Tensor:
    s = scores.masked_fill(~seen, float("-inf"))
    e = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    return e / e.sum(dim=-1, keepdim=True)


def map_weight(p: Dict[str, torch.Tensor], diff: float) -> torch.Tensor:
    """What the second map counts against the first: one number per layer."""
    return torch.exp((p["lq1"] * p["lk1"]).sum()) - torch.exp((p["lq2"] * p["lk2"]).sum()) + diff


def combine_maps(a1: torch.Tensor, a2: torch.Tensor, weight, diff: float, eps: float) -> torch.Tensor:
    """A head's output from its two maps' (over the last axis)."""
    return rms(a1 - weight * a2, eps) * (1.0 - diff)


def differential_attention(h: torch.Tensor, p: Dict[str, torch.Tensor], m: Dict, eps: float) -> torch.Tensor:
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate((h @ p["q"].T).view(T, H * 2, d), m.get("rot")).view(T, H, 2, d)
    k = rotate((h @ p["k"].T).view(T, G * 2, d), m.get("rot")).view(T, G, 2, d)
    v = (h @ p["v"].T).view(T, G, dv)
    seen = window_seen(T, m["mask"]["size"] if m.get("mask") is not None else T)
    weight = map_weight(p, m["diff"])
    out = []
    for a in range(H):
        g = a // (H // G)
        maps = [softmax_seen((q[:, a, i] @ k[:, g, i].T) * m["scale"], seen) @ v[:, g] for i in (0, 1)]
        out.append(combine_maps(maps[0], maps[1], weight, m["diff"], eps))
    return torch.cat(out, dim=1) @ p["o"].T


# ---- gated linear attention ----------------------------------------------------------------
def key_decay(h: torch.Tensor, a1: torch.Tensor, a2: torch.Tensor, b: torch.Tensor, tau: float) -> torch.Tensor:
    """A factor per token and key channel: ``sigmoid(z)^(1/tau)``."""
    z = (h @ a1.T) @ a2.T + b
    return torch.exp(torch.nn.functional.logsigmoid(z) / tau)


def decayed_recurrence(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: torch.Tensor) -> torch.Tensor:
    """``q, k, decay [T, H, d]``, ``v [T, H, dv]``: ``S_t = diag(decay_t) S_(t-1) + k_t v_t^T``, ``o_t = S_t^T q_t``."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        S = decay[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(dim=1)
    return out


def gated_linear_attention(h: torch.Tensor, p: Dict[str, torch.Tensor], m: Dict, eps: float) -> torch.Tensor:
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ p["q"].T).view(T, H, d) * d ** -0.5
    k = (h @ p["k"].T).view(T, H, d)
    v = (h @ p["v"].T).view(T, H, dv)
    decay = key_decay(h, p["a1"], p["a2"], p["a2.b"], m["tau"]).view(T, H, d)
    o = norm(decayed_recurrence(q, k, v, decay), p["norm"], eps).reshape(T, H * dv)
    return (o * silu(h @ p["g"].T)) @ p["o"].T


# ---- experts -------------------------------------------------------------------------------
def expert(h: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor, limit: Optional[float]) -> torch.Tensor:
    g, u = h @ gate.T, h @ up.T
    if limit is not None:
        g, u = torch.clamp(g, max=limit), torch.clamp(u, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def choose_experts(logits: torch.Tensor, correction: torch.Tensor, top: int, scale: float) -> Tuple[torch.Tensor, torch.Tensor]:
    """Experts and weights ``[T, top]`` from the router's logits ``[T, n]``."""
    e = torch.exp(logits - logits.max(dim=-1, keepdim=True).values)
    s = e / e.sum(dim=-1, keepdim=True)
    chosen = torch.topk(s + correction, top, dim=-1).indices
    w = torch.gather(s, 1, chosen)
    return chosen, w / (w.sum(dim=-1, keepdim=True) + 1e-20) * scale


def experts(h: torch.Tensor, p: Dict[str, torch.Tensor], m: Dict) -> torch.Tensor:
    r = m["router"]
    chosen, w = choose_experts(h @ p["router"].T, p["correction"], r["top"], 1.0 if r.get("scale") is None else r["scale"])
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for c in range(r["top"]):
            e = int(chosen[t, c])
            if e < r["experts"]:
                out = expert(h[t:t + 1], p[f"e{e}.gate"], p[f"e{e}.up"], p[f"e{e}.down"], m["expert"]["limit"])[0]
            else:
                out = h[t]
            y[t] = y[t] + w[t, c] * out
    if m.get("shared") is not None:
        y = y + expert(h, p["shared.gate"], p["shared.up"], p["shared.down"], m["shared"]["limit"])
    return y


# ---- the model -----------------------------------------------------------------------------
def _under(tensors: Dict[str, torch.Tensor], prefix: str) -> Dict[str, torch.Tensor]:
    return {k[len(prefix):]: v for k, v in tensors.items() if k.startswith(prefix)}


def forward(cfg: Dict, tensors: Dict[str, torch.Tensor], tokens, streams: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits ``[T, vocab]`` of one sequence; ``streams`` collects the sum of the streams after every layer."""
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x = tensors["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    xs = [x for _ in range(cfg["streams"])]
    for i, lay in enumerate(cfg["layers"]):
        t = _under(tensors, f"l{i}.")
        mixer: Callable = {"attention": differential_attention, "gla": gated_linear_attention}[lay["type"]]
        y = mixer(norm(streams_input(xs, t["hc1.in"]), t["norm1"], eps), _under(t, "mix."), lay["mixer"], eps)
        xs = streams_update(xs, y, t["hc1.mix"], t["hc1.out"], m)
        if lay.get("mlp") is not None:
            y = experts(norm(streams_input(xs, t["hc2.in"]), t["norm2"], eps), _under(t, "mlp."), lay["mlp"])
            xs = streams_update(xs, y, t["hc2.mix"], t["hc2.out"], m)
        if streams is not None:
            streams.append(sum(xs))
    return (norm(sum(xs), tensors["final.norm"], eps) @ tensors["head"].T) * cfg["logit_scale"]


def greedy(cfg: Dict, tensors: Dict[str, torch.Tensor], prompt, n: int) -> List[int]:
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(forward(cfg, tensors, seq)[-1].argmax()))
    return seq[len(prompt):]
