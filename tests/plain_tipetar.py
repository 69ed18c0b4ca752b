"""Plain, slow implementation of the Tipetar decoder: whole sequences, no
cache, one function per mechanism, in float64 on the CPU.  It shares no code
with the engine; the tests compare the engine against it.

A Tipetar layer has no norm in front of its sublayers: they read the residual
stream itself, and what is normed is their result, which then joins the stream
times a constant.  The mixer is causal softmax attention over a window, with a
slope per head that takes a multiple of the distance off every score, and with
queries and keys that are divided by the root mean square of the whole
projection (all heads at once).  A layer may attend over the keys and values
that an earlier layer made.  The feed-forward is a mixture of experts: a
softmax router, a correction that takes part in the choice only, groups of
which the best are eligible, choices that hand the input through instead of
running an expert, and a shared expert that every token runs.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

from plain_model import read_folder  # noqa: F401  (own safetensors reader of the tests)

DT = torch.float64


def over_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def offset_rmsnorm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """What is stored is the gain less one."""
    return over_rms(x, eps) * (1.0 + w)


def plain_rmsnorm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return over_rms(x, eps) * w


def head_slope(h: int, heads: int) -> float:
    return 2.0 ** (-8.0 * (h + 1) / heads)


def queries(x: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    """[T, heads, dim], normed over all heads at once."""
    return plain_rmsnorm(x @ w[p + "q"].T, w[p + "q.norm"], eps).reshape(x.shape[0], m["heads"], m["dim"])


def keys_values(x: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> Tuple[torch.Tensor, torch.Tensor]:
    k = plain_rmsnorm(x @ w[p + "k"].T, w[p + "k.norm"], eps).reshape(x.shape[0], m["kv_heads"], m["dim"])
    return k, (x @ w[p + "v"].T).reshape(x.shape[0], m["kv_heads"], m["vdim"])


def attend(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, window: int) -> torch.Tensor:
    """q [T, H, D], k [T, G, D], v [T, G, Dv] -> [T, H, Dv]; window 0: every earlier key is seen."""
    t, heads, _ = q.shape
    share = heads // k.shape[1]
    out = torch.zeros(t, heads, v.shape[2], dtype=q.dtype)
    dist = torch.arange(t)[:, None] - torch.arange(t)[None, :]
    seen = dist >= 0
    if window:
        seen = seen & (dist < window)
    for h in range(heads):
        g = h // share
        score = (q[:, h] @ k[:, g].T) * scale - head_slope(h, heads) * dist.to(q.dtype)
        out[:, h] = torch.softmax(score.masked_fill(~seen, -math.inf), dim=-1) @ v[:, g]
    return out


def gated_unit(x: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    g = x @ w[p + "gate"].T
    return (g * torch.sigmoid(g) * (x @ w[p + "up"].T)) @ w[p + "down"].T


def choose(scores: torch.Tensor, correction: torch.Tensor, top: int, count: int, keep: int) -> Tuple[List[int], float]:
    """One token's chosen outputs, and how clearly they are chosen: the distance of the last group kept from the first
    left out and of the last output chosen from the first eligible one left out, the smaller of the two, over the scores
    that stand against each other (a choice that rounding may turn has a small one)."""
    n = scores.numel()
    c = scores + correction
    size = n // count
    best = [max(range(g * size, (g + 1) * size), key=lambda e: float(c[e])) for g in range(count)]
    order = sorted(range(count), key=lambda g: (-float(c[best[g]]), g))
    kept = set(order[:keep])

    def clear(a, b):
        return float(c[a] - c[b]) / float(scores[a] + scores[b])
    margin = clear(best[order[keep - 1]], best[order[keep]]) if keep < count else math.inf
    eligible = sorted((e for e in range(n) if e // size in kept), key=lambda e: (-float(c[e]), e))
    if top < len(eligible):
        margin = min(margin, clear(eligible[top - 1], eligible[top]))
    return eligible[:top], margin


def mixture(x: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mlp: dict, margins: Optional[list] = None) -> torch.Tensor:
    ro = mlp["router"]
    n_experts, top = int(ro["experts"]), int(ro["top"])
    groups = ro.get("groups") or {"count": 1, "keep": 1}
    scores = torch.softmax(x @ w[p + "router"].T, dim=-1)
    out = torch.zeros_like(x)
    least = []
    for t in range(x.shape[0]):
        chosen, margin = choose(scores[t], w[p + "correction"], top, int(groups["count"]), int(groups["keep"]))
        least.append(margin)
        total = float(sum(scores[t, e] for e in chosen)) + 1e-20
        for e in chosen:
            weight = scores[t, e] / total * float(ro.get("scale", 1.0))
            out[t] += weight * (gated_unit(x[t], w, f"{p}e{e}.") if e < n_experts else x[t])
    if margins is not None:
        margins.append(torch.tensor(least, dtype=DT))
    if mlp.get("shared"):
        out = out + gated_unit(x, w, p + "shared.")
    return out


def forward(cfg: dict, w: Dict[str, torch.Tensor], ids: List[int], streams: Optional[list] = None,
            margins: Optional[list] = None, rounded: bool = False) -> torch.Tensor:
    """Logits [T, vocab] of one sequence from position 0.  streams: a list that receives the residual stream after
    every layer; margins: a list that receives, per mixture, every token's margin of choice (`choose`);
    rounded: every sublayer's input and result, the queries, keys, values and heads' outputs and the last norm's
    output are rounded to bfloat16, which shows how far rounding alone moves this model's logits."""
    def r16(x):
        return x.to(torch.bfloat16).to(DT) if rounded else x

    w = {k: v.to(DT) for k, v in w.items()}
    eps, mult = float(cfg["norm"]["eps"]), float(cfg.get("residual_mult", 1.0))
    x = w["embed"][torch.tensor(ids, dtype=torch.long)]
    kept = {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = r16(x)
        src = m.get("kv_from")
        if src is None:
            k, v = keys_values(h, w, p + "mix.", m, eps)
            kept[i] = (r16(k), r16(v))
        k, v = kept[i if src is None else int(src)]
        window = int(m["mask"]["size"]) if m.get("mask") else 0
        o = attend(r16(queries(h, w, p + "mix.", m, eps)), k, v, float(m["scale"]), window)
        y = r16(o.reshape(len(ids), -1)) @ w[p + "mix.o"].T
        x = x + mult * offset_rmsnorm(r16(y), w[p + "norm1"], eps)
        if layer.get("mlp") is not None:
            y = mixture(r16(x), w, p + "mlp.", layer["mlp"], margins)
            x = x + mult * offset_rmsnorm(r16(y), w[p + "norm2"], eps)
        if streams is not None:
            streams.append(x.clone())
    return r16(offset_rmsnorm(x, w["final.norm"], eps)) @ w["head"].T


def greedy(cfg: dict, w: Dict[str, torch.Tensor], prompt: List[int], n_new: int) -> List[int]:
    ids = list(prompt)
    for _ in range(n_new):
        ids.append(int(torch.argmax(forward(cfg, w, ids)[-1])))
    return ids[len(prompt):]
