"""Plain, slow implementation of the Lilatar decoder: whole sequences, no
cache, one function per mechanism, in float64 on the CPU.  It shares no code
with the engine; the tests compare the engine against it.

A Lilatar layer norms both ends of its sublayers: what goes in and what comes
out, before it joins the residual stream.  Two mixers: "lightning", linear
attention with a constant decay per head; and "parallel", capped softmax
attention over a window that also keeps a sequence's first tokens, beside a
gated delta rule with a decay per key channel, each normed over the model's
width and the two averaged.  The feed-forwards have no gate: relu squared of
one projection, dense or as a softmax-routed mixture of experts.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

from plain_model import read_folder  # noqa: F401  (own safetensors reader of the tests)

DT = torch.float64
UNIT_EPS = 1e-6


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt(x.square().mean(-1, keepdim=True) + eps)


def silu(x: torch.Tensor) -> torch.Tensor:
    return x * torch.sigmoid(x)


def softplus(x: torch.Tensor) -> torch.Tensor:
    return torch.logaddexp(x, torch.zeros_like(x))


# -- rotation ---------------------------------------------------------------
def pair_frequencies(dims: int, base: float, scaling: Optional[dict]) -> List[float]:
    """Radians per position of every rotated pair; long wavelengths are slowed down by `factor`, short ones kept, and
    those between original/high and original/low mixed."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling:
            wave = 2.0 * math.pi / f
            orig, lo, hi, factor = (float(scaling[k]) for k in ("original", "low", "high", "factor"))
            if wave > orig / lo:
                f = f / factor
            elif wave >= orig / hi:
                s = (orig / wave - lo) / (hi - lo)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return out


def rotate(x: torch.Tensor, rot: Optional[dict]) -> torch.Tensor:
    """x [T, heads, D] at positions 0 .. T-1: element 2i turns with element 2i + 1."""
    if not rot:
        return x
    n = int(rot["dims"])
    freq = torch.tensor(pair_frequencies(n, float(rot["base"]), rot.get("scaling")), dtype=DT)
    turn = torch.polar(torch.ones(x.shape[0], n // 2, dtype=DT), torch.arange(x.shape[0], dtype=DT)[:, None] * freq)
    pairs = torch.view_as_complex(x[..., :n].reshape(*x.shape[:-1], n // 2, 2).contiguous())
    turned = torch.view_as_real(pairs * turn[:, None]).reshape(*x.shape[:-1], n)
    return torch.cat([turned, x[..., n:]], dim=-1)


# -- attention with a window that keeps the first tokens -----------------------
def visible(t: int, window: int, keep: int) -> torch.Tensor:
    """[T, T] bool: key j from position i.  window 0: every earlier key."""
    i, j = torch.arange(t)[:, None], torch.arange(t)[None, :]
    seen = j <= i
    return seen & ((i - j < window) | (j < keep)) if window else seen


def attend(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, cap: float, seen: torch.Tensor) -> torch.Tensor:
    """q [T, H, D], k [T, G, D], v [T, G, Dv] -> [T, H, Dv]."""
    share = q.shape[1] // k.shape[1]
    outs = []
    for h in range(q.shape[1]):
        s = scale * (q[:, h] @ k[:, h // share].T)
        if cap:
            s = cap * torch.tanh(s / cap)
        outs.append(torch.softmax(s.masked_fill(~seen, -math.inf), dim=-1) @ v[:, h // share])
    return torch.stack(outs, dim=1)


def left_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, r=lambda x: x) -> torch.Tensor:
    t, (H, G) = h.shape[0], (m["heads"], m["kv_heads"])
    q, k, v = ((h @ w[p + n].T + w[p + n + ".b"]).reshape(t, heads, size)
               for n, heads, size in (("q", H, m["dim"]), ("k", G, m["dim"]), ("v", G, m["vdim"])))
    mask = m.get("mask") or {}
    o = attend(r(rotate(q, m.get("rot"))), r(rotate(k, m.get("rot"))), r(v), float(m["scale"]), float(m.get("softcap") or 0.0),
               visible(t, int(mask.get("size") or 0), int(mask.get("keep_first") or 0)))
    return r(o.reshape(t, -1)) @ w[p + "o"].T + w[p + "o.b"]


# -- gated delta rule with a decay per key channel -------------------------------
def conv_silu(x: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """x [T, C], taps [C, K], the last of which is the current token's."""
    k = taps.shape[1]
    wide = torch.cat([x.new_zeros(k - 1, x.shape[1]), x])
    return silu((wide.unfold(0, k, 1) * taps[None]).sum(-1))


def delta_rule(q, k, v, beta, g) -> torch.Tensor:
    """q, k, g [T, H, D], v [T, H, Dv], beta [T, H] -> [T, H, Dv]."""
    S = torch.zeros(v.shape[1], q.shape[2], v.shape[2], dtype=DT)
    out = []
    for t in range(q.shape[0]):
        S = S * g[t][:, :, None]
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def right_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float, r=lambda x: x) -> torch.Tensor:
    t, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (r(conv_silu(r(h @ w[p + n].T), w[p + n + ".conv"])) for n in "qkv")
    owner = torch.arange(H) // (H // G)
    q, k = (x.reshape(t, G, D)[:, owner] for x in (q, k))
    q, k = (x / torch.sqrt(x.square().sum(-1, keepdim=True) + UNIT_EPS) for x in (q, k))
    z = r(h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    g = torch.exp(-torch.exp(w[p + "A_log"])[None, :, None] * softplus(z).reshape(t, H, D))
    o = delta_rule(q * D ** -0.5, k, v.reshape(t, H, Dv), torch.sigmoid(r(h @ w[p + "b"].T)), g)
    gate = torch.sigmoid(r(h @ w[p + "g1"].T) @ w[p + "g2"].T)
    return r((unit_rms(o, eps) * w[p + "norm"]).reshape(t, -1) * gate) @ w[p + "o"].T


def pair_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float, r=lambda x: x) -> torch.Tensor:
    left = unit_rms(r(left_mixer(h, w, p + "left.", m["left"], r)), eps) * w[p + "left.out"]
    right = unit_rms(r(right_mixer(h, w, p + "right.", m["right"], eps, r)), eps) * w[p + "right.out"]
    return 0.5 * (left + right)


# -- linear attention with a constant decay per head --------------------------------
def decayed_attention(q, k, v, decay) -> torch.Tensor:
    """q, k [T, H, D], v [T, H, Dv], decay [H]: o_t = sum_{s <= t} decay^(t-s) (q_t . k_s) v_s, one sum per token."""
    age = (torch.arange(q.shape[0])[:, None] - torch.arange(q.shape[0])[None, :]).to(DT)
    out = []
    for h in range(q.shape[1]):
        weight = torch.where(age >= 0, torch.as_tensor(float(decay[h]), dtype=DT) ** age.clamp(min=0), 0.0)
        out.append(((q[:, h] @ k[:, h].T) * weight) @ v[:, h])
    return torch.stack(out, dim=1)


def lightning_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float, r=lambda x: x) -> torch.Tensor:
    t, H = h.shape[0], m["heads"]
    q, k, v = (silu(r(h @ w[p + n].T)).reshape(t, H, -1) for n in "qkv")
    o = decayed_attention(q, k, v, m["decay"]).reshape(t, -1)
    return r(unit_rms(o, eps) * w[p + "norm"] * torch.sigmoid(r(h @ w[p + "g"].T))) @ w[p + "o"].T


# -- feed-forwards ----------------------------------------------------------------
def squared_relu_mlp(x: torch.Tensor, w: Dict[str, torch.Tensor], p: str, r=lambda x: x) -> torch.Tensor:
    return r(torch.relu(x @ w[p + "up"].T).square()) @ w[p + "down"].T


def mixture(x: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mlp: dict, margins: Optional[list] = None,
            r=lambda x: x) -> torch.Tensor:
    n_experts, top = int(mlp["router"]["experts"]), int(mlp["router"]["top"])
    s = torch.softmax(x @ w[p + "router"].T, dim=-1)
    out, least = torch.zeros_like(x), []
    for t in range(x.shape[0]):
        order = sorted(range(n_experts), key=lambda e: (-float(s[t, e]), e))
        for e in order[:top]:
            out[t] += s[t, e] * squared_relu_mlp(x[t], w, f"{p}e{e}.", r)
        least.append(float(s[t, order[top - 1]] - s[t, order[top]]) / float(s[t, order[top - 1]] + s[t, order[top]])
                     if top < n_experts else math.inf)
    if margins is not None:
        margins.append(torch.tensor(least, dtype=DT))
    return out


def forward(cfg: dict, w: Dict[str, torch.Tensor], ids: List[int], streams: Optional[list] = None,
            margins: Optional[list] = None, rounded: bool = False) -> torch.Tensor:
    """Logits [T, vocab] of one sequence from position 0.  streams: a list that receives the residual stream after
    every layer; margins: a list that receives, per mixture, how clearly every token's last choice beat the first left
    out; rounded: sublayers' inputs and results and what passes between their products are rounded to bfloat16, which
    shows how far rounding alone moves this model's logits."""
    def r(x):
        return x.to(torch.bfloat16).to(DT) if rounded else x

    w = {k: v.to(DT) for k, v in w.items()}
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][torch.tensor(ids, dtype=torch.long)]
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h = r(unit_rms(x, eps) * w[p + "norm1"])
        if layer["type"] == "lightning":
            y = r(lightning_mixer(h, w, p + "mix.", m, eps, r))
        elif layer["type"] == "parallel":
            y = pair_mixer(h, w, p + "mix.", m, eps, r)
        else:
            raise ValueError(layer["type"])
        x = x + unit_rms(y, eps) * w[p + "norm1b"]
        mlp = layer.get("mlp")
        if mlp:
            h = r(unit_rms(x, eps) * w[p + "norm2"])
            y = mixture(h, w, p + "mlp.", mlp, margins, r) if mlp["kind"] == "moe" else r(squared_relu_mlp(h, w, p + "mlp.", r))
            x = x + unit_rms(y, eps) * w[p + "norm2b"]
        if streams is not None:
            streams.append(x.clone())
    return r(unit_rms(x, eps) * w["final.norm"]) @ w["head"].T * float(cfg.get("logit_scale") or 1.0)


def greedy(cfg: dict, w: Dict[str, torch.Tensor], prompt: List[int], n_new: int) -> Tuple[List[int], float]:
    """The new tokens, and the smallest lead that a chosen token had over the next best."""
    ids, lead = list(prompt), math.inf
    for _ in range(n_new):
        two = torch.topk(forward(cfg, w, ids)[-1], 2)
        lead = min(lead, float(two.values[0] - two.values[1]))
        ids.append(int(two.indices[0]))
    return ids[len(prompt):], lead
