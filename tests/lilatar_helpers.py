"""Small Lilatar configurations, weights that make every mechanism matter, and the comparison of logits with the plain
implementation (plain_lilatar.py)."""
from __future__ import annotations

import copy
import json
import os
from typing import Dict, List

import numpy as np
import torch

import plain_lilatar as pl

# root mean square of a row's error (its mean taken off) over the root mean square of the row's logits (theirs too)
TOL = {"float32": 4e-5, "bfloat16": 3e-2, "float16": 4e-3}
# A router's choice that float32's rounding might turn: from that position on nothing is compared (the recurrent layers
# carry it to every later one).  Models that are compared in 16 bits have "clear routes" (make_weights) and no such token.
CLOSE_CALL = 2e-5
ROUTE_CHANNELS = 16     # leading channels of the stream that nothing but the embedding writes where routes are clear


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def lightning(heads=3, dim=16, vdim=24, decay=None, mlp=None):
    decay = decay if decay is not None else [round(0.5 + 0.499 * (h + 1) / heads, 6) for h in range(heads)]
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, "mlp": mlp}


def pair(heads=4, kv_heads=2, dim=16, vdim=32, scale=0.3, softcap=6.0, window=12, keep=5, rot_dims=8, base=3000.0,
         scaling=(4.0, 64.0, 1.0, 4.0), r_heads=2, r_kv=1, r_dim=16, r_vdim=24, conv=3, a_rank=6, g_rank=5, mlp=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if softcap:
        left["softcap"] = softcap
    if window:
        left["mask"] = {"size": window}
        if keep:
            left["mask"]["keep_first"] = keep
    if rot_dims:
        left["rot"] = {"dims": rot_dims, "base": base}
        if scaling:
            left["rot"]["scaling"] = dict(zip(("factor", "original", "low", "high"), scaling))
    return {"type": "parallel", "mlp": mlp,
            "mixer": {"left": left, "right": {"heads": r_heads, "kv_heads": r_kv, "dim": r_dim, "vdim": r_vdim, "conv": conv,
                                              "a_rank": a_rank, "g_rank": g_rank}}}


# every form once: grouped heads on both sides, a layer without a feed-forward, dense and expert feed-forwards, windows
# that are no multiple of a page, kept tokens that end inside a page and at a page's edge
CFG_A = {"architecture": "Lilatar", "vocab": 203, "width": 96, "norm": {"eps": 1e-5}, "logit_scale": 0.3,
         "layers": [pair(mlp=dense(80)), lightning(mlp=moe(6, 2, 40)), pair(window=30, keep=16, heads=8, mlp=moe(5, 1, 24)),
                    lightning(heads=2, dim=24, vdim=16, decay=[0.9, 0.999])]}
# what can be left out is left out: no cap, no mask, no rotation in one layer, no scaling of frequencies in another; as
# many key heads as heads, a window and a kept run of one token, one tap, ranks of one, every expert chosen, factor 1
CFG_B = {"architecture": "Lilatar", "vocab": 131, "width": 80, "norm": {"eps": 1e-6}, "logit_scale": 1.0,
         "layers": [lightning(heads=1, dim=8, vdim=40, decay=[1.0], mlp=dense(48)),
                    pair(heads=3, kv_heads=3, dim=16, vdim=16, softcap=0, window=0, rot_dims=0, r_heads=3, r_kv=3, r_dim=32, r_vdim=16,
                         conv=1, a_rank=1, g_rank=12, mlp=moe(4, 4, 16)),
                    pair(heads=5, kv_heads=1, dim=48, vdim=80, scale=0.1, window=1, keep=1, rot_dims=48, scaling=None, r_heads=1, r_kv=1,
                         r_dim=8, r_vdim=8, conv=5, mlp=dense(56)),
                    lightning(heads=4, dim=16, vdim=16, decay=[0.0, 0.25, 0.75, 1.0], mlp=moe(9, 3, 32))]}
# heads in multiples of 16, four to a key head (they share what they read); more tokens kept than the window holds; heads
# of the linear attention that fill several tiles
CFG_C = {"architecture": "Lilatar", "vocab": 97, "width": 128, "norm": {"eps": 1e-4}, "logit_scale": 2.0,
         "layers": [pair(heads=4, kv_heads=1, dim=64, vdim=32, scale=0.125, window=33, keep=40, rot_dims=32, r_heads=4, r_kv=2, r_dim=20,
                         r_vdim=12, conv=4, mlp=moe(8, 2, 32)),
                    lightning(heads=2, dim=64, vdim=48, mlp=dense(96)),
                    pair(heads=16, kv_heads=1, dim=32, vdim=16, window=17, keep=3, rot_dims=16, mlp=moe(8, 3, 16))]}
# sizes that no vector access divides: widths, heads, experts and ranks
CFG_D = {"architecture": "Lilatar", "vocab": 150, "width": 100, "norm": {"eps": 1e-6}, "logit_scale": 0.7,
         "layers": [lightning(heads=3, dim=10, vdim=7, mlp=moe(7, 2, 20)),
                    pair(heads=6, kv_heads=3, dim=20, vdim=10, window=40, keep=9, rot_dims=6, r_heads=3, r_kv=1, r_dim=10, r_vdim=22,
                         conv=2, a_rank=7, g_rank=3, mlp=dense(36)),
                    lightning(heads=5, dim=20, vdim=12, mlp=dense(20))]}
CONFIGS = {"A": CFG_A, "B": CFG_B, "C": CFG_C, "D": CFG_D}


def make_weights(cfg: dict, seed: int, clear_routes: bool = False, idle: bool = False) -> Dict[str, torch.Tensor]:
    """Weights at scales at which every mechanism shows in the logits, rounded to bfloat16.
    clear_routes: a token's choice of experts hangs on its embedding alone and is never close: the leading channels of the
    stream are the embedding's (the norms on the sublayers' results have a gain of zero there) and hold every token's
    levels in an order of its own, and an expert's router row reads one of them.
    idle: also the second norms of layers without a feed-forward, which a model tolerates and does not read."""
    from vt_transformer_amd.config import config_from_dict
    from vt_transformer_amd.weights.random_init import declared_tensors
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, decl in declared_tensors(config_from_dict(copy.deepcopy(cfg))).items():
        shape, leaf = tuple(decl.shape), name.rsplit(".", 1)[-1]
        if decl.optional and not idle:
            continue
        if decl.role == "matrix32":
            t = torch.randn(shape, generator=g) * 1.5 / shape[-1] ** 0.5
            if clear_routes:
                assert shape[0] <= ROUTE_CHANNELS
                t = torch.zeros(shape)
                t[torch.arange(shape[0]), torch.randperm(ROUTE_CHANNELS, generator=g)[:shape[0]]] = 2.0
        elif leaf == "A_log":
            t = torch.log(torch.rand(shape, generator=g) * 2.0 + 0.01)
        elif leaf == "dt_bias":
            t = torch.randn(shape, generator=g) - 2.0
        elif leaf == "conv":
            t = torch.randn(shape, generator=g) * 0.6
        elif decl.role == "gain":
            t = 1.0 + torch.randn(shape, generator=g) * 0.3
            if clear_routes and leaf in ("norm1b", "norm2b"):
                t[:ROUTE_CHANNELS] = 0.0
            if clear_routes and leaf == "norm2":
                t[:ROUTE_CHANNELS] = 1.0
        elif decl.role == "bias":
            t = torch.randn(shape, generator=g) * 0.3
        elif name == "embed":
            t = torch.randn(shape, generator=g)
            if clear_routes:
                levels = (torch.arange(ROUTE_CHANNELS) - ROUTE_CHANNELS / 2 + 0.5) * 0.25
                for row in t:
                    row[:ROUTE_CHANNELS] = levels[torch.randperm(ROUTE_CHANNELS, generator=g)]
        else:
            t = torch.randn(shape, generator=g) / shape[-1] ** 0.5
        out[name] = t.to(torch.bfloat16)
    return out


def write_model(cfg: dict, folder: str, seed: int, clear_routes: bool = False, idle: bool = False, keep_ranks: bool = False) -> str:
    """The folder as a checkpoint has it: the sizes of the low-rank projections are not in config.json (the tensors'
    shapes say them) unless keep_ranks."""
    from vt_transformer_amd.weights.safetensors_io import write_safetensors
    os.makedirs(folder, exist_ok=True)
    stored = copy.deepcopy(cfg)
    if not keep_ranks:
        for L in stored["layers"]:
            if L["type"] == "parallel":
                L["mixer"]["right"].pop("a_rank", None)
                L["mixer"]["right"].pop("g_rank", None)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(stored, f)
    write_safetensors(os.path.join(folder, "model.safetensors"), make_weights(cfg, seed, clear_routes, idle).items(),
                      metadata={"format": "pt"})
    return folder


def row_errors(got: np.ndarray, ref: np.ndarray) -> np.ndarray:
    """Per row: root mean square of the difference (its mean taken off) over that of the reference (its mean too)."""
    d = got.astype(np.float64) - ref
    d = d - d.mean(axis=-1, keepdims=True)
    c = ref - ref.mean(axis=-1, keepdims=True)
    return np.sqrt((d * d).mean(axis=-1)) / np.maximum(np.sqrt((c * c).mean(axis=-1)), 1e-30)


def check_logits(model_dir: str, reqs: Dict[str, List[int]], steps: List[dict], got: Dict[int, np.ndarray], dtype: str,
                 cache: dict = None) -> float:
    """Every wanted row against the plain implementation's logits at that place; raises at the first row beyond its limit,
    naming step, request and position.  In float32 that is the tolerance.  In 16 bits a position's limit is the tolerance,
    or three times what rounding alone does to it where that is more; one position in twenty (or two) may be over it, one
    in fifty (or one) half again: rounding moves a few positions a long way (a recurrent read-out is divided by its size),
    while a lost state, a missed key or a wrong edge moves every position behind it.  Returns the worst error."""
    cfg, w = pl.read_folder(model_dir)
    cache = cache if cache is not None else {}
    ref, known, limit = {}, {}, {}
    for rid, toks in reqs.items():
        key = (model_dir, tuple(toks), dtype != "float32")
        if key not in cache:
            margins: list = []
            logits = pl.forward(cfg, w, toks, margins=margins).numpy()
            least = torch.stack(margins).min(dim=0).values.numpy() if margins else np.full(len(toks), np.inf)
            doubt = np.nonzero(least < CLOSE_CALL)[0]
            moved = 3.0 * row_errors(pl.forward(cfg, w, toks, rounded=True).numpy(), logits) if dtype != "float32" else np.zeros(len(toks))
            if dtype != "float32":
                assert least.min() > 1e-2, "a model that is compared in 16 bits has clear routes"
            cache[key] = (logits, int(doubt[0]) if len(doubt) else len(toks), moved)
        ref[rid], known[rid], limit[rid] = cache[key]
    pos = {r: 0 for r in reqs}
    worst, over, far, count, skipped = 0.0, 0, [], 0, 0
    for s in steps:
        row = 0
        for e in s["entries"]:
            for wi in e["want"]:
                p = pos[e["id"]] + wi
                gl = got[s["step"]][row]
                assert np.isfinite(gl).all(), f"step {s['step']} request {e['id']} position {p}: logits are not finite"
                row += 1
                count += 1
                if p >= known[e["id"]]:
                    skipped += 1
                    continue
                err = float(row_errors(gl[None], ref[e["id"]][p][None])[0])
                where = f"step {s['step']} request {e['id']} position {p} (portion starts at {pos[e['id']]})"
                if dtype == "float32":
                    assert err < TOL[dtype], f"{where}: error {err:.3e} > {TOL[dtype]:.1e}"
                else:
                    # (float16 rounds eight times finer than bfloat16)
                    lim = max(TOL[dtype], float(limit[e["id"]][p]) / (8.0 if dtype == "float16" else 1.0))
                    over += err >= lim
                    if err >= 1.5 * lim:
                        far.append((where, round(err, 4), round(lim, 4)))
                worst = max(worst, err)
            pos[e["id"]] += len(e["tokens"])
    assert skipped <= count // 5, f"{skipped} of {count} positions hang on close choices"
    assert over <= max(2, count // 20), f"{over} of {count} positions are over their limit (worst {worst:.3e})"
    assert len(far) <= max(1, count // 50), f"{len(far)} of {count} positions are far over their limit: {far[:8]}"
    return worst
