"""Small Tipetar configurations, weights that make every mechanism matter, and the comparison of logits with the
plain implementation (plain_tipetar.py)."""
from __future__ import annotations

import copy
import json
import os
from typing import Dict, List, Optional

import numpy as np
import torch

import plain_tipetar as pt

# root mean square of a row's error (its mean taken off) over the root mean square of the row's logits (theirs too)
TOL = {"float32": 3e-5, "bfloat16": 2e-2, "float16": 4e-3}
# Rounding may send a token whose choice of experts is nearly a tie to other experts than the plain implementation
# sends it to.  Two measures: models that are compared in bfloat16 have "fixed routes" (make_weights), whose routers read
# numbers that bfloat16 holds exactly, so that their logits are float32's in both dtypes; and a position that a token can
# reach (itself, and the later ones that see it through the layers' windows) whose choice float32's rounding might turn
# is left out.
CLOSE_CALL = 2e-5


def moe(experts, top, ff, identity=0, groups=None, scale=1.0, shared=None):
    router = {"experts": experts, "top": top, "identity": identity, "scale": scale}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": router, "shared": {"ff": shared} if shared else None}


def layer(heads=4, kv_heads=2, dim=16, vdim=32, window=12, scale=0.3, kv_from=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if window:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": mlp}


# keys of layer 0 are read through a wider window (with more heads) and through a narrower one, those of layer 2, whose
# head sizes are no multiples of 16, by a layer that sees everything; a layer without a feed-forward; every form of the
# router in one, four groups of two of which the last is identity choices alone
CFG_A = {"architecture": "Tipetar", "vocab": 211, "width": 96, "norm": {"eps": 1e-5}, "residual_mult": 0.8,
         "layers": [layer(mlp=moe(6, 2, 40, identity=2, groups=(4, 2), scale=1.7, shared=56)),
                    layer(heads=8, window=30, kv_from=0),
                    layer(heads=3, kv_heads=1, dim=20, vdim=10, window=7, scale=0.2, mlp=moe(5, 3, 24, identity=1, scale=0.6)),
                    layer(heads=3, kv_heads=1, dim=20, vdim=10, window=0, scale=0.25, kv_from=2, mlp=moe(4, 1, 32, shared=20)),
                    layer(window=5, kv_from=0, mlp=moe(3, 2, 16, identity=3, groups=(2, 1), scale=2.5, shared=16))]}
# everything that can be left out is: no groups, no identity choices, no shared expert, no factor, one expert a token, a
# window of one position, as many key heads as query heads
CFG_B = {"architecture": "Tipetar", "vocab": 131, "width": 80, "norm": {"eps": 1e-6},
         "layers": [layer(heads=2, kv_heads=2, dim=64, vdim=32, window=20, scale=0.125, mlp=moe(4, 1, 24)),
                    layer(heads=1, kv_heads=1, dim=48, vdim=80, window=1, scale=0.3, mlp=moe(7, 7, 16)),
                    layer(heads=5, kv_heads=5, dim=16, vdim=16, window=0, scale=0.4, mlp=moe(9, 3, 32))]}
# sixteen heads on one key head; a shared expert of an expert's size; one group of three kept; all layers but the first
# read its keys
CFG_C = {"architecture": "Tipetar", "vocab": 97, "width": 128, "norm": {"eps": 1e-4}, "residual_mult": 1.3,
         "layers": [layer(heads=16, kv_heads=1, dim=32, vdim=16, window=17, scale=0.2,
                          mlp=moe(10, 2, 16, identity=2, groups=(3, 1), scale=1.2, shared=16))]
         + [layer(heads=16, kv_heads=1, dim=32, vdim=16, window=w, scale=0.2, kv_from=0,
                  mlp=moe(10, 2, 16, identity=2, groups=(3, 2), scale=1.2, shared=64)) for w in (17, 16, 33)]}
# a width that is no multiple of 8 and expert sizes that are none either
CFG_D = {"architecture": "Tipetar", "vocab": 150, "width": 100, "norm": {"eps": 1e-6}, "residual_mult": 0.45,
         "layers": [layer(heads=6, kv_heads=3, dim=64, vdim=80, window=40, scale=0.1,
                          mlp=moe(8, 4, 20, identity=4, groups=(3, 2), scale=3.0, shared=36)),
                    layer(heads=6, kv_heads=3, dim=64, vdim=80, window=64, scale=0.15, kv_from=0, mlp=moe(2, 1, 12, shared=28))]}
CONFIGS = {"A": CFG_A, "B": CFG_B, "C": CFG_C, "D": CFG_D}

ROUTE_CHANNELS = 16     # leading channels of the stream that nothing but the embedding writes where routes are fixed


def make_weights(cfg: dict, seed: int, fixed_routes: bool = False, idle: bool = False) -> Dict[str, torch.Tensor]:
    """Weights at scales at which every mechanism shows in the logits, rounded to bfloat16: routers that spread their
    scores, corrections of the scores' size and mostly negative (choice scores below zero), gains away from 1.
    fixed_routes: the leading channels of the stream are the embedding's alone (the norms on the sublayers' outputs have
    a gain of zero there) and the routers read only them, so that a token's choices do not depend on rounding.
    idle: also the second norm of layers without a feed-forward, which a model tolerates and does not read."""
    from vt_transformer_amd.config import config_from_dict
    from vt_transformer_amd.weights.random_init import declared_tensors
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, decl in declared_tensors(config_from_dict(copy.deepcopy(cfg))).items():
        shape = tuple(decl.shape)
        if decl.optional and not idle:
            continue
        if decl.role == "matrix32":
            t = torch.randn(shape, generator=g) * 1.5 / shape[-1] ** 0.5
            if fixed_routes:
                t = torch.zeros(shape)
                t[:, :ROUTE_CHANNELS] = torch.randn((shape[0], ROUTE_CHANNELS), generator=g) * 1.5 / ROUTE_CHANNELS ** 0.5
        elif name.endswith(".correction"):
            t = (torch.rand(shape, generator=g) - 0.8) * 2.0 / shape[0]
        elif decl.role == "gain":
            t = 1.0 + torch.randn(shape, generator=g) * 0.3
        elif decl.role == "bias":
            t = torch.randn(shape, generator=g) * 0.3
            if fixed_routes and name.rsplit(".", 1)[-1] in ("norm1", "norm2"):
                t[:ROUTE_CHANNELS] = -1.0
        elif name == "embed":
            t = torch.randn(shape, generator=g)
        else:
            t = torch.randn(shape, generator=g) / shape[-1] ** 0.5
        out[name] = t.to(torch.bfloat16)
    return out


def write_model(cfg: dict, folder: str, seed: int, fixed_routes: bool = False, idle: bool = False) -> str:
    from vt_transformer_amd.weights.safetensors_io import write_safetensors
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(folder, "model.safetensors"), make_weights(cfg, seed, fixed_routes, idle).items(),
                      metadata={"format": "pt"})
    return folder


def row_errors(got: np.ndarray, ref: np.ndarray) -> np.ndarray:
    """Per row: root mean square of the difference (its mean taken off) over that of the reference (its mean too)."""
    d = got.astype(np.float64) - ref
    d = d - d.mean(axis=-1, keepdims=True)
    c = ref - ref.mean(axis=-1, keepdims=True)
    return np.sqrt((d * d).mean(axis=-1)) / np.maximum(np.sqrt((c * c).mean(axis=-1)), 1e-30)


def _in_doubt(cfg: dict, least: Optional[np.ndarray], n: int) -> np.ndarray:
    """Positions that a token with a close choice can reach."""
    doubt = np.zeros(n, dtype=bool)
    if least is None:
        return doubt
    windows = [layer["mixer"]["mask"]["size"] if layer["mixer"].get("mask") else n for layer in cfg["layers"]]
    reach = sum(w - 1 for w in windows)
    for p in np.nonzero(least < CLOSE_CALL)[0]:
        doubt[p:p + reach + 1] = True
    return doubt


def check_logits(model_dir: str, reqs: Dict[str, List[int]], steps: List[dict], got: Dict[int, np.ndarray], dtype: str,
                 cache: dict = None, least_compared: float = 0.9) -> float:
    """Every wanted row against the plain implementation's logits at that place; raises at the first row beyond
    its limit, naming step, request and position.  In 16 bits a position's limit is the tolerance, or three times what
    rounding alone does to it where that is more.  Returns the worst error."""
    cfg, w = pt.read_folder(model_dir)
    cache = cache if cache is not None else {}
    ref, doubt, limit = {}, {}, {}
    for rid, toks in reqs.items():
        key = (model_dir, tuple(toks))
        if key not in cache:
            margins = []
            logits = pt.forward(cfg, w, toks, margins=margins).numpy()
            least = torch.stack(margins).min(dim=0).values.numpy() if margins else None
            # (float16 rounds eight times finer than bfloat16)
            moved = row_errors(pt.forward(cfg, w, toks, rounded=True).numpy(), logits)
            cache[key] = (logits, least, 3.0 * moved)
        ref[rid], least, limit[rid] = cache[key]
        doubt[rid] = _in_doubt(cfg, least, len(toks))
    pos = {r: 0 for r in reqs}
    worst, count, skipped = 0.0, 0, 0
    for s in steps:
        row = 0
        for e in s["entries"]:
            for wi in e["want"]:
                p = pos[e["id"]] + wi
                r = ref[e["id"]][p]
                gl = got[s["step"]][row].astype(np.float64)
                assert np.isfinite(gl).all(), f"step {s['step']} request {e['id']} position {p}: logits are not finite"
                row += 1
                count += 1
                if doubt[e["id"]][p]:
                    skipped += 1
                    continue
                err = float(row_errors(gl[None], r[None])[0])
                lim = TOL[dtype]
                if dtype != "float32":
                    lim = max(lim, float(limit[e["id"]][p]) / (8.0 if dtype == "float16" else 1.0))
                assert err < lim, (f"step {s['step']} request {e['id']} position {p} "
                                   f"(portion starts at {pos[e['id']]}): error {err:.3e} > {lim:.1e}")
                worst = max(worst, err)
            pos[e["id"]] += len(e["tokens"])
    assert skipped <= (1.0 - least_compared) * count, f"{skipped} of {count} positions hang on close choices"
    return worst
