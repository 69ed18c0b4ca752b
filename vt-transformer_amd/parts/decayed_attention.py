"""Linear attention with a constant decay per head ("lightning" attention): a
token mixer with a matrix state per head instead of a cache of keys and values.

Per head, with S [D, Dv] (float32, zero at the start of a sequence) carried from token to token and x the mixer's input:

    q, k = silu(W_q x), silu(W_k x)  (D each),   v = silu(W_v x)  (Dv)
    S <- g S + k v^T                  g a constant of the model, one per head
    o  = S^T q                        read out after the write

Behind it the concatenated heads are divided by their common root mean square, multiplied by a gain per channel and by
sigmoid(W_g x), and projected back to the model's width.  The activations of q, k and v, the state, the read-out and
the norm are float32 whatever the runtime's dtype.

Steps of single tokens and short portions move the state token by token; a step that brings a longer portion goes
through chunks of 64 tokens, inside which the same sums are products of matrices (float32 on the matrix cores).

A request's state slot holds the heads' matrices ([H][Dv][D]); the mixer has no pages.
"""
from __future__ import annotations

from typing import Callable, Dict, Optional, Sequence

import numpy as np
import torch

from ..kernels import ops
from .base import MIXERS, CacheNeed, Part, Runtime, StateNeed, TensorDecl
from .linear import linear


CHUNKS_KEY = ("decayed_attention.chunks", ops.DECAYED_CHUNK)
CHUNKS_FROM = ops.DECAYED_CHUNK     # tokens of a step's longest portion from which the step goes through chunks


def plan_chunks(entry_start) -> np.ndarray:
    """Every entry's tokens in runs of up to a chunk: where each entry's runs start (entries + 1 numbers), then per run its
    first row and its rows."""
    start = np.asarray(entry_start, dtype=np.int64)
    runs = -(-(start[1:] - start[:-1]) // ops.DECAYED_CHUNK)
    first_run = np.concatenate([[0], np.cumsum(runs)])
    owner = np.repeat(np.arange(len(runs)), runs)
    row = start[:-1][owner] + (np.arange(first_run[-1]) - first_run[:-1][owner]) * ops.DECAYED_CHUNK
    rows = np.minimum(ops.DECAYED_CHUNK, start[1:][owner] - row)
    return np.concatenate([first_run, np.stack([row, rows], axis=1).reshape(-1)]).astype(np.int32)


@MIXERS.register("decayed_attention")
class DecayedAttentionMixer(Part):
    replayable = True       # a decoding step's launches depend on the number of entries only; the state lies in device
                            # memory and is found by the slots of the step's metadata

    def __init__(self, *, rt: Runtime, width: int, prefix: str, num_heads: int, key_dim: int, decay: Sequence[float],
                 norm_eps: float, value_dim: Optional[int] = None, activation: Optional[str] = "silu",
                 shared: Optional[dict] = None, names: Optional[Dict[str, str]] = None):
        """num_heads heads with queries and keys of key_dim and values of value_dim (default: the same); decay: the heads'
        factors g; norm_eps: eps of the output's norm; activation: "silu" (on q, k and v) or None; names: tensor names
        behind the prefix for q, k, v, g, o (matrices) and norm (per value channel of all heads)."""
        self.rt, self.width = rt, int(width)
        self.nh, self.d = int(num_heads), int(key_dim)
        self.dv = int(value_dim) if value_dim is not None else self.d
        if min(self.nh, self.d, self.dv) <= 0:
            raise ValueError("decayed attention: heads and sizes must be positive")
        if self.d > ops.DELTA_MAX_KEY_DIM:
            raise ValueError(f"key size {self.d}: the kernel takes up to {ops.DELTA_MAX_KEY_DIM}")
        self.decays = [float(g) for g in decay]
        if len(self.decays) != self.nh or not all(0.0 <= g <= 1.0 for g in self.decays):
            raise ValueError(f"{len(self.decays)} decays for {self.nh} heads (each between 0 and 1)")
        if activation not in ("silu", None):
            raise ValueError(f"activation {activation!r} ('silu' or None)")
        self.eps, self.silu = float(norm_eps), activation == "silu"
        n = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "norm": "norm"}
        n.update(names or {})
        self.names = {k: prefix + v for k, v in n.items()}
        kd, vd = self.nh * self.d, self.nh * self.dv
        # columns of the input product: queries, keys, values, the output's gate
        self.col = {"q": 0, "k": kd, "v": 2 * kd, "g": 2 * kd + vd}
        self.w_in = self.p_in = self.w_o = self.p_o = self.norm_w = self.decay = self.powers = None

    def cache_need(self) -> Optional[CacheNeed]:
        return None

    def state_need(self) -> Optional[StateNeed]:
        """One float32 row per request: the heads' matrices [H][Dv][D]."""
        return StateNeed((self.nh * self.d * self.dv,), torch.float32)

    def prepare_step(self, ctx) -> Optional[Dict[tuple, np.ndarray]]:
        """The chunks of a step with a portion long enough (one list for every layer that wants it)."""
        if CHUNKS_KEY in ctx.extra_host or not ops.decayed_attention_chunks_take(self.d, self.dv):
            return None
        start = np.asarray(ctx.h_entry_start)
        return {CHUNKS_KEY: plan_chunks(start)} if int((start[1:] - start[:-1]).max()) >= CHUNKS_FROM else None

    def tensors(self) -> Dict[str, TensorDecl]:
        nm, kd, vd = self.names, self.nh * self.d, self.nh * self.dv
        return {
            nm["q"]: TensorDecl((kd, self.width), "matrix"),
            nm["k"]: TensorDecl((kd, self.width), "matrix"),
            nm["v"]: TensorDecl((vd, self.width), "matrix"),
            nm["g"]: TensorDecl((vd, self.width), "matrix"),
            nm["o"]: TensorDecl((self.width, vd), "matrix"),
            nm["norm"]: TensorDecl((vd,), "gain"),
        }

    def load(self, get: Callable[[str], torch.Tensor], rt: Runtime) -> None:
        nm = self.names
        # one product for everything that reads the mixer's input
        self.w_in = torch.cat([rt.place(get(nm[k]), "matrix") for k in ("q", "k", "v", "g")], dim=0).contiguous()
        self.w_o = rt.place(get(nm["o"]), "matrix")
        self.p_in, self.p_o = rt.pack(self.w_in), rt.pack(self.w_o)
        self.w_in, self.w_o = rt.row_major(self.w_in, self.p_in), rt.row_major(self.w_o, self.p_o)
        self.norm_w = rt.place(get(nm["norm"]), "gain")
        self.decay = torch.tensor(self.decays, dtype=torch.float32, device=rt.device)
        powers = np.asarray(self.decays, dtype=np.float64)[:, None] ** np.arange(ops.DECAYED_CHUNK + 1)
        self.powers = torch.from_numpy(powers.astype(np.float32)).to(rt.device)

    def forward(self, x, ctx, cache, state):
        rt, c, vd = self.rt, self.col, self.nh * self.dv
        n = x.shape[0]
        if state is None or state.dim() != 2 or state.shape[1] != self.d * vd:
            raise RuntimeError("the decayed attention mixer was given no state of its shape")
        y = linear(rt, x, self.w_in, None, "dattn.in", packed=self.p_in)        # q, k, v, gate
        o = rt.buffer("dattn.o", (n, vd), torch.float32)
        plan = ctx.extra.get(CHUNKS_KEY) if ops.decayed_attention_chunks_take(self.d, self.dv) else None
        if plan is not None:
            n_chunks = (plan.numel() - ctx.n_entries - 1) // 2
            work = rt.buffer("dattn.chunks", (n_chunks * vd * self.d,), torch.float32)
            ops.decayed_attention_chunked(y, c["q"], c["k"], c["v"], self.powers, state, plan, n_chunks, ctx.state_slots, work, o,
                                          self.nh, self.d, self.dv, silu=self.silu)
        else:
            ops.decayed_attention(y, c["q"], c["k"], c["v"], self.decay, state, ctx.entry_start, ctx.state_slots, o, self.nh,
                                  self.d, self.dv, silu=self.silu, single=ctx.single_token)
        gated = rt.buffer("dattn.gated", (n, vd), rt.dtype)
        # (one norm over all heads: a single head of H Dv channels)
        ops.gated_rmsnorm(o, self.norm_w, y, c["g"], gated, 1, vd, self.eps, gate_kind="sigmoid")
        return linear(rt, gated, self.w_o, None, "dattn.o_proj", packed=self.p_o)
