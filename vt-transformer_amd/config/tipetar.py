"""Tipetar: typed configuration read from the keys of its config.json.

A Tipetar layer has no norm in front of its sublayers: they read the float32
residual stream itself, and their results are normed and join the stream times
a constant (`parts/block.py`: "output_norm"; the norms' tensors hold the gains
less one).  The mixer is softmax attention over a window with a slope per head
on the distance, and with queries and keys normed over the whole projection;
a layer may take the keys and values of an earlier one
(`parts/masked_attention.py`).  The feed-forward is a mixture of SiLU experts
with a softmax router, a correction that takes part in the choice only, groups
of which the best are eligible, choices that hand the input through, and a
shared expert (`parts/moe.py`).

config.json:
  architecture            "Tipetar"
  vocab, width            sizes of the vocabulary and of the stream
  norm.eps                eps of every norm of the model
  residual_mult           factor on a sublayer's normed result (absent: 1)
  layers[i].type          "attention"
  layers[i].mixer         heads, kv_heads, dim, vdim, scale, mask.size (no mask: every earlier key is seen), kv_from (absent
                          or null: keys and values of its own; else the index of the earlier layer that made them)
  layers[i].mlp           null | {kind: "moe", expert.ff, router.{experts, top, scale, identity, groups.{count, keep}},
                          shared: null | {ff}}

Tensor names: embed, head, final.norm, and per layer l<i>.norm1, l<i>.norm2, l<i>.mix.{q, k, v, o, q.norm, k.norm} (a layer
with kv_from: without k, v and k.norm), l<i>.mlp.router, l<i>.mlp.correction, l<i>.mlp.e<j>.{gate, up, down},
l<i>.mlp.shared.{gate, up, down}.

Fixed by the architecture: slopes 2^(-8 (h + 1) / heads); SiLU; a softmax over all of the router's outputs; the chosen
scores divided by their sum + 1e-20; no biases, no rotation.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .base import (ConfigError, LayerSpec, ModelConfig, ModelSpec, PartSpec, ScheduleEntry, read_key, require_positive)

_ATTENTION_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm"}
_MLP_NAMES = {"gate": "gate", "up": "up", "down": "down"}

SLOPE_STEEPNESS = 8.0       # slope of head h: 2^(-SLOPE_STEEPNESS (h + 1) / heads)
RENORM_EPS = 1e-20


def _sub(d: Dict[str, Any], key: str, where: str, optional: bool = False) -> Optional[Dict[str, Any]]:
    v = d.get(key)
    if v is None:
        if optional:
            return None
        raise ConfigError(f"{where}: required key '{key}' is missing")
    if not isinstance(v, dict):
        raise ConfigError(f"{where}: key '{key}' must be an object, got {v!r}")
    return v


@dataclass
class TipetarConfig(ModelConfig):
    vocab: int
    width: int
    norm_eps: float
    layers: List[Dict[str, Any]]
    residual_mult: float = 1.0
    max_positions: int = 1 << 20          # the design sets no limit; the engine's max_seq_len bounds what is run
    eos_token_id: List[int] = field(default_factory=list)

    architecture = "Tipetar"

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "TipetarConfig":
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers or not all(isinstance(x, dict) for x in layers):
            raise ConfigError("config.json: key 'layers' must be a non-empty list of objects")
        eos = d.get("eos_token_id")
        eos_list = [] if eos is None else ([eos] if isinstance(eos, int) else list(eos))
        cfg = cls(
            vocab=read_key(d, "vocab", int),
            width=read_key(d, "width", int),
            norm_eps=read_key(_sub(d, "norm", "config.json"), "eps", float, where="config.json: norm"),
            layers=copy.deepcopy(layers),
            residual_mult=read_key(d, "residual_mult", float, 1.0),
            max_positions=read_key(d, "max_positions", int, 1 << 20),
            eos_token_id=eos_list,
        )
        cfg.check()
        return cfg

    # ------------------------------------------------------------------
    def check(self) -> None:
        require_positive("vocab", self.vocab)
        require_positive("width", self.width)
        require_positive("norm.eps", self.norm_eps)
        for i, L in enumerate(self.layers):
            where = f"config.json: layers[{i}]"
            kind = read_key(L, "type", str, where=where)
            if kind != "attention":
                raise ConfigError(f"{where}: mixer type '{kind}' is not known ('attention' is)")
            m, mw = _sub(L, "mixer", where), where + ".mixer"
            heads, kv = read_key(m, "heads", int, where=mw), read_key(m, "kv_heads", int, where=mw)
            if heads <= 0 or kv <= 0 or heads % kv:
                raise ConfigError(f"{mw}: heads {heads} must be a positive multiple of kv_heads {kv}")
            for key in ("dim", "vdim"):
                require_positive(f"layers[{i}].mixer.{key}", read_key(m, key, int, where=mw))
            require_positive(f"layers[{i}].mixer.scale", read_key(m, "scale", float, where=mw))
            mask = _sub(m, "mask", mw, optional=True)
            if mask is not None:
                require_positive(f"layers[{i}].mixer.mask.size", read_key(mask, "size", int, where=mw + ".mask"))
            self._check_source(i, m, mw)
            mlp = _sub(L, "mlp", where, optional=True)
            if mlp is not None:
                self._check_mlp(i, mlp, where + ".mlp")

    def _check_source(self, i: int, m: Dict[str, Any], where: str) -> None:
        src = read_key(m, "kv_from", int, None, where=where)
        if src is None:
            return
        if not 0 <= src < i:
            raise ConfigError(f"{where}: kv_from {src} is not a layer in front of layer {i}")
        other = self.layers[src]["mixer"]
        if other.get("kv_from") is not None:
            raise ConfigError(f"{where}: kv_from {src} names a layer that has no keys and values of its own")
        for key in ("kv_heads", "dim", "vdim"):
            if int(other[key]) != int(m[key]):
                raise ConfigError(f"{where}: {key} {m[key]}, but layer {src}, whose keys and values it reads, has {other[key]}")

    def _check_mlp(self, i: int, mlp: Dict[str, Any], where: str) -> None:
        kind = read_key(mlp, "kind", str, "moe", where=where)
        if kind != "moe":
            raise ConfigError(f"{where}: kind '{kind}' is not known ('moe' is)")
        expert, ro, rw = _sub(mlp, "expert", where), _sub(mlp, "router", where), where + ".router"
        require_positive(f"layers[{i}].mlp.expert.ff", read_key(expert, "ff", int, where=where + ".expert"))
        experts, top = read_key(ro, "experts", int, where=rw), read_key(ro, "top", int, where=rw)
        identity = read_key(ro, "identity", int, 0, where=rw)
        require_positive(f"layers[{i}].mlp.router.experts", experts)
        if identity < 0:
            raise ConfigError(f"{rw}: identity {identity} must not be negative")
        read_key(ro, "scale", float, 1.0, where=rw)
        groups = _sub(ro, "groups", rw, optional=True)
        count, keep = 1, 1
        if groups is not None:
            count, keep = read_key(groups, "count", int, where=rw + ".groups"), read_key(groups, "keep", int, where=rw + ".groups")
        outputs = experts + identity
        if count < 1 or outputs % count or not 1 <= keep <= count:
            raise ConfigError(f"{rw}.groups: {keep} of {count} equal groups of {outputs} outputs")
        if not 1 <= top <= keep * (outputs // count):
            raise ConfigError(f"{rw}: top {top} of {keep * (outputs // count)} eligible outputs")
        shared = _sub(mlp, "shared", where, optional=True)
        if shared is not None:
            require_positive(f"layers[{i}].mlp.shared.ff", read_key(shared, "ff", int, where=where + ".shared"))

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {
            "architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
            "residual_mult": self.residual_mult, "layers": copy.deepcopy(self.layers),
        }
        if self.max_positions != 1 << 20:
            d["max_positions"] = self.max_positions
        if self.eos_token_id:
            d["eos_token_id"] = list(self.eos_token_id)
        return d

    # ------------------------------------------------------------------
    def _mixer_spec(self, m: Dict[str, Any]) -> PartSpec:
        mask = m.get("mask")
        return PartSpec("masked_attention", {
            "num_heads": int(m["heads"]), "num_kv_heads": int(m["kv_heads"]), "key_dim": int(m["dim"]),
            "value_dim": int(m["vdim"]), "scale": float(m["scale"]), "window": int(mask["size"]) if mask else 0,
            "distance_slopes": SLOPE_STEEPNESS, "whole_norm_eps": self.norm_eps, "own_keys": m.get("kv_from") is None,
            "names": dict(_ATTENTION_NAMES), "prefix": "mix.",
        })

    def _mlp_spec(self, mlp: Dict[str, Any]) -> PartSpec:
        ro, groups, shared = mlp["router"], mlp["router"].get("groups"), mlp.get("shared")
        return PartSpec("expert_mixture", {
            "num_experts": int(ro["experts"]), "top": int(ro["top"]), "intermediate_size": int(mlp["expert"]["ff"]),
            "score": "softmax", "renormalize": True, "renorm_eps": RENORM_EPS, "weight_on": "output", "activation": "silu",
            "correction": True, "groups": {k: int(groups[k]) for k in ("count", "keep")} if groups else None,
            "router_scale": float(ro["scale"]) if ro.get("scale") is not None else 1.0,
            "identity": int(ro.get("identity") or 0),
            "shared_expert": PartSpec("gated_mlp", {"intermediate_size": int(shared["ff"]), "activation": "silu",
                                                    "names": dict(_MLP_NAMES), "weight_suffix": "", "prefix": "shared."})
            if shared else None,
            "prefix": "mlp.",
        })

    def to_spec(self) -> ModelSpec:
        layers, schedule = [], []
        for i, L in enumerate(self.layers):
            mlp = L.get("mlp")
            norms = {"mixer_output": PartSpec("rmsnorm", {"eps": self.norm_eps, "name": "norm1", "unit_offset": True})}
            if mlp is not None:
                norms["feed_forward_output"] = PartSpec("rmsnorm", {"eps": self.norm_eps, "name": "norm2", "unit_offset": True})
            layers.append(LayerSpec(block=PartSpec("output_norm", {"residual_mult": self.residual_mult, "idle_norm": "norm2"}),
                                    mixer=self._mixer_spec(L["mixer"]),
                                    feed_forward=self._mlp_spec(mlp) if mlp is not None else None, norms=norms, prefix=f"l{i}."))
            src = L["mixer"].get("kv_from")
            schedule.append(ScheduleEntry(i, cache_from=int(src) if src is not None else None))
        spec = ModelSpec(
            architecture=self.architecture,
            vocab_size=self.vocab,
            hidden_size=self.width,
            embedding=PartSpec("embedding", {"name": "embed"}),
            layers=layers,
            schedule=schedule,
            final_norm=PartSpec("rmsnorm", {"eps": self.norm_eps, "name": "final.norm", "unit_offset": True}),
            head=PartSpec("linear_head", {"name": "head", "tied_to": None}),
            max_positions=self.max_positions,
            eos_token_ids=list(self.eos_token_id),
        )
        spec.validate()
        return spec
