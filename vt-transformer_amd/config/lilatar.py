"""Lilatar: typed configuration read from the keys of its config.json.

A Lilatar layer norms what goes into a sublayer and what comes out of it
(`parts/block.py`: "sandwich") around a float32 residual stream.  Two mixers:
"lightning", linear attention with a constant decay per head
(`parts/decayed_attention.py`), and "parallel", two mixers side by side whose
results are normed and averaged (`parts/mixer_pair.py`): capped softmax
attention in a window that keeps a sequence's first tokens, with biases and
rotation of neighbouring elements (`parts/masked_attention.py`), beside a gated
delta rule with a decay per key channel (`parts/gated_delta.py`).  The
feed-forwards have no gate: the square of ReLU, dense or as a mixture of
softmax-routed experts (`parts/feedforward.py`, `parts/moe.py`).  The logits
are multiplied by a constant.

config.json:
  architecture            "Lilatar"
  vocab, width            sizes of the vocabulary and of the stream
  norm.eps                eps of every norm of the model (also of the mixers' own)
  logit_scale             factor on the logits (absent: 1)
  layers[i].type          "lightning" | "parallel"
  layers[i].mixer         lightning: heads, dim, vdim, decay (one factor per head)
                          parallel:  left.{heads, kv_heads, dim, vdim, scale, softcap, mask.{size, keep_first}, rot.{dims, base,
                                     scaling.{factor, original, low, high}}} (softcap, mask, rot and rot.scaling may be absent),
                                     right.{heads, kv_heads, dim, vdim, conv} (and optionally a_rank, g_rank)
  layers[i].mlp           null | {kind: "dense", ff} | {kind: "moe", expert.ff, router.{experts, top}}

The sizes of the delta rule's two low-rank projections are the rows of its tensors a1 and g1; a config.json that is
written for random weights says them as right.a_rank and right.g_rank.

Tensor names: embed, head, final.norm, and per layer l<i>.{norm1, norm1b, norm2, norm2b}; l<i>.mix.{q, k, v, g, o, norm}
(lightning), l<i>.mix.left.{q, k, v, o} and their biases with ".b", l<i>.mix.right.{q, k, v, b, a1, a2, g1, g2, o, A_log,
dt_bias, norm} and convolutions with ".conv", l<i>.mix.{left, right}.out; l<i>.mlp.{up, down} or l<i>.mlp.router and
l<i>.mlp.e<j>.{up, down}.

Fixed by the architecture: SiLU on the lightning mixer's projections; the mean of the pair; sigmoid gates; a softmax over
all experts whose chosen scores are the weights; 1e-6 inside the root of the delta rule's unit vectors (in the kernel).
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .base import (ConfigError, LayerSpec, ModelConfig, ModelSpec, PartSpec, ScheduleEntry, read_key, require_positive)

_LIGHTNING_NAMES = {"q": "q", "k": "k", "v": "v", "g": "g", "o": "o", "norm": "norm"}
_LEFT_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_bias": "q.b", "k_bias": "k.b", "v_bias": "v.b", "o_bias": "o.b"}
_RIGHT_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_conv": "q.conv", "k_conv": "k.conv", "v_conv": "v.conv",
                "b": "b", "a1": "a1", "a2": "a2", "g1": "g1", "g2": "g2", "A_log": "A_log", "dt_bias": "dt_bias", "norm": "norm"}
_SCALING_KEYS = ("factor", "original", "low", "high")


def _sub(d: Dict[str, Any], key: str, where: str, optional: bool = False) -> Optional[Dict[str, Any]]:
    v = d.get(key)
    if v is None:
        if optional:
            return None
        raise ConfigError(f"{where}: required key '{key}' is missing")
    if not isinstance(v, dict):
        raise ConfigError(f"{where}: key '{key}' must be an object, got {v!r}")
    return v


def _positive(d: Dict[str, Any], key: str, typ, where: str):
    v = read_key(d, key, typ, where=where)
    if not v > 0:
        raise ConfigError(f"{where}: '{key}' must be positive, got {v!r}")
    return v


def _grouped_heads(m: Dict[str, Any], where: str) -> None:
    heads, kv = _positive(m, "heads", int, where), _positive(m, "kv_heads", int, where)
    if heads % kv:
        raise ConfigError(f"{where}: heads {heads} must be a multiple of kv_heads {kv}")
    for key in ("dim", "vdim"):
        _positive(m, key, int, where)


@dataclass
class LilatarConfig(ModelConfig):
    vocab: int
    width: int
    norm_eps: float
    layers: List[Dict[str, Any]]
    logit_scale: float = 1.0
    max_positions: int = 1 << 20          # the design sets no limit; the engine's max_seq_len bounds what is run
    eos_token_id: List[int] = field(default_factory=list)

    architecture = "Lilatar"

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "LilatarConfig":
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
            logit_scale=read_key(d, "logit_scale", float, 1.0),
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
            m, mw = _sub(L, "mixer", where), where + ".mixer"
            if kind == "lightning":
                self._check_lightning(m, mw)
            elif kind == "parallel":
                self._check_left(_sub(m, "left", mw), mw + ".left")
                self._check_right(_sub(m, "right", mw), mw + ".right")
            else:
                raise ConfigError(f"{where}: mixer type '{kind}' is not known ('lightning' and 'parallel' are)")
            mlp = _sub(L, "mlp", where, optional=True)
            if mlp is not None:
                self._check_mlp(mlp, where + ".mlp")

    @staticmethod
    def _check_lightning(m: Dict[str, Any], where: str) -> None:
        heads = _positive(m, "heads", int, where)
        for key in ("dim", "vdim"):
            _positive(m, key, int, where)
        decay = read_key(m, "decay", list, where=where)
        if len(decay) != heads or not all(isinstance(g, (int, float)) and not isinstance(g, bool) and 0 <= g <= 1 for g in decay):
            raise ConfigError(f"{where}: 'decay' must hold a factor between 0 and 1 for each of {heads} heads, got {decay!r}")

    @staticmethod
    def _check_left(m: Dict[str, Any], where: str) -> None:
        _grouped_heads(m, where)
        _positive(m, "scale", float, where)
        if read_key(m, "softcap", float, 0.0, where=where) < 0:
            raise ConfigError(f"{where}: softcap must not be negative")
        mask = _sub(m, "mask", where, optional=True)
        if mask is not None:
            _positive(mask, "size", int, where + ".mask")
            if read_key(mask, "keep_first", int, 0, where=where + ".mask") < 0:
                raise ConfigError(f"{where}.mask: keep_first must not be negative")
        rot = _sub(m, "rot", where, optional=True)
        if rot is not None:
            dims = read_key(rot, "dims", int, where=where + ".rot")
            if dims <= 0 or dims % 2 or dims > m["dim"]:
                raise ConfigError(f"{where}.rot: dims {dims} must be even, positive and at most dim {m['dim']}")
            _positive(rot, "base", float, where + ".rot")
            sc = _sub(rot, "scaling", where + ".rot", optional=True)
            if sc is not None:
                for key in _SCALING_KEYS:
                    _positive(sc, key, float, where + ".rot.scaling")

    @staticmethod
    def _check_right(m: Dict[str, Any], where: str) -> None:
        _grouped_heads(m, where)
        _positive(m, "conv", int, where)
        for key in ("a_rank", "g_rank"):
            if m.get(key) is not None:
                _positive(m, key, int, where)

    @staticmethod
    def _check_mlp(mlp: Dict[str, Any], where: str) -> None:
        kind = read_key(mlp, "kind", str, where=where)
        if kind == "dense":
            _positive(mlp, "ff", int, where)
        elif kind == "moe":
            _positive(_sub(mlp, "expert", where), "ff", int, where + ".expert")
            ro, rw = _sub(mlp, "router", where), where + ".router"
            experts, top = _positive(ro, "experts", int, rw), _positive(ro, "top", int, rw)
            if top > experts:
                raise ConfigError(f"{rw}: top {top} of {experts} experts")
        else:
            raise ConfigError(f"{where}: kind '{kind}' is not known ('dense' and 'moe' are)")

    def take_tensor_shapes(self, shapes: Dict[str, Any]) -> None:
        """The sizes of a delta rule's low-rank projections are the rows of its tensors a1 (decay) and g1 (gate)."""
        for i, L in enumerate(self.layers):
            if L["type"] != "parallel":
                continue
            right = L["mixer"]["right"]
            for key, tensor in (("a_rank", f"l{i}.mix.right.a1"), ("g_rank", f"l{i}.mix.right.g1")):
                shape = shapes.get(tensor)
                if shape is None or len(shape) != 2:
                    continue
                said = right.get(key)
                if said is not None and int(said) != int(shape[0]):
                    raise ConfigError(f"config.json: layers[{i}].mixer.right.{key} is {said}, the tensor {tensor} has {shape[0]} rows")
                right[key] = int(shape[0])

    def to_dict(self) -> Dict[str, Any]:
        d: Dict[str, Any] = {
            "architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
            "logit_scale": self.logit_scale, "layers": copy.deepcopy(self.layers),
        }
        if self.max_positions != 1 << 20:
            d["max_positions"] = self.max_positions
        if self.eos_token_id:
            d["eos_token_id"] = list(self.eos_token_id)
        return d

    # ------------------------------------------------------------------
    def _mixer_spec(self, i: int, L: Dict[str, Any]) -> PartSpec:
        m = L["mixer"]
        if L["type"] == "lightning":
            return PartSpec("decayed_attention", {
                "num_heads": int(m["heads"]), "key_dim": int(m["dim"]), "value_dim": int(m["vdim"]),
                "decay": [float(g) for g in m["decay"]], "norm_eps": self.norm_eps, "names": dict(_LIGHTNING_NAMES), "prefix": "mix.",
            })
        left, right = m["left"], m["right"]
        if right.get("a_rank") is None or right.get("g_rank") is None:
            raise ConfigError(f"config.json: layers[{i}].mixer.right: the sizes of the low-rank projections are not known "
                              f"(the tensors l{i}.mix.right.a1 and g1 give them, or the keys a_rank and g_rank)")
        mask, rot, position = left.get("mask"), left.get("rot"), None
        if rot is not None:
            sc = rot.get("scaling")
            scaling = {"kind": "bands", **{k: float(sc[k]) for k in _SCALING_KEYS}} if sc else None
            position = PartSpec("rotary", {"theta": float(rot["base"]), "dim": int(rot["dims"]), "scaling": scaling})
        left_spec = PartSpec("masked_attention", {
            "num_heads": int(left["heads"]), "num_kv_heads": int(left["kv_heads"]), "key_dim": int(left["dim"]),
            "value_dim": int(left["vdim"]), "qkv_bias": True, "o_bias": True, "position": position, "rot_pairs": "neighbours",
            "scale": float(left["scale"]), "softcap": float(left.get("softcap") or 0.0),
            "window": int(mask["size"]) if mask else 0, "keep_first": int(mask.get("keep_first") or 0) if mask else 0,
            "names": dict(_LEFT_NAMES), "prefix": "left.",
        })
        right_spec = PartSpec("gated_delta", {
            "num_heads": int(right["heads"]), "num_kv_heads": int(right["kv_heads"]), "key_dim": int(right["dim"]),
            "value_dim": int(right["vdim"]), "conv_taps": int(right["conv"]), "norm_eps": self.norm_eps,
            "decay": "channel", "decay_rank": int(right["a_rank"]), "gate_rank": int(right["g_rank"]), "gate_act": "sigmoid",
            "names": dict(_RIGHT_NAMES), "prefix": "right.",
        })
        return PartSpec("mixer_pair", {
            "left": left_spec, "right": right_spec, "left_scale": 0.5, "right_scale": 0.5,
            "out_norms": {"eps": self.norm_eps, "left": "left.out", "right": "right.out"}, "prefix": "mix.",
        })

    @staticmethod
    def _mlp_spec(mlp: Dict[str, Any]) -> PartSpec:
        if mlp["kind"] == "dense":
            return PartSpec("plain_mlp", {"intermediate_size": int(mlp["ff"]), "activation": "squared_relu", "prefix": "mlp."})
        ro = mlp["router"]
        return PartSpec("expert_mixture", {
            "num_experts": int(ro["experts"]), "top": int(ro["top"]), "intermediate_size": int(mlp["expert"]["ff"]),
            "score": "softmax", "weight_on": "output", "activation": "squared_relu", "prefix": "mlp.",
        })

    def to_spec(self) -> ModelSpec:
        def norm(name: str) -> PartSpec:
            return PartSpec("rmsnorm", {"eps": self.norm_eps, "name": name})
        layers = []
        for i, L in enumerate(self.layers):
            mlp = L.get("mlp")
            norms = {"input": norm("norm1"), "mixer_output": norm("norm1b")}
            if mlp is not None:
                norms.update({"post_mixer": norm("norm2"), "feed_forward_output": norm("norm2b")})
            layers.append(LayerSpec(block=PartSpec("sandwich", {"idle_norms": ("norm2", "norm2b")}), mixer=self._mixer_spec(i, L),
                                    feed_forward=self._mlp_spec(mlp) if mlp is not None else None, norms=norms, prefix=f"l{i}."))
        spec = ModelSpec(
            architecture=self.architecture,
            vocab_size=self.vocab,
            hidden_size=self.width,
            embedding=PartSpec("embedding", {"name": "embed"}),
            layers=layers,
            schedule=[ScheduleEntry(i) for i in range(len(layers))],
            # (the factor on the logits goes in with the gains of the norm in front of the head)
            final_norm=PartSpec("rmsnorm", {"eps": self.norm_eps, "name": "final.norm", "factor": self.logit_scale}),
            head=PartSpec("linear_head", {"name": "head", "tied_to": None}),
            max_positions=self.max_positions,
            eos_token_ids=list(self.eos_token_id),
        )
        spec.validate()
        return spec
