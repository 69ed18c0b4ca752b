"""Tipetar without a GPU: its configuration (keys, run order, tensors, errors), what its layers ask of the cache, and the
plain implementation's mechanisms on cases whose answers are known."""
import copy
import json
import math
import os
import subprocess
import sys
from types import SimpleNamespace

import pytest
import torch

import plain_tipetar as pt
from tipetar_helpers import CONFIGS, make_weights, moe
from vt_transformer_amd.config import ConfigError, config_from_dict
from vt_transformer_amd.weights.random_init import declared_tensors

DT = torch.float64


def test_parts_schedule_and_tensors_follow_the_configuration():
    cfg = config_from_dict(copy.deepcopy(CONFIGS["A"]))
    spec = cfg.to_spec()
    assert [(e.layer, e.cache_from) for e in spec.schedule] == [(0, None), (1, 0), (2, None), (3, 2), (4, 0)]
    assert all(ls.block.kind == "output_norm" and ls.block.params["residual_mult"] == 0.8 for ls in spec.layers)
    assert [ls.feed_forward is None for ls in spec.layers] == [False, True, False, False, False]
    assert set(spec.layers[0].norms) == {"mixer_output", "feed_forward_output"} and set(spec.layers[1].norms) == {"mixer_output"}
    att = [ls.mixer.params for ls in spec.layers]
    assert [(a["num_heads"], a["key_dim"], a["value_dim"], a["window"], a["own_keys"]) for a in att] == [
        (4, 16, 32, 12, True), (8, 16, 32, 30, False), (3, 20, 10, 7, True), (3, 20, 10, 0, False), (4, 16, 32, 5, False)]
    assert all(a["whole_norm_eps"] == 1e-5 and a["distance_slopes"] == 8.0 for a in att)
    ff = spec.layers[0].feed_forward.params
    assert (ff["num_experts"], ff["top"], ff["identity"], ff["groups"], ff["router_scale"], ff["correction"], ff["score"],
            ff["renormalize"], ff["renorm_eps"], ff["weight_on"]) == (6, 2, 2, {"count": 4, "keep": 2}, 1.7, True, "softmax", True, 1e-20,
                                                                      "output")
    assert ff["shared_expert"].params["intermediate_size"] == 56 and spec.layers[2].feed_forward.params["shared_expert"] is None
    t = declared_tensors(cfg)
    assert t["l0.mix.q.norm"].shape == (64,) and t["l0.mix.k.norm"].shape == (32,) and t["l0.mix.v"].shape == (64, 96)
    assert t["l1.mix.q"].shape == (128, 96) and t["l1.mix.q.norm"].shape == (128,) and t["l1.mix.o"].shape == (96, 8 * 32)
    assert not any(n in t for n in ("l1.mix.k", "l1.mix.v", "l1.mix.k.norm", "l1.mlp.router", "l0.mlp.e6.gate"))
    assert t["l1.norm2"].optional and not t["l0.norm2"].optional
    assert t["l0.mlp.router"].shape == (8, 96) and t["l0.mlp.correction"].shape == (8,) and t["l0.mlp.e5.down"].shape == (96, 40)
    assert t["l0.mlp.shared.gate"].shape == (56, 96) and t["l0.mlp.shared.down"].shape == (96, 56)
    assert t["head"].shape == (211, 96) and t["final.norm"].shape == (96,)
    assert set(make_weights(CONFIGS["A"], 0)) == {k for k, d in t.items() if not d.optional}
    assert config_from_dict(cfg.to_dict()).to_dict() == cfg.to_dict()


def test_what_is_left_out_has_its_neutral_value():
    spec = config_from_dict(copy.deepcopy(CONFIGS["B"])).to_spec()
    assert spec.layers[0].block.params["residual_mult"] == 1.0
    ff = spec.layers[0].feed_forward.params
    assert (ff["identity"], ff["groups"], ff["router_scale"], ff["shared_expert"]) == (0, None, 1.0, None)
    raw = copy.deepcopy(CONFIGS["B"])
    for key in ("identity", "scale"):
        raw["layers"][0]["mlp"]["router"].pop(key)
    raw["layers"][0]["mlp"].pop("shared")
    raw["layers"][0]["mixer"]["kv_from"] = None
    raw["layers"][0]["mixer"]["mask"] = None
    spec = config_from_dict(raw).to_spec()
    assert spec.layers[0].feed_forward.params == ff
    assert spec.layers[0].mixer.params["window"] == 0 and spec.layers[0].mixer.params["own_keys"]


@pytest.mark.parametrize("change,text", [
    (lambda c: c["layers"][0].update(type="delta"), "mixer type"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "multiple"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][1]["mixer"].update(kv_from=1), "in front of"),
    (lambda c: c["layers"][4]["mixer"].update(kv_from=3), "of its own"),
    (lambda c: c["layers"][1]["mixer"].update(vdim=24), "vdim"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=4), "kv_heads"),
    (lambda c: c.pop("norm"), "norm"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "kind"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=3), "equal groups"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=5), "equal groups"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=5), "eligible"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(identity=-1), "identity"),
    (lambda c: c["layers"][0]["mlp"]["shared"].update(ff=0), "shared.ff"),
])
def test_configuration_errors(change, text):
    cfg = copy.deepcopy(CONFIGS["A"])
    change(cfg)
    with pytest.raises(ConfigError, match=text):
        config_from_dict(cfg)


def test_parts_refuse_what_they_do_not_combine():
    from vt_transformer_amd.config.base import PartSpec
    from vt_transformer_amd.parts import FEED_FORWARDS, MIXERS, Runtime
    rt = Runtime(torch.device("cpu"), torch.float32)
    base = dict(num_heads=2, num_kv_heads=1, key_dim=8, whole_norm_eps=1e-5)
    for more in (dict(unit_rms_eps=1e-5), dict(position=PartSpec("rotary", {"theta": 1e4, "dim": 8})), dict(value_mix="source")):
        with pytest.raises(ValueError, match="whole projection"):
            MIXERS.build(PartSpec("masked_attention", {**base, **more}), rt=rt, width=16, prefix="a.", shared={})
    # (a norm over the whole projection has no limit from the kernel that norms heads: larger keys are taken)
    MIXERS.build(PartSpec("masked_attention", {**base, "key_dim": 320}), rt=rt, width=16, prefix="a.", shared={})
    ff = dict(num_experts=4, top=2, intermediate_size=8)
    with pytest.raises(ValueError, match="on the output"):
        FEED_FORWARDS.build(PartSpec("expert_mixture", {**ff, "identity": 1, "weight_on": "input"}), rt=rt, width=16, prefix="f.")
    with pytest.raises(ValueError, match="equal groups"):
        FEED_FORWARDS.build(PartSpec("expert_mixture", {**ff, "groups": {"count": 3, "keep": 1}}), rt=rt, width=16, prefix="f.")
    with pytest.raises(ValueError, match="choices from"):
        FEED_FORWARDS.build(PartSpec("expert_mixture", {**ff, "top": 3, "groups": {"count": 2, "keep": 1}}), rt=rt, width=16, prefix="f.")


def test_a_cache_keeps_what_its_widest_reader_sees():
    """Entries that read another entry's pages widen its window; a reader without a window removes it."""
    from vt_transformer_amd.cache.storage import CacheStorage
    from vt_transformer_amd.config.base import ScheduleEntry
    from vt_transformer_amd.parts import CacheNeed, PageTensor, Runtime
    rt = Runtime(torch.device("cpu"), torch.float32)

    def storage(windows, sources):
        need = lambda w: CacheNeed((PageTensor("k", (1, 4), 1), PageTensor("v", (1, 4), 2)), window=w)     # noqa: E731
        layers = [SimpleNamespace(mixer=SimpleNamespace(cache_need=lambda w=w: need(w))) for w in windows]
        model = SimpleNamespace(layers=layers, schedule=[ScheduleEntry(i, cache_from=s) for i, s in enumerate(sources)])
        return CacheStorage(rt, model, 16, 256, 2, 256)
    s = storage([12, 30, 5, 12], [None, 0, 0, None])
    assert [n.window for n in s.group_needs] == [30, 12] and s.entry_group == [0, 0, 0, 1]
    assert s.entry_index == [0, 0, 0, 0] and s.writes == [True, False, False, True]
    s = storage([12, 0, 5, 0], [None, 0, 0, None])
    assert [n.window for n in s.group_needs] == [0] and s.entry_group == [0, 0, 0, 0] and s.entry_index == [0, 0, 0, 1]
    s = storage([0, 7], [None, 0])
    assert [n.window for n in s.group_needs] == [0]


# ---------------------------------------------------------------------------
# the plain mechanisms on cases with known answers
# ---------------------------------------------------------------------------
def test_norms_known_values():
    x = torch.tensor([[3.0, 4.0, 0.0, 0.0]], dtype=DT)
    assert torch.allclose(pt.over_rms(x, 0.0), x / 2.5)
    assert torch.allclose(pt.over_rms(x, 2.75), x / 3.0)                 # (eps inside the root: 6.25 + 2.75 = 9)
    w = torch.tensor([1.0, -1.0, 0.5, 0.0], dtype=DT)
    assert torch.allclose(pt.offset_rmsnorm(x, w, 0.0), torch.tensor([[2.4, 0.0, 0.0, 0.0]], dtype=DT))
    assert torch.allclose(pt.plain_rmsnorm(x, w, 0.0), torch.tensor([[1.2, -1.6, 0.0, 0.0]], dtype=DT))
    # over the whole projection: a head that is zero leaves its share of the root to the others
    wq = {"q": torch.eye(4, dtype=DT), "q.norm": torch.tensor([1.0, 2.0, 3.0, 4.0], dtype=DT)}
    q = pt.queries(x, wq, "", {"heads": 2, "dim": 2}, 0.0)
    assert torch.allclose(q, torch.tensor([[[1.2, 3.2], [0.0, 0.0]]], dtype=DT))


def test_window_and_slopes():
    assert [pt.head_slope(h, 4) for h in range(4)] == [2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8]
    assert abs(pt.head_slope(0, 3) - 2.0 ** (-8.0 / 3.0)) < 1e-15
    t = 9
    q, k = torch.zeros(t, 8, 2, dtype=DT), torch.zeros(t, 1, 2, dtype=DT)
    v = torch.arange(t, dtype=DT).reshape(t, 1, 1)
    out = pt.attend(q, k, v, 1.0, 3)
    # head 0 of 8 has slope 1/2: weights e^0, e^(-1/2), e^(-1)
    w = [1.0, math.exp(-0.5), math.exp(-1.0)]
    assert abs(float(out[8, 0, 0]) - (8 * w[0] + 7 * w[1] + 6 * w[2]) / sum(w)) < 1e-12
    w = [1.0, math.exp(-1.0 / 256), math.exp(-2.0 / 256)]
    assert abs(float(out[8, 7, 0]) - (8 * w[0] + 7 * w[1] + 6 * w[2]) / sum(w)) < 1e-12
    assert torch.allclose(pt.attend(q, k, v, 1.0, 1)[:, 3, 0], v[:, 0, 0])      # a window of one: the position's own value
    # heads share key heads in runs: of 4 heads on 2 key heads the first two read head 0
    v2 = torch.tensor([1.0, 5.0], dtype=DT).reshape(1, 2, 1).expand(t, 2, 1)
    assert pt.attend(q[:, :4], torch.zeros(t, 2, 2, dtype=DT), v2, 1.0, 0)[4, :, 0].round(decimals=9).tolist() == [1.0, 1.0, 5.0, 5.0]


def test_choice_with_correction_and_groups():
    s = torch.tensor([0.30, 0.05, 0.25, 0.10, 0.20, 0.10], dtype=DT)
    zero = torch.zeros(6, dtype=DT)
    assert pt.choose(s, zero, 2, 1, 1)[0] == [0, 2]
    # the correction turns the choice
    assert pt.choose(s, torch.tensor([-1.0, 0, 0, 0, 0.3, 0], dtype=DT), 2, 1, 1)[0] == [4, 2]
    # three groups of two, two kept: {4, 5} (best 0.2) is left out, so 3 is chosen although 4 scores higher
    assert pt.choose(s, zero, 4, 3, 2)[0] == [0, 2, 3, 1]
    # choice scores below zero: a group left out counts as minus infinity, not as zero
    assert pt.choose(s, torch.full((6,), -2.0, dtype=DT), 4, 3, 2)[0] == [0, 2, 3, 1]
    # a group's score is its largest, not its sum
    assert pt.choose(torch.tensor([0.4, 0.0, 0.0, 0.3, 0.3, 0.0], dtype=DT), zero, 1, 2, 1)[0] == [0]
    # equal scores: the lower index
    assert pt.choose(torch.full((6,), 1 / 6, dtype=DT), zero, 3, 3, 2)[0] == [0, 1, 2]
    assert abs(pt.choose(s, zero, 2, 1, 1)[1] - (0.25 - 0.20) / 0.45) < 1e-12


def test_mixture_weights_identity_and_shared():
    """A router whose logits are the input's channels and experts that write one channel each: the sums are written out."""
    width, ff = 4, 1
    x = torch.tensor([[math.log(4.0), math.log(2.0), 0.0, 0.0]], dtype=DT)       # scores 4/8, 2/8, 1/8, 1/8
    w = {"router": torch.eye(4, dtype=DT), "correction": torch.zeros(4, dtype=DT)}
    silu = lambda z: z / (1.0 + math.exp(-z))       # noqa: E731
    for e in range(2):
        w[f"e{e}.gate"], w[f"e{e}.up"] = torch.tensor([[1.0, 0, 0, 0]], dtype=DT), torch.tensor([[0, 1.0, 0, 0]], dtype=DT)
        w[f"e{e}.down"] = torch.zeros(width, ff, dtype=DT)
        w[f"e{e}.down"][e, 0] = 1.0
    unit = silu(math.log(4.0)) * math.log(2.0)
    mlp = moe(2, 3, ff, identity=2, scale=1.5)
    got = pt.mixture(x, w, "", mlp)
    # chosen: outputs 0, 1 (experts) and 2 (the input itself), weights 4/7, 2/7, 1/7 times 1.5
    want = torch.zeros(1, 4, dtype=DT)
    want[0, 0] += 1.5 * 4 / 7 * unit
    want[0, 1] += 1.5 * 2 / 7 * unit
    want += 1.5 / 7 * x
    assert torch.allclose(got, want)
    w["shared.gate"], w["shared.up"], w["shared.down"] = w["e0.gate"], w["e0.up"], torch.ones(width, ff, dtype=DT)
    mlp["shared"] = {"ff": ff}
    assert torch.allclose(pt.mixture(x, w, "", mlp), want + unit)
    # the correction turns the choice to output 3 and leaves the weights' scores alone
    w["correction"] = torch.tensor([0.0, -1.0, 0.0, 0.5], dtype=DT)
    mlp = moe(2, 2, ff, identity=2)
    got = pt.mixture(x, w, "", mlp)
    want = 1 / 5 * x
    want[0, 0] += 4 / 5 * unit
    assert torch.allclose(got, want)


def test_whole_model_prefix_property_and_layers():
    """Logits at a position depend on the tokens up to it only, every tensor has an effect, and the stream after every
    layer is handed out."""
    cfg = copy.deepcopy(CONFIGS["A"])
    w = {k: v.float() for k, v in make_weights(cfg, 3).items()}
    ids = torch.randint(0, cfg["vocab"], (40,), generator=torch.Generator().manual_seed(1)).tolist()
    streams, margins = [], []
    full = pt.forward(cfg, w, ids, streams, margins)
    assert len(streams) == 5 and streams[0].shape == (40, 96) and len(margins) == 4 and margins[0].shape == (40,)
    assert torch.allclose(pt.forward(cfg, w, ids[:17]), full[:17], atol=1e-9)
    for name in w:
        if ".mlp.e" in name:
            continue
        changed = dict(w)
        changed[name] = w[name] + 0.25 * torch.linspace(-1.0, 1.0, w[name].numel()).reshape(w[name].shape)
        assert float((pt.forward(cfg, changed, ids) - full).abs().max()) > 1e-4, name
    less = copy.deepcopy(cfg)
    less["residual_mult"] = 0.79
    assert float((pt.forward(less, w, ids) - full).abs().max()) > 1e-4
    # an expert of every mixture was somebody's choice, and so was handing the input through
    for i in (0, 2, 4):
        x = streams[i]
        ro = cfg["layers"][i]["mlp"]["router"]
        groups = ro.get("groups") or {"count": 1, "keep": 1}
        chosen = [e for row in torch.softmax(x @ w[f"l{i}.mlp.router"].double().T, dim=-1)
                  for e in pt.choose(row, w[f"l{i}.mlp.correction"].double(), ro["top"], groups["count"], groups["keep"])[0]]
        assert min(chosen) < ro["experts"] <= max(chosen)


def test_random_model_from_the_command_line(tmp_path):
    """`--write-random-model` on a Tipetar config.json: every declared tensor is written and the folder loads back."""
    from vt_transformer_amd.config import load_config
    from vt_transformer_amd.weights import WeightStore
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg_path = tmp_path / "c.json"
    cfg_path.write_text(json.dumps(CONFIGS["A"]))
    out = tmp_path / "m"
    r = subprocess.run([sys.executable, "-m", "vt_transformer_amd", "--write-random-model", str(out), "--config", str(cfg_path),
                        "--seed", "4"], capture_output=True, text=True, env=dict(os.environ, PYTHONPATH=root), timeout=300)
    assert r.returncode == 0, r.stderr
    cfg = load_config(str(out))
    assert cfg.to_dict() == config_from_dict(copy.deepcopy(CONFIGS["A"])).to_dict()
    assert set(WeightStore(str(out)).names()) == {k for k, d in declared_tensors(cfg).items() if not d.optional}
    _, w = pt.read_folder(str(out))
    assert torch.isfinite(pt.forward(cfg.to_dict(), w, [3, 1, 4, 1, 5, 9, 2, 6])).all()
