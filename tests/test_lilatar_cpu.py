"""Lilatar without a GPU: its configuration (keys, parts, tensors, errors), what its layers ask of the cache, the pages
that a window with kept tokens holds, the chunks of a step, the table of angles, and the plain implementation's mechanisms
on cases whose answers are known."""
import copy
import json
import math
import os
import random
import subprocess
import sys
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import plain_lilatar as pl
from lilatar_helpers import CONFIGS, lightning, make_weights, moe, pair
from vt_transformer_amd.config import ConfigError, config_from_dict
from vt_transformer_amd.weights.random_init import declared_tensors

DT = torch.float64


def test_parts_and_tensors_follow_the_configuration():
    cfg = config_from_dict(copy.deepcopy(CONFIGS["A"]))
    spec = cfg.to_spec()
    assert [ls.mixer.kind for ls in spec.layers] == ["mixer_pair", "decayed_attention", "mixer_pair", "decayed_attention"]
    assert [ls.feed_forward.kind if ls.feed_forward else None for ls in spec.layers] == ["plain_mlp", "expert_mixture", "expert_mixture", None]
    assert all(ls.block.kind == "sandwich" for ls in spec.layers)
    assert set(spec.layers[0].norms) == {"input", "mixer_output", "post_mixer", "feed_forward_output"}
    assert set(spec.layers[3].norms) == {"input", "mixer_output"}
    left, right = spec.layers[0].mixer.params["left"].params, spec.layers[0].mixer.params["right"].params
    assert (left["num_heads"], left["num_kv_heads"], left["key_dim"], left["value_dim"], left["scale"], left["softcap"], left["window"],
            left["keep_first"], left["rot_pairs"], left["qkv_bias"], left["o_bias"]) == (4, 2, 16, 32, 0.3, 6.0, 12, 5, "neighbours", True, True)
    assert left["position"].params == {"theta": 3000.0, "dim": 8, "scaling": {"kind": "bands", "factor": 4.0, "original": 64.0, "low": 1.0,
                                                                            "high": 4.0}}
    assert (right["num_heads"], right["num_kv_heads"], right["conv_taps"], right["decay_rank"], right["gate_rank"]) == (2, 1, 3, 6, 5)
    assert spec.layers[0].mixer.params["out_norms"] == {"eps": 1e-5, "left": "left.out", "right": "right.out"}
    assert spec.layers[3].mixer.params["decay"] == [0.9, 0.999]
    assert spec.final_norm.params["factor"] == 0.3
    tensors = declared_tensors(cfg)
    assert tensors["l0.mix.left.o.b"].shape == (96,) and tensors["l0.mix.right.a2"].shape == (32, 6)
    assert tensors["l0.mix.right.dt_bias"].shape == (32,) and tensors["l0.mix.right.A_log"].shape == (2,)
    assert tensors["l0.mix.left.out"].shape == tensors["l0.mix.right.out"].shape == (96,)
    assert tensors["l1.mix.norm"].shape == (72,) and tensors["l1.mix.g"].shape == (72, 96)
    assert "l0.mlp.gate" not in tensors and "l1.mlp.e0.gate" not in tensors and tensors["l1.mlp.e5.down"].shape == (96, 40)
    assert tensors["l3.norm2"].optional and tensors["l3.norm2b"].optional and not tensors["l0.norm2b"].optional
    assert cfg.to_dict() == config_from_dict(cfg.to_dict()).to_dict()


def test_what_may_be_left_out_has_its_neutral_value():
    left = config_from_dict(copy.deepcopy(CONFIGS["B"])).to_spec().layers[1].mixer.params["left"].params
    assert (left["softcap"], left["window"], left["keep_first"], left["position"]) == (0.0, 0, 0, None)
    raw = copy.deepcopy(CONFIGS["B"])
    raw.pop("logit_scale")
    raw["layers"][1]["mixer"]["left"].update(softcap=None, mask=None, rot=None)
    raw["layers"][2]["mixer"]["left"]["rot"]["scaling"] = None
    spec = config_from_dict(raw).to_spec()
    assert spec.final_norm.params["factor"] == 1.0 and spec.layers[1].mixer.params["left"].params == left
    assert spec.layers[2].mixer.params["left"].params["position"].params["scaling"] is None


def test_low_rank_sizes_come_from_the_tensors():
    raw = copy.deepcopy(CONFIGS["A"])
    for i in (0, 2):
        raw["layers"][i]["mixer"]["right"].pop("a_rank"), raw["layers"][i]["mixer"]["right"].pop("g_rank")
    cfg = config_from_dict(raw)
    with pytest.raises(ConfigError, match="low-rank"):
        cfg.to_spec()
    cfg.take_tensor_shapes({k: v.shape for k, v in make_weights(CONFIGS["A"], 1).items()})
    assert cfg.to_dict() == config_from_dict(copy.deepcopy(CONFIGS["A"])).to_dict()
    with pytest.raises(ConfigError, match="rows"):
        cfg.take_tensor_shapes({"l0.mix.right.a1": (9, 96)})


@pytest.mark.parametrize("change,text", [
    (lambda c: c["layers"][0].update(type="attention"), "mixer type"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=3), "multiple"),
    (lambda c: c["layers"][0]["mixer"]["left"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(softcap=-1.0), "softcap"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(keep_first=-1), "keep_first"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=18), "dims"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"]["scaling"].pop("low"), "low"),
    (lambda c: c["layers"][0]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(conv=0), "conv"),
    (lambda c: c["layers"][1]["mixer"].update(decay=[0.5]), "decay"),
    (lambda c: c["layers"][1]["mixer"]["decay"].__setitem__(0, 1.5), "decay"),
    (lambda c: c["layers"][1]["mixer"].update(vdim=0), "vdim"),
    (lambda c: c["layers"][1]["mlp"].update(kind="gated"), "kind"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=7), "top"),
    (lambda c: c["layers"][0]["mlp"].update(ff=0), "ff"),
    (lambda c: c.pop("norm"), "norm"),
    (lambda c: c.update(layers=[]), "layers"),
])
def test_configuration_errors(change, text):
    cfg = copy.deepcopy(CONFIGS["A"])
    change(cfg)
    with pytest.raises(ConfigError, match=text):
        config_from_dict(cfg)


def test_parts_refuse_what_they_do_not_combine():
    from vt_transformer_amd.config.base import PartSpec
    from vt_transformer_amd.parts import FEED_FORWARDS, MIXERS, POSITIONS, Runtime
    rt = Runtime(torch.device("cpu"), torch.float32)
    base = dict(num_heads=2, num_kv_heads=1, key_dim=8)
    for more in (dict(keep_first=4), dict(keep_first=4, window=8, chunk=8), dict(keep_first=-1, window=8)):
        with pytest.raises(ValueError, match="keep_first"):
            MIXERS.build(PartSpec("masked_attention", {**base, **more}), rt=rt, width=16, prefix="a.", shared={})
    for decay in ([0.5], [0.5, 1.1], [0.5, -0.1]):
        with pytest.raises(ValueError, match="decays"):
            MIXERS.build(PartSpec("decayed_attention", dict(num_heads=2, key_dim=8, decay=decay, norm_eps=1e-5)), rt=rt, width=16, prefix="a.")
    with pytest.raises(ValueError, match="without a gate"):
        FEED_FORWARDS.build(PartSpec("expert_mixture", dict(num_experts=4, top=2, intermediate_size=8, activation="squared_relu")), rt=rt,
                            width=16, prefix="f.")
    with pytest.raises(ValueError, match="scaling"):
        POSITIONS.build(PartSpec("rotary", dict(theta=1e4, dim=8, scaling={"kind": "bands", "factor": 2.0, "original": 8, "low": 1.0})), rt=rt)
    with pytest.raises(ValueError, match="not known"):
        POSITIONS.build(PartSpec("rotary", dict(theta=1e4, dim=8, scaling={"kind": "steps", "factor": 2.0})), rt=rt)


# ---------------------------------------------------------------------------
# pages of a window that keeps a sequence's first tokens
# ---------------------------------------------------------------------------
def kept_manager(keep, window=5, page=4, pages=16):
    from vt_transformer_amd.cache.pages import CacheManager, GroupSpec
    return CacheManager([GroupSpec("k", window, pages, keep)], page, 4, 4096)


def test_the_first_pages_stay_and_the_middle_is_given_back():
    from vt_transformer_amd.cache.pages import NO_PAGE
    for keep, stay in ((0, 0), (1, 1), (4, 1), (5, 2), (9, 3)):
        m = kept_manager(keep)
        m.admit("r")
        first = None
        for n in range(1, 60):
            assert m.reserve([("r", n)])
            m.commit("r", n)
            m.check()
            table = m.get("r").tables[0]
            if n == 12:
                first = table[:stay]
            if n >= 12:
                assert table[:stay] == first and NO_PAGE not in first        # the same pages, never moved
            oldest_seen = max(0, n - 5 + 1) // 4
            assert all(p == NO_PAGE for p in table[stay:oldest_seen]) and NO_PAGE not in table[max(stay, oldest_seen):]
            assert m.held_pages()[0] <= m.max_held_pages(0, 1)
        m.release("r")
        assert m.available_pages() == [16]


def test_pages_through_random_traffic_with_kept_tokens():
    from vt_transformer_amd.cache.pages import NO_PAGE
    rng = random.Random(7)
    m = kept_manager(keep=10, window=17, page=8, pages=40)
    live = {}
    for step in range(400):
        if len(live) < 4 and rng.random() < 0.4:
            rid = f"q{step}"
            m.admit(rid)
            live[rid] = 0
        for rid in list(live):
            grow = rng.choice([1, 1, 2, 9, 30])
            if m.reserve([(rid, live[rid] + grow)]):
                live[rid] += grow
                m.commit(rid, live[rid])
            m.check()
            n, table = live[rid], m.get(rid).tables[0]
            needed = {j // 8 for j in range(n) if j < 10 or j > n - 17}
            assert all(table[b] != NO_PAGE for b in needed)
            assert m.held_pages()[0] <= 40
            if n > 150 or rng.random() < 0.05:
                m.release(rid)
                del live[rid]
    for rid in list(live):
        m.release(rid)
    assert m.available_pages() == [40]


def test_groups_and_budget_know_the_kept_tokens():
    from vt_transformer_amd.cache.storage import CacheStorage, group_pages
    from vt_transformer_amd.config.base import ScheduleEntry
    from vt_transformer_amd.parts import CacheNeed, PageTensor, Runtime
    rt = Runtime(torch.device("cpu"), torch.float32)

    def need(window, keep):
        return CacheNeed((PageTensor("k", (1, 4), 1), PageTensor("v", (1, 4), 2)), window=window, keep_first=keep)

    def storage(needs, sources):
        layers = [SimpleNamespace(mixer=SimpleNamespace(cache_need=lambda n=n: n)) for n in needs]
        return CacheStorage(rt, SimpleNamespace(layers=layers, schedule=[ScheduleEntry(i, cache_from=s) for i, s in enumerate(sources)]),
                            16, 256, 2, 256)
    s = storage([need(12, 4), need(12, 4), need(12, 0), need(30, 4)], [None] * 4)
    assert s.entry_group == [0, 0, 1, 2] and [g.keep_first for g in s.manager.groups] == [4, 0, 4]
    # a reader that keeps more of the first tokens, and one that sees everything
    s = storage([need(12, 4), need(9, 20), need(12, 4)], [None, 0, None])
    assert [(g.window, g.keep_first) for g in s.manager.groups] == [(12, 20), (12, 4)]
    s = storage([need(12, 4), need(0, 0)], [None, 0])
    assert [(g.window, g.keep_first) for g in s.manager.groups] == [(0, 0)]
    # three requests, window 8 and portions of 8 in pages of 4: 5 pages and one of head-room each, and 3 for ten kept tokens
    assert group_pages([need(8, 0)], [100], 4, 3, 256, 8, 10 ** 6) == [18]
    assert group_pages([need(8, 10)], [100], 4, 3, 256, 8, 10 ** 6) == [27]


def test_chunks_of_a_step():
    from vt_transformer_amd.parts.decayed_attention import plan_chunks
    got = plan_chunks([0, 1, 130, 194, 195, 259])
    assert got[:6].tolist() == [0, 1, 4, 5, 6, 7]
    assert got[6:].reshape(-1, 2).tolist() == [[0, 1], [1, 64], [65, 64], [129, 1], [130, 64], [194, 1], [195, 64]]
    for seed in range(20):
        rs = np.random.RandomState(seed)
        start = np.concatenate([[0], np.cumsum(rs.randint(1, 300, size=rs.randint(1, 6)))])
        got = plan_chunks(start)
        first, runs = got[:len(start)], got[len(start):].reshape(-1, 2)
        for e in range(len(start) - 1):
            mine = runs[first[e]:first[e + 1]]
            rows = [r for a, n in mine for r in range(a, a + n)]
            assert rows == list(range(start[e], start[e + 1])) and all(n == 64 for _, n in mine[:-1])


def test_table_of_angles_in_bands():
    from vt_transformer_amd.parts.rotary import rotary_table
    for dims, base, sc in ((16, 10000.0, dict(factor=8.0, original=100.0, low=1.0, high=4.0)),
                           (64, 700.0, dict(factor=2.5, original=33.0, low=0.5, high=9.0)),
                           (8, 50.0, dict(factor=4.0, original=4.0, low=1.0, high=4.0))):
        cos, sin = rotary_table(50, dims, base, {"kind": "bands", **sc})
        freq = pl.pair_frequencies(dims, base, sc)
        ang = np.arange(50)[:, None] * np.asarray(freq)[None]
        assert np.abs(cos - np.cos(ang)).max() < 1e-6 and np.abs(sin - np.sin(ang)).max() < 1e-6
        plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
        ratio = np.asarray(freq) / np.asarray(plain)
        assert ratio.max() <= 1.0 + 1e-12 and ratio.min() >= 1.0 / sc["factor"] - 1e-12 and (np.diff(ratio) <= 1e-12).all()
    # the three bands by hand: wavelengths of 2 pi (kept), 2 pi 5 (mixed) and 2 pi 25 (slowed down) against 30 positions
    f = pl.pair_frequencies(6, 125.0, dict(factor=10.0, original=60.0, low=1.0, high=4.0))
    turns = 60.0 / (2.0 * math.pi * 5.0)
    s = (turns - 1.0) / 3.0
    assert abs(f[0] - 1.0) < 1e-12 and abs(f[1] - 0.2 * (s + (1.0 - s) / 10.0)) < 1e-12 and abs(f[2] - 0.004) < 1e-12


# ---------------------------------------------------------------------------
# the plain mechanisms on cases with known answers
# ---------------------------------------------------------------------------
def test_window_with_kept_tokens():
    seen = pl.visible(9, 3, 2)
    assert [seen[8].nonzero().flatten().tolist(), seen[3].nonzero().flatten().tolist(), seen[1].nonzero().flatten().tolist()] == [
        [0, 1, 6, 7, 8], [0, 1, 2, 3], [0, 1]]
    assert torch.equal(pl.visible(9, 0, 0), torch.ones(9, 9).tril().bool()) and torch.equal(pl.visible(9, 20, 0), pl.visible(9, 0, 0))
    v = torch.arange(9, dtype=DT).reshape(9, 1, 1)
    zero = torch.zeros(9, 2, 4, dtype=DT)
    out = pl.attend(zero, zero[:, :1], v, 1.0, 0.0, seen)
    assert torch.allclose(out[8, :, 0], torch.full((2,), (0 + 1 + 6 + 7 + 8) / 5.0, dtype=DT))


def test_capped_scores():
    q = torch.tensor([[[1.0]], [[3.0]]], dtype=DT)
    k, v = torch.tensor([[[2.0]], [[-1.0]]], dtype=DT), torch.tensor([[[1.0]], [[0.0]]], dtype=DT)
    s0, s1 = 5.0 * math.tanh(0.5 * 6.0 / 5.0), 5.0 * math.tanh(0.5 * -3.0 / 5.0)
    want = math.exp(s0) / (math.exp(s0) + math.exp(s1))
    assert abs(float(pl.attend(q, k, v, 0.5, 5.0, pl.visible(2, 0, 0))[1, 0, 0]) - want) < 1e-12


def test_rotation_of_neighbours():
    x = torch.zeros(4, 1, 6, dtype=DT)
    x[..., 0], x[..., 2], x[..., 4] = 1.0, 1.0, 7.0
    y = pl.rotate(x, {"dims": 4, "base": 100.0})
    assert torch.allclose(y[3, 0], torch.tensor([math.cos(3.0), math.sin(3.0), math.cos(0.3), math.sin(0.3), 7.0, 0.0], dtype=DT))
    assert torch.equal(pl.rotate(x, None), x)
    # a score hangs on the distance alone
    a = pl.rotate(torch.randn(1, 1, 6, generator=torch.Generator().manual_seed(1), dtype=DT).expand(9, 1, 6), {"dims": 6, "base": 20.0})
    b = pl.rotate(torch.randn(1, 1, 6, generator=torch.Generator().manual_seed(2), dtype=DT).expand(9, 1, 6), {"dims": 6, "base": 20.0})
    assert abs(float((a[7] * b[4]).sum() - (a[5] * b[2]).sum())) < 1e-12


def test_decayed_attention_is_its_recurrence():
    g = torch.Generator().manual_seed(3)
    q, k, v = (torch.randn(12, 2, n, generator=g, dtype=DT) for n in (3, 3, 5))
    out = pl.decayed_attention(q, k, v, [0.7, 1.0])
    for h, decay in enumerate((0.7, 1.0)):
        S = torch.zeros(3, 5, dtype=DT)
        for t in range(12):
            S = decay * S + torch.outer(k[t, h], v[t, h])
            assert torch.allclose(out[t, h], S.T @ q[t, h])
    # one key that lies along one element: its value returns times decay^distance
    k = torch.zeros(8, 1, 2, dtype=DT)
    k[2, 0, 0] = 1.0
    q, v = torch.ones(8, 1, 2, dtype=DT), torch.full((8, 1, 1), 3.0, dtype=DT)
    assert torch.allclose(pl.decayed_attention(q, k, v, [0.5])[:, 0, 0], torch.tensor([0, 0, 3, 1.5, 0.75, 0.375, 0.1875, 0.09375], dtype=DT))
    # nothing is kept at a decay of zero
    assert pl.decayed_attention(q, k, v, [0.0])[:, 0, 0].tolist() == [0, 0, 3, 0, 0, 0, 0, 0]


def test_delta_rule_and_convolution():
    # writing the same key twice with full strength leaves the second value; the decay acts on its own channel only
    q = torch.tensor([[1.0, 0], [1.0, 0], [0, 1.0], [1.0, 0]], dtype=DT).reshape(4, 1, 2)
    k = torch.tensor([[1.0, 0], [1.0, 0], [0, 1.0], [0, 1.0]], dtype=DT).reshape(4, 1, 2)
    v = torch.tensor([2.0, 5.0, 7.0, 9.0], dtype=DT).reshape(4, 1, 1)
    g = torch.ones(4, 1, 2, dtype=DT)
    g[3, 0, 0] = 0.5
    assert pl.delta_rule(q, k, v, torch.ones(4, 1, dtype=DT), g)[:, 0, 0].tolist() == [2.0, 5.0, 7.0, 2.5]
    taps = torch.tensor([[0.5, 2.0, 1.0]], dtype=DT)
    x = torch.tensor([[1.0], [10.0], [100.0]], dtype=DT)
    assert torch.allclose(pl.conv_silu(x, taps)[:, 0], pl.silu(torch.tensor([1.0, 12.0, 120.5], dtype=DT)))


def test_mixture_weights_are_not_renormalized():
    width = 4
    x = torch.tensor([[math.log(4.0), math.log(2.0), 0.0, 0.0]], dtype=DT)       # scores 4/8, 2/8, 1/8, 1/8
    w = {"router": torch.eye(4, dtype=DT)}
    for e in range(4):
        w[f"e{e}.up"] = torch.tensor([[1.0, 0, 0, 0], [-1.0, 0, 0, 0]], dtype=DT)       # (the second unit is cut off)
        w[f"e{e}.down"] = torch.zeros(width, 2, dtype=DT)
        w[f"e{e}.down"][e] = 1.0
    unit = math.log(4.0) ** 2
    assert torch.allclose(pl.mixture(x, w, "", moe(4, 2, 2)), torch.tensor([[0.5 * unit, 0.25 * unit, 0.0, 0.0]], dtype=DT))
    margins = []
    pl.mixture(x, w, "", moe(4, 2, 2), margins)
    assert abs(float(margins[0][0]) - (2 - 1) / (2 + 1)) < 1e-12
    pl.mixture(x, w, "", moe(4, 4, 2), margins)
    assert float(margins[1][0]) == math.inf


def test_whole_model_prefix_property_and_layers():
    """Logits at a position depend on the tokens up to it only, every tensor has an effect, and the stream after every
    layer is handed out."""
    cfg = copy.deepcopy(CONFIGS["A"])
    w = {k: v.float() for k, v in make_weights(cfg, 3).items()}
    ids = torch.randint(0, cfg["vocab"], (40,), generator=torch.Generator().manual_seed(1)).tolist()
    streams, margins = [], []
    full = pl.forward(cfg, w, ids, streams, margins)
    assert len(streams) == 4 and streams[0].shape == (40, 96) and len(margins) == 2 and margins[0].shape == (40,)
    assert torch.allclose(pl.forward(cfg, w, ids[:17]), full[:17], atol=1e-9)
    for name in w:
        if ".mlp.e" in name:
            continue
        changed = dict(w)
        changed[name] = w[name] + 0.25 * torch.linspace(-1.0, 1.0, w[name].numel()).reshape(w[name].shape)
        assert float((pl.forward(cfg, changed, ids) - full).abs().max()) > 1e-4, name
    for change in (lambda c: c.update(logit_scale=0.29), lambda c: c["layers"][0]["mixer"]["left"].update(softcap=5.0),
                   lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(keep_first=4),
                   lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(size=11),
                   lambda c: c["layers"][0]["mixer"]["left"]["rot"]["scaling"].update(factor=5.0),
                   lambda c: c["layers"][1]["mixer"]["decay"].__setitem__(2, 0.9)):
        other = copy.deepcopy(cfg)
        change(other)
        assert float((pl.forward(other, w, ids) - full).abs().max()) > 1e-4


def test_clear_routes_are_clear_and_varied():
    for name, cfg in CONFIGS.items():
        w = {k: v.float() for k, v in make_weights(cfg, 5, clear_routes=True).items()}
        margins = []
        pl.forward(cfg, w, torch.randint(0, cfg["vocab"], (60,), generator=torch.Generator().manual_seed(2)).tolist(), margins=margins)
        assert margins and float(torch.stack(margins).min()) > 1e-2, name


def test_random_model_from_the_command_line(tmp_path):
    """`--write-random-model` on a Lilatar config.json: every declared tensor is written and the folder loads back."""
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
    _, w = pl.read_folder(str(out))
    assert torch.isfinite(pl.forward(cfg.to_dict(), w, [3, 1, 4, 1, 5, 9, 2, 6])).all()


def test_helpers_name_every_key():
    """The small configurations' builders write what the configuration reads back."""
    cfg = {"architecture": "Lilatar", "vocab": 9, "width": 16, "norm": {"eps": 1e-5}, "layers": [pair(), lightning(), pair(window=0, keep=0)]}
    spec = config_from_dict(cfg).to_spec()
    assert [ls.mixer.params.get("left") is not None for ls in spec.layers] == [True, False, True]
    assert spec.layers[2].mixer.params["left"].params["keep_first"] == 0
