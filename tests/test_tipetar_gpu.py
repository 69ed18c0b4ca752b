"""Tipetar on the GPU against the plain implementation (plain_tipetar.py): each mechanism alone, keys just inside and
just outside windows and at pages' borders, prompts against token-by-token decoding, portions down to two tokens, unequal
batches, pages and slots used again, the first tokens, long decoding, generation through the engine and through
bin/trace_run, configurations drawn at random."""
import copy
import math
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import plain_tipetar as pt
import replay_helpers as rh
from test_parts_gpu import DEV, OneMixer, rel, runtime
from tipetar_helpers import CONFIGS, check_logits, layer, moe, write_model
from vt_transformer_amd.config.base import PartSpec, ScheduleEntry

pytestmark = pytest.mark.gpu
PART_TOL = {torch.float32: 1e-5, torch.bfloat16: 2.5e-2}
NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm"}
CUTS = [(0, 20), (20, 21), (21, 23), (23, 70), (70, 71), (71, 83)]


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    """Every configuration twice: as it is, and with fixed routes (what the 16-bit types compare)."""
    root = tmp_path_factory.mktemp("tipetar")
    out = {}
    for i, (k, cfg) in enumerate(CONFIGS.items()):
        out[k, "float32"] = write_model(copy.deepcopy(cfg), str(root / k), seed=41 + i, idle=k == "A")
        out[k, "bfloat16"] = out[k, "float16"] = write_model(copy.deepcopy(cfg), str(root / (k + "f")), seed=51 + i, fixed_routes=True)
    return out


def make_runner(folder, dtype, pool_tokens, max_requests=4, page_size=16, max_seq_len=None):
    from vt_transformer_amd.engine import load_model, make_runner as mk
    model = load_model(folder, dtype, page_size=page_size)
    return mk(model, pool_tokens=pool_tokens, page_size=page_size, max_requests=max_requests,
              max_seq_len=max_seq_len or pool_tokens)


def weights_for(part, seed, scale):
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, decl in part.tensors().items():
        if decl.role == "matrix32":
            t = torch.randn(decl.shape, generator=g) * 2.0 / decl.shape[-1] ** 0.5
        elif name.endswith("correction"):
            t = (torch.rand(decl.shape, generator=g) - 0.8) * 2.0 / decl.shape[0]
        else:
            t = torch.randn(decl.shape, generator=g) * (scale if decl.role == "matrix" else 0.4)
        if decl.role == "gain":
            t += 1.0
        out[name] = t.to(torch.bfloat16).float()
    return out


class MixerAndReader(OneMixer):
    """Two schedule entries: a mixer and one that reads its keys and values."""

    def __init__(self, mixer, reader):
        super().__init__(mixer)
        self.schedule = [ScheduleEntry(0), ScheduleEntry(1, cache_from=0)]
        self.layers = [SimpleNamespace(mixer=mixer), SimpleNamespace(mixer=reader)]


def step_mixers(runner, mixers, x, cuts, rid="r"):
    """Every mixer of the runner's model on x [T, width] of one request, in the portions `cuts`."""
    from vt_transformer_amd.engine.step import StepEntry
    runner.admit(rid)
    outs = [[] for _ in mixers]
    for a, b in cuts:
        assert runner.cache.reserve([(rid, b)])
        ctx = runner.build_context([StepEntry(rid, [0] * (b - a), [])])
        for mixer, cache, o in zip(mixers, runner.storage.layer_caches(ctx.block_tables), outs):
            o.append(mixer.forward(x[a:b].to(DEV).contiguous(), ctx, cache, None).float().cpu().clone())
        runner.cache.commit(rid, b)
    runner.release(rid)
    return [torch.cat(o) for o in outs]


def build_mixer(rt, width, prefix, nh, nkv, d, dv, window, scale, own=True, eps=1e-5):
    from vt_transformer_amd.parts import MIXERS
    return MIXERS.build(PartSpec("masked_attention", dict(
        num_heads=nh, num_kv_heads=nkv, key_dim=d, value_dim=dv, scale=scale, window=window, distance_slopes=8.0,
        whole_norm_eps=eps, own_keys=own, names=dict(NAMES))), rt=rt, width=width, prefix=prefix, shared={})


# ---------------------------------------------------------------------------
# the mechanisms alone
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nh,nkv,d,dv,window,readers", [
    (4, 2, 16, 32, 12, [(4, 12), (8, 30)]),     # a reader of the same form; one with more heads and a wider window
    (3, 1, 20, 10, 7, [(3, 0)]),                # sizes that are no multiples of 16; a reader that sees everything
    (16, 1, 32, 16, 17, [(16, 5)]),             # a full tile of heads; a narrower reader
    (5, 5, 16, 16, 0, [(5, 1)]),                # a reader that sees itself alone
    (6, 3, 64, 80, 40, [(12, 64)]),             # four heads to a key head: they share what they read
    (2, 1, 18, 6, 23, [(20, 23)]),              # rows that are no multiples of 4; more heads than a tile's 16 rows
])
def test_attention_with_a_norm_over_the_whole_projection(dtype, nh, nkv, d, dv, window, readers):
    from vt_transformer_amd.engine.step import ModelRunner
    width, t, eps = 72, 83, 1e-3
    x = (torch.randn(t, width, generator=torch.Generator().manual_seed(4)) * 0.2).to(dtype)
    for rh_, rw in readers:
        rt = runtime(dtype)
        mixer = build_mixer(rt, width, "a.", nh, nkv, d, dv, window, 0.3, eps=eps)
        reader = build_mixer(rt, width, "b.", rh_, nkv, d, dv, rw, 0.2, own=False, eps=eps)
        assert "b.k" not in reader.tensors() and "b.k.norm" not in reader.tensors()
        w = {**weights_for(mixer, 3, 0.3), **weights_for(reader, 5, 0.3)}
        mixer.load(w.__getitem__, rt)
        reader.load(w.__getitem__, rt)
        runner = ModelRunner(MixerAndReader(mixer, reader), rt, 16, 256, 4, 256)
        assert runner.storage.n_groups == 1
        got = step_mixers(runner, [mixer, reader], x, CUTS)
        wd, xd = {k: v.double() for k, v in w.items()}, x.double()
        m = {"heads": nh, "kv_heads": nkv, "dim": d, "vdim": dv}
        k, v = pt.keys_values(xd, wd, "a.", m, eps)
        refs = [pt.attend(pt.queries(xd, wd, "a.", m, eps), k, v, 0.3, window).reshape(t, -1) @ wd["a.o"].T,
                pt.attend(pt.queries(xd, wd, "b.", dict(m, heads=rh_), eps), k, v, 0.2, rw).reshape(t, -1) @ wd["b.o"].T]
        for g, r in zip(got, refs):
            assert rel(g, r) < PART_TOL[dtype]
        if dtype == torch.float32:      # the same operations whatever the cut
            for cuts in ([(0, t)], [(0, 50)] + [(i, i + 1) for i in range(50, t)]):
                for g, r in zip(got, step_mixers(runner, [mixer, reader], x, cuts)):
                    assert rel(g, r) < 1e-6


def test_a_reader_without_a_writer_is_refused():
    from vt_transformer_amd.engine.step import ModelRunner
    rt = runtime(torch.float32)
    reader = build_mixer(rt, 24, "b.", 2, 1, 8, 8, 4, 0.3, own=False)
    reader.load(weights_for(reader, 1, 0.3).__getitem__, rt)
    runner = ModelRunner(OneMixer(reader), rt, 16, 64, 1, 64)
    with pytest.raises(RuntimeError, match="cache of its own"):
        step_mixers(runner, [reader], torch.zeros(3, 24), [(0, 3)])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nh,window,reader_window", [(2, 37, 21), (4, 33, 50), (4, 16, 0), (8, 100, 101)])
def test_one_key_inside_and_outside_the_windows(dtype, nh, window, reader_window):
    """A mixer and a reader with weights that pass their input through: one token's key points along element 0, every
    query asks for element 0, and that token's value is the only one that is not zero.  Every position that the window
    reaches returns it (the score stands far above what the slope takes off), the first one behind it nothing; the token
    sits in the last slot of a page; in one portion, in portions that end around the window's edge, and decoded one by
    one across it."""
    from vt_transformer_amd.engine.step import ModelRunner
    rt = runtime(dtype)
    d, t, star = 16, 190, 31
    width = nh * d + 2 * d
    mixer = build_mixer(rt, width, "a.", nh, 1, d, d, window, 4.0, eps=1e-6)
    reader = build_mixer(rt, width, "b.", nh, 1, d, d, reader_window, 4.0, own=False, eps=1e-6)
    eye = torch.eye(width)
    o = torch.cat([torch.eye(nh * d), torch.zeros(2 * d, nh * d)])
    w = {"a.q": eye[:nh * d], "a.k": eye[nh * d:nh * d + d], "a.v": eye[nh * d + d:], "a.o": o, "b.q": eye[:nh * d], "b.o": o,
         "a.q.norm": torch.ones(nh * d), "b.q.norm": torch.ones(nh * d), "a.k.norm": torch.ones(d)}
    mixer.load(w.__getitem__, rt)
    reader.load(w.__getitem__, rt)
    runner = ModelRunner(MixerAndReader(mixer, reader), rt, 16, 256, 2, 256)
    x = torch.zeros(t, width)
    for h in range(nh):
        x[:, h * d] = 6.0
    x[:, nh * d + 1:nh * d + d] = torch.randn(t, d - 1, generator=torch.Generator().manual_seed(6))
    x[star, nh * d:nh * d + d] = 0.0
    x[star, nh * d] = 1.0
    x[star, nh * d + d:] = torch.linspace(1.0, 2.0, d)
    x = x.to(dtype)
    value = x[star, nh * d + d:].float()
    edges = sorted({min(t, star + w_) for w_ in (window, reader_window or t)})
    steps = [(0, t)], [(0, star), (star, star + 1), (star + 1, edges[0] - 1), (edges[0] - 1, edges[0] + 1), (edges[0] + 1, t)], \
        [(0, edges[0] - 3)] + [(i, i + 1) for i in range(edges[0] - 3, min(t, edges[-1] + 3))]
    for cuts in steps:
        end = cuts[-1][1]
        for got, w_ in zip(step_mixers(runner, [mixer, reader], x, cuts), (window, reader_window or t)):
            got = got[:, :nh * d].reshape(end, nh, d)
            assert float(got[:star].abs().max()) < 1e-6
            inside = got[star:min(end, star + w_)]
            assert float((inside - value).abs().max()) < (1e-3 if dtype == torch.float32 else 2e-2), "a position lost the key"
            if end > star + w_:
                assert float(got[star + w_:].abs().max()) < 1e-6, "a position sees beyond its window"


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_slope_is_taken_off_the_distance(dtype):
    """Queries and keys are the same everywhere, so a weight is e^(-slope * distance) alone and the output a known mean
    of the values, which grow with the position; 3 heads (slopes that are no powers of two) and 12."""
    from vt_transformer_amd.engine.step import ModelRunner
    for nh, window in ((3, 0), (12, 50)):
        rt = runtime(dtype)
        d, t = 16, 150
        width = nh * d + 2 * d
        mixer = build_mixer(rt, width, "a.", nh, 1, d, d, window, 1.0)
        eye = torch.eye(width)
        w = {"a.q": eye[:nh * d], "a.k": eye[nh * d:nh * d + d], "a.v": eye[nh * d + d:], "a.q.norm": torch.ones(nh * d),
             "a.k.norm": torch.ones(d), "a.o": torch.cat([torch.eye(nh * d), torch.zeros(2 * d, nh * d)])}
        mixer.load(w.__getitem__, rt)
        runner = ModelRunner(OneMixer(mixer), rt, 16, 256, 1, 256)
        x = torch.ones(t, width)
        x[:, nh * d + d:] = (torch.arange(t) / 64.0)[:, None]
        x = x.to(dtype)
        values = x[:, nh * d + d].double()
        dist = (torch.arange(t)[:, None] - torch.arange(t)[None, :]).double()
        seen = (dist >= 0) & (dist < (window or t))
        for cuts in ([(0, t)], [(0, 100)] + [(i, i + 1) for i in range(100, t)]):
            got = step_mixers(runner, [mixer], x, cuts)[0][:, :nh * d].reshape(t, nh, d)
            for h in range(nh):
                p = torch.exp(-(2.0 ** (-8.0 * (h + 1) / nh)) * dist) * seen
                want = (p @ values) / p.sum(dim=1)
                assert rel(got[:, h, 0], want) < (2e-6 if dtype == torch.float32 else 1e-2), h


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("experts,identity,top,groups,width,with_bias", [
    (6, 2, 2, (4, 2), 96, True), (5, 1, 3, (1, 1), 72, True), (12, 4, 4, (4, 1), 100, True), (7, 0, 7, (1, 1), 80, False),
    (60, 4, 8, (8, 3), 128, True), (250, 6, 6, (32, 4), 64, True), (3, 3, 2, (2, 1), 52, True), (1, 0, 1, (1, 1), 40, False),
])
def test_router_forms(dtype, experts, identity, top, groups, width, with_bias):
    """Chosen outputs and weights of the router alone: correction, groups, choices without an expert, the factor; choice
    scores below zero, where leaving a group out must mean minus infinity."""
    from vt_transformer_amd.kernels import ops
    n, n_out = 90, experts + identity
    g = torch.Generator().manual_seed(experts)
    x = (torch.randn(n, width, generator=g)).to(dtype)
    wr = torch.randn(n_out, width, generator=g) * 2.0 / width ** 0.5
    bias = (torch.rand(n_out, generator=g) - 0.9) * 2.0 / n_out if with_bias else None
    ids = torch.full((n, top), -7, dtype=torch.int32, device=DEV)
    wts, idw = torch.full((n, top), -1.0, device=DEV), torch.full((n,), -1.0, device=DEV)
    ops.moe_route(x.to(DEV), wr.to(DEV), ids, wts, "softmax", True, 1e-20, 1.7, bias.to(DEV) if with_bias else None, groups[0],
                  groups[1], identity, idw)
    # many tokens go four to a block, a few hundred one to a block of fewer waves: the same bits for a token
    for rows in (300, 1030):
        place = torch.arange(rows) % n
        more = [torch.full((rows, top), -7, dtype=torch.int32, device=DEV), torch.full((rows, top), -1.0, device=DEV),
                torch.full((rows,), -1.0, device=DEV)]
        ops.moe_route(x[place].to(DEV), wr.to(DEV), more[0], more[1], "softmax", True, 1e-20, 1.7,
                      bias.to(DEV) if with_bias else None, groups[0], groups[1], identity, more[2])
        assert all(torch.equal(a, b[place.to(DEV)]) for a, b in zip(more, (ids, wts, idw)))
    ids, wts, idw = ids.cpu(), wts.cpu().double(), idw.cpu().double()
    scores = torch.softmax(x.double() @ wr.double().T, dim=-1)
    compared = handed = 0
    for t in range(n):
        chosen, margin = pt.choose(scores[t], (bias if with_bias else torch.zeros(n_out)).double(), top, *groups)
        if margin < 2e-5:
            continue
        compared += 1
        total = sum(float(scores[t, e]) for e in chosen)
        assert ids[t].tolist() == [e if e < experts else -1 for e in chosen], t
        want = torch.tensor([float(scores[t, e]) / total * 1.7 for e in chosen], dtype=torch.float64)
        assert torch.allclose(wts[t], want, rtol=2e-5), t
        lent = sum(float(v) for v, e in zip(want, chosen) if e >= experts)
        assert abs(float(idw[t]) - lent) < 4e-5, t
        handed += lent > 0
    assert compared > 0.9 * n and (handed > 0) == (identity > 0)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("experts,identity,top,groups,inter,shared,width", [
    (6, 2, 2, (4, 2), 40, 56, 96),          # every form
    (5, 1, 3, None, 24, None, 72),          # no shared expert, no groups
    (4, 0, 1, None, 32, 20, 64),            # one choice a token and no choice without an expert
    (3, 3, 2, (2, 1), 16, 16, 128),         # tokens all of whose choices hand the input through
    (2, 4, 1, (3, 1), 16, None, 64),        # ... one choice a token
    (8, 4, 4, (3, 2), 20, 36, 100),         # sizes that are no multiples of 8: the any-shape kernels
    (16, 0, 4, (4, 2), 48, 96, 256),
])
def test_mixture_forms(dtype, experts, identity, top, groups, inter, shared, width):
    """The whole feed-forward, few rows and many, added up by itself and handed on in pieces."""
    from vt_transformer_amd.parts import FEED_FORWARDS
    from vt_transformer_amd.parts.base import SublayerPieces
    rt = runtime(dtype)
    sh = PartSpec("gated_mlp", dict(intermediate_size=shared, weight_suffix="", prefix="shared.",
                                    names={"gate": "gate", "up": "up", "down": "down"})) if shared else None
    ff = FEED_FORWARDS.build(PartSpec("expert_mixture", dict(
        num_experts=experts, top=top, intermediate_size=inter, score="softmax", renormalize=True, renorm_eps=1e-20,
        weight_on="output", correction=True, groups={"count": groups[0], "keep": groups[1]} if groups else None,
        router_scale=1.6, identity=identity, shared_expert=sh)), rt=rt, width=width, prefix="f.")
    assert ff.replayable and f"f.e{experts}.gate" not in ff.tensors() and ("f.shared.up" in ff.tensors()) == bool(shared)
    w = weights_for(ff, 12, 0.2)
    ff.load(w.__getitem__, rt)
    wd = {k: v.double() for k, v in w.items()}
    mlp = moe(experts, top, inter, identity, groups, 1.6, shared)
    for rows in (1, 3, 7, 30, 150, 700):
        x = torch.randn(rows, width, generator=torch.Generator().manual_seed(rows)).to(dtype)
        margins = []
        ref = pt.mixture(x.double(), wd, "f.", mlp, margins)
        sure = margins[0] > 2e-5
        got = ff.forward(x.to(DEV)).float().cpu().clone()
        assert rel(got[sure], ref[sure]) < PART_TOL[dtype], rows
        pieces = ff.forward(x.to(DEV), None, pieces=True)
        assert isinstance(pieces, SublayerPieces)
        assert torch.equal(pieces.materialize().float().cpu(), got) or rel(pieces.materialize(), got) < 1e-6


def test_a_plain_mixture_keeps_its_own_sum():
    from vt_transformer_amd.parts import FEED_FORWARDS
    rt = runtime(torch.bfloat16)
    ff = FEED_FORWARDS.build(PartSpec("expert_mixture", dict(num_experts=4, top=2, intermediate_size=16)), rt=rt, width=64, prefix="f.")
    ff.load(weights_for(ff, 2, 0.3).__getitem__, rt)
    x = torch.randn(9, 64, generator=torch.Generator().manual_seed(1)).to(torch.bfloat16).to(DEV)
    whole = ff.forward(x)
    assert isinstance(whole, torch.Tensor) and rel(ff.forward(x, None, pieces=True).materialize(), whole.clone()) < 1e-6


@pytest.mark.parametrize("width", [40, 96, 100, 1024, 2048, 2052, 4096, 8192, 8196, 51])
def test_norm_on_the_output(width):
    """u added up from its pieces, normed, times the factor, added to the stream, and the stream's copy; the pieces'
    sum alone; widths for every number of registers and none."""
    from vt_transformer_amd.kernels import ops
    g = torch.Generator().manual_seed(width)
    n, top, eps, mult = 5, 3, 1e-2, 0.7
    gain = 1.0 + torch.randn(width, generator=g) * 0.3
    h = torch.randn(n, width, generator=g)
    choices = torch.randn(n * top, width, generator=g)
    ids = torch.tensor([[0, -1, 2], [1, 1, 0], [-1, -1, -1], [3, 0, -1], [-1, 2, 2]], dtype=torch.int32)
    idw = torch.tensor([0.5, 0.0, 2.0, 0.25, 1.0])
    dead = choices.clone()
    dead[ids.flatten() < 0] = float("nan")          # (rows that nobody has written must not be read)
    for y_dtype in (torch.float32, torch.bfloat16):
        y, x = torch.randn(n, width, generator=g).to(y_dtype), torch.randn(n, width, generator=g).to(y_dtype)
        forms = [dict(y=y), dict(choices=choices), dict(choices=dead, ids=ids, id_weights=idw, x=x, y=y),
                 dict(choices=dead, ids=ids, id_weights=idw, x=x), dict(id_weights=idw, x=x, y=y), dict(choices=choices, y=y)]
        for form in forms:
            u = torch.zeros(n, width, dtype=torch.float64)
            if "choices" in form:
                rows = choices.double().reshape(n, top, width)
                u = u + (rows * (ids >= 0)[:, :, None] if "ids" in form else rows).sum(dim=1)
            if "id_weights" in form:
                u = u + idw.double()[:, None] * x.double()
            if "y" in form:
                u = u + y.double()
            dev = {k: v.to(DEV) for k, v in form.items()}
            out = ops.sublayer_sum(torch.full((n, width), 9.0, device=DEV), **dev)
            assert rel(out, u) < 1e-6
            ref = h.double() + mult * pt.plain_rmsnorm(u, gain.double(), eps)
            for copy_dtype in (None, torch.float32, torch.bfloat16):
                hd = h.to(DEV).clone()
                copy_ = torch.empty(n, width, dtype=copy_dtype, device=DEV) if copy_dtype else None
                ops.output_norm_add(hd, gain.to(DEV), eps, mult, copy=copy_, **dev)
                assert rel(hd, ref) < 2e-6
                if copy_ is not None:
                    assert torch.equal(copy_, hd.to(copy_dtype))
    # the sublayer's input is the stream itself: read before it is changed
    hd = h.to(DEV).clone()
    ops.output_norm_add(hd, gain.to(DEV), eps, mult, y=y.to(DEV), id_weights=idw.to(DEV), x=hd)
    u = idw.double()[:, None] * h.double() + y.double()
    assert rel(hd, h.double() + mult * pt.plain_rmsnorm(u, gain.double(), eps)) < 2e-6


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_stream_after_every_layer(folders, dtype):
    from vt_transformer_amd.engine.step import StepEntry
    folder = folders["A", dtype]
    cfg, w = pt.read_folder(folder)
    toks = rh.random_requests(cfg["vocab"], [29], seed=1)["r0"]
    streams = []
    pt.forward(cfg, w, toks, streams)
    runner = make_runner(folder, dtype, pool_tokens=64, max_requests=1)
    seen = []
    for block in runner.model.layers:
        def wrapped(h, delta, ctx, cache, state, inner=block.forward):
            h, d = inner(h, delta, ctx, cache, state)
            assert torch.equal(d.x, h.to(d.x.dtype))
            seen.append(h.cpu().double())
            return h, d
        block.forward = wrapped
    runner.admit("r")
    runner.step([StepEntry("r", toks, [len(toks) - 1])])
    assert len(seen) == len(streams) == 5
    for i, (a, b) in enumerate(zip(seen, streams)):
        assert rel(a, b) < (2e-5 if dtype == "float32" else 3e-2), f"layer {i}"


def test_blocks_of_other_kinds_around_this_one(tmp_path):
    """A model whose layers are of two kinds, a norm in front of the sublayers and a norm behind them in turn: what one
    kind hands on, the other goes on from (float32 and bfloat16 agree with the arrangement written out)."""
    from vt_transformer_amd.config.base import LayerSpec, ModelSpec
    from vt_transformer_amd.engine.step import StepEntry, ModelRunner
    from vt_transformer_amd.models.model import DecoderModel
    width, vocab = 64, 50

    def mlp_spec():
        return PartSpec("gated_mlp", dict(intermediate_size=40, weight_suffix="", prefix="mlp.", names={"gate": "gate", "up": "up", "down": "down"}))

    def mixer_spec():
        return PartSpec("masked_attention", dict(num_heads=2, num_kv_heads=1, key_dim=16, value_dim=16, scale=0.3,
                                                 distance_slopes=8.0, whole_norm_eps=1e-5, names=dict(NAMES), prefix="mix."))
    norm = lambda name: PartSpec("rmsnorm", {"eps": 1e-5, "name": name, "unit_offset": True})      # noqa: E731
    pre = {"input": norm("norm1"), "post_mixer": norm("norm2")}
    post = {"mixer_output": norm("norm1"), "feed_forward_output": norm("norm2")}
    kinds = ["prenorm", "output_norm", "output_norm", "prenorm", "output_norm"]
    spec = ModelSpec("mixed", vocab, width, PartSpec("embedding", {"name": "embed"}),
                     [LayerSpec(PartSpec(k, {"residual_mult": 0.6} if k == "output_norm" else {}), mixer_spec(), mlp_spec(),
                                post if k == "output_norm" else pre, f"l{i}.") for i, k in enumerate(kinds)],
                     [ScheduleEntry(i) for i in range(len(kinds))], norm("final.norm"),
                     PartSpec("linear_head", {"name": "head", "tied_to": None}), 256)
    ids = rh.random_requests(vocab, [21], seed=3)["r0"]
    for dtype in (torch.float32, torch.bfloat16):
        rt = runtime(dtype)
        model = DecoderModel(spec, rt)
        g = torch.Generator().manual_seed(1)
        w = {}
        for name, decl in model.tensors().items():
            t = torch.randn(decl.shape, generator=g) * (0.3 if decl.role != "matrix" else 1.0 if name == "embed" else decl.shape[-1] ** -0.5)
            w[name] = (t + 1.0 if decl.role == "gain" else t).to(torch.bfloat16).float()
        model.load(w.__getitem__)
        wd = {k: v.double() for k, v in w.items()}
        x = wd["embed"][torch.tensor(ids)]
        m = {"heads": 2, "kv_heads": 1, "dim": 16, "vdim": 16}

        def mix(h, p):
            k, v = pt.keys_values(h, wd, p + "mix.", m, 1e-5)
            return pt.attend(pt.queries(h, wd, p + "mix.", m, 1e-5), k, v, 0.3, 0).reshape(len(ids), -1) @ wd[p + "mix.o"].T
        for i, k in enumerate(kinds):
            p = f"l{i}."
            if k == "prenorm":
                x = x + mix(pt.offset_rmsnorm(x, wd[p + "norm1"], 1e-5), p)
                x = x + pt.gated_unit(pt.offset_rmsnorm(x, wd[p + "norm2"], 1e-5), wd, p + "mlp.")
            else:
                x = x + 0.6 * pt.offset_rmsnorm(mix(x, p), wd[p + "norm1"], 1e-5)
                x = x + 0.6 * pt.offset_rmsnorm(pt.gated_unit(x, wd, p + "mlp."), wd[p + "norm2"], 1e-5)
        ref = pt.offset_rmsnorm(x, wd["final.norm"], 1e-5) @ wd["head"].T
        runner = ModelRunner(model, rt, 16, 64, 1, 64)
        runner.admit("r")
        got = [runner.step([StepEntry("r", ids[a:b], list(range(b - a)))]).float().cpu() for a, b in ((0, 17), (17, 18), (18, 21))]
        assert rel(torch.cat(got), ref) < (2e-5 if dtype == torch.float32 else 3e-2)


# ---------------------------------------------------------------------------
# whole models: schedules against the plain implementation
# ---------------------------------------------------------------------------
LENGTHS = [61, 1, 23, 90, 2, 47]


@pytest.mark.parametrize("name,dtype", [(n, d) for n in "ABCD" for d in ("float32", "bfloat16")] + [("A", "float16"), ("D", "float16")])
def test_schedules(folders, name, dtype):
    """Whole prompts; most of a prompt and then its last tokens one by one; portions of changing sizes down to two
    tokens; unequal requests side by side with three slots and few pages, so that both are used again."""
    folder, vocab = folders[name, dtype], CONFIGS[name]["vocab"]
    reqs = rh.random_requests(vocab, LENGTHS, seed=3)
    cache = {}
    runner = make_runner(folder, dtype, pool_tokens=256, max_requests=3)
    runner.decode_graphs = True
    whole = rh.trace_alone(reqs, {r: [(0, len(t))] for r, t in reqs.items()})
    got_whole = rh.run_in_process(runner, whole)
    check_logits(folder, reqs, whole, got_whole, dtype, cache)
    decode = rh.trace_alone(reqs, {r: ([(0, max(1, len(t) - 30))] + [(i, i + 1) for i in range(max(1, len(t) - 30), len(t))])
                                   for r, t in reqs.items()})
    got_decode = rh.run_in_process(runner, decode)
    check_logits(folder, reqs, decode, got_decode, dtype, cache)
    chunked = rh.trace_alone(reqs, {r: rh.cut(t, [7, 2, 16, 3, 2, 33, 1, 5]) for r, t in reqs.items()})
    got_chunked = rh.run_in_process(runner, chunked)
    check_logits(folder, reqs, chunked, got_chunked, dtype, cache)
    mixed = rh.trace_mixed(reqs, {r: rh.cut(t, [9, 2, 1, 1, 20, 1, 1, 1, 4]) for r, t in reqs.items()}, max_live=3, seed=5)
    assert rh.max_live_tokens(mixed) <= 256
    got_mixed = rh.run_in_process(runner, mixed)
    check_logits(folder, reqs, mixed, got_mixed, dtype, cache)
    if dtype == "float32":
        # a position's logits do not depend on the cut, the batch, the pages or the slots
        flat = {}
        for steps, got in ((whole, got_whole), (decode, got_decode), (chunked, got_chunked), (mixed, got_mixed)):
            pos = {r: 0 for r in reqs}
            for s in steps:
                row = 0
                for e in s["entries"]:
                    for wi in e["want"]:
                        flat.setdefault((e["id"], pos[e["id"]] + wi), []).append(got[s["step"]][row])
                        row += 1
                    pos[e["id"]] += len(e["tokens"])
        for key, rows in flat.items():
            assert len(rows) == 4
            for r in rows[1:]:
                assert float(np.abs(rows[0] - r).max()) <= 1e-5 * float(np.abs(rows[0]).max()), f"{key} depends on the schedule"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_across_windows_and_pages(folders, dtype):
    folder, vocab = folders["A", dtype], CONFIGS["A"]["vocab"]
    reqs = rh.random_requests(vocab, [150], seed=9)
    steps = rh.trace_alone(reqs, {"r0": [(0, 5)] + [(i, i + 1) for i in range(5, 150)]})
    runner = make_runner(folder, dtype, pool_tokens=192, max_requests=1)
    runner.decode_graphs = True
    check_logits(folder, reqs, steps, rh.run_in_process(runner, steps), dtype)
    assert sum(runner.cache.available_pages()) == sum(p.num_pages for p in runner.cache.pools)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_pages_stay_as_long_as_their_widest_reader_needs_them(tmp_path, dtype):
    """A pool that holds less than a request, since every key dies in the end; keys of the first layer are read through
    a window of three pages by a later one, long after the layer that made them has passed them."""
    cfg = {"architecture": "Tipetar", "vocab": 61, "width": 64, "norm": {"eps": 1e-5}, "residual_mult": 0.9,
           "layers": [layer(window=4, mlp=moe(4, 2, 16)), layer(window=45, scale=0.05, kv_from=0, mlp=moe(3, 1, 16, identity=1)),
                      layer(window=9, kv_from=0)]}
    folder = write_model(cfg, str(tmp_path / "m"), seed=77, fixed_routes=True)
    reqs = rh.random_requests(61, [180], seed=13)
    for cuts in ([10], [50, 1, 1, 2, 1, 1, 1, 1, 3, 16]):
        steps = rh.trace_alone(reqs, {"r0": rh.cut(reqs["r0"], cuts)})
        runner = make_runner(folder, dtype, pool_tokens=112, max_requests=1, max_seq_len=192)
        check_logits(folder, reqs, steps, rh.run_in_process(runner, steps), dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_many_tokens_at_once(tmp_path, dtype):
    """Prompts of some hundred tokens (tiles of many pairs of an expert, key ranges of many pages) against the same
    prompts in portions."""
    cfg = {"architecture": "Tipetar", "vocab": 90, "width": 64, "norm": {"eps": 1e-6}, "residual_mult": 0.5,
           "layers": [layer(heads=4, kv_heads=1, dim=64, vdim=32, window=130, scale=0.1,
                            mlp=moe(4, 2, 24, identity=2, groups=(2, 1), scale=2.0, shared=48)),
                      layer(heads=4, kv_heads=1, dim=64, vdim=32, window=0, scale=0.1, kv_from=0, mlp=moe(2, 1, 48, shared=8))]}
    folder = write_model(cfg, str(tmp_path / "m"), seed=77, fixed_routes=True)
    reqs = rh.random_requests(90, [300, 170], seed=2)
    runner = make_runner(folder, dtype, pool_tokens=512, max_requests=2)
    cache = {}
    whole = rh.trace_alone(reqs, {r: [(0, len(t))] for r, t in reqs.items()})
    check_logits(folder, reqs, whole, rh.run_in_process(runner, whole), dtype, cache)
    mixed = rh.trace_mixed(reqs, {r: rh.cut(t, [130, 2, 1, 64, 1, 1, 50]) for r, t in reqs.items()}, max_live=2, seed=4)
    check_logits(folder, reqs, mixed, rh.run_in_process(runner, mixed), dtype, cache)


def test_captured_decoding_steps_equal_launched_ones(folders):
    """bfloat16: the same decoding steps through captured graphs and launch by launch, bit for bit, with three requests
    (a captured step of four entries, one of them padding)."""
    folder, vocab = folders["A", "bfloat16"], CONFIGS["A"]["vocab"]
    reqs = rh.random_requests(vocab, [40, 25, 31], seed=19)
    portions = {r: [(0, len(t) - 16)] + [(i, i + 1) for i in range(len(t) - 16, len(t))] for r, t in reqs.items()}
    steps = rh.trace_mixed(reqs, portions, max_live=3, seed=1, skip_prob=0.0)
    got = []
    for graphs in (False, True):
        runner = make_runner(folder, "bfloat16", pool_tokens=192, max_requests=3)
        runner.decode_graphs = graphs
        assert runner.replays(3) == graphs
        got.append(rh.run_in_process(runner, steps))
        assert bool(runner._graphs) == graphs
    assert all(np.array_equal(got[0][k], got[1][k]) for k in got[0])
    check_logits(folder, reqs, steps, got[1], "bfloat16")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_generation_through_the_engine(folders, dtype):
    """Greedy tokens through Engine.generate (scheduler with short portions, two slots for three requests)."""
    from vt_transformer_amd.engine import Engine
    from vt_transformer_amd.sampling import SamplingParams
    folder = folders["C", dtype]
    cfg, w = pt.read_folder(folder)
    prompts = [r for r in rh.random_requests(cfg["vocab"], [19, 3, 41], seed=21).values()]
    eng = Engine(folder, dtype=dtype, num_pages=16, max_running_reqs=2, max_seq_len=128, chunk_size=16, max_extend_tokens=24)
    got = eng.generate(prompts, SamplingParams(max_tokens=8, ignore_eos=True))
    for p, g in zip(prompts, got):
        assert len(g) == 8
        if dtype == "float32":
            assert g == pt.greedy(cfg, w, p, 8)
        else:
            logits = pt.forward(cfg, w, p + g)
            for i, tok in enumerate(g):
                row = logits[len(p) - 1 + i]
                assert float(row.max() - row[tok]) <= 3e-2 * float(row.abs().max())


def test_trace_run_with_a_tipetar_folder(folders, tmp_path):
    folder, vocab = folders["D", "float32"], CONFIGS["D"]["vocab"]
    reqs = rh.random_requests(vocab, [40, 9, 27], seed=17)
    steps = rh.trace_mixed(reqs, {r: rh.cut(t, [6, 2, 11, 1]) for r, t in reqs.items()}, max_live=2, seed=2)
    got = rh.run_trace_run(folder, "float32", steps, str(tmp_path / "out"), rh.max_live_tokens(steps), vocab,
                           extra_args=("--max-requests", "2"))
    check_logits(folder, reqs, steps, got, "float32")


# ---------------------------------------------------------------------------
# configurations drawn at random
# ---------------------------------------------------------------------------
def random_tipetar_config(seed: int) -> dict:
    rs = np.random.RandomState(seed)
    pick = lambda xs: xs[rs.randint(len(xs))]      # noqa: E731
    layers = []
    for i in range(rs.randint(2, 7)):
        if rs.rand() < 0.8:
            count, size = int(pick([1, 1, 2, 3, 4])), int(pick([1, 2, 3, 5]))
            keep = int(rs.randint(1, count + 1))
            n_out = count * size
            identity = int(rs.randint(0, n_out)) if rs.rand() < 0.6 else 0
            mlp = moe(n_out - identity, int(rs.randint(1, keep * size + 1)), int(pick([8, 24, 40, 52])), identity,
                      (count, keep) if count > 1 or rs.rand() < 0.5 else None, float(pick([1.0, 0.5, 2.3])),
                      int(pick([8, 16, 60])) if rs.rand() < 0.6 else None)
        else:
            mlp = None
        window = int(pick([0, 1, 3, 16, 17, 50, 1000]))
        own = [j for j, x in enumerate(layers) if "kv_from" not in x["mixer"]]
        if own and rs.rand() < 0.5:
            src = int(pick(own))
            m = layers[src]["mixer"]
            layers.append(layer(heads=m["kv_heads"] * int(pick([1, 2, 3, 4])), kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"],
                                window=window, scale=float(pick([0.1, 0.3])), kv_from=src, mlp=mlp))
        else:
            kv = int(pick([1, 2, 3]))
            dim, vdim = pick([(16, 16), (16, 32), (64, 32), (20, 24), (48, 80), (8, 40), (13, 7), (64, 80)])
            layers.append(layer(heads=kv * int(pick([1, 2, 4, 5])), kv_heads=kv, dim=dim, vdim=vdim, window=window,
                                scale=float(pick([0.1, 0.3, 0.6])), mlp=mlp))
    cfg = {"architecture": "Tipetar", "vocab": int(pick([29, 100, 257])), "width": int(pick([40, 52, 64, 96, 100, 136])),
           "norm": {"eps": float(pick([1e-6, 1e-5, 1e-2]))}, "layers": layers}
    if rs.rand() < 0.8:
        cfg["residual_mult"] = float(pick([0.3, 0.8, 1.0, 1.5]))
    return cfg


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(tmp_path, seed):
    cfg = random_tipetar_config(seed)
    free = write_model(cfg, str(tmp_path / "m"), seed=100 + seed, idle=bool(seed % 2))
    fixed = write_model(cfg, str(tmp_path / "f"), seed=200 + seed, fixed_routes=True)
    reqs = rh.random_requests(cfg["vocab"], [70, 33, 5], seed=seed)
    for folder, dtype in ((free, "float32"), (fixed, "bfloat16")):
        runner = make_runner(folder, dtype, pool_tokens=192, max_requests=2)
        runner.decode_graphs = True
        cache = {}
        whole = rh.trace_alone(reqs, {r: [(0, len(t))] for r, t in reqs.items()})
        check_logits(folder, reqs, whole, rh.run_in_process(runner, whole), dtype, cache)
        mixed = rh.trace_mixed(reqs, {r: rh.cut(t, [11, 2, 1, 1, 17, 1, 1, 3]) for r, t in reqs.items()}, max_live=2, seed=seed)
        check_logits(folder, reqs, mixed, rh.run_in_process(runner, mixed), dtype, cache)
