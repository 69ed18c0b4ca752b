"""Lilatar on the GPU against the plain implementation (plain_lilatar.py): each mechanism alone, keys just inside and just
outside a window and its kept tokens, prompts against token-by-token decoding, portions down to two tokens, unequal batches,
pages and slots used again, the first tokens, long decoding, generation through the engine and through bin/trace_run,
configurations drawn at random."""
import copy
import math

import numpy as np
import pytest
import torch

import plain_lilatar as pl
import replay_helpers as rh
from lilatar_helpers import CONFIGS, check_logits, dense, lightning, moe, pair, write_model
from test_parts_gpu import DEV, OneMixer, rel, runtime
from vt_transformer_amd.config.base import PartSpec, ScheduleEntry

pytestmark = pytest.mark.gpu
DT = torch.float64
PART_TOL = {torch.float32: 2e-5, torch.bfloat16: 2.5e-2, torch.float16: 4e-3}
CUTS = [(0, 20), (20, 21), (21, 23), (23, 70), (70, 71), (71, 83)]


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    """Every configuration twice: as it is, and with clear routes (what the 16-bit types compare)."""
    root = tmp_path_factory.mktemp("lilatar")
    out = {}
    for i, (k, cfg) in enumerate(CONFIGS.items()):
        out[k, "float32"] = write_model(copy.deepcopy(cfg), str(root / k), seed=41 + i, idle=k == "A")
        out[k, "bfloat16"] = out[k, "float16"] = write_model(copy.deepcopy(cfg), str(root / (k + "c")), seed=51 + i, clear_routes=True,
                                                             keep_ranks=k == "B")
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
        else:
            t = torch.randn(decl.shape, generator=g) * (scale if decl.role == "matrix" else 0.4)
        if decl.role == "gain":
            t += 1.0
        out[name] = t.to(torch.bfloat16).float()
    return out


def strip(w, prefix):
    return {k[len(prefix):]: v.double() for k, v in w.items() if k.startswith(prefix)}


def step_part(runner, mixer, x, cuts, rid="r", **kw):
    """The runner's one mixer on x [T, width] of one request, in the portions `cuts`."""
    from vt_transformer_amd.engine.step import StepEntry
    runner.admit(rid)
    runner.storage.clear_state([runner.cache.get(rid).slot])
    out = []
    for a, b in cuts:
        assert runner.cache.reserve([(rid, b)])
        ctx = runner.build_context([StepEntry(rid, [0] * (b - a), [])])
        y = mixer.forward(x[a:b].to(DEV).contiguous(), ctx, runner.storage.layer_caches(ctx.block_tables)[0], runner.storage.state[0], **kw)
        out.append((y if isinstance(y, torch.Tensor) else y.materialize()).float().cpu().clone())
        runner.cache.commit(rid, b)
    runner.release(rid)
    return torch.cat(out)


def one_by_one(a, b):
    return [(i, i + 1) for i in range(a, b)]


# ---------------------------------------------------------------------------
# the mechanisms alone
# ---------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nh,d,dv,decay", [
    (3, 16, 24, [0.5, 0.93, 0.999]), (2, 64, 128, [0.8, 1.0]), (1, 128, 144, [0.99]), (4, 20, 12, [0.0, 0.3, 0.97, 1.0]),
    (2, 10, 7, [0.6, 0.95]),            # sizes that the chunks do not take: token by token
    (2, 256, 20, [0.7, 0.998]), (1, 8, 4, [0.9]), (5, 32, 32, [0.1, 0.6, 0.9, 0.99, 0.9999]),
])
def test_decayed_attention_part(dtype, nh, d, dv, decay):
    """A prompt in one step (chunks of 64, the last of them short), in portions around the chunks' edges and down to one and
    two tokens, and token by token, all against the sums written out."""
    from vt_transformer_amd.engine.step import ModelRunner
    from vt_transformer_amd.parts import MIXERS
    rt = runtime(dtype)
    width, t = 56, 210
    mixer = MIXERS.build(PartSpec("decayed_attention", dict(num_heads=nh, key_dim=d, value_dim=dv, decay=decay, norm_eps=1e-5)), rt=rt,
                         width=width, prefix="m.", shared={})
    w = weights_for(mixer, 7, 0.25)
    mixer.load(w.__getitem__, rt)
    runner = ModelRunner(OneMixer(mixer), rt, 16, 256, 3, 256)
    assert runner.storage.state[0].shape == (3 + 1, nh * d * dv) and runner.storage.n_groups == 0
    x = (torch.randn(t, width, generator=torch.Generator().manual_seed(8)) * 0.8).to(dtype)
    ref = pl.lightning_mixer(x.double(), strip(w, "m."), "", dict(heads=nh, decay=decay), 1e-5)
    whole = step_part(runner, mixer, x, [(0, t)])
    assert rel(whole, ref) < PART_TOL[dtype]
    for cuts in ([(0, 64), (64, 128), (128, t)], [(0, 63), (63, 65), (65, 130), (130, 131), (131, t)],
                 [(0, 1), (1, 3), (3, 4), (4, 6), (6, 80), (80, 81), (81, 83), (83, 100), (100, t)], [(0, 150)] + one_by_one(150, t),
                 one_by_one(0, t)):
        assert rel(step_part(runner, mixer, x, cuts), ref) < PART_TOL[dtype], cuts[:6]
    if d % 4 or dv % 4:
        assert dtype != torch.float32 or torch.equal(whole, step_part(runner, mixer, x, one_by_one(0, t)))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_decayed_attention_unequal_requests_in_a_step(dtype):
    """Portions of several lengths beside single tokens in one step, some of which go through chunks with them, against each
    request alone; a slot that another request has used."""
    from vt_transformer_amd.engine.step import ModelRunner, StepEntry
    from vt_transformer_amd.parts import MIXERS
    rt = runtime(dtype)
    width, nh, d, dv, decay = 40, 2, 20, 36, [0.9, 0.995]
    mixer = MIXERS.build(PartSpec("decayed_attention", dict(num_heads=nh, key_dim=d, value_dim=dv, decay=decay, norm_eps=1e-5)), rt=rt,
                         width=width, prefix="m.", shared={})
    w = weights_for(mixer, 5, 0.3)
    mixer.load(w.__getitem__, rt)
    runner = ModelRunner(OneMixer(mixer), rt, 16, 512, 4, 512)
    step_part(runner, mixer, torch.ones(30, width, dtype=dtype), [(0, 30)], rid="old")
    lens = [200, 5, 130, 66]
    xs = [(torch.randn(n, width, generator=torch.Generator().manual_seed(n)) * 0.8).to(dtype) for n in lens]
    refs = [pl.lightning_mixer(x.double(), strip(w, "m."), "", dict(heads=nh, decay=decay), 1e-5) for x in xs]
    sizes = [[130, 1, 1, 68], [2, 1, 1, 1], [1, 128, 1], [65, 1]]
    slots = []
    for i in range(4):
        runner.admit(i)
        slots.append(runner.cache.get(i).slot)
    runner.storage.clear_state(slots)
    at, got = [0] * 4, [[] for _ in lens]
    for s in range(4):
        live = [i for i in range(4) if s < len(sizes[i])]
        ctx = runner.build_context([StepEntry(i, [0] * sizes[i][s], []) for i in live])
        y = mixer.forward(torch.cat([xs[i][at[i]:at[i] + sizes[i][s]] for i in live]).to(DEV), ctx, None, runner.storage.state[0])
        row = 0
        for i in live:
            got[i].append(y[row:row + sizes[i][s]].float().cpu().clone())
            row += sizes[i][s]
            at[i] += sizes[i][s]
            runner.cache.commit(i, at[i])
    for i in range(4):
        assert rel(torch.cat(got[i]), refs[i][:at[i]]) < PART_TOL[dtype], i


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16, torch.float16])
def test_decayed_attention_known_answer(dtype):
    """Weights that pass their input through, one token whose key points along element 0: every later position returns its
    value times decay^distance (without the activation and the norm: the kernels alone), hundreds of positions on, in a
    prompt, across portions and token by token."""
    from vt_transformer_amd.kernels import ops
    from vt_transformer_amd.parts.decayed_attention import plan_chunks
    nh, d, dv, t, star = 2, 16, 12, 400, 5
    decay = torch.tensor([0.5, 0.995])
    powers = (decay.double()[:, None] ** torch.arange(ops.DECAYED_CHUNK + 1)).float().to(DEV)
    x = torch.zeros(t, nh * (2 * d + dv))
    x[:, 0], x[:, d] = 1.0, 2.0                       # queries
    x[star, nh * d], x[star, nh * d + d] = 1.0, 0.5   # the keys
    x[:, 2 * nh * d:] = 3.0
    x = x.to(dtype)
    dist = (torch.arange(t) - star).double()
    want = torch.stack([3.0 * decay.double()[h] ** dist.clamp(min=0) * (dist >= 0) for h in range(nh)], dim=1)
    for cuts in ([(0, t)], [(0, 3), (3, 70), (70, 71), (71, 300), (300, t)], one_by_one(0, t)):
        state = torch.zeros(2, nh * d * dv, device=DEV)
        slots = torch.tensor([1], dtype=torch.int32, device=DEV)
        out = []
        for a, b in cuts:
            xx = x[a:b].to(DEV).contiguous()
            o = torch.full((b - a, nh * dv), 9.0, device=DEV)
            if b - a > 1:
                plan = torch.from_numpy(plan_chunks([0, b - a])).to(DEV)
                n_chunks = (plan.numel() - 2) // 2
                work = torch.full((n_chunks * nh * d * dv,), float("nan"), device=DEV)
                ops.decayed_attention_chunked(xx, 0, nh * d, 2 * nh * d, powers, state, plan, n_chunks, slots, work, o, nh, d, dv, silu=False)
            else:
                start = torch.tensor([0, 1], dtype=torch.int32, device=DEV)
                ops.decayed_attention(xx, 0, nh * d, 2 * nh * d, decay.to(DEV), state, start, slots, o, nh, d, dv, silu=False, single=True)
            out.append(o.cpu())
        got = torch.cat(out).reshape(t, nh, dv)
        assert rel(got, want[:, :, None].expand(t, nh, dv)) < 1e-5
        assert float(state[0].abs().max()) == 0.0


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("nh,kvh,d,dv,window,keep,rot", [
    (4, 2, 16, 32, 12, 5, 8), (4, 1, 64, 32, 33, 40, 32), (3, 3, 20, 10, 7, 3, 6), (16, 1, 32, 16, 17, 16, 32), (8, 2, 48, 80, 1, 1, 0),
    (5, 1, 48, 80, 40, 17, 48), (4, 1, 16, 16, 50, 33, 8), (2, 1, 18, 6, 23, 0, 4), (4, 2, 16, 16, 0, 0, 16),
])
def test_attention_with_kept_tokens(dtype, nh, kvh, d, dv, window, keep, rot):
    """The left mixer of a pair (biases everywhere, neighbours rotated, banded frequencies, capped scores) under windows with
    kept tokens, in portions that cut pages, and decoded one by one."""
    from vt_transformer_amd.engine.step import ModelRunner
    from vt_transformer_amd.parts import MIXERS
    rt = runtime(dtype)
    width, t = 72, 200
    scaling = dict(factor=4.0, original=64.0, low=1.0, high=4.0)
    position = PartSpec("rotary", dict(theta=500.0, dim=rot, scaling=dict(kind="bands", **scaling))) if rot else None
    mixer = MIXERS.build(PartSpec("masked_attention", dict(
        num_heads=nh, num_kv_heads=kvh, key_dim=d, value_dim=dv, qkv_bias=True, o_bias=True, position=position, rot_pairs="neighbours",
        scale=0.3, softcap=5.0, window=window, keep_first=keep, names={"q": "q", "k": "k", "v": "v", "o": "o", "q_bias": "q.b",
                                                                       "k_bias": "k.b", "v_bias": "v.b", "o_bias": "o.b"})),
        rt=rt, width=width, prefix="a.", shared={})
    w = weights_for(mixer, 3, 0.3)
    mixer.load(w.__getitem__, rt)
    need = mixer.cache_need()
    assert (need.window, need.keep_first) == (window, keep)
    runner = ModelRunner(OneMixer(mixer), rt, 16, 256, 4, 256)
    x = (torch.randn(t, width, generator=torch.Generator().manual_seed(6)) * 0.7).to(dtype)
    m = {"heads": nh, "kv_heads": kvh, "dim": d, "vdim": dv, "scale": 0.3, "softcap": 5.0}
    if rot:
        m["rot"] = {"dims": rot, "base": 500.0, "scaling": scaling}
    if window:
        m["mask"] = {"size": window, "keep_first": keep}
    ref = pl.left_mixer(x.double(), strip(w, "a."), "", m)
    for cuts in ([(0, t)], CUTS + [(83, 130), (130, t)], [(0, 1), (1, 3), (3, 40), (40, 41), (41, 150)] + one_by_one(150, t),
                 one_by_one(0, t)):
        assert rel(step_part(runner, mixer, x, cuts), ref) < PART_TOL[dtype], cuts[:6]
        runner.cache.check()


@pytest.mark.parametrize("dtype,nh,d", [(torch.float32, 2, 12), (torch.bfloat16, 2, 12), (torch.bfloat16, 2, 16), (torch.bfloat16, 4, 16)])
@pytest.mark.parametrize("star,window,keep", [(3, 20, 4), (3, 20, 3), (15, 33, 16), (16, 33, 16), (16, 33, 17), (31, 50, 32), (32, 50, 32),
                                              (0, 7, 1), (40, 70, 33), (63, 64, 64), (64, 64, 64)])
def test_one_key_inside_and_outside_of_what_is_kept(dtype, nh, d, star, window, keep):
    """One key takes nearly all the weight from whoever sees it: the last kept token is seen from everywhere, the first one
    that is not kept until the window has passed it, to the position.  On the plain kernel (float32, and heads of 12), the
    one for portions (2 heads), the one whose waves share keys (4) and the one for single tokens; whole prompts, portions
    that end around the window's edge, and decoding across it while the pages in between go to another request."""
    from vt_transformer_amd.engine.step import ModelRunner, StepEntry
    from vt_transformer_amd.kernels import ops
    from vt_transformer_amd.parts import MIXERS
    from vt_transformer_amd.parts.masked_attention import run_masked_attention
    rt = runtime(dtype)
    dv, t = 16, 260
    mixer = MIXERS.build(PartSpec("masked_attention", dict(num_heads=nh, num_kv_heads=1, key_dim=d, value_dim=dv, scale=1.0, window=window,
                                                           keep_first=keep)), rt=rt, width=8, prefix="a.", shared={})
    runner = ModelRunner(OneMixer(mixer), rt, 16, 512, 2, 512)
    y = torch.randn(t, (nh + 1) * d + dv, generator=torch.Generator().manual_seed(5)) * 0.1
    y[:, :nh * d] = 0
    for h in range(nh):
        y[:, h * d] = 6.0
    y[star, nh * d] = 6.0
    y[star, (nh + 1) * d:] = 50.0
    last = t - 1 if star < keep else star + window - 1        # the last position that sees it
    edge = min(last, star + window - 1)

    def run(rid, rows, at):
        ctx = runner.build_context([StepEntry(rid, [0] * len(rows), [])])
        cache = runner.storage.layer_caches(ctx.block_tables)[0]
        yy = rows.to(DEV).to(dtype).contiguous()
        q = torch.empty(len(rows), nh * d, dtype=dtype, device=DEV)
        out = torch.empty(len(rows), nh * dv, dtype=dtype, device=DEV)
        ops.qk_prepare(yy, None, None, ctx.positions, ctx.tok_entry, cache.block_table, q, cache["k"], cache["v"], nh, 1, d, dv, None)
        run_masked_attention(rt, ctx, cache, q, out, nh, 1, d, dv, 1.0, window=window, keep_first=keep)
        runner.cache.commit(rid, at + len(rows))
        return out.float().cpu()
    for cuts in ([(0, t)], [(0, star + 1), (star + 1, edge), (edge, edge + 2), (edge + 2, t)],
                 [(0, max(1, edge - 2))] + one_by_one(max(1, edge - 2), edge + 4) + [(edge + 4, t - 2), (t - 2, t - 1), (t - 1, t)]):
        runner.admit("r")
        runner.admit("other")
        outs, other = [], 0
        for a, b in cuts:
            assert runner.cache.reserve([("r", b), ("other", other + 16)])
            outs.append(run("r", y[a:b], a))
            # another request writes large keys into the pages that the window has given back
            run("other", torch.full((16, y.shape[1]), 7.0), other)
            other += 16
        for rid in ("r", "other"):
            runner.release(rid)
        got = torch.cat(outs)
        assert float(got[star:last + 1].min()) > 49.0, "a position that should see the key lost it"
        assert float(got[last + 1:].abs().max() if last + 1 < t else 0.0) < 1.0, "a position saw a key beyond its window"
        assert float(got[:star].abs().max() if star else 0.0) < 1.0


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [56, 100, 1040])
def test_pair_of_normed_mixers(dtype, width):
    """The whole pair: both results normed over the width and averaged, handed on whole and in pieces."""
    from vt_transformer_amd.engine.step import ModelRunner
    from vt_transformer_amd.config import config_from_dict
    from vt_transformer_amd.parts import MIXERS
    L = pair(window=20, keep=7, r_heads=3, r_kv=1, r_dim=12, r_vdim=20, conv=4, a_rank=9, g_rank=3)
    cfg = {"architecture": "Lilatar", "vocab": 20, "width": width, "norm": {"eps": 1e-3}, "layers": [L]}
    spec = config_from_dict(copy.deepcopy(cfg)).to_spec().layers[0].mixer
    params = dict(spec.params)
    params.pop("prefix")
    rt = runtime(dtype)
    mixer = MIXERS.build(PartSpec(spec.kind, params), rt=rt, width=width, prefix="p.", shared={})
    w = weights_for(mixer, 13, 0.3 * (56 / width) ** 0.5)
    w["p.right.A_log"] = torch.log(torch.linspace(0.02, 1.5, 3)).to(torch.bfloat16).float()
    mixer.load(w.__getitem__, rt)
    runner = ModelRunner(OneMixer(mixer), rt, 16, 256, 3, 256)
    assert runner.storage.manager.groups[0].keep_first == 7 and mixer.replayable and mixer.hands_pieces
    t = 110
    x = (torch.randn(t, width, generator=torch.Generator().manual_seed(14)) * 0.8).to(dtype)
    ref = pl.pair_mixer(x.double(), strip(w, "p."), "", L["mixer"], 1e-3)
    for cuts in ([(0, t)], CUTS, [(0, 50)] + one_by_one(50, t)):
        end = cuts[-1][1]
        got = step_part(runner, mixer, x, cuts)
        assert rel(got, ref[:end]) < 2 * PART_TOL[dtype]
        assert torch.equal(step_part(runner, mixer, x, cuts, pieces=True), got)


@pytest.mark.parametrize("width", [40, 51, 100, 1024, 2048, 2052, 4096, 8192, 8196])
def test_norm_on_the_output_with_a_pair_and_the_norm_behind(width):
    """A pair of normed results in the place of one, alone and beside other pieces; the norm behind in the copy's place."""
    from vt_transformer_amd.kernels import ops
    g = torch.Generator().manual_seed(width)
    n, top, eps = 5, 2, 1e-2
    gain, g1, g2, gn = (1.0 + torch.randn(width, generator=g) * 0.3 for _ in range(4))
    h, choices = torch.randn(n, width, generator=g), torch.randn(n * top, width, generator=g)
    for da, db in ((torch.float32, torch.float32), (torch.bfloat16, torch.float32), (torch.bfloat16, torch.bfloat16)):
        a, b = torch.randn(n, width, generator=g).to(da), (torch.randn(n, width, generator=g) * 3.0).to(db)
        u = 0.5 * pl.unit_rms(a.double(), 1e-3) * g1.double() - 1.5 * pl.unit_rms(b.double(), 1e-3) * g2.double()
        spec = ((a.to(DEV), g1.to(DEV), 0.5), (b.to(DEV), g2.to(DEV), -1.5), 1e-3)
        assert rel(ops.sublayer_sum(torch.full((n, width), 9.0, device=DEV), pair=spec), u) < 1e-6
        for with_choices in (False, True):
            uu = u + choices.double().reshape(n, top, width).sum(1) if with_choices else u
            more = {"choices": choices.to(DEV)} if with_choices else {}
            ref = h.double() + 0.7 * pl.unit_rms(uu, eps) * gain.double()
            for copy_dtype in (torch.float32, torch.bfloat16):
                for behind in (False, True):
                    hd, cp = h.to(DEV).clone(), torch.empty(n, width, dtype=copy_dtype, device=DEV)
                    kw = dict(next_gain=gn.to(DEV), next_eps=1e-4) if behind else {}
                    ops.output_norm_add(hd, gain.to(DEV), eps, 0.7, copy=cp, pair=spec, **more, **kw)
                    assert rel(hd, ref) < 2e-6
                    want = pl.unit_rms(ref, 1e-4) * gn.double() if behind else ref
                    assert rel(cp, want) < (3e-6 if copy_dtype == torch.float32 else 6e-3)
    # a single result with the norm behind
    y = torch.randn(n, width, generator=g)
    hd, cp = h.to(DEV).clone(), torch.empty(n, width, device=DEV)
    ops.output_norm_add(hd, gain.to(DEV), eps, 1.0, y=y.to(DEV), copy=cp, next_gain=gn.to(DEV), next_eps=1e-4)
    ref = h.double() + pl.unit_rms(y.double(), eps) * gain.double()
    assert rel(hd, ref) < 2e-6 and rel(cp, pl.unit_rms(ref, 1e-4) * gn.double()) < 3e-6


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width,inter", [(96, 80), (64, 200), (100, 36), (52, 20), (256, 1040)])
def test_feed_forward_without_a_gate(dtype, width, inter):
    from vt_transformer_amd.parts import FEED_FORWARDS
    rt = runtime(dtype)
    ff = FEED_FORWARDS.build(PartSpec("plain_mlp", dict(intermediate_size=inter)), rt=rt, width=width, prefix="f.")
    assert set(ff.tensors()) == {"f.up", "f.down"} and ff.replayable
    w = weights_for(ff, 12, 0.2)
    ff.load(w.__getitem__, rt)
    for rows in (1, 5, 16, 17, 33, 64, 65, 130, 300):
        x = torch.randn(rows, width, generator=torch.Generator().manual_seed(rows)).to(dtype)
        assert rel(ff.forward(x.to(DEV)), pl.squared_relu_mlp(x.double(), strip(w, "f."), "")) < PART_TOL[dtype], rows


@pytest.mark.parametrize("rows,m,k", [(5, 200, 96), (16, 48, 4096), (30, 96, 128), (64, 4096, 256), (40, 128, 16384), (50, 132, 16384),
                                      (64, 9000, 64), (100, 160, 1024), (9, 40, 100)])
def test_squared_relu_on_a_products_sums(rows, m, k):
    """The few-row products in all their arrangements (k split over waves, over blocks, not at all; any shape)."""
    from vt_transformer_amd.kernels import ops
    g = torch.Generator().manual_seed(m)
    x, w = torch.randn(rows, k, generator=g).to(torch.bfloat16), (torch.randn(m, k, generator=g) / k ** 0.5).to(torch.bfloat16)
    bias = torch.randn(m, generator=g)
    packed = ops.pack_matrix_bf16(w.to(DEV))
    need = ops.linear_bf16_workspace(rows, m, k) if rows > 16 else 0
    work = torch.empty(need, device=DEV) if need else None
    ref = torch.relu(x.double() @ w.double().T + bias.double()).square()
    for out_dtype, tol in ((torch.float32, 1e-4), (torch.bfloat16, 6e-3)):
        out = torch.empty(rows, m, dtype=out_dtype, device=DEV)
        ops.linear_bf16(x.to(DEV), packed, bias.to(DEV), out, work, act="squared_relu")
        assert rel(out, ref) < tol


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("experts,top,inter,width", [(6, 2, 40, 96), (5, 1, 24, 64), (4, 4, 16, 128), (7, 2, 20, 100), (16, 4, 48, 256),
                                                     (2, 1, 200, 72), (12, 3, 136, 136)])
def test_experts_without_a_gate(dtype, experts, top, inter, width):
    """Softmax scores of the chosen experts as weights, as they are; few rows and many, whole and in pieces."""
    from vt_transformer_amd.parts import FEED_FORWARDS
    from vt_transformer_amd.parts.base import SublayerPieces
    rt = runtime(dtype)
    ff = FEED_FORWARDS.build(PartSpec("expert_mixture", dict(num_experts=experts, top=top, intermediate_size=inter, score="softmax",
                                                             weight_on="output", activation="squared_relu")), rt=rt, width=width, prefix="f.")
    assert "f.e0.gate" not in ff.tensors()
    w = weights_for(ff, 12, 0.2)
    ff.load(w.__getitem__, rt)
    for rows in (1, 3, 7, 30, 150, 700):
        x = torch.randn(rows, width, generator=torch.Generator().manual_seed(rows)).to(dtype)
        margins = []
        ref = pl.mixture(x.double(), strip(w, "f."), "", moe(experts, top, inter), margins)
        sure = margins[0] > 2e-5
        got = ff.forward(x.to(DEV)).float().cpu().clone()
        assert rel(got[sure], ref[sure]) < PART_TOL[dtype], rows
        pieces = ff.forward(x.to(DEV), None, pieces=True)
        assert isinstance(pieces, SublayerPieces) and rel(pieces.materialize(), got) < 1e-6


@pytest.mark.parametrize("heads,dim", [(1, 40), (3, 200), (1, 513), (1, 900), (1, 2048), (2, 700), (1, 3000), (1, 4100)])
def test_gated_norm_over_wide_heads(heads, dim):
    from vt_transformer_amd.kernels import ops
    g = torch.Generator().manual_seed(dim)
    o, gate, w = torch.randn(6, heads * dim, generator=g), torch.randn(6, heads * dim + 8, generator=g), torch.randn(heads * dim, generator=g)
    for column in (4, 5):       # (16-byte accesses, and not)
        for gdt, odt in ((torch.float32, torch.float32), (torch.float32, torch.bfloat16), (torch.bfloat16, torch.bfloat16)):
            gd, out = gate.to(gdt), torch.empty(6, heads * dim, dtype=odt, device=DEV)
            for kind, f in (("sigmoid", torch.sigmoid), ("silu", pl.silu)):
                ops.gated_rmsnorm(o.to(DEV), w.to(DEV), gd.to(DEV), column, out, heads, dim, 1e-3, gate_kind=kind)
                ref = pl.unit_rms(o.double().reshape(6, heads, dim), 1e-3).reshape(6, -1) * w.double() * f(gd.double()[:, column:column + heads * dim])
                assert rel(out, ref) < (3e-6 if odt == torch.float32 else 6e-3)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_stream_after_every_layer(folders, dtype):
    """And what a layer hands on is the norm that the next one starts with."""
    from vt_transformer_amd.engine.step import StepEntry
    folder = folders["A", dtype]
    cfg, w = pl.read_folder(folder)
    toks = rh.random_requests(cfg["vocab"], [29], seed=1)["r0"]
    streams = []
    pl.forward(cfg, w, toks, streams)
    runner = make_runner(folder, dtype, pool_tokens=64, max_requests=1)
    seen, layers = [], runner.model.layers
    for i, block in enumerate(layers):
        def wrapped(h, delta, ctx, cache, state, next_norm=None, inner=block.forward, i=i):
            h, d = inner(h, delta, ctx, cache, state, next_norm=next_norm)
            seen.append(h.cpu().double())
            if i + 1 < len(layers):
                assert d.norm is layers[i + 1].norm_in
                assert rel(d.x, pl.unit_rms(seen[-1], 1e-5) * w[f"l{i + 1}.norm1"]) < (1e-5 if dtype == "float32" else 6e-3)
            else:
                assert d is None
            return h, d
        block.forward = wrapped
    runner.admit("r")
    runner.step([StepEntry("r", toks, [len(toks) - 1])])
    assert len(seen) == len(streams) == 4
    for i, (a, b) in enumerate(zip(seen, streams)):
        assert rel(a, b) < (3e-5 if dtype == "float32" else 4e-2), f"layer {i}"


def test_blocks_of_other_kinds_around_this_one():
    """A model whose layers are of three kinds (a norm in front of the sublayers, behind them, on both ends) in turn: what
    one kind hands on, the other goes on from."""
    from vt_transformer_amd.config.base import LayerSpec, ModelSpec
    from vt_transformer_amd.engine.step import ModelRunner, StepEntry
    from vt_transformer_amd.models.model import DecoderModel
    width, vocab, eps = 64, 50, 1e-5

    def norm(name):
        return PartSpec("rmsnorm", {"eps": eps, "name": name})
    mixer = PartSpec("decayed_attention", dict(num_heads=2, key_dim=8, value_dim=12, decay=[0.8, 0.99], norm_eps=eps, prefix="mix."))
    mlp = PartSpec("plain_mlp", dict(intermediate_size=40, prefix="mlp."))
    norms = {"prenorm": {"input": norm("n1"), "post_mixer": norm("n2")},
             "output_norm": {"mixer_output": norm("n1b"), "feed_forward_output": norm("n2b")},
             "sandwich": {"input": norm("n1"), "mixer_output": norm("n1b"), "post_mixer": norm("n2"), "feed_forward_output": norm("n2b")}}
    kinds = ["sandwich", "prenorm", "sandwich", "output_norm", "sandwich", "sandwich", "prenorm", "output_norm"]
    spec = ModelSpec("mixed", vocab, width, PartSpec("embedding", {"name": "embed"}),
                     [LayerSpec(PartSpec(k, {}), mixer, mlp, norms[k], f"l{i}.") for i, k in enumerate(kinds)],
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

        def around(x, f, before, after):
            y = f(pl.unit_rms(x, eps) * wd[before] if before in wd else x)
            return x + (pl.unit_rms(y, eps) * wd[after] if after in wd else y)
        for i in range(len(kinds)):
            p = f"l{i}."
            x = around(x, lambda h: pl.lightning_mixer(h, wd, p + "mix.", dict(heads=2, decay=[0.8, 0.99]), eps), p + "n1", p + "n1b")
            x = around(x, lambda h: pl.squared_relu_mlp(h, wd, p + "mlp."), p + "n2", p + "n2b")
        ref = pl.unit_rms(x, eps) * wd["final.norm"] @ wd["head"].T
        runner = ModelRunner(model, rt, 16, 64, 1, 64)
        runner.admit("r")
        got = [runner.step([StepEntry("r", ids[a:b], list(range(b - a)))]).float().cpu() for a, b in ((0, 17), (17, 18), (18, 21))]
        assert rel(torch.cat(got), ref) < (2e-5 if dtype == torch.float32 else 4e-2)


# ---------------------------------------------------------------------------
# whole models: schedules against the plain implementation
# ---------------------------------------------------------------------------
LENGTHS = [150, 1, 23, 90, 2, 70]


@pytest.mark.parametrize("name,dtype", [(n, d) for n in "ABCD" for d in ("float32", "bfloat16")] + [("A", "float16"), ("D", "float16")])
def test_schedules(folders, name, dtype):
    """Whole prompts; most of a prompt and then its last tokens one by one; portions of changing sizes down to two
    tokens; unequal requests side by side with three slots and few pages, so that both are used again."""
    folder, vocab = folders[name, dtype], CONFIGS[name]["vocab"]
    reqs = rh.random_requests(vocab, LENGTHS, seed=3)
    cache = {}
    runner = make_runner(folder, dtype, pool_tokens=320, max_requests=3)
    runner.decode_graphs = True
    traces = [
        rh.trace_alone(reqs, {r: [(0, len(t))] for r, t in reqs.items()}),
        rh.trace_alone(reqs, {r: [(0, max(1, len(t) - 30))] + one_by_one(max(1, len(t) - 30), len(t)) for r, t in reqs.items()}),
        rh.trace_alone(reqs, {r: rh.cut(t, [7, 2, 16, 3, 2, 33, 1, 5, 66]) for r, t in reqs.items()}),
        rh.trace_mixed(reqs, {r: rh.cut(t, [9, 2, 1, 1, 70, 1, 1, 1, 4]) for r, t in reqs.items()}, max_live=3, seed=5),
    ]
    assert rh.max_live_tokens(traces[3]) <= 320
    gots = []
    for steps in traces:
        gots.append(rh.run_in_process(runner, steps))
        check_logits(folder, reqs, steps, gots[-1], dtype, cache)
    if dtype == "float32":
        # a position's logits do not depend on the cut, the batch, the pages or the slots
        flat = {}
        for steps, got in zip(traces, gots):
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
                assert float(np.abs(rows[0] - r).max()) <= 4e-5 * float(np.abs(rows[0]).max()), f"{key} depends on the schedule"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_across_windows_and_pages(folders, dtype):
    folder, vocab = folders["A", dtype], CONFIGS["A"]["vocab"]
    reqs = rh.random_requests(vocab, [190], seed=9)
    steps = rh.trace_alone(reqs, {"r0": [(0, 5)] + one_by_one(5, 190)})
    runner = make_runner(folder, dtype, pool_tokens=192, max_requests=1)
    runner.decode_graphs = True
    check_logits(folder, reqs, steps, rh.run_in_process(runner, steps), dtype)
    assert sum(runner.cache.available_pages()) == sum(p.num_pages for p in runner.cache.pools)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_request_longer_than_its_pool(tmp_path, dtype):
    """Pages for a window, a portion and the kept tokens suffice for a request several times as long: the kept ones stay,
    those in between are used again (a second request writes into them)."""
    cfg = {"architecture": "Lilatar", "vocab": 61, "width": 64, "norm": {"eps": 1e-5}, "logit_scale": 0.5,
           "layers": [pair(window=20, keep=18, mlp=dense(40)), lightning(), pair(window=9, keep=33, mlp=moe(4, 2, 16))]}
    folder = write_model(cfg, str(tmp_path / "m"), seed=77, clear_routes=True)
    reqs = rh.random_requests(61, [230, 150], seed=13)
    for cuts in ([10], [50, 1, 1, 2, 1, 1, 1, 1, 3, 16]):
        runner = make_runner(folder, dtype, pool_tokens=224, max_requests=2, max_seq_len=256)
        runner.decode_graphs = True
        steps = rh.trace_mixed(reqs, {r: rh.cut(t, cuts) for r, t in reqs.items()}, max_live=2, seed=3)
        check_logits(folder, reqs, steps, rh.run_in_process(runner, steps), dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_many_tokens_at_once(tmp_path, dtype):
    """Prompts of some hundred tokens (several chunks, tiles of many pairs of an expert, key ranges of many pages) against the
    same prompts in portions."""
    cfg = {"architecture": "Lilatar", "vocab": 90, "width": 64, "norm": {"eps": 1e-6}, "logit_scale": 0.25,
           "layers": [lightning(heads=2, dim=32, vdim=64, decay=[0.95, 0.999], mlp=moe(4, 2, 48)),
                      pair(heads=4, kv_heads=1, dim=64, vdim=32, window=130, keep=20, scale=0.1, rot_dims=32, r_dim=32, r_vdim=32,
                           mlp=moe(3, 1, 48))]}
    folder = write_model(cfg, str(tmp_path / "m"), seed=77, clear_routes=True)
    reqs = rh.random_requests(90, [330, 170], seed=2)
    runner = make_runner(folder, dtype, pool_tokens=576, max_requests=2)
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
    portions = {r: [(0, len(t) - 16)] + one_by_one(len(t) - 16, len(t)) for r, t in reqs.items()}
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
    cfg, w = pl.read_folder(folder)
    prompts = [r for r in rh.random_requests(cfg["vocab"], [19, 3, 75], seed=21).values()]
    eng = Engine(folder, dtype=dtype, num_pages=24, max_running_reqs=2, max_seq_len=128, chunk_size=16, max_extend_tokens=24)
    got = eng.generate(prompts, SamplingParams(max_tokens=8, ignore_eos=True))
    for p, g in zip(prompts, got):
        assert len(g) == 8
        if dtype == "float32":
            want, lead = pl.greedy(cfg, w, p, 8)
            assert lead > 1e-3 and g == want
        else:
            logits = pl.forward(cfg, w, p + g)
            for i, tok in enumerate(g):
                row = logits[len(p) - 1 + i]
                assert float(row.max() - row[tok]) <= 5e-2 * float(row.abs().max())


def test_trace_run_with_a_lilatar_folder(folders, tmp_path):
    folder, vocab = folders["D", "float32"], CONFIGS["D"]["vocab"]
    reqs = rh.random_requests(vocab, [90, 9, 27], seed=17)
    steps = rh.trace_mixed(reqs, {r: rh.cut(t, [6, 2, 11, 1, 65]) for r, t in reqs.items()}, max_live=2, seed=2)
    got = rh.run_trace_run(folder, "float32", steps, str(tmp_path / "out"), rh.max_live_tokens(steps), vocab,
                           extra_args=("--max-requests", "2"))
    check_logits(folder, reqs, steps, got, "float32")


# ---------------------------------------------------------------------------
# configurations drawn at random
# ---------------------------------------------------------------------------
def random_lilatar_config(seed: int) -> dict:
    rs = np.random.RandomState(seed)
    pick = lambda xs: xs[rs.randint(len(xs))]      # noqa: E731
    layers = []
    for _ in range(rs.randint(2, 6)):
        u = rs.rand()
        experts = int(rs.randint(1, 13))
        mlp = None if u < 0.15 else dense(int(pick([8, 36, 64, 104]))) if u < 0.5 else moe(experts, int(rs.randint(1, experts + 1)),
                                                                                            int(pick([8, 20, 48])))
        if rs.rand() < 0.45:
            heads = int(rs.randint(1, 6))
            dim, vdim = pick([(8, 8), (16, 32), (64, 20), (12, 100), (6, 5), (48, 144), (4, 16)])
            layers.append(lightning(heads, dim, vdim, [float(x) for x in np.round(1.0 - 10.0 ** -rs.uniform(0.0, 4.0, heads), 6)], mlp))
        else:
            kv, r_kv = int(pick([1, 2, 3])), int(pick([1, 2, 3]))
            dim, vdim = pick([(16, 16), (16, 32), (64, 32), (20, 24), (48, 80), (8, 40), (14, 7), (64, 80)])
            window = int(pick([0, 1, 3, 16, 17, 50, 1000]))
            layers.append(pair(
                heads=kv * int(pick([1, 2, 4, 5])), kv_heads=kv, dim=dim, vdim=vdim, scale=float(pick([0.1, 0.3, 0.6])),
                softcap=float(pick([0.0, 2.0, 20.0])), window=window, keep=int(pick([0, 1, 5, 16, 40])), rot_dims=int(pick([0, 2, dim // 2 // 2 * 2, dim])),
                base=float(pick([100.0, 10000.0])), scaling=pick([None, (8.0, 40.0, 1.0, 4.0), (1.0, 32.0, 1.0, 2.0), (3.0, 200.0, 0.5, 16.0)]),
                r_heads=r_kv * int(pick([1, 2, 3])), r_kv=r_kv, r_dim=int(pick([8, 16, 20, 40])), r_vdim=int(pick([8, 16, 33])),
                conv=int(pick([1, 2, 4, 5])), a_rank=int(pick([1, 6, 20])), g_rank=int(pick([1, 5, 12])), mlp=mlp))
    return {"architecture": "Lilatar", "vocab": int(pick([29, 100, 257])), "width": int(pick([40, 52, 64, 96, 100, 136])),
            "norm": {"eps": float(pick([1e-6, 1e-5, 1e-3]))}, "logit_scale": float(pick([0.1, 1.0, 3.0])), "layers": layers}


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(tmp_path, seed):
    cfg = random_lilatar_config(seed)
    free = write_model(cfg, str(tmp_path / "m"), seed=100 + seed, idle=bool(seed % 2))
    clear = write_model(cfg, str(tmp_path / "f"), seed=200 + seed, clear_routes=True)
    reqs = rh.random_requests(cfg["vocab"], [100, 33, 5], seed=seed)
    for folder, dtype in ((free, "float32"), (clear, "bfloat16")):
        runner = make_runner(folder, dtype, pool_tokens=192, max_requests=2)
        runner.decode_graphs = True
        cache = {}
        whole = rh.trace_alone(reqs, {r: [(0, len(t))] for r, t in reqs.items()})
        check_logits(folder, reqs, whole, rh.run_in_process(runner, whole), dtype, cache)
        mixed = rh.trace_mixed(reqs, {r: rh.cut(t, [11, 2, 1, 1, 70, 1, 1, 3]) for r, t in reqs.items()}, max_live=2, seed=seed)
        check_logits(folder, reqs, mixed, rh.run_in_process(runner, mixed), dtype, cache)
