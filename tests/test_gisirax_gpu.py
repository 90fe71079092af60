"""Gisirax on the GPU: the HIP kernels against the oracle's functions at odd, unaligned and
real-layer sizes in both element types, on the chunked and the single-row path; every mixer alone;
planted keys and memories far back, at page and at chunk borders, in prompts and decoding; models
served in float32 on every schedule within fp32 rounding of the oracle; bf16 models through
HIP-graph decode and eager mixed steps against the oracle and across schedules; graph vs eager;
greedy generation."""
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import gisirax_cases as gc  # noqa: E402
import gisirax_oracle as go  # noqa: E402
from ome_amd import ops  # noqa: E402

pytestmark = pytest.mark.gpu
DEV = "cuda"
BF, F32 = torch.bfloat16, torch.float32
DTYPES = [F32, BF]
TOL, TYPICAL = 0.2, 0.03     # 16-bit whole-model runs: every position / the median of a request


# ------------------------------------------------------------------------------ kernels
@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,W", [(7, 24), (3, 33), (5, 1032), (33, 2048), (4, 4096), (2, 8192), (2, 9000)])
def test_tanh_stream_kernel(dt, T, W):
    gc.tanh_stream_case(DEV, dt, T=T, W=W)


LONG = ([100, 33, 16], [1, 1, 1], [31, 1, 200])


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("kw", [dict(), dict(H=1, Hk=1, dk=1, dv=1, K=1), dict(H=6, Hk=2, dk=17, dv=9, K=5), dict(H=2, Hk=1, dk=33, dv=70, K=9),
                                dict(H=4, Hk=4, dk=64, dv=64, K=3, steps=LONG), dict(H=8, Hk=8, dk=128, dv=128, K=4, steps=LONG),
                                dict(H=4, Hk=2, dk=128, dv=80, K=2, steps=LONG), dict(H=2, Hk=2, dk=256, dv=64, K=4),
                                dict(H=2, Hk=1, dk=200, dv=130, K=3), dict(H=3, Hk=3, dk=100, dv=34, K=4), dict(H=2, Hk=2, dk=16, dv=300, K=32)])
def test_channel_delta_kernels(dt, kw):
    gc.delta_case(DEV, dt, **kw)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("kw", [dict(rate=30.0), dict(rate=200.0, bias_spread=6.0), dict(H=2, Hk=2, dk=128, dv=64, K=4, rate=30.0, steps=LONG),
                                dict(H=4, Hk=4, dk=64, dv=16, K=3, rate=3.0, bias_spread=8.0, steps=LONG), dict(rate=1e-4)])
def test_channel_delta_forgets_fast_or_never(dt, kw):
    """Decays beyond the range of the factored form, chunks on both sides of it, and hardly any."""
    gc.delta_case(DEV, dt, **kw)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("kw", [dict(), dict(H=1, dk=1, dv=1, decay=(1.0,)), dict(H=2, dk=17, dv=33, decay=(1e-3, 0.999)),
                                dict(H=4, dk=64, dv=64, steps=LONG), dict(H=8, dk=128, dv=128, steps=LONG), dict(H=2, dk=256, dv=48),
                                dict(H=2, dk=100, dv=130, decay=(0.0, 0.7), steps=LONG)])
def test_lightning_kernels(dt, kw):
    gc.lightning_case(DEV, dt, **kw)


@pytest.mark.parametrize("dt", DTYPES)
def test_memories_far_back(dt):
    steps = ([280, 0, 1],) + ([1, 1, 1],) * 24 + ([5, 2, 2],)
    for wr in (0, 15, 16):
        gc.delta_case(DEV, dt, steps=steps, memory=(wr, 303))
        gc.delta_case(DEV, dt, H=2, Hk=2, dk=64, dv=32, steps=steps, memory=(wr, 308))
        gc.lightning_case(DEV, dt, steps=steps, memory=(wr, 308))
        gc.lightning_case(DEV, dt, H=2, dk=64, dv=32, steps=steps, memory=(wr, 303))


def test_many_sequences():
    """More sequences than one wave scans at a time, unequal lengths, against the reference ops."""
    g = torch.Generator().manual_seed(1)
    n = [1] * 70 + [40] + [1] * 30 + [97, 2, 16, 17]
    T, H, dk, dv, K = sum(n), 2, 12, 10, 3
    C = 2 * H * dk + H * dv
    x, z, b = torch.randn(T, C, generator=g), torch.randn(T, H * (dk + dv), generator=g), torch.randn(T, H, generator=g)
    cw, st, tail = torch.randn(C, K, generator=g), torch.randn(len(n) + 3, H, dv, dk, generator=g), torch.randn(len(n) + 3, C, K - 1, generator=g)
    A, db, nw = torch.tensor([-1.0, 0.5]), torch.randn(H * dk, generator=g), torch.ones(dv)
    cu = torch.tensor([0] + torch.tensor(n).cumsum(0).tolist(), dtype=torch.int32)
    slot = torch.randperm(len(n) + 3, generator=g)[:len(n)].to(torch.int32)
    reset = (torch.rand(len(n), generator=g) < 0.3).to(torch.int32)
    res = {}
    for dev in ("cpu", DEV):
        to = lambda t: t.clone().to(dev)   # noqa: E731
        sq = tuple(map(to, (cu, slot, reset)))
        s1, s2, tl, xd = to(st), to(st), to(tail), to(x)
        o1 = ops.channel_delta(xd, to(cw), tl, to(z), to(b), to(A), to(db), to(nw), 1e-5, s1, sq, H)
        o2 = ops.lightning_scan(xd[:, :H * dk], xd[:, H * dk:2 * H * dk], xd[:, 2 * H * dk:], torch.tensor([0.9, 0.5], device=dev), s2, sq)
        res[dev] = [t.cpu() for t in (o1, s1, tl, o2, s2)]
    for a, c in zip(res["cpu"], res[DEV]):
        assert (a - c).abs().max() < 1e-4 * a.abs().max()


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,I,group", [(5, 21, 21), (4, 24, 6), (33, 4096, 128), (3, 1024, 1024), (2, 4096, 4096), (9, 96, 32), (2, 15, 5), (3, 1000, 500)])
def test_sigmoid_gate_norm_kernel(dt, T, I, group):
    gc.sigmoid_gate_norm_case(DEV, dt, T=T, I=I, group=group)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("I,group", [(96, 32), (4096, 128), (512, 512), (18, 6)])
def test_silu_gate_norm_small_groups(dt, I, group):
    """The wave-per-group kernel with the SiLU gate (the gated delta rule of other models)."""
    g = torch.Generator().manual_seed(3)
    y, z = torch.randn(7, I, generator=g).to(dt), torch.randn(7, I, generator=g).to(dt)
    w = torch.randn(group, generator=g).to(dt)
    got = ops.gated_rmsnorm(y.to(DEV), z.to(DEV), w.to(DEV), group, 1e-5, norm_first=True, exact=True)
    want = go.rms_unit(y.double().view(7, -1, group), 1e-5) * w.double()
    assert gc.rel(got, want.reshape(7, I) * go.silu(z.double())) < (0.01 if dt == BF else 1e-5)


def test_group_routing():
    gc.group_route_case(DEV)


# ------------------------------------------------------------------------------ mixers alone
@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("kw", [dict(), dict(heads=1, kv_heads=1, dim=8, vdim=8, rot_dims=8, r_heads=1, r_dim=2, r_vdim=2, decay=(1.0,)),
                                dict(heads=3, kv_heads=3, dim=10, vdim=4, rot_dims=0, scale=1.3),
                                dict(heads=4, kv_heads=1, dim=70, vdim=12, rot_dims=6, base=5000.0, scaling=None),
                                dict(heads=2, kv_heads=2, dim=6, vdim=6, rot_dims=6, scaling=(3.0, 1.0, 2.0, 8)),
                                dict(heads=8, kv_heads=2, dim=128, vdim=128, rot_dims=128, base=10000.0, scale=0.09, r_heads=2, r_dim=128,
                                     r_vdim=64, decay=(0.9, 0.999)),
                                dict(heads=34, kv_heads=2, dim=8, vdim=8, rot_dims=8, base=10000.0, r_heads=2, decay=(0.1, 0.999))])
def test_parallel_mixers_alone(kw, dt):
    gc.mixer_alone(DEV, dt, go.parallel_layer(**kw), T=70)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("kw", [dict(), dict(heads=1, kv_heads=1, dim=8, vdim=8, conv=1), dict(heads=6, kv_heads=2, dim=7, vdim=3, conv=6),
                                dict(heads=2, kv_heads=2, dim=70, vdim=5, conv=2), dict(heads=4, kv_heads=4, dim=64, vdim=96, conv=4)])
def test_channel_delta_mixer_alone(kw, dt):
    gc.mixer_alone(DEV, dt, go.delta_layer(**kw), T=70)


@pytest.mark.parametrize("dt", DTYPES)
def test_feed_forward_alone(dt):
    for f, width in ((go.moe(), 24), (go.moe(6, 3, 9, 2, 1), 24), (go.moe(2, 2, 8, 1, 1), 24), (go.moe(1, 1, 8, 1, 1), 24),
                     (go.moe(8, 3, 32, 4, 2), 64), (go.moe(4, 2, 8, 4, 4, 1.0), 24), (go.moe(6, 2, 64, 3, 2, 0.6), 96)):
        grouped = gc.moe_case(DEV, dt, f, width)
        assert grouped == (dt == BF and width % 32 == 0 and f["expert"]["ff"] % 32 == 0)


@pytest.mark.parametrize("dt", DTYPES)
def test_one_in_the_denominator(dt):
    gc.plus_one_case(DEV, dt)


@pytest.mark.parametrize("dt", DTYPES)
def test_far_key_and_page_borders(dt):
    for j in (131, 128, 127, 112, 0):
        gc.planted_case(DEV, dt, 432, 431, j, [400] + [1] * 32)
    gc.planted_case(DEV, dt, 432, 431, 16, gc.portions(432, [64, 35, 2, 17]))


# ------------------------------------------------------------------------------ whole models
@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, cfg in (("a", gc.config_a()), ("b", gc.config_b()), ("c", gc.config_c()), ("h", gc.config_bf16())):
        w = go.make_weights(cfg, seed=11)
        out[name] = (cfg, w, go.write_model(str(tmp_path_factory.mktemp("gis_" + name)), cfg, w), {})
    return out


def _schedules(toks):
    return (gc.whole_schedule(toks), gc.decode_schedule(toks, 24), gc.chunked_schedule(toks, [2, 3, 17, 1, 32, 2]),
            gc.mixed_schedule(toks, [1, 2, 5, 16, 1, 31]))


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_float32_schedules_match_oracle(models, name):
    cfg, w, path, cache = models[name]
    toks = dict(zip("pqrstu", gc.prompts(cfg, w, [1, 2, 37, 70, 16, 33], min_margin=1e-4)))
    eng = gc.make_engine(path, DEV, "float32", max_tokens=192)
    for sched in _schedules(toks):
        gc.assert_matches_oracle(eng, cfg, w, toks, sched, 2e-4, cache)
    assert eng.runner.launch_stats["decode-graph"] > 0


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_bfloat16_odd_sizes_run_every_schedule(models, name):
    """Sizes no vector kernel takes, in 16 bits, on every schedule: the typical position against
    the oracle and against the whole-prompt run (single positions of a tiny random model may flip a
    router decision in 16 bits, so only medians are pinned here)."""
    cfg, w, path, cache = models[name]
    toks = dict(zip("pqrs", gc.prompts(cfg, w, [1, 2, 37, 50], min_margin=2e-3)))
    outs = []
    for sched in _schedules(toks):
        eng = gc.make_engine(path, DEV, "bfloat16", max_tokens=192)
        outs.append(gc.assert_matches_oracle(eng, cfg, w, toks, sched, 1e9, cache, 0.1))
    for o in outs[1:]:
        errs = torch.cat([gc.logit_errors(o[rid], outs[0][rid].double()) for rid in toks])
        assert errs.median().item() < 0.05


def test_bfloat16_schedules_match_oracle(models):
    cfg, w, path, cache = models["h"]
    toks = dict(zip("pqrstu", gc.prompts(cfg, w, [1, 2, 37, 60, 16, 33], min_margin=0.004)))
    outs = []
    for sched in _schedules(toks):
        eng = gc.make_engine(path, DEV, "bfloat16", max_tokens=192)
        outs.append(gc.assert_matches_oracle(eng, cfg, w, toks, sched, TOL, cache, TYPICAL))
    for o in outs[1:]:          # the same tokens under another schedule: only summation orders differ
        errs = torch.cat([gc.logit_errors(o[rid], outs[0][rid].double()) for rid in toks])
        assert errs.max().item() < TOL and errs.median().item() < 0.02


def test_planted_keys_through_the_engine(tmp_path):
    both = lambda t: (gc.whole_schedule(t), gc.decode_schedule(t, 41), gc.mixed_schedule(t, [2, 1, 19, 3]))   # noqa: E731
    for dtype, tol in (("float32", 2e-4), ("bfloat16", 0.08)):
        gc.planted_engine_case(DEV, dtype, both, tmp_path / dtype, tol)


def test_slots_and_pages_are_reused(models):
    cfg, w, path, cache = models["h"]
    ps = gc.prompts(cfg, w, [20, 3, 41, 17, 2, 33, 9, 48, 1, 25, 16, 30], seed=5, min_margin=0.004)
    toks = {f"r{i}": t for i, t in enumerate(ps)}
    for dt, tol, typ in (("bfloat16", TOL, TYPICAL), ("float32", 2e-4, None)):
        eng = gc.make_engine(path, DEV, dt, max_tokens=160)
        gc.assert_matches_oracle(eng, cfg, w, toks, gc.mixed_schedule(toks, [2, 7, 1, 16, 3], seed=8), tol, cache, typ)
        assert eng.runner.pages.num_free == eng.runner.pages.num_pages - 1 and not eng.scheduler.running


def test_graph_and_eager_decode_agree(models):
    cfg, w, path, cache = models["h"]
    toks = {"x": gc.prompts(cfg, w, [100], seed=9, min_margin=0.004)[0]}
    outs = []
    for graphs in (True, False):
        eng = gc.make_engine(path, DEV, "bfloat16", max_tokens=128, graphs=graphs)
        outs.append(gc.assert_matches_oracle(eng, cfg, w, toks, gc.decode_schedule(toks, 80), TOL, cache, TYPICAL)["x"])
        assert eng.runner.launch_stats["decode-graph"] > 0 if graphs else not eng.runner.launch_stats["decode-graph"]
    errs = gc.logit_errors(outs[0], outs[1].double())
    assert errs.max().item() < TOL and errs.median().item() < 0.01


def test_greedy_generation(models):
    cfg, w, path, _ = models["h"]
    ps = gc.prompts(cfg, w, [5, 19, 1], seed=13)
    for dt, clear in (("bfloat16", 0.25), ("float32", 1e-3)):
        eng = gc.make_engine(path, DEV, dt, max_tokens=256)
        got = gc.greedy_engine(eng, ps, 12)
        for p, g in zip(ps, got):
            want, gap = gc.greedy_reference(cfg, w, p, 12)
            assert len(g) == 12
            if gap > clear:                 # only clear-cut argmaxes are pinned
                assert g == want
