"""Pagatar on the GPU: the HIP kernels against the oracle's functions at odd, unaligned and
real-layer sizes in both element types; every mixer alone; planted keys at chunk edges, far back
and at page borders, in prompts and decoding; models served in float32 on every schedule within
fp32 rounding of the oracle; bf16 models through HIP-graph decode and eager mixed steps against the
oracle and across schedules; graph vs eager; greedy generation."""
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import pagatar_cases as pc  # noqa: E402
import pagatar_oracle as po  # noqa: E402
from ome_amd import ops  # noqa: E402

pytestmark = pytest.mark.gpu
DEV = "cuda"
BF, F32 = torch.bfloat16, torch.float32
DTYPES = [F32, BF]
TOL, TYPICAL = 0.2, 0.03     # 16-bit whole-model runs: every position / the median of a request


# ------------------------------------------------------------------------------ kernels
@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,W,groups,n", [(7, 24, 3, 4), (3, 40, 1, 1), (5, 16, 16, 7), (4, 21, 7, 3), (9, 64, 2, 9), (33, 2048, 4, 8),
                                          (5, 4096, 2, 17), (2, 8192, 16, 2), (3, 1032, 3, 5), (2, 9000, 5, 2), (4, 96, 32, 2)])
def test_stream_step_kernel(dt, T, W, groups, n):
    pc.stream_case(DEV, dt, T=T, W=W, groups=groups, n=n)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("width,a,b,bias", [(20, (5, 0, 3), (4, 6, 1), -1.0), (7, (33, 0, 64), (1, 1, 1), -6.0),
                                            (513, (32, 31, 33), (1, 0, 1), -5.0), (64, (700, 5, 321), (2, 65, 1), -6.0),
                                            (1030, (1500, 3000, 1), (200, 1, 129), -7.0), (96, (5000, 1, 700), (1, 1, 300), -7.0)])
def test_mingru_kernel(dt, width, a, b, bias):
    pc.mingru_case(DEV, dt, width=width, lens_a=a, lens_b=b, bias=bias)


def test_mingru_many_sequences():
    """More sequences than one wave scans at a time, unequal lengths, against the reference op."""
    g = torch.Generator().manual_seed(1)
    n = [1] * 150 + [40] + [1] * 30 + [97, 2]
    T, W = sum(n), 34
    x = torch.randn(T, 3 * W, generator=g)
    zb, xb = torch.randn(W, generator=g) - 2, torch.randn(W, generator=g)
    cu = torch.tensor([0] + torch.tensor(n).cumsum(0).tolist(), dtype=torch.int32)
    slot = torch.randperm(len(n) + 3, generator=g)[:len(n)].to(torch.int32)
    reset = (torch.rand(len(n), generator=g) < 0.3).to(torch.int32)
    st = torch.randn(len(n) + 3, W, generator=g)
    res = {}
    for dev in ("cpu", DEV):
        s = st.clone().to(dev)
        xd = x.to(dev)
        o = ops.mingru_scan(xd[:, :W], xd[:, W:2 * W], xd[:, 2 * W:], zb.to(dev), xb.to(dev), s, cu.to(dev), slot.to(dev), reset.to(dev))
        res[dev] = (o.cpu(), s.cpu())
    for a, b in zip(res["cpu"], res[DEV]):
        assert (a - b).abs().max() < 1e-5


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,H,D,vdim", [(5, 3, 64, 10), (4, 6, 64, 56), (33, 32, 128, 128), (2, 1, 64, 1), (3, 5, 256, 200), (9, 16, 64, 64)])
def test_head_gate_kernel(dt, T, H, D, vdim):
    pc.head_gate_case(DEV, dt, T=T, H=H, D=D, vdim=vdim)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("kw", [dict(), dict(K=4, dim=16, vdim=8, rot=16), dict(K=1, rot=0), dict(K=0, il=True), dict(K=7, dim=10, vdim=70),
                                dict(Hq=32, Hkv=8, dim=128, vdim=128, rot=128, K=4), dict(dim=48, vdim=40, rot=32, K=2),
                                dict(dim=48, vdim=16, rot=24, K=3), dict(dim=200, vdim=256, rot=160, K=5), dict(dim=64, vdim=64, rot=8, K=6, il=True),
                                dict(Hq=6, Hkv=3, dim=72, vdim=24, rot=48, K=0), dict(dim=130, vdim=6, rot=130, K=3),
                                dict(dim=16, vdim=8, rot=12, K=4)])
def test_conv_rope_cache_options_kernel(dt, kw):
    pc.conv_options_case(DEV, dt, **kw)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("Hq,Hkv,D,size", [(4, 2, 64, 7), (8, 2, 128, 48), (4, 1, 256, 33), (32, 8, 128, 100), (3, 3, 64, 2)])
def test_chunked_paged_attention_kernel(dt, Hq, Hkv, D, size):
    """Prompt rows that start inside a chunk and cross several, and single rows at a chunk's first
    and last position, against the reference op."""
    from ome_amd.models.common import PagedKVCache

    g = torch.Generator().manual_seed(D + size)
    P, ql, kl = 16, [70, 3, 131], [200, 103, 131]
    kv = PagedKVCache(1, 60, Hkv, D, P, dt, DEV)
    kv.k[0].copy_(torch.randn(kv.k[0].shape, generator=g))
    kv.v[0].copy_(torch.randn(kv.v[0].shape, generator=g))
    bt = (torch.randperm(59, generator=g)[:39] + 1).view(3, 13).to(torch.int32)
    cu = torch.tensor([0] + torch.tensor(ql).cumsum(0).tolist(), dtype=torch.int32)
    q = torch.randn(sum(ql), Hq, D, generator=g).to(dt)
    items = torch.tensor([[s, r] for s in range(3) for r in range(0, ql[s], 32)], dtype=torch.int32)
    c = lambda t: t.to(DEV)   # noqa: E731
    k, v = kv.layer(0)
    args = (0.3, -size)
    want = ops.paged_prefill(q, k.cpu(), v.cpu(), bt, cu, torch.tensor(kl, dtype=torch.int32), items, *args)
    got = ops.paged_prefill(c(q), k, v, c(bt), c(cu), c(torch.tensor(kl, dtype=torch.int32)), c(items), *args)
    tol = 0.03 if dt == BF else 1e-4
    assert pc.rel(got, want.double()) < tol
    for lens in ([size + 1, 2 * size, 1], [3 * size, size, min(8 * size + 1, 208)]):
        sl = torch.tensor([min(n, 208) for n in lens], dtype=torch.int32)
        qd = q[:3].contiguous()
        want = ops.paged_decode(qd, k.cpu(), v.cpu(), bt, sl, *args[:1], window=-size)
        got = ops.paged_decode(c(qd), k, v, c(bt), c(sl), *args[:1], window=-size)
        assert pc.rel(got, want.double()) < tol, lens


def test_router_with_a_correction():
    pc.router_correction_case(DEV)
    g = torch.Generator().manual_seed(2)
    for E, k in ((16, 3), (12, 2), (64, 8), (5, 5), (1, 1), (300, 16)):
        logits, corr = torch.randn(33, E, generator=g), torch.randn(E, generator=g)
        a = ops.moe_route(logits, k, False, "sigmoid", bias=corr)
        b = ops.moe_route(logits.to(DEV), k, False, "sigmoid", bias=corr.to(DEV))
        assert torch.equal(a[1].sort(-1).values, b[1].cpu().sort(-1).values)
        assert (a[0].sort(-1).values - b[0].cpu().sort(-1).values).abs().max() < 1e-6


# ------------------------------------------------------------------------------ mixers alone
@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("kw", [dict(), dict(heads=1, kv_heads=1, dim=8, vdim=8, rot_dims=8, scaling=pc.YARN),
                                dict(heads=3, kv_heads=3, dim=10, vdim=4, chunk=1000, conv=1, rot_dims=0, scale=1.3),
                                dict(heads=4, kv_heads=1, dim=70, vdim=12, chunk=3, conv=5, rot_dims=6, base=5000.0),
                                dict(heads=2, kv_heads=2, dim=6, vdim=6, chunk=1, rot_dims=6),
                                dict(heads=8, kv_heads=2, dim=128, vdim=128, chunk=40, conv=4, rot_dims=128, scaling=pc.YARN, scale=0.09),
                                dict(heads=34, kv_heads=2, dim=8, vdim=8, chunk=20, rot_dims=4, scaling=(8.0, 16, 2.0, 0.5))])
def test_chunked_attention_alone(kw, dt):
    pc.mixer_alone(DEV, dt, po.attn_layer(**kw), T=70)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("kw", [dict(), dict(heads=1, dim=8, rot_dim=8, vdim=8, kv_rank=8, q_rank=8),
                                dict(heads=5, dim=4, rot_dim=2, vdim=12, kv_rank=70, q_rank=3, scale=0.7),
                                dict(heads=18, dim=6, rot_dim=12, vdim=4, kv_rank=16, q_rank=9),
                                dict(heads=8, dim=64, rot_dim=32, vdim=64, kv_rank=256, q_rank=96, scale=0.1)])
def test_latent_attention_alone(kw, dt):
    pc.mixer_alone(DEV, dt, po.latent_layer(**kw), T=70)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("inner", [20, 1, 33, 256])
def test_mingru_alone(inner, dt):
    pc.mixer_alone(DEV, dt, po.gru_layer(inner), T=70)


@pytest.mark.parametrize("dt", DTYPES)
def test_feed_forward_alone(dt):
    for f, width in ((po.moe(), 24), (po.moe(6, 3, 9), 24), (po.moe(2, 2, 8), 24), (po.moe(1, 1, 8), 24), (po.moe(8, 3, 32), 64),
                     (po.moe(6, 2, 64), 96)):
        grouped = pc.moe_case(DEV, dt, f, width)
        assert grouped == (dt == BF and width % 32 == 0 and f["expert"]["ff"] % 32 == 0)


@pytest.mark.parametrize("dt", DTYPES)
def test_chunk_edge(dt):
    for cuts in ([60], [50] + [1] * 10, [16, 16, 16, 12], pc.portions(60, [2, 3, 7])):
        pc.planted_case(DEV, dt, "attention", 60, 53, 45, cuts, other_chunk=8)      # a chunk's first row from its last
        pc.planted_case(DEV, dt, "attention", 60, 53, 44, cuts, other_chunk=54)     # the row before: not seen
        pc.planted_case(DEV, dt, "attention", 60, 55, 54, cuts, other_chunk=11)     # in the open chunk
        pc.planted_case(DEV, dt, "attention", 60, 54, 53, cuts, other_chunk=55)     # neighbours across the edge


@pytest.mark.parametrize("dt", DTYPES)
def test_far_key_and_page_borders(dt):
    for j in (131, 128, 127, 112, 0):
        pc.planted_case(DEV, dt, "attention", 432, 431, j, [400] + [1] * 32, chunk=1000, other_chunk=210)
        pc.planted_case(DEV, dt, "latent_attention", 432, 431, j, [400] + [1] * 32)
    pc.planted_case(DEV, dt, "latent_attention", 432, 431, 16, pc.portions(432, [64, 35, 2, 17]))
    pc.planted_case(DEV, dt, "attention", 432, 431, 400, pc.portions(432, [64, 35, 2, 17]), chunk=192, other_chunk=401)


# ------------------------------------------------------------------------------ whole models
@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, cfg in (("a", pc.config_a()), ("b", pc.config_b()), ("c", pc.config_c()), ("h", pc.config_bf16())):
        w = po.make_weights(cfg, seed=11)
        out[name] = (cfg, w, po.write_model(str(tmp_path_factory.mktemp("pag_" + name)), cfg, w), {})
    return out


def _schedules(toks):
    return (pc.whole_schedule(toks), pc.decode_schedule(toks, 24), pc.chunked_schedule(toks, [2, 3, 17, 1, 32, 2]),
            pc.mixed_schedule(toks, [1, 2, 5, 16, 1, 31]))


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_float32_schedules_match_oracle(models, name):
    cfg, w, path, cache = models[name]
    toks = dict(zip("pqrstu", pc.prompts(cfg, w, [1, 2, 37, 70, 16, 33], min_margin=1e-4)))
    eng = pc.make_engine(path, DEV, "float32", max_tokens=192)
    for sched in _schedules(toks):
        pc.assert_matches_oracle(eng, cfg, w, toks, sched, 2e-4, cache)
    assert eng.runner.launch_stats["decode-graph"] > 0


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_bfloat16_odd_sizes_run_every_schedule(models, name):
    """Sizes no vector kernel takes, in 16 bits, on every schedule: the typical position against
    the oracle and against the whole-prompt run (single positions of a tiny random model may flip a
    router decision in 16 bits, so only medians are pinned here)."""
    cfg, w, path, cache = models[name]
    toks = dict(zip("pqrs", pc.prompts(cfg, w, [1, 2, 37, 50], min_margin=1e-3)))
    outs = []
    for sched in _schedules(toks):
        eng = pc.make_engine(path, DEV, "bfloat16", max_tokens=192)
        outs.append(pc.assert_matches_oracle(eng, cfg, w, toks, sched, 1e9, cache, 0.1))
    for o in outs[1:]:
        errs = torch.cat([pc.logit_errors(o[rid], outs[0][rid].double()) for rid in toks])
        assert errs.median().item() < 0.05


def test_bfloat16_schedules_match_oracle(models):
    cfg, w, path, cache = models["h"]
    toks = dict(zip("pqrstu", pc.prompts(cfg, w, [1, 2, 37, 70, 16, 33], min_margin=0.004)))
    outs = []
    for sched in _schedules(toks):
        eng = pc.make_engine(path, DEV, "bfloat16", max_tokens=192)
        outs.append(pc.assert_matches_oracle(eng, cfg, w, toks, sched, TOL, cache, TYPICAL))
    for o in outs[1:]:          # the same tokens under another schedule: only summation orders differ
        errs = torch.cat([pc.logit_errors(o[rid], outs[0][rid].double()) for rid in toks])
        assert errs.max().item() < TOL and errs.median().item() < 0.02


def test_chunk_edges_through_the_engine(tmp_path):
    both = lambda t: (pc.whole_schedule(t), pc.decode_schedule(t, 41), pc.mixed_schedule(t, [2, 1, 19, 3]))   # noqa: E731
    for dtype, tol in (("float32", 2e-4), ("bfloat16", 0.08)):
        for chunk in (16, 21, 33):
            pc.planted_engine_case(DEV, dtype, chunk, both, tmp_path / f"{dtype}{chunk}", tol)


def test_slots_and_pages_are_reused(models):
    cfg, w, path, cache = models["h"]
    ps = pc.prompts(cfg, w, [20, 3, 41, 17, 2, 33, 9, 48, 1, 25, 16, 30], seed=5, min_margin=0.004)
    toks = {f"r{i}": t for i, t in enumerate(ps)}
    for dt, tol, typ in (("bfloat16", TOL, TYPICAL), ("float32", 2e-4, None)):
        eng = pc.make_engine(path, DEV, dt, max_tokens=160)
        pc.assert_matches_oracle(eng, cfg, w, toks, pc.mixed_schedule(toks, [2, 7, 1, 16, 3], seed=8), tol, cache, typ)
        assert eng.runner.pages.num_free == eng.runner.pages.num_pages - 1 and not eng.scheduler.running


def test_graph_and_eager_decode_agree(models):
    cfg, w, path, cache = models["h"]
    toks = {"x": pc.prompts(cfg, w, [100], seed=9, min_margin=0.003)[0]}
    outs = []
    for graphs in (True, False):
        eng = pc.make_engine(path, DEV, "bfloat16", max_tokens=128, graphs=graphs)
        outs.append(pc.assert_matches_oracle(eng, cfg, w, toks, pc.decode_schedule(toks, 80), TOL, cache, TYPICAL)["x"])
        assert eng.runner.launch_stats["decode-graph"] > 0 if graphs else not eng.runner.launch_stats["decode-graph"]
    errs = pc.logit_errors(outs[0], outs[1].double())
    assert errs.max().item() < TOL and errs.median().item() < 0.01


def test_greedy_generation(models):
    cfg, w, path, _ = models["h"]
    ps = pc.prompts(cfg, w, [5, 19, 1], seed=13)
    for dt, clear in (("bfloat16", 0.25), ("float32", 1e-3)):
        eng = pc.make_engine(path, DEV, dt, max_tokens=256)
        got = pc.greedy_engine(eng, ps, 12)
        for p, g in zip(ps, got):
            want, gap = pc.greedy_reference(cfg, w, p, 12)
            assert len(g) == 12
            if gap > clear:                 # only clear-cut argmaxes are pinned
                assert g == want

