"""Pagatar on the CPU path (fp32 reference ops) against the slow oracle: every mechanism alone,
then whole models through the engine's replay entry -- whole prompts, prefill + token-by-token
decoding, portions down to two tokens, batches of unequal requests, reused state slots and pages,
planted keys at chunk edges, far back and at page borders -- and greedy generation through the
scheduler."""
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import pagatar_cases as pc  # noqa: E402
import pagatar_oracle as po  # noqa: E402
from ome_amd.models.config import ModelConfig  # noqa: E402

DEV, DT = "cpu", torch.float32


def test_oracle_sanity():
    pc.constants_matter_case()


def test_config_envelope():
    cfg = ModelConfig.from_hf(pc.config_a())
    assert cfg.num_layers == 6 and cfg.architecture == "Pagatar" and cfg.num_heads == 6 and cfg.num_kv_heads == 1


@pytest.mark.parametrize("W,groups,n", [(24, 3, 4), (40, 1, 1), (16, 16, 7), (21, 7, 3), (64, 2, 9)])
def test_stream_step(W, groups, n):
    pc.stream_case(DEV, DT, W=W, groups=groups, n=n)


def test_mingru_scan():
    pc.mingru_case(DEV, DT)
    pc.mingru_case(DEV, DT, width=7, lens_a=(33, 0, 64), lens_b=(1, 1, 1), bias=-6.0)


def test_head_gate_per_head():
    pc.head_gate_case(DEV, DT)


@pytest.mark.parametrize("kw", [dict(), dict(K=4, dim=16, vdim=8, rot=16), dict(K=1, rot=0), dict(K=0, il=True), dict(K=7, dim=10, vdim=70)])
def test_conv_rope_cache_options(kw):
    pc.conv_options_case(DEV, DT, **kw)


@pytest.mark.parametrize("kw", [dict(), dict(heads=1, kv_heads=1, dim=8, vdim=8, rot_dims=8, scaling=pc.YARN),
                                dict(heads=3, kv_heads=3, dim=10, vdim=4, chunk=1000, conv=1, rot_dims=0, scale=1.3),
                                dict(heads=4, kv_heads=1, dim=70, vdim=12, chunk=3, conv=5, rot_dims=6, base=5000.0),
                                dict(heads=2, kv_heads=2, dim=6, vdim=6, chunk=1, rot_dims=6),
                                dict(heads=34, kv_heads=2, dim=8, vdim=8, chunk=20, rot_dims=4, scaling=(8.0, 16, 2.0, 0.5))])
def test_chunked_attention_alone(kw):
    pc.mixer_alone(DEV, DT, po.attn_layer(**kw))


@pytest.mark.parametrize("kw", [dict(), dict(heads=1, dim=8, rot_dim=8, vdim=8, kv_rank=8, q_rank=8),
                                dict(heads=5, dim=4, rot_dim=2, vdim=12, kv_rank=70, q_rank=3, scale=0.7),
                                dict(heads=18, dim=6, rot_dim=12, vdim=4, kv_rank=16, q_rank=9),
                                dict(heads=2, dim=12, rot_dim=6, vdim=1, kv_rank=130, q_rank=40)])
def test_latent_attention_alone(kw):
    pc.mixer_alone(DEV, DT, po.latent_layer(**kw))


@pytest.mark.parametrize("inner", [20, 1, 33])
def test_mingru_alone(inner):
    pc.mixer_alone(DEV, DT, po.gru_layer(inner))


def test_feed_forward_alone():
    for f, width in ((po.moe(), 24), (po.moe(6, 3, 9), 24), (po.moe(2, 2, 8), 24), (po.moe(1, 1, 8), 24), (po.moe(8, 3, 32), 64)):
        assert not pc.moe_case(DEV, DT, f, width)
    pc.router_correction_case(DEV)


def test_chunk_edge():
    """Chunks of nine rows: 45 .. 53 closed, 54 .. 59 the open last one."""
    for cuts in ([60], [50] + [1] * 10, [16, 16, 16, 12], pc.portions(60, [2, 3, 7])):
        pc.planted_case(DEV, DT, "attention", 60, 53, 45, cuts, other_chunk=8)      # a chunk's first row from its last
        pc.planted_case(DEV, DT, "attention", 60, 53, 44, cuts, other_chunk=54)     # the row before: not seen
        pc.planted_case(DEV, DT, "attention", 60, 55, 54, cuts, other_chunk=11)     # in the open chunk
        pc.planted_case(DEV, DT, "attention", 60, 54, 53, cuts, other_chunk=55)     # neighbours across the edge


def test_far_key_and_page_borders():
    for j in (131, 128, 127, 112, 0):                              # keys of row 431, one long chunk / the latent layer
        pc.planted_case(DEV, DT, "attention", 432, 431, j, [400] + [1] * 32, chunk=1000, other_chunk=210)
        pc.planted_case(DEV, DT, "latent_attention", 432, 431, j, [400] + [1] * 32)
    pc.planted_case(DEV, DT, "latent_attention", 432, 431, 16, pc.portions(432, [64, 35, 2, 17]))
    pc.planted_case(DEV, DT, "attention", 432, 431, 400, pc.portions(432, [64, 35, 2, 17]), chunk=192, other_chunk=401)


# ------------------------------------------------------------------------------ whole models
@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, cfg in (("a", pc.config_a()), ("b", pc.config_b()), ("c", pc.config_c())):
        w = po.make_weights(cfg, seed=11)
        out[name] = (cfg, w, po.write_model(str(tmp_path_factory.mktemp("pag_" + name)), cfg, w), {})
    return out


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_schedules_match_oracle(models, name):
    cfg, w, path, cache = models[name]
    toks = dict(zip("pqrstu", pc.prompts(cfg, w, [1, 2, 37, 70, 16, 33], min_margin=1e-4)))
    eng = pc.make_engine(path, DEV, "float32", max_tokens=192)
    for sched in (pc.whole_schedule(toks), pc.decode_schedule(toks, 24),
                  pc.chunked_schedule(toks, [2, 3, 17, 1, 32, 2]), pc.mixed_schedule(toks, [1, 2, 5, 16, 1, 31])):
        pc.assert_matches_oracle(eng, cfg, w, toks, sched, 2e-4, cache)


def test_chunk_edges_through_the_engine(tmp_path):
    pc.planted_engine_case(DEV, "float32", 16, lambda t: (pc.whole_schedule(t), pc.decode_schedule(t, 30)), tmp_path / "p", 2e-4)
    pc.planted_engine_case(DEV, "float32", 21, lambda t: (pc.decode_schedule(t, 41), pc.mixed_schedule(t, [2, 1, 19, 3])),
                           tmp_path / "o", 2e-4)


def test_slots_and_pages_are_reused(models):
    cfg, w, path, cache = models["a"]
    ps = pc.prompts(cfg, w, [20, 3, 41, 17, 2, 33, 9, 48, 1, 25], seed=5, min_margin=1e-4)
    toks = {f"r{i}": t for i, t in enumerate(ps)}
    eng = pc.make_engine(path, DEV, "float32", max_tokens=160)
    pc.assert_matches_oracle(eng, cfg, w, toks, pc.mixed_schedule(toks, [2, 7, 1, 16, 3], seed=8), 2e-4, cache)
    assert eng.runner.pages.num_free == eng.runner.pages.num_pages - 1 and not eng.scheduler.running


def test_long_decoding(models):
    """Eighty tokens one by one: every chunk of the stack opens and closes over decoded tokens."""
    cfg, w, path, cache = models["a"]
    toks = {"x": pc.prompts(cfg, w, [100], seed=9, min_margin=1e-4)[0]}
    eng = pc.make_engine(path, DEV, "float32", max_tokens=128)
    pc.assert_matches_oracle(eng, cfg, w, toks, pc.decode_schedule(toks, 80), 2e-4, cache)


def test_residual_stream_after_every_layer(models):
    cfg, w, path, _ = models["a"]
    t = pc.prompts(cfg, w, [23], seed=3, min_margin=1e-4)[0]
    res = []
    po.forward(cfg, w, t, residuals=res)
    eng = pc.make_engine(path, DEV, "float32")
    eng.runner.model.debug_residuals = got = []
    pc.replay(eng, {"x": t}, pc.whole_schedule({"x": t}))
    assert len(got) == len(res) == 6
    for a, b in zip(got, res):
        assert pc.rel(a, b) < 1e-4


def test_greedy_generation(models):
    cfg, w, path, _ = models["a"]
    ps = pc.prompts(cfg, w, [5, 19, 1], seed=13)
    eng = pc.make_engine(path, DEV, "float32", max_tokens=256)
    got = pc.greedy_engine(eng, ps, 10)
    for p, g in zip(ps, got):
        want, gap = pc.greedy_reference(cfg, w, p, 10)
        assert len(g) == 10
        if gap > 1e-3:                 # only clear-cut argmaxes are pinned
            assert g == want


def test_incomplete_checkpoint_is_refused(models, tmp_path):
    cfg, w, _, _ = models["a"]
    for gone in ("l1.mix.q.b", "l4.mix.vmix", "l2.mix.z", "l3.dwa", "embed.norm", "l0.mix.dkv.norm", "l0.mlp.correction", "l2.norm2"):
        path = po.write_model(str(tmp_path / gone), cfg, {k: v for k, v in w.items() if k != gone})
        with pytest.raises(ValueError, match=gone.split(".")[-1]):
            pc.make_engine(path, DEV, "float32")
    with pytest.raises(ValueError, match="coefficients"):
        pc.make_engine(po.write_model(str(tmp_path / "dwa"), cfg, dict(w, **{"l3.dwa": w["l2.dwa"].clone()})), DEV, "float32")
    bad = pc.config_a()
    bad["layers"][5]["mixer"]["vdim"] = 10
    with pytest.raises(ValueError, match="mix"):
        pc.make_engine(po.write_model(str(tmp_path / "vdim"), bad, po.make_weights(bad)), DEV, "float32")
