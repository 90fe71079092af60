"""Gisirax on the CPU path (fp32 reference ops) against the slow oracle: every mechanism alone,
then whole models through the engine's replay entry -- whole prompts, prefill + token-by-token
decoding, portions down to two tokens, batches of unequal requests, reused state slots and pages,
planted keys and memories far back and at page borders -- and greedy generation through the
scheduler."""
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import gisirax_cases as gc  # noqa: E402
import gisirax_oracle as go  # noqa: E402
from ome_amd.models import model_class, supported  # noqa: E402
from ome_amd.models.config import ModelConfig  # noqa: E402

DEV, DT = "cpu", torch.float32


def test_oracle_sanity():
    gc.constants_matter_case()


def test_config_envelope():
    cfg = ModelConfig.from_hf(gc.config_a())
    assert cfg.num_layers == 5 and cfg.architecture == "Gisirax" and cfg.num_heads == 4 and cfg.num_kv_heads == 2
    assert model_class(cfg).__name__ == "GisiraxForCausalLM" and supported("Gisirax")


@pytest.mark.parametrize("W", [24, 33, 64])
def test_tanh_stream(W):
    gc.tanh_stream_case(DEV, DT, W=W)


@pytest.mark.parametrize("kw", [dict(), dict(H=1, Hk=1, dk=1, dv=1, K=1), dict(H=6, Hk=2, dk=17, dv=9, K=5),
                                dict(H=2, Hk=2, dk=16, dv=16, K=2, rate=30.0, bias_spread=4.0)])
def test_channel_delta(kw):
    gc.delta_case(DEV, DT, **kw)


@pytest.mark.parametrize("kw", [dict(), dict(H=1, dk=1, dv=1, decay=(1.0,)), dict(H=2, dk=17, dv=33, decay=(1e-3, 0.999))])
def test_lightning_scan(kw):
    gc.lightning_case(DEV, DT, **kw)


def test_memories_far_back():
    """A value written at the first token, beside a chunk's edge, and read three hundred tokens later."""
    steps = ([280, 0, 1],) + ([1, 1, 1],) * 24 + ([5, 2, 2],)
    for wr in (0, 15, 16):
        gc.delta_case(DEV, DT, steps=steps, memory=(wr, 303))
        gc.lightning_case(DEV, DT, steps=steps, memory=(wr, 308))


def test_sigmoid_gate_norm():
    gc.sigmoid_gate_norm_case(DEV, DT)
    gc.sigmoid_gate_norm_case(DEV, DT, I=24, group=6)


def test_rope_table():
    gc.rope_table_case()


def test_group_routing():
    gc.group_route_case(DEV)


@pytest.mark.parametrize("kw", [dict(), dict(heads=1, kv_heads=1, dim=8, vdim=8, rot_dims=8, r_heads=1, r_dim=2, r_vdim=2, decay=(1.0,)),
                                dict(heads=3, kv_heads=3, dim=10, vdim=4, rot_dims=0, scale=1.3),
                                dict(heads=4, kv_heads=1, dim=70, vdim=12, rot_dims=6, base=5000.0, scaling=None),
                                dict(heads=2, kv_heads=2, dim=6, vdim=6, rot_dims=6, scaling=(3.0, 1.0, 2.0, 8)),
                                dict(heads=34, kv_heads=2, dim=8, vdim=8, rot_dims=8, base=10000.0, r_heads=2, decay=(0.1, 0.999))])
def test_parallel_mixers_alone(kw):
    gc.mixer_alone(DEV, DT, go.parallel_layer(**kw))


@pytest.mark.parametrize("kw", [dict(), dict(heads=1, kv_heads=1, dim=8, vdim=8, conv=1), dict(heads=6, kv_heads=2, dim=7, vdim=3, conv=6),
                                dict(heads=2, kv_heads=2, dim=70, vdim=5, conv=2)])
def test_channel_delta_mixer_alone(kw):
    gc.mixer_alone(DEV, DT, go.delta_layer(**kw))


def test_feed_forward_alone():
    for f, width in ((go.moe(), 24), (go.moe(6, 3, 9, 2, 1), 24), (go.moe(2, 2, 8, 1, 1), 24), (go.moe(1, 1, 8, 1, 1), 24),
                     (go.moe(8, 3, 32, 4, 2), 64), (go.moe(4, 2, 8, 4, 4, 1.0), 24)):
        assert not gc.moe_case(DEV, DT, f, width)


def test_one_in_the_denominator():
    gc.plus_one_case(DEV, DT)


def test_far_key_and_page_borders():
    for j in (131, 128, 127, 112, 0):                              # keys of row 431
        gc.planted_case(DEV, DT, 432, 431, j, [400] + [1] * 32)
    gc.planted_case(DEV, DT, 432, 431, 16, gc.portions(432, [64, 35, 2, 17]))


# ------------------------------------------------------------------------------ whole models
@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, cfg in (("a", gc.config_a()), ("b", gc.config_b()), ("c", gc.config_c())):
        w = go.make_weights(cfg, seed=11)
        out[name] = (cfg, w, go.write_model(str(tmp_path_factory.mktemp("gis_" + name)), cfg, w), {})
    return out


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_schedules_match_oracle(models, name):
    cfg, w, path, cache = models[name]
    toks = dict(zip("pqrstu", gc.prompts(cfg, w, [1, 2, 37, 70, 16, 33], min_margin=1e-4)))
    eng = gc.make_engine(path, DEV, "float32", max_tokens=192)
    for sched in (gc.whole_schedule(toks), gc.decode_schedule(toks, 24),
                  gc.chunked_schedule(toks, [2, 3, 17, 1, 32, 2]), gc.mixed_schedule(toks, [1, 2, 5, 16, 1, 31])):
        gc.assert_matches_oracle(eng, cfg, w, toks, sched, 2e-4, cache)


def test_planted_keys_through_the_engine(tmp_path):
    gc.planted_engine_case(DEV, "float32", lambda t: (gc.whole_schedule(t), gc.decode_schedule(t, 30), gc.mixed_schedule(t, [2, 1, 19, 3])),
                           tmp_path / "p", 2e-4)


def test_slots_and_pages_are_reused(models):
    cfg, w, path, cache = models["a"]
    ps = gc.prompts(cfg, w, [20, 3, 41, 17, 2, 33, 9, 48, 1, 25], seed=5, min_margin=1e-4)
    toks = {f"r{i}": t for i, t in enumerate(ps)}
    eng = gc.make_engine(path, DEV, "float32", max_tokens=160)
    gc.assert_matches_oracle(eng, cfg, w, toks, gc.mixed_schedule(toks, [2, 7, 1, 16, 3], seed=8), 2e-4, cache)
    assert eng.runner.pages.num_free == eng.runner.pages.num_pages - 1 and not eng.scheduler.running


def test_long_decoding(models):
    cfg, w, path, cache = models["a"]
    toks = {"x": gc.prompts(cfg, w, [100], seed=9, min_margin=1e-4)[0]}
    eng = gc.make_engine(path, DEV, "float32", max_tokens=128)
    gc.assert_matches_oracle(eng, cfg, w, toks, gc.decode_schedule(toks, 80), 2e-4, cache)


def test_residual_stream_after_every_layer(models):
    cfg, w, path, _ = models["a"]
    t = gc.prompts(cfg, w, [23], seed=3, min_margin=1e-4)[0]
    res = []
    go.forward(cfg, w, t, residuals=res)
    eng = gc.make_engine(path, DEV, "float32")
    eng.runner.model.debug_residuals = got = []
    gc.replay(eng, {"x": t}, gc.whole_schedule({"x": t}))
    assert len(got) == len(res) == 5
    for a, b in zip(got, res):
        assert gc.rel(a, b) < 1e-4


def test_greedy_generation(models):
    cfg, w, path, _ = models["a"]
    ps = gc.prompts(cfg, w, [5, 19, 1], seed=13)
    eng = gc.make_engine(path, DEV, "float32", max_tokens=256)
    got = gc.greedy_engine(eng, ps, 10)
    for p, g in zip(ps, got):
        want, gap = gc.greedy_reference(cfg, w, p, 10)
        assert len(g) == 10
        if gap > 1e-3:                 # only clear-cut argmaxes are pinned
            assert g == want


def test_incomplete_checkpoint_is_refused(models, tmp_path):
    cfg, w, _, _ = models["a"]
    for gone in ("l0.mix.q.conv", "l2.mix.a2", "l1.mix.right.norm", "l3.mix.left.out", "bigram", "head", "l0.norm1b.alpha",
                 "l2.norm2b", "final.norm.b", "l2.mlp.router", "l0.mlp.e1.up"):
        path = go.write_model(str(tmp_path / gone), cfg, {k: v for k, v in w.items() if k != gone})
        with pytest.raises(ValueError, match=gone.split(".")[-1]):
            gc.make_engine(path, DEV, "float32")
    for name, bad in (("l0.mix.dt_bias", w["l0.mix.dt_bias"][:-1]), ("bigram", w["bigram"][:-1]), ("l0.mix.k.conv", w["l0.mix.k.conv"][:, 1:])):
        with pytest.raises(ValueError, match=name.split(".", 2)[-1]):
            gc.make_engine(go.write_model(str(tmp_path / ("bad" + name)), cfg, dict(w, **{name: bad.clone()})), DEV, "float32")
    odd = gc.config_a()
    odd["layers"][1]["mixer"]["right"]["decay"] = [0.5, 0.9]
    with pytest.raises(ValueError, match="decays"):
        gc.make_engine(go.write_model(str(tmp_path / "decay"), odd, w), DEV, "float32")
