"""Scenarios shared by the CPU (fp32 reference ops) and GPU (HIP kernels) Gisirax tests: every
mechanism alone against the slow oracle of ``gisirax_oracle``, small random models run through the
engine's replay entry under different schedules, planted keys and planted memories far back, at page
and at chunk borders.  The schedule builders are the ones of ``zavilorn_cases`` (they know nothing of
a design).  Every function takes the device and element type, so the two test files only bind them."""
from __future__ import annotations

import random

import torch

import gisirax_oracle as go
from ome_amd import ops
from ome_amd.models.common import AttnMeta, PagedKVCache
from ome_amd.models.mixers import (ChannelDeltaMixer, GatedWindowAttention, GroupRoutedMoE, LightningAttention, MixerCtx,
                                   ParallelMixers)
from zavilorn_cases import (chunked_schedule, decode_schedule, greedy_engine, make_engine, mixed_schedule,  # noqa: F401
                            portions, replay, whole_schedule)

F64 = torch.float64
BF = torch.bfloat16
EPS = 1e-5


def tol_of(dt):
    return 0.04 if dt == BF else 1e-4


def rel(got, want):
    return ((got.detach().cpu().to(F64) - want).abs().max() / want.abs().max()).item()


def w64(w):
    return {k: v.to(F64) for k, v in w.items()}


# ------------------------------------------------------------------------------------ configs
def config_a():
    """Both mixers, sizes that all differ from each other, one layer without a feed-forward, delta
    rule first."""
    return go.make_config([
        go.delta_layer(mlp=go.moe()),
        go.parallel_layer(mlp=None),
        go.delta_layer(heads=6, kv_heads=3, dim=10, vdim=4, conv=4, mlp=go.moe(8, 3, 9, 4, 2, 0.8)),
        go.parallel_layer(heads=3, kv_heads=3, dim=10, vdim=4, rot_dims=8, base=10000.0, scaling=(8.0, 2.0, 4.0, 100), scale=0.7,
                          r_heads=2, r_dim=9, r_vdim=3, decay=(0.999, 0.3), mlp=go.moe(6, 3, 7, 2, 1, 2.5)),
        go.delta_layer(heads=2, kv_heads=1, dim=6, vdim=12, conv=2, mlp=None),
    ])


def config_b():
    """Other sizes, and what the first config keeps apart made equal, 1 or absent: one tap, one
    head, kv heads = heads, dim = vdim, one group, every group kept, every expert chosen, groups of
    one expert, nothing rotated, rotated but not scaled, no token-pair table, no factors, head widths
    beyond one 64-wide tile, more than 16 query heads per kv head, a decay of one and of almost zero."""
    return go.make_config([
        go.parallel_layer(heads=1, kv_heads=1, dim=8, vdim=8, rot_dims=0, scale=1.0, r_heads=1, r_dim=8, r_vdim=8, decay=(1.0,),
                          mlp=go.moe(3, 3, 8, 1, 1, 1.0)),
        go.delta_layer(heads=1, kv_heads=1, dim=8, vdim=8, conv=1, mlp=go.moe(4, 2, 8, 4, 3, 1.0)),
        go.parallel_layer(heads=34, kv_heads=2, dim=4, vdim=4, rot_dims=4, scaling=None, r_heads=2, r_dim=70, r_vdim=33,
                          decay=(1e-4, 0.95), mlp=go.moe(4, 1, 5, 2, 2, 3.0)),
        go.delta_layer(heads=3, kv_heads=3, dim=70, vdim=20, conv=6, mlp=go.moe(1, 1, 5, 1, 1, 1.0)),
        go.parallel_layer(heads=2, kv_heads=1, dim=72, vdim=36, rot_dims=72, scaling=(2.0, 1.0, 1.0, 16), scale=0.2, mlp=None),
    ], width=40, vocab=37, eps=1e-6, scale=1.0, mult=1.0, bigram=None)


def config_c():
    """Only recurrent layers: no KV page at all."""
    return go.make_config([go.delta_layer(heads=3, kv_heads=1, dim=5, vdim=7, conv=5, mlp=go.moe(3, 2, 6, 1, 1)),
                           go.delta_layer(heads=2, kv_heads=2, dim=16, vdim=16, conv=2, mlp=None)], width=16, vocab=29, bigram=(7, 3, 2))


def config_bf16():
    """For 16-bit runs: kernel-friendly widths (grouped expert GEMMs, 16-byte-vector kernels, key
    widths that are a padded width), few routed evaluations."""
    return go.make_config([
        go.delta_layer(heads=4, kv_heads=2, dim=32, vdim=16, conv=4, mlp=go.moe(4, 1, 32, 2, 1, 1.5)),
        go.parallel_layer(heads=4, kv_heads=1, dim=32, vdim=16, rot_dims=16, scale=0.18, r_heads=2, r_dim=16, r_vdim=32,
                          decay=(0.8, 0.98), mlp=go.moe(4, 2, 32, 1, 1, 1.0)),
        go.delta_layer(heads=2, kv_heads=2, dim=128, vdim=16, conv=3, mlp=None),
        go.parallel_layer(heads=4, kv_heads=2, dim=16, vdim=8, rot_dims=16, scaling=None, scale=0.25, r_heads=4, r_dim=8, r_vdim=8,
                          decay=(0.5, 0.7, 0.9, 0.95), mlp=go.moe(2, 1, 64, 1, 1, 2.0)),
    ], width=64, vocab=53)


def prompts(cfg, weights, lengths, seed=1, min_margin=0.0):
    """Random prompts whose routed evaluations all have a clear router margin (a smaller one is a
    coin toss between the oracle and a 16- or 32-bit run)."""
    g = random.Random(seed)
    out = []
    for n in lengths:
        for _ in range(300):
            t = [g.randrange(cfg["vocab"]) for _ in range(n)]
            if min_margin <= 0 or go.router_margin(cfg, weights, t) > min_margin:
                break
        else:
            raise AssertionError("no prompt with the wanted router margin")
        out.append(t)
    return out


def logit_errors(got, want):
    """Per position: rms over the vocabulary of the centred difference / rms of the oracle's
    centred logits over the request."""
    got, want = got.detach().cpu().to(F64), want.to(F64)
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    ref = want - want.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / ref.pow(2).mean().sqrt()


def assert_matches_oracle(eng, cfg, weights, toks, schedule, tol, cache, typical=None):
    got = replay(eng, toks, schedule)
    for rid, t in toks.items():
        key = tuple(t)
        if key not in cache:
            cache[key] = go.forward(cfg, weights, t)
        e = logit_errors(got[rid], cache[key])
        assert e.max().item() < tol, f"request {rid} ({len(t)} tokens): position {int(e.argmax())} differs from " \
                                     f"the oracle by {e.max().item():.3g} (limit {tol})"
        if typical is not None and len(t) > 4:
            assert e.median().item() < typical, f"request {rid}: median error {e.median().item():.3g}"
    return got


def greedy_reference(cfg, weights, prompt, n):
    t, gap = list(prompt), float("inf")
    for _ in range(n):
        lg = go.forward(cfg, weights, t)[-1]
        top = torch.topk(lg, 2).values
        gap = min(gap, float(top[0] - top[1]))
        t.append(int(lg.argmax()))
    return t[len(prompt):], gap


# ------------------------------------------------------------------------------------ one mechanism
def tanh_stream_case(dev, dt, T=7, W=24, seed=5):
    """The stream step in all its uses: norm alone, sum after one output, sum after two joined ones,
    with small, ordinary and saturating arguments of the curves."""
    g = torch.Generator().manual_seed(seed)

    def curve(alpha):
        return (alpha, (1 + 0.3 * torch.randn(W, generator=g)).to(dt), (0.2 * torch.randn(W, generator=g)).to(dt))

    spread = torch.logspace(-3, 1, W)[torch.randperm(W, generator=g)]
    y, y2 = ((torch.randn(T, W, generator=g) * spread).to(dt) for _ in range(2))
    x0 = torch.randn(T, W, generator=g) * spread
    jw = ((1 + 0.3 * torch.randn(W, generator=g)).to(dt), torch.randn(W, generator=g).to(dt))
    pre, post, mult = curve(0.8), curve(1.7), 0.37
    D = lambda v, c: torch.tanh(c[0] * v) * c[1].to(F64) + c[2].to(F64)   # noqa: E731
    to = lambda c: (c[0], c[1].to(dev), c[2].to(dev))   # noqa: E731
    tol = 0.01 if dt == BF else 1e-5
    x = x0.clone().to(dev)
    h = ops.tanh_stream(x, to(pre), dt)
    assert torch.equal(x.cpu(), x0) and h.dtype == dt and rel(h, D(x0.to(F64), pre)) < tol
    h = ops.tanh_stream(x, to(pre), dt, post=to(post), mult=mult, y=y.to(dev))
    x1 = x0.to(F64) + mult * D(y.to(F64), post)
    assert rel(x, x1) < 1e-6 and rel(h, D(x1, pre)) < tol
    joined = 0.5 * (go.rms_unit(y.to(F64), EPS) * jw[0].to(F64) + go.rms_unit(y2.to(F64), EPS) * jw[1].to(F64))
    h = ops.tanh_stream(x, to(pre), dt, post=to(post), mult=mult, y=y.to(dev), y2=y2.to(dev), join=(jw[0].to(dev), jw[1].to(dev), EPS))
    x2 = x1 + mult * D(joined, post)
    assert rel(x, x2) < 2e-6 and rel(h, D(x2, pre)) < tol
    # small arguments keep their relative accuracy
    tiny = (torch.randn(T, W, generator=g) * 1e-4).to(dev)
    zero = torch.zeros(W, dtype=dt, device=dev)
    h = ops.tanh_stream(tiny, (1.0, torch.ones(W, dtype=dt, device=dev), zero), dt)
    assert ((h.float().cpu() - tiny.cpu()).abs() <= tiny.cpu().abs() * (2 ** -8 if dt == BF else 1e-6)).all()


def _steps(step_lens, dev):
    """Several steps over some sequences (rows per sequence and step; 0 = not in the step): per step
    (live sequences, rows before the step, rows, cu, reset)."""
    done = [0] * len(step_lens[0])
    for lens in step_lens:
        live = [s for s, n in enumerate(lens) if n > 0]
        cu = torch.tensor([0] + list(torch.tensor([lens[s] for s in live]).cumsum(0)), dtype=torch.int32, device=dev)
        reset = torch.tensor([int(done[s] == 0) for s in live], dtype=torch.int32, device=dev)
        yield live, list(done), lens, cu, reset
        done = [a + b for a, b in zip(done, lens)]


def _run_steps(step_lens, rows, slots, dev, fn):
    """``fn(x, seqs, single)`` over every step; rows: per sequence a tensor, returns the outputs per sequence."""
    got = [[] for _ in slots]
    for live, done, lens, cu, reset in _steps(step_lens, dev):
        x = torch.cat([rows[s][done[s]:done[s] + lens[s]] for s in live]).to(dev)
        slot = torch.tensor([slots[s] for s in live], dtype=torch.int32, device=dev)
        o = fn(x, (cu, slot, reset), max(lens) == 1)
        a = 0
        for s in live:
            got[s].append(o[a:a + lens[s]].cpu())
            a += lens[s]
    return [torch.cat(o) for o in got]


STEPS = ([5, 0, 17], [1, 1, 1], [1, 0, 1], [4, 36, 1], [2, 1, 16])


def delta_case(dev, dt, H=4, Hk=2, dk=8, dv=6, K=3, steps=STEPS, rate=0.3, bias_spread=1.0, seed=5, memory=None):
    """The delta rule's op over three sequences in several steps (one that starts late on a dirty
    slot, portions shorter than the taps, single rows on the one-launch path), against the oracle.
    ``rate``: size of exp(A_log) (30: a state that forgets within a token).  ``memory`` = (row written,
    row read) of sequence 0: nothing decays, hardly anything else is written and the reader's query is
    the writer's key, so its output is that one value."""
    g = torch.Generator().manual_seed(seed)
    n = [sum(s[i] for s in steps) for i in range(3)]
    C, off = 2 * Hk * dk + H * dv, 8
    zw = H * (dk + dv)
    rows = [torch.randn(k, off + C + zw + H, generator=g) for k in n]
    cw = torch.randn(C, K, generator=g) * 0.6
    A_log = torch.log(rate * (0.2 + torch.rand(H, generator=g)))
    dtb = torch.randn(H * dk, generator=g) * bias_spread
    nw = (1 + 0.3 * torch.randn(dv, generator=g)).to(dt)
    if memory is not None:
        wr, rd = memory
        A_log, cw = torch.full((H,), -20.0), torch.zeros(C, K)
        cw[:, -1] = 1.0
        rows[0][:, off + C + zw:] = -7.0
        rows[0][wr, off + C + zw:] = 6.0
        rows[0][rd, off:off + Hk * dk] = rows[0][wr, off + Hk * dk:off + 2 * Hk * dk]
    rows, cw = [r.to(dt) for r in rows], cw.to(dt)

    def oracle(q):
        T = q.shape[0]
        u = go.silu(go.causal_conv(q[:, off:off + C].to(F64), cw.to(F64)))
        qq = go.unit_vector(u[:, :Hk * dk].view(T, Hk, dk)).repeat_interleave(H // Hk, 1) * dk ** -0.5
        kk = go.unit_vector(u[:, Hk * dk:2 * Hk * dk].view(T, Hk, dk)).repeat_interleave(H // Hk, 1)
        z = q[:, off + C:off + C + zw].to(F64)
        dec = torch.exp(-torch.exp(A_log.to(F64))[:, None] * go.softplus(z[:, :H * dk] + dtb.to(F64)).view(T, H, dk))
        o, S = go.delta_core(qq, kk, u[:, 2 * Hk * dk:].view(T, H, dv), dec, go.sigmoid(q[:, off + C + zw:].to(F64)))
        y = go.rms_unit(o, EPS) * nw.to(F64) * go.sigmoid(z[:, H * dk:]).view(T, H, dv)
        return y.reshape(T, H * dv), S

    want = [oracle(r) for r in rows]
    state = torch.full((6, H, dv, dk), 3.0, dtype=torch.float32, device=dev)
    tail = torch.full((6, C, K - 1), 3.0, dtype=dt, device=dev)
    slots = [4, 2, 1]
    d = lambda t: t.to(dev)   # noqa: E731

    def fn(x, seqs, single):
        return ops.channel_delta(x[:, off:off + C], d(cw), tail, x[:, off + C:off + C + zw].contiguous(), x[:, off + C + zw:], d(A_log),
                                 d(dtb), d(nw), EPS, state, seqs, Hk, single_rows=single)

    got = _run_steps(steps, rows, slots, dev, fn)
    for s in range(3):
        assert rel(got[s], want[s][0]) < (0.03 if dt == BF else 2e-4), (s, rel(got[s], want[s][0]))
        assert rel(state[slots[s]].transpose(1, 2), want[s][1]) < (0.01 if dt == BF else 2e-5), s
        if K > 1 and n[s] >= K - 1:
            assert torch.equal(tail[slots[s]].cpu(), rows[s][n[s] - K + 1:, off:off + C].T)
    assert float(state[0].min()) == float(state[5].max()) == 3.0            # other slots are untouched
    if memory is not None:      # with another value written there the reader answers something else
        rows[0] = rows[0].clone()
        rows[0][wr, off + 2 * Hk * dk:off + C] = -rows[0][wr, off + 2 * Hk * dk:off + C]
        assert (oracle(rows[0])[0][rd] - want[0][0][rd]).abs().max() > 0.5 * want[0][0][rd].abs().max()


def lightning_case(dev, dt, H=3, dk=5, dv=7, decay=(0.5, 0.9, 0.99), steps=STEPS, seed=5, memory=None):
    """Lightning attention's op as in :func:`delta_case`.  ``memory`` = (row written, row read): the
    written row's key and value are large and the decay is one."""
    g = torch.Generator().manual_seed(seed)
    n = [sum(s[i] for s in steps) for i in range(3)]
    off, w = 3, H * (2 * dk + dv)
    rows = [torch.randn(k, off + w, generator=g) for k in n]
    dec = torch.tensor((list(decay) * H)[:H])
    if memory is not None:
        wr, rd = memory
        dec = torch.ones(H)
        for r in rows:
            r[:, off:] -= 2.0
        rows[0][wr, off:] = 12.0 * torch.rand(w, generator=g)
        rows[0][rd, off:off + H * dk] = 3.0
    rows = [r.to(dt) for r in rows]

    def oracle(q):
        T = q.shape[0]
        u = go.silu(q[:, off:].to(F64))
        o, S = go.lightning_core(u[:, :H * dk].view(T, H, dk), u[:, H * dk:2 * H * dk].view(T, H, dk), u[:, 2 * H * dk:].view(T, H, dv),
                                 dec.to(F64))
        return o.reshape(T, H * dv), S

    want = [oracle(r) for r in rows]
    state = torch.full((6, H, dv, dk), 3.0, dtype=torch.float32, device=dev)
    slots = [4, 2, 1]

    def fn(x, seqs, single):
        return ops.lightning_scan(x[:, off:off + H * dk], x[:, off + H * dk:off + 2 * H * dk], x[:, off + 2 * H * dk:], dec.to(dev), state,
                                  seqs, single_rows=single)

    got = _run_steps(steps, rows, slots, dev, fn)
    for s in range(3):
        assert rel(got[s], want[s][0]) < (0.01 if dt == BF else 2e-5), (s, rel(got[s], want[s][0]))
        assert rel(state[slots[s]].transpose(1, 2), want[s][1]) < (1e-4 if dt == BF else 2e-5), s
    assert float(state[0].min()) == float(state[5].max()) == 3.0
    if memory is not None:
        rows[0] = rows[0].clone()
        rows[0][wr, off + 2 * H * dk:] = 1.0
        assert (oracle(rows[0])[0][rd] - want[0][0][rd]).abs().max() > 0.3 * want[0][0][rd].abs().max()


def sigmoid_gate_norm_case(dev, dt, T=5, I=21, group=21, seed=4):
    """Norm over groups of channels times a weight shared by the groups times sigmoid(gate)."""
    g = torch.Generator().manual_seed(seed)
    y, z = torch.randn(T, I, generator=g).to(dt), torch.randn(T, I + 8, generator=g).to(dt)
    w = (1 + 0.3 * torch.randn(group, generator=g)).to(dt)
    got = ops.gated_rmsnorm(y.to(dev), z.to(dev)[:, 8:], w.to(dev), group, EPS, norm_first=True, exact=True, gate="sigmoid")
    want = go.rms_unit(y.to(F64).view(T, I // group, group), EPS) * w.to(F64)
    assert rel(got, want.reshape(T, I) * go.sigmoid(z[:, 8:].to(F64))) < (0.01 if dt == BF else 1e-5)


def rope_table_case():
    """The scaled table against the oracle's angles: pairs of short wavelength untouched, of long one
    slowed by the factor, the ones between blended; every band occurs."""
    from ome_amd.models.config import plain_rope_table

    rot = {"base": 10000.0, "dims": 16, "scaling": {"factor": 8.0, "low": 1.5, "high": 4.0, "original": 200}}
    f, f0 = go.frequencies(rot), go.frequencies(dict(rot, scaling=None))
    ratio = f / f0
    assert float(ratio[0]) == 1.0 and abs(float(ratio[-1]) - 1 / 8) < 1e-12 and ((ratio > 0.13) & (ratio < 0.99)).any()
    cs = plain_rope_table(10000.0, 16, 500, None, rot["scaling"])
    a = torch.arange(500, dtype=F64)[:, None] * f
    assert (cs.to(F64) - torch.cat([a.cos(), a.sin()], -1)).abs().max() < 1e-6


def group_route_case(dev):
    """A group is chosen by the SUM of its two best scores (not by its best), experts of the other
    groups never, however high; the weights are the plain scores over their sum."""
    logit = lambda p: torch.log(p / (1 - p))   # noqa: E731
    s = torch.tensor([[0.9, 0.1, 0.6, 0.6, 0.3, 0.2], [0.5, 0.5, 0.1, 0.95, 0.7, 0.2]], dtype=F64)
    w, ids = ops.moe_route(logit(s).float().to(dev), 2, True, "sigmoid", n_group=3, topk_group=1, group_mode=4)
    assert sorted(ids[0].tolist()) == [2, 3] and sorted(ids[1].tolist()) == [2, 3]
    assert abs(float(w[0, 0]) - 0.5) < 1e-6
    top = {int(i): float(x) for i, x in zip(ids[1], w[1])}
    assert abs(top[3] - 0.95 / 1.05) < 1e-6 and abs(top[2] - 0.1 / 1.05) < 1e-6
    g = torch.Generator().manual_seed(2)
    for E, k, n, keep in ((16, 3, 4, 2), (12, 2, 12, 5), (64, 8, 8, 4), (6, 6, 2, 2), (8, 2, 2, 1)):
        lg = torch.randn(33, E, generator=g)
        chosen, _ = go.choose(go.sigmoid(lg.to(F64)), {"groups": {"count": n, "keep": keep}, "top": k})
        ids = ops.moe_route(lg.to(dev), k, True, "sigmoid", n_group=n, topk_group=keep, group_mode=4)[1].cpu().long()
        assert torch.equal(torch.zeros(33, E, dtype=torch.bool).scatter_(1, ids, True), chosen), (E, k, n, keep)


def moe_block(f, width, dev, dt):
    r = f["router"]
    return GroupRoutedMoE(width, r["experts"], r["top"], f["expert"]["ff"], 0.0, r["groups"]["count"], r["groups"]["keep"], 0, 0.0, dev,
                          dt, act=0, renorm=True, correction=False, scoring="sigmoid", group_score="top2", routed_scale=r["scale"])


def moe_case(dev, dt, f, width, rows=13):
    """The routed feed-forward alone, on inputs whose router decisions are clear of ties."""
    cfg = go.make_config([go.delta_layer(mlp=f)], width=width)
    w = go.sub(go.make_weights(cfg, 9), "l0.mlp.")
    for seed in range(7, 600):
        h = torch.randn(rows, width, generator=torch.Generator().manual_seed(seed))
        hq = h.to(dt).to(F64)
        if go.choose(go.sigmoid(hq @ w["router"].to(F64).T), f["router"])[1] > (5e-3 if dt == BF else 1e-4):
            break
    else:
        raise AssertionError("no input with the wanted router margin")
    blk = moe_block(f, width, dev, dt)
    blk.load(w)
    hd = h.to(device=dev, dtype=dt)
    assert rel(blk.forward(hd), go.moe_ff(hq, w64(w), f)) < tol_of(dt)
    return blk.grouped_ok(hd)


# ------------------------------------------------------------------------------------ mixers alone
class Joined:
    """A parallel block whose two outputs stand side by side."""

    def __init__(self, blk):
        self.blk = blk
        self.alloc_state = blk.alloc_state

    def forward(self, h, ctx):
        return torch.cat(self.blk.forward(h, ctx), -1)


def block_of(layer, width, dev, dt, max_pos=1024, pages=80):
    """The framework's block of a layer entry, with a one-layer paged cache of its shape."""
    m = layer["mixer"]
    if layer["type"] == "channel_delta":
        return ChannelDeltaMixer(width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], EPS, dev, dt), None
    a, r = m["left"], m["right"]
    rot = a.get("rot") or {}
    left = GatedWindowAttention(0, width, a["heads"], a["kv_heads"], a["dim"], a["vdim"], -1, 0, rot.get("base", 1.0),
                                rot.get("dims", 0), a["scale"], EPS, max_pos, dev, dt, interleaved=False, wide_norm=False, gated=False,
                                rot_scaling=rot.get("scaling"), sink=0.0)
    right = LightningAttention(width, r["heads"], r["dim"], r["vdim"], r["decay"], EPS, dev, dt)
    return ParallelMixers(left, right, dev, dt), PagedKVCache(1, pages, a["kv_heads"], left.D, 16, dt, dev)


def load_block(blk, w):
    if isinstance(blk, ParallelMixers):
        blk.load(go.sub(w, "left."), go.sub(w, "right."))
        return Joined(blk)
    blk.load(w)
    return blk


def oracle_mixer(layer, h, w):
    m = layer["mixer"]
    if layer["type"] == "channel_delta":
        return go.channel_delta(h, w, m, EPS)
    return torch.cat([go.attention(h, go.sub(w, "left."), m["left"]), go.lightning_attention(h, go.sub(w, "right."), m["right"], EPS)], -1)


def run_chunks(block, h, cuts, kv=None, page=16):
    """One sequence through ``block`` in portions ``cuts`` (state slot 1, a scattered page table); a
    portion of one row runs as a decode step."""
    T = h.shape[0]
    dev = h.device
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)   # noqa: E731
    table = i32([[7 + 2 * i for i in range(-(-T // page))]])
    block.alloc_state(3)
    outs, a = [], 0
    for n in cuts:
        pos = torch.arange(a, a + n, dtype=torch.int32, device=dev)
        slots = (table[0, (pos // page).long()] * page + pos % page).to(torch.int32)
        if n == 1:
            meta = AttnMeta("decode", pos, slots, table, seq_lens=i32([a + 1]))
        else:
            meta = AttnMeta("prefill", pos, slots, table, cu_q=i32([0, n]), kv_lens=i32([a + n]),
                            items=i32([[0, r] for r in range(0, n, 32)]))
        outs.append(block.forward(h[a:a + n].contiguous(), MixerCtx(meta, kv, (i32([0, n]), i32([1]), i32([int(a == 0)])))))
        a += n
    return torch.cat(outs)


def mixer_alone(dev, dt, layer, width=24, T=45, cut_sets=None, seed=3):
    """One mixer over one sequence, whole and in portions, against the oracle."""
    cfg = go.make_config([layer], width=width, eps=EPS)
    w = go.sub(go.make_weights(cfg, seed), "l0.mix.")
    h = torch.randn(T, width, generator=torch.Generator().manual_seed(seed))
    want = oracle_mixer(layer, h.to(dt).to(F64), w64(w))
    for cuts in cut_sets or ([T], [T - 5] + [1] * 5, portions(T, [2, 3, 17, 16, 1, 6]), [1] * T):
        blk, kv = block_of(layer, width, dev, dt)
        got = run_chunks(load_block(blk, w), h.to(device=dev, dtype=dt), cuts, kv)
        for part in ((slice(0, width), slice(width, 2 * width)) if layer["type"] == "parallel" else (slice(0, width),)):
            assert rel(got[:, part], want[:, part]) < tol_of(dt), (cuts, rel(got[:, part], want[:, part]))


# ------------------------------------------------------------------------------------ planted keys
def planted_layer():
    """A parallel layer whose keys are made by the NEGATED query weights, with a sharp scale and
    nothing rotated: a row that is the negated input of another one owns that one's softmax, and the
    row itself scores lowest."""
    L = go.parallel_layer(heads=2, kv_heads=2, dim=16, vdim=12, rot_dims=0, scale=1.2)
    w = go.sub(go.make_weights(go.make_config([L], width=24), 6), "l0.mix.")
    w["left.k"] = -w["left.q"]
    return L, w


def planted_case(dev, dt, T, i, j, cuts, moved=0.08):
    """Row j is the planted key of row i; with the key's row replaced the oracle's answer must be
    another one, so the case would notice a key that is not seen."""
    L, w = planted_layer()
    h = torch.randn(T, 24, generator=torch.Generator().manual_seed(4))
    h[j] = -h[i]
    hq = h.to(dt).to(F64)
    left = L["mixer"]["left"]
    lw = w64(go.sub(w, "left."))
    want = go.attention(hq, lw, left)
    blk, kv = block_of(L, 24, dev, dt, pages=2 * (T // 16) + 12)
    got = run_chunks(load_block(blk, w), h.to(device=dev, dtype=dt), cuts, kv)[:, :24]
    assert rel(got[i:i + 1], want[i:i + 1]) < tol_of(dt), rel(got[i:i + 1], want[i:i + 1])
    h2 = hq.clone()
    h2[j] = hq[j - 1 if j else 1]
    assert (go.attention(h2, lw, left)[i] - want[i]).abs().max() > moved * want[i].abs().max()


def plus_one_case(dev, dt):
    """Scores all near zero: the one in the denominator takes half of the first token's weight, a
    third of the second's, ...; and scores far below zero: next to nothing is left."""
    for scale, far in ((1e-4, False), (6.0, True)):
        L = go.parallel_layer(heads=1, kv_heads=1, dim=8, vdim=8, rot_dims=0, scale=scale)
        w = go.sub(go.make_weights(go.make_config([L], width=24), 6), "l0.mix.")
        w["left.k"] = -w["left.q"].clone()
        h = torch.randn(1, 24, generator=torch.Generator().manual_seed(4)).expand(20, 24) * torch.linspace(0.9, 1.1, 20)[:, None]
        hq = h.to(dt).to(F64)
        lw, m = w64(go.sub(w, "left.")), L["mixer"]["left"]
        want = go.attention(hq, lw, m)
        v = (hq @ lw["v"].T) @ lw["o"].T     # the first token's output if nothing were added: its own value
        assert want.abs().max() < 1e-6 * v.abs().max() if far else (want[0] - 0.5 * v[0]).abs().max() < 1e-3 * v.abs().max()
        for cuts in ([20], [1] * 20, [2, 3, 1, 14]):
            blk, kv = block_of(L, 24, dev, dt)
            got = run_chunks(load_block(blk, w), h.to(device=dev, dtype=dt).contiguous(), cuts, kv)[:, :24]
            if far:
                assert float(got.abs().max()) < 1e-5 * float(v.abs().max())
            else:
                assert rel(got, want) < tol_of(dt)


def planted_model(vocab=60):
    """A one-layer model on planted weights; token 1 embeds as the negated token 0 (no token-pair
    rows, a norm that is odd), so the two are each other's planted keys."""
    L, mw = planted_layer()
    cfg = go.make_config([L], width=24, vocab=vocab, bigram=None)
    w = go.make_weights(cfg, 6)
    for k, v in mw.items():
        w["l0.mix." + k] = v
    w["l0.norm1.b"] = torch.zeros_like(w["l0.norm1.b"])
    w["embed"][1] = -w["embed"][0]
    return cfg, w


def planted_engine_case(dev, dtype, schedules, tmp, tol, length=75, vocab=60):
    """Token 0 (the query) at the end and in the middle, token 1 (its key) once, at the first token,
    at a page's last and first row, in the middle."""
    cfg, w = planted_model(vocab)
    path = go.write_model(str(tmp), cfg, w)
    g = random.Random(3)
    toks, want = {}, {}
    for at in (0, 15, 16, 31, 40):
        t = [g.randrange(2, vocab) for _ in range(length)]
        t[at] = 1
        t[50] = t[length - 1] = 0
        toks[f"k{at}"] = t
        want[f"k{at}"] = go.forward(cfg, w, t)
        t2 = list(t)
        t2[at] = 2 if t[at - 1] != 2 else 3
        e = logit_errors(go.forward(cfg, w, t2), want[f"k{at}"])
        assert e[50] > 0.03 and e[length - 1] > 0.03
    for sched in schedules(toks):
        eng = make_engine(path, dev, dtype, max_tokens=4 * 16 * (-(-length // 16)))
        got = replay(eng, toks, sched)
        for k in toks:
            e = logit_errors(got[k], want[k])
            assert e.max().item() < tol, (k, int(e.argmax()), e.max().item())


def constants_matter_case():
    """Oracle sanity: every constant and every small tensor moves the result by an amount of its own
    size (or, where it must not, not at all)."""
    cfg = config_a()
    wt = go.make_weights(cfg, 2)
    t = [3, 9, 1, 30, 7, 12, 2, 2, 19, 5]
    a = go.forward(cfg, wt, t)

    def moved(cfg2=cfg, **kw):
        return float((go.forward(cfg2, dict(wt, **kw), t) - a).abs().max())

    def layer(i, **kw):
        L = dict(cfg["layers"][i])
        L["mixer"] = dict(L["mixer"], **kw)
        return dict(cfg, layers=cfg["layers"][:i] + [L] + cfg["layers"][i + 1:])

    left, right = cfg["layers"][3]["mixer"]["left"], cfg["layers"][3]["mixer"]["right"]
    assert moved(dict(cfg, residual_mult=0.5)) > 0.02
    assert moved(dict(cfg, embedding=dict(cfg["embedding"], scale=2.0))) > 0.02
    assert moved(dict(cfg, embedding=dict(cfg["embedding"], bigram={"buckets": 29, "mul_prev": 12, "mul_cur": 5}))) > 0.02
    assert moved(layer(3, left=dict(left, rot={"base": 10000.0, "dims": 8}))) > 1e-4
    assert moved(layer(3, left=dict(left, scale=0.2))) > 0.005
    assert moved(layer(3, right=dict(right, decay=[0.9, 0.3]))) > 0.005
    for name in ("l0.norm1.alpha", "l0.norm1b.b", "l2.norm2b.alpha", "l2.norm2.b", "final.norm.b", "l0.mix.dt_bias", "l0.mix.A_log",
                 "l2.mix.a1", "l2.mix.g1", "l2.mix.b", "l0.mix.norm", "l1.mix.right.norm", "l1.mix.left.out", "l1.mix.right.out",
                 "l1.mix.right.g"):
        assert moved(**{name: torch.zeros_like(wt[name])}) > 0.005, name
