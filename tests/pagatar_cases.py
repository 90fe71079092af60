"""Scenarios shared by the CPU (fp32 reference ops) and GPU (HIP kernels) Pagatar tests: every
mechanism alone against the slow oracle of ``pagatar_oracle``, small random models run through the
engine's replay entry under different schedules, planted keys at chunk edges, far back and at page
borders.  The schedule builders are the ones of ``zavilorn_cases`` (they know nothing of a design).
Every function takes the device and element type, so the two test files only bind them."""
from __future__ import annotations

import random

import torch

import pagatar_oracle as po
from ome_amd import ops
from ome_amd.models.common import PagedKVCache
from ome_amd.models.mixers import ConvRotaryAttention, GroupRoutedMoE, LatentAttention, MinGruMixer
from zavilorn_cases import (chunked_schedule, decode_schedule, greedy_engine, make_engine, mixed_schedule,  # noqa: F401
                            portions, replay, run_chunks, whole_schedule)

F64 = torch.float64
BF = torch.bfloat16
EPS = 1e-5
YARN = (4.0, 64, 8.0, 1.0)       # (factor, original, fast, slow)


def tol_of(dt):
    return 0.04 if dt == BF else 1e-4


def rel(got, want):
    return ((got.detach().cpu().to(F64) - want).abs().max() / want.abs().max()).item()


def w64(w):
    return {k: v.to(F64) for k, v in w.items()}


# ------------------------------------------------------------------------------------ configs
def config_a():
    """All three mixers, sizes that all differ from each other, value mixing across a layer that
    does not mix, one layer without a feed-forward, latent attention first."""
    return po.make_config([
        po.latent_layer(mlp=po.moe(5, 2, 12)),
        po.attn_layer(v_mix=True, scaling=YARN, mlp=None),
        po.gru_layer(mlp=po.moe(6, 3, 9)),
        po.attn_layer(heads=3, kv_heads=3, dim=10, vdim=4, chunk=11, conv=4, rot_dims=10, base=33.0, scale=0.4,
                      mlp=po.moe(4, 1, 7)),
        po.attn_layer(heads=6, kv_heads=2, dim=12, vdim=6, chunk=9, conv=2, rot_dims=8, v_mix=True, mlp=po.moe(4, 2, 8)),
        po.attn_layer(heads=2, kv_heads=1, dim=6, vdim=12, chunk=16, conv=5, rot_dims=2, v_mix=True, scaling=(2.0, 32, 4.0, 1.0),
                      mlp=None),
    ])


def config_b():
    """Other sizes, and what the first config keeps apart made equal, 1 or absent: one norm group,
    one tap, one head, kv heads = heads, dim = vdim, chunks longer than every prompt or of one
    token, every expert chosen, nothing rotated, head widths beyond one 64-wide tile, a latent wider
    than the heads, a rotated part wider than the unrotated one, no value mixing at all."""
    return po.make_config([
        po.gru_layer(inner=1, mlp=po.moe(2, 2, 8)),
        po.attn_layer(heads=1, kv_heads=1, dim=8, vdim=8, chunk=1000, conv=1, rot_dims=8, base=7.0, scale=1.0, mlp=po.moe(3, 1, 16)),
        po.latent_layer(heads=1, dim=4, rot_dim=8, vdim=8, kv_rank=8, q_rank=8, scale=1.0, mlp=po.moe(1, 1, 5)),
        po.attn_layer(heads=2, kv_heads=2, dim=72, vdim=36, chunk=1, conv=6, rot_dims=0, scale=0.3, mlp=po.moe(4, 4, 5)),
        po.latent_layer(heads=18, dim=4, rot_dim=2, vdim=3, kv_rank=70, q_rank=3, scale=0.7, mlp=None),
        po.attn_layer(heads=34, kv_heads=2, dim=4, vdim=4, chunk=12, conv=7, rot_dims=2, mlp=None),
    ], width=40, vocab=37, eps=1e-6, groups=1)


def config_c():
    """Only recurrent layers: no KV page at all; as many norm groups as channels."""
    return po.make_config([po.gru_layer(inner=33, mlp=po.moe(3, 2, 6)), po.gru_layer(inner=16, mlp=None)], width=16, vocab=29,
                          groups=16)


def config_bf16():
    """For 16-bit runs: kernel-friendly widths (grouped expert GEMMs, the 16-byte-vector kernels,
    the latent kernel's row shapes), few routed evaluations."""
    return po.make_config([
        po.attn_layer(heads=4, kv_heads=1, dim=32, vdim=16, chunk=24, conv=4, rot_dims=16, scale=0.18, v_mix=True, scaling=YARN,
                      mlp=po.moe(4, 1, 32)),
        po.gru_layer(inner=96, mlp=po.moe(4, 2, 32)),
        po.latent_layer(heads=4, dim=16, rot_dim=8, vdim=16, kv_rank=48, q_rank=24, scale=0.2, mlp=None),
        po.attn_layer(heads=4, kv_heads=2, dim=16, vdim=8, chunk=40, conv=2, rot_dims=16, scale=0.25, v_mix=True, mlp=po.moe(2, 1, 64)),
    ], width=64, vocab=53, groups=2)


def prompts(cfg, weights, lengths, seed=1, min_margin=0.0):
    """Random prompts whose routed evaluations all have a clear router margin (a smaller one is a
    coin toss between the oracle and a 16- or 32-bit run)."""
    g = random.Random(seed)
    out = []
    for n in lengths:
        for _ in range(300):
            t = [g.randrange(cfg["vocab"]) for _ in range(n)]
            if min_margin <= 0 or po.router_margin(cfg, weights, t) > min_margin:
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
            cache[key] = po.forward(cfg, weights, t)
        e = logit_errors(got[rid], cache[key])
        assert e.max().item() < tol, f"request {rid} ({len(t)} tokens): position {int(e.argmax())} differs from " \
                                     f"the oracle by {e.max().item():.3g} (limit {tol})"
        if typical is not None and len(t) > 4:
            assert e.median().item() < typical, f"request {rid}: median error {e.median().item():.3g}"
    return got


def greedy_reference(cfg, weights, prompt, n):
    t, gap = list(prompt), float("inf")
    for _ in range(n):
        lg = po.forward(cfg, weights, t)[-1]
        top = torch.topk(lg, 2).values
        gap = min(gap, float(top[0] - top[1]))
        t.append(int(lg.argmax()))
    return t[len(prompt):], gap


# ------------------------------------------------------------------------------------ one mechanism
def block_of(layer, width, dev, dt, max_pos=1024, pages=80):
    """The framework's block of a layer entry, with a one-layer paged cache of its shape."""
    m, kind = layer["mixer"], layer["type"]
    rot = m.get("rot") or {}
    if kind == "attention":
        blk = ConvRotaryAttention(0, width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["mask"]["size"], m["conv"],
                                  rot.get("base", 1.0), rot.get("dims", 0), m["scale"], EPS, max_pos, dev, dt,
                                  interleaved=False, unit_norm=False, rot_scaling=rot.get("scaling"), chunked=True, bias=True,
                                  head_norm=True, sink=False, gated=True)
        return blk, PagedKVCache(1, pages, m["kv_heads"], blk.D, 16, dt, dev)
    if kind == "mingru":
        return MinGruMixer(width, m["width"], dev, dt), None
    blk = LatentAttention(0, 0, width, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"],
                          rot.get("base", 1.0), None, m["scale"], EPS, max_pos, dev, dt, None, sink=False, gated="head",
                          interleaved=True)
    return blk, PagedKVCache(1, pages, 1, blk.D, 16, dt, dev, v_dim=0 if blk.latent_cache else None)


def oracle_mixer(layer, h, w):
    m = layer["mixer"]
    if layer["type"] == "attention":
        return po.attention(h, w, m, EPS)
    if layer["type"] == "mingru":
        return po.mingru(h, w)
    return po.latent_attention(h, w, m, EPS)


def mixer_alone(dev, dt, layer, width=24, T=45, cut_sets=None, seed=3):
    """One mixer over one sequence, whole and in portions, against the oracle."""
    cfg = po.make_config([layer], width=width, eps=EPS, groups=1)
    w = po.sub(po.make_weights(cfg, seed), "l0.mix.")
    h = torch.randn(T, width, generator=torch.Generator().manual_seed(seed))
    want = oracle_mixer(layer, h.to(dt).to(F64), w64(w))
    for cuts in cut_sets or ([T], [T - 5] + [1] * 5, portions(T, [2, 3, 17, 16, 1, 6])):
        blk, kv = block_of(layer, width, dev, dt)
        blk.load(w)
        got = run_chunks(blk, h.to(device=dev, dtype=dt), cuts, kv)
        assert rel(got, want) < tol_of(dt), (cuts, rel(got, want))


def stream_case(dev, dt, T=7, W=24, groups=3, n=4, seed=5):
    """The stream step in all its uses: gathered embedding, sum after a mixer, layer result into
    the history + average over depth, final norm; out-of-place and through the history."""
    g = torch.Generator().manual_seed(seed)
    w = (1.0 + 0.3 * torch.randn(W, generator=g)).to(dt)
    y = (torch.randn(T, W, generator=g) * torch.linspace(0.2, 4.0, W)).to(dt)       # groups of unlike size
    table = torch.randn(11, W, generator=g).to(dt)
    ids = torch.randint(0, 11, (T,), generator=g).to(torch.int32)
    res = torch.randn(T, W, generator=g)
    coef = torch.randn(n + 1, generator=g)
    old = torch.randn(n + 2, T, W, generator=g)
    tol = 0.01 if dt == BF else 1e-5
    d = lambda t: t.to(dev)   # noqa: E731
    N = lambda t: po.group_norm(t.to(F64), w.to(F64), groups, EPS)   # noqa: E731
    hist = d(old.clone())
    out = ops.stream_step(d(table), d(w), groups, EPS, ids=d(ids), hist=hist, k=0, out_dtype=dt)
    x0 = N(table[ids.long()])
    assert rel(hist[0], x0) < 1e-5 and rel(out, x0) < tol and rel(hist[1:], old[1:].to(F64)) < 1e-12
    hist = d(old.clone())       # after a mixer: the sum goes to the history entry of the layer's result
    out = ops.stream_step(d(y), d(w), groups, EPS, res=d(res), x_out=hist[n], out_dtype=dt)
    x1 = res.to(F64) + N(y)
    assert rel(hist[n], x1) < 1e-5 and rel(out, x1) < tol
    x = torch.full((T, W), 7.0, device=dev)
    cur = hist[n]               # the layer's result over it, and the average
    out = ops.stream_step(d(y), d(w), groups, EPS, res=cur, hist=hist, k=n, coef=d(coef), x_out=x, out_dtype=dt)
    X = x1 + N(y)
    want = po.depth_average(coef.to(F64), [old[j].to(F64) for j in range(n)] + [X])
    assert rel(hist[n], X) < 1e-5 and rel(x, want) < 1e-5 and rel(out, want) < tol
    assert rel(hist[:n], old[:n].to(F64)) < 1e-12 and rel(hist[n + 1], old[n + 1].to(F64)) < 1e-12
    assert ops.stream_step(d(y), d(w), groups, EPS, res=d(res), x_out=x) is None and rel(x, res.to(F64) + N(y)) < 1e-5
    fin = ops.stream_step(x, d(w), groups, EPS, out_dtype=dt)
    assert fin.dtype == dt and rel(fin, N(res.to(F64) + N(y))) < tol
    # the groups matter
    if groups > 1 and W > groups:
        assert (po.group_norm(y.to(F64), w.to(F64), 1, EPS) - N(y)).abs().max() > 0.1


def _batches(lens_a, lens_b, dev):
    """Two steps over three sequences (rows per sequence and step; 0 = not in the step): per step
    (live sequences, row offsets, rows, cu, reset)."""
    for step, lens in enumerate((lens_a, lens_b)):
        off = [0, 0, 0] if step == 0 else lens_a
        live = [s for s in range(3) if lens[s] > 0]
        cu = torch.tensor([0] + list(torch.tensor([lens[s] for s in live]).cumsum(0)), dtype=torch.int32, device=dev)
        reset = torch.tensor([int(off[s] == 0) for s in live], dtype=torch.int32, device=dev)
        yield live, off, lens, cu, reset


def mingru_case(dev, dt, width=20, lens_a=(5, 0, 3), lens_b=(4, 6, 1), bias=-1.0, seed=5):
    """The scan over a batch of three sequences in two steps: one that continues, one that starts
    on a dirty slot, row counts around the kernel's chunk lengths; a slow gate keeps the first
    token's write visible at the end."""
    g = torch.Generator().manual_seed(seed)
    lens_a, lens_b = list(lens_a), list(lens_b)
    n = [a + b for a, b in zip(lens_a, lens_b)]
    p = [torch.randn(k, 3 * width + 5, generator=g).to(dt) for k in n]
    zb, xb = (bias + torch.rand(width, generator=g)).to(dt), torch.randn(width, generator=g).to(dt)

    def oracle(q):
        z = po.sigmoid(q[:, :width] + zb.to(F64))
        c = po.mingru_candidate(q[:, width:2 * width] + xb.to(F64))
        S, out = torch.zeros(width, dtype=F64), []
        for t in range(q.shape[0]):
            S = (1 - z[t]) * S + z[t] * c[t]
            out.append(S * po.silu(q[t, 2 * width:3 * width]))
        return torch.stack(out), S

    want = [oracle(q.to(F64)) for q in p]
    state = torch.full((6, width), 3.0, dtype=torch.float32, device=dev)
    slots = [4, 2, 1]
    got = [[] for _ in range(3)]
    for live, off, lens, cu, reset in _batches(lens_a, lens_b, dev):
        x = torch.cat([p[s][off[s]:off[s] + lens[s]] for s in live]).to(dev)
        slot = torch.tensor([slots[s] for s in live], dtype=torch.int32, device=dev)
        o = ops.mingru_scan(x[:, :width], x[:, width:2 * width], x[:, 2 * width:3 * width], zb.to(dev), xb.to(dev), state, cu,
                            slot, reset, single_rows=max(lens) == 1)
        a = 0
        for s in live:
            got[s].append(o[a:a + lens[s]].cpu())
            a += lens[s]
    for s in range(3):
        assert rel(torch.cat(got[s]), want[s][0]) < (0.01 if dt == BF else 2e-5), s
        assert rel(state[slots[s]], want[s][1]) < 2e-5, s
    assert float(state[0].min()) == float(state[5].max()) == 3.0            # other slots are untouched


def head_gate_case(dev, dt, T=5, H=3, D=64, vdim=10, seed=4):
    g = torch.Generator().manual_seed(seed)
    a, gate = torch.randn(T, H, D, generator=g).to(dt), torch.randn(T, H + 3, generator=g).to(dt)
    want = (a[..., :vdim].to(F64) * po.sigmoid(gate[:, 3:].to(F64))[:, :, None]).reshape(T, H * vdim)
    assert rel(ops.head_gate(a.to(dev), gate.to(dev)[:, 3:], vdim, 0), want) < (0.01 if dt == BF else 1e-6)
    gate = torch.randn(T, H * vdim + 8, generator=g).to(dt)
    want = (a[..., :vdim].to(F64).reshape(T, -1) * po.sigmoid(gate[:, 8:].to(F64)))
    assert rel(ops.head_gate(a.to(dev), gate.to(dev)[:, 8:], vdim, 0), want) < (0.01 if dt == BF else 1e-6)


def conv_options_case(dev, dt, Hq=4, Hkv=2, dim=8, vdim=6, K=3, rot=4, il=False, seed=2):
    """Attention input with every option at once -- biases, head norms before the rotation, value
    mix, values handed out -- over three sequences in two steps (a one-row first step: the bias must
    not reach the rows before position 0), against the oracle's functions."""
    g = torch.Generator().manual_seed(seed)
    P, D = 16, 64 if max(dim, vdim) <= 64 else (128 if max(dim, vdim) <= 128 else 256)
    nq, nk, nv = Hq * dim, Hkv * dim, Hkv * vdim
    C = nq + nk + nv
    lens_a, lens_b = [1, 0, 19], [2, 6, 1]
    n = [a + b for a, b in zip(lens_a, lens_b)]
    p = [torch.randn(k, C + 8, generator=g).to(dt) for k in n]
    vf = [torch.randn(k, nv, generator=g).to(dt) for k in n]
    b = torch.randn(C, generator=g).to(dt)
    cw = (torch.randn(C, K, generator=g) * 0.6).to(dt) if K else None
    qn, kn = ((1 + 0.3 * torch.randn(dim, generator=g)).to(dt) for _ in range(2))
    lam = torch.tensor([0.35])
    rope = {"base": 90.0, "dims": rot, "scaling": dict(zip(("factor", "original", "fast", "slow"), YARN))} if rot else None
    from ome_amd.models.config import yarn_rope_table

    cs = yarn_rope_table(90.0, rot, 64, rope["scaling"], dev) if rot else torch.zeros(64, 0, device=dev)
    want = []
    for s in range(3):
        u = p[s][:, :C].to(F64) + b.to(F64)
        u = po.causal_conv(u, cw.to(F64)) if K else u
        turn = po.rotate_neighbours if il else po.rotate_halves
        q = turn(po.rms_unit(u[:, :nq].view(n[s], Hq, dim), EPS) * qn.to(F64), rope)
        k = turn(po.rms_unit(u[:, nq:nq + nk].view(n[s], Hkv, dim), EPS) * kn.to(F64), rope)
        v = 0.65 * u[:, nq + nk:] + 0.35 * vf[s].to(F64)
        want.append((q, k, v))
    tail = torch.full((6, max(K - 1, 0), C), 3.0, dtype=dt, device=dev) if K > 1 else None
    slots_of = [4, 2, 1]
    kc = torch.zeros(12, Hkv, P, D, dtype=dt, device=dev)
    vc = torch.zeros(12, Hkv, D, P, dtype=dt, device=dev)
    page0 = [3, 7, 9]            # two pages per sequence
    dd = lambda t: None if t is None else t.contiguous().to(dev)   # noqa: E731
    tol = 0.03 if dt == BF else 2e-5
    taps = (dd(cw[:nq]), dd(cw[nq:nq + nk]), dd(cw[nq + nk:])) if K else (None,) * 3
    for live, off, lens, cu, reset in _batches(lens_a, lens_b, dev):
        cat = lambda seqs: torch.cat([seqs[s][off[s]:off[s] + lens[s]] for s in live]).to(dev)   # noqa: E731
        x = cat(p)
        T = x.shape[0]
        pos = torch.cat([torch.arange(off[s], off[s] + lens[s]) for s in live]).to(torch.int32)
        pg = torch.cat([torch.full((lens[s],), page0[s]) for s in live])
        where = ((pg + pos // P) * P + pos % P).to(torch.int32).to(dev)
        slot = torch.tensor([slots_of[s] for s in live], dtype=torch.int32, device=dev)
        q = torch.empty(T, Hq, D, dtype=dt, device=dev)
        v_out = torch.empty(T, nv, dtype=dt, device=dev)
        ops.conv_rope_cache(x[:, :nq], x[:, nq:nq + nk], x[:, nq + nk:C], *taps, tail, (cu, slot, reset), pos.to(dev), cs, rot,
                            il, False, EPS, q, kc, vc, where, Hq, Hkv, dim, vdim, bias=(dd(b[:nq]), dd(b[nq:nq + nk]), dd(b[nq + nk:])),
                            head_norm=(dd(qn), dd(kn)), v_mix=(lam.to(dev), cat(vf)), v_out=v_out)
        a = 0
        for s in live:
            sl = slice(off[s], off[s] + lens[s])
            assert rel(q[a:a + lens[s], :, :dim], want[s][0][sl]) < tol, s
            assert rel(v_out[a:a + lens[s]], want[s][2][sl]) < tol, s
            a += lens[s]
        assert float(q[:, :, dim:].float().abs().max() if dim < D else 0.0) == 0.0
    for s in range(3):
        at = [((page0[s] + t // P), t % P) for t in range(n[s])]
        k = torch.stack([kc[i, :, j, :dim] for i, j in at])
        v = torch.stack([vc[i, :, :vdim, j].reshape(-1) for i, j in at])
        assert rel(k, want[s][1]) < tol and rel(v, want[s][2]) < tol, s


def moe_block(f, width, dev, dt):
    r = f["router"]
    return GroupRoutedMoE(width, r["experts"], r["top"], f["expert"]["ff"], 0.0, 1, 1, 0, 0.0, dev, dt, act=0, scoring="sigmoid")


def moe_case(dev, dt, f, width, rows=13):
    """The routed feed-forward alone, on inputs whose router decisions are clear of ties."""
    cfg = po.make_config([po.gru_layer(mlp=f)], width=width, groups=1)
    w = po.sub(po.make_weights(cfg, 9), "l0.mlp.")
    r = f["router"]
    for seed in range(7, 600):
        h = torch.randn(rows, width, generator=torch.Generator().manual_seed(seed))
        hq = h.to(dt).to(F64)
        c = po.router_scores(hq, w64(w))[1].sort(-1, descending=True).values
        t = r["top"]
        if t == r["experts"] or float((c[:, t - 1] - c[:, t]).min()) > (5e-3 if dt == BF else 1e-4):
            break
    else:
        raise AssertionError("no input with the wanted router margin")
    blk = moe_block(f, width, dev, dt)
    blk.load(w)
    hd = h.to(device=dev, dtype=dt)
    got = blk.forward(hd)
    assert rel(got, po.moe_ff(hq, w64(w), f)) < tol_of(dt)
    return blk.grouped_ok(hd)


def router_correction_case(dev):
    """The correction changes who is chosen, not the weights: those are the plain sigmoid scores,
    not renormalised."""
    logits = torch.tensor([[2.0, 1.5, 0.1, 0.0, 1.0], [0.0, 0.1, 0.2, 0.3, 3.0]], device=dev)
    corr = torch.tensor([-0.9, 0.0, 0.0, 0.6, 0.0], device=dev)
    w, ids = ops.moe_route(logits, 2, False, "sigmoid", bias=corr)
    assert sorted(ids[0].tolist()) == [1, 3] and sorted(ids[1].tolist()) == [3, 4]
    s = po.sigmoid(logits.cpu().double())
    for t in range(2):
        for j in range(2):
            assert abs(float(w[t, j]) - float(s[t, int(ids[t, j])])) < 1e-6
    assert sorted(ops.moe_route(logits, 2, False, "sigmoid")[1][0].tolist()) == [0, 1]


# ------------------------------------------------------------------------------------ planted keys
def planted_layer(kind, chunk):
    """A layer whose keys are made by the NEGATED query weights, with a sharp scale and nothing
    rotated, convolved or biased: a row that is the negated input of another one owns that one's
    softmax whenever visible, and the row itself scores lowest."""
    if kind == "attention":
        L = po.attn_layer(heads=2, kv_heads=2, dim=16, vdim=12, chunk=chunk, conv=3, rot_dims=0, scale=1.2)
    else:
        L = po.latent_layer(heads=2, dim=16, rot_dim=4, vdim=12, kv_rank=20, q_rank=20, scale=0.6)
    w = po.sub(po.make_weights(po.make_config([L], width=24), 6), "l0.mix.")
    if kind == "attention":
        w["k"], w["k.norm"] = -w["q"], w["q.norm"].clone()
        for n in "qkv":
            w[n + ".b"] = torch.zeros_like(w[n + ".b"])
            w[n + ".conv"] = torch.zeros_like(w[n + ".conv"])
            w[n + ".conv"][:, -1] = 1.0
    else:
        r = L["mixer"]["rot_dim"]
        w["dkv"] = torch.cat([w["dq"], torch.zeros(r, 24, dtype=w["dq"].dtype)])
        w["dkv.norm"] = w["dq.norm"].clone()
        w["uk"] = -w["uq"].view(2, 16 + r, -1)[:, :16].reshape(32, -1)
    return L, w


def planted_case(dev, dt, kind, T, i, j, cuts, chunk=9, other_chunk=None, moved=0.08):
    """Row j is the planted key of row i.  ``other_chunk``: a chunk size under which the key's
    visibility differs; the oracle's answer under it (for the latent layer: with the key's row
    replaced) must be another one, so the case would notice a wrong edge."""
    L, w = planted_layer(kind, chunk)
    h = torch.randn(T, 24, generator=torch.Generator().manual_seed(4))
    h[j] = -h[i]
    hq = h.to(dt).to(F64)
    want = oracle_mixer(L, hq, w64(w))
    blk, kv = block_of(L, 24, dev, dt, pages=2 * (T // 16) + 12)
    blk.load(w)
    got = run_chunks(blk, h.to(device=dev, dtype=dt), cuts, kv)
    assert rel(got[i:i + 1], want[i:i + 1]) < tol_of(dt), rel(got[i:i + 1], want[i:i + 1])
    if other_chunk is not None:
        other = oracle_mixer(dict(L, mixer=dict(L["mixer"], mask={"size": other_chunk})), hq, w64(w))
    else:
        h2 = hq.clone()
        h2[j] = hq[j - 1 if j else 1]
        other = oracle_mixer(L, h2, w64(w))
    assert (other[i] - want[i]).abs().max() > moved * want[i].abs().max()


def planted_model(chunk, kind="attention", vocab=60):
    """A one-layer model on planted weights; token 1 embeds as the negated token 0, so the two are
    each other's planted keys."""
    L, mw = planted_layer(kind, chunk)
    cfg = po.make_config([L], width=24, vocab=vocab, groups=2)
    w = po.make_weights(cfg, 6)
    for k, v in mw.items():
        w["l0.mix." + k] = v
    w["embed"][1] = -w["embed"][0]
    return cfg, w


def planted_prompts(chunk, n_chunks, vocab=60, seed=3):
    """{id: tokens}: random tokens with token 0 (the query) at places just behind a chunk's first
    row, in its middle and at its last row, and token 1 (its key) at the chunk's first row (seen) or
    at the last row of the chunk before (not seen)."""
    g = random.Random(seed)
    out = {}
    for name, key_off in (("in", 0), ("out", -1)):
        for at in (1, chunk // 2, chunk - 1):
            t = [g.randrange(2, vocab) for _ in range(chunk * n_chunks)]
            for c in range(1, n_chunks):
                t[c * chunk + key_off] = 1
                t[c * chunk + at] = 0
            out[f"{name}{at}"] = t
    return out


def planted_engine_case(dev, dtype, chunk, schedules, tmp, tol, n_chunks=3):
    cfg, w = planted_model(chunk)
    path = po.write_model(str(tmp), cfg, w)
    toks = planted_prompts(chunk, n_chunks)
    want = {k: po.forward(cfg, w, t) for k, t in toks.items()}
    shifted = dict(cfg, layers=[dict(cfg["layers"][0], mixer=dict(cfg["layers"][0]["mixer"], mask={"size": chunk * n_chunks}))])
    for k, t in toks.items():
        if k.startswith("out"):      # with the chunks' edge gone the key is seen and the answer is another one
            e = logit_errors(po.forward(shifted, w, t), want[k])
            assert e[t.index(0)] > 0.05
    for sched in schedules(toks):
        eng = make_engine(path, dev, dtype, max_tokens=4 * 16 * (-(-chunk * n_chunks // 16)))
        got = replay(eng, toks, sched)
        for k in toks:
            e = logit_errors(got[k], want[k])
            assert e.max().item() < tol, (k, int(e.argmax()), e.max().item())


def constants_matter_case():
    """Oracle sanity: the value mix, the layer's unused mix factor, the depth coefficients, YaRN,
    the gates and the norm groups each move the result by an amount of their own size (or not)."""
    cfg = config_a()
    wt = po.make_weights(cfg, 2)
    t = [3, 9, 1, 30, 7, 12, 2, 2, 19, 5]
    a = po.forward(cfg, wt, t)

    def moved(cfg2=cfg, **kw):
        return float((po.forward(cfg2, dict(wt, **kw), t) - a).abs().max())

    assert moved(**{"l4.mix.vmix": torch.tensor(0.0)}) > 0.02 and moved(**{"l1.mix.vmix": torch.tensor(0.0)}) == 0.0
    assert moved(**{"l5.dwa": torch.cat([torch.zeros(6), torch.ones(1)])}) > 0.05
    assert moved(**{"l2.mix.z.b": torch.zeros(20)}) > 0.02
    assert moved(dict(cfg, norm={"eps": 1e-5, "groups": 1})) > 0.02
    L1 = dict(cfg["layers"][1], mixer=dict(cfg["layers"][1]["mixer"], rot={"base": 100.0, "dims": 4}))
    assert moved(dict(cfg, layers=cfg["layers"][:1] + [L1] + cfg["layers"][2:])) > 0.01
    assert moved(**{"l0.mix.g": torch.zeros_like(wt["l0.mix.g"])}) > 0.02
