"""Slow fp64 implementation of the Pagatar design, one function per mechanism, written from the
equations alone (no code shared with ``ome_amd``), plus makers of small random configs and
checkpoints for the tests.  Everything works on one whole sequence at a time."""
from __future__ import annotations

import json
import math
import os

import torch

F64 = torch.float64


# ------------------------------------------------------------------------------------ pieces
def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_norm(x, w, groups, eps):
    """Every one of ``groups`` equal consecutive parts by its own root mean square, then the weight."""
    T, W = x.shape
    return rms_unit(x.reshape(T, groups, W // groups), eps).reshape(T, W) * w


def sigmoid(x):
    return 1 / (1 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def depth_average(coef, history):
    return sum(coef[j] * x for j, x in enumerate(history))


def mingru_candidate(u):
    return torch.where(u >= 0, u + 0.5, sigmoid(u))


def mingru(h, w):
    """S_t = (1 - z_t) S_{t-1} + z_t c_t element by element; the output is gated by silu."""
    z = sigmoid(h @ w["z"].T + w["z.b"])
    c = mingru_candidate(h @ w["x"].T + w["x.b"])
    S, out = torch.zeros_like(z[0]), []
    for t in range(h.shape[0]):
        S = (1 - z[t]) * S + z[t] * c[t]
        out.append(S)
    return (torch.stack(out) * silu(h @ w["g"].T)) @ w["o"].T


def causal_conv(u, w):
    """y_t = sum_j w[:, j] u_{t - K + 1 + j}, rows before the start are zero; u [T, C], w [C, K]."""
    T, K = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for j in range(K):
        back = K - 1 - j                      # tap j reads the row `back` steps before
        if back < T:
            y[back:] += w[:, j] * u[:T - back]
    return y


def frequencies(dims, base, scaling=None):
    """([dims / 2] frequencies, factor of cos and sin); ``scaling`` = YaRN's {factor, original, fast, slow}."""
    f = [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return torch.tensor(f, dtype=F64), 1.0

    def turns_at(t):
        return dims * math.log(scaling["original"] / (2 * math.pi * t)) / (2 * math.log(base))

    lo, hi = max(math.floor(turns_at(scaling["fast"])), 0), min(math.ceil(turns_at(scaling["slow"])), dims - 1)
    out = []
    for i, x in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(x / scaling["factor"] * r + x * (1 - r))
    return torch.tensor(out, dtype=F64), 0.1 * math.log(scaling["factor"]) + 1.0


def angles(T, rot):
    f, m = frequencies(rot["dims"], rot["base"], rot.get("scaling"))
    a = torch.arange(T, dtype=F64)[:, None] * f[None]
    return torch.cos(a)[:, None] * m, torch.sin(a)[:, None] * m


def rotate_halves(x, rot):
    """x [T, H, d]: dim i pairs with dim i + dims/2 (i < dims/2); the rest passes."""
    n = (rot or {}).get("dims", 0)
    if not n:
        return x
    c, s = angles(x.shape[0], rot)
    u, v = x[..., :n // 2], x[..., n // 2:n]
    out = x.clone()
    out[..., :n // 2] = u * c - v * s
    out[..., n // 2:n] = v * c + u * s
    return out


def rotate_neighbours(x, rot):
    """x [T, H, d]: dims (2i, 2i+1), i < dims/2; the rest passes."""
    n = (rot or {}).get("dims", 0)
    if not n:
        return x
    c, s = angles(x.shape[0], rot)
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out = x.clone()
    out[..., 0:n:2] = u * c - v * s
    out[..., 1:n:2] = v * c + u * s
    return out


def chunk_mask(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None]
    vis = j <= i
    return vis & (i // size == j // size) if size else vis


def softmax_over(score, visible):
    s = score.masked_fill(~visible[None], -math.inf)
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def conv_projection(h, w, n):
    u = h @ w[n].T + w[n + ".b"]
    return causal_conv(u, w[n + ".conv"]) if n + ".conv" in w else u


def attention(h, w, m, eps, first=None):
    """Grouped-query attention within chunks: biased projections, short convolutions, q / k norms
    and rotation; ``first``: a list that receives the values of the first value-mixing layer and
    hands them to the later ones.  Output gated element by element."""
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (conv_projection(h, w, n) for n in "qkv")
    if m.get("v_mix") and first is not None:
        if first:
            lam = w["vmix"]
            v = (1 - lam) * v + lam * first[0]
        else:
            first.append(v)
    q = rms_unit(q.view(T, H, d), eps) * w["q.norm"]
    k = rms_unit(k.view(T, G, d), eps) * w["k.norm"]
    q, k, v = rotate_halves(q, m.get("rot")), rotate_halves(k, m.get("rot")), v.view(T, G, dv)
    kk, vv = k.repeat_interleave(H // G, 1), v.repeat_interleave(H // G, 1)
    p = softmax_over(torch.einsum("ihd,jhd->hij", q, kk) * m["scale"], chunk_mask(T, (m.get("mask") or {}).get("size", 0)))
    o = torch.einsum("hij,jhd->ihd", p, vv).reshape(T, H * dv)
    return (o * sigmoid(h @ w["g"].T)) @ w["o"].T


def latent_attention(h, w, m, eps):
    """Queries and keys / values through normed low-rank latents, one rotated key part shared by
    all heads, full causal softmax, one output gate per head."""
    T = h.shape[0]
    H, d, r, dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    rot = m.get("rot") or {}
    q = ((rms_unit(h @ w["dq"].T, eps) * w["dq.norm"]) @ w["uq"].T).view(T, H, d + r)
    kv = h @ w["dkv"].T
    c = rms_unit(kv[:, :R], eps) * w["dkv.norm"]
    k, v = (c @ w["uk"].T).view(T, H, d), (c @ w["uv"].T).view(T, H, dv)
    qr, kr = rotate_neighbours(q[..., d:], rot), rotate_neighbours(kv[:, None, R:], rot)
    score = torch.einsum("ihd,jhd->hij", q[..., :d], k) + torch.einsum("ihd,jd->hij", qr, kr[:, 0])
    p = softmax_over(score * m["scale"], chunk_mask(T, 0))
    o = torch.einsum("hij,jhd->ihd", p, v) * sigmoid(h @ w["g"].T)[:, :, None]
    return o.reshape(T, H * dv) @ w["o"].T


def glu_expert(h, w, pre):
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def router_scores(h, w):
    """(scores, choice scores)"""
    s = sigmoid(h @ w["router"].T)
    return s, s + w["correction"]


def moe_ff(h, w, f):
    """The ``top`` experts by corrected score, each weighted by its plain score."""
    s, c = router_scores(h, w)
    idx = c.topk(f["router"]["top"], -1).indices
    y = torch.zeros_like(h)
    for e in range(f["router"]["experts"]):
        rows = (idx == e).any(-1)
        if rows.any():
            y[rows] += s[rows, e, None] * glu_expert(h[rows], w, f"e{e}.")
    return y


def sub(w, prefix):
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, residuals=None, margins=None):
    """Logits [T, vocab] (fp64) of one whole sequence; ``residuals``: a list that receives the
    stream after every layer (averaged over depth); ``margins``: a one-element list that receives
    the smallest gap between the last chosen and the first unchosen choice score."""
    W = {k: v.to(F64) for k, v in weights.items()}
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = group_norm(W["embed"][list(tokens)], W["embed.norm"], groups, eps)
    history, first = [x], []
    for i, L in enumerate(cfg["layers"]):
        w = sub(W, f"l{i}.")
        mw, m = sub(w, "mix."), L["mixer"]
        if L["type"] == "mingru":
            y = mingru(x, mw)
        elif L["type"] == "attention":
            y = attention(x, mw, m, eps, first)
        elif L["type"] == "latent_attention":
            y = latent_attention(x, mw, m, eps)
        else:
            raise ValueError(L["type"])
        x = x + group_norm(y, w["norm1"], groups, eps)
        f = L.get("mlp")
        if f:
            fw = sub(w, "mlp.")
            t = f["router"]["top"]
            if margins is not None and t < f["router"]["experts"]:
                srt = router_scores(x, fw)[1].sort(-1, descending=True).values
                margins[0] = min(margins[0], float((srt[:, t - 1] - srt[:, t]).min()))
            x = x + group_norm(moe_ff(x, fw, f), w["norm2"], groups, eps)
        history.append(x)
        x = depth_average(w["dwa"], history)
        if residuals is not None:
            residuals.append(x.clone())
    return group_norm(x, W["final.norm"], groups, eps) @ W["embed"].T


# ------------------------------------------------------------------------------------ makers
def moe(experts=5, top=2, ff=12):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def attn_layer(heads=4, kv_heads=2, dim=8, vdim=6, chunk=7, conv=3, rot_dims=4, base=100.0, scaling=None, scale=0.5,
               v_mix=False, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk}, "scale": scale,
         "conv": conv, "v_mix": v_mix}
    if rot_dims:
        m["rot"] = {"base": base, "dims": rot_dims}
        if scaling:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "attention", "mixer": m, "mlp": mlp}


def latent_layer(heads=3, dim=8, rot_dim=4, vdim=6, kv_rank=10, q_rank=12, base=50.0, scale=0.4, mlp=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "scale": scale,
         "rot": {"base": base, "dims": rot_dim}}
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def gru_layer(inner=20, mlp=None):
    return {"type": "mingru", "mixer": {"width": inner}, "mlp": mlp}


def make_config(layers, width=24, vocab=41, eps=1e-5, groups=3):
    return {"architecture": "Pagatar", "layers": layers, "norm": {"eps": eps, "groups": groups}, "vocab": vocab, "width": width}


def make_weights(cfg, seed=0, dtype=torch.bfloat16):
    """Random checkpoint tensors (values exactly representable in ``dtype``), sized so that the
    stream stays O(1), scores spread over a few units and states remember a few dozen tokens."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def rnd(*shape, s=1.0):
        return (torch.randn(*shape, generator=g) * s).to(dtype)

    def lin(o, i, gain=1.0):
        return rnd(o, i, s=gain / math.sqrt(i))

    def gain(n, at=1.0):
        return (at + 0.2 * torch.randn(n, generator=g)).to(dtype)

    t = {"embed": rnd(V, W, s=0.7), "embed.norm": gain(W), "final.norm": gain(W)}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        t[p + "norm1"] = gain(W, 0.8)
        if L["type"] == "attention":
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for n, c in (("q", H * d), ("k", G * d), ("v", G * dv)):
                t[p + "mix." + n], t[p + "mix." + n + ".b"] = lin(c, W), rnd(c, s=0.5)
                if m.get("conv"):
                    t[p + "mix." + n + ".conv"] = rnd(c, m["conv"], s=0.6)
            t[p + "mix.q.norm"], t[p + "mix.k.norm"] = gain(d), gain(d)
            t[p + "mix.g"], t[p + "mix.o"] = lin(H * dv, W), lin(W, H * dv)
            if m.get("v_mix"):
                t[p + "mix.vmix"] = (0.3 + 0.4 * torch.rand((), generator=g)).to(dtype)
        elif L["type"] == "latent_attention":
            H, d, r, dv, R, Q = (m[n] for n in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
            t[p + "mix.dq"], t[p + "mix.dq.norm"], t[p + "mix.uq"] = lin(Q, W), gain(Q), lin(H * (d + r), Q, 1.5)
            t[p + "mix.dkv"], t[p + "mix.dkv.norm"] = lin(R + r, W), gain(R)
            t[p + "mix.uk"], t[p + "mix.uv"] = lin(H * d, R, 1.5), lin(H * dv, R)
            t[p + "mix.g"], t[p + "mix.o"] = lin(H, W), lin(W, H * dv)
        else:
            n = m["width"]
            t[p + "mix.z"], t[p + "mix.x"], t[p + "mix.g"] = lin(n, W), lin(n, W), lin(n, W)
            t[p + "mix.z.b"] = (-3 + 3 * torch.rand(n, generator=g)).to(dtype)
            t[p + "mix.x.b"], t[p + "mix.o"] = rnd(n, s=0.5), lin(W, n)
        t[p + "dwa"] = torch.cat([rnd(i + 1, s=0.2), torch.ones(1, dtype=dtype)])
        f = L.get("mlp")
        if not f:
            continue
        E, ff = f["router"]["experts"], f["expert"]["ff"]
        t[p + "norm2"] = gain(W, 0.8)
        t[p + "mlp.router"], t[p + "mlp.correction"] = lin(E, W, 2.0), rnd(E, s=0.3)
        for j in range(E):
            t[p + f"mlp.e{j}.gate"], t[p + f"mlp.e{j}.up"], t[p + f"mlp.e{j}.down"] = lin(ff, W), lin(ff, W), lin(W, ff)
    return t


def write_model(folder, cfg, weights):
    from safetensors.torch import save_file

    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in weights.items()}, os.path.join(folder, "model.safetensors"))
    return folder


def router_margin(cfg, weights, tokens):
    """Smallest gap between the last chosen and the first unchosen choice score over all routed
    evaluations of a prompt (infinite when every expert is always chosen)."""
    m = [math.inf]
    forward(cfg, weights, tokens, margins=m)
    return m[0]
