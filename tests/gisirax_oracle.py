"""Slow fp64 implementation of the Gisirax design, one function per mechanism, written from the
equations alone (no code shared with ``ome_amd``), plus makers of small random configs and
checkpoints for the tests.  Everything works on one whole sequence at a time."""
from __future__ import annotations

import json
import math
import os

import torch

F64 = torch.float64


# ------------------------------------------------------------------------------------ pieces
def sigmoid(x):
    return 1 / (1 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return torch.clamp(x, min=0) + torch.log1p(torch.exp(-x.abs()))


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def unit_vector(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def tanh_norm(x, w, name):
    """tanh(alpha x) w + b with one scalar alpha and a vector b beside the weight."""
    return torch.tanh(w[name + ".alpha"] * x) * w[name] + w[name + ".b"]


def embed_rows(cfg, W, tokens):
    e = cfg["embedding"]
    rows = []
    big = e.get("bigram")
    for t, tok in enumerate(tokens):
        x = W["embed"][tok] * e["scale"]
        if big:
            r = (tokens[t - 1] * big["mul_prev"] + tok * big["mul_cur"]) % big["buckets"] if t else big["buckets"]
            x = x + W["bigram"][r]
        rows.append(x)
    return torch.stack(rows)


def frequencies(rot):
    """Angle per position of every pair; ``scaling`` slows the pairs whose wavelength is long
    against ``original`` by ``factor``, leaves the short ones and blends the ones between."""
    n, sc, out = rot["dims"], rot.get("scaling"), []
    for i in range(n // 2):
        f = float(rot["base"]) ** (-2.0 * i / n)
        if sc:
            lam = 2 * math.pi / f
            if lam > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif lam >= sc["original"] / sc["high"]:
                s = (sc["original"] / lam - sc["low"]) / (sc["high"] - sc["low"])
                f = (1 - s) * f / sc["factor"] + s * f
        out.append(f)
    return torch.tensor(out, dtype=F64)


def rotate_halves(x, rot):
    """x [T, H, d]: dim i pairs with dim i + dims/2 (i < dims/2); the rest passes."""
    n = (rot or {}).get("dims", 0)
    if not n:
        return x
    a = torch.arange(x.shape[0], dtype=F64)[:, None, None] * frequencies(rot)
    u, v = x[..., :n // 2], x[..., n // 2:n]
    out = x.clone()
    out[..., :n // 2] = u * torch.cos(a) - v * torch.sin(a)
    out[..., n // 2:n] = v * torch.cos(a) + u * torch.sin(a)
    return out


def softmax_plus_one(score):
    """Causal softmax over the last axis with one more exp(0) in the denominator."""
    T = score.shape[-1]
    s = score.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1)[None], -math.inf)
    m = torch.clamp(s.max(-1, keepdim=True).values, min=0.0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def attention(h, w, m):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate_halves((h @ w["q"].T).view(T, H, d), m.get("rot"))
    k = rotate_halves((h @ w["k"].T).view(T, G, d), m.get("rot")).repeat_interleave(H // G, 1)
    v = (h @ w["v"].T).view(T, G, dv).repeat_interleave(H // G, 1)
    p = softmax_plus_one(torch.einsum("ihd,jhd->hij", q, k) * m["scale"])
    return torch.einsum("hij,jhd->ihd", p, v).reshape(T, H * dv) @ w["o"].T


def lightning_core(q, k, v, decay):
    """o_t = S_t^T q_t, S_t = decay_h S_{t-1} + k_t v_t^T; q, k [T, H, d], v [T, H, dv] -> ([T, H, dv], S)."""
    T, H, d = q.shape
    S, out = torch.zeros(H, d, v.shape[-1], dtype=F64), []
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def lightning_attention(h, w, m, eps):
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q, k, v = silu(h @ w["q"].T).view(T, H, d), silu(h @ w["k"].T).view(T, H, d), silu(h @ w["v"].T).view(T, H, dv)
    o = lightning_core(q, k, v, torch.tensor(m["decay"], dtype=F64))[0].reshape(T, H * dv)
    return (rms_unit(o, eps) * w["norm"] * sigmoid(h @ w["g"].T)) @ w["o"].T


def parallel(h, w, m, eps):
    left = attention(h, sub(w, "left."), m["left"])
    right = lightning_attention(h, sub(w, "right."), m["right"], eps)
    return 0.5 * (rms_unit(left, eps) * w["left.out"] + rms_unit(right, eps) * w["right.out"])


def causal_conv(u, w):
    """y_t = sum_j w[:, j] u_{t - K + 1 + j}, rows before the start are zero; u [T, C], w [C, K]."""
    T, K = u.shape[0], w.shape[1]
    y = torch.zeros_like(u)
    for j in range(K):
        back = K - 1 - j                      # tap j reads the row `back` steps before
        if back < T:
            y[back:] += w[:, j] * u[:T - back]
    return y


def channel_decay(h, w, H, d):
    """[T, H, d] factors by which the state's rows (key channels) shrink."""
    z = (h @ w["a1"].T) @ w["a2"].T + w["dt_bias"]
    return torch.exp(-torch.exp(w["A_log"])[:, None] * softplus(z).view(-1, H, d))


def delta_core(q, k, v, g, beta):
    """q, k, g [T, H, d], v [T, H, dv], beta [T, H] -> ([T, H, dv], S [H, d, dv])."""
    T, H, d = q.shape
    S, out = torch.zeros(H, d, v.shape[-1], dtype=F64), []
    for t in range(T):
        S = S * g[t][:, :, None]
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def channel_delta(h, w, m, eps):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ w[n].T, w[n + ".conv"])) for n in "qkv")
    q = unit_vector(q.view(T, G, d)).repeat_interleave(H // G, 1) * d ** -0.5
    k = unit_vector(k.view(T, G, d)).repeat_interleave(H // G, 1)
    o = delta_core(q, k, v.view(T, H, dv), channel_decay(h, w, H, d), sigmoid(h @ w["b"].T))[0]
    gate = sigmoid((h @ w["g1"].T) @ w["g2"].T).view(T, H, dv)
    return (rms_unit(o, eps) * w["norm"] * gate).reshape(T, H * dv) @ w["o"].T


def glu_expert(h, w, pre):
    return (silu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def choose(s, r):
    """([T, E] bool: the chosen experts, smallest margin of the two choices): groups by the sum of
    their two best scores, then the best experts of the kept groups."""
    T, E = s.shape
    grp = r.get("groups") or {"count": 1, "keep": 1}
    n, keep, top = grp["count"], grp["keep"], r["top"]
    best = s.view(T, n, E // n).sort(-1, descending=True).values
    score = best[:, :, :2].sum(-1)
    kept = torch.zeros(T, n, dtype=torch.bool).scatter_(1, score.topk(keep, -1).indices, True)
    c = s.masked_fill(~kept.repeat_interleave(E // n, 1), -math.inf)
    chosen = torch.zeros(T, E, dtype=torch.bool).scatter_(1, c.topk(top, -1).indices, True)
    margin = math.inf
    if keep < n:
        o = score.sort(-1, descending=True).values
        margin = min(margin, float((o[:, keep - 1] - o[:, keep]).min()))
    if top < keep * (E // n):
        o = c.sort(-1, descending=True).values
        margin = min(margin, float((o[:, top - 1] - o[:, top]).min()))
    return chosen, margin


def moe_ff(h, w, f):
    r = f["router"]
    s = sigmoid(h @ w["router"].T)
    chosen = choose(s, r)[0]
    p = s * chosen
    p = p / (p.sum(-1, keepdim=True) + 1e-20) * r["scale"]
    y = torch.zeros_like(h)
    for e in range(r["experts"]):
        rows = chosen[:, e]
        if rows.any():
            y[rows] += p[rows, e, None] * glu_expert(h[rows], w, f"e{e}.")
    return y


def sub(w, prefix):
    return {k[len(prefix):]: v for k, v in w.items() if k.startswith(prefix)}


def forward(cfg, weights, tokens, residuals=None, margins=None):
    """Logits [T, vocab] (fp64) of one whole sequence; ``residuals``: a list that receives the
    stream after every layer; ``margins``: a one-element list that receives the smallest gap of any
    router decision (groups or experts)."""
    W = {k: v.to(F64) for k, v in weights.items()}
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x = embed_rows(cfg, W, list(tokens))
    for i, L in enumerate(cfg["layers"]):
        w = sub(W, f"l{i}.")
        h, mw = tanh_norm(x, w, "norm1"), sub(w, "mix.")
        if L["type"] == "parallel":
            y = parallel(h, mw, L["mixer"], eps)
        elif L["type"] == "channel_delta":
            y = channel_delta(h, mw, L["mixer"], eps)
        else:
            raise ValueError(L["type"])
        x = x + m * tanh_norm(y, w, "norm1b")
        f = L.get("mlp")
        if f:
            h, fw = tanh_norm(x, w, "norm2"), sub(w, "mlp.")
            if margins is not None:
                margins[0] = min(margins[0], choose(sigmoid(h @ fw["router"].T), f["router"])[1])
            x = x + m * tanh_norm(moe_ff(h, fw, f), w, "norm2b")
        if residuals is not None:
            residuals.append(x.clone())
    return tanh_norm(x, W, "final.norm") @ W["head"].T


# ------------------------------------------------------------------------------------ makers
def moe(experts=6, top=2, ff=12, groups=3, keep=2, scale=1.7):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top, "groups": {"count": groups, "keep": keep}, "scale": scale}}


def parallel_layer(heads=4, kv_heads=2, dim=8, vdim=6, rot_dims=4, base=100.0, scaling=(4.0, 1.0, 4.0, 64), scale=0.4,
                   r_heads=3, r_dim=5, r_vdim=7, decay=(0.5, 0.9, 0.99), mlp=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if rot_dims:
        left["rot"] = {"base": base, "dims": rot_dims}
        if scaling:
            left["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return {"type": "parallel", "mlp": mlp,
            "mixer": {"left": left, "right": {"heads": r_heads, "dim": r_dim, "vdim": r_vdim, "decay": list(decay)}}}


def delta_layer(heads=4, kv_heads=2, dim=8, vdim=6, conv=3, mlp=None):
    return {"type": "channel_delta", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def make_config(layers, width=24, vocab=41, eps=1e-5, scale=3.0, mult=0.4, bigram=(29, 13, 5)):
    emb = {"scale": scale}
    if bigram:
        emb["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))
    return {"architecture": "Gisirax", "embedding": emb, "layers": layers, "norm": {"eps": eps}, "residual_mult": mult,
            "vocab": vocab, "width": width}


def make_weights(cfg, seed=0, dtype=torch.bfloat16, ranks=(5, 7)):
    """Random checkpoint tensors (values exactly representable in ``dtype``), sized so that the
    stream stays O(1), scores spread over a few units and states remember a few dozen tokens.
    ``ranks``: rows of the low-rank projections a1 and g1."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def rnd(*shape, s=1.0):
        return (torch.randn(*shape, generator=g) * s).to(dtype)

    def lin(o, i, gain=1.0):
        return rnd(o, i, s=gain / math.sqrt(i))

    def gain(n, at=1.0):
        return (at + 0.2 * torch.randn(n, generator=g)).to(dtype)

    t = {"embed": rnd(V, W, s=0.7 / cfg["embedding"]["scale"]), "head": lin(V, W)}
    if cfg["embedding"].get("bigram"):
        t["bigram"] = rnd(cfg["embedding"]["bigram"]["buckets"] + 1, W, s=0.5)

    def norm(name, at=1.0):
        t[name], t[name + ".b"] = gain(W, at), rnd(W, s=0.1)
        t[name + ".alpha"] = (0.6 + 0.5 * torch.rand((), generator=g)).to(dtype)

    norm("final.norm")
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        norm(p + "norm1")
        norm(p + "norm1b", 1.5)
        x = p + "mix."
        if L["type"] == "parallel":
            a, r = m["left"], m["right"]
            H, G = a["heads"], a["kv_heads"]
            t[x + "left.q"], t[x + "left.k"] = lin(H * a["dim"], W, 1.5), lin(G * a["dim"], W, 1.5)
            t[x + "left.v"], t[x + "left.o"] = lin(G * a["vdim"], W), lin(W, H * a["vdim"])
            t[x + "right.q"], t[x + "right.k"] = lin(r["heads"] * r["dim"], W), lin(r["heads"] * r["dim"], W)
            n = r["heads"] * r["vdim"]
            t[x + "right.v"], t[x + "right.g"] = lin(n, W), lin(n, W)
            t[x + "right.norm"], t[x + "right.o"] = gain(n), lin(W, n)
            t[x + "left.out"], t[x + "right.out"] = gain(W), gain(W)
        else:
            H, G, d, dv, K = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            for n, c in (("q", G * d), ("k", G * d), ("v", H * dv)):
                t[x + n], t[x + n + ".conv"] = lin(c, W, 1.5), rnd(c, K, s=0.6)
            t[x + "b"] = lin(H, W)
            t[x + "A_log"] = torch.log(0.05 + 0.4 * torch.rand(H, generator=g)).to(dtype)
            t[x + "a1"], t[x + "a2"] = lin(ranks[0], W), lin(H * d, ranks[0], 1.5)
            t[x + "dt_bias"] = rnd(H * d)
            t[x + "g1"], t[x + "g2"] = lin(ranks[1], W), lin(H * dv, ranks[1], 1.5)
            t[x + "norm"], t[x + "o"] = gain(dv), lin(W, H * dv)
        f = L.get("mlp")
        if not f:
            continue
        norm(p + "norm2")
        norm(p + "norm2b", 1.5)
        E, ff = f["router"]["experts"], f["expert"]["ff"]
        t[p + "mlp.router"] = lin(E, W, 2.0)
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
    """Smallest gap of any group or expert choice over all routed evaluations of a prompt."""
    m = [math.inf]
    forward(cfg, weights, tokens, margins=m)
    return m[0]
