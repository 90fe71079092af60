"""Gisirax: a layer-list decoder (``architecture: Gisirax``) whose norms are tanh curves, before AND
after every sublayer, with a hashed token-pair embedding and group-routed experts.

``layers[i]`` = {``type``, ``mixer`` (that mixer's own sizes), ``mlp`` (or null)}.  Mixer types:

* ``channel_delta`` -- ``mixers.ChannelDeltaMixer``: gated delta rule with a decay per head and key
  channel behind short convolutions;
* ``parallel`` -- ``mixers.ParallelMixers``: causal grouped-query attention (``mixers.
  GatedWindowAttention`` without window, norms or gate; half-split rotary pairs scaled by wavelength
  bands; one added to the softmax denominator) beside ``mixers.LightningAttention``; the block's
  output is half the sum of the two outputs, each RMS-normed over the width with its own weight.

Feed-forward (``mlp.kind: moe``): ``mixers.GroupRoutedMoE`` with sigmoid scores, groups that score by
the sum of their two best experts, renormalised weights times ``router.scale``, SiLU-GLU experts.

With D(v) = tanh(alpha v) w + b (scalar alpha, vectors w and b per norm) and c = ``residual_mult``:

  x += c D1b(mixer(D1(x)));   x += c D2b(ff(D2(x)))            (no ``mlp``: the first half only)

x starts as ``embed[token] * embedding.scale + bigram[r]``, r = (previous token * mul_prev + token *
mul_cur) mod buckets, the table's extra last row for a sequence's first token.  logits = ``head`` .
D_final(x).

Numerics: x is fp32 from the embedding to the final norm.  ``ops.tanh_stream`` norms a sublayer's
output (joining the two outputs of a parallel block first), adds it, norms the sum and rounds once
to the next GEMM's input, one launch per sublayer.  Convolutions, unit norms, decays, write
strengths, both recurrences and their states, rotary angles, attention scores / softmax, router
logits and scores are fp32 inside the kernels; logits leave the head in fp32.  The previous token
of every request slot is part of the state (``prev_token``).  Prefix caching is off (``stateful``).
The model has no cache, loop over steps or scheduler of its own: ``ModelRunner`` drives it like the
other layer-list designs.
"""
from __future__ import annotations

import torch

from ome_amd import ops
from ome_amd.models.common import AttnMeta, PagedKVCache
from ome_amd.models.config import ModelConfig
from ome_amd.models.llama import LlamaForCausalLM
from ome_amd.models.mixers import (ChannelDeltaMixer, GatedWindowAttention, GroupRoutedMoE, LightningAttention, MixerCtx,
                                   ParallelMixers)
from ome_amd.parallel import state as pstate

GISIRAX_ARCHS = {"Gisirax"}
NORMS = ("norm1", "norm1b", "norm2", "norm2b")


class GisiraxForCausalLM(LlamaForCausalLM):
    stateful = True
    tune_gemms = False   # odd projection widths: the library heuristic, no TunableOp pass

    def __init__(self, cfg: ModelConfig, device="cuda", dtype=torch.bfloat16, max_positions: int | None = None):
        st = pstate.get()
        if st.tp_size > 1 or st.pp_size > 1:
            raise NotImplementedError("Gisirax: tensor / pipeline parallelism (one GPU holds the model)")
        super().__init__(cfg, device, dtype, 1)   # (the base's rotary table is unused: one row)
        hf = cfg.extra or {}
        W, eps = cfg.hidden_size, cfg.rms_norm_eps
        mp = max_positions or cfg.max_position_embeddings
        emb = hf.get("embedding") or {}
        self.embed_scale = float(emb.get("scale", 1.0))
        self.pair = dict(emb["bigram"]) if emb.get("bigram") else None      # {buckets, mul_prev, mul_cur}
        self.mult = float(hf.get("residual_mult", 1.0))
        self.specs = list(hf["layers"])
        self.mix: list[ChannelDeltaMixer | ParallelMixers] = []
        self.ff: dict[int, GroupRoutedMoE] = {}
        for i, spec in enumerate(self.specs):
            m, kind = spec["mixer"], spec["type"]
            if kind == "channel_delta":
                self.mix.append(ChannelDeltaMixer(W, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], eps,
                                                  self.device, dtype))
            elif kind == "parallel":
                a, r = m["left"], m["right"]
                rot = a.get("rot") or {}
                left = GatedWindowAttention(i, W, a["heads"], a["kv_heads"], a["dim"], a["vdim"], -1, 0,
                                            rot.get("base", 10000.0), rot.get("dims", 0), a["scale"], eps, mp, self.device,
                                            dtype, interleaved=False, wide_norm=False, gated=False,
                                            rot_scaling=rot.get("scaling"), sink=0.0)
                right = LightningAttention(W, r["heads"], r["dim"], r["vdim"], r["decay"], eps, self.device, dtype)
                self.mix.append(ParallelMixers(left, right, self.device, dtype))
            else:
                raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
            f = spec.get("mlp")
            if f:
                if f.get("kind", "moe") != "moe":
                    raise ValueError(f"layer {i}: unknown feed-forward kind {f.get('kind')!r}")
                ro = f["router"]
                g = ro.get("groups") or {}
                self.ff[i] = GroupRoutedMoE(W, ro["experts"], ro["top"], f["expert"]["ff"], 0.0, int(g.get("count", 1)),
                                            int(g.get("keep", 1)), 0, 0.0, self.device, dtype, act=0, renorm=True,
                                            correction=False, scoring="sigmoid", group_score="top2",
                                            routed_scale=ro.get("scale", 1.0))
        self.norms: dict[str, tuple] = {}     # "l<i>.norm1" ...: (alpha, w, b)
        self.out_w: dict[int, tuple] = {}     # parallel layers: weights of the left / right output norms
        self.pair_table = None
        self.prev_token = None                # [slots] int32: every request's last token
        attn = {i: b.left for i, b in enumerate(self.mix) if isinstance(b, ParallelMixers)}
        self.kv_layers = sorted(attn)
        self.kv_heads_per_layer = {i: a.Hkv for i, a in attn.items()}
        self.kv_dims_per_layer = {i: a.D for i, a in attn.items()}
        self.debug_residuals: list | None = None   # set to []: the stream after every layer is appended

    def prefill_item_rows(self, page: int) -> int:
        """Query rows per prefill work item: one plan serves all attention layers, so the 64-row
        item needs every layer to have the shape its kernel is built for."""
        attn = [b.left for b in self.mix if isinstance(b, ParallelMixers)]
        rows = {ops.prefill_rows(a.Hq, a.Hkv, a.D, page) for a in attn}
        return rows.pop() if len(rows) == 1 else 32

    def _blocks(self):
        yield from self.mix
        yield from self.ff.values()

    def alloc_state(self, slots: int) -> None:
        for b in self.mix:
            b.alloc_state(slots)
        self.prev_token = torch.zeros(slots, dtype=torch.int32, device=self.device)

    # ------------------------------------------------------------------ weights
    def _norm_names(self) -> list[str]:
        return [f"l{i}.{n}" for i in range(len(self.specs)) for n in (NORMS if i in self.ff else NORMS[:2])] + ["final.norm"]

    def init_random(self, seed: int = 0, std: float = 0.02) -> "GisiraxForCausalLM":
        gen = torch.Generator(device=self.device)
        gen.manual_seed(seed)
        W, V = self.cfg.hidden_size, self.cfg.vocab_size
        for n in self._norm_names():
            self.norms[n] = (0.5, self._alloc(W, std=None, gen=gen), self._alloc(W, std=0.02, gen=gen))
        for i, b in enumerate(self.mix):
            if isinstance(b, ParallelMixers):
                self.out_w[i] = (self._alloc(W, std=None, gen=gen), self._alloc(W, std=None, gen=gen))
        for b in self._blocks():
            b.init_random(gen, std)
        self.embed = self._alloc(V, W, std=1.0 / max(self.embed_scale, 1e-6), gen=gen)
        if self.pair:
            self.pair_table = self._alloc(int(self.pair["buckets"]) + 1, W, std=0.5, gen=gen)
        self.lm_head = self._alloc(V, W, std=std, gen=gen)
        return self

    def load_hf_weights(self, weights) -> "GisiraxForCausalLM":
        put = lambda w: w.to(device=self.device, dtype=self.dtype).contiguous()   # noqa: E731
        top = {"embed": "embed", "bigram": "pair_table", "head": "lm_head"}
        wanted = {f"{n}{suffix}" for n in self._norm_names() for suffix in ("", ".b", ".alpha")}
        curves: dict[str, torch.Tensor] = {}
        groups: dict[tuple[int, str], dict[str, torch.Tensor]] = {}
        for name, w in weights:
            if name in top:
                setattr(self, top[name], put(w))
            elif name in wanted:
                curves[name] = w
            elif name.startswith("l") and "." in name:
                head, rest = name.split(".", 1)
                if not head[1:].isdigit() or int(head[1:]) >= len(self.specs):
                    continue
                for pre in ("mix.", "mlp."):
                    if rest.startswith(pre):
                        groups.setdefault((int(head[1:]), pre), {})[rest[len(pre):]] = w
                        break
        W = self.cfg.hidden_size
        missing = [k for k, v in (("embed", self.embed), ("head", self.lm_head)) if v is None]
        missing += sorted(wanted - set(curves))
        if self.pair and self.pair_table is None:
            missing.append("bigram")
        for i, b in enumerate(self.mix):
            t = groups.get((i, "mix."), {})
            try:
                if isinstance(b, ParallelMixers):
                    part = {s: {k[len(s):]: w for k, w in t.items() if k.startswith(s)} for s in ("left.", "right.")}
                    self.out_w[i] = tuple(put(t[n]) for n in ("left.out", "right.out"))
                    b.load(part["left."], part["right."])
                else:
                    b.load(t)
            except KeyError as e:
                missing.append(f"l{i}.mix.{e.args[0]}")
        for i, b in self.ff.items():
            try:
                b.load(groups.get((i, "mlp."), {}))
            except KeyError as e:
                missing.append(f"l{i}.mlp.{e.args[0]}")
        if missing:
            raise ValueError(f"checkpoint incomplete: {', '.join(missing[:6])} missing")
        if self.pair and tuple(self.pair_table.shape) != (int(self.pair["buckets"]) + 1, W):
            raise ValueError(f"bigram: shape {tuple(self.pair_table.shape)} != [buckets + 1, width]")
        for n in self._norm_names():
            if curves[n + ".alpha"].numel() != 1 or curves[n].numel() != W or curves[n + ".b"].numel() != W:
                raise ValueError(f"{n}: one alpha and {W}-wide weight and bias expected")
            self.norms[n] = (float(curves[n + ".alpha"].float().reshape(())), put(curves[n]), put(curves[n + ".b"]))
        return self

    def weight_bytes(self) -> int:
        own = [self.embed, self.lm_head, self.pair_table] + [t for _, w, b in self.norms.values() for t in (w, b)]
        own += [t for pair in self.out_w.values() for t in pair]
        n = sum(t.numel() * t.element_size() for t in own if t is not None)
        return n + sum(t.numel() * t.element_size() for b in self._blocks() for t in b.tensors())

    def gemm_probe_widths(self):
        return None

    # ------------------------------------------------------------------ forward
    def forward(self, ids: torch.Tensor, meta: AttnMeta, kv: PagedKVCache,
                input_embeds: torch.Tensor | None = None) -> torch.Tensor:
        """ids [T] int32 -> final normed hidden [T, W] (model dtype)."""
        if input_embeds is not None:
            raise NotImplementedError("Gisirax: the token-pair embedding needs token ids")
        ctx = MixerCtx(meta, kv, meta.extra["ssm"])
        dt, norms = self.dtype, self.norms
        if self.pair:
            x = ops.pair_embedding_f32(ids, self.embed, self.embed_scale, self.pair_table, int(self.pair["buckets"]),
                                       int(self.pair["mul_prev"]), int(self.pair["mul_cur"]), self.prev_token, ctx.seqs)
        else:
            x = ops.embedding_f32(ids, self.embed, self.embed_scale)          # fp32 stream
        step: dict = {}                              # the sublayer output not yet added to x
        dbg = self.debug_residuals
        for i in range(len(self.specs)):
            h = ops.tanh_stream(x, norms[f"l{i}.norm1"], dt, **step)
            if dbg is not None and i:
                dbg.append(x.clone())
            y = self.mix[i].forward(h, ctx)
            step = dict(post=norms[f"l{i}.norm1b"], mult=self.mult)
            if i in self.out_w:
                step.update(y=y[0], y2=y[1], join=(*self.out_w[i], self.eps))
            else:
                step["y"] = y
            if i in self.ff:
                h = ops.tanh_stream(x, norms[f"l{i}.norm2"], dt, **step)
                step = dict(post=norms[f"l{i}.norm2b"], mult=self.mult, y=self.ff[i].forward(h))
        h = ops.tanh_stream(x, norms["final.norm"], dt, **step)
        if dbg is not None:
            dbg.append(x.clone())
        return h

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """fp32 logits ``head . hidden``."""
        return ops.lm_head_f32(hidden, self.lm_head)
