"""Pagatar: a layer-list decoder (``architecture: Pagatar``) whose sublayers read the raw stream, are
normed on their OUTPUT in groups of channels, and whose layers pass on a learned average over depth.

``layers[i]`` = {``type``, ``mixer`` (that mixer's own sizes), ``mlp`` (or null)}.  Mixer types:

* ``attention`` -- ``mixers.ConvRotaryAttention`` with biased projections, per-head q / k norms
  before the (half-split, YaRN-scaled) rotation, chunked mask, element-wise output gate and value
  mixing with the first layer whose ``mixer.v_mix`` is set;
* ``latent_attention`` -- ``mixers.LatentAttention``, full causal, interleaved rotary pairs, no
  sink, one output gate per head;
* ``mingru`` -- ``mixers.MinGruMixer``.

Feed-forward (``mlp.kind: moe``): ``mixers.GroupRoutedMoE`` as one group of SiLU-GLU experts, chosen
by sigmoid score + correction and weighted by the plain score.

With G(y) w the norm in ``norm.groups`` equal parts, X_0 = G(embed[token]) ``embed.norm`` and x = X_0,
layer i computes

  x += G(mixer(x)) norm1;   x += G(ff(x)) norm2          (no ``mlp``: the first half only)
  X_{i+1} = x;   x = sum_{j <= i+1} dwa_i[j] X_j

and logits = ``embed`` . (G(x) ``final.norm``): the embedding table is the head.

Numerics: x and every X_j are fp32 (``ops.stream_step``: norm of the sublayer's output, residual
sum, depth average and the one rounding of the next GEMM's input in one launch); convolution sums,
q / k norms, rotary angles, attention scores / softmax, router logits and scores, minGRU gates and
state are fp32 inside the kernels; logits leave the head in fp32.  The depth history [layers + 1, T,
W] lives for one step.  Prefix caching is off (``stateful``).  The model has no cache, loop over
steps or scheduler of its own: ``ModelRunner`` drives it like the other layer-list designs.
"""
from __future__ import annotations

import torch

from ome_amd import ops
from ome_amd.models.common import AttnMeta, PagedKVCache
from ome_amd.models.config import ModelConfig
from ome_amd.models.llama import LlamaForCausalLM
from ome_amd.models.mixers import ConvRotaryAttention, GroupRoutedMoE, LatentAttention, MinGruMixer, MixerCtx
from ome_amd.parallel import state as pstate

PAGATAR_ARCHS = {"Pagatar"}


class PagatarForCausalLM(LlamaForCausalLM):
    stateful = True
    tune_gemms = False   # odd projection widths: the library heuristic, no TunableOp pass

    def __init__(self, cfg: ModelConfig, device="cuda", dtype=torch.bfloat16, max_positions: int | None = None):
        st = pstate.get()
        if st.tp_size > 1 or st.pp_size > 1:
            raise NotImplementedError("Pagatar: tensor / pipeline parallelism (one GPU holds the model)")
        super().__init__(cfg, device, dtype, 1)   # (the base's rotary table is unused: one row)
        hf = cfg.extra or {}
        W, eps = cfg.hidden_size, cfg.rms_norm_eps
        mp = max_positions or cfg.max_position_embeddings
        self.groups = int(hf["norm"].get("groups", 1))
        if self.groups < 1 or W % self.groups:
            raise ValueError(f"norm.groups {self.groups} does not divide the width {W}")
        self.specs = list(hf["layers"])
        L = len(self.specs)
        lat = [s["mixer"] for s in self.specs if s["type"] == "latent_attention"]
        # key rows that carry their values (the latent kernel, bf16) when every latent layer's width has a
        # kernel shape, else key rows + value columns of the generic kernels
        self.latent_cache = dtype == torch.bfloat16 and bool(lat) and all(ops.latent_shape(m["kv_rank"], m["rot_dim"])
                                                                          for m in lat)
        self.mix: list[ConvRotaryAttention | LatentAttention | MinGruMixer] = []
        self.ff: dict[int, GroupRoutedMoE] = {}
        first = None                                       # the layer whose values the later v_mix layers mix in
        for i, spec in enumerate(self.specs):
            m, kind = spec["mixer"], spec["type"]
            rot = m.get("rot") or {}
            if kind == "attention":
                mixes = None
                if m.get("v_mix"):
                    if first is not None and first.nv != m["kv_heads"] * m["vdim"]:
                        raise ValueError(f"layer {i}: {m['kv_heads']} x {m['vdim']} values cannot mix with layer "
                                         f"{first.layer}'s {first.nv}")
                    mixes = "first" if first is None else "mix"
                self.mix.append(ConvRotaryAttention(
                    i, W, m["heads"], m["kv_heads"], m["dim"], m["vdim"], (m.get("mask") or {}).get("size", 0),
                    m.get("conv", 0), rot.get("base", 10000.0), rot.get("dims", 0), m["scale"], eps, mp, self.device,
                    dtype, interleaved=False, unit_norm=False, rot_scaling=rot.get("scaling"), chunked=True, bias=True,
                    head_norm=True, sink=False, gated=True, v_mix=mixes))
                if mixes == "first":
                    first = self.mix[-1]
            elif kind == "latent_attention":
                if int(rot.get("dims", m["rot_dim"])) != int(m["rot_dim"]):
                    raise ValueError(f"layer {i}: rot.dims {rot.get('dims')} != rot_dim {m['rot_dim']}")
                self.mix.append(LatentAttention(
                    i, i, W, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"],
                    rot.get("base", 10000.0), rot.get("scaling"), m["scale"], eps, mp, self.device, dtype,
                    self.latent_cache, sink=False, gated="head", interleaved=True))
            elif kind == "mingru":
                self.mix.append(MinGruMixer(W, m["width"], self.device, dtype))
            else:
                raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
            f = spec.get("mlp")
            if f:
                if f.get("kind", "moe") != "moe":
                    raise ValueError(f"layer {i}: unknown feed-forward kind {f.get('kind')!r}")
                self.ff[i] = GroupRoutedMoE(W, f["router"]["experts"], f["router"]["top"], f["expert"]["ff"], 0.0, 1, 1,
                                            0, 0.0, self.device, dtype, act=0, scoring="sigmoid")
        self.embed_norm = None
        self.dwa: list = [None] * L                        # fp32 [i + 2] per layer
        kv = {i: b for i, b in enumerate(self.mix) if not isinstance(b, MinGruMixer)}
        rows_only = {i for i, b in kv.items() if isinstance(b, LatentAttention) and b.latent_cache}
        self.kv_layers = sorted(kv)
        self.kv_heads_per_layer = {i: 1 if isinstance(b, LatentAttention) else b.Hkv for i, b in kv.items()}
        self.kv_dims_per_layer = {i: b.D for i, b in kv.items()}
        # (a latent layer's key rows carry their values: no value array)
        self.kv_value_dim = {i: 0 if i in rows_only else b.D for i, b in kv.items()}
        # fewest kv heads among the layers that run the split-K decode kernel (layers on the latent kernel
        # bring their own workspace): the runner partitions its decode workspace by it
        self.decode_ws_kv_heads = min((self.kv_heads_per_layer[i] for i in kv if i not in rows_only), default=None)
        self.debug_residuals: list | None = None   # set to []: the stream after every layer is appended

    def prefill_item_rows(self, page: int) -> int:
        """Query rows per prefill work item: one plan serves all attention layers, so the 64-row
        item needs every layer that reads the plan to have the shape its kernel is built for."""
        rows = set()
        for a in self.mix:
            if isinstance(a, ConvRotaryAttention):
                rows.add(ops.prefill_rows(a.Hq, a.Hkv, a.D, page))
            elif isinstance(a, LatentAttention) and not a.latent_cache:
                rows.add(ops.prefill_rows(a.H, 1, a.D, page) if a.H <= LatentAttention.HEAD_GROUP else 32)
        return rows.pop() if len(rows) == 1 else 32

    def _blocks(self):
        yield from self.mix
        yield from self.ff.values()

    def alloc_state(self, slots: int) -> None:
        for b in self.mix:
            b.alloc_state(slots)

    # ------------------------------------------------------------------ weights
    def init_random(self, seed: int = 0, std: float = 0.02) -> "PagatarForCausalLM":
        gen = torch.Generator(device=self.device)
        gen.manual_seed(seed)
        W, V = self.cfg.hidden_size, self.cfg.vocab_size
        for i in range(len(self.specs)):
            self.ln1[i] = self._alloc(W, std=None, gen=gen)
            if i in self.ff:
                self.ln2[i] = self._alloc(W, std=None, gen=gen)
            w = torch.full((i + 2,), 0.1, dtype=torch.float32, device=self.device)
            w[-1] = 1.0
            self.dwa[i] = w
        for b in self._blocks():
            b.init_random(gen, std)
        self.embed = self._alloc(V, W, std=std, gen=gen)
        self.embed_norm = self._alloc(W, std=None, gen=gen)
        self.norm = self._alloc(W, std=None, gen=gen)
        self.lm_head = self.embed
        return self

    def load_hf_weights(self, weights) -> "PagatarForCausalLM":
        put = lambda w: w.to(device=self.device, dtype=self.dtype).contiguous()   # noqa: E731
        top = {"embed": "embed", "embed.norm": "embed_norm", "final.norm": "norm"}
        per_layer = {"norm1": self.ln1, "norm2": self.ln2}
        groups: dict[tuple[int, str], dict[str, torch.Tensor]] = {}
        for name, w in weights:
            if name in top:
                setattr(self, top[name], put(w))
            elif name.startswith("l") and "." in name:
                head, rest = name.split(".", 1)
                if not head[1:].isdigit() or int(head[1:]) >= len(self.specs):
                    continue
                i = int(head[1:])
                if rest in per_layer:
                    per_layer[rest][i] = put(w)
                elif rest == "dwa":
                    self.dwa[i] = w.reshape(-1).to(device=self.device, dtype=torch.float32).contiguous()
                else:
                    for pre in ("mix.", "mlp."):
                        if rest.startswith(pre):
                            groups.setdefault((i, pre), {})[rest[len(pre):]] = w
                            break
        for i in range(len(self.specs)):
            for kind, b in (("mix.", self.mix[i]), ("mlp.", self.ff.get(i))):
                if b is None:
                    continue
                try:
                    b.load(groups.get((i, kind), {}))
                except KeyError as e:
                    raise ValueError(f"checkpoint incomplete: l{i}.{kind}{e.args[0]} is missing") from None
        n = range(len(self.specs))
        missing = [k for k, v in (("embed", self.embed), ("embed.norm", self.embed_norm), ("final.norm", self.norm))
                   if v is None]
        missing += [f"l{i}.norm1" for i in n if self.ln1[i] is None] + [f"l{i}.norm2" for i in self.ff if self.ln2[i] is None]
        missing += [f"l{i}.dwa" for i in n if self.dwa[i] is None]
        if missing:
            raise ValueError(f"checkpoint incomplete: {', '.join(missing[:6])} missing")
        for i in n:
            if self.dwa[i].numel() != i + 2:
                raise ValueError(f"l{i}.dwa: {self.dwa[i].numel()} coefficients, {i + 2} expected")
        self.lm_head = self.embed
        return self

    def weight_bytes(self) -> int:
        own = [self.embed, self.embed_norm, self.norm] + self.ln1 + self.ln2 + self.dwa
        n = sum(t.numel() * t.element_size() for t in own if t is not None)
        return n + sum(t.numel() * t.element_size() for b in self._blocks() for t in b.tensors())

    def gemm_probe_widths(self):
        return None

    # ------------------------------------------------------------------ forward
    def forward(self, ids: torch.Tensor, meta: AttnMeta, kv: PagedKVCache,
                input_embeds: torch.Tensor | None = None) -> torch.Tensor:
        """ids [T] int32 -> final normed hidden [T, W] (model dtype)."""
        ctx = MixerCtx(meta, kv, meta.extra["ssm"])
        eps, dt, G = self.eps, self.dtype, self.groups
        T, W, L = ids.shape[0], self.cfg.hidden_size, len(self.specs)
        hist = torch.empty(L + 1, T, W, dtype=torch.float32, device=ids.device)   # X_0 .. X_L
        x = torch.empty(T, W, dtype=torch.float32, device=ids.device)
        if input_embeds is None:
            h = ops.stream_step(self.embed, self.embed_norm, G, eps, ids=ids, hist=hist, k=0, out_dtype=dt)
        else:
            h = ops.stream_step(input_embeds, self.embed_norm, G, eps, hist=hist, k=0, out_dtype=dt)
        cur = hist[0]
        dbg = self.debug_residuals
        for i in range(L):
            y = self.mix[i].forward(h, ctx)
            w = self.ln1[i]
            if i in self.ff:      # (the sum after the mixer rests in the history entry the layer's result will take)
                h = ops.stream_step(y, w, G, eps, res=cur, x_out=hist[i + 1], out_dtype=dt)
                y, w, cur = self.ff[i].forward(h), self.ln2[i], hist[i + 1]
            h = ops.stream_step(y, w, G, eps, res=cur, hist=hist, k=i + 1, coef=self.dwa[i], x_out=x,
                                out_dtype=dt if i + 1 < L else None)
            cur = x
            if dbg is not None:
                dbg.append(x.clone())
        return ops.stream_step(cur, self.norm, G, eps, out_dtype=dt)

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        """fp32 logits ``embed . hidden``."""
        return ops.lm_head_f32(hidden, self.lm_head)
