"""Gefilix decoder on the fp32-residual kernel set (``ops/res32.py``, ``csrc/kernels/res32``).

The residual stream x is fp32 and is normed AFTER every residual sum; the sublayers read x itself, as the rows h of the
activation type that the norm's kernel writes beside it.  A layer over the T rows of a step (decode rows and
prompt-portion rows alike):

    low-rank attention layer (models/latent.py):
      proj = h @ [Wq | Wg | Wdkv]^T                      ONE GEMM (Wg: one gate logit per head)
      cache <- [rms_norm(c) * w | rot(k_r)], c again as the value row           res32.latent_kv_write
      o    = softmax over the cached latents             queries absorbed, or keys / values up-projected (wide portions);
                                                         a layer with ``kv_from`` has no Wdkv and reads that layer's rows
      a    = o * sigmoid(proj_g) per head                res32.head_gate_rows (reads the batched product as it lies)
    lightning layer:
      proj = h @ [Wq | Wk | Wv | Wg]^T                   ONE GEMM
      o    = S <- a_h S + k v^T, S^T q over the slot     res32.lightning (silu of q, k, v inside; state fp32 [H, D, Dv])
      a    = o / rms(o) over all heads * w * sigmoid(proj_g)                    res32.head_norm_gate (one "head" of H Dv)
    x, h = rms_norm(alpha x + a @ Wo^T) * w1             res32.post_norm
    dense:   y = gelu(h @ Wup^T) @ Wdown^T               res32.gelu;  x, h = rms_norm(alpha x + y) * w2
    experts: z = h @ [Wrouter | Wsg]^T                   fp32: the router's logits and the shared expert's gate logit
             groups, top-k, weights                      res32.router (sigmoid scores)
             Y = clamped experts of the chosen rows      res32.expert_rows / grouped GEMMs + res32.glu
             x, h = rms_norm(alpha x + sum_j w_j Y_j + sigmoid(z_sg) shared(h)) * w2     res32.post_norm_experts

Logits = (rms_norm(x) * w) @ head^T; the embedding is scaled by ``embed_scale``.  ``dtype=torch.float32`` runs every
GEMM, activation and the cache in true fp32.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field
from typing import Dict, List, Optional

import torch

from .. import ops
from ..ops import res32
from .cache import PagedLayerCache
from .config import GefilixConfig, GeluFfSpec, GroupedExpertsSpec
from .latent import LatentDecoder, StepAttention, up
from .state import RecurrentStatePool


@dataclass
class GefilixLayer:
    norm1: torch.Tensor                  # fp32
    norm2: Optional[torch.Tensor]
    w_in: torch.Tensor                   # fused input-side projections of the mixer
    w_o: torch.Tensor
    extra: Dict[str, object] = field(default_factory=dict)


class GefilixModel(LatentDecoder):
    design = "Gefilix"

    def __init__(self, cfg: GefilixConfig, device="cuda", dtype=torch.bfloat16, seed: int = 0,
                 weights_path: Optional[str] = None, max_position: Optional[int] = None):
        self._setup(cfg, device, dtype)
        K = res32.kernels()
        for L in cfg.layer_specs:
            if L.type == "lightning" and L.mixer.dim > K.retention_max_dim():
                raise ValueError("Gefilix: lightning head size beyond what the kernel is built for")
            if L.type == "latent_attention" and up(L.mixer.kv_rank, 8) > 512:
                raise ValueError("Gefilix: kv_rank beyond what the attention kernels are built for")
            if isinstance(L.mlp, GroupedExpertsSpec) and L.mlp.experts > K.router_max_outputs():
                raise ValueError("Gefilix: too many router outputs")
        # layer -> index of its pages' views in the paged cache; a layer with kv_from shares its source's
        self.cache_index: Dict[int, int] = {}
        self.cache_layers: List[int] = []
        for i, L in enumerate(cfg.layer_specs):
            if L.type == "latent_attention":
                if L.mixer.kv_from is None:
                    self.cache_index[i] = len(self.cache_layers)
                    self.cache_layers.append(i)
                else:
                    self.cache_index[i] = self.cache_index[L.mixer.kv_from]
        self._assemble(self._read(weights_path) if weights_path else self._random(seed))

    # ------------------------------------------------------------------ weights
    def tensor_shapes(self) -> dict:
        """name -> shape of every tensor of a checkpoint of this config."""
        cfg, d = self.cfg, self.cfg.hidden
        out = {"embed": (cfg.vocab_size, d), "final.norm": (d,), "head": (cfg.vocab_size, d)}
        for i, L in enumerate(cfg.layer_specs):
            m, e, p = L.mixer, L.mlp, f"l{i}."
            out[p + "norm1"] = (d,)
            if L.type == "latent_attention":
                out[p + "mix.q"] = (m.nq, d)
                if m.kv_from is None:
                    out.update({p + "mix.dkv": (m.kv_rank + m.rot_dim, d), p + "mix.dkv.norm": (m.kv_rank,)})
                out.update({p + "mix.uk": (m.heads * m.dim, m.kv_rank), p + "mix.uv": (m.nv, m.kv_rank),
                            p + "mix.g": (m.heads, d), p + "mix.o": (d, m.nv)})
            else:
                out.update({p + "mix.q": (m.nq, d), p + "mix.k": (m.nq, d), p + "mix.v": (m.nv, d), p + "mix.g": (m.nv, d),
                            p + "mix.o": (d, m.nv), p + "mix.norm": (m.nv,)})
            if e is None:
                continue
            out[p + "norm2"] = (d,)
            if isinstance(e, GeluFfSpec):
                out.update({p + "mlp.up": (e.ff, d), p + "mlp.down": (d, e.ff)})
                continue
            out[p + "mlp.router"] = (e.experts, d)
            units = [(f"e{j}", e.ff) for j in range(e.experts)] + ([("shared", e.shared_ff)] if e.shared_ff else [])
            for name, ff in units:
                out.update({f"{p}mlp.{name}.gate": (ff, d), f"{p}mlp.{name}.up": (ff, d), f"{p}mlp.{name}.down": (d, ff)})
            if e.shared_ff:
                out[p + "mlp.shared.sg"] = (1, d)
        return out

    def _random(self, seed: int) -> dict:
        """Random weights of the config's shapes (benchmarks, tests): bf16-representable values."""
        g = torch.Generator(device="cpu")
        g.manual_seed(seed)
        d = self.cfg.hidden
        out = {}
        for name, shape in self.tensor_shapes().items():
            if len(shape) == 1:
                t = 1.0 + 0.1 * torch.randn(shape, generator=g)
            elif name == "embed":
                t = torch.randn(shape, generator=g) / math.sqrt(d)
            else:
                t = torch.randn(shape, generator=g) / math.sqrt(shape[1])
            out[name] = t.to(torch.bfloat16)
        return out

    def _assemble(self, sd: dict) -> None:
        cfg, dev, dt = self.cfg, self.device, self.dtype

        def t(name):
            return sd[name].to(device=dev, dtype=dt).contiguous()

        def f32(name):
            return sd[name].to(device=dev, dtype=torch.float32).contiguous()

        def gate_up(name):
            return torch.cat([t(name + ".gate"), t(name + ".up")], 0)

        self.embed, self.head, self.final_w = t("embed"), t("head"), f32("final.norm")
        self.layers: List[GefilixLayer] = []
        for i, L in enumerate(cfg.layer_specs):
            m, e, p = L.mixer, L.mlp, f"l{i}."
            x: Dict[str, object] = {}
            if L.type == "latent_attention":
                x["freq"], x["rot_mult"] = res32.rope_frequencies(m.rot.dims, m.rot.base, m.rot.scaling_dict(), dev)
                parts = [t(p + "mix.q"), t(p + "mix.g")]
                x["pad"] = up(m.nq + m.heads, 8) - m.nq - m.heads   # the latent's columns start on a 16-byte boundary
                if m.kv_from is None:
                    if x["pad"]:
                        parts.append(torch.zeros(x["pad"], cfg.hidden, dtype=dt, device=dev))
                    parts.append(t(p + "mix.dkv"))
                    x["dkv_norm"] = f32(p + "mix.dkv.norm")
                self._latent_weights(x, m, t(p + "mix.uk"), t(p + "mix.uv"))
            else:
                parts = [t(p + "mix." + n) for n in ("q", "k", "v", "g")]
                x["decay"] = torch.tensor(m.decay, dtype=torch.float32, device=dev)
                x["norm"] = f32(p + "mix.norm")
            if isinstance(e, GeluFfSpec):
                x["w_up"], x["w_down"] = t(p + "mlp.up"), t(p + "mlp.down")
            elif isinstance(e, GroupedExpertsSpec):
                rows = [f32(p + "mlp.router")] + ([f32(p + "mlp.shared.sg")] if e.shared_ff else [])
                self._router_weight(x, torch.cat(rows, 0).contiguous())
                x["w_gu"] = torch.stack([gate_up(f"{p}mlp.e{j}") for j in range(e.experts)]).contiguous()
                x["w_down"] = torch.stack([t(f"{p}mlp.e{j}.down") for j in range(e.experts)]).contiguous()
                if e.shared_ff:
                    x["ws_gu"], x["ws_down"] = gate_up(p + "mlp.shared").contiguous(), t(p + "mlp.shared.down")
            self.layers.append(GefilixLayer(norm1=f32(p + "norm1"), norm2=f32(p + "norm2") if e is not None else None,
                                            w_in=torch.cat(parts, 0).contiguous(), w_o=t(p + "mix.o"), extra=x))

    def _gemm_weights(self) -> list:
        ws = [w for L in self.layers for w in (L.w_in, L.w_o, L.extra.get("w_up"), L.extra.get("ws_gu"), L.extra.get("ws_down"))]
        return ws + [L.extra["w_down"] for L in self.layers if "w_up" in L.extra]

    def _head(self) -> torch.Tensor:
        return self.head

    # ------------------------------------------------------------------ cache and state
    def _layer_dims(self):
        return [self.latent_row_sizes(self.cfg.layer_specs[i].mixer) for i in self.cache_layers]

    def state_fields(self):
        """(name, shape) of every per-sequence state tensor: one matrix per lightning layer and head."""
        return [(f"S.{i}", (L.mixer.heads, L.mixer.dim, L.mixer.vdim)) for i, L in enumerate(self.cfg.layer_specs)
                if L.type == "lightning"]

    # ------------------------------------------------------------------ forward
    def _latent_mixer(self, h, L: GefilixLayer, m, li: int, positions, slots, cache, plan: StepAttention) -> torch.Tensor:
        x, ci = L.extra, self.cache_index[li]
        proj = self._linear(h, L.w_in)
        if m.kv_from is None:
            res32.latent_kv_write(proj[:, m.nq + m.heads + x["pad"]:], 0, m.kv_rank, m.rot_dim, None, x["dkv_norm"], x["freq"],
                                  x["rot_mult"], positions, slots, cache.k[ci], cache.v[ci], self.cfg.norm_eps)
        a = torch.empty(h.shape[0], m.nv, dtype=self.dtype, device=self.device)
        for rows, o in self._latent_attention(proj[:, :m.nq], x, m, ci, positions, cache, plan):
            res32.head_gate_rows(o, proj[rows, m.nq:m.nq + m.heads], a[rows])
        return a

    def _lightning_mixer(self, h, L: GefilixLayer, m, li: int, state, items) -> torch.Tensor:
        x = L.extra
        proj = self._linear(h, L.w_in)
        o = res32.lightning(proj, state[f"S.{li}"], x["decay"], items, m.heads)
        a = torch.empty(h.shape[0], m.nv, dtype=self.dtype, device=self.device)
        return res32.head_norm_gate(o, a, 1, self.cfg.norm_eps, w=x["norm"], gate=proj[:, 2 * m.nq + m.nv:], mode="sigmoid")

    def _feed_forward(self, x, h, L: GefilixLayer, e, cast) -> None:
        """x, cast <- the layer's second post-norm of the feed-forward's result."""
        w, eps, alpha = L.extra, self.cfg.norm_eps, self.cfg.alpha
        if isinstance(e, GeluFfSpec):
            y = self._linear(res32.gelu(self._linear(h, w["w_up"])), w["w_down"])
            res32.post_norm(x, y, alpha, L.norm2, eps, cast=cast)
            return
        z = self._router_logits(h, w)
        _ids, wts, row_off, src, row_expert, inv = res32.router(z[:, :e.experts], None, e.experts, e.top, renorm=True,
                                                                scores="sigmoid", floor=e.floor, scale=e.scale, groups=e.groups,
                                                                keep=e.keep)
        if self._use_grouped(self.cfg.hidden, e.ff):
            gu = ops.grouped_gemm(h, w["w_gu"], row_off, a_rows=src, rows=src.numel())
            Y = ops.grouped_gemm(res32.glu(gu, mode="clamped", alpha=e.alpha, limit=e.limit), w["w_down"], row_off)
        else:
            Y = res32.expert_rows(h, src, row_expert, row_off, w["w_gu"], w["w_down"], mode="clamped", alpha=e.alpha, limit=e.limit)
        shared = gate = None
        if e.shared_ff:
            act = res32.glu(self._linear(h, w["ws_gu"]), mode="clamped", alpha=e.alpha, limit=e.shared_limit)
            shared, gate = self._linear(act, w["ws_down"]), z[:, e.experts]
        res32.post_norm_experts(x, Y, inv, wts, h, alpha, L.norm2, eps, shared=shared, gate=gate, cast=cast)

    def _forward(self, tokens, positions, slots, cache: PagedLayerCache, state: RecurrentStatePool,
                 items: res32.StepItems, plan: StepAttention, keep: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Every layer over the step's rows; ``plan`` says how the rows reach the paged cache.  Returns the fp32 stream
        that the output norm reads, [T, d].

        ``keep`` (int64 rows): only these rows' final states are wanted (a prompt's last token).  The LAST layer then
        still runs its mixer on every row (the cached rows and the recurrent state are what later steps read) but the
        output projection and the feed-forward on the kept rows only; returns [len(keep), d]."""
        cfg, eps, n = self.cfg, self.cfg.norm_eps, len(self.layers)
        T, d, half = tokens.shape[0], self.cfg.hidden, self.dtype == torch.bfloat16
        # h: the stream as the GEMMs read it (fp32: the stream itself; every reader is done before it changes)
        h = torch.empty(T, d, dtype=self.dtype, device=self.device) if half else None
        x = res32.embed_rows(self.embed, tokens, scale=cfg.embed_scale, cast=h)
        for li, (S, L) in enumerate(zip(cfg.layer_specs, self.layers)):
            rows = h if half else x
            if S.type == "latent_attention":
                a = self._latent_mixer(rows, L, S.mixer, li, positions, slots, cache, plan)
            else:
                a = self._lightning_mixer(rows, L, S.mixer, li, state, items)
            if keep is not None and li + 1 == n:   # from here on only the kept rows
                a, x = a.index_select(0, keep), x.index_select(0, keep)
                h = torch.empty(x.shape[0], d, dtype=self.dtype, device=self.device) if half else None
            res32.post_norm(x, self._linear(a, L.w_o), cfg.alpha, L.norm1, eps, cast=h)
            if S.mlp is not None:
                self._feed_forward(x, h if half else x, L, S.mlp, h)
            if self.on_layer is not None:
                self.on_layer(li, x)
        return x
