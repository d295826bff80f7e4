"""Limatar decoder on the fp32-residual kernel set (``ops/res32.py``, ``csrc/kernels/res32``).

The residual stream x is fp32; every norm is x / rms(x) * (1 + w) (the stored weights are offsets from one, the sum
is formed once at load).  A layer run over the T rows of a step (decode rows and prompt-portion rows alike):

    h      = norm1(x)                                   res32.rmsnorm_rows
    low-rank attention layer:
      proj = h @ [Wdq | Wdkv | Wg]^T                     ONE GEMM
      cq   = rms_norm(proj_dq) * w;  cache <- [rms_norm(c) * w | rot(k_r)] and c again as the value row
                                                         res32.latent_kv_write (one cached row serves every head)
      q    = cq @ Wuq^T                                  GEMM
      qf   = [ (q_unrotated Wuk) * scale | rot(q_r) * scale ]   batched GEMM per head + res32.latent_q_rows: the keys'
                                                         up-projection is applied to the query, so scores are taken
                                                         against the cached latent itself
      o_c  = softmax with a sink over the cache          res32.window_attn (G = 1: all heads read the one cached row)
      a    = (o_c Wuv^T per head) * sigmoid(proj_g)      batched GEMM + res32.gate_mul
      (bf16, cached rows wider than the portion kernel takes: prompt portions instead attend per head over keys
       [Wuk c | rotated part] and values Wuv c up-projected from their sequences' cached rows into pages of their own,
       res32.latent_expand_write; decode rows stay on the cached rows)
    retention layer:
      proj = h @ [Wq | Wk | Wv | Wg]^T                   ONE GEMM
      o    = S <- a_h S + k v^T, S^T q over the slot     res32.retention (rotation of q, k inside; state fp32 [H, D, Dv])
      a    = o / rms(o) per head * silu(proj_g)          res32.head_norm_gate
    x     += norm1b(a @ Wo^T);  h2 = norm2(x)            res32.gated_norm_residual (no gate; both norms in one pass)
    dense:   y = (glu_clamped(h2 @ [Wgate | Wup]^T)) @ Wdown^T             res32.glu
    experts: top-k of the router's logits + bias, softmax over the chosen  res32.router (fp32)
             y = sum_j s_j expert_j(h2) + shared(h2)                       res32.expert_rows / grouped GEMMs, moe_combine
    x     += norm2b(y);  h = the next run's norm1(x)     res32.gated_norm_residual

``cfg.runs`` lists the layer of every run: a looped span repeats in a row with the same weights, and every run has its
own pages in the paged cache (attention) or its own matrix in the recurrent-state slots (retention).
Logits = norm(x) @ embed^T (tied).  ``dtype=torch.float32`` runs every GEMM, activation and the cache in true fp32.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field
from typing import Dict, List, Optional

import torch

from .. import ops
from ..ops import res32
from .cache import PagedLayerCache
from .config import ClampedGluSpec, LimatarConfig, TopkExpertsSpec
from .latent import LatentDecoder, StepAttention, up
from .state import RecurrentStatePool


@dataclass
class LimatarLayer:
    norm1: torch.Tensor                  # fp32, 1 + w
    norm1b: torch.Tensor
    norm2: Optional[torch.Tensor]
    norm2b: Optional[torch.Tensor]
    w_in: torch.Tensor                   # fused input-side projections of the mixer
    w_o: torch.Tensor
    extra: Dict[str, torch.Tensor] = field(default_factory=dict)


class LimatarModel(LatentDecoder):
    design = "Limatar"

    def __init__(self, cfg: LimatarConfig, device="cuda", dtype=torch.bfloat16, seed: int = 0,
                 weights_path: Optional[str] = None, max_position: Optional[int] = None):
        self._setup(cfg, device, dtype)
        K = res32.kernels()
        for L in cfg.layer_specs:
            if L.type == "retention" and L.mixer.dim > K.retention_max_dim():
                raise ValueError("Limatar: retention head size beyond what the kernel is built for")
            if L.type == "latent_attention" and up(L.mixer.kv_rank, 8) > 512:
                raise ValueError("Limatar: kv_rank beyond what the attention kernels are built for")
            if isinstance(L.mlp, TopkExpertsSpec) and L.mlp.experts > K.router_max_outputs():
                raise ValueError("Limatar: too many router outputs")
        self.runs = cfg.runs
        # run -> index of its pages' views in the paged cache (attention runs only)
        self.cache_index = {}
        for ri, li in enumerate(self.runs):
            if cfg.layer_specs[li].type == "latent_attention":
                self.cache_index[ri] = len(self.cache_index)
        self._assemble(self._read(weights_path) if weights_path else self._random(seed))

    # ------------------------------------------------------------------ weights
    def tensor_shapes(self) -> dict:
        """name -> shape of every tensor of a checkpoint of this config."""
        cfg, d = self.cfg, self.cfg.hidden
        out = {"embed": (cfg.vocab_size, d), "embed.norm": (d,), "final.norm": (d,)}
        for i, L in enumerate(cfg.layer_specs):
            m, p = L.mixer, f"l{i}."
            out.update({p + "norm1": (d,), p + "norm1b": (d,)})
            if L.type == "latent_attention":
                out.update({p + "mix.dq": (m.q_rank, d), p + "mix.dq.norm": (m.q_rank,), p + "mix.uq": (m.nq, m.q_rank),
                            p + "mix.dkv": (m.kv_rank + m.rot_dim, d), p + "mix.dkv.norm": (m.kv_rank,),
                            p + "mix.uk": (m.heads * m.dim, m.kv_rank), p + "mix.uv": (m.nv, m.kv_rank),
                            p + "mix.sink": (m.heads,), p + "mix.g": (m.nv, d), p + "mix.o": (d, m.nv)})
            else:
                out.update({p + "mix.q": (m.nq, d), p + "mix.k": (m.nq, d), p + "mix.v": (m.nv, d), p + "mix.g": (m.nv, d),
                            p + "mix.o": (d, m.nv)})
            e = L.mlp
            if e is not None:
                out.update({p + "norm2": (d,), p + "norm2b": (d,)})
            if isinstance(e, ClampedGluSpec):
                out.update({p + "mlp.gate": (e.ff, d), p + "mlp.up": (e.ff, d), p + "mlp.down": (d, e.ff)})
            elif isinstance(e, TopkExpertsSpec):
                out.update({p + "mlp.router": (e.experts, d), p + "mlp.router.b": (e.experts,)})
                for x in range(e.experts):
                    out.update({f"{p}mlp.e{x}.gate": (e.ff, d), f"{p}mlp.e{x}.up": (e.ff, d), f"{p}mlp.e{x}.down": (d, e.ff)})
                if e.shared_ff:
                    out.update({p + "mlp.shared.gate": (e.shared_ff, d), p + "mlp.shared.up": (e.shared_ff, d),
                                p + "mlp.shared.down": (d, e.shared_ff)})
        return out

    def _random(self, seed: int) -> dict:
        """Random weights of the config's shapes (benchmarks, tests): bf16-representable values."""
        g = torch.Generator(device="cpu")
        g.manual_seed(seed)
        d = self.cfg.hidden
        out = {}
        for name, shape in self.tensor_shapes().items():
            leaf = name.split(".")[-1]
            if leaf in ("norm1", "norm2", "norm1b", "norm2b") or name in ("final.norm", "embed.norm"):
                t = 0.1 * torch.randn(shape, generator=g)            # stored around zero
            elif leaf == "norm":
                t = 1.0 + 0.1 * torch.randn(shape, generator=g)      # the latents' plain weights
            elif leaf == "sink":
                t = torch.randn(shape, generator=g)
            elif leaf == "b":
                t = 0.1 * torch.randn(shape, generator=g)
            elif name == "embed":
                t = torch.randn(shape, generator=g)
            else:
                t = torch.randn(shape, generator=g) / math.sqrt(shape[-1] if len(shape) > 1 else d)
            out[name] = t.to(torch.bfloat16)
        return out

    def _assemble(self, sd: dict) -> None:
        cfg, dev, dt = self.cfg, self.device, self.dtype

        def t(name):
            return sd[name].to(device=dev, dtype=dt).contiguous()

        def f32(name):
            return sd[name].to(device=dev, dtype=torch.float32).contiguous()

        def one_plus(name):
            return (1.0 + f32(name)).contiguous()

        self.embed = t("embed")
        self.embed_norm, self.final_w = one_plus("embed.norm"), one_plus("final.norm")
        self.layers: List[LimatarLayer] = []
        for i, L in enumerate(cfg.layer_specs):
            m, p = L.mixer, f"l{i}."
            x: Dict[str, torch.Tensor] = {}
            x["freq"], x["rot_mult"] = res32.rope_frequencies(m.rot.dims, m.rot.base, m.rot.scaling_dict(), dev)
            if L.type == "latent_attention":
                w_in = torch.cat([t(p + "mix.dq"), t(p + "mix.dkv"), t(p + "mix.g")], 0).contiguous()
                x["dq_norm"], x["dkv_norm"], x["sink"] = f32(p + "mix.dq.norm"), f32(p + "mix.dkv.norm"), f32(p + "mix.sink")
                x["w_uq"] = t(p + "mix.uq")
                self._latent_weights(x, m, t(p + "mix.uk"), t(p + "mix.uv"))
            else:
                w_in = torch.cat([t(p + "mix.q"), t(p + "mix.k"), t(p + "mix.v"), t(p + "mix.g")], 0).contiguous()
                x["decay"] = torch.tensor(m.decay, dtype=torch.float32, device=dev)
            e = L.mlp
            if isinstance(e, ClampedGluSpec):
                x["w_gu"] = torch.cat([t(p + "mlp.gate"), t(p + "mlp.up")], 0).contiguous()
                x["w_down"] = t(p + "mlp.down")
            elif isinstance(e, TopkExpertsSpec):
                self._router_weight(x, f32(p + "mlp.router"))
                x["router_b"] = f32(p + "mlp.router.b")
                x["w_gu"] = torch.stack([torch.cat([t(f"{p}mlp.e{j}.gate"), t(f"{p}mlp.e{j}.up")], 0)
                                         for j in range(e.experts)]).contiguous()
                x["w_down"] = torch.stack([t(f"{p}mlp.e{j}.down") for j in range(e.experts)]).contiguous()
                if e.shared_ff:
                    x["ws_gu"] = torch.cat([t(p + "mlp.shared.gate"), t(p + "mlp.shared.up")], 0).contiguous()
                    x["ws_down"] = t(p + "mlp.shared.down")
            has = e is not None
            self.layers.append(LimatarLayer(norm1=one_plus(p + "norm1"), norm1b=one_plus(p + "norm1b"),
                                            norm2=one_plus(p + "norm2") if has else None,
                                            norm2b=one_plus(p + "norm2b") if has else None, w_in=w_in, w_o=t(p + "mix.o"),
                                            extra=x))

    def _gemm_weights(self) -> list:
        ws = [w for L in self.layers for w in (L.w_in, L.w_o, L.extra.get("w_uq"), L.extra.get("ws_gu"), L.extra.get("ws_down"))]
        return ws + [L.extra[k] for L in self.layers for k in ("w_gu", "w_down") if k in L.extra and L.extra[k].dim() == 2]

    def _head(self) -> torch.Tensor:
        return self.embed

    # ------------------------------------------------------------------ cache and state
    def _layer_dims(self):
        return [self.latent_row_sizes(self.cfg.layer_specs[self.runs[ri]].mixer) for ri in sorted(self.cache_index)]

    def state_fields(self):
        """(name, shape) of every per-sequence state tensor: one retention matrix set per retention RUN."""
        out = []
        for ri, li in enumerate(self.runs):
            L = self.cfg.layer_specs[li]
            if L.type == "retention":
                out.append((f"S.{ri}", (L.mixer.heads, L.mixer.dim, L.mixer.vdim)))
        return out

    # ------------------------------------------------------------------ forward
    def _latent_mixer(self, h, L: LimatarLayer, m, ri: int, positions, slots, cache, plan: StepAttention) -> torch.Tensor:
        x, T, dt = L.extra, h.shape[0], self.dtype
        C, R, H, ci = m.kv_rank, m.rot_dim, m.heads, self.cache_index[ri]
        proj = self._linear(h, L.w_in)
        cq = res32.latent_kv_write(proj, m.q_rank, C, R, x["dq_norm"], x["dkv_norm"], x["freq"], x["rot_mult"], positions,
                                   slots, cache.k[ci], cache.v[ci], self.cfg.norm_eps)
        q = self._linear(cq, x["w_uq"])                                            # [T, H (D + R)]
        a = torch.empty(T, H * m.vdim, dtype=dt, device=self.device)
        for rows, o in self._latent_attention(q, x, m, ci, positions, cache, plan, sink=x["sink"]):
            a[rows].view(-1, H, m.vdim).copy_(o)
        res32.gate_mul(a, proj[:, m.q_rank + C + R:], "sigmoid")
        return a

    def _retention_mixer(self, h, L: LimatarLayer, m, ri: int, state, items) -> torch.Tensor:
        x, T = L.extra, h.shape[0]
        proj = self._linear(h, L.w_in)
        nq, nv = m.nq, m.nv
        o = res32.retention(proj, nq, proj[:, 2 * nq:2 * nq + nv], x["freq"], x["rot_mult"], m.rot.dims, x["decay"],
                            state[f"S.{ri}"], items, m.heads)
        a = torch.empty(T, nv, dtype=self.dtype, device=self.device)
        res32.head_norm_gate(o, a, m.heads, self.cfg.norm_eps, w=None, gate=proj[:, 2 * nq + nv:], mode="silu")
        return a

    def _feed_forward(self, h2: torch.Tensor, L: LimatarLayer, e) -> torch.Tensor:
        x = L.extra
        if isinstance(e, ClampedGluSpec):
            act = res32.glu(self._linear(h2, x["w_gu"]), mode="clamped", alpha=e.alpha, limit=e.limit)
            return self._linear(act, x["w_down"])
        z = self._router_logits(h2, x)
        _ids, w, row_off, src, row_expert, inv = res32.router(z, None, e.experts, e.top, bias=x["router_b"], renorm=True)
        if self._use_grouped(self.cfg.hidden, e.ff):
            gu = ops.grouped_gemm(h2, x["w_gu"], row_off, a_rows=src, rows=src.numel())
            Y = ops.grouped_gemm(res32.glu(gu), x["w_down"], row_off)
        else:
            Y = res32.expert_rows(h2, src, row_expert, row_off, x["w_gu"], x["w_down"])
        shared = None
        if e.shared_ff:
            shared = self._linear(res32.glu(self._linear(h2, x["ws_gu"])), x["ws_down"])
        return res32.moe_combine(Y, inv, w, h2, add=shared)

    def _forward(self, tokens, positions, slots, cache: PagedLayerCache, state: RecurrentStatePool,
                 items: res32.StepItems, plan: StepAttention, keep: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Every layer run over the step's rows; ``plan`` says how the rows reach the paged cache.
        Returns the fp32 stream that the output norm reads, [T, d].

        ``keep`` (int64 rows): only these rows' final states are wanted (a prompt's last token).  The LAST run then
        still runs its mixer on every row (the cached rows and the recurrent state are what later steps read) but the
        output projection and the feed-forward on the kept rows only; returns [len(keep), d]."""
        cfg, dt, eps = self.cfg, self.dtype, self.cfg.norm_eps
        x = res32.rmsnorm_rows(res32.embed_rows(self.embed, tokens), self.embed_norm, eps, torch.float32)
        n = len(self.runs)
        h = res32.rmsnorm_rows(x, self.layers[self.runs[0]].norm1, eps, dt) if n else None
        for ri, li in enumerate(self.runs):
            S, L = cfg.layer_specs[li], self.layers[li]
            if S.type == "latent_attention":
                a = self._latent_mixer(h, L, S.mixer, ri, positions, slots, cache, plan)
            else:
                a = self._retention_mixer(h, L, S.mixer, ri, state, items)
            last = ri + 1 == n
            if keep is not None and last:   # from here on only the kept rows
                a, x = a.index_select(0, keep), x.index_select(0, keep)
            nxt = None if last else self.layers[self.runs[ri + 1]].norm1
            y = self._linear(a, L.w_o)
            if S.mlp is not None:
                h2 = self._add_norm(x, y, L.norm1b, L.norm2)
                h = self._add_norm(x, self._feed_forward(h2, L, S.mlp), L.norm2b, nxt)
            else:
                h = self._add_norm(x, y, L.norm1b, nxt)
            if self.on_layer is not None:
                self.on_layer(ri, x)
        return x

    def _add_norm(self, x: torch.Tensor, y: torch.Tensor, w: torch.Tensor, next_w: Optional[torch.Tensor]):
        """x += y / rms(y) * w; returns the next sublayer's input x / rms(x) * next_w (None without ``next_w``): one
        pass over the stream in bf16 (the new x stays in registers between the two norms)."""
        eps = self.cfg.norm_eps
        if next_w is None:
            res32.gated_norm_residual(x, y, w, eps)
            return None
        if self.dtype == torch.bfloat16:
            h = torch.empty(x.shape[0], x.shape[1], dtype=self.dtype, device=self.device)
            res32.gated_norm_residual(x, y, w, eps, x_cast=h, next_w=next_w)
            return h
        res32.gated_norm_residual(x, y, w, eps)
        return res32.rmsnorm_rows(x, next_w, eps, self.dtype)
