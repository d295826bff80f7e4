"""Semuzen decoder on the fp32-residual kernel set (``ops/res32.py``, ``csrc/kernels/res32``).

The residual is S parallel fp32 streams X[s].  Every sublayer reads u = sum_s in_s X_s through an elementwise norm
dyt(u) = tanh(a u) * w + b, and its result y enters all streams at once, X_t <- sum_s mix[s, t] X_s + out_t y.  Neither
needs a statistic over the row, so what lies between two sublayers is ONE elementwise pass (``res32.hyper_step``): the
streams' update, the next sublayer's u and its norm.  A layer over the T rows of a step (decode rows and prompt-portion
rows alike):

    windowed low-rank attention layer (models/latent.py):
      proj = h @ [Wq | Wdkv]^T                           ONE GEMM (rotated rows reordered at load: pairs adjacent)
      cache <- [rms_norm(c) * w | rot(k_r)], c again as the value row           res32.latent_kv_write
      a    = softmax over the window's cached latents    queries absorbed, or keys / values up-projected (wide portions)
    attention layer:
      proj = h @ [Wq | Wk | Wv | Wg]^T                   ONE GEMM; a layer with ``kv_from`` has no Wk and Wv
      q    = rot(rms_norm(proj_q + b) over all heads) * scale;  cache <- rot(rms_norm(proj_k + b)), proj_v + b
                                                         res32.norm_rot_kv_write (heads padded to the kernels' sizes)
      o    = softmax of softcap * tanh(s / softcap) over the cache (a layer with ``kv_from``: that layer's)   res32.window_attn
      a    = o * sigmoid(proj_g)                         res32.head_gate_rows (reads the padded heads as they lie)
    X, h = update with a @ Wo^T (+ the output bias), next u, next norm          res32.hyper_step
    y    = relu(h @ Wup^T)^2 @ Wdown^T                   res32.relu2
    X, h = update with y, next u, next norm              res32.hyper_step

The embedding is scaled, goes through a norm of its own and starts every stream (``res32.embed_streams``); the output reads
the streams' sum (a step whose in-weights are ones) through ``final.norm``: logits = dyt(sum_t X_t) @ head^T.  A step's last
update only forms the rows whose logits are wanted and does not store the streams.  ``dtype=torch.float32`` runs every GEMM,
activation and the cache in true fp32.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple

import torch

from ..ops import res32
from .cache import PagedLayerCache
from .config import CappedAttentionSpec, SemuzenConfig
from .latent import LatentDecoder, StepAttention, adjacent_pairs, core_size, up


@dataclass
class SemuzenLayer:
    w_in: torch.Tensor                   # fused input-side projections of the mixer
    w_o: torch.Tensor
    w_up: Optional[torch.Tensor] = None
    w_down: Optional[torch.Tensor] = None
    w_down_split: Optional[torch.Tensor] = None
    extra: Dict[str, object] = field(default_factory=dict)


@dataclass
class StreamUpdate:
    """What follows a sublayer: the coefficients of its update and of the next reader's input, and that reader's norm."""
    coef: torch.Tensor
    norm: res32.Dyt
    bias: Optional[torch.Tensor] = None


class SemuzenModel(LatentDecoder):
    design = "Semuzen"
    has_state = False   # everything a sequence carries is in the paged cache

    def __init__(self, cfg: SemuzenConfig, device="cuda", dtype=torch.bfloat16, seed: int = 0,
                 weights_path: Optional[str] = None, max_position: Optional[int] = None):
        self._setup(cfg, device, dtype)
        if cfg.streams > res32.kernels().hyper_max_streams():
            raise ValueError("Semuzen: more streams than the kernels are built for")
        for L in cfg.layer_specs:
            if L.type == "latent_attention" and up(L.mixer.kv_rank, 8) > 512:
                raise ValueError("Semuzen: kv_rank beyond what the attention kernels are built for")
            if L.type == "attention" and L.mixer.vdim > 512:
                raise ValueError("Semuzen: vdim beyond what the attention kernels are built for")
        # layer -> index of its pages' views in the paged cache; a layer with kv_from shares its source's
        self.cache_index: Dict[int, int] = {}
        self.cache_layers: List[int] = []
        for i, L in enumerate(cfg.layer_specs):
            if L.mixer.kv_from is None:
                self.cache_index[i] = len(self.cache_layers)
                self.cache_layers.append(i)
            else:
                self.cache_index[i] = self.cache_index[L.mixer.kv_from]
        self._assemble(self._read(weights_path) if weights_path else self._random(seed))

    # ------------------------------------------------------------------ weights
    def tensor_shapes(self) -> dict:
        """name -> shape of every tensor of a checkpoint of this config."""
        cfg, d, S = self.cfg, self.cfg.hidden, self.cfg.streams
        out = {"embed": (cfg.vocab_size, d), "head": (cfg.vocab_size, d)}

        def norm(name):
            out.update({name: (d,), name + ".b": (d,), name + ".alpha": ()})

        norm("embed.norm")
        norm("final.norm")
        for i, L in enumerate(cfg.layer_specs):
            m, p = L.mixer, f"l{i}."
            for n in ("1", "2") if L.mlp is not None else ("1",):
                norm(p + "norm" + n)
                out.update({f"{p}hc{n}.in": (S,), f"{p}hc{n}.out": (S,), f"{p}hc{n}.mix": (S, S)})
            out[p + "mix.q"] = (m.nq, d)
            if L.type == "latent_attention":
                out.update({p + "mix.dkv": (m.kv_rank + m.rot_dim, d), p + "mix.dkv.norm": (m.kv_rank,),
                            p + "mix.uk": (m.heads * m.dim, m.kv_rank), p + "mix.uv": (m.nv, m.kv_rank), p + "mix.o": (d, m.nv)})
            else:
                out.update({p + "mix.q.b": (m.nq,), p + "mix.q.norm": (m.nq,), p + "mix.g": (m.no, d), p + "mix.o": (d, m.no),
                            p + "mix.o.b": (d,)})
                if m.kv_from is None:
                    out.update({p + "mix.k": (m.nk, d), p + "mix.k.b": (m.nk,), p + "mix.k.norm": (m.nk,), p + "mix.v": (m.nv, d),
                                p + "mix.v.b": (m.nv,)})
            if L.mlp is not None:
                out.update({p + "mlp.up": (L.mlp.ff, d), p + "mlp.down": (d, L.mlp.ff)})
        return out

    def _random(self, seed: int) -> dict:
        """Random weights of the config's shapes (benchmarks, tests): bf16-representable values."""
        g = torch.Generator(device="cpu")
        g.manual_seed(seed)
        S = self.cfg.streams
        out = {}
        for name, shape in self.tensor_shapes().items():
            leaf = name.split(".")[-1]
            if leaf == "mix":
                t = torch.eye(S) + 0.1 * torch.randn(shape, generator=g)
            elif leaf in ("in", "out"):
                t = 1.0 / S + 0.1 * torch.randn(shape, generator=g) if leaf == "in" else 1.0 + 0.1 * torch.randn(shape, generator=g)
            elif leaf == "alpha":
                t = torch.tensor(0.5)
            elif leaf == "b":
                t = 0.05 * torch.randn(shape, generator=g)
            elif len(shape) == 1:
                t = 1.0 + 0.1 * torch.randn(shape, generator=g)
            elif name == "embed":
                t = torch.randn(shape, generator=g)
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

        def dyt(name):
            return res32.Dyt(float(sd[name + ".alpha"].float()), f32(name), f32(name + ".b"))

        self.embed, self.head = t("embed"), t("head")
        self.embed_norm = dyt("embed.norm")
        self.layers: List[SemuzenLayer] = []
        subs: List[str] = []                  # the sublayers' tensor suffixes in order
        for i, L in enumerate(cfg.layer_specs):
            m, p = L.mixer, f"l{i}."
            x: Dict[str, object] = {}
            x["freq"], x["rot_mult"] = res32.rope_frequencies(m.rot.dims, m.rot.base, m.rot.scaling_dict(), dev) if m.rot.dims else (None, 1.0)
            if L.type == "latent_attention":
                x["pad"] = up(m.nq, 8) - m.nq   # the latent's columns start on a 16-byte boundary
                parts = [adjacent_pairs(t(p + "mix.q"), m.rot_dim, m.heads), torch.zeros(x["pad"], cfg.hidden, dtype=dt, device=dev),
                         adjacent_pairs(t(p + "mix.dkv"), m.rot_dim)]
                x["dkv_norm"] = f32(p + "mix.dkv.norm")
                self._latent_weights(x, m, t(p + "mix.uk"), t(p + "mix.uv"))
            else:
                own = m.kv_from is None
                parts = [t(p + "mix." + n) for n in (("q", "k", "v") if own else ("q",))]
                x["cols"] = sum(w.shape[0] for w in parts)
                x["pad"] = up(x["cols"], 8) - x["cols"]
                parts += [torch.zeros(x["pad"], cfg.hidden, dtype=dt, device=dev), t(p + "mix.g")]
                x["bias"] = torch.cat([f32(f"{p}mix.{n}.b") for n in (("q", "k", "v") if own else ("q",))]).contiguous()
                x["wq"], x["wk"] = f32(p + "mix.q.norm"), f32(p + "mix.k.norm") if own else None
                x["bias_o"] = f32(p + "mix.o.b")
            lay = SemuzenLayer(w_in=torch.cat(parts, 0).contiguous(), w_o=t(p + "mix.o"), extra=x)
            subs.append(p + "{}1")
            if L.mlp is not None:
                lay.w_up, lay.w_down = t(p + "mlp.up"), t(p + "mlp.down")
                lay.w_down_split = self.split_weight(lay.w_down)
                subs.append(p + "{}2")
            self.layers.append(lay)
        ones = torch.ones(cfg.streams, dtype=torch.float32, device=dev)
        norms = [dyt(s.format("norm")) for s in subs] + [dyt("final.norm")]
        ins = [f32(s.format("hc") + ".in") for s in subs] + [ones]
        self.first_in, self.first_norm = ins[0], norms[0]
        self.updates: List[Tuple[StreamUpdate, Optional[StreamUpdate]]] = []   # per layer: behind the mixer, behind the feed-forward
        k = 0
        for L, lay in zip(cfg.layer_specs, self.layers):
            ups: List[Optional[StreamUpdate]] = []
            for _ in range(1 if L.mlp is None else 2):
                hc = subs[k].format("hc")
                ups.append(StreamUpdate(res32.hyper_coef(f32(hc + ".mix"), f32(hc + ".out"), ins[k + 1]), norms[k + 1],
                                        None if ups else lay.extra.get("bias_o")))
                k += 1
            self.updates.append((ups[0], ups[1] if len(ups) > 1 else None))

    def _gemm_weights(self) -> list:
        return [w for L in self.layers for w in (L.w_in, L.w_o, L.w_up, L.w_down)]

    def _split_weights(self) -> list:
        return [(L.w_down, L.w_down_split) for L in self.layers if L.w_down is not None]

    def _head(self) -> torch.Tensor:
        return self.head

    # ------------------------------------------------------------------ cache
    def attention_row_sizes(self, m: CappedAttentionSpec) -> Tuple[int, int]:
        """(key, value) sizes per head in the cache: bf16 heads are padded with zeros to the next sizes that the matrix-core
        attention kernels are built for (up to 192 / 128), else as they are."""
        if self.dtype == torch.bfloat16 and m.vdim <= 128 and m.dim <= 192:
            return core_size(m.dim) if m.dim <= 128 else 192, core_size(m.vdim)
        return m.dim, m.vdim

    def _layer_dims(self):
        out = []
        for i in self.cache_layers:
            m = self.cfg.layer_specs[i].mixer
            if isinstance(m, CappedAttentionSpec):
                dk, dv = self.attention_row_sizes(m)
                out.append((m.kv_heads * dk, m.kv_heads * dv))
            else:
                out.append(self.latent_row_sizes(m))
        return out

    # ------------------------------------------------------------------ forward
    @staticmethod
    def _kept_plan(keep: torch.Tensor, plan: StepAttention) -> StepAttention:
        """The attention of a few of a step's portion rows alone: each reads its own sequence's pages like a decode row."""
        item = torch.bucketize(keep, plan.chunk["cu_q"][1:].to(torch.int64), right=True)
        return StepAttention(keep.numel(), plan.chunk["block_tables"].index_select(0, item), None)

    def _latent_mixer(self, h, L: SemuzenLayer, m, li: int, positions, slots, cache, plan: StepAttention, keep) -> torch.Tensor:
        x, ci = L.extra, self.cache_index[li]
        proj = self._linear(h, L.w_in)
        res32.latent_kv_write(proj[:, m.nq + x["pad"]:], 0, m.kv_rank, m.rot_dim, None, x["dkv_norm"], x["freq"], x["rot_mult"],
                              positions, slots, cache.k[ci], cache.v[ci], self.cfg.norm_eps)
        q = proj[:, :m.nq]
        if keep is not None:
            q, positions, plan = q.index_select(0, keep), positions.index_select(0, keep), self._kept_plan(keep, plan)
        parts = self._latent_attention(q, x, m, ci, positions, cache, plan)
        if len(parts) == 1 and parts[0][1].is_contiguous():
            return parts[0][1].view(q.shape[0], m.nv)
        a = torch.empty(q.shape[0], m.nv, dtype=self.dtype, device=self.device)
        for rows, o in parts:
            a[rows].view(-1, m.heads, m.vdim).copy_(o)
        return a

    def _attention_mixer(self, h, L: SemuzenLayer, m, li: int, positions, slots, cache, plan: StepAttention, keep) -> torch.Tensor:
        x, ci, H, G = L.extra, self.cache_index[li], m.heads, m.kv_heads
        dk, dv = self.attention_row_sizes(m)
        proj = self._linear(h, L.w_in)
        own = dict(k_cache=cache.k[ci], v_cache=cache.v[ci], G=G, Dv=m.vdim) if m.kv_from is None else {}
        q = res32.norm_rot_kv_write(proj[:, :x["cols"]], positions, slots, H, m.dim, dk, m.scale, eps=self.cfg.norm_eps, wq=x["wq"],
                                    wk=x["wk"], bias=x["bias"], rot_dims=m.rot.dims, freq=x["freq"], mult=x["rot_mult"], **own)
        gate = proj[:, x["cols"] + x["pad"]:]
        if keep is not None:
            q, gate, positions, plan = (q.index_select(0, keep), gate.index_select(0, keep), positions.index_select(0, keep),
                                        self._kept_plan(keep, plan))
        n = q.shape[0]
        o = torch.empty(n, H * dv, dtype=self.dtype, device=self.device)
        self._paged_attention(q.view(n, H * dk), positions, cache, ci, plan, o, H, G, cap=m.softcap)
        a = torch.empty(n, m.no, dtype=self.dtype, device=self.device)
        return res32.head_gate_rows(o.view(n, H, dv)[:, :, :m.vdim], gate, a)

    def _forward(self, tokens, positions, slots, cache: PagedLayerCache, state, items, plan: StepAttention,
                 keep: Optional[torch.Tensor] = None):
        """Every layer over the step's rows; ``plan`` says how the rows reach the paged cache.  Returns what the output needs:
        (streams before the last update, the last sublayer's result, that update).

        ``keep`` (int64 rows): only these rows' final states are wanted (a prompt's last token).  The LAST layer then still
        projects every row and writes its keys and values (later steps read them), but attends, and runs everything behind,
        on the kept rows only; the result holds these rows."""
        cfg, n, dt = self.cfg, len(self.layers), self.dtype
        X, h = res32.embed_streams(self.embed, tokens, cfg.embed_scale, self.embed_norm, self.first_in, self.first_norm)
        y = u = None
        for li, (S, L) in enumerate(zip(cfg.layer_specs, self.layers)):
            few = keep if li + 1 == n else None
            mixer = self._latent_mixer if S.type == "latent_attention" else self._attention_mixer
            y = self._linear(mixer(h, L, S.mixer, li, positions, slots, cache, plan, few), L.w_o)
            if few is not None:
                X = X.index_select(1, keep)
            u, ff = self.updates[li]
            if ff is not None:
                h = res32.hyper_step(X, y, u.coef, u.norm, dt, bias=u.bias)
                y, u = self._linear_parts(res32.relu2(self._linear(h, L.w_up)), L.w_down, L.w_down_split), ff
            if li + 1 < n:
                h = res32.hyper_step(X, y, u.coef, u.norm, dt, bias=u.bias)
            if self.on_layer is not None:
                self.on_layer(li, self._stream_sum(X, y, u) if li + 1 == n else X.sum(0))
        return X, y, u

    @staticmethod
    def _stream_sum(X: torch.Tensor, y: torch.Tensor, u: StreamUpdate) -> torch.Tensor:
        """The streams' sum behind an update that the forward pass leaves to the output rows (for ``on_layer``)."""
        X = X.clone()
        res32.hyper_step(X, y, u.coef, u.norm, y.dtype, bias=u.bias)
        return X.sum(0)

    def _output_rows(self, x, rows: Optional[torch.Tensor]) -> torch.Tensor:
        X, y, u = x
        return res32.hyper_step(X, y, u.coef, u.norm, self.dtype, bias=u.bias, rows=rows, write=False)
