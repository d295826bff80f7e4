"""What decoder designs with low-rank ("latent") attention share, with recurrent layers or without: the step functions over
the paged cache and the state slots, and the attention over cached latents (causal, or within a sliding window).

A low-rank attention layer caches ONE row per token for all heads, [latent c | rotated key part], and c again as the value
row.  Two ways to attend (``LatentDecoder._latent_attention``):

  * over the cached rows themselves: the keys' up-projection is applied to the query ("absorbed"), the values' to the
    result; decode rows always, prompt portions where the portion kernel takes the cached rows;
  * over keys and values up-projected per head from their sequences' cached rows into pages of their own: prompt portions
    whose cached rows are too wide for the portion kernel.

A layer may read rows that another layer cached: the caller names the cache layer, not the model layer.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from pathlib import Path
from typing import Callable, Dict, List, Optional, Tuple

import numpy as np
import torch
import torch.nn.functional as F

from .. import ops
from ..ops import gemm_plan, res32
from .cache import PagedLayerCache
from .state import RecurrentStatePool

UNBOUNDED = 1 << 30  # "window" of a causal attention without one


def up(n: int, m: int) -> int:
    return -(-n // m) * m


def adjacent_pairs(w: torch.Tensor, R: int, heads: int = 1) -> torch.Tensor:
    """Rows of a projection whose last R rows per head are rotated in "rotate half" pairs (i, i + R/2), reordered so that a
    pair is adjacent (2i, 2i + 1).  Applied to the query and the key side alike it changes no score."""
    o = w.view(heads, -1, w.shape[-1])
    n = o.shape[1] - R
    rot = o[:, n:].view(heads, 2, R // 2, -1).transpose(1, 2).reshape(heads, R, -1)
    return torch.cat([o[:, :n], rot], 1).reshape(w.shape).contiguous()


def core_size(n: int) -> int:
    """The next head size the matrix-core attention kernels are built for (beyond 128: a multiple of 8)."""
    for c in (32, 64, 128):
        if n <= c:
            return c
    return up(n, 8)


@dataclass
class StepAttention:
    """How a step's rows reach the paged cache: ``n_dec`` decode rows (row b reads ``dec_tables[b]``), then prompt
    portions described by ``chunk`` (block tables, row offsets, key counts; host copies of the counts in "lens")."""
    n_dec: int
    dec_tables: Optional[torch.Tensor]
    chunk: Optional[dict]
    scratch: Dict[object, object] = field(default_factory=dict)   # per-step data shared by the layer runs


class LatentDecoder:
    """Base of the designs: subclasses set ``cfg``, ``device``, ``dtype``, ``logit_width``, the weights, and implement
    ``tensor_shapes``, ``_layer_dims`` (cache rows), ``_forward``, ``_gemm_weights``, ``_head`` and, with recurrent layers,
    ``state_fields`` (without: ``has_state = False``, and the step functions take no state)."""

    paged_prefill = True      # whole prompts run as one portion over the paged cache (engine._run_prefill)
    supports_cascade = False
    graph_safe = True
    float_logits = True
    has_state = True          # the engine gives every sequence a recurrent-state slot
    design = "decoder"        # the design's name in error messages

    # experts at least this large (d * ff) go through the grouped matrix-core GEMMs of the full kernel extension
    GROUPED_MIN = 1 << 18

    def _setup(self, cfg, device, dtype) -> None:
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"{self.design} runs in bfloat16 or float32")
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        if self.device.type != "cuda":
            raise RuntimeError(f"{self.design} runs on the GPU kernels only (no CPU path)")
        if dtype == torch.float32:
            torch.backends.cuda.matmul.allow_tf32 = False
        self.logit_width = up(cfg.vocab_size, 32)
        self._mm32 = self._probe_mm32()
        self.g8_ws = None
        self.on_layer: Optional[Callable[[int, torch.Tensor], None]] = None
        self._zeros_h: Dict[int, torch.Tensor] = {}
        self._split_for: set = set()    # (M, N, K) whose split product was timed faster
        self._split_seen: set = set()

    # ------------------------------------------------------------------ weights
    def _read(self, path: str) -> dict:
        """The tensors of a checkpoint folder (or file), checked against ``tensor_shapes``."""
        from safetensors.torch import load_file

        p = Path(path)
        files = sorted(p.glob("*.safetensors")) if p.is_dir() else [p]
        if not files:
            raise FileNotFoundError(f"no .safetensors under {path}")
        sd = {}
        for f in files:
            sd.update(load_file(str(f), device="cpu"))
        for name, shape in self.tensor_shapes().items():
            if name not in sd:
                raise KeyError(f"{path}: tensor {name} missing")
            if tuple(sd[name].shape) != tuple(shape):
                raise ValueError(f"{path}: {name} has shape {tuple(sd[name].shape)}, the config says {tuple(shape)}")
        return sd

    def _latent_weights(self, x: Dict[str, object], m, uk: torch.Tensor, uv: torch.Tensor) -> None:
        """The up-projections of a low-rank attention layer in the layouts that ``_latent_attention`` reads."""
        x["w_uk"] = uk.view(m.heads, m.dim, m.kv_rank)                                          # [H, D, C]
        x["w_uv_t"] = uv.view(m.heads, m.vdim, m.kv_rank).transpose(1, 2).contiguous()          # [H, C, Dv]
        if self.expanded_head_sizes(m) is not None:
            x["w_ukv"] = torch.cat([uk, uv], 0).contiguous()

    # ------------------------------------------------------------------ GEMMs
    def _probe_mm32(self) -> bool:
        """Whether this torch build multiplies bf16 matrices into an fp32 result (router logits, absorbed queries)."""
        if self.dtype != torch.bfloat16:
            return False
        try:
            a = torch.zeros(2, 8, 16, dtype=self.dtype, device=self.device)
            b = torch.zeros(2, 16, 8, dtype=self.dtype, device=self.device)
            return (torch.mm(a[0], a[0].t(), out_dtype=torch.float32).dtype == torch.float32
                    and torch.bmm(a, b, out_dtype=torch.float32).dtype == torch.float32)
        except (TypeError, RuntimeError):
            return False

    def _linear(self, x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
        if self.g8_ws is not None:
            return gemm_plan.linear(x, w, ws=self.g8_ws)
        return F.linear(x, w)

    def _bmm32(self, a: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
        """Batched a @ b with an fp32 result."""
        if self.dtype == torch.float32:
            return torch.bmm(a, b)
        if self._mm32:
            return torch.bmm(a, b, out_dtype=torch.float32)
        return torch.bmm(a.float(), b.float())

    def _router_weight(self, x: Dict[str, object], w: torch.Tensor) -> None:
        """Router rows (fp32 [NE, d]): also kept as a bf16 operand when that holds them exactly."""
        x["router"] = w
        if self._mm32 and bool((w.to(self.dtype).float() == w).all()):
            x["router_t"] = w.to(self.dtype).t().contiguous()

    def _router_logits(self, h: torch.Tensor, x: Dict[str, object]) -> torch.Tensor:
        if "router_t" in x:   # bf16 operands, fp32 accumulation AND output
            return torch.mm(h, x["router_t"], out_dtype=torch.float32)
        return F.linear(h.float(), x["router"])

    def _use_grouped(self, d: int, ff: int) -> bool:
        """Whether experts of these sizes run on the grouped matrix-core GEMMs."""
        return self.dtype == torch.bfloat16 and d * ff >= self.GROUPED_MIN and d % 64 == 0 and ff % 64 == 0 and ops.available()

    # Few rows against a long reduction (a feed-forward's down projection in a decode step) leave most CUs idle in one GEMM:
    # such a weight is kept a second time as S slices of the reduction [S, K / S, N] (S = 4, or 8 for at most 2048 outputs),
    # run as ONE batched GEMM with fp32 partial products that the consumer adds up.  Which row counts take it is timed (tune_gemms).
    SPLIT_ROWS, SPLIT_MIN_K = 256, 4096

    def split_weight(self, w: torch.Tensor) -> Optional[torch.Tensor]:
        """``w`` [N, K] in slices of the reduction, [S, K / S, N] (None where the split does not apply)."""
        N, K = w.shape
        S = 4 if N > 2048 else 8
        if not self._mm32 or K < self.SPLIT_MIN_K or K % (8 * S) or N % 8:
            return None
        return w.t().contiguous().view(S, K // S, N)

    @staticmethod
    def _split_product(x: torch.Tensor, ws: torch.Tensor) -> torch.Tensor:
        S, Ks, _ = ws.shape
        return torch.bmm(x.view(x.shape[0], S, Ks).transpose(0, 1), ws, out_dtype=torch.float32)

    def _linear_parts(self, x: torch.Tensor, w: torch.Tensor, ws: Optional[torch.Tensor]) -> torch.Tensor:
        """x @ w^T as rows [M, N], or as fp32 partial products [S, M, N] where the split was timed faster for this M."""
        if ws is not None and (x.shape[0], *w.shape) in self._split_for:
            return self._split_product(x, ws)
        return self._linear(x, w)

    def _tune_split(self, M: int, w: torch.Tensor, ws: Optional[torch.Tensor]) -> None:
        key = (M, *w.shape)
        if ws is None or M > self.SPLIT_ROWS or key in self._split_seen:
            return
        self._split_seen.add(key)
        x = torch.randn(M, w.shape[1], device=self.device).to(self.dtype)
        t = {"one": [], "split": []}
        for _ in range(5):
            t["one"].append(gemm_plan._time(lambda: self._linear(x, w), iters=5, rounds=1))
            t["split"].append(gemm_plan._time(lambda: self._split_product(x, ws), iters=5, rounds=1))
        if sorted(t["split"])[2] < sorted(t["one"])[2]:
            self._split_for.add(key)

    def tune_gemms(self, M: int, bucket: bool = False, lm_head: bool = True, only=None) -> None:
        """Pick the backend of the projections at M rows by timing the library and the hand-written cores (the engine
        calls this before it captures a decode bucket's graph).  bf16 only, and only where the full kernel extension is
        built; otherwise every GEMM stays on the library."""
        if self.dtype != torch.bfloat16 or only is not None or not ops.available():
            return
        if self.g8_ws is None:
            self.g8_ws = ops.new_gemm8p_workspace(self.device)
        seen = set()
        for w in self._gemm_weights() + ([self._head()] if lm_head else []):
            if w is not None and tuple(w.shape) not in seen and w.shape[0] % 8 == 0 and w.shape[1] % 8 == 0:
                seen.add(tuple(w.shape))
                gemm_plan.tune(torch.randn(M, w.shape[1], device=self.device).to(self.dtype), w, ws=self.g8_ws, bucket=bucket)
        for w, ws in self._split_weights():
            self._tune_split(M, w, ws)

    def _split_weights(self) -> list:
        """(weight, its split form or None) of the projections that :meth:`_linear_parts` runs."""
        return []

    # ------------------------------------------------------------------ cache and state
    def latent_row_sizes(self, m) -> Tuple[int, int]:
        """(key row, value row) sizes of a low-rank attention layer's cached token: [latent | rotated part] and the
        latent, padded with zeros.  bf16: up to the next size the matrix-core attention kernels are built for (32, 64,
        128; 192 / 128; one wide row of 320 / 256 or 576 / 512), else to a multiple of 8 (16-byte rows).  A wide row is
        taken where it pads at most by half (latents far below it stay on the general kernel)."""
        nk, nv = m.kv_rank + m.rot_dim, m.kv_rank
        if self.dtype == torch.bfloat16:
            if nk <= 128:
                return core_size(nk), core_size(nv)
            for rk, rv in ((192, 128), (320, 256)):
                if nk <= rk and nv <= rv and 2 * rk <= 3 * up(nk, 8):
                    return rk, rv
            if 288 < nk <= 576 and nv <= 512:
                return 576, 512
        return up(nk, 8), up(nv, 8)

    def expanded_head_sizes(self, m) -> Optional[Tuple[int, int]]:
        """(key, value) sizes per head of the up-projected keys [unrotated | rotated part] and values that prompt
        portions attend over when the cached rows themselves are too wide for the portion kernel; None: not used."""
        K = res32.kernels()
        if self.dtype != torch.bfloat16 or K.window_attn_mfma_ok(*self.latent_row_sizes(m)):
            return None
        dk = core_size(m.dim + m.rot_dim) if m.dim + m.rot_dim <= 128 else up(m.dim + m.rot_dim, 64)
        dv = core_size(m.vdim)
        return (dk, dv) if K.window_attn_mfma_ok(dk, dv) else None

    def new_cache(self, num_blocks: int, block_size: int) -> PagedLayerCache:
        return PagedLayerCache(self._layer_dims(), num_blocks, block_size, self.device, self.dtype)

    def bytes_per_block(self, block_size: int) -> int:
        n = PagedLayerCache.elems_per_block(self._layer_dims(), block_size) * (4 if self.dtype == torch.float32 else 2)
        return max(n, 16)

    def new_state(self, num_slots: int) -> RecurrentStatePool:
        return RecurrentStatePool(self.state_fields(), num_slots, self.device)

    def bytes_per_state_slot(self) -> int:
        return RecurrentStatePool.bytes_per_slot(self.state_fields())

    # ------------------------------------------------------------------ attention over the paged cache
    def _no_bias(self, H: int) -> torch.Tensor:
        z = self._zeros_h.get(H)
        if z is None:
            z = self._zeros_h[H] = torch.zeros(H, dtype=torch.float32, device=self.device)
        return z

    def _paged_attention(self, q: torch.Tensor, positions: torch.Tensor, cache: PagedLayerCache, ci: int, plan: StepAttention,
                         out: torch.Tensor, H: int, G: int, window: Optional[int] = None, cap: float = 0.0,
                         sink: Optional[torch.Tensor] = None, values_in_keys: bool = False) -> torch.Tensor:
        """Softmax attention of a step's rows (fp32 ``q`` [n, H * key size]; decode rows first, then portion rows if ``n``
        reaches them) over cache layer ``ci`` into ``out`` [n, H * value size]."""
        n, n_dec = q.shape[0], plan.n_dec
        z, kc, vc, win = self._no_bias(H), cache.k[ci], cache.v[ci], UNBOUNDED if window is None else window
        if n_dec:
            res32.window_attn(q[:n_dec], kc, vc, positions[:n_dec], plan.dec_tables, z, z, win, out[:n_dec], H, G, cores=True,
                              sink=sink, values_in_keys=values_in_keys, cap=cap)
        if n > n_dec:
            ch = plan.chunk
            res32.window_attn(q[n_dec:], kc, vc, positions[n_dec:], ch["block_tables"], z, z, win, out[n_dec:], H, G, cu_q=ch["cu_q"],
                              k_lens=ch.get("k_lens"), max_q=int(ch.get("max_q", 0)), cores=True, sink=sink, cap=cap)
        return out

    def _latent_attention(self, q: torch.Tensor, x: Dict[str, object], m, ci: int, positions, cache: PagedLayerCache,
                          plan: StepAttention, sink: Optional[torch.Tensor] = None) -> List[Tuple[slice, torch.Tensor]]:
        """Attention of a step's rows: ``q`` [T, H (D + R)] (row-dense columns are fine) as projected, over the rows of
        cache layer ``ci``.  Returns [(rows, o [n, H, Dv])]: the heads' results of these rows, in whatever strides they
        come (a batched product's transpose, padded heads)."""
        T, dt = q.shape[0], self.dtype
        C, R, D, H, Dv = m.kv_rank, m.rot_dim, m.dim, m.heads, m.vdim
        Dk, Cv = self.latent_row_sizes(m)
        n_dec = plan.n_dec
        wide = T > n_dec and self.expanded_head_sizes(m) is not None and cache.block_size & (cache.block_size - 1) == 0
        n_abs = n_dec if wide else T   # rows that attend over the cached latent rows themselves
        out: List[Tuple[slice, torch.Tensor]] = []
        if n_abs:
            qa, pa = q[:n_abs], positions[:n_abs]
            qn = self._bmm32(qa.view(n_abs, H, D + R)[:, :, :D].transpose(0, 1), x["w_uk"])  # [H, n, C]: keys' up-projection on q
            qf = res32.latent_q_rows(qa, D, R, qn, x["freq"], x["rot_mult"], m.scale, pa, H, Dk).view(n_abs, H * Dk)
            oc = torch.empty(n_abs, H * Cv, dtype=dt, device=self.device)
            self._paged_attention(qf, pa, cache, ci, plan, oc, H, 1, window=m.window, sink=sink, values_in_keys=True)
            o = torch.bmm(oc.view(n_abs, H, Cv)[:, :, :C].transpose(0, 1), x["w_uv_t"])      # [H, n, Dv]
            out.append((slice(0, n_abs), o.transpose(0, 1)))
        if wide:
            out.append((slice(n_dec, T), self._expanded_attention(q[n_dec:], positions[n_dec:], x, m, ci, cache, plan, sink)))
        return out

    def _context_rows(self, plan: StepAttention, bs: int, window: Optional[int] = None) -> dict:
        """For the prompt portions of a step: where every token that their rows may see lies in the paged cache (the whole
        sequences, or with ``window`` from the page of the first portion row's first key on), and a dense page numbering of
        those tokens, sequence after sequence (built once per step and window).  Tables are indexed by position as usual;
        entries of pages before the first visible key are not read."""
        ctx = plan.scratch.get(("ctx", window))
        if ctx is None:
            ch = plan.chunk
            q_lens, k_lens = (np.asarray(ch["lens"][i], dtype=np.int64) for i in (0, 1))
            lo = np.zeros_like(k_lens)
            if window is not None:   # (the portion kernel walks tiles of 32 keys from a multiple of 32 on)
                align = max(bs, 32)
                lo = np.maximum(k_lens - q_lens - window + 1, 0) // align * align
            skip, last = lo // bs, -(-k_lens // bs)
            first = np.concatenate([[0], np.cumsum(last - skip)])
            item = np.repeat(np.arange(len(k_lens)), k_lens - lo)
            pos = np.concatenate([np.arange(a, n) for a, n in zip(lo, k_lens)]) if len(k_lens) else np.zeros(0, np.int64)
            dev = self.device
            item_d, pos_d = torch.from_numpy(item).to(dev), torch.from_numpy(pos).to(dev)
            blk = ch["block_tables"][item_d, pos_d // bs].long()
            tables = np.zeros((len(k_lens), max(1, int(last.max()))), np.int32)
            for i in range(len(k_lens)):
                tables[i, skip[i]:last[i]] = first[i] + np.arange(last[i] - skip[i])
            ctx = plan.scratch[("ctx", window)] = {
                "blk": blk, "off": pos_d % bs, "slots": torch.from_numpy((first[item] - skip[item]) * bs + pos).to(dev),
                "tables": torch.from_numpy(tables).to(dev), "pages": int(first[-1])}
        return ctx

    def _expanded_attention(self, q, positions, x, m, ci: int, cache: PagedLayerCache, plan: StepAttention, sink) -> torch.Tensor:
        """Prompt portions over keys and values up-projected from the cached latents of their sequences: per head the
        key [W_uk c | rotated part] and the value W_uv c, laid out as pages of their own for the portion kernel."""
        Tq, bs = q.shape[0], cache.block_size
        C, R, D, H, Dv = m.kv_rank, m.rot_dim, m.dim, m.heads, m.vdim
        dk, dv = self.expanded_head_sizes(m)
        ctx = self._context_rows(plan, bs, m.window)
        rows = plan.scratch.get(("rows", ci, m.window))                            # [N, row]: latent | rotated part
        if rows is None:   # (a later layer that reads the same cached rows finds them gathered)
            rows = plan.scratch[("rows", ci, m.window)] = cache.k[ci][ctx["blk"], ctx["off"]]
        kv = F.linear(rows[:, :C], x["w_ukv"])                                     # [N, H D + H Dv]
        key = ("pages", H * dk, H * dv, ctx["pages"])
        tmp = plan.scratch.get(key)
        if tmp is None:
            tmp = plan.scratch[key] = PagedLayerCache([(H * dk, H * dv)], ctx["pages"], bs, self.device, self.dtype)
        res32.latent_expand_write(kv, rows, C, R, ctx["slots"], tmp.k[0], tmp.v[0], H, D, Dv)
        qf = res32.latent_q_rows(q, D, R, None, x["freq"], x["rot_mult"], m.scale, positions, H, dk)
        out = torch.empty(Tq, H * dv, dtype=self.dtype, device=self.device)
        ch, z = plan.chunk, self._no_bias(H)
        res32.window_attn(qf.view(Tq, H * dk), tmp.k[0], tmp.v[0], positions, ctx["tables"], z, z,
                          UNBOUNDED if m.window is None else m.window, out, H, H,
                          cu_q=ch["cu_q"], k_lens=ch["k_lens"], max_q=int(ch["max_q"]), cores=True, sink=sink)
        return out.view(Tq, H, dv)[:, :, :Dv]

    # ------------------------------------------------------------------ step functions
    def _output_rows(self, x, rows: Optional[torch.Tensor]) -> torch.Tensor:
        """What the output weights read: the output norm of what ``_forward`` returned, optionally of ``rows`` only."""
        return res32.rmsnorm_rows(x, self.final_w, self.cfg.norm_eps, self.dtype, rows=rows)

    def _logits(self, x, rows: Optional[torch.Tensor], float_logits: bool) -> torch.Tensor:
        lg = self._linear(self._output_rows(x, rows), self._head()).float()
        if float_logits:
            return lg
        V, Vp = self.cfg.vocab_size, self.logit_width
        if Vp == V:
            return lg.to(torch.bfloat16)
        out = torch.full((lg.shape[0], Vp), float("-inf"), dtype=torch.bfloat16, device=lg.device)
        out[:, :V] = lg
        return out

    def decode(self, tokens: torch.Tensor, positions: torch.Tensor, slots: torch.Tensor, block_tables: torch.Tensor,
               ctx_lens: torch.Tensor, cache: PagedLayerCache, num_splits: int = 1, cascade_tiles=None,
               float_logits: bool = False, state: Optional[RecurrentStatePool] = None,
               state_slots: Optional[torch.Tensor] = None) -> torch.Tensor:
        """One decode step for B sequences -> logits [B, V]; device tensors only (hipGraph-capturable).  Row b
        reads table row b and the state slot ``state_slots[b]``; its key range ends at its own position."""
        items = None
        if self.has_state:
            if state is None or state_slots is None:
                raise RuntimeError(f"{self.design}: a decode step needs the recurrent-state pool and the rows' slots")
            items = res32.StepItems.rows(state_slots, positions)
        x = self._forward(tokens, positions, slots, cache, state, items, StepAttention(tokens.shape[0], block_tables, None))
        return self._logits(x, None, float_logits)

    def forward_mixed(self, tokens: torch.Tensor, positions: torch.Tensor, slots: torch.Tensor, cache: PagedLayerCache,
                      n_dec: int, dec: Optional[dict], chunk: Optional[dict], logit_rows: torch.Tensor,
                      float_logits: bool = False, state: Optional[RecurrentStatePool] = None,
                      state_slots: Optional[torch.Tensor] = None) -> torch.Tensor:
        """ONE forward over [n_dec decode rows || prompt-portion rows]: every projection is one GEMM over both, the
        recurrence walks decode rows and portions alike as items; the attention runs per part over the paged cache
        that this step's rows were just written to.  ``state_slots``: int32, the slot of every decode row, then of
        every portion (designs without recurrent layers: no state, no slots).  Logits of ``logit_rows``."""
        T = tokens.shape[0]
        items = self._step_items(chunk, T, n_dec, positions, state, state_slots) if self.has_state else None
        plan = StepAttention(n_dec, dec["block_tables"] if n_dec else None, chunk if T > n_dec else None)
        keep = logit_rows if n_dec == 0 and self.on_layer is None and 4 * logit_rows.numel() <= T else None
        x = self._forward(tokens, positions, slots, cache, state, items, plan, keep=keep)
        return self._logits(x, None if keep is not None else logit_rows, float_logits)

    def _step_items(self, chunk, T: int, n_dec: int, positions, state, state_slots) -> res32.StepItems:
        """The step's rows grouped by sequence for the recurrent layers: decode rows, then portions."""
        if state is None or state_slots is None:
            raise RuntimeError(f"{self.design}: a step needs the recurrent-state pool and the sequences' slots")
        q_lens = list(chunk["lens"][0]) if T > n_dec else []
        cu = np.concatenate([np.arange(n_dec, dtype=np.int64), n_dec + np.concatenate([[0], np.cumsum(q_lens, dtype=np.int64)])])
        if cu[-1] != T or state_slots.numel() != n_dec + len(q_lens):
            raise ValueError(f"{self.design}: rows, portions and state slots disagree")
        row_item = np.concatenate([np.arange(n_dec, dtype=np.int64), n_dec + np.repeat(np.arange(len(q_lens)), q_lens)])
        dev = self.device
        return res32.StepItems(torch.from_numpy(row_item.astype(np.int32)).to(dev), torch.from_numpy(cu.astype(np.int32)).to(dev),
                               state_slots, positions)

    def prefill(self, tokens, positions, slots, cu_seqlens, max_seqlen, last_idx, cache, ctx=None):
        raise RuntimeError(f"{self.design} prefills through forward_mixed over the paged cache (paged_prefill)")
