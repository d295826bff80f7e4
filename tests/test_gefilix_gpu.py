"""Gefilix on the GPU against the plain fp64 oracle (tests/gefilix_oracle.py): each mechanism alone, then the model
through the engine — whole prompts, token-by-token decoding, portions, unequal batches, pages and state slots used
again, the first tokens of a sequence, keys far away and at page borders, long decoding, layers that read another
layer's latents and greedy generation through the scheduler.  Small configurations with random weights; sizes chosen so
that nothing the design allows to differ happens to be equal or 1."""
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import gefilix_oracle as O

pytestmark = pytest.mark.gpu

DTYPES = [(torch.float32, 2e-5), (torch.bfloat16, 2e-2)]


def _items(lens, slots, starts, gpu):
    """StepItems of portions with ``lens`` rows starting at positions ``starts`` in state slots ``slots``."""
    from llm_weighted_consensus_amd.ops import res32

    cu, row_item, pos = [0], [], []
    for i, (n, p0) in enumerate(zip(lens, starts)):
        cu.append(cu[-1] + n)
        row_item += [i] * n
        pos += list(range(p0, p0 + n))
    t = lambda v: torch.tensor(v, dtype=torch.int32, device=gpu)  # noqa: E731
    return res32.StepItems(t(row_item), t(cu), t(slots), t(pos))


def _paged(n_tokens, bs, nk, nv, dtype, gpu, seed=0):
    """A cache of shuffled pages for one sequence of n_tokens: (cache, table row, slots)."""
    from llm_weighted_consensus_amd.models.cache import PagedLayerCache

    nb = -(-n_tokens // bs)
    perm = torch.randperm(nb + 3, generator=torch.Generator().manual_seed(seed))[:nb]
    cache = PagedLayerCache([(nk, nv)], nb + 3, bs, gpu, dtype)
    return cache, perm.to(torch.int32), torch.tensor([int(perm[j // bs]) * bs + j % bs for j in range(n_tokens)])


# ------------------------------------------------------------------ mechanisms, one by one
@pytest.mark.parametrize("ydt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("d", [46, 64, 1028, 2052, 5120])
def test_norm_after_the_sum(gpu, d, ydt):
    """x <- norm(alpha x + y) in place with a bf16 copy, y of either type (a column slice too), rows of every path."""
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(d)
    T, eps, alpha = 7, 1e-3, 2.75
    x, y, w = 0.1 * torch.randn(T, d, generator=g), torch.randn(T, d + 4, generator=g).to(ydt), torch.randn(d, generator=g)
    x[2], y[2] = 0.0, 0.0   # a zero row: eps alone under the root
    ref = O.rms_norm(alpha * x.double() + y.double()[:, :d], w, eps)
    xg, h = x.to(gpu), torch.empty(T, d, dtype=torch.bfloat16, device=gpu)
    res32.post_norm(xg, y.to(gpu)[:, :d], alpha, w.to(gpu), eps, cast=h)
    assert (xg.cpu().double() - ref).abs().max() < 1e-5 * 4
    assert torch.equal(h, xg.to(torch.bfloat16))
    xg = x.to(gpu)
    res32.post_norm(xg, y.to(gpu)[:, :d], alpha, w.to(gpu), eps)
    assert (xg.cpu().double() - ref).abs().max() < 1e-5 * 4


@pytest.mark.parametrize("act,ydt", [(torch.float32, torch.float32), (torch.bfloat16, torch.float32), (torch.bfloat16, torch.bfloat16)])
@pytest.mark.parametrize("d", [46, 64, 2052])
def test_norm_after_a_routed_sum(gpu, d, act, ydt):
    """The weighted experts' rows and the gated shared rows formed inside the norm's pass; without shared rows; with
    shared rows but no gate."""
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(d)
    T, k, eps, alpha = 9, 3, 1e-5, 0.6
    x, w = torch.randn(T, d, generator=g), 1 + 0.2 * torch.randn(d, generator=g)
    Y, inv = torch.randn(T * k, d, generator=g).to(ydt), torch.randperm(T * k, generator=g).to(torch.int32)
    wts, sh = torch.rand(T, k, generator=g), torch.randn(T, d, generator=g).to(act)
    z = torch.randn(T, 5, generator=g)
    sums = (Y.double()[inv.long()].view(T, k, d) * wts.double()[..., None]).sum(1)
    for shared, gate in ((sh, z), (None, None), (sh, None)):
        y = sums if shared is None else sums + sh.double() * (torch.sigmoid(z.double()[:, 4:]) if gate is not None else 1.0)
        ref = O.rms_norm(alpha * x.double() + y, w, eps)
        xg, h = x.to(gpu), torch.empty(T, d, dtype=torch.bfloat16, device=gpu)
        res32.post_norm_experts(xg, Y.to(gpu), inv.to(gpu), wts.to(gpu), torch.zeros(T, d, dtype=act, device=gpu), alpha, w.to(gpu), eps,
                                shared=None if shared is None else shared.to(gpu),
                                gate=None if gate is None else z.to(gpu)[:, 4], cast=h)
        assert (xg.cpu().double() - ref).abs().max() < 1e-5 * 4
        assert torch.equal(h, xg.to(torch.bfloat16))


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-5), (torch.bfloat16, 3e-2)])
@pytest.mark.parametrize("H,D,R,C", [(3, 20, 6, 28), (2, 32, 16, 104), (5, 8, 2, 5)])
def test_cached_rows_without_a_query_latent(gpu, dtype, tol, H, D, R, C):
    """What a layer's down-projection leaves in the cache: the normed latent and the rotated part behind it, padding
    zero, the latent again in the value row; a slot of -1 writes nothing; positions far from zero."""
    from llm_weighted_consensus_amd.models.cache import PagedLayerCache
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(C)
    T, bs, eps, off = 8, 8, 1e-5, 3
    Dk, Cv = -(-(C + R) // 8) * 8, -(-C // 8) * 8
    proj, wc = torch.randn(T, off + C + R, generator=g).to(dtype), 1 + 0.2 * torch.randn(C, generator=g)
    pos = torch.tensor([0, 1, 2, 63, 64, 500, 1500, 4000])
    slots = torch.randperm(4 * bs, generator=g)[:T].to(torch.int32)
    slots[3] = -1
    cache = PagedLayerCache([(Dk, Cv)], 4, bs, gpu, dtype)
    cache.pool.fill_(7.0)  # stale contents
    f, m = res32.rope_frequencies(R, 777.0, None, gpu)
    assert m == 1.0
    assert res32.latent_kv_write(proj.to(gpu)[:, off:], 0, C, R, None, wc.to(gpu), f, m, pos.int().to(gpu), slots.to(gpu), cache.k[0],
                                 cache.v[0], eps) is None
    live = slots >= 0
    p64 = proj.double()[:, off:]
    c, kr = O.rms_norm(p64[:, :C], wc, eps), O.rotate_pairs(p64[:, C:], pos, 777.0)
    krow, vrow = (a.cpu().double() for a in cache.rows(0, slots[live].long().to(gpu)))
    assert (krow[:, :C] - c[live]).abs().max() < tol * 4 and (vrow[:, :C] - c[live]).abs().max() < tol * 4
    # (angles are fp32 products: 4000 rad has a spacing of 2.4e-4)
    assert (krow[:, C:C + R] - kr[live]).abs().max() < tol * 4 + 5e-4 * float(kr.abs().max())
    assert float(krow[:, C + R:].abs().sum()) == 0 and float(vrow[:, C:].abs().sum()) == 0
    assert int((cache.k[0] == 7.0).all(-1).sum()) == 4 * bs - int(live.sum())   # no other token was touched


@pytest.mark.parametrize("dtype,tol", DTYPES)
@pytest.mark.parametrize("H,Dv", [(3, 10), (5, 24), (16, 64)])
def test_gate_per_head(gpu, dtype, tol, H, Dv):
    """One sigmoid gate per head over results as a batched product leaves them ([H, T, Dv]) or with padded heads."""
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(H)
    T = 13
    z = (3 * torch.randn(T, 4 + H, generator=g)).to(dtype)
    for o in (torch.randn(H, T, Dv, generator=g).to(dtype).transpose(0, 1), torch.randn(T, H, Dv + 6, generator=g).to(dtype)[:, :, :Dv]):
        out = torch.empty(T, H * Dv, dtype=dtype, device=gpu)
        og = (o.transpose(0, 1).contiguous().to(gpu).transpose(0, 1) if o.stride(0) == Dv
              else torch.nn.functional.pad(o, (0, 6)).to(gpu)[:, :, :Dv])
        assert og.stride() == o.stride()
        res32.head_gate_rows(og, z.to(gpu)[:, 4:], out)
        ref = (o.double() * torch.sigmoid(z.double()[:, 4:])[..., None]).reshape(T, H * Dv)
        assert (out.cpu().double() - ref).abs().max() < tol * 4


@pytest.mark.parametrize("dtype,tol", DTYPES)
@pytest.mark.parametrize("H,D,Dv", [(3, 160, 128), (7, 192, 128), (20, 192, 64), (5, 320, 256), (17, 320, 256), (33, 320, 256), (2, 168, 136)])
def test_attention_over_one_shared_wide_row(gpu, dtype, tol, H, D, Dv):
    """All heads read ONE cached row per token whose head is the value: decode rows (in bf16 on the split-key kernels of
    192 and 320 entries where they are built, else and in fp32 on the general kernel) and a portion behind cached keys."""
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(D + H)
    n, bs = 145, 16
    cache, table, slots = _paged(n, bs, D, Dv, dtype, gpu, seed=D)
    K = torch.randn(n, D, generator=g).to(dtype)
    V = K[:, :Dv].clone()
    cache.set_rows(0, slots.to(gpu), K.to(gpu), V.to(gpu))
    q = torch.randn(n, H, D, generator=g) * 2 * D ** -0.5
    ref = torch.einsum("hij,jv->ihv", O.causal_softmax(torch.einsum("ihd,jd->hij", q.double(), K.double())), V.double())
    z, tab = torch.zeros(H, device=gpu), table[None].to(gpu)
    rows = [0, 1, 15, 16, 17, 31, 32, 127, 128, 144]
    out = torch.empty(len(rows), H * Dv, dtype=dtype, device=gpu)
    res32.window_attn(q[rows].reshape(len(rows), -1).to(gpu), cache.k[0], cache.v[0], torch.tensor(rows, dtype=torch.int32, device=gpu),
                      tab.expand(len(rows), -1).contiguous(), z, z, 1 << 30, out, H, 1, cores=True, values_in_keys=True)
    assert (out.cpu().double().view(len(rows), H, Dv) - ref[rows]).abs().max() < tol * 4
    a = 30
    out = torch.empty(n - a, H * Dv, dtype=dtype, device=gpu)
    res32.window_attn(q[a:].reshape(n - a, -1).to(gpu), cache.k[0], cache.v[0], torch.arange(a, n, dtype=torch.int32, device=gpu), tab, z, z,
                      1 << 30, out, H, 1, cu_q=torch.tensor([0, n - a], dtype=torch.int32, device=gpu),
                      k_lens=torch.tensor([n], dtype=torch.int32, device=gpu), max_q=n - a, cores=True)
    assert (out.cpu().double().view(n - a, H, Dv) - ref[a:]).abs().max() < tol * 4


@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("dtype,D,Dv", [(torch.float32, 40, 24), (torch.bfloat16, 128, 64), (torch.bfloat16, 192, 128), (torch.bfloat16, 320, 256)])
def test_far_key_and_page_borders_stand_out(gpu, decode, dtype, D, Dv):
    """One cached row made to stand out (parallel to the query, scaled up) at the first token, at both sides of page
    borders, hundreds of tokens back and at the row itself, over shuffled pages: the result is that row's value."""
    from llm_weighted_consensus_amd.ops import res32

    H, n, bs = 3, 530, 16
    g = torch.Generator().manual_seed(5)
    z = torch.zeros(H, device=gpu)
    for target in (0, 15, 16, 31, 32, 255, 256, 511, 512, 528, 529):
        cache, table, slots = _paged(n, bs, D, Dv, dtype, gpu, seed=target)
        K = 0.05 * torch.randn(n, D, generator=g)
        qv = torch.randn(D, generator=g)
        qv = qv / qv.norm()
        K[target] = 12.0 * qv
        K = K.to(dtype)
        cache.set_rows(0, slots.to(gpu), K.to(gpu), K[:, :Dv].to(gpu))
        q = (qv[None, None] * 3.0).expand(1, H, D).reshape(1, H * D).contiguous().to(gpu)
        out = torch.empty(1, H * Dv, dtype=dtype, device=gpu)
        kw = dict(values_in_keys=True) if decode else dict(cu_q=torch.tensor([0, 1], dtype=torch.int32, device=gpu),
                                                           k_lens=torch.tensor([n], dtype=torch.int32, device=gpu), max_q=1)
        res32.window_attn(q, cache.k[0], cache.v[0], torch.tensor([n - 1], dtype=torch.int32, device=gpu), table[None].to(gpu), z, z,
                          1 << 30, out, H, 1, cores=True, **kw)
        assert (out.cpu().double().view(H, Dv) - K[target, :Dv].double()).abs().max() < 2e-2, target


@pytest.mark.parametrize("dtype,tol", DTYPES)
@pytest.mark.parametrize("H,D,Dv", [(3, 12, 20), (2, 64, 64), (4, 64, 48), (2, 80, 72), (1, 130, 8), (2, 200, 40), (5, 128, 128), (2, 32, 96)])
def test_lightning_portions_single_tokens_and_stale_slots(gpu, dtype, tol, H, D, Dv):
    """The recurrence over activated rows: sequences cut into portions (single rows, two tokens, several in one step,
    tiles of the kernels crossed) in slots that held other data, against the whole-sequence oracle; the state left in
    the slot is the oracle's."""
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(D + Dv)
    lens = {"a": 230, "b": 9, "c": 140}
    decay = [1.0 - 2.0 ** (-1 - 2 * h) for h in range(H)]
    nq, nv = H * D, H * Dv
    seqs = {k: torch.randn(n, 2 * nq + nv + 3, generator=g).to(dtype) for k, n in lens.items()}
    state = (torch.randn(5, H, D, Dv, generator=g) * 50).to(gpu)  # stale contents of earlier sequences
    ref, ref_S = {}, {}
    for k, x in seqs.items():
        a = O.silu(x.double()[:, :2 * nq + nv])
        T = lens[k]
        ref[k], ref_S[k] = O.lightning_scan(a[:, :nq].reshape(T, H, D), a[:, nq:2 * nq].reshape(T, H, D), a[:, 2 * nq:].reshape(T, H, Dv), decay)
    plan = [[("a", 1)], [("a", 2), ("b", 1)], [("b", 2), ("a", 1)], [("a", 17)], [("b", 6), ("a", 33)], [("c", 129), ("a", 64)],
            [("a", 63)], [("a", 1), ("c", 10)], [("a", 48), ("c", 1)]]
    at, got, slot = {k: 0 for k in seqs}, {k: [] for k in seqs}, {"a": 2, "b": 0, "c": 3}
    dec = torch.tensor(decay, dtype=torch.float32, device=gpu)
    for step in plan:
        x = torch.cat([seqs[k][at[k]:at[k] + n] for k, n in step]).to(gpu)
        out = res32.lightning(x, state, dec, _items([n for _, n in step], [slot[k] for k, _ in step], [at[k] for k, _ in step], gpu), H)
        o = 0
        for k, n in step:
            got[k].append(out[o:o + n].cpu())
            o, at[k] = o + n, at[k] + n
    assert at == lens
    for k in seqs:
        r = ref[k].reshape(-1, nv)
        assert (torch.cat(got[k]).double() - r).abs().max() < tol * max(4.0, float(r.abs().max())), k
        assert (state[slot[k]].cpu().double() - ref_S[k]).abs().max() < tol * max(4.0, float(ref_S[k].abs().max())), k


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_lightning_far_token_survives_a_slow_decay(gpu, dtype):
    """One early token made large: after hundreds of tokens its share of the result is a^n times its value, for a fast,
    a slow and a lossless head (one portion; portions; then single tokens)."""
    from llm_weighted_consensus_amd.ops import res32

    H, D, Dv, n = 3, 32, 32, 400
    decay = [0.9, 0.9990234375, 1.0]
    x = torch.full((n, 2 * H * D + H * Dv), -30.0)                 # silu(-30) = -3e-12
    x[5, H * D + 3:2 * H * D:D] = 50.0                              # k of token 5: entry 3 of every head
    x[5, 2 * H * D:] = 2.0                                          # v of token 5
    x[n - 1, 3:H * D:D] = 40.0                                      # q of the last token
    v2 = 2.0 / (1.0 + math.exp(-2.0))
    xs, dec = x.to(dtype).to(gpu), torch.tensor(decay, device=gpu)
    for cuts in ([n], [6, 100, n - 106], [3, 2, n - 25] + [1] * 20):
        state, a, out = torch.zeros(2, H, D, Dv, device=gpu), 0, None
        for c in cuts:
            out = res32.lightning(xs[a:a + c], state, dec, _items([c], [1], [a], gpu), H)
            a += c
        assert a == n
        last = out[-1].cpu().view(H, Dv)
        for h in range(H):
            want = 40.0 * 50.0 * v2 * decay[h] ** (n - 1 - 5)
            assert (last[h] - want).abs().max() < 1e-6 + 6e-3 * want, (cuts[:3], h)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-5), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("n", [30, 96, 260, 1300, 3000])
def test_norm_over_all_heads_with_a_gate(gpu, dtype, tol, n):
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(n)
    T, eps = 6, 1e-4
    o, w, z = 0.05 * torch.randn(T, n, generator=g), torch.randn(n, generator=g), (2 * torch.randn(T, n + 4, generator=g)).to(dtype)
    out = torch.empty(T, n, dtype=dtype, device=gpu)
    res32.head_norm_gate(o.to(gpu), out, 1, eps, w=w.to(gpu), gate=z.to(gpu)[:, 4:], mode="sigmoid")
    ref = O.rms_norm(o.double(), w, eps) * torch.sigmoid(z.double()[:, 4:])
    assert (out.cpu().double() - ref).abs().max() < tol * 4


@pytest.mark.parametrize("E,top,groups,keep", [(6, 2, 3, 1), (8, 3, 2, 2), (12, 5, 4, 3), (16, 1, 8, 2), (5, 5, 1, 1), (7, 2, 7, 3),
                                               (40, 4, 5, 2), (96, 6, 8, 3), (300, 7, 30, 4), (128, 3, 64, 9)])
def test_router_scores_groups_and_weights(gpu, E, top, groups, keep):
    """Sigmoid scores, the open groups, the choice and the weights on both router kernels (up to 16 outputs a thread per
    token, above a wave per token); z comes as columns of a wider product; the row lists are consistent."""
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(E)
    T, scale = 67, 1.9
    z = 2 * torch.randn(T, E + 1, generator=g)
    ids, w, row_off, src, row_expert, inv = res32.router(z.to(gpu)[:, :E], None, E, top, renorm=True, scores="sigmoid", floor=1e-20,
                                                         scale=scale, groups=groups, keep=keep)
    r = {"experts": E, "top": top, "scale": scale, "groups": {"count": groups, "keep": keep}}
    ref_ids, ref_w = O.route(z.double()[:, :E], lambda n: torch.eye(E, dtype=torch.float64), r)
    assert torch.equal(ids.cpu().long(), ref_ids)
    assert (w.cpu().double() - ref_w).abs().max() < 1e-5
    assert groups in (1, E) or keep == groups or not torch.equal(ref_ids, torch.topk(z[:, :E], top).indices)  # the groups matter
    rows = inv.cpu().view(T, top)
    assert sorted(rows.flatten().tolist()) == list(range(T * top)) and int(row_off[-1]) == T * top
    assert torch.equal(src.cpu()[rows.flatten().long()].view(T, top), torch.arange(T)[:, None].expand(T, top).int())
    assert torch.equal(row_expert.cpu()[rows.flatten().long()].view(T, top), ids.cpu())


@pytest.mark.parametrize("E,size", [(8, 4), (96, 12)])
def test_a_group_wins_by_its_two_best_scores(gpu, E, size):
    """Hand-made scores: a group with the single best expert loses to one with the best pair; a third high score in a
    group does not count."""
    from llm_weighted_consensus_amd.ops import res32

    z = torch.full((3, E), -3.0)
    z[0, 0] = 4.0                                    # group 0: one star
    z[0, size], z[0, size + 1] = 1.0, 1.2            # group 1: the best pair
    z[1, :3] = torch.tensor([0.5, 0.5, 0.5])         # three middling experts
    z[1, size], z[1, size + size - 1] = 0.6, 0.6     # two slightly better ones
    z[2, E - 1], z[2, E - 2], z[2, 1] = 2.0, 1.0, 2.5  # the last group wins
    ids, w, *_ = res32.router(z.to(gpu), None, E, 2, renorm=True, scores="sigmoid", floor=1e-20, scale=1.0, groups=E // size, keep=1)
    assert ids.cpu().tolist() == [[size + 1, size], [size, 2 * size - 1], [E - 1, E - 2]]
    s = torch.sigmoid(torch.tensor([1.2, 1.0]))
    assert (w[0].cpu() - s / s.sum()).abs().max() < 1e-6


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-5), (torch.bfloat16, 3e-2)])
@pytest.mark.parametrize("d,ff", [(24, 10), (64, 40), (50, 33)])
def test_clamped_experts(gpu, dtype, tol, d, ff):
    """Experts' rows with inputs far beyond the limits on both sides, and the shared expert's fused unit."""
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(d)
    T, E, top, limit = 11, 4, 2, 0.8
    h = torch.randn(T, d, generator=g).to(dtype)
    W = {f"e{e}.{n}": (torch.randn(*s, generator=g) * 3 / math.sqrt(s[1])).to(dtype) for e in range(E)
         for n, s in (("gate", (ff, d)), ("up", (ff, d)), ("down", (d, ff)))}
    gu = torch.stack([torch.cat([W[f"e{e}.gate"], W[f"e{e}.up"]]) for e in range(E)]).contiguous().to(gpu)
    dn = torch.stack([W[f"e{e}.down"] for e in range(E)]).contiguous().to(gpu)
    z = torch.randn(T, E, generator=g).to(gpu)
    ids, w, row_off, src, row_expert, inv = res32.router(z, None, E, top, renorm=True, scores="sigmoid")
    Y = res32.expert_rows(h.to(gpu), src, row_expert, row_off, gu, dn, mode="clamped", alpha=1.702, limit=limit).cpu().double()
    for r in range(T * top):
        e, t = int(row_expert[r]), int(src[r])
        ref = O.expert(h[t].double(), lambda n: W[n].double(), f"e{e}", limit)
        assert (Y[r] - ref).abs().max() < tol * 8
    a = (h.to(gpu) @ gu[0].T).contiguous()
    got = res32.glu(a, mode="clamped", alpha=1.702, limit=limit).cpu().double()
    assert (got - O.clamped_unit(a.cpu().double()[:, :ff], a.cpu().double()[:, ff:], limit)).abs().max() < tol * 8


def test_scaled_embedding_rows_with_a_copy(gpu):
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(1)
    E, tok = torch.randn(30, 46, generator=g).to(torch.bfloat16), torch.tensor([3, 29, 0, 3], dtype=torch.int32)
    h = torch.empty(4, 46, dtype=torch.bfloat16, device=gpu)
    x = res32.embed_rows(E.to(gpu), tok.to(gpu), scale=7.5, cast=h)
    assert torch.equal(x.cpu(), E[tok.long()].float() * 7.5) and torch.equal(h, x.to(torch.bfloat16))


# ------------------------------------------------------------------ the model through the engine
def _configs():
    m8 = O.moe(8, 3, 24, 40, groups=(4, 2))
    return {
        # both mixers, both feed-forwards, a layer without feed-forward, a layer that reads the latents of an earlier one
        # with other heads and sizes of its own, and one that reads layer 0's
        "mixed": dict(width=72, vocab=250, layers=[
            O.latent_layer(4, 16, 8, 24, 40, m8, scale=0.21, base=900.0), O.lightning_layer(2, 32, 16, O.dense(56)),
            O.latent_layer(3, 24, 16, 20, 48, O.dense(90)), O.lightning_layer(3, 24, 40, None),
            O.latent_layer(6, 12, 16, 28, 48, m8, kv_from=2), O.latent_layer(2, 20, 8, 16, 40, None, base=900.0, kv_from=0)]),
        # odd sizes everywhere: nothing a multiple of 8, one head, one expert chosen, groups of one
        "odd": dict(width=46, vocab=131, layers=[
            O.lightning_layer(1, 20, 12, O.moe(5, 1, 18, 7, groups=(5, 2), scale=0.8)),
            O.latent_layer(3, 10, 6, 14, 27, O.dense(33), scale=0.3), O.latent_layer(1, 12, 6, 5, 27, O.moe(6, 4, 9, 11, groups=(2, 2)), kv_from=1),
            O.lightning_layer(5, 7, 9, None)]),
        # lightning only (no paged keys at all)
        "recurrent": dict(width=48, vocab=200, layers=[
            O.lightning_layer(2, 64, 32, O.dense(64)), O.lightning_layer(4, 16, 24, O.moe(4, 2, 16, 20)), O.lightning_layer(2, 128, 64, None)]),
        # attention only (no recurrent state), sizes of the matrix-core paths (rows of 128 / 96 -> 128)
        "attentive": dict(width=64, vocab=200, layers=[
            O.latent_layer(4, 32, 32, 32, 96, O.dense(64)), O.latent_layer(8, 16, 32, 16, 96, m8, kv_from=0)]),
        # rows of 192 / 128 (portions and decode rows on the matrix cores), two layers over one cache
        "rows192": dict(width=64, vocab=200, layers=[
            O.latent_layer(5, 24, 40, 32, 120, m8), O.lightning_layer(2, 32, 32, O.dense(48)), O.latent_layer(18, 8, 40, 12, 120, O.dense(40), kv_from=0)]),
        # rows of 320 / 256: decode rows on the staged kernel, portions over up-projected keys and values, shared too
        "rows320": dict(width=64, vocab=200, layers=[
            O.latent_layer(3, 48, 24, 40, 232, O.dense(64)), O.latent_layer(18, 16, 24, 32, 232, m8, kv_from=0)]),
        # rows of 576 / 512, and rows no kernel is built for (general kernel in decoding)
        "rows576": dict(width=64, vocab=200, layers=[
            O.latent_layer(17, 16, 64, 16, 328, O.dense(40)), O.latent_layer(2, 40, 8, 24, 140, m8)]),
        # experts past the grouped-GEMM threshold
        "grouped": dict(width=256, vocab=200, layers=[
            O.latent_layer(2, 32, 16, 32, 48, O.dense(64)), O.lightning_layer(2, 32, 32, O.moe(4, 2, 1024, 64, groups=(2, 1)))]),
        # 33 router outputs in 11 groups (the wave-wide router), 20 heads, a lightning head wider than 128
        "ragged": dict(width=50, vocab=97, layers=[
            O.latent_layer(20, 6, 4, 5, 26, O.moe(33, 4, 10, 14, groups=(11, 3))), O.lightning_layer(2, 136, 20, O.dense(30))]),
    }


CONFIGS = _configs()


def _make(name, seed=0, every_expert=False):
    """``every_expert``: all groups open and all experts chosen, so that no choice is there for bf16 rounding to flip (a
    flipped choice changes whole rows and, through the recurrent state, the rows after them).  The choice itself is the
    same fp32 kernel in both modes; the fp32 cases and the router's own tests cover it."""
    cfg = json.loads(json.dumps(O.make_config(**CONFIGS[name])))
    for L in cfg["layers"]:
        if every_expert and L["mlp"] and L["mlp"]["kind"] == "moe":
            r = L["mlp"]["router"]
            r["top"], r["groups"]["keep"] = r["experts"], r["groups"]["count"]
    return cfg, O.make_weights(cfg, seed)


def _save(path, cfg, W):
    from safetensors.torch import save_file

    path.mkdir(exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in W.items()}, str(path / "model.safetensors"))
    return str(path)


def _build(tmp_path, name, dtype, seed=0, **engine_kw):
    from llm_weighted_consensus_amd.engine.engine import LLMEngine
    from llm_weighted_consensus_amd.engine.tokenizer import load_tokenizer
    from llm_weighted_consensus_amd.models.registry import load_model

    cfg, W = _make(name, seed, every_expert=dtype == torch.bfloat16)
    model = load_model(_save(tmp_path / f"{name}-{seed}", cfg, W), dtype=dtype)
    kw = dict(block_size=16, num_blocks=24, max_batch=4, max_model_len=256, use_graphs=False, prefix_sharing=False, tune_gc=False)
    kw.update(engine_kw)
    return cfg, W, model, LLMEngine(model, load_tokenizer({}, cfg["vocab"]), **kw)


def _tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def _err(got, ref, dtype=torch.float32):
    """fp32: the largest difference relative to the reference's largest entry (at least 1).  bf16: the row-wise
    relative RMS difference that 95 % of the rows stay under, and no row may be off by more than its own size.  (Where a
    sequence's first q and k are nearly orthogonal, rounding decides the sign of a lightning head's q . k, which the norm
    behind it blows up to full size: single rows are then far off without a fault.)"""
    d, ref = got.cpu().double() - ref, ref.double()
    if dtype == torch.float32:
        return float(d.abs().max()) / max(1.0, float(ref.abs().max()))
    rel = (d.pow(2).mean(-1).sqrt() / ref.pow(2).mean(-1).sqrt().clamp_min(1e-3)).flatten()
    assert float(rel.max()) < 1.0
    return float(rel.quantile(0.95))


TOL = {torch.float32: 1e-4, torch.bfloat16: 0.15}
F32, BF16 = torch.float32, torch.bfloat16
ALL = ("mixed", "odd", "recurrent", "attentive", "rows192", "rows320", "rows576", "ragged")


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", ALL)
def test_whole_prompt_and_every_layer(gpu, tmp_path, name, dtype):
    """A whole prompt in one step: the stream after every layer and the logits."""
    cfg, W, model, eng = _build(tmp_path, name, dtype)
    toks = _tokens(70, cfg["vocab"], 1)
    streams, seen = [], []
    ref = O.forward(cfg, W, toks, streams)
    model.on_layer = lambda i, x: seen.append(x.detach().cpu().double())
    got = eng.step_tokens([("w", toks, list(range(len(toks))))], ["w"])
    model.on_layer = None
    assert len(seen) == len(streams) == len(cfg["layers"])
    for a, b in zip(seen, streams):
        assert _err(a, b, dtype) < TOL[dtype]
    assert _err(got, ref, dtype) < TOL[dtype]
    assert eng.bm.num_free == eng.bm.num_blocks and eng.bm.num_free_state_slots == 4


def test_row_sizes_and_shared_caches(gpu, tmp_path):
    """Which cached row sizes the configurations above reach, and that a layer with kv_from has no pages of its own."""
    want = {"rows192": [(192, 128)], "rows320": [(320, 256)], "rows576": [(576, 512), (152, 144)], "attentive": [(128, 128)],
            "mixed": [(64, 64), (64, 64)], "recurrent": []}
    for name, dims in want.items():
        _, _, model, _ = _build(tmp_path, name, BF16)
        assert [tuple(d) for d in model._layer_dims()] == dims, name
    _, _, model, _ = _build(tmp_path, "mixed", F32)
    assert model.cache_index == {0: 0, 2: 1, 4: 1, 5: 0} and len(model.state_fields()) == 2


def test_a_layer_reads_the_named_layers_latents(gpu, tmp_path):
    """The oracle with kv_from pointing at the other source differs (so the test would see it); the model follows the
    right one, in a prompt and in decoding."""
    base = dict(heads=3, dim=12, rot_dim=8, vdim=10, kv_rank=24)
    layers = [O.latent_layer(mlp=None, **base), O.latent_layer(mlp=O.dense(40), **base), O.latent_layer(mlp=None, **dict(base, heads=5), kv_from=0)]
    cfg = O.make_config(40, 90, layers)
    W = O.make_weights(cfg, 3)
    other = json.loads(json.dumps(cfg))
    other["layers"][2]["mixer"]["kv_from"] = 1
    toks = _tokens(30, 90, 4)
    ref, wrong = O.forward(cfg, W, toks), O.forward(other, W, toks)
    assert float((ref - wrong).abs().max()) > 0.1
    from llm_weighted_consensus_amd.engine.engine import LLMEngine
    from llm_weighted_consensus_amd.engine.tokenizer import load_tokenizer
    from llm_weighted_consensus_amd.models.registry import load_model

    for c, r in ((cfg, ref), (other, wrong)):
        model = load_model(_save(tmp_path / str(c["layers"][2]["mixer"]["kv_from"]), c, W), dtype=F32)
        eng = LLMEngine(model, load_tokenizer({}, 90), block_size=16, num_blocks=8, max_batch=4, max_model_len=64, use_graphs=False,
                        prefix_sharing=False, tune_gc=False)
        got = [eng.step_tokens([("s", toks[:20], list(range(20)))])]
        got += [eng.step_tokens([("s", [t], [0])]) for t in toks[20:]]
        assert _err(torch.cat(got), r) < TOL[F32]


@pytest.mark.parametrize("change", ["alpha", "eps", "decay", "limit", "shared_limit", "router_scale", "keep", "scale", "base", "embed"])
def test_every_constant_is_read_from_the_config(gpu, tmp_path, change):
    """One constant changed in the folder's config: the model's logits follow the oracle's, which move."""
    from llm_weighted_consensus_amd.engine.engine import LLMEngine
    from llm_weighted_consensus_amd.engine.tokenizer import load_tokenizer
    from llm_weighted_consensus_amd.models.registry import load_model

    cfg, W = _make("mixed", 6)
    toks = _tokens(40, cfg["vocab"], 7)
    before = O.forward(cfg, W, toks)
    c = json.loads(json.dumps(cfg))
    mlp = c["layers"][0]["mlp"]
    if change == "alpha":
        c["postln_alpha"] = 0.8
    elif change == "eps":
        c["norm"]["eps"] = 0.3
    elif change == "decay":
        c["layers"][1]["mixer"]["decay"] = [0.99, 0.3]
    elif change == "limit":
        mlp["expert"]["limit"] = 0.4
    elif change == "shared_limit":
        mlp["shared"]["limit"] = 3.0
    elif change == "router_scale":
        mlp["router"]["scale"] = 0.5
    elif change == "keep":
        mlp["router"]["groups"]["keep"] = 4
    elif change == "scale":
        c["layers"][0]["mixer"]["scale"] = 0.05
    elif change == "base":
        for i in (0, 5):
            c["layers"][i]["mixer"]["rot"]["base"] = 11.0
    else:
        c["embedding"]["scale"] = 1.5
    ref = O.forward(c, W, toks)
    assert float((ref - before).abs().max()) > 0.02
    model = load_model(_save(tmp_path / change, c, W), dtype=F32)
    eng = LLMEngine(model, load_tokenizer({}, c["vocab"]), block_size=16, num_blocks=8, max_batch=4, max_model_len=64, use_graphs=False,
                    prefix_sharing=False, tune_gc=False)
    got = eng.step_tokens([("w", toks, list(range(40)))], ["w"])
    assert _err(got, ref) < TOL[F32]


def test_grouped_expert_path(gpu, tmp_path):
    """Experts past the size threshold run through the framework's grouped GEMMs (bf16): a portion and single tokens."""
    from llm_weighted_consensus_amd import ops

    assert ops.available()
    cfg, W, model, eng = _build(tmp_path, "grouped", BF16)
    assert model._use_grouped(cfg["width"], cfg["layers"][1]["mlp"]["expert"]["ff"])
    toks = _tokens(48, cfg["vocab"], 3)
    ref = O.forward(cfg, W, toks)
    got = [eng.step_tokens([("g", toks[:40], list(range(40)))])]
    for i in range(40, 48):
        got.append(eng.step_tokens([("g", [toks[i]], [0])], ["g"] if i == 47 else []))
    assert _err(torch.cat(got), ref, BF16) < TOL[BF16]


@pytest.mark.parametrize("name,dtype", [("mixed", F32), ("odd", F32), ("attentive", F32), ("rows320", BF16)])
def test_few_wanted_rows_and_what_they_leave(gpu, tmp_path, name, dtype):
    """A prompt of which only the last row is wanted (the last layer's output side then runs on that row only): the same
    logits, and the cache and state it leaves carry the decoding that follows."""
    cfg, W, model, eng = _build(tmp_path, name, dtype)
    toks = _tokens(60, cfg["vocab"], 6)
    ref = O.forward(cfg, W, toks)
    got = [eng.step_tokens([("k", toks[:50], [49])])]
    for i in range(50, 60):
        got.append(eng.step_tokens([("k", [toks[i]], [0])], ["k"] if i == 59 else []))
    assert _err(torch.cat(got), ref[49:], dtype) < TOL[dtype]


@pytest.mark.parametrize("name,dtype", [(n, F32) for n in ("mixed", "odd", "recurrent", "ragged")]
                         + [(n, BF16) for n in ("mixed", "recurrent", "attentive", "rows192", "rows320", "rows576", "ragged")])
def test_decode_token_by_token_and_portions(gpu, tmp_path, name, dtype):
    """The same logits whether a prompt comes whole, token by token from the first token on, or in portions of
    changing sizes (down to two tokens; cut inside pages and inside the recurrence kernels' tiles)."""
    cfg, W, model, eng = _build(tmp_path, name, dtype)
    toks = _tokens(75, cfg["vocab"], 2)
    ref = O.forward(cfg, W, toks)
    rows = []
    for i, t in enumerate(toks):
        rows.append(eng.step_tokens([("d", [t], [0])], ["d"] if i + 1 == len(toks) else []))
    assert _err(torch.cat(rows), ref, dtype) < TOL[dtype]
    for sizes in ([2, 2, 13, 3, 16, 2, 30, 7], [17, 16, 15, 2, 25], [1, 2, 5, 67]):
        assert sum(sizes) == len(toks)
        rows, a = [], 0
        for n in sizes:
            rows.append(eng.step_tokens([("p", toks[a:a + n], list(range(n)))], ["p"] if a + n == len(toks) else []))
            a += n
        assert _err(torch.cat(rows), ref, dtype) < TOL[dtype]
    assert eng.bm.num_free == eng.bm.num_blocks and eng.bm.num_free_state_slots == 4


@pytest.mark.parametrize("name,dtype", [("mixed", F32), ("odd", F32), ("mixed", BF16), ("attentive", BF16), ("rows192", BF16),
                                        ("rows320", BF16), ("rows576", BF16)])
def test_unequal_batches_pages_and_slots_used_again(gpu, tmp_path, name, dtype):
    """Up to four live sequences of unequal lengths, portions beside single tokens, one sitting steps out, in a pool
    so small that pages and state slots are freed and taken again; every position equals the sequence run alone."""
    cfg, W, model, eng = _build(tmp_path, name, dtype, num_blocks=14)
    seqs = {k: _tokens(n, cfg["vocab"], 10 + i) for i, (k, n) in enumerate([("a", 70), ("b", 12), ("c", 40), ("d", 33), ("e", 58), ("f", 1)])}
    ref = {k: O.forward(cfg, W, t) for k, t in seqs.items()}
    at = {k: 0 for k in seqs}
    plan = [[("a", 30), ("b", 2)], [("a", 1), ("b", 7), ("c", 17)], [("a", 1), ("c", 1), ("d", 33), ("b", 3)], [("a", 2), ("c", 22)],
            [("a", 36)], [("e", 20), ("f", 1)], [("e", 1)], [("e", 37)]]
    gots, refs, free = [], [], set()
    for step in plan:
        entries, end, spans = [], [], []
        for k, n in step:
            a = at[k]
            entries.append((k, seqs[k][a:a + n], list(range(n))))
            spans.append((k, a, n))
            at[k] = a + n
            if at[k] == len(seqs[k]):
                end.append(k)
        got = eng.step_tokens(entries, end)
        o = 0
        for k, a, n in spans:
            gots.append(got[o:o + n].cpu())
            refs.append(ref[k][a:a + n])
            o += n
        free.add(eng.bm.num_free_state_slots)
    assert all(at[k] == len(seqs[k]) for k in seqs)
    assert _err(torch.cat(gots), torch.cat(refs), dtype) < TOL[dtype]
    assert eng.bm.num_free == eng.bm.num_blocks and eng.bm.num_free_state_slots == 4 and min(free) == 1
    with pytest.raises(RuntimeError):  # a fifth live sequence: no state slot
        eng.step_tokens([(k, [1, 2], []) for k in "vwxyz"])


@pytest.mark.parametrize("name,dtype", [("mixed", F32), ("rows192", BF16)])
def test_long_decoding(gpu, tmp_path, name, dtype):
    """220 tokens decoded one by one after a short prompt (pages cross, the recurrent state runs long)."""
    cfg, W, model, eng = _build(tmp_path, name, dtype, num_blocks=20, max_model_len=320)
    toks = _tokens(230, cfg["vocab"], 9)
    ref = O.forward(cfg, W, toks)
    got = [eng.step_tokens([("l", toks[:10], list(range(10)))])]
    for i in range(10, 230):
        got.append(eng.step_tokens([("l", [toks[i]], [0])], ["l"] if i == 229 else []))
    assert _err(torch.cat(got), ref, dtype) < TOL[dtype]


def _check_greedy(cfg, W, prompt, got, slack=0.04):
    """Every generated token is the oracle's best next token GIVEN the engine's own tokens so far, up to near-ties
    (the sampler reads bf16 logits: two logits closer than their rounding may swap); most are the exact argmax."""
    lg = O.forward(cfg, W, list(prompt) + list(got[:-1]))[len(prompt) - 1:]
    exact = 0
    for t, tok in enumerate(got):
        assert 0 <= tok < cfg["vocab"]
        assert float(lg[t].max() - lg[t, tok]) < slack, f"token {t}: {tok} is {float(lg[t].max() - lg[t, tok])} below the best"
        exact += int(lg[t].argmax()) == tok
    assert exact >= 0.8 * len(got)


@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation_through_the_scheduler(gpu, tmp_path, graphs):
    """engine.generate (admission, paged prefill, state slots from the block manager, batched decode steps, the fused
    sampler at temperature 0; with hipGraph replay of the decode step when ``graphs``: its warm-up run must not advance
    the sequences' states) against the oracle's greedy continuation, twice on one engine so that slots and pages come
    back dirty."""
    from llm_weighted_consensus_amd.engine.sampling import SamplingParams

    cfg, W, model, eng = _build(tmp_path, "mixed", F32, use_graphs=graphs, num_blocks=40)
    for seeds in ((21, 22), (23, 24)):
        prompts = [_tokens(23, 250, seeds[0]), _tokens(5, 250, seeds[1])]
        out = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=40, ignore_eos=True))
        for p, o in zip(prompts, out):
            assert len(o[0]) == 40
            _check_greedy(cfg, W, p, o[0])
    assert eng.bm.num_free == eng.bm.num_blocks and eng.bm.num_free_state_slots == 4


@pytest.mark.parametrize("name", ["rows192", "rows320"])
def test_captured_decode_steps_equal_eager_ones(gpu, tmp_path, name):
    """bf16 generation with and without hipGraph replay over the matrix-core paths: the same tokens."""
    from llm_weighted_consensus_amd.engine.sampling import SamplingParams

    outs = []
    for graphs in (False, True):
        cfg, W, model, eng = _build(tmp_path, name, BF16, use_graphs=graphs, num_blocks=40)
        prompts = [_tokens(23, 200, 51), _tokens(7, 200, 52), _tokens(60, 200, 53)]
        outs.append([o[0] for o in eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=24, ignore_eos=True))])
        if not graphs:
            for p, o in zip(prompts, outs[0]):
                _check_greedy(cfg, W, p, o, slack=0.6)
    same = sum(a == b for x, y in zip(*outs) for a, b in zip(x, y))
    assert same >= 0.9 * 72   # (the captured step may run other GEMM backends: a near-tie may fall the other way)


def test_generation_chunked_prefill_and_forks(gpu, tmp_path):
    """Chunked prefill (prompt portions beside running decodes) and n > 1 (forked sequences: shared prompt pages, the
    prompt's recurrent state copied to every child) give the greedy continuation too."""
    from llm_weighted_consensus_amd.engine.sampling import SamplingParams

    cfg, W, model, eng = _build(tmp_path, "mixed", F32, num_blocks=48, chunked_prefill=8, max_batch=8)
    prompts = [_tokens(37, 250, 31), _tokens(12, 250, 32)]
    out = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=20, ignore_eos=True), n=2)
    for p, o in zip(prompts, out):
        assert len(o) == 2 and o[0] == o[1]  # greedy forks of one prompt agree
        _check_greedy(cfg, W, p, o[0])
    assert eng.bm.num_free == eng.bm.num_blocks and eng.bm.num_free_state_slots == 8


def test_server_worker_factory_and_seeded_sampling(gpu, tmp_path):
    """The server's worker factory on a model folder of the design: prefix caching is switched off for it (a cached
    head brings no recurrent state), the state pool is there, greedy and seeded top-k generation work."""
    from llm_weighted_consensus_amd.engine.group import build_engine
    from llm_weighted_consensus_amd.engine.sampling import SamplingParams

    cfg, W = _make("mixed", 2)
    eng = build_engine({"model_dir": _save(tmp_path / "m", cfg, W), "dtype": "float32", "max_batch": 4, "max_model_len": 128,
                        "kv_fraction": 0.001}, 0)
    assert eng.state is not None and not eng.prefix_caching and eng.bm.num_state_slots == 4
    prompt = _tokens(20, cfg["vocab"], 8)
    out = eng.generate([prompt], SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True))
    _check_greedy(cfg, W, prompt, out[0][0])
    draws = [eng.generate([prompt], SamplingParams(temperature=1.0, top_k=5, seed=77, max_tokens=10, ignore_eos=True))[0][0] for _ in range(2)]
    assert draws[0] == draws[1]
    lg = O.forward(cfg, W, prompt + draws[0][:-1])[len(prompt) - 1:]
    for t, tok in enumerate(draws[0]):
        assert float(lg[t, tok]) > float(lg[t].topk(5).values[-1]) - 0.04


def test_trace_replay_command_line(gpu, tmp_path):
    """bin/trace_run as a user runs it: JSON lines in, ``done <step>`` lines and <step>.f32 files out; two sequences
    interleaved (portions beside single tokens, one sitting a step out), pages and slots given back at ``end``."""
    cfg, W = _make("mixed", 4)
    mdir, out = _save(tmp_path / "model", cfg, W), tmp_path / "out"
    a, b = _tokens(40, cfg["vocab"], 1), _tokens(21, cfg["vocab"], 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:30], "want": [0, 29]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:20], "want": []}, {"id": "a", "tokens": a[30:31], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[20:], "want": [0]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": a[31:], "want": [8, 2]}], "end": ["a"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", mdir, "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(4)]
    ra, rb = O.forward(cfg, W, a), O.forward(cfg, W, b)
    for step, ref in {0: ra[[0, 29]], 1: ra[[30]], 2: rb[[20]], 3: ra[[39, 33]]}.items():
        got = torch.from_numpy(np.fromfile(out / f"{step}.f32", dtype="<f4")).view(-1, cfg["vocab"])
        assert _err(got, ref) < TOL[F32]
    assert sorted(os.listdir(out)) == ["0.f32", "1.f32", "2.f32", "3.f32"]


def test_loader_refuses_wrong_shapes(gpu, tmp_path):
    from llm_weighted_consensus_amd.models.registry import load_model

    cfg, W = _make("odd", 0)
    bad = dict(W)
    bad["l1.mix.g"] = torch.zeros(5, cfg["width"], dtype=torch.bfloat16)
    with pytest.raises(ValueError):
        load_model(_save(tmp_path / "bad", cfg, bad))
    bad["l1.mix.g"] = W["l1.mix.g"]
    del bad["l0.mlp.shared.sg"]
    with pytest.raises(KeyError):
        load_model(_save(tmp_path / "bad2", cfg, bad))
