"""Semuzen on the GPU against the plain fp64 oracle (tests/semuzen_oracle.py): each mechanism alone, then the model
through the engine — whole prompts, token-by-token decoding, portions, unequal batches, pages used again, the first tokens
of a sequence, keys far away, at page borders and at both sides of a window's edge, long decoding, layers that read another
layer's keys and values, and greedy generation through the scheduler.  Small configurations with random weights; sizes
chosen so that nothing the design allows to differ happens to be equal or 1."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import semuzen_oracle as O

pytestmark = pytest.mark.gpu

F32, BF16 = torch.float32, torch.bfloat16
DTYPES = [(F32, 2e-5), (BF16, 2e-2)]
NO_WINDOW = 1 << 30


def _paged(n_tokens, bs, nk, nv, dtype, gpu, seed=0):
    """A cache of shuffled pages for one sequence of n_tokens: (cache, table row, slots)."""
    from llm_weighted_consensus_amd.models.cache import PagedLayerCache

    nb = -(-n_tokens // bs)
    perm = torch.randperm(nb + 3, generator=torch.Generator().manual_seed(seed))[:nb]
    cache = PagedLayerCache([(nk, nv)], nb + 3, bs, gpu, dtype)
    return cache, perm.to(torch.int32), torch.tensor([int(perm[j // bs]) * bs + j % bs for j in range(n_tokens)])


def _dyt(d, g, gpu, a):
    """(product parameters, oracle triple) of one elementwise norm."""
    from llm_weighted_consensus_amd.ops import res32

    w, b = torch.randn(d, generator=g), torch.randn(d, generator=g)
    return res32.Dyt(a, w.to(gpu), b.to(gpu)), (torch.tensor(a), w, b)


# ------------------------------------------------------------------ mechanisms, one by one
@pytest.mark.parametrize("act,ydt", [(F32, F32), (BF16, BF16), (BF16, F32)])
@pytest.mark.parametrize("S,d", [(1, 64), (2, 46), (3, 64), (4, 1028), (4, 33), (5, 48), (8, 30), (11, 64), (16, 24)])
def test_streams_update_and_next_norm(gpu, S, d, act, ydt):
    """One pass behind a sublayer: all streams from the old ones, the next input, its norm; with and without a bias; y as a
    column slice; rows chosen without storing; large inputs (a saturated tanh)."""
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(10 * S + d)
    T = 21
    X, y = torch.randn(S, T, d, generator=g), torch.randn(T, d + 4, generator=g).to(ydt)
    X[:, 3] *= 1e3
    mix, out, w_in, bias = torch.randn(S, S, generator=g), torch.randn(S, generator=g), torch.randn(S, generator=g), torch.randn(d, generator=g)
    nxt, ref_norm = _dyt(d, g, gpu, 0.7)
    coef = res32.hyper_coef(mix.to(gpu), out.to(gpu), w_in.to(gpu))
    tol = 2e-5 if act == F32 else 2e-2
    for bs in (bias, None):
        y64 = y.double()[:, :d] + (bs.double() if bs is not None else 0.0)
        Xr = O.hyper_out(X.double(), y64, mix.double(), out.double())
        hr = O.dyt(O.hyper_in(Xr, w_in.double()), *ref_norm)
        size = Xr.abs().amax((0, 2), keepdim=True).clamp_min(1.0)[0]                  # per row
        bad = 4e-7 * float(w_in.abs().sum()) * size * (S + 2)                          # fp32 sums in front of the tanh
        lim = tol * 4 + bad * float(ref_norm[1].abs().max())
        Xg = X.to(gpu)
        kw = dict(bias=None if bs is None else bs.to(gpu))
        h = res32.hyper_step(Xg, y.to(gpu)[:, :d], coef, nxt, act, **kw)
        assert ((Xg.cpu().double() - Xr).abs() / size).max() < 4e-6 and ((h.cpu().double() - hr).abs() < lim).all()
        for rows in ([20, 0, 7], None):
            Xg = X.to(gpu)
            h = res32.hyper_step(Xg, y.to(gpu)[:, :d], coef, nxt, act, rows=None if rows is None else torch.tensor(rows, device=gpu),
                                 write=False, **kw)
            assert torch.equal(Xg.cpu(), X) and ((h.cpu().double() - hr[rows or slice(None)]).abs() < lim[rows or slice(None)]).all()


@pytest.mark.parametrize("S,d,P", [(2, 64, 4), (3, 46, 2), (6, 40, 3)])
def test_streams_update_from_partial_products(gpu, S, d, P):
    """The result as planes of a split GEMM: their sum enters the streams."""
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(d)
    X, y = torch.randn(S, 5, d, generator=g), torch.randn(P, 5, d, generator=g)
    coef, bias = torch.randn(S * S + 2 * S, generator=g).to(gpu), torch.randn(d, generator=g).to(gpu)
    nxt, _ = _dyt(d, g, gpu, 0.7)
    a, b = X.to(gpu), X.to(gpu)
    ha = res32.hyper_step(a, y.to(gpu), coef, nxt, BF16, bias=bias)
    hb = res32.hyper_step(b, y.to(gpu).sum(0), coef, nxt, BF16, bias=bias)
    assert (a - b).abs().max() < 1e-5 * S and (ha.float() - hb.float()).abs().max() < 0.05
    rows = torch.tensor([4, 1], device=gpu)
    assert torch.equal(res32.hyper_step(X.to(gpu), y.to(gpu), coef, nxt, BF16, bias=bias, rows=rows, write=False), ha[rows])


def test_split_down_projection(gpu, tmp_path):
    """A feed-forward wide enough for the split form: decode steps with it (forced) and without give the oracle's logits."""
    cfg = O.make_config(64, 90, [O.attention_layer(2, 1, 16, 16, 4096), O.latent_layer(2, 16, 8, 16, 32, 9, 4160)], streams=2)
    W = O.make_weights(cfg, 2)
    model, eng = _engine(_save(tmp_path / "m", cfg, W), 90, BF16)
    pairs = model._split_weights()
    assert len(pairs) == 2 and all(s is not None and s.shape == (8, w.shape[1] // 8, 64) for w, s in pairs)
    toks = _tokens(30, 90, 3)
    ref = O.forward(cfg, W, toks)
    for forced in (False, True):
        model._split_for = {(1, *w.shape) for w, _ in pairs} if forced else set()
        got = [eng.step_tokens([("s", toks[:20], list(range(20)))])]
        got += [eng.step_tokens([("s", [t], [0])], ["s"] if i == 9 else []) for i, t in enumerate(toks[20:])]
        assert _err(torch.cat(got), ref, BF16) < TOL[BF16]


@pytest.mark.parametrize("dtype,tol", DTYPES)
@pytest.mark.parametrize("S,d", [(1, 46), (3, 64), (6, 40)])
def test_streams_start_as_the_normed_embedding(gpu, S, d, dtype, tol):
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(d)
    E, tok, w_in = torch.randn(30, d, generator=g).to(dtype), torch.tensor([3, 29, 0, 3], dtype=torch.int32), torch.randn(S, generator=g)
    ne, re = _dyt(d, g, gpu, 0.3)
    nx, rx = _dyt(d, g, gpu, 1.4)
    X, h = res32.embed_streams(E.to(gpu), tok.to(gpu), 6.5, ne, w_in.to(gpu), nx)
    x = O.dyt(E[tok.long()].double() * 6.5, *re)
    assert X.shape == (S, 4, d) and (X.cpu().double() - x[None]).abs().max() < 1e-5
    assert h.dtype == dtype and (h.cpu().double() - O.dyt(x * float(w_in.double().sum()), *rx)).abs().max() < tol * 4


@pytest.mark.parametrize("dtype,tol", DTYPES)
@pytest.mark.parametrize("n", [64, 30, 513])
def test_squared_relu(gpu, dtype, tol, n):
    from llm_weighted_consensus_amd.ops import res32

    z = (3 * torch.randn(9, n + 4, generator=torch.Generator().manual_seed(n))).to(dtype)
    z[2, 4:] = -z[2, 4:].abs()
    got = res32.relu2(z.to(gpu)[:, 4:]).cpu().double()
    ref = torch.relu(z.double()[:, 4:]) ** 2
    assert ((got - ref).abs() < tol * ref.clamp_min(1.0)).all() and float(got[2].abs().sum()) == 0


@pytest.mark.parametrize("dtype,tol", DTYPES)
@pytest.mark.parametrize("H,Dv", [(3, 10), (5, 24), (16, 64)])
def test_gate_per_entry(gpu, dtype, tol, H, Dv):
    """A sigmoid gate for every entry over heads that lie padded, or as a batched product left them."""
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(H)
    T = 13
    z = (3 * torch.randn(T, 4 + H * Dv, generator=g)).to(dtype)
    o = torch.randn(T, H, Dv, generator=g).to(dtype)
    ref = (o.double().reshape(T, -1) * torch.sigmoid(z.double()[:, 4:]))
    for og in (torch.nn.functional.pad(o, (0, 6)).to(gpu)[:, :, :Dv], o.transpose(0, 1).contiguous().to(gpu).transpose(0, 1)):
        out = res32.head_gate_rows(og, z.to(gpu)[:, 4:], torch.empty(T, H * Dv, dtype=dtype, device=gpu))
        assert (out.cpu().double() - ref).abs().max() < tol * 4


@pytest.mark.parametrize("dtype,tol", [(F32, 2e-5), (BF16, 3e-2)])
@pytest.mark.parametrize("H,G,D,Dv,rd,Dk,Dvp", [(6, 2, 20, 12, 16, 32, 32), (4, 4, 32, 32, 32, 32, 32), (3, 1, 10, 7, 6, 10, 7),
                                                (8, 2, 64, 48, 0, 64, 64), (2, 1, 96, 128, 96, 128, 128), (5, 5, 12, 20, 4, 16, 20)])
def test_whole_projection_norms_rotation_and_cache_rows(gpu, dtype, tol, H, G, D, Dv, rd, Dk, Dvp):
    """q out, k and v in the cache: biases, norms over all heads at once, rotated first entries, zero padding; a slot of -1
    writes nothing; positions far from zero; without keys and values (another layer's are read)."""
    from llm_weighted_consensus_amd.models.cache import PagedLayerCache
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(D + H)
    T, bs, eps, scale, base = 8, 8, 1e-3, 0.37, 900.0
    nq, nk, nv = H * D, G * D, G * Dv
    src, bias = torch.randn(T, nq + nk + nv + 4, generator=g).to(dtype), torch.randn(nq + nk + nv, generator=g)
    wq, wk = torch.randn(nq, generator=g), torch.randn(nk, generator=g)
    pos = torch.tensor([0, 1, 2, 63, 64, 500, 1500, 4000])
    slots = torch.randperm(4 * bs, generator=g)[:T].to(torch.int32)
    slots[3] = -1
    live = slots >= 0
    cache = PagedLayerCache([(G * Dk, G * Dvp)], 4, bs, gpu, dtype)
    cache.pool.fill_(7.0)  # stale contents
    sc = {"factor": 4.0, "original": 50, "low": 1.0, "high": 3.0}
    f, m = res32.rope_frequencies(rd, base, sc, gpu) if rd else (None, 1.0)
    kw = dict(eps=eps, wq=wq.to(gpu), rot_dims=rd, freq=f, mult=m)
    args = (pos.int().to(gpu), slots.to(gpu), H, D, Dk, scale)
    q = res32.norm_rot_kv_write(src.to(gpu)[:, :nq + nk + nv], *args, wk=wk.to(gpu), bias=bias.to(gpu), k_cache=cache.k[0], v_cache=cache.v[0],
                                G=G, Dv=Dv, **kw)
    x = src.double()[:, :nq + nk + nv] + bias.double()
    fr = O.banded_frequencies(rd, base, sc) if rd else []
    qr = O.rotate_half(O.rms_norm(x[:, :nq], wq, eps).view(T, H, D), pos, fr) * scale
    kr = O.rotate_half(O.rms_norm(x[:, nq:nq + nk], wk, eps).view(T, G, D), pos, fr)
    vr = x[:, nq + nk:].view(T, G, Dv)
    far = 5e-4   # (angles are fp32 products: 4000 rad has a spacing of 2.4e-4)
    q = q.cpu().double()
    assert (q[..., :D] - qr).abs().max() < 2e-5 * 4 + far * float(qr.abs().max()) and float(q[..., D:].abs().sum()) == 0
    krow, vrow = (a.cpu().double() for a in cache.rows(0, slots[live].long().to(gpu)))
    krow, vrow = krow.view(-1, G, Dk), vrow.view(-1, G, Dvp)
    assert (krow[..., :D] - kr[live]).abs().max() < tol * 4 + far * float(kr.abs().max()) and float(krow[..., D:].abs().sum()) == 0
    assert (vrow[..., :Dv] - vr[live]).abs().max() < tol * 4 and float(vrow[..., Dv:].abs().sum()) == 0
    assert int((cache.k[0] == 7.0).all(-1).sum()) == 4 * bs - int(live.sum())   # no other token was touched
    only = res32.norm_rot_kv_write(src.to(gpu)[:, :nq], *args, bias=bias[:nq].contiguous().to(gpu), **kw)
    assert torch.equal(only.cpu().double(), q)
    bare = res32.norm_rot_kv_write(src.to(gpu)[:, :nq], *args, rot_dims=rd, freq=f)     # no norm, no bias
    ref = O.rotate_half(src.double()[:, :nq].view(T, H, D), pos, fr) * scale
    assert (bare.cpu().double()[..., :D] - ref).abs().max() < 1e-4 + far * float(ref.abs().max())


@pytest.mark.parametrize("dtype,tol", DTYPES)
@pytest.mark.parametrize("H,G,D,Dv,cap", [(6, 2, 32, 64, 1.5), (3, 1, 128, 128, 30.0), (20, 1, 64, 32, 0.3), (4, 4, 20, 12, 5.0),
                                          (5, 1, 320, 256, 2.0), (18, 1, 576, 512, 2.0)])
def test_capped_scores(gpu, dtype, tol, H, G, D, Dv, cap):
    """Scores far beyond the cap and well inside it: decode rows and a portion behind cached keys, in bf16 on every
    matrix-core kernel (one wide row shared by all heads too) and on the general kernel."""
    from llm_weighted_consensus_amd.ops import res32

    g = torch.Generator().manual_seed(D + H)
    n, bs = 145, 16
    cache, table, slots = _paged(n, bs, G * D, G * Dv, dtype, gpu, seed=D)
    K = torch.randn(n, G, D, generator=g).to(dtype)
    V = K[..., :Dv].clone() if D > 192 else torch.randn(n, G, Dv, generator=g).to(dtype)
    cache.set_rows(0, slots.to(gpu), K.view(n, -1).to(gpu), V.reshape(n, -1).to(gpu))
    q = torch.randn(n, H, D, generator=g) * 3 * cap * D ** -0.5
    q[40] *= 100.0
    if D == 576:
        q = q.to(BF16).float()   # (this row size takes q as its bf16 rounding)
    grp = [h // (H // G) for h in range(H)]
    s = torch.einsum("ihd,jhd->hij", q.double(), K.double()[:, grp])
    ref = torch.einsum("hij,jhv->ihv", O.masked_softmax(O.softcap(s, cap), O.visible(n)), V.double()[:, grp])
    plain = torch.einsum("hij,jhv->ihv", O.masked_softmax(s, O.visible(n)), V.double()[:, grp])
    assert (ref - plain).abs().max() > 0.1
    z, tab = torch.zeros(H, device=gpu), table[None].to(gpu)
    rows = [0, 1, 15, 16, 31, 32, 40, 127, 128, 144]
    out = torch.empty(len(rows), H * Dv, dtype=dtype, device=gpu)
    res32.window_attn(q[rows].reshape(len(rows), -1).to(gpu), cache.k[0], cache.v[0], torch.tensor(rows, dtype=torch.int32, device=gpu),
                      tab.expand(len(rows), -1).contiguous(), z, z, NO_WINDOW, out, H, G, cores=True, values_in_keys=D > 192, cap=cap)
    assert (out.cpu().double().view(len(rows), H, Dv) - ref[rows]).abs().max() < tol * 4
    a = 30
    out = torch.empty(n - a, H * Dv, dtype=dtype, device=gpu)
    res32.window_attn(q[a:].reshape(n - a, -1).to(gpu), cache.k[0], cache.v[0], torch.arange(a, n, dtype=torch.int32, device=gpu), tab, z, z,
                      NO_WINDOW, out, H, G, cu_q=torch.tensor([0, n - a], dtype=torch.int32, device=gpu),
                      k_lens=torch.tensor([n], dtype=torch.int32, device=gpu), max_q=n - a, cores=True, cap=cap)
    assert (out.cpu().double().view(n - a, H, Dv) - ref[a:]).abs().max() < tol * 4


# ------------------------------------------------------------------ the model through the engine
def _configs():
    return {
        # both mixers, layers without feed-forward, two layers that read another one's keys and values, partial rotation
        "mixed": dict(width=72, vocab=250, streams=3, layers=[
            O.attention_layer(6, 2, 20, 12, 56, rot_dims=16), O.latent_layer(4, 16, 8, 24, 40, 21, 90, scale=0.21, base=900.0),
            O.attention_layer(3, 3, 24, 28, None, softcap=1.1), O.attention_layer(6, 2, 20, 12, 40, rot_dims=16, softcap=9.0, kv_from=0),
            O.latent_layer(3, 24, 16, 20, 48, 37, None), O.attention_layer(3, 3, 24, 28, 33, kv_from=2, scale=0.3)]),
        # odd sizes everywhere: nothing a multiple of 8, one head, one stream, a window of 1 and of 2
        "odd": dict(width=46, vocab=131, streams=1, layers=[
            O.latent_layer(3, 10, 6, 14, 27, 1, 33, scale=0.3), O.attention_layer(5, 1, 9, 7, 19, rot_dims=6),
            O.latent_layer(1, 12, 2, 5, 26, 2, None), O.attention_layer(5, 1, 9, 7, None, rot_dims=6, kv_from=1), O.latent_layer(2, 7, 4, 9, 11, 30, 50)]),
        # attention only, five streams, heads of the matrix-core sizes as they are
        "dense": dict(width=64, vocab=200, streams=5, layers=[
            O.attention_layer(4, 2, 32, 64, 64), O.attention_layer(8, 1, 64, 32, 48, scaling=None), O.attention_layer(2, 1, 128, 128, 40)]),
        # latents only, two streams, a window longer than every prompt
        "latents": dict(width=64, vocab=200, streams=2, layers=[
            O.latent_layer(4, 32, 32, 32, 96, 20, 64), O.latent_layer(8, 16, 32, 16, 96, 400, 40, scaling=None)]),
        # cached rows of 192 / 128 and 320 / 256: portions over up-projected keys and values, decode rows on the staged kernel
        "rows": dict(width=64, vocab=200, streams=4, layers=[
            O.latent_layer(5, 24, 40, 32, 120, 33, 50), O.latent_layer(3, 48, 24, 40, 232, 17, 64), O.latent_layer(18, 16, 24, 32, 232, 50, 30)]),
        # 576 / 512 rows, rows that no kernel is built for (general kernel in decoding), 136-entry heads
        "rows576": dict(width=64, vocab=200, streams=2, layers=[
            O.latent_layer(17, 16, 64, 16, 328, 40, 40), O.latent_layer(2, 40, 8, 24, 140, 24, 50), O.attention_layer(3, 1, 136, 72, 24, rot_dims=40),
            O.attention_layer(2, 1, 200, 140, 24, rot_dims=64)]),
        # twenty heads over two, nine streams, a wide feed-forward
        "ragged": dict(width=50, vocab=97, streams=9, layers=[
            O.attention_layer(20, 2, 6, 5, 130, rot_dims=4), O.latent_layer(20, 6, 4, 5, 26, 9, 30)]),
    }


CONFIGS = _configs()


def _make(name, seed=0):
    cfg = json.loads(json.dumps(O.make_config(**CONFIGS[name])))
    return cfg, O.make_weights(cfg, seed)


def _save(path, cfg, W):
    from safetensors.torch import save_file

    path.mkdir(exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in W.items()}, str(path / "model.safetensors"))
    return str(path)


def _engine(mdir, vocab, dtype, **engine_kw):
    from llm_weighted_consensus_amd.engine.engine import LLMEngine
    from llm_weighted_consensus_amd.engine.tokenizer import load_tokenizer
    from llm_weighted_consensus_amd.models.registry import load_model

    model = load_model(mdir, dtype=dtype)
    kw = dict(block_size=16, num_blocks=24, max_batch=4, max_model_len=256, use_graphs=False, prefix_sharing=False, tune_gc=False)
    kw.update(engine_kw)
    return model, LLMEngine(model, load_tokenizer({}, vocab), **kw)


def _build(tmp_path, name, dtype, seed=0, **engine_kw):
    cfg, W = _make(name, seed)
    return (cfg, W, *_engine(_save(tmp_path / f"{name}-{seed}", cfg, W), cfg["vocab"], dtype, **engine_kw))


def _tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def _err(got, ref, dtype=F32):
    """fp32: the largest difference relative to the reference's largest entry (at least 1).  bf16: the largest row-wise
    relative RMS difference."""
    d, ref = got.cpu().double() - ref, ref.double()
    if dtype == F32:
        return float(d.abs().max()) / max(1.0, float(ref.abs().max()))
    return float((d.pow(2).mean(-1).sqrt() / ref.pow(2).mean(-1).sqrt().clamp_min(1e-3)).max())


TOL = {F32: 1e-4, BF16: 0.12}
ALL = tuple(CONFIGS)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("name", ALL)
def test_whole_prompt_and_every_layer(gpu, tmp_path, name, dtype):
    """A whole prompt in one step: the streams' sum after every layer and the logits."""
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
    assert eng.bm.num_free == eng.bm.num_blocks and eng.state is None


def test_row_sizes_and_shared_caches(gpu, tmp_path):
    """Which cached row sizes the configurations above reach, and that a layer with kv_from has no pages of its own."""
    want = {"dense": [(64, 128), (64, 32), (128, 128)], "latents": [(128, 128), (128, 128)], "rows": [(192, 128), (320, 256), (320, 256)],
            "rows576": [(576, 512), (152, 144), (192, 128), (200, 140)], "mixed": [(64, 64), (64, 64), (96, 96), (64, 64)]}
    for name, dims in want.items():
        _, _, model, _ = _build(tmp_path, name, BF16)
        assert [tuple(d) for d in model._layer_dims()] == dims, name
    _, _, model, _ = _build(tmp_path, "mixed", F32)
    assert model.cache_index == {0: 0, 1: 1, 2: 2, 3: 0, 4: 3, 5: 2} and not model.has_state


def test_a_layer_reads_the_named_layers_keys(gpu, tmp_path):
    """The oracle with kv_from pointing at the other source differs (so the test would see it); the model follows the
    right one, in a prompt and in decoding."""
    layers = [O.attention_layer(4, 2, 12, 10, None), O.attention_layer(4, 2, 12, 10, 40), O.attention_layer(4, 2, 12, 10, None, softcap=2.0, kv_from=0)]
    cfg = O.make_config(40, 90, layers, streams=2)
    W = O.make_weights(cfg, 3)
    other = json.loads(json.dumps(cfg))
    other["layers"][2]["mixer"]["kv_from"] = 1
    toks = _tokens(30, 90, 4)
    ref, wrong = O.forward(cfg, W, toks), O.forward(other, W, toks)
    assert float((ref - wrong).abs().max()) > 0.1
    for c, r in ((cfg, ref), (other, wrong)):
        model, eng = _engine(_save(tmp_path / str(c["layers"][2]["mixer"]["kv_from"]), c, W), 90, F32, num_blocks=8, max_model_len=64)
        got = [eng.step_tokens([("s", toks[:20], list(range(20)))])]
        got += [eng.step_tokens([("s", [t], [0])]) for t in toks[20:]]
        assert _err(torch.cat(got), r) < TOL[F32]


CHANGES = {
    "eps": lambda c: c["norm"].update(eps=0.5), "embed": lambda c: c["embedding"].update(scale=1.5),
    "softcap": lambda c: c["layers"][0]["mixer"].update(softcap=0.4), "no_softcap": lambda c: c["layers"][0]["mixer"].update(softcap=1e4),
    "scale": lambda c: c["layers"][0]["mixer"].update(scale=0.05), "latent_scale": lambda c: c["layers"][1]["mixer"].update(scale=0.03),
    "window": lambda c: c["layers"][1]["mixer"]["mask"].update(size=20), "base": lambda c: c["layers"][0]["mixer"]["rot"].update(base=31.0),
    "latent_base": lambda c: c["layers"][1]["mixer"]["rot"].update(base=41.0), "rot_dims": lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10),
    "factor": lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=1.5),
    "low": lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(low=0.2), "high": lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(high=60.0),
    "original": lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(original=700),
    "latent_factor": lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(factor=8.0),
    "fast": lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(fast=1.5), "slow": lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(slow=0.01),
    "latent_original": lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(original=4000),
    "plain": lambda c: [c["layers"][i]["mixer"]["rot"].pop("scaling") for i in (0, 1, 3)]}


@pytest.mark.parametrize("change", sorted(CHANGES))
def test_every_constant_is_read_from_the_config(gpu, tmp_path, change):
    """One constant changed in the folder's config: the model's logits follow the oracle's, which move."""
    cfg, W = _make("mixed", 6)
    toks = _tokens(40, cfg["vocab"], 7)
    before = O.forward(cfg, W, toks)
    c = json.loads(json.dumps(cfg))
    CHANGES[change](c)
    ref = O.forward(c, W, toks)
    assert float((ref - before).abs().max()) > 4e-3
    model, eng = _engine(_save(tmp_path / change, c, W), c["vocab"], F32, num_blocks=8, max_model_len=64)
    got = eng.step_tokens([("w", toks, list(range(40)))], ["w"])
    assert _err(got, ref) < TOL[F32]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("C,R,window", [(24, 8, 19), (40, 24, 32), (120, 40, 33), (232, 24, 17), (328, 64, 48), (28, 4, 1)])
def test_window_edges(gpu, tmp_path, C, R, window, dtype):
    """One windowed layer whose scores single out one marked token by far: rows that still see it differ from rows that do
    not, at both sides of the window's edge, with the mark at page and tile borders and at the first token; portions cut in
    the window and single tokens give the same.  The oracle with a window one longer or shorter differs at the edge."""
    d, V, n = 32, 12, 120
    cfg = O.make_config(d, V, [O.latent_layer(2, 16, R, 16, C, window, None, scale=0.5, scaling=None)], streams=2)
    W = O.make_weights(cfg, 5)
    g = torch.Generator().manual_seed(C)
    # token 1's latent is parallel to every query's absorbed direction: the embedding of token 1 is set apart
    W["embed"][:] = (0.02 * torch.randn(V, d, generator=g)).to(BF16)
    W["embed"][:, 0] = 1.0
    W["embed"][1, 1] = 4.0
    W["embed.norm.alpha"] = torch.tensor(1.0, dtype=BF16)
    for nm in ("embed.norm", "l0.norm1"):
        W[nm][:], W[nm + ".b"][:] = 1.0, 0.0
    W["l0.norm1.alpha"], W["l0.hc1.in"] = torch.tensor(1.0, dtype=BF16), torch.tensor([1.0, 0.0], dtype=BF16)
    q, dkv, uk = torch.zeros(2 * (16 + R), d), 0.05 * torch.randn(C + R, d, generator=g), torch.zeros(2 * 16, C)
    q[0, 0] = q[16 + R, 0] = 6.0            # every query: entry 0 of both heads
    dkv[0, :], dkv[0, 1] = 0.0, 8.0         # the marked token's latent: entry 0
    dkv[1, 0] = 1.0
    uk[0, 0] = uk[16, 0] = 1.0
    W["l0.mix.q"], W["l0.mix.dkv"], W["l0.mix.uk"] = q.to(BF16), dkv.to(BF16), uk.to(BF16)
    W["l0.mix.dkv.norm"][:] = 1.0
    for mark in (0, 15, 16, 31, 32, 40):
        toks = _tokens(n, V - 2, mark)
        toks = [t + 2 for t in toks]
        toks[mark] = 1
        ref = O.forward(cfg, W, toks)
        for other in (window - 1, window + 1):
            if other:
                c2 = json.loads(json.dumps(cfg))
                c2["layers"][0]["mixer"]["mask"]["size"] = other
                e = (O.forward(c2, W, toks) - ref).abs().amax(-1)
                edge = mark + min(other, window)
                assert edge >= n or e[edge] > 0.1, (mark, other, float(e[edge]))
        if mark == 0:
            model, eng = _engine(_save(tmp_path / "m", cfg, W), V, dtype)
        for sizes in ([n], [mark + max(window - 2, 1), 2, 3] + [1] * 6 + [n], [7, 30, 2, 2, 41, n]):
            rows, a = [], 0
            for k in sizes:
                k = min(k, n - a)
                if k:
                    rows.append(eng.step_tokens([("s", toks[a:a + k], list(range(k)))], ["s"] if a + k == n else []))
                    a += k
            assert _err(torch.cat(rows), ref, dtype) < (TOL[F32] if dtype == F32 else 0.05), (mark, sizes[:2])


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_far_key_of_an_attention_layer(gpu, tmp_path, dtype):
    """An attention layer whose marked token takes almost all the weight hundreds of tokens later, through the cap: at the
    first token, at page borders and next to the row, in a prompt and in decoding; a second layer reads the same cache."""
    d, V, n = 32, 12, 300
    cfg = O.make_config(d, V, [O.attention_layer(4, 2, 16, 12, None, softcap=12.0, scale=1.0, rot_dims=4),
                               O.attention_layer(4, 2, 16, 12, None, softcap=10.0, scale=1.0, rot_dims=4, kv_from=0)], streams=2)
    W = O.make_weights(cfg, 8)
    g = torch.Generator().manual_seed(1)
    W["embed"][:] = (0.02 * torch.randn(V, d, generator=g)).to(BF16)
    W["embed"][:, 0], W["embed"][:, 1] = 1.0, 0.0
    W["embed"][1, 1] = 4.0
    for nm in ("embed.norm", "l0.norm1", "l1.norm1"):
        W[nm][:], W[nm + ".b"][:], W[nm + ".alpha"] = 1.0, 0.0, torch.tensor(1.0, dtype=BF16)
    W["l0.hc1.in"] = torch.tensor([1.0, 0.0], dtype=BF16)
    for p in ("l0.", "l1."):
        q = torch.zeros(64, d)
        q[8::16, 0] = 3.0                        # every head's entry 8 (not rotated)
        W[p + "mix.q"], W[p + "mix.q.b"] = q.to(BF16), torch.zeros(64, dtype=BF16)
        W[p + "mix.q.norm"] = torch.full((64,), 3.0, dtype=BF16)
    k = 0.3 * torch.randn(32, d, generator=g)
    k[8::16, :] = 0.0
    k[8::16, 1] = 20.0                           # the marked token's keys: entry 8
    W["l0.mix.v"] = (W["l0.mix.v"].float() * 3).to(BF16)
    W["l0.mix.k"], W["l0.mix.k.b"], W["l0.mix.k.norm"] = k.to(BF16), torch.randn(32, generator=g).to(BF16), torch.full((32,), 1.0, dtype=BF16)
    W["l0.mix.k.b"][8::16] = 0.0
    model, eng = _engine(_save(tmp_path / "m", cfg, W), V, dtype, num_blocks=40, max_model_len=512)
    for mark in (0, 15, 16, 31, 128, 298):
        toks = [t + 2 for t in _tokens(n, V - 2, 50 + mark)]
        toks[mark] = 1
        ref = O.forward(cfg, W, toks)
        without = O.forward(cfg, W, toks[:mark] + [2] + toks[mark + 1:])
        assert float((ref[-1] - without[-1]).abs().max()) > 0.3, float((ref[-1] - without[-1]).abs().max())
        rows = [eng.step_tokens([("s", toks[:n - 30], list(range(n - 30)))])]
        rows += [eng.step_tokens([("s", [t], [0])], ["s"] if i == 29 else []) for i, t in enumerate(toks[n - 30:])]
        assert _err(torch.cat(rows), ref, dtype) < (TOL[F32] if dtype == F32 else 0.06), mark


@pytest.mark.parametrize("name,dtype", [("mixed", F32), ("odd", F32), ("dense", BF16), ("rows", BF16), ("latents", BF16)])
def test_few_wanted_rows_and_what_they_leave(gpu, tmp_path, name, dtype):
    """A prompt of which only a few rows are wanted (the last layer then attends on these rows only): the same logits, and
    the cache it leaves carries the decoding that follows; two prompts in one step."""
    cfg, W, model, eng = _build(tmp_path, name, dtype)
    toks, more = _tokens(60, cfg["vocab"], 6), _tokens(33, cfg["vocab"], 61)
    ref, ref2 = O.forward(cfg, W, toks), O.forward(cfg, W, more)
    got = eng.step_tokens([("k", toks[:50], [49, 3]), ("j", more, [32, 0, 17])], ["j"])
    assert _err(got, torch.cat([ref[[49, 3]], ref2[[32, 0, 17]]]), dtype) < TOL[dtype]
    got = [eng.step_tokens([("k", [toks[i]], [0])], ["k"] if i == 59 else []) for i in range(50, 60)]
    assert _err(torch.cat(got), ref[50:], dtype) < TOL[dtype]


@pytest.mark.parametrize("name,dtype", [(n, F32) for n in ("mixed", "odd", "ragged")]
                         + [(n, BF16) for n in ("mixed", "dense", "latents", "rows", "rows576", "ragged")])
def test_decode_token_by_token_and_portions(gpu, tmp_path, name, dtype):
    """The same logits whether a prompt comes whole, token by token from the first token on, or in portions of
    changing sizes (down to two tokens; cut inside pages and windows)."""
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
    assert eng.bm.num_free == eng.bm.num_blocks


@pytest.mark.parametrize("name,dtype", [("mixed", F32), ("odd", F32), ("mixed", BF16), ("dense", BF16), ("rows", BF16), ("rows576", BF16)])
def test_unequal_batches_and_pages_used_again(gpu, tmp_path, name, dtype):
    """Up to four live sequences of unequal lengths, portions beside single tokens, one sitting steps out, in a pool
    so small that pages are freed and taken again; every position equals the sequence run alone."""
    cfg, W, model, eng = _build(tmp_path, name, dtype, num_blocks=8)   # (the sequences take 17 pages altogether)
    seqs = {k: _tokens(n, cfg["vocab"], 10 + i) for i, (k, n) in enumerate([("a", 70), ("b", 12), ("c", 40), ("d", 33), ("e", 58), ("f", 1)])}
    ref = {k: O.forward(cfg, W, t) for k, t in seqs.items()}
    at = {k: 0 for k in seqs}
    plan = [[("a", 30), ("b", 2)], [("a", 1), ("b", 7), ("c", 17)], [("a", 1), ("c", 1), ("d", 33), ("b", 3)], [("a", 2), ("c", 22)],
            [("a", 36)], [("e", 20), ("f", 1)], [("e", 1)], [("e", 37)]]
    gots, refs = [], []
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
    assert all(at[k] == len(seqs[k]) for k in seqs)
    assert _err(torch.cat(gots), torch.cat(refs), dtype) < TOL[dtype]
    assert eng.bm.num_free == eng.bm.num_blocks


@pytest.mark.parametrize("name,dtype", [("mixed", F32), ("rows", BF16)])
def test_long_decoding(gpu, tmp_path, name, dtype):
    """220 tokens decoded one by one after a short prompt (pages cross, windows pass over decoded tokens)."""
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
    """engine.generate (admission, paged prefill, batched decode steps, the fused sampler at temperature 0; with hipGraph
    replay of the decode step when ``graphs``) against the oracle's greedy continuation, twice on one engine so that pages
    come back dirty."""
    from llm_weighted_consensus_amd.engine.sampling import SamplingParams

    cfg, W, model, eng = _build(tmp_path, "mixed", F32, use_graphs=graphs, num_blocks=40)
    for seeds in ((21, 22), (23, 24)):
        prompts = [_tokens(23, 250, seeds[0]), _tokens(5, 250, seeds[1])]
        out = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=40, ignore_eos=True))
        for p, o in zip(prompts, out):
            assert len(o[0]) == 40
            _check_greedy(cfg, W, p, o[0])
    assert eng.bm.num_free == eng.bm.num_blocks


@pytest.mark.parametrize("name", ["dense", "rows"])
def test_captured_decode_steps_equal_eager_ones(gpu, tmp_path, name):
    """bf16 generation with and without hipGraph replay over the matrix-core paths: the same tokens."""
    from llm_weighted_consensus_amd.engine.sampling import SamplingParams

    outs = []
    for graphs in (False, True):
        cfg, W, model, eng = _build(tmp_path, name, BF16, use_graphs=graphs, num_blocks=40)
        prompts = [_tokens(23, 200, 51), _tokens(7, 200, 52), _tokens(60, 200, 53)]
        outs.append([o[0] for o in eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=24, ignore_eos=True))])
    same = sum(a == b for x, y in zip(*outs) for a, b in zip(x, y))
    assert same >= 0.8 * 72   # (the captured step may run other GEMM backends: a near-tie may fall the other way)


def test_generation_chunked_prefill_prefix_cache_and_forks(gpu, tmp_path):
    """Chunked prefill (prompt portions beside running decodes), n > 1 (forked sequences on shared prompt pages) and a prefix
    cache (this design carries nothing beside its pages, so a second prompt starts behind the first one's blocks) give the
    greedy continuation too."""
    from llm_weighted_consensus_amd.engine.sampling import SamplingParams

    cfg, W, model, eng = _build(tmp_path, "mixed", F32, num_blocks=64, chunked_prefill=8, max_batch=8, prefix_caching=True)
    prompts = [_tokens(37, 250, 31), _tokens(12, 250, 32)]
    for _ in range(2):
        out = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=20, ignore_eos=True), n=2)
        for p, o in zip(prompts, out):
            assert len(o) == 2 and o[0] == o[1]  # greedy forks of one prompt agree
            _check_greedy(cfg, W, p, o[0])
    assert eng.stats["prefix_cache_tokens"] >= 32


def test_server_worker_factory_and_seeded_sampling(gpu, tmp_path):
    """The server's worker factory on a model folder of the design: prefix caching stays on, no state pool; greedy and
    seeded top-k generation work."""
    from llm_weighted_consensus_amd.engine.group import build_engine
    from llm_weighted_consensus_amd.engine.sampling import SamplingParams

    cfg, W = _make("mixed", 2)
    eng = build_engine({"model_dir": _save(tmp_path / "m", cfg, W), "dtype": "float32", "max_batch": 4, "max_model_len": 128,
                        "kv_fraction": 0.001}, 0)
    assert eng.state is None and eng.prefix_caching
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
    interleaved (portions beside single tokens, one sitting a step out), pages given back at ``end``."""
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
    bad["l1.mix.g"] = torch.zeros(5, cfg["width"], dtype=BF16)
    with pytest.raises(ValueError):
        load_model(_save(tmp_path / "bad", cfg, bad))
    bad["l1.mix.g"] = W["l1.mix.g"]
    del bad["l0.hc2.mix"]
    with pytest.raises(KeyError):
        load_model(_save(tmp_path / "bad2", cfg, bad))
