"""Plain float64 oracle of the Gefilix design, one function per mechanism (CPU, slow, whole sequences at once).

It shares no code with the product path: weights come as a dict name -> tensor, the configuration as the dict that
a model folder's config.json holds.  Notation: T tokens of ONE sequence at positions 0 .. T-1, d the width.

    norm         x / sqrt(mean(x^2) + eps) * w
    layer        x = norm1(alpha x + mixer(x));  x = norm2(alpha x + ff(x))        (no norm in front of a sublayer)
    latent attn  keys / values through one low-rank latent per token, one rotated key part shared by all heads, causal
                 softmax, one sigmoid gate per head; a layer may read another layer's latents
    lightning    q, k, v = silu(projections);  S_t = a_h S_(t-1) + k_t v_t^T;  o_t = S_t^T q_t;  one RMS norm over all
                 heads together, sigmoid gate per entry
    dense ff     Wd gelu(Wu h)                                                     (erf form)
    experts      sigmoid scores, the best groups by the sum of their two largest scores, top-k among their experts,
                 weights = scores / (their sum + 1e-20) * scale; clamped gated experts + a gated shared expert
"""
from __future__ import annotations

import math
from typing import Callable, Dict, List, Optional

import torch

F64 = torch.float64


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w.to(F64)


def silu(z):
    return z / (1.0 + torch.exp(-z))


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def rotate_pairs(x, positions, base: float):
    """x [T, ..., n]: the pair (2i, 2i + 1) turned by position * base^(-2i / n)."""
    n = x.shape[-1]
    i = torch.arange(n // 2, dtype=F64)
    a = positions.to(F64)[:, None] * (base ** (-2.0 * i / n))[None, :]
    shape = [x.shape[0]] + [1] * (x.dim() - 2) + [n // 2]
    c, s = torch.cos(a).view(shape), torch.sin(a).view(shape)
    u, v = x[..., 0::2], x[..., 1::2]
    return torch.stack([u * c - v * s, v * c + u * s], -1).flatten(-2)


def latents(h, W: Callable[[str], torch.Tensor], m: dict, eps: float):
    """(c [T, kv_rank], rotated key part [T, rot_dim]) of a layer that has its own down-projection."""
    C = int(m["kv_rank"])
    z = h @ W("dkv").T
    return rms_norm(z[:, :C], W("dkv.norm"), eps), rotate_pairs(z[:, C:], torch.arange(h.shape[0]), float(m["rot"]["base"]))


def causal_softmax(s):
    """s [H, T, T] -> weights over the keys j <= i."""
    T = s.shape[-1]
    s = s.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), -math.inf)
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def latent_attention(h, W, m: dict, c, k_rot):
    """h [T, d], the latents and rotated key parts it attends over -> [T, d]."""
    T = h.shape[0]
    H, D, R, Dv = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"])
    q = (h @ W("q").T).view(T, H, D + R)
    q_rot = rotate_pairs(q[..., D:], torch.arange(T), float(m["rot"]["base"]))
    k = (c @ W("uk").T).view(T, H, D)
    v = (c @ W("uv").T).view(T, H, Dv)
    s = (torch.einsum("ihd,jhd->hij", q[..., :D], k) + torch.einsum("ihr,jr->hij", q_rot, k_rot)) * float(m["scale"])
    o = torch.einsum("hij,jhv->ihv", causal_softmax(s), v)
    o = o * torch.sigmoid(h @ W("g").T)[..., None]
    return o.reshape(T, H * Dv) @ W("o").T


def lightning_scan(q, k, v, decay, S=None):
    """q, k [T, H, D], v [T, H, Dv] -> (o [T, H, Dv], final state [H, D, Dv]), token by token."""
    T, H, D = q.shape
    a = torch.tensor(list(decay), dtype=F64)[:, None, None]
    S = torch.zeros(H, D, v.shape[-1], dtype=F64) if S is None else S.clone()
    o = torch.empty(T, H, v.shape[-1], dtype=F64)
    for t in range(T):
        S = a * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    return o, S


def lightning(h, W, m: dict, eps: float):
    T = h.shape[0]
    H, D, Dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q, k = (silu(h @ W(n).T).view(T, H, D) for n in "qk")
    o, _ = lightning_scan(q, k, silu(h @ W("v").T).view(T, H, Dv), m["decay"])
    o = rms_norm(o.reshape(T, H * Dv), W("norm"), eps) * torch.sigmoid(h @ W("g").T)
    return o @ W("o").T


def dense_ff(h, W, mlp: dict):
    return gelu_erf(h @ W("up").T) @ W("down").T


def clamped_unit(g, u, limit: float):
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def expert(h, W, name: str, limit: float):
    return clamped_unit(h @ W(name + ".gate").T, h @ W(name + ".up").T, limit) @ W(name + ".down").T


def route(h, W, r: dict):
    """(ids [T, top] from the largest score down, weights [T, top])."""
    s = torch.sigmoid(h @ W("router").T)
    E, n, keep = int(r["experts"]), int(r["groups"]["count"]), int(r["groups"]["keep"])
    size = E // n
    ids, wts = [], []
    for row in s:
        group = [sum(sorted(row[g * size:(g + 1) * size].tolist())[-2:]) for g in range(n)]
        best = sorted(range(n), key=lambda g: -group[g])[:keep]
        open_ = [e for e in range(E) if e // size in best]
        pick = sorted(open_, key=lambda e: -float(row[e]))[:int(r["top"])]
        w = row[pick]
        ids.append(pick)
        wts.append(w / (w.sum() + 1e-20) * float(r["scale"]))
    return torch.tensor(ids), torch.stack(wts)


def moe_ff(h, W, mlp: dict):
    ids, w = route(h, W, mlp["router"])
    out = torch.zeros_like(h)
    for e in range(int(mlp["router"]["experts"])):
        t, j = (ids == e).nonzero(as_tuple=True)
        if t.numel():
            out.index_add_(0, t, expert(h[t], W, f"e{e}", float(mlp["expert"]["limit"])) * w[t, j][:, None])
    return out + torch.sigmoid(h @ W("shared.sg").T) * expert(h, W, "shared", float(mlp["shared"]["limit"]))


def forward(cfg: dict, sd: Dict[str, torch.Tensor], tokens, streams: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence; ``streams`` collects the residual after every layer."""
    eps, alpha = float(cfg["norm"]["eps"]), float(cfg["postln_alpha"])

    def w(name):
        return sd[name].to(F64)

    x = w("embed")[torch.as_tensor(tokens, dtype=torch.long)] * float(cfg["embedding"]["scale"])
    lat: List = []
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        W = lambda n, p=p: w(p + "mix." + n)  # noqa: E731
        lat.append(None)
        if L["type"] == "latent_attention":
            lat[i] = lat[m["kv_from"]] if m.get("kv_from") is not None else latents(x, W, m, eps)
            y = latent_attention(x, W, m, *lat[i])
        elif L["type"] == "lightning":
            y = lightning(x, W, m, eps)
        else:
            raise ValueError(L["type"])
        x = rms_norm(alpha * x + y, w(p + "norm1"), eps)
        if L.get("mlp") is not None:
            ff = dense_ff if L["mlp"]["kind"] == "dense" else moe_ff
            x = rms_norm(alpha * x + ff(x, lambda n, p=p: w(p + "mlp." + n), L["mlp"]), w(p + "norm2"), eps)
        if streams is not None:
            streams.append(x.clone())
    return rms_norm(x, w("final.norm"), eps) @ w("head").T


# ------------------------------------------------------------------ small configurations and random weights for tests
def latent_layer(heads, dim, rot_dim, vdim, kv_rank, mlp, scale=None, base=3000.0, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
         "scale": scale if scale is not None else (dim + rot_dim) ** -0.5, "rot": {"base": base, "dims": rot_dim}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mlp": mlp, "mixer": m}


def lightning_layer(heads, dim, vdim, mlp, decay=None):
    decay = decay or [1.0 - 2.0 ** (-1 - 1.7 * h) for h in range(heads)]
    return {"type": "lightning", "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared, groups=(1, 1), limit=1.3, shared_limit=0.9, scale=1.7):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "shared": {"ff": shared, "limit": shared_limit},
            "router": {"experts": experts, "top": top, "scale": scale, "groups": {"count": groups[0], "keep": groups[1]}}}


def make_config(width, vocab, layers, eps=1e-5, alpha=1.6, embed_scale=5.0):
    return {"architecture": "Gefilix", "embedding": {"scale": embed_scale}, "layers": layers, "norm": {"eps": eps},
            "postln_alpha": alpha, "vocab": vocab, "width": width}


def make_weights(cfg: dict, seed: int = 0) -> Dict[str, torch.Tensor]:
    """bf16 tensors under the names a checkpoint of the design uses."""
    g = torch.Generator().manual_seed(seed)
    d, V = int(cfg["width"]), int(cfg["vocab"])

    def mat(o, i, s=1.0):
        return (torch.randn(o, i, generator=g) * s / math.sqrt(i)).to(torch.bfloat16)

    def vec(n, s=0.2, mean=1.0):
        return (mean + s * torch.randn(n, generator=g)).to(torch.bfloat16)

    W = {"embed": mat(V, d, 3.0), "final.norm": vec(d), "head": mat(V, d)}
    for i, L in enumerate(cfg["layers"]):
        p, m, e = f"l{i}.", L["mixer"], L.get("mlp")
        W[p + "norm1"] = vec(d)
        H, D, Dv = m["heads"], m["dim"], m["vdim"]
        if L["type"] == "latent_attention":
            R, C = m["rot_dim"], m["kv_rank"]
            W[p + "mix.q"] = mat(H * (D + R), d, 1.3)
            if m.get("kv_from") is None:
                W[p + "mix.dkv"], W[p + "mix.dkv.norm"] = mat(C + R, d, 2.0), vec(C)
            W[p + "mix.uk"], W[p + "mix.uv"], W[p + "mix.g"] = mat(H * D, C, 2.0), mat(H * Dv, C, 2.0), mat(H, d, 2.0)
        else:
            W[p + "mix.q"], W[p + "mix.k"], W[p + "mix.v"] = mat(H * D, d), mat(H * D, d), mat(H * Dv, d)
            W[p + "mix.g"], W[p + "mix.norm"] = mat(H * Dv, d, 2.0), vec(H * Dv)
        W[p + "mix.o"] = mat(d, H * Dv, 2.0)
        if e is None:
            continue
        W[p + "norm2"] = vec(d)
        if e["kind"] == "dense":
            W[p + "mlp.up"], W[p + "mlp.down"] = mat(e["ff"], d, 2.0), mat(d, e["ff"], 2.0)
        else:
            W[p + "mlp.router"] = mat(e["router"]["experts"], d, 2.0)
            for name, ff in [(f"e{x}", e["expert"]["ff"]) for x in range(e["router"]["experts"])] + [("shared", e["shared"]["ff"])]:
                W[f"{p}mlp.{name}.gate"], W[f"{p}mlp.{name}.up"], W[f"{p}mlp.{name}.down"] = mat(ff, d, 2.0), mat(ff, d, 2.0), mat(d, ff, 2.0)
            W[p + "mlp.shared.sg"] = mat(1, d, 2.0)
    return W
