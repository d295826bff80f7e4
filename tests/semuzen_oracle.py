"""Plain float64 oracle of the Semuzen design, one function per mechanism (CPU, slow, whole sequences at once).

It shares no code with the product path: weights come as a dict name -> tensor, the configuration as the dict that
a model folder's config.json holds.  Notation: T tokens of ONE sequence at positions 0 .. T-1, d the width, S the
number of parallel streams.

    dyt          tanh(a x) * w + b                                            (stands where other designs have a norm)
    sublayer     u = sum_s in_s X_s;  y = f(dyt(u));  X_t <- sum_s M[s, t] X_s + out_t y
    windowed     keys / values through one low-rank latent per token, one rotated key part shared by all heads, softmax
    latent attn  over the last `size` positions
    attention    grouped queries, biases, RMS norms over whole projections, partial rotation, capped scores, causal
                 softmax, a sigmoid gate per entry; a layer may read another layer's keys and values
    feed-forward Wd relu(Wu h)^2
"""
from __future__ import annotations

import math
from typing import Callable, Dict, Optional

import torch

F64 = torch.float64


def dyt(x, alpha, w, b):
    return torch.tanh(alpha.to(F64) * x) * w.to(F64) + b.to(F64)


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w.to(F64)


def plain_frequencies(n: int, base: float):
    return [base ** (-2.0 * i / n) for i in range(n // 2)]


def yarn_frequencies(n: int, base: float, sc: Optional[dict]):
    """(frequencies, multiplier of cos and sin): slow pairs divided by the factor, a linear ramp of the pair index."""
    f = plain_frequencies(n, base)
    if not sc:
        return f, 1.0
    turns = lambda t: n * math.log(sc["original"] / (2 * math.pi * t)) / (2 * math.log(base))  # noqa: E731
    lo, hi = max(math.floor(turns(sc["fast"])), 0), min(math.ceil(turns(sc["slow"])), n - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * r + fi * (1.0 - r))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def banded_frequencies(n: int, base: float, sc: Optional[dict]):
    """Short wavelengths kept, long ones stretched by the factor, a blend by original / wavelength between the two."""
    out = []
    for fi in plain_frequencies(n, base):
        if sc:
            wave = 2 * math.pi / fi
            if wave > sc["original"] / sc["low"]:
                fi = fi / sc["factor"]
            elif wave >= sc["original"] / sc["high"]:
                s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
                fi = (1.0 - s) * fi / sc["factor"] + s * fi
        out.append(fi)
    return out


def rotate_half(x, positions, freq, mult: float = 1.0):
    """x [T, ..., n]: entries (i, i + len(freq)) turned by position * freq[i], cos and sin times mult; the entries
    behind 2 len(freq) stay."""
    m = len(freq)
    a = positions.to(F64)[:, None] * torch.tensor(freq, dtype=F64)[None, :]
    shape = [x.shape[0]] + [1] * (x.dim() - 2) + [m]
    c, s = (torch.cos(a) * mult).view(shape), (torch.sin(a) * mult).view(shape)
    u, v = x[..., :m], x[..., m:2 * m]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * m:]], -1)


def visible(T: int, window: Optional[int] = None):
    """[T, T] bool: row i sees key j."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    ok = j <= i
    return ok if window is None else ok & (i - j < window)


def masked_softmax(s, ok):
    s = s.masked_fill(~ok, -math.inf)
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def softcap(s, cap: float):
    return cap * torch.tanh(s / cap)


def latent_attention(h, W: Callable[[str], torch.Tensor], m: dict, eps: float):
    T = h.shape[0]
    H, D, R, Dv, C = (int(m[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    pos = torch.arange(T)
    f, mult = yarn_frequencies(R, float(m["rot"]["base"]), m["rot"].get("scaling"))
    q = (h @ W("q").T).view(T, H, D + R)
    z = h @ W("dkv").T
    c, k_rot = rms_norm(z[:, :C], W("dkv.norm"), eps), rotate_half(z[:, C:], pos, f, mult)
    q_rot = rotate_half(q[..., D:], pos, f, mult)
    k = (c @ W("uk").T).view(T, H, D)
    v = (c @ W("uv").T).view(T, H, Dv)
    s = (torch.einsum("ihd,jhd->hij", q[..., :D], k) + torch.einsum("ihr,jr->hij", q_rot, k_rot)) * float(m["scale"])
    p = masked_softmax(s, visible(T, int(m["mask"]["size"])))
    return torch.einsum("hij,jhv->ihv", p, v).reshape(T, H * Dv) @ W("o").T


def keys_and_values(h, W, m: dict, eps: float):
    """(k [T, G, D] after norm and rotation, v [T, G, Dv]) of a layer with projections of its own."""
    T, G, D, Dv = h.shape[0], int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    k = rms_norm(h @ W("k").T + W("k.b"), W("k.norm"), eps).view(T, G, D)
    f = banded_frequencies(int(m["rot"]["dims"]), float(m["rot"]["base"]), m["rot"].get("scaling"))
    return rotate_half(k, torch.arange(T), f), (h @ W("v").T + W("v.b")).view(T, G, Dv)


def attention(h, W, m: dict, eps: float, k, v):
    T, H, G, D = h.shape[0], int(m["heads"]), int(m["kv_heads"]), int(m["dim"])
    q = rms_norm(h @ W("q").T + W("q.b"), W("q.norm"), eps).view(T, H, D)
    f = banded_frequencies(int(m["rot"]["dims"]), float(m["rot"]["base"]), m["rot"].get("scaling"))
    q = rotate_half(q, torch.arange(T), f)
    group = [x // (H // G) for x in range(H)]
    s = softcap(torch.einsum("ihd,jhd->hij", q, k[:, group]) * float(m["scale"]), float(m["softcap"]))
    o = torch.einsum("hij,jhv->ihv", masked_softmax(s, visible(T)), v[:, group]).reshape(T, -1)
    return (o * torch.sigmoid(h @ W("g").T)) @ W("o").T + W("o.b")


def relu2_ff(h, W):
    return torch.relu(h @ W("up").T) ** 2 @ W("down").T


def hyper_in(X, w_in):
    """X [S, T, d] -> the sublayer's input row before its norm."""
    return torch.einsum("s,std->td", w_in, X)


def hyper_out(X, y, mix, out):
    """All streams at once: X'_t = sum_s mix[s, t] X_s + out[t] y."""
    return torch.einsum("sr,std->rtd", mix, X) + out[:, None, None] * y[None]


def forward(cfg: dict, sd: Dict[str, torch.Tensor], tokens, streams: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence; ``streams`` collects the sum of the streams after every layer."""
    eps, S = float(cfg["norm"]["eps"]), int(cfg["streams"])

    def w(name):
        return sd[name].to(F64)

    def norm(name, x):
        return dyt(x, w(name + ".alpha"), w(name), w(name + ".b"))

    x = w("embed")[torch.as_tensor(tokens, dtype=torch.long)] * float(cfg["embedding"]["scale"])
    X = norm("embed.norm", x)[None].repeat(S, 1, 1)
    kv: Dict[int, tuple] = {}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        W = lambda n, p=p: w(p + "mix." + n)  # noqa: E731

        def mixer(h):
            if L["type"] == "latent_attention":
                return latent_attention(h, W, m, eps)
            if L["type"] != "attention":
                raise ValueError(L["type"])
            kv[i] = kv[m["kv_from"]] if m.get("kv_from") is not None else keys_and_values(h, W, m, eps)
            return attention(h, W, m, eps, *kv[i])

        subs = [("1", mixer)]
        if L.get("mlp") is not None:
            subs.append(("2", lambda h, p=p: relu2_ff(h, lambda n: w(p + "mlp." + n))))
        for n, f in subs:
            y = f(norm(p + "norm" + n, hyper_in(X, w(f"{p}hc{n}.in"))))
            X = hyper_out(X, y, w(f"{p}hc{n}.mix"), w(f"{p}hc{n}.out"))
        if streams is not None:
            streams.append(X.sum(0))
    return norm("final.norm", X.sum(0)) @ w("head").T


# ------------------------------------------------------------------ small configurations and random weights for tests
def latent_layer(heads, dim, rot_dim, vdim, kv_rank, window, ff, scale=None, base=3000.0, scaling=(3.0, 64, 8.0, 1.0)):
    """``scaling``: (factor, original, fast, slow) or None."""
    rot = {"base": base, "dims": rot_dim}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "mask": {"size": window},
         "scale": scale if scale is not None else (dim + rot_dim) ** -0.5, "rot": rot}
    return {"type": "latent_attention", "mlp": {"kind": "dense", "ff": ff} if ff else None, "mixer": m}


def attention_layer(heads, kv_heads, dim, vdim, ff, rot_dims=None, scale=None, softcap=4.0, base=2000.0, scaling=(5.0, 96, 1.0, 4.0),
                    kv_from=None):
    """``scaling``: (factor, original, low, high) or None."""
    rot = {"base": base, "dims": dim if rot_dims is None else rot_dims}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "original", "low", "high"), scaling))
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5,
         "softcap": softcap, "rot": rot}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mlp": {"kind": "dense", "ff": ff} if ff else None, "mixer": m}


def make_config(width, vocab, layers, streams=3, eps=1e-5, embed_scale=5.0):
    return {"architecture": "Semuzen", "embedding": {"scale": embed_scale}, "layers": layers, "norm": {"eps": eps},
            "streams": streams, "vocab": vocab, "width": width}


def make_weights(cfg: dict, seed: int = 0) -> Dict[str, torch.Tensor]:
    """bf16 tensors under the names a checkpoint of the design uses."""
    g = torch.Generator().manual_seed(seed)
    d, V, S = int(cfg["width"]), int(cfg["vocab"]), int(cfg["streams"])
    bf = torch.bfloat16

    def mat(o, i, s=1.0):
        return (torch.randn(o, i, generator=g) * s / math.sqrt(i)).to(bf)

    def vec(n, s=0.2, mean=1.0):
        return (mean + s * torch.randn(n, generator=g)).to(bf)

    W = {"embed": mat(V, d, 3.0), "head": mat(V, d)}

    def norm(name):
        W[name], W[name + ".b"] = vec(d), vec(d, 0.1, 0.0)
        W[name + ".alpha"] = (0.4 + 0.4 * torch.rand((), generator=g)).to(bf)

    norm("embed.norm")
    norm("final.norm")
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        for n in ("1", "2") if L["mlp"] else ("1",):
            norm(p + "norm" + n)
            W[f"{p}hc{n}.in"], W[f"{p}hc{n}.out"] = vec(S, 0.4, 1.0 / S), vec(S, 0.4, 0.8)
            W[f"{p}hc{n}.mix"] = (0.9 * torch.eye(S) + 0.25 * torch.randn(S, S, generator=g)).to(bf)
        H, D, Dv = m["heads"], m["dim"], m["vdim"]
        if L["type"] == "latent_attention":
            R, C = m["rot_dim"], m["kv_rank"]
            W[p + "mix.q"], W[p + "mix.dkv"], W[p + "mix.dkv.norm"] = mat(H * (D + R), d, 2.0), mat(C + R, d, 2.0), vec(C)
            W[p + "mix.uk"], W[p + "mix.uv"] = mat(H * D, C, 2.0), mat(H * Dv, C, 2.0)
        else:
            G = m["kv_heads"]
            W[p + "mix.q"], W[p + "mix.q.b"], W[p + "mix.q.norm"] = mat(H * D, d), vec(H * D, 0.4, 0.0), vec(H * D, 0.3, 1.6)
            if m.get("kv_from") is None:
                W[p + "mix.k"], W[p + "mix.k.b"], W[p + "mix.k.norm"] = mat(G * D, d), vec(G * D, 0.4, 0.0), vec(G * D, 0.3, 1.6)
                W[p + "mix.v"], W[p + "mix.v.b"] = mat(G * Dv, d), vec(G * Dv, 0.4, 0.0)
            W[p + "mix.g"], W[p + "mix.o.b"] = mat(H * Dv, d, 2.0), vec(d, 0.3, 0.0)
        W[p + "mix.o"] = mat(d, H * Dv, 1.5)
        if L["mlp"]:
            W[p + "mlp.up"], W[p + "mlp.down"] = mat(L["mlp"]["ff"], d, 1.2), mat(d, L["mlp"]["ff"], 1.2)
    return W
