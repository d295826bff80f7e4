"""Gefilix on the CPU: config parsing, the registry, and the plain oracle's own consistency (the GPU tests cover the
kernels and the model)."""
import json

import pytest
import torch

import gefilix_oracle as O

M = O.moe(8, 3, 24, 40, groups=(4, 2), limit=1.25, shared_limit=0.75, scale=1.5)
LAYERS = [O.lightning_layer(3, 20, 12, O.dense(50)), O.latent_layer(4, 16, 8, 24, 40, M, scale=0.21, base=700.0),
          O.latent_layer(2, 10, 6, 14, 27, None), O.latent_layer(3, 12, 8, 10, 40, O.dense(30), base=700.0, kv_from=1)]


def test_config_from_json_and_registry(tmp_path):
    from llm_weighted_consensus_amd.models.config import GefilixConfig, GeluFfSpec, GroupedExpertsSpec, load_model_config
    from llm_weighted_consensus_amd.models.registry import model_class

    cfg = O.make_config(44, 77, LAYERS, eps=1e-4, alpha=2.25, embed_scale=3.5)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    c = load_model_config(tmp_path)
    assert isinstance(c, GefilixConfig) and (c.vocab_size, c.hidden, c.norm_eps, c.alpha, c.embed_scale) == (77, 44, 1e-4, 2.25, 3.5)
    r, a, b, s = c.layer_specs
    assert (r.type, r.mixer.nq, r.mixer.nv, len(r.mixer.decay)) == ("lightning", 60, 36, 3)
    assert isinstance(r.mlp, GeluFfSpec) and r.mlp.ff == 50
    assert (a.mixer.nq, a.mixer.nv, a.mixer.kv_rank, a.mixer.scale, a.mixer.rot.base, a.mixer.kv_from) == (96, 96, 40, 0.21, 700.0, None)
    e = a.mlp
    assert isinstance(e, GroupedExpertsSpec)
    assert (e.experts, e.top, e.ff, e.limit, e.groups, e.keep, e.scale) == (8, 3, 24, 1.25, 4, 2, 1.5)
    assert (e.shared_ff, e.shared_limit, e.alpha) == (40, 0.75, 1.702)
    assert b.mlp is None and s.mixer.kv_from == 1 and b.mixer.rot.dims == 6
    assert model_class(c).__name__ == "GefilixModel" and c.layers == 4
    assert c.params() == sum(t.numel() for t in O.make_weights(cfg, 0).values())
    zero = json.loads(json.dumps(cfg))
    zero["layers"] = [LAYERS[2], dict(LAYERS[2], mixer=dict(LAYERS[2]["mixer"], kv_from=0))]
    assert GefilixConfig.from_dict(zero).layer_specs[1].mixer.kv_from == 0      # layer 0 is a source like any other


@pytest.mark.parametrize("path,value", [
    (("layers", 1, "mixer", "rot", "dims"), 6), (("layers", 0, "mixer", "decay"), [0.5]), (("layers", 0, "type"), "other"),
    (("layers", 1, "mlp", "kind"), "other"), (("layers", 1, "mlp", "router", "top"), 5),           # two groups of two hold 4
    (("layers", 1, "mlp", "router", "groups", "count"), 3), (("layers", 1, "mlp", "router", "groups", "keep"), 5),
    (("layers", 3, "mixer", "kv_from"), 0), (("layers", 3, "mixer", "kv_from"), 2), (("layers", 3, "mixer", "kv_from"), 3),
    (("layers", 3, "mixer", "rot", "base"), 701.0)])
def test_config_refuses_what_does_not_fit(path, value):
    from llm_weighted_consensus_amd.models.config import GefilixConfig

    bad = json.loads(json.dumps(O.make_config(44, 77, LAYERS)))
    node = bad
    for k in path[:-1]:
        node = node[k]
    node[path[-1]] = value
    with pytest.raises(ValueError):
        GefilixConfig.from_dict(bad)


def test_oracle_mechanisms_agree_with_their_definitions():
    """The oracle's own pieces: the scan equals the explicit double sum with decay powers and continues from a state;
    rotations keep lengths and depend on position differences only; softmax rows sum to one; the group choice against a
    hand-made case."""
    g = torch.Generator().manual_seed(0)
    T, H, D, Dv = 9, 2, 4, 3
    q, k, v = (torch.randn(T, H, n, generator=g, dtype=torch.float64) for n in (D, D, Dv))
    decay = [0.5, 0.9]
    o, S = O.lightning_scan(q, k, v, decay)
    for h in range(H):
        for i in range(T):
            ref = sum(decay[h] ** (i - j) * float(q[i, h] @ k[j, h]) * v[j, h] for j in range(i + 1))
            assert (o[i, h] - ref).abs().max() < 1e-12
    o2, S2 = O.lightning_scan(q[5:], k[5:], v[5:], decay, S=O.lightning_scan(q[:5], k[:5], v[:5], decay)[1])
    assert (o2 - o[5:]).abs().max() < 1e-12 and (S2 - S).abs().max() < 1e-12
    x, y = torch.randn(2, 1, 6, generator=g, dtype=torch.float64)
    at = lambda p, v: O.rotate_pairs(v, torch.tensor([p]), 100.0)[0]  # noqa: E731
    assert abs(float(at(7, x).norm() - x.norm())) < 1e-12
    assert abs(float(at(9, x) @ at(4, y) - at(5, x) @ at(0, y))) < 1e-12
    assert abs(float(at(3, torch.tensor([[1.0, 0, 0, 0]], dtype=torch.float64))[1]) - float(torch.sin(torch.tensor(3.0, dtype=torch.float64)))) < 1e-12
    p = O.causal_softmax(torch.randn(2, 5, 5, generator=g, dtype=torch.float64))
    assert (p.sum(-1) - 1).abs().max() < 1e-12 and float(p[:, 0, 1:].abs().sum()) == 0
    # three groups of two: group 0 holds the single best score, group 1 the best pair; one group kept
    z = torch.tensor([[2.0, -9.0, 1.0, 0.9, -1.0, -1.0]], dtype=torch.float64)
    ids, w = O.route(z, lambda n: torch.eye(6, dtype=torch.float64), {"experts": 6, "top": 2, "scale": 3.0, "groups": {"count": 3, "keep": 1}})
    s = torch.sigmoid(z[0, 2:4])
    assert ids.tolist() == [[2, 3]] and (w[0] - 3.0 * s / s.sum()).abs().max() < 1e-12
