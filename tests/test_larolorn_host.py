"""Larolorn without a GPU: configuration round trip, tensor inventory, the oracle's mechanisms on hand-made inputs whose results are
known by construction, and faults planted in the oracle, which must move the results of the models that the GPU tests run by far
more than those tests tolerate."""
import math

import pytest
import torch

from tests import larolorn_oracle as orc
from tests import test_gpu_larolorn as gt

F = torch.float64


def test_config_round_trip():
    from vllm_rust_amd.larolorn import LarolornSpec
    spec = gt.small_spec()
    cfg = spec.to_config()
    assert cfg["architecture"] == "Larolorn" and [e["type"] for e in cfg["layers"]] == ["latent_attention", "parallel", "latent_attention", "parallel", "parallel", "latent_attention"]
    assert cfg["layers"][5]["mlp"] is None and "weights_of" not in cfg["layers"][0] and cfg["layers"][2]["weights_of"] == 0
    assert set(cfg["layers"][1]["mixer"]) == {"left", "right"} and cfg["layers"][1]["mixer"]["left"]["mask"] == {"size": 9}
    again = LarolornSpec.from_config(cfg)
    assert again.to_config() == cfg and again.layers[2].weights_of == 0 and again.layers[0].weights_of is None and again.layers[1].decay == spec.layers[1].decay
    # what a configuration may leave out
    e = {"type": "parallel", "mixer": {"left": {"heads": 2, "dim": 16}, "right": {"heads": 1, "dim": 4, "decay": [0.5]}}, "mlp": None}
    f = {"type": "latent_attention", "mixer": {"heads": 2, "dim": 6, "rot_dim": 10, "kv_rank": 5}}
    p, l = LarolornSpec.from_config({"vocab": 5, "width": 8, "norm": {"eps": 1e-5}, "layers": [e, f]}).layers
    assert (p.kv_heads, p.vdim, p.scale, p.mask, p.rot.dims, p.r_vdim, p.mlp) == (2, 16, 0.25, 0, 0, 4, None)
    assert (l.vdim, l.scale, l.mask, l.mlp, l.weights_of) == (6, 0.25, 0, None, None)
    two = {"left": e["mixer"]["left"], "right": dict(e["mixer"]["right"], decay=[0.5, 0.5])}
    for bad in (dict(e, type="lightning"), dict(f, mlp={"kind": "moe"}), dict(e, mixer=two)):
        with pytest.raises(ValueError):
            LarolornSpec.from_config({"vocab": 5, "width": 8, "norm": {"eps": 1e-5}, "layers": [bad]})


def test_tensor_inventory_registry_and_oracle_runs():
    from vllm_rust_amd.larolorn import synthetic_weights
    from vllm_rust_amd.models import REGISTRY
    spec = gt.small_spec()
    shapes = spec.tensor_shapes()
    assert shapes["embed"] == shapes["head"] == (67, 40) and shapes["final.norm"] == (40,)
    assert shapes["l0.mix.q"] == (48, 40) and shapes["l0.mix.dkv"] == (26, 40) and shapes["l0.mix.uk"] == (30, 20) and shapes["l0.mix.uv"] == (42, 20)
    assert shapes["l0.mix.g"] == (3, 40) and shapes["l0.mix.o"] == (40, 42) and shapes["l0.mlp.down"] == (40, 36)
    assert shapes["l1.mix.left.k"] == (20, 40) and shapes["l1.mix.left.k.b"] == (20,) and shapes["l1.mix.left.q.norm"] == (60,) and shapes["l1.mix.left.v"] == (14, 40)
    assert shapes["l1.mix.left.o"] == (40, 42) and shapes["l1.mix.left.o.b"] == (40,) and shapes["l1.mix.left.sink"] == (6,) and shapes["l1.mix.left.out"] == (40,)
    assert shapes["l1.mix.right.q"] == (27, 40) and shapes["l1.mix.right.g"] == (33, 40) and shapes["l1.mix.right.norm"] == (33,) and shapes["l1.mix.right.out"] == (40,)
    assert not any(k.startswith(("l2.", "l4.")) for k in shapes) and "l5.norm2" not in shapes and shapes["l5.norm1"] == (40,)
    ck = synthetic_weights(spec, 0)
    assert set(ck) == set(shapes) and all(tuple(ck[k].shape) == shapes[k] and ck[k].dtype == torch.bfloat16 for k in ck)
    assert "Larolorn" in REGISTRY
    lg, tr = orc.forward(spec.to_config(), ck, [3, 1, 4, 1, 5, 9, 2, 6, 5, 3])
    assert lg.shape == (10, 67) and tr.shape == (6, 10, 40) and bool(torch.isfinite(lg).all())
    with orc.rounded_operands():
        lo, _ = orc.forward(spec.to_config(), ck, [3, 1, 4, 1, 5, 9, 2, 6, 5, 3])
    assert 1e-4 < float(gt.row_errs(lo, lg).mean()) < 0.1 and orc._rounding is None


def test_oracle_norm_rotation_and_activation():
    x = torch.tensor([[1.0, 3.0, 5.0, 7.0]], dtype=F)
    assert torch.allclose(orc.rms_unit(x, 0.0), x / math.sqrt(21.0)) and torch.allclose(orc.rms_norm(x, torch.full((4,), 2.0, dtype=F), 4.0), 2 * x / 5.0)
    v = torch.zeros(2, 1, 6, dtype=F)
    v[:, 0, 0], v[:, 0, 4], v[:, 0, 5] = 1.0, 7.0, 8.0
    r = orc.rotate_halves(v, [0, 3], dict(dims=4, base=10.0))
    assert torch.allclose(r[0], v[0]) and torch.allclose(r[1, 0], torch.tensor([math.cos(3.0), 0, math.sin(3.0), 0, 7.0, 8.0], dtype=F))
    r = orc.rotate_neighbours(v, [0, 3], dict(dims=4, base=10.0))
    assert torch.allclose(r[0], v[0]) and torch.allclose(r[1, 0], torch.tensor([math.cos(3.0), math.sin(3.0), 0, 0, 7.0, 8.0], dtype=F))
    v[:, 0] = 0.0
    v[:, 0, 1] = 1.0
    s = 3.0 * 10.0 ** -0.5                                         # the second pair's angle
    assert torch.allclose(orc.rotate_halves(v, [0, 3], dict(dims=4, base=10.0))[1, 0, :4], torch.tensor([0, math.cos(s), 0, math.sin(s)], dtype=F))
    # gate cut above only, up value cut on both sides
    g = torch.tensor([5.0, -5.0, 1.0, 1.0], dtype=F)
    u = torch.tensor([0.5, 0.5, 9.0, -9.0], dtype=F)
    sg = lambda z: z / (1 + math.exp(-1.702 * z))   # noqa: E731
    assert torch.allclose(orc.clamped_glu(g, u, 2.0), torch.tensor([sg(2.0) * 1.5, sg(-5.0) * 1.5, sg(1.0) * 3.0, -sg(1.0)], dtype=F))


def test_oracle_attention_and_memory_by_hand():
    assert [orc.window_start(i, 3) for i in range(6)] == [0, 0, 0, 1, 2, 3] and orc.window_start(9, 0) == 0
    assert [orc.chunk_start(i, 3) for i in range(7)] == [0, 0, 0, 3, 3, 3, 6] and orc.chunk_start(9, 0) == 0
    q, k = torch.zeros(4, 1, 2, dtype=F), torch.zeros(4, 1, 2, dtype=F)
    v = torch.tensor([1.0, 2.0, 4.0, 8.0], dtype=F).reshape(4, 1, 1)
    assert orc.softmax_attention(q, k, v, 1.0, lambda i: orc.window_start(i, 2)).flatten().tolist() == [1.0, 1.5, 3.0, 6.0]
    assert orc.softmax_attention(q, k, v, 1.0, lambda i: orc.chunk_start(i, 2)).flatten().tolist() == [1.0, 1.5, 4.0, 6.0]
    sink = torch.tensor([math.log(2.0)], dtype=F)                  # two more keys without a value
    assert torch.allclose(orc.softmax_attention(q, k, v, 1.0, lambda i: 0, sink).flatten(), torch.tensor([1 / 3, 3 / 4, 7 / 5, 15 / 6], dtype=F))
    k, v, q = (torch.tensor(x, dtype=F).reshape(3, 1, 1) for x in ([1.0, 2.0, -1.0], [5.0, -3.0, 4.0], [1.0, 1.0, 2.0]))
    assert orc.decayed_memory(q, k, v, [0.5]).flatten().tolist() == [5.0, 2.5 - 6.0, 2 * (0.5 * -3.5 - 4.0)]


def _per_head_norm(x, w, eps, f=orc.rms_norm):
    return f(x.reshape(x.shape[0], -1, 5), w.reshape(-1, 5), eps).reshape(x.shape) if x.shape[-1] in (60, 20) else f(x, w, eps)


FAULTS = {
    "window a token too long": ("window_start", lambda i, size, f=orc.window_start: f(i, size + 1)),
    "window a token too short": ("window_start", lambda i, size, f=orc.window_start: f(i, size - 1)),
    "no window": ("window_start", lambda i, size: 0),
    "chunks one position late": ("chunk_start", lambda i, size, f=orc.chunk_start: max(0, f(i + 1, size) - 1)),
    "a chunk as a window": ("chunk_start", lambda i, size, f=orc.window_start: f(i, size)),
    "no chunks": ("chunk_start", lambda i, size: 0),
    "sink left out": ("softmax_attention", lambda q, k, v, s, st, sink=None, f=orc.softmax_attention: f(q, k, v, s, st)),
    "sink scaled like a score": ("softmax_attention", lambda q, k, v, s, st, sink=None, f=orc.softmax_attention: f(q, k, v, s, st, None if sink is None else sink * s)),
    "neighbours rotated instead of halves": ("rotate_halves", orc.rotate_neighbours),
    "halves rotated instead of neighbours": ("rotate_neighbours", orc.rotate_halves),
    "key part one position late": ("rotate_neighbours", lambda x, p, rot, f=orc.rotate_neighbours: f(x, [i + 1 for i in p], rot) if x.shape[1] == 1 else f(x, p, rot)),
    "q and k normed in parts": ("rms_norm", _per_head_norm),
    "memory forgets before nothing": ("decayed_memory", lambda q, k, v, d, f=orc.decayed_memory: f(q, k, v, [1.0] * len(d))),
    "decays of the heads swapped": ("decayed_memory", lambda q, k, v, d, f=orc.decayed_memory: f(q, k, v, list(d)[::-1])),
    "read before the write": ("decayed_memory", lambda q, k, v, d, f=orc.decayed_memory: f(q, k, v, d) - (q * k).sum(-1, keepdim=True) * v),
    "no SiLU on the memory's inputs": ("silu", lambda z: z),
    "gate cut on both sides": ("clamped_glu", lambda g, u, c, f=orc.clamped_glu: f(torch.clamp(g, min=-c), u, c)),
    "no limit": ("clamped_glu", lambda g, u, c, f=orc.clamped_glu: f(g, u, 1e9)),
    "plain sigmoid slope": ("clamped_glu", lambda g, u, c: torch.clamp(g, max=c) * torch.sigmoid(torch.clamp(g, max=c)) * (torch.clamp(u, -c, c) + 1)),
    "no one added": ("clamped_glu", lambda g, u, c: torch.clamp(g, max=c) * torch.sigmoid(1.702 * torch.clamp(g, max=c)) * torch.clamp(u, -c, c)),
    "branches not normed": ("parallel", lambda h, w, p, m, eps: 0.5 * (orc.chunked_attention(h, w, p + "left.", m["left"], eps) + orc.lightning_attention(h, w, p + "right.", m["right"], eps))),
    "left branch alone": ("lightning_attention", lambda h, w, p, m, eps: torch.zeros_like(h)),
    "right branch alone": ("chunked_attention", lambda h, w, p, m, eps: torch.zeros_like(h)),
}


@pytest.mark.parametrize("name", list(FAULTS))
def test_planted_faults_show(monkeypatch, name):
    from vllm_rust_amd.larolorn import synthetic_weights
    spec = gt.small_spec()
    ck = synthetic_weights(spec, 0)
    toks = gt.tokens_for(spec, 53, 2)
    want = orc.forward(spec.to_config(), ck, toks)[0]
    monkeypatch.setattr(orc, *FAULTS[name])
    assert float(gt.row_errs(orc.forward(spec.to_config(), ck, toks)[0], want).max()) > 100 * gt.TOL["float32"]


@pytest.mark.parametrize("name,skip", [("l1.mix.left.q.b", 0.0), ("l1.mix.left.k.b", 0.0), ("l1.mix.left.v.b", 0.0), ("l1.mix.left.o.b", 0.0), ("l0.mix.dkv.norm", 1.0),
                                       ("l1.mix.left.out", 1.0), ("l1.mix.right.out", 1.0), ("l1.mix.right.norm", 1.0), ("l1.norm1", 1.0), ("l0.norm2", 1.0), ("final.norm", 1.0),
                                       ("l0.mix.g", 0.0), ("l1.mix.right.g", 0.0)])
def test_every_small_tensor_counts(name, skip):
    from vllm_rust_amd.larolorn import synthetic_weights
    spec = gt.small_spec()
    ck = synthetic_weights(spec, 0)
    toks = gt.tokens_for(spec, 53, 2)
    want = orc.forward(spec.to_config(), ck, toks)[0]
    ck[name] = torch.full_like(ck[name], skip)
    assert float(gt.row_errs(orc.forward(spec.to_config(), ck, toks)[0], want).max()) > 20 * gt.TOL["float32"]


def test_scale_faults_show_where_eps_is_large(monkeypatch):
    """The norm behind the two branches hides a missing half, and the one behind the memory its scale, unless eps is of the order of
    the squares: what the large-eps GPU test relies on."""
    from vllm_rust_amd.larolorn import synthetic_weights
    spec = gt.small_spec(norm_eps=0.5)
    ck = synthetic_weights(spec, 0)
    toks = gt.tokens_for(spec, 48, 3)
    real_p, real_m = orc.parallel, orc.decayed_memory
    want = orc.forward(spec.to_config(), ck, toks)[0]
    for fault in (("parallel", lambda *a: 2.0 * real_p(*a)), ("decayed_memory", lambda q, *a: real_m(q * q.shape[2] ** -0.5, *a))):
        with pytest.MonkeyPatch.context() as mp:
            mp.setattr(orc, *fault)
            assert float(gt.row_errs(orc.forward(spec.to_config(), ck, toks)[0], want).max()) > 100 * gt.TOL["float32"]
