"""Fofinex without a GPU: configuration round trip, tensor inventory, the oracle's mechanisms on hand-made inputs whose results are
known by construction, and faults planted in the oracle, which must move the results of the models that the GPU tests run by far
more than those tests tolerate."""
import dataclasses
import math

import pytest
import torch

from tests import fofinex_oracle as orc
from tests import test_gpu_fofinex as gt

F = torch.float64


def test_config_round_trip():
    from vllm_rust_amd.fofinex import FofinexSpec
    spec = gt.small_spec()
    cfg = spec.to_config()
    assert cfg["architecture"] == "Fofinex" and [e["type"] for e in cfg["layers"]] == ["latent_attention", "mlstm", "latent_attention", "mlstm", "latent_attention"]
    assert cfg["layers"][4]["mlp"] is None and "kv_from" not in cfg["layers"][0]["mixer"] and cfg["layers"][2]["mixer"]["kv_from"] == 0
    assert cfg["layers"][0]["mixer"]["rot"]["scaling"] == gt.STRETCH and "scaling" not in cfg["layers"][4]["mixer"]["rot"]
    again = FofinexSpec.from_config(cfg)
    assert again.to_config() == cfg and again.layers[2].kv_from == 0 and again.layers[0].kv_from is None
    # what a configuration may leave out
    e = {"type": "mlstm", "mixer": {"heads": 2, "dim": 6, "gate_cap": 5.0}, "mlp": {"kind": "moe", "expert": {"ff": 4}, "router": {"experts": 4, "top": 2}}}
    l = FofinexSpec.from_config({"vocab": 5, "width": 8, "norm": {"eps": 1e-5}, "layers": [e]}).layers[0]
    assert (l.vdim, l.groups, l.keep_groups, l.router_scale, l.shared_ff) == (6, 1, 1, 1.0, 0)
    for bad in (dict(e, type="lstm"), dict(e, mlp={"kind": "sparse"})):
        with pytest.raises(ValueError):
            FofinexSpec.from_config({"vocab": 5, "width": 8, "norm": {"eps": 1e-5}, "layers": [bad]})


def test_tensor_inventory_registry_and_oracle_runs():
    from vllm_rust_amd.fofinex import synthetic_weights
    from vllm_rust_amd.models import REGISTRY
    spec = gt.small_spec()
    shapes = spec.tensor_shapes()
    assert shapes["embed"] == (67, 40) and shapes["embed.norm"] == (40,) and "head" not in shapes
    assert shapes["l0.mix.uq"] == (48, 18) and shapes["l0.mix.dkv"] == (26, 40) and shapes["l0.mix.uk"] == (30, 20) and shapes["l0.mix.uv"] == (42, 20)
    assert "l2.mix.dkv" not in shapes and "l2.mix.dkv.norm" not in shapes and shapes["l2.mix.uk"] == (35, 20) and shapes["l2.mix.dq.norm"] == (11,)
    assert shapes["l1.mix.norm"] == (48,) and shapes["l1.mix.f.b"] == (3,) and shapes["l1.mlp.correction"] == (12,) and shapes["l1.mlp.shared.sg"] == (1, 40)
    assert shapes["l0.mlp.down.b"] == (40,) and "l1.mlp.e0.gate" not in shapes and "l4.norm2b" not in shapes and shapes["l4.norm1b"] == (40,)
    ck = synthetic_weights(spec, 0)
    assert set(ck) == set(shapes) and all(tuple(ck[k].shape) == shapes[k] and ck[k].dtype == torch.bfloat16 for k in ck)
    assert "Fofinex" in REGISTRY
    lg, tr = orc.forward(spec.to_config(), ck, [3, 1, 4, 1, 5, 9, 2, 6, 5, 3])
    assert lg.shape == (10, 67) and tr.shape == (5, 10, 40) and bool(torch.isfinite(lg).all())
    with orc.rounded_operands():
        lo, _ = orc.forward(spec.to_config(), ck, [3, 1, 4, 1, 5, 9, 2, 6, 5, 3])
    assert 1e-4 < float(gt.row_errs(lo, lg).mean()) < 0.1 and orc._rounding is None


def test_oracle_norm_rotation_and_activations():
    x = torch.tensor([[1.0, 3.0, 5.0, 7.0]], dtype=F)
    assert torch.allclose(orc.layer_norm(x, torch.ones(4, dtype=F), 0.0), (x - 4) / math.sqrt(5.0))
    assert torch.allclose(orc.layer_norm(x + 100, torch.full((4,), 2.0, dtype=F), 4.0), 2 * (x - 4) / 3.0)
    assert torch.allclose(orc.rms_unit(x, 0.0), x / math.sqrt(21.0))
    assert torch.equal(orc.relu_squared(torch.tensor([-2.0, 0.0, 3.0])), torch.tensor([0.0, 0.0, 9.0]))
    z = torch.linspace(-4, 4, 33, dtype=F)
    assert torch.allclose(orc.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    # coordinate 0 turns with coordinate 2 (dims 4), coordinates 4, 5 pass
    v = torch.zeros(2, 1, 6, dtype=F)
    v[:, 0, 0], v[:, 0, 4], v[:, 0, 5] = 1.0, 7.0, 8.0
    r = orc.rotate(v, [0, 3], dict(dims=4, base=10.0))
    assert torch.allclose(r[0], v[0]) and torch.allclose(r[1, 0], torch.tensor([math.cos(3.0), 0, math.sin(3.0), 0, 7.0, 8.0], dtype=F))
    # stretched: the fastest pair keeps its step, the slowest turns `factor` times slower, cos and sin carry the multiplier
    rot = dict(dims=24, base=2e4, scaling=dict(factor=8.0, original=1024, fast=16.0, slow=2.0))
    plain, one = orc.rotation_steps(dict(dims=24, base=2e4))
    steps, mul = orc.rotation_steps(rot)
    assert one == 1.0 and mul == pytest.approx(0.1 * math.log(8) + 1) and steps[0] == plain[0] and steps[-1] == pytest.approx(plain[-1] / 8)
    u = torch.zeros(1, 1, 24, dtype=F)
    u[0, 0, 3] = 1.0
    assert float(orc.rotate(u, [17], rot).norm()) == pytest.approx(mul)


def test_oracle_exponential_memory_by_hand():
    # one head of size one: S and n are numbers
    k, v, q = (torch.tensor(x, dtype=F).reshape(3, 1, 1) for x in ([1.0, 2.0, -1.0], [5.0, -3.0, 4.0], [1.0, 1.0, 2.0]))
    li, lf = torch.tensor([[-2.0], [1.0], [0.5]], dtype=F), torch.tensor([[-0.5], [-1.0], [-0.25]], dtype=F)
    o = orc.exponential_gate_memory(q, k, v, li, lf).reshape(3)
    m0 = max(-0.5 + 0.0, -2.0)                                     # the maximum starts at 0, so the forget gate holds it up
    s0, n0 = math.exp(-2 - m0) * 5, math.exp(-2 - m0) * 1
    assert o[0] == pytest.approx(s0 / (max(abs(n0), math.exp(-m0)) + 1e-6)) and math.exp(-m0) > n0
    m1 = max(-1.0 + m0, 1.0)
    d, a = math.exp(-1 + m0 - m1), math.exp(1 - m1)
    s1, n1 = d * s0 + a * 2 * -3, d * n0 + a * 2
    assert o[1] == pytest.approx(s1 / (max(abs(n1), math.exp(-m1)) + 1e-6))
    m2 = max(-0.25 + m1, 0.5)
    d, a = math.exp(-0.25 + m1 - m2), math.exp(0.5 - m2)
    s2, n2 = d * s1 + a * -1 * 4, d * n1 + a * -1
    assert o[2] == pytest.approx(2 * s2 / (max(abs(2 * n2), math.exp(-m2)) + 1e-6))
    li, lf = orc.log_gates(torch.tensor([100.0]), torch.tensor([-100.0]), 6.0)
    assert float(li) == pytest.approx(6.0) and float(lf) == pytest.approx(-6.0, abs=3e-3)


def test_oracle_router_by_hand():
    z = torch.logit(torch.tensor([[0.9, 0.1, 0.6, 0.6, 0.2, 0.3]], dtype=F))
    none = torch.zeros(6, dtype=F)
    ids, w = orc.route(z, none, 2, 1, 1, 2.0)
    assert ids.tolist() == [[0, 2]] and torch.allclose(w, torch.tensor([[1.8, 1.2]], dtype=F))
    ids, w = orc.route(z, none, 2, 3, 1, 1.0)                      # group sums 1.0, 1.2, 0.5
    assert ids.tolist() == [[2, 3]] and torch.allclose(w, torch.tensor([[0.6, 0.6]], dtype=F))
    low = torch.full((6,), -2.0, dtype=F)
    low[5] = 0.5
    ids, w = orc.route(z, low, 3, 3, 2, 1.0)                       # negative choice scores still beat a dropped group
    assert ids.tolist() == [[5, 2, 3]] and torch.allclose(w, torch.tensor([[0.3, 0.6, 0.6]], dtype=F))
    assert orc.router_margin(z, none, 2, 3, 1) == pytest.approx(0.2) and orc.router_margin(z, none, 6, 1, 1) == math.inf


FAULTS = {
    "uncentred norm": ("layer_norm", lambda x, w, eps: orc.rms_unit(x, eps) * w),
    "neighbouring pairs rotated": ("rotate", lambda x, p, rot: _neighbours(x, p, rot)),
    "angles one position late": ("rotate", lambda x, p, rot, f=orc.rotate: f(x, [i + 1 for i in p], rot) if x.shape[1] == 1 else f(x, p, rot)),
    "cos and sin without the multiplier": ("rotation_steps", lambda rot, f=orc.rotation_steps: (f(rot)[0], 1.0)),
    "steps not stretched": ("rotation_steps", lambda rot, f=orc.rotation_steps: (f({k: v for k, v in rot.items() if k != "scaling"})[0], f(rot)[1])),
    "a key too few": ("causal_softmax_attention", lambda q, k, v, s, f=orc.causal_softmax_attention: f(q, torch.cat([k[:1], k[:-1]]), torch.cat([v[:1], v[:-1]]), s)),
    "other activation of the dense part": ("gelu_tanh", lambda z: z * torch.sigmoid(z)),
    "experts not squared": ("relu_squared", lambda z: torch.clamp(z, min=0.0)),
    "weights with the correction": ("route", lambda z, c, t, g, k, s, f=orc.route: (f(z, c, t, g, k, s)[0], torch.gather(torch.sigmoid(z) + c, 1, f(z, c, t, g, k, s)[0]) * s)),
    "weights renormalised": ("route", lambda z, c, t, g, k, s, f=orc.route: (f(z, c, t, g, k, s)[0], f(z, c, t, g, k, s)[1] / f(z, c, t, g, k, s)[1].sum(-1, keepdim=True))),
    "choice without the correction": ("route", lambda z, c, t, g, k, s, f=orc.route: f(z, 0 * c, t, g, k, s)),
    "groups ignored": ("route", lambda z, c, t, g, k, s, f=orc.route: f(z, c, t, 1, 1, s)),
    "forget gate from the raw logit": ("log_gates", lambda i, f, cap, g=orc.log_gates: (g(i, f, cap)[0], torch.nn.functional.logsigmoid(2 * f))),
    "input gate not capped": ("log_gates", lambda i, f, cap, g=orc.log_gates: (2.0 * i, g(i, f, cap)[1])),
}


def _neighbours(x, positions, rot):
    if not rot or not rot.get("dims"):
        return x.clone()
    n = rot["dims"]
    order = list(range(0, n, 2)) + list(range(1, n, 2)) + list(range(n, x.shape[2]))
    back = [order.index(i) for i in range(x.shape[2])]
    return _halves(x[:, :, order], positions, rot)[:, :, back]


_halves = orc.rotate


@pytest.mark.parametrize("name", list(FAULTS))
def test_planted_faults_show(monkeypatch, name):
    from vllm_rust_amd.fofinex import synthetic_weights
    spec = gt.small_spec()
    ck = synthetic_weights(spec, 0)
    toks = gt.tokens_for(spec, 53, 2)
    want = orc.forward(spec.to_config(), ck, toks)[0]
    monkeypatch.setattr(orc, *FAULTS[name])
    assert float(gt.row_errs(orc.forward(spec.to_config(), ck, toks)[0], want).max()) > 20 * gt.TOL["float32"]


def test_planted_memory_faults_show_where_eps_is_large():
    """The per-head norm behind the memory hides its scale unless eps is of the order of the squares: what the large-eps GPU test
    relies on, checked for a floor that ignores the running maximum, a read-out without its normaliser and an unscaled query."""
    from vllm_rust_amd.fofinex import synthetic_weights
    spec = gt.small_spec(layers=[gt.mem_layer(mlp=None), gt.att_layer(mlp=None), gt.mem_layer(heads=2, dim=40, **gt.DENSE)], norm_eps=0.5)
    ck = synthetic_weights(spec, 0)
    toks = gt.tokens_for(spec, 48, 3)
    real = orc.exponential_gate_memory
    want = orc.forward(spec.to_config(), ck, toks)[0]

    def floor_of_one(q, k, v, li, lf, parts=None):
        parts = []
        real(q, k, v, li, lf, parts)
        return torch.stack([top / (torch.clamp(nq.abs(), min=1.0) + 1e-6).unsqueeze(-1) for top, nq, _, _ in parts])

    def no_normaliser(q, k, v, li, lf, parts=None):
        parts = []
        real(q, k, v, li, lf, parts)
        return torch.stack([p[0] for p in parts])
    for fault in (floor_of_one, no_normaliser, lambda q, *a: real(q * q.shape[2] ** 0.5, *a)):
        with pytest.MonkeyPatch.context() as mp:
            mp.setattr(orc, "exponential_gate_memory", fault)
            assert float(gt.row_errs(orc.forward(spec.to_config(), ck, toks)[0], want).max()) > 20 * gt.TOL["float32"]


def test_rotated_and_shared_layers_differ_in_the_oracle():
    spec = gt.small_spec()
    from vllm_rust_amd.fofinex import synthetic_weights
    ck = synthetic_weights(spec, 1)
    toks = gt.tokens_for(spec, 20, 1)
    want = orc.forward(spec.to_config(), ck, toks)[0]
    layers = list(spec.layers)
    layers[0] = dataclasses.replace(layers[0], scale=0.31)
    assert float(gt.row_errs(orc.forward(dataclasses.replace(spec, layers=layers).to_config(), ck, toks)[0], want).max()) > 1e-3
