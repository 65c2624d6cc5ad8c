"""Fofinex on the GPU against the float64 oracle (tests/fofinex_oracle.py): every mechanism alone (corrected group-limited routing,
latent preparation part by part, causal latent attention with a needle key, the exponential-gate scan, the matrix memory with its
normaliser fed in portions through dirty state slots, the read-out), then the executor through the engine's step function under
different cuttings of the same tokens (whole prompts, token-by-token decoding, portions down to two tokens, unequal batches,
recycled cache blocks and state slots), layers that share latents, norms of every row width, other sizes, random models, and greedy
generation through the scheduler.  Small random models built here; float32 mode is held to 2e-4 of the logits' spread, bfloat16
mode to 4e-2 or three times what rounding alone does."""
import ctypes as C
import dataclasses
import json
import math
import subprocess
import sys
from pathlib import Path

import numpy as np
import pytest

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
TOL = {"float32": 2e-4, "bfloat16": 4e-2}


@pytest.fixture(scope="module")
def gpu():
    import torch
    import vllm_rust_amd as vmx
    assert torch.cuda.is_available()
    vmx.init(0)
    return vmx, torch


def rot(dims, base=500.0, **scaling):
    from vllm_rust_amd.rotation import RotationSpec
    return RotationSpec(dims, base, dict(scaling) if scaling else None)


STRETCH = dict(factor=4.0, original=64.0, fast=8.0, slow=1.0)
MOE = dict(mlp="moe", experts=12, top=3, groups=4, keep_groups=2, expert_ff=20, shared_ff=28, router_scale=1.7)
DENSE = dict(mlp="dense", ff=36)


def att_layer(**kw):
    from vllm_rust_amd.fofinex import FofinexLayerSpec
    d = dict(mixer="latent_attention", heads=3, dim=10, rot_dim=6, vdim=14, kv_rank=20, q_rank=18, scale=0.3, rot=rot(6, 300.0, **STRETCH), **DENSE)
    d.update(kw)
    return FofinexLayerSpec(**d)


def mem_layer(**kw):
    from vllm_rust_amd.fofinex import FofinexLayerSpec
    d = dict(mixer="mlstm", heads=3, dim=12, vdim=16, gate_cap=9.0, **MOE)
    d.update(kw)
    return FofinexLayerSpec(**d)


def small_spec(layers=None, **kw):
    from vllm_rust_amd.fofinex import FofinexSpec
    layers = layers or [att_layer(), mem_layer(), att_layer(kv_from=0, heads=5, dim=7, vdim=9, q_rank=11, **MOE), mem_layer(heads=2, dim=7, vdim=5, **DENSE),
                        att_layer(kv_rank=33, rot_dim=10, rot=rot(4, 100.0), mlp=None)]
    d = dict(vocab=67, width=40, layers=layers, norm_eps=1e-5)
    d.update(kw)
    return FofinexSpec(**d)


def sure_routing(spec):
    """The same model with every expert chosen: long bfloat16 runs, where some router decision among hundreds is always a close
    call, then test everything but the choice."""
    return dataclasses.replace(spec, layers=[dataclasses.replace(l, top=l.experts, keep_groups=l.groups) if l.mlp == "moe" else l for l in spec.layers])


def routed(spec, dtype):
    """The model as it is in float32; in bfloat16 with every expert chosen (the choice itself is tested in float32, on single
    layers in bfloat16, and by the router's own test)."""
    return sure_routing(spec) if dtype == "bfloat16" else spec


def build(spec, dtype="float32", seed=0, tweak=None, block_size=4, num_blocks=96, max_tokens=320, max_seqs=6):
    from vllm_rust_amd.engine import Engine
    from vllm_rust_amd.fofinex import FofinexForCausalLM, synthetic_weights
    ck = synthetic_weights(spec, seed)
    if tweak:
        tweak(ck)
    model = FofinexForCausalLM(spec, dtype=dtype, block_size=block_size, num_blocks=num_blocks, max_tokens=max_tokens, max_seqs=max_seqs)
    model.load_state(ck)
    return model, Engine(model), {k: v.double() for k, v in ck.items()}


def tokens_for(spec, n, seed, weights=None, dtype="bfloat16"):
    """n random token ids.  With the model's weights: the first draw on which no router decision of the oracle is a close call
    (score gap above 0.01 for bfloat16 runs, 1e-5 for float32 ones), since a decision that rounding can flip says nothing about
    the kernels."""
    from tests import fofinex_oracle as orc
    gap = 0.01 if dtype == "bfloat16" else 1e-5
    for attempt in range(200):
        toks = np.random.default_rng(seed + 1000 * attempt).integers(0, spec.vocab, n).tolist()
        if weights is None:
            return toks
        margins = []
        orc.forward(spec.to_config(), weights, toks, margins)
        if not margins or min(margins) > gap:
            return toks
    raise AssertionError("no token draw with safe router margins")


def row_errs(got, want):
    """Difference of two logits arrays per row, row means removed, relative to the spread of the expected row."""
    g, w = np.asarray(got, np.float64), np.asarray(want, np.float64)
    d = g - w
    d = d - d.mean(-1, keepdims=True)
    return np.sqrt((d ** 2).mean(-1)) / (w.std(-1) + 1e-12)


class Expected:
    """The oracle's logits and streams of a token sequence, and how far a run may be from them: float32 2e-4 in every row; bfloat16
    4e-2 in every row and 1.5e-2 in the mean, or three times what rounding the operands alone does to this model and these tokens
    (a memory's read-out is divided by its own size, so some rows amplify rounding a lot)."""

    def __init__(self, spec, weights, toks, dtype):
        from tests import fofinex_oracle as orc
        lg, tr = orc.forward(spec.to_config(), weights, toks)
        self.logits, self.trace, self.dtype = lg.numpy(), tr.numpy(), dtype
        self.rounded = None
        if dtype == "bfloat16":
            with orc.rounded_operands():
                lg, tr = orc.forward(spec.to_config(), weights, toks)
            self.rounded = (lg.numpy(), tr.numpy())

    def _check(self, got, want, rounded, rows, what):
        err = row_errs(got, want[rows])
        if self.dtype == "float32":
            assert err.max() < TOL["float32"], (what, err.max())
            return
        alone = row_errs(rounded, want)          # every row of the sequence: the worst one says what this model can amplify
        assert err.max() < max(TOL["bfloat16"], 3 * alone.max()), (what, err.max(), alone.max())
        assert len(err) < 8 or err.mean() < max(1.5e-2, 3 * alone.mean()), (what, err.mean(), alone.mean())

    def check(self, got, rows=slice(None), what=""):
        self._check(got, self.logits, self.rounded and self.rounded[0], rows, what)

    def check_layer(self, i, got, what=""):
        self._check(got, self.trace[i], self.rounded and self.rounded[1][i], slice(None), (what, "layer", i))


def oracle(spec, weights, toks):
    from tests import fofinex_oracle as orc
    lg, tr = orc.forward(spec.to_config(), weights, toks)
    return lg.numpy(), tr.numpy()


def feed(engine, seq_id, toks, cuts, finish=True):
    """Feed toks to one sequence in pieces of the given sizes (the last size repeats); logits of every position."""
    out, at, i = [], 0, 0
    while at < len(toks):
        n = min(cuts[min(i, len(cuts) - 1)], len(toks) - at)
        lg, _, _ = engine.step([(seq_id, toks[at:at + n], list(range(n)))])
        out.append(lg.cpu().numpy())
        at += n
        i += 1
    if finish:
        engine.finish(seq_id)
    return np.concatenate(out)


# ----------------------------------------------------------------------------- mechanisms alone

@pytest.mark.parametrize("E,top,groups,keep", [(20, 3, 5, 3), (12, 2, 3, 1), (8, 8, 4, 4), (70, 4, 7, 2), (256, 6, 16, 4), (6, 2, 6, 3), (5, 2, 1, 1), (64, 1, 2, 1),
                                               (1, 1, 1, 1), (200, 12, 2, 2)])
@pytest.mark.parametrize("shift", [0.0, -0.9, 0.4])
def test_corrected_router(gpu, E, top, groups, keep, shift):
    """Choice by score + correction inside the best groups (shift -0.9: almost every choice score is negative, so a dropped group
    must lose to them), weights from the plain scores, rows with a stride of their own."""
    _, torch = gpu
    from tests import fofinex_oracle as orc
    from vllm_rust_amd._lib import check, lib
    g = torch.Generator().manual_seed(E + top)
    T, ld = 23, E + 3
    z = torch.full((T, ld), 1e9)
    z[:, :E] = 2 * torch.randn((T, E), generator=g)
    corr = (0.4 * torch.randn(E, generator=g) + shift).to(torch.bfloat16)
    z[5, :E] = torch.logit(torch.full((E,), 0.5))                  # equal scores: the correction alone decides
    ids, w = orc.route(z[:, :E].double(), corr.double(), top, groups, keep, 1.7)
    zc, cc = z.cuda(), corr.cuda()
    wo, io = torch.empty(T, top, device="cuda"), torch.empty(T, top, dtype=torch.int32, device="cuda")
    check(lib.vmx_grouped_topk_sigmoid(zc.data_ptr(), ld, cc.data_ptr(), wo.data_ptr(), io.data_ptr(), T, E, top, groups, keep, 1.7, None))
    torch.cuda.synchronize()
    for t in range(T):
        if orc.router_margin(z[t:t + 1, :E].double(), corr.double(), top, groups, keep) > 1e-6:
            assert io[t].tolist() == ids[t].tolist()
            assert float((wo[t].cpu().double() - w[t]).abs().max()) < 1e-6
        assert len(set(io[t].tolist())) == top and all(0 <= e < E for e in io[t].tolist())


def test_corrected_router_ties_and_group_sums(gpu):
    """Equal choice scores go to the smaller index; a group wins by the sum of its two best, not by its best or its total."""
    _, torch = gpu
    from vllm_rust_amd._lib import check, lib

    def run(choice, top, groups, keep):
        E = len(choice)
        z = torch.zeros(1, E, device="cuda")                       # every plain score 0.5
        c = (torch.tensor(choice) - 0.5).to(torch.bfloat16).cuda()
        wo, io = torch.empty(1, top, device="cuda"), torch.empty(1, top, dtype=torch.int32, device="cuda")
        check(lib.vmx_grouped_topk_sigmoid(z.data_ptr(), E, c.data_ptr(), wo.data_ptr(), io.data_ptr(), 1, E, top, groups, keep, 2.0, None))
        torch.cuda.synchronize()
        assert float((wo - 1.0).abs().max()) < 1e-6
        return io[0].tolist()
    assert run([0.5] * 9, 4, 3, 2) == [0, 1, 2, 3]
    assert run([1.0, 0.0, 0.0, 0.75, 0.5, 0.0, 0.5, 0.5, 0.5], 1, 3, 1) == [3]                      # 1.0 < 1.25 > 1.0
    assert run([-1.0, -2.0, -1.5, -1.25, -4.0, -0.5], 2, 3, 1) == [3, 2]                             # -3, -2.75, -4.5
    assert run([-1.0, -2.0, -1.5, -1.25, -4.0, -0.5], 3, 3, 2) == [0, 3, 2]


@pytest.mark.parametrize("H,dim,rd,rdims,R,Q,stretch", [(3, 10, 6, 6, 20, 18, True), (5, 64, 24, 24, 112, 72, True), (2, 0, 8, 8, 16, 5, False), (4, 7, 10, 4, 33, 7, False),
                                                        (1, 16, 0, 0, 24, 300, False), (2, 4, 300, 300, 512, 1, True)])
@pytest.mark.parametrize("dtype", [0, 1])
def test_latent_preparation_part_by_part(gpu, H, dim, rd, rdims, R, Q, stretch, dtype):
    """Query latent norm, latent + rotated key part to the cache rows, rotated query parts: each alone and all together give the
    same numbers; nothing else is written."""
    _, torch = gpu
    from tests import fofinex_oracle as orc
    from vllm_rust_amd._lib import LatentPrepare, Rotation, check, lib
    T, eps = 9, 1e-5
    g = torch.Generator().manual_seed(H * R + Q)
    rn = lambda *s: torch.randn(*s, generator=g).float()   # noqa: E731
    kv, q, ql = rn(T, R + rd + 3), rn(T, H * (dim + rd) + 2), rn(T, Q + 1)
    kn, qn = (1 + 0.2 * rn(R)).to(torch.bfloat16), (1 + 0.2 * rn(Q)).to(torch.bfloat16)
    pos = [0, 1, 2, 3, 50, 51, 1000, 1001, 5000]
    slots = [5, 4, -1, 0, 1, 2, 11, 10, 7]
    rotd = dict(dims=rdims, base=777.0, **({"scaling": STRETCH} if stretch else {})) if rdims else None
    steps, mul = None, 1.0
    if rdims:
        sc = rotd.get("scaling") or {}
        r = Rotation(rdims, 777.0, sc.get("factor", 0.0), sc.get("original", 0.0), sc.get("fast", 0.0), sc.get("slow", 0.0))
        buf, m = (C.c_float * (rdims // 2))(), C.c_float()
        check(lib.vmx_rotation_steps(C.byref(r), buf, C.byref(m)))
        steps, mul = torch.tensor(list(buf), dtype=torch.float32, device="cuda"), m.value
    cdt = torch.float32 if dtype == 0 else torch.bfloat16
    i32 = lambda a: torch.tensor(a, dtype=torch.int32, device="cuda")   # noqa: E731
    P, S = i32(pos), i32(slots)
    kvc, qc, qlc, knc, qnc = kv.cuda(), q.cuda(), ql.cuda(), kn.cuda(), qn.cuda()

    def run(parts):
        cache = torch.full((13, R + rd), 7.0, dtype=cdt, device="cuda")
        qrot, qlo = torch.full((T * H * rd + 1,), 7.0, device="cuda"), torch.full((T * Q + 1,), 7.0, dtype=cdt, device="cuda")
        p = LatentPrepare(kvc.data_ptr() if "kv" in parts else None, R + rd + 3, knc.data_ptr(), qc.data_ptr() if "q" in parts else None, H * (dim + rd) + 2, H, dim,
                          qrot.data_ptr(), qlc.data_ptr() if "ql" in parts else None, Q + 1, Q, qnc.data_ptr(), R, rd, eps,
                          None if steps is None else steps.data_ptr(), rdims, 1, mul)
        check(lib.vmx_latent_prepare_rows(C.byref(p), P.data_ptr(), S.data_ptr(), cache.data_ptr(), dtype, qlo.data_ptr(), T, None))
        torch.cuda.synchronize()
        return cache.cpu().double(), qrot.cpu().double(), qlo.cpu().double()
    cache, qrot, qlo = run({"kv", "q", "ql"})
    for part, i in (("kv", 0), ("q", 1), ("ql", 2)):
        alone = run({part})
        assert bool((alone[i] == (cache, qrot, qlo)[i]).all())
        for j in range(3):
            if j != i:
                assert bool((alone[j] == 7.0).all())
    # angles are f32 products of a position and an f32 step: at position 5000 they carry an error of about 5000 * 2^-24
    tol = 6e-3 if rdims else 1e-5
    low = 0.04 if dtype == 1 else 0.0
    c = orc.rms_unit(kv[:, :R].double(), eps) * kn.double()
    kr = orc.rotate(kv[:, R:R + rd].double().unsqueeze(1), pos, rotd).squeeze(1)
    for t, s in enumerate(slots):
        if s >= 0:
            assert float((cache[s, :R] - c[t]).abs().max()) < 1e-5 + low
            assert rd == 0 or float((cache[s, R:] - kr[t]).abs().max()) < tol + low
    for s in (3, 6, 8, 9, 12):
        assert bool((cache[s] == 7.0).all())                       # rows no token owns
    if rd:
        qr = orc.rotate(q[:, :H * (dim + rd)].double().reshape(T, H, dim + rd)[:, :, dim:], pos, rotd)
        assert float((qrot[:-1].reshape(T, H, rd) - qr).abs().max()) < tol
    assert qrot[-1] == 7.0 and qlo[-1] == 7.0
    assert float((qlo[:-1].reshape(T, Q) - orc.rms_unit(ql[:, :Q].double(), eps) * qn.double()).abs().max()) < 1e-5 + low


@pytest.mark.parametrize("H,R,rd", [(3, 24, 8), (7, 112, 40), (16, 64, 16), (20, 16, 0), (2, 33, 6), (5, 256, 64)])
@pytest.mark.parametrize("dtype,bs", [(0, 16), (1, 16), (1, 5), (0, 1)])
def test_causal_latent_attention_with_a_needle(gpu, H, R, rd, dtype, bs):
    """No window: one key whose score stands out is found from its own position to 400 keys later, at page borders, as the first
    token and in the last row, in a prompt (all queries at once), in a late portion and as single decoded rows; a query one
    position earlier does not see it."""
    _, torch = gpu
    from vllm_rust_amd._lib import check, lib
    T = 430
    g = torch.Generator().manual_seed(R + H)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)   # noqa: E731
    q, row = 0.2 * rn(T, H, R + rd), 0.2 * rn(T, R + rd)
    needles = [0, 16, 31, 256]
    for n in needles:
        d = rn(R + rd)
        row[n] = d * (5 / d.norm())
        for i in [j for j in (n - 1, n, n + 1, n + 63, n + 64, n + 150, T - 1 - needles.index(n)) if 0 <= j < T and j not in needles]:
            q[i] = row[n] * 4                                       # score 50 against the needle, of order 1 against the rest
        q[n] = row[n] * 4
    bf = lambda t: t.to(torch.bfloat16).double()   # noqa: E731
    q, row = bf(q), bf(row)
    scale = 0.5
    s = torch.einsum("ihd,jd->hij", q, row) * scale
    s = s.masked_fill(torch.triu(torch.ones(T, T, dtype=torch.bool), 1), -math.inf)
    want = torch.einsum("hij,jr->ihr", torch.softmax(s, -1), row[:, :R])
    nb = (T + bs - 1) // bs
    perm = np.random.default_rng(1).permutation(nb + 5)[:nb].astype(np.int32)
    pos = np.arange(T)
    cache = torch.full(((nb + 5) * bs, R + rd), float("nan"), dtype=torch.float32)
    cache[perm[pos // bs] * bs + pos % bs] = row.float()
    cache = cache.to(torch.float32 if dtype == 0 else torch.bfloat16).cuda()
    bt = torch.from_numpy(perm[None]).cuda()
    tol = (3e-5 if dtype == 0 else 2e-2) * float(want.abs().max())
    for a, b in [(0, T), (300, T), (17, 19)] + [(i, i + 1) for i in (0, 16, 17, 31, 94, 255, 256, 320, 429)]:
        n = b - a
        qa, qr = q[a:b, :, :R].float().contiguous().cuda(), q[a:b, :, R:].float().contiguous().cuda() if rd else torch.zeros(1, device="cuda")
        out = torch.empty(n, H, R, device="cuda")
        P, sid = torch.arange(a, b, dtype=torch.int32, device="cuda"), torch.zeros(n, dtype=torch.int32, device="cuda")
        ws = torch.empty(lib.vmx_latent_attention_workspace_bytes(n, H, R, 0, nb, bs) // 4 + 1, device="cuda")
        check(lib.vmx_latent_attention(out.data_ptr(), qa.data_ptr(), qr.data_ptr(), cache.data_ptr(), dtype, bt.data_ptr(), nb, sid.data_ptr(), P.data_ptr(), None,
                                       scale, 0, n, H, R, rd, bs, ws.data_ptr(), ws.numel() * 4, None))
        torch.cuda.synchronize()
        assert float((out.cpu().double() - want[a:b]).abs().max()) < tol, (a, b)


def _run_exp_memory(torch, q, k, v, zi, zf, cap, portions, slot_of, q_mul, chunks=False):
    """vmx_exp_gate_scan + vmx_matrix_memory_recurrence_ex over several sequences fed in unequal portions through slots that start
    full of NaN.  Lists of [n, H, D], [n, H, D], [n, H, V], [n, H], [n, H]; per sequence [o / (max(|n . q|, e^-m) + 1e-6), o, n . q, e^-m].
    chunks: let steps with enough tokens take the chunked form (which rounds q, k and v to bf16)."""
    from vllm_rust_amd._lib import MatrixMemoryOpts, check, lib
    H, D, V = k[0].shape[1], k[0].shape[2], v[0].shape[2]
    nslots = max(slot_of) + 2
    nan = lambda n: torch.full((n,), float("nan"), dtype=torch.float32, device="cuda")   # noqa: E731
    state, maxima = nan(lib.vmx_gated_delta_rule_state_bytes(nslots, H, D, V + 1) // 4), nan(nslots * H)
    lens = [x.shape[0] for x in q]
    got, fed = [[] for _ in lens], [0] * len(lens)
    i32 = lambda a: torch.tensor(a, dtype=torch.int32, device="cuda")   # noqa: E731
    for step in range(max(len(p) for p in portions)):
        parts, starts, slots, posn, owners = [], [0], [], [], []
        for s, n in enumerate(lens):
            if step < len(portions[s]) and fed[s] < n:
                c = min(portions[s][step], n - fed[s])
                a, b = fed[s], fed[s] + c
                parts.append(torch.cat([x[s][a:b].reshape(c, -1) for x in (q, k, v, zi, zf)], 1))
                posn += list(range(a, b))
                starts.append(starts[-1] + c)
                slots.append(slot_of[s])
                owners.append((s, c))
                fed[s] = b
        x = torch.cat(parts).float().cuda()
        T, ld = x.shape
        o, norm, floor = torch.empty(T, H * V, device="cuda"), torch.empty(T, H + 1, device="cuda"), torch.empty(T, H + 2, device="cuda")
        P, S, L = i32(posn), i32(starts), i32(slots)
        ok, ov, oi = H * D, 2 * H * D, 2 * H * D + H * V
        at = lambda off: x.data_ptr() + 4 * off   # noqa: E731
        check(lib.vmx_exp_gate_scan(at(oi), ld, at(oi + H), ld, floor.data_ptr(), H + 2, maxima.data_ptr(), cap, P.data_ptr(), S.data_ptr(), L.data_ptr(), len(slots),
                                    H, None))
        mo = MatrixMemoryOpts(at(oi), ld, norm.data_ptr(), H + 1, 1 if chunks else 0, T)
        check(lib.vmx_matrix_memory_recurrence_ex(o.data_ptr(), H * V, at(0), ld, q_mul, at(ok), ld, at(ov), ld, at(oi + H), ld, 1, None, 0, state.data_ptr(),
                                                  P.data_ptr(), S.data_ptr(), L.data_ptr(), len(slots), H, H, D, V, C.byref(mo), None))
        torch.cuda.synchronize()
        den = torch.maximum(norm[:, :H].abs(), floor[:, :H]).cpu().double() + 1e-6
        res = [o.cpu().double().reshape(T, H, V) / den.unsqueeze(-1), o.cpu().double().reshape(T, H, V), norm[:, :H].cpu().double(), floor[:, :H].cpu().double()]
        row = 0
        for s, c in owners:
            got[s].append([r[row:row + c] for r in res])
            row += c
    assert fed == lens
    return [[torch.cat([x[j] for x in g]) for j in range(4)] for g in got]


@pytest.mark.parametrize("H,D,V,cap", [(2, 32, 32, 15.0), (3, 5, 7, 4.0), (4, 64, 47, 11.0), (1, 130, 16, 8.0), (2, 16, 1, 1.0), (6, 40, 56, 10.0)])
@pytest.mark.parametrize("bias", [(0.0, 2.0), (-6.0, 0.0), (8.0, 4.0)])
@pytest.mark.parametrize("chunks", [False, True])
def test_exponential_memory_in_portions_through_dirty_slots(gpu, H, D, V, cap, bias, chunks):
    """Both forms of the recurrence (with q, k and v that are bf16 numbers the chunked one is held to the same bounds; steps of few
    tokens take the other form, so the two also hand the memory to each other).  Three sequences of unequal length in portions of 1 .. 90 rows; input gates around zero, far below (the maximum then falls
    from its start at 0 and the floor e^-m counts) and far above."""
    _, torch = gpu
    from tests import fofinex_oracle as orc
    gen = torch.Generator().manual_seed(H * D + V)
    lens = [331, 1, 70]
    rn = lambda *s: torch.randn(*s, generator=gen, dtype=torch.float64).float().double()   # noqa: E731
    bf = lambda *s: rn(*s).to(torch.bfloat16).double()   # noqa: E731
    q, k, v = [bf(n, H, D) for n in lens], [bf(n, H, D) for n in lens], [bf(n, H, V) for n in lens]
    zi, zf = [(2 * rn(n, H) + bias[0]).float().double() for n in lens], [(2 * rn(n, H) + bias[1]).float().double() for n in lens]
    got = _run_exp_memory(torch, q, k, v, zi, zf, cap, [[90, 1, 1, 37, 2, 200], [1], [2, 3, 63, 1, 1]], [3, 0, 4], D ** -0.5, chunks)
    for s in range(3):
        parts = []
        want = orc.exponential_gate_memory(q[s] * D ** -0.5, k[s], v[s], *orc.log_gates(zi[s], zf[s], cap), parts)
        o, nq, floor, size = (torch.stack([p[j] for p in parts]) for j in range(4))
        ref = max(1.0, float(size.max()))                          # the terms that o and n . q are sums of
        assert float((got[s][1] - o).abs().max()) < 3e-5 * ref * max(1.0, float(v[s].abs().max())), s
        assert float((got[s][2] - nq).abs().max()) < 2e-5 * ref, s
        assert float((got[s][3] / floor - 1).abs().max()) < 3e-5, s
        sound = (torch.maximum(nq.abs(), floor) > 0.05 * size).unsqueeze(-1)   # elsewhere the quotient is as exact as a cancellation
        assert float(((got[s][0] - want) * sound).abs().max()) < 1e-3 * max(1.0, float((want * sound).abs().max())), s


@pytest.mark.parametrize("chunks", [False, True])
def test_exponential_memory_keeps_a_far_key_and_starts_at_zero(gpu, chunks):
    """A key written at position 5 with the largest input gate and asked for 290 tokens and four portions later, through a forget
    gate of nearly one on head 0 and of one half on head 1; before it the memory is empty of it.  The first token's floor is
    e^-max(f, i), which leaves a small write small."""
    _, torch = gpu
    from tests import fofinex_oracle as orc
    n, D, V, cap = 300, 16, 8, 10.0
    gen = torch.Generator().manual_seed(0)
    k = torch.zeros(n, 2, D, dtype=torch.float64)
    k[:, :, 1:] = torch.randn(n, 2, D - 1, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()
    k[5, :, 0] = 1.0
    v = torch.randn(n, 2, V, generator=gen, dtype=torch.float64).to(torch.bfloat16).double()
    q = torch.zeros(n, 2, D, dtype=torch.float64)
    q[:, :, 0] = 1.0
    zi, zf = torch.full((n, 2), -4.0, dtype=torch.float64), torch.zeros(n, 2, dtype=torch.float64)
    zi[5], zf[:, 0] = 6.0, 90.0
    got = _run_exp_memory(torch, [q], [k], [v], [zi], [zf], cap, [[4, 100, 1, 150, 45]], [1], 1.0, chunks)[0][0]
    want = orc.exponential_gate_memory(q, k, v, *orc.log_gates(zi, zf, cap))
    assert float(got[:5].abs().max()) == 0 and float((got - want).abs().max()) < 1e-5
    for t in (5, 6, 104, 105, 295, 299):
        assert float((got[t, 0] - v[5, 0]).abs().max()) < 0.05 * float(v[5, 0].abs().max())      # still there, nearly whole
    assert float(got[40:, 1].abs().max()) < 1e-3 * float(v[5, 1].abs().max())
    k[0, :, 0] = 1.0                                                                               # the very first token, a small input gate
    got = _run_exp_memory(torch, [q[:1]], [k[:1]], [v[:1]], [zi[:1]], [zf[:1]], cap, [[1]], [0], 1.0, chunks)[0][0]
    m = torch.maximum(orc.log_gates(zi[0], zf[0], cap)[1], orc.log_gates(zi[0], zf[0], cap)[0])
    w = torch.exp(orc.log_gates(zi[0], zf[0], cap)[0])
    assert float((got[0] - v[0] * (w / torch.maximum(w, torch.ones(2, dtype=torch.float64))).unsqueeze(-1)).abs().max()) < 1e-5 and float(m[1]) < 0


def test_read_out_with_normaliser_and_head_gains(gpu):
    _, torch = gpu
    from tests import fofinex_oracle as orc
    from vllm_rust_amd._lib import ReadOutOpts, check, lib
    gen = torch.Generator().manual_seed(4)
    for H, V in ((3, 10), (2, 70), (5, 1), (1, 200)):
        for per_head in (0, 1):
            for silu in (0, 1):
                o = torch.randn(6, H * V + 2, generator=gen).cuda() * 1e-2
                gate = torch.randn(6, H * V + 4, generator=gen).cuda()
                norm, floor = torch.randn(6, H + 1, generator=gen).cuda(), torch.rand(6, H, generator=gen).cuda()
                norm[:, 0] = 0.0
                w = (1 + 0.2 * torch.randn(H * V if per_head else V, generator=gen)).to(torch.bfloat16).cuda()
                y = torch.empty(6, H * V, dtype=torch.float32, device="cuda")
                ro = ReadOutOpts(silu, per_head, norm.data_ptr(), H + 1, floor.data_ptr(), H, 1e-6)
                check(lib.vmx_head_read_out(y.data_ptr(), 0, o.data_ptr(), H * V + 2, w.data_ptr(), gate.data_ptr(), H * V + 4, 1e-4, 6, H, V, C.byref(ro), None))
                torch.cuda.synchronize()
                den = torch.maximum(norm[:, :H].abs(), floor).cpu().double() + 1e-6
                ref = orc.rms_unit(o.cpu().double()[:, :H * V].reshape(6, H, V) / den.unsqueeze(-1), 1e-4)
                wr = w.cpu().double().reshape(H, V) if per_head else w.cpu().double().reshape(1, V)
                gz = gate.cpu().double()[:, :H * V]
                ref = (ref * wr).reshape(6, H * V) * torch.sigmoid(gz) * (gz if silu else 1.0)
                assert float((y.cpu().double() - ref).abs().max()) < 1e-5


# ----------------------------------------------------------------------------- the executor through the engine

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_layers_and_logits_against_the_oracle(gpu, dtype):
    spec = routed(small_spec(), dtype)
    model, eng, w = build(spec, dtype)
    toks = tokens_for(spec, 41, 1, w, dtype)
    lg, _, tr = eng.step([("a", toks, list(range(len(toks))))], layer_trace=True)
    want = Expected(spec, w, toks, dtype)
    assert tr.shape[0] == len(spec.layers) == 5
    for r in range(tr.shape[0]):
        want.check_layer(r, tr[r].cpu().numpy())
    want.check(lg.cpu().numpy())


@pytest.mark.parametrize("kind", ["latent_attention", "mlstm"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_every_layer_kind_alone(gpu, dtype, kind):
    """One layer of each kind with every feed-forward, with and without groups and the shared expert: the stream after the layer."""
    make = att_layer if kind == "latent_attention" else mem_layer
    for ff in (DENSE, MOE, dict(mlp=None), dict(MOE, shared_ff=0, groups=1, keep_groups=1, router_scale=1.0), dict(MOE, experts=3, groups=3, keep_groups=2, top=1)):
        spec = small_spec(layers=[make(**ff)])
        model, eng, w = build(spec, dtype)
        toks = tokens_for(spec, 26, 2, w, dtype)
        lg, _, tr = eng.step([("a", toks, list(range(26)))], layer_trace=True)
        want = Expected(spec, w, toks, dtype)
        want.check_layer(0, tr[0].cpu().numpy())
        want.check(lg.cpu().numpy(), what=(kind, ff))
        model.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prompt_decode_and_portions_agree(gpu, dtype):
    spec = routed(small_spec(), dtype)
    model, eng, w = build(spec, dtype)
    toks = tokens_for(spec, 53, 2, w, dtype)
    want = Expected(spec, w, toks, dtype)
    for cuts in ([53], [1], [2], [3], [7, 16], [16, 1], [20, 2, 1]):
        got = feed(eng, "s", toks, cuts)
        want.check(got, what=f"cuts {cuts}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_batches_and_recycled_blocks_and_slots(gpu, dtype):
    """Three requests of unequal length in one batch, then decoded together while the short ones finish early; five generations of
    requests through 3 state slots and few blocks, freed blocks and slots handed out again in another order."""
    spec = routed(small_spec(), dtype)
    model, eng, w = build(spec, dtype, num_blocks=40, max_seqs=3)
    for gen in range(5):
        lens = [(29, 6), (3, 2), (14, 9)]
        reqs = {f"g{gen}r{i}": tokens_for(spec, n + d, 100 * gen + i, w, dtype) for i, (n, d) in enumerate(lens)}
        want = {k: Expected(spec, w, t, dtype) for k, t in reqs.items()}
        got = {k: [] for k in reqs}
        lg, _, _ = eng.step([(k, reqs[k][:n], list(range(n))) for k, (n, _) in zip(reqs, lens)])
        at = 0
        for k, (n, _) in zip(reqs, lens):
            got[k].append(lg[at:at + n].cpu().numpy())
            at += n
        fed = {k: n for k, (n, _) in zip(reqs, lens)}
        while True:
            live = [k for k in reqs if fed[k] < len(reqs[k])]
            if not live:
                break
            lg, _, _ = eng.step([(k, [reqs[k][fed[k]]], [0]) for k in live])
            for j, k in enumerate(live):
                got[k].append(lg[j:j + 1].cpu().numpy())
                fed[k] += 1
                if fed[k] == len(reqs[k]):
                    eng.finish(k)     # leaves the batch early; its blocks and slot go back
        for k in reqs:
            want[k].check(np.concatenate(got[k]), what=k)
    assert len(eng.blocks.free) == 40 and len(eng.states.free) == 3


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_steps_of_portions_and_decoding(gpu, dtype):
    """Steps that hold a fresh prompt, a later portion and a decoding token of different requests at once."""
    spec = routed(small_spec(), dtype)
    model, eng, w = build(spec, dtype)
    reqs = {k: tokens_for(spec, n, 30 + n, w, dtype) for k, n in (("a", 31), ("b", 26), ("c", 18))}
    plan = [{"a": 10}, {"a": 1, "b": 7}, {"b": 2, "a": 1, "c": 5}, {"c": 1, "a": 6, "b": 1}, {"a": 1, "b": 15, "c": 1}, {"c": 11, "b": 1, "a": 12}]
    fed, got = {k: 0 for k in reqs}, {k: [] for k in reqs}
    for step in plan:
        lg, _, _ = eng.step([(k, reqs[k][fed[k]:fed[k] + n], list(range(n))) for k, n in step.items()])
        at = 0
        for k, n in step.items():
            got[k].append(lg[at:at + n].cpu().numpy())
            at, fed[k] = at + n, fed[k] + n
    for k in reqs:
        assert fed[k] == len(reqs[k])
        Expected(spec, w, reqs[k], dtype).check(np.concatenate(got[k]), what=k)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_layers_that_share_latents(gpu, dtype):
    """Two layers attend over the first layer's latents and one over a later layer's, with other head counts, sizes, scales and
    query latents; swapping the sources changes the logits, so the test would notice a wrong cache."""
    common = dict(rot_dim=6, rot=rot(6, 300.0, **STRETCH), kv_rank=24)
    layers = [att_layer(**common), mem_layer(mlp=None), att_layer(**common, heads=2, dim=6), att_layer(**common, kv_from=0, heads=7, dim=3, vdim=4, q_rank=9, scale=0.5),
              att_layer(**common, kv_from=2, heads=1, dim=30, mlp=None), att_layer(**common, kv_from=0, heads=2, vdim=40)]
    spec = small_spec(layers=layers)
    model, eng, w = build(spec, dtype)
    toks = tokens_for(spec, 45, 7)
    want = Expected(spec, w, toks, dtype)
    other = dataclasses.replace(spec, layers=[dataclasses.replace(l, kv_from=2) if l.kv_from == 0 else l for l in layers])
    assert row_errs(oracle(other, w, toks)[0], want.logits).mean() > 0.2
    for cuts in ([45], [20, 1], [2]):
        want.check(feed(eng, "a", toks, cuts))
    model.close()
    from vllm_rust_amd._lib import VmxError
    from vllm_rust_amd.fofinex import FofinexForCausalLM
    for bad in ([att_layer(kv_from=0)], [mem_layer(), att_layer(kv_from=0)], [att_layer(), att_layer(kv_from=0), att_layer(kv_from=1)],
                [att_layer(), att_layer(kv_from=0, kv_rank=21)], [att_layer(), att_layer(kv_from=2), att_layer()]):
        with pytest.raises(VmxError):
            FofinexForCausalLM(small_spec(layers=bad), dtype=dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width", [1, 40, 256, 257, 1000, 1500, 2600, 4100])
def test_norms_of_every_row_width(gpu, dtype, width):
    """Rows of one number up to rows wider than the norm kernels keep in registers; every sublayer's result and the table get a
    large common offset, which only a norm that takes the mean off removes."""
    def offset(ck):
        ck["embed"] = (ck["embed"].float() + 3).to(ck["embed"].dtype)
        ck["l0.mlp.down.b"] = (ck["l0.mlp.down.b"].float() + 20).to(ck["l0.mlp.down.b"].dtype)
    spec = sure_routing(small_spec(layers=[att_layer(heads=2), mem_layer(heads=2, experts=3, groups=1, keep_groups=1)], width=width, vocab=31))
    model, eng, w = build(spec, dtype, tweak=offset, max_tokens=32, num_blocks=16)
    toks = tokens_for(spec, 9, width)
    want = Expected(spec, w, toks, dtype)
    lg, _, tr = eng.step([("a", toks, list(range(9)))], layer_trace=True)
    if width > 1:
        want.check_layer(-1, tr[-1].cpu().numpy())
        want.check(lg.cpu().numpy())
    else:
        assert float(tr.abs().max()) == 0 and float(lg.abs().max()) == 0          # one number minus itself
    model.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_large_eps_shows_the_scales_that_norms_hide(gpu, dtype):
    """With eps of the order of the squares, the query scale, the normaliser and the floor of the memory, and the scales of both
    latents reach the logits instead of cancelling in the norm that follows them."""
    spec = routed(small_spec(layers=[mem_layer(mlp=None), att_layer(mlp=None), mem_layer(heads=2, dim=40, **DENSE)], norm_eps=0.5), dtype)
    model, eng, w = build(spec, dtype)
    toks = tokens_for(spec, 48, 3, w, dtype)
    want = Expected(spec, w, toks, dtype)
    for cuts in ([48], [20, 1]):
        want.check(feed(eng, "a", toks, cuts))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", ["any", "eights"])
def test_sharp_attention_over_300_tokens_and_long_decoding(gpu, dtype, sizes):
    """Queries scaled up so that single keys decide rows over all 300 tokens, forget gates close to one in the memories, 220 tokens
    as a prompt and 80 decoded one by one; every expert chosen (no close calls)."""
    def sharpen(ck):
        for k in ck:
            if k.endswith("mix.dq.norm"):
                ck[k] = (ck[k].float() * 3).to(ck[k].dtype)
            if k.endswith("mix.f.b"):
                ck[k] = (ck[k].float() + 4).to(ck[k].dtype)       # old writes stay in the memory
    if sizes == "any":
        layers = [att_layer(), mem_layer(), att_layer(kv_from=0, mlp=None)]
    else:    # multiples of 8: the matrix-core forms in bfloat16
        layers = [att_layer(heads=4, dim=16, rot_dim=8, vdim=24, kv_rank=64, q_rank=32, rot=rot(8, 1e4)), mem_layer(dim=32, vdim=32),
                  att_layer(heads=8, dim=24, rot_dim=8, vdim=8, kv_rank=64, q_rank=32, rot=rot(8, 1e4), kv_from=0, mlp=None)]
    spec = sure_routing(small_spec(layers=layers))
    model, eng, w = build(spec, dtype, tweak=sharpen, block_size=16, num_blocks=64, max_tokens=512)
    toks = tokens_for(spec, 300, 9)
    want = Expected(spec, w, toks, dtype)
    want.check(feed(eng, "a", toks, [220, 1]))
    want.check(feed(eng, "b", toks, [300]))


OTHER_SIZES = {
    "one layer of each": dict(layers=[att_layer, mem_layer]),
    "reverse order": dict(layers=[mem_layer, att_layer]),
    "only memories": dict(layers=[mem_layer, lambda: mem_layer(heads=1, dim=1, vdim=33, **DENSE), mem_layer]),
    "only attention": dict(layers=[att_layer, lambda: att_layer(**MOE)]),
    "one head": dict(layers=[lambda: att_layer(heads=1), lambda: mem_layer(heads=1)]),
    "many heads": dict(layers=[lambda: att_layer(heads=20, dim=8, rot_dim=8, rot=rot(8), vdim=8, kv_rank=32), lambda: mem_layer(heads=9, dim=8, vdim=8)]),
    "sizes of 8s": dict(layers=[lambda: att_layer(heads=8, dim=32, rot_dim=16, rot=rot(16, 1e4, **STRETCH), vdim=32, kv_rank=64, q_rank=48, ff=64),
                                lambda: mem_layer(heads=4, dim=32, vdim=64, expert_ff=32, shared_ff=48),
                                lambda: att_layer(heads=16, dim=32, rot_dim=16, rot=rot(16, 1e4, **STRETCH), vdim=16, kv_rank=64, q_rank=64, kv_from=0, ff=64)], width=64),
    "odd sizes": dict(layers=[lambda: att_layer(heads=3, dim=7, rot_dim=2, rot=rot(2), vdim=3, kv_rank=9, q_rank=5, ff=11), lambda: mem_layer(dim=5, vdim=3, expert_ff=7, shared_ff=1)],
                      width=33, vocab=101),
    "no unrotated part": dict(layers=[lambda: att_layer(dim=0, rot_dim=16, rot=rot(16))]),
    "no rotated part": dict(layers=[lambda: att_layer(rot_dim=0, rot=rot(0))]),
    "partly rotated, plain steps": dict(layers=[lambda: att_layer(rot_dim=12, rot=rot(4)), lambda: att_layer(rot_dim=8, rot=rot(0))]),
    "wide latents": dict(layers=[lambda: att_layer(kv_rank=264, q_rank=3, rot_dim=64, rot=rot(64, 1e4, **STRETCH)), lambda: att_layer(kv_rank=512, rot_dim=64, rot=rot(64))]),
    "key size 130 and 200": dict(layers=[lambda: mem_layer(heads=2, dim=130, vdim=8), lambda: mem_layer(heads=1, dim=200, vdim=150)]),
    "value sizes at a tile's edge": dict(layers=[lambda: mem_layer(vdim=15), lambda: mem_layer(vdim=16), lambda: mem_layer(vdim=31), lambda: mem_layer(vdim=1)]),
    "tight and loose gate caps": dict(layers=[lambda: mem_layer(gate_cap=0.5), lambda: mem_layer(gate_cap=30.0)]),
    "one expert": dict(layers=[lambda: mem_layer(experts=1, top=1, groups=1, keep_groups=1), lambda: att_layer(**dict(MOE, experts=2, top=2, groups=2, keep_groups=2, shared_ff=0))]),
    "many experts": dict(layers=[lambda: mem_layer(experts=40, top=4, groups=8, keep_groups=3, expert_ff=8), lambda: att_layer(**dict(MOE, experts=256, top=2, groups=1, keep_groups=1, expert_ff=4))]),
    "no feed-forward anywhere": dict(layers=[lambda: att_layer(mlp=None), lambda: mem_layer(mlp=None), lambda: att_layer(mlp=None, kv_from=0)]),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(OTHER_SIZES))
def test_other_sizes(gpu, dtype, name):
    kw = dict(OTHER_SIZES[name])
    kw["layers"] = [f() for f in kw["layers"]]
    spec = routed(small_spec(**kw), dtype)
    model, eng, w = build(spec, dtype)
    toks = tokens_for(spec, 37, 4, w, dtype)
    want = Expected(spec, w, toks, dtype)
    lg, _, tr = eng.step([("a", toks, list(range(37)))], layer_trace=True)
    assert tr.shape[0] == len(spec.layers)
    want.check_layer(-1, tr[-1].cpu().numpy())
    want.check(lg.cpu().numpy())
    eng.finish("a")
    want.check(feed(eng, "b", toks, [30, 1]))
    want.check(feed(eng, "c", toks, [2]))


def random_spec(rng):
    pick = lambda *a: a[int(rng.integers(0, len(a)))]   # noqa: E731
    layers = []
    for i in range(int(rng.integers(1, 6))):
        mult8 = rng.random() < 0.5
        size = lambda lo, hi: 8 * int(rng.integers(1, 6)) if mult8 else int(rng.integers(lo, hi))   # noqa: E731
        kind = pick("none", "dense", "moe", "moe")
        if kind == "moe":
            groups = int(rng.integers(1, 5))
            per = int(rng.integers(1, 6))
            keep = int(rng.integers(1, groups + 1))
            ff = dict(mlp="moe", experts=groups * per, groups=groups, keep_groups=keep, top=int(rng.integers(1, keep * per + 1)), expert_ff=size(4, 40),
                      shared_ff=int(pick(0, 8, 21)), router_scale=float(pick(1.0, 2.5)))
        else:
            ff = dict(mlp="dense", ff=size(5, 70)) if kind == "dense" else dict(mlp=None)
        if rng.random() < 0.5:
            layers.append(mem_layer(heads=int(rng.integers(1, 6)), dim=size(3, 60), vdim=size(4, 50), gate_cap=float(pick(3.0, 10.0, 15.0)), **ff))   # a norm over 1 .. 3 numbers turns rounding into sign flips
            continue
        own = [j for j, l in enumerate(layers) if l.mixer == "latent_attention" and l.kv_from is None]
        a = dict(heads=int(rng.integers(1, 8)), dim=size(2, 40), vdim=size(3, 40), q_rank=size(5, 40), scale=float(rng.uniform(0.1, 0.5)), **ff)
        if own and rng.random() < 0.6:
            src = layers[int(pick(*own))]
            a.update(kv_rank=src.kv_rank, rot_dim=src.rot_dim, rot=src.rot, kv_from=layers.index(src))
        else:
            rd = 8 * int(rng.integers(0, 4)) if mult8 else 2 * int(rng.integers(0, 12))
            st = dict(factor=float(pick(2.0, 4.0, 16.0)), original=float(pick(16, 64, 2048)), fast=float(pick(4.0, 32.0)), slow=float(pick(0.5, 1.0, 2.0))) if rng.random() < 0.5 else {}
            a.update(kv_rank=size(6, 70), rot_dim=rd, rot=rot(rd, float(pick(100.0, 1e4, 1e6)), **st) if rd else rot(0))
        layers.append(att_layer(**a))
    return small_spec(layers=layers, width=8 * int(rng.integers(2, 12)) if rng.random() < 0.5 else int(rng.integers(12, 90)), vocab=int(rng.integers(20, 300)),
                      norm_eps=float(pick(1e-6, 1e-5)))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(14))
def test_random_models(gpu, dtype, seed):
    """Models drawn at random (layer order, shared latents, head counts, sizes, rotations, gates, experts) on random page sizes: two
    unequal requests decoding together, a third fed in portions."""
    rng = np.random.default_rng(seed)
    spec = routed(random_spec(rng), dtype)
    bs = int(rng.choice([1, 3, 4, 8, 16]))
    model, eng, w = build(spec, dtype, seed=seed, block_size=bs, num_blocks=600 // bs + 8)
    ta, tb, tc = tokens_for(spec, 75, seed, w, dtype), tokens_for(spec, 33, seed + 50, w, dtype), tokens_for(spec, 60, seed + 99, w, dtype)
    wa, wb, wc = (Expected(spec, w, t, dtype) for t in (ta, tb, tc))
    lg, _, _ = eng.step([("a", ta[:60], list(range(60))), ("b", tb[:20], list(range(20)))])
    ga, gb = [lg[:60].cpu().numpy()], [lg[60:].cpu().numpy()]
    for i in range(15):
        ent = [("a", [ta[60 + i]], [0])] + ([("b", [tb[20 + i]], [0])] if i < 13 else [])
        lg, _, _ = eng.step(ent)
        ga.append(lg[:1].cpu().numpy())
        if i < 13:
            gb.append(lg[1:2].cpu().numpy())
        if i == 12:
            eng.finish("b")
    wa.check(np.concatenate(ga))
    wb.check(np.concatenate(gb))
    wc.check(feed(eng, "c", tc, [int(rng.integers(2, 20)), int(rng.integers(1, 9))]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decode_step_replays_as_a_graph(gpu, dtype):
    """A captured decode step of two sequences, replayed with eager work between the replays, gives the eager step's logits; the
    recurrent state moves on with every replay, so each is compared with an eager run of the same number of steps."""
    _, torch = gpu
    spec = routed(small_spec(), dtype)
    outs = []
    for graph in (False, True):
        model, eng, w = build(spec, dtype)
        toks = [tokens_for(spec, 21, 5), tokens_for(spec, 9, 6)]
        eng.step([("a", toks[0], []), ("b", toks[1], [])])
        for s in ("a", "b"):                                       # room for the decoded rows
            eng.seqs[s].blocks.extend(eng.blocks.allocate(2))
        i32 = lambda a: torch.tensor(a, dtype=torch.int32, device="cuda")   # noqa: E731
        wd = max(len(eng.seqs[s].blocks) for s in ("a", "b"))
        bt = i32([eng.seqs[s].blocks + [0] * (wd - len(eng.seqs[s].blocks)) for s in ("a", "b")])
        tok, pos, slots = i32([3, 4]), i32([0, 0]), i32([0, 0])
        sid, starts, states, rows = i32([0, 1]), i32([0, 1, 2]), i32([eng.seqs[s].state_slot for s in ("a", "b")]), i32([0, 1])

        def place(step):
            p = [21 + step, 9 + step]
            pos.copy_(i32(p))
            slots.copy_(i32([eng.seqs[s].blocks[q // 4] * 4 + q % 4 for s, q in zip(("a", "b"), p)]))
            tok.copy_(i32([3 + step, 4 + 2 * step]))
        run = lambda: model.forward(tok, None, pos, slots, sid, bt, rows, seq_starts=starts, state_slots=states)[0]   # noqa: E731
        place(0)
        got = []
        if graph:
            stream = torch.cuda.Stream()
            with torch.cuda.stream(stream):
                got.append(run().cpu())                            # step 0 eagerly
                g = torch.cuda.CUDAGraph()
                with torch.cuda.graph(g, stream=stream):
                    lg = run()
                for step in range(1, 5):
                    place(step)
                    g.replay()
                    torch.cuda.synchronize()
                    got.append(lg.cpu())
        else:
            for step in range(5):
                place(step)
                got.append(run().cpu())
        outs.append(torch.stack(got))
        model.close()
    assert bool((outs[0] == outs[1]).all())


def test_greedy_generation_through_the_scheduler(gpu):
    """Engine.generate (scheduler, block pressure, prompt portions, greedy ids from the executor) against the oracle's argmax
    continuation; sampled generation runs and stays in the vocabulary."""
    from tests import fofinex_oracle as orc
    from vllm_rust_amd.engine import SamplingParams
    spec = small_spec()
    model, eng, w = build(spec, "float32", num_blocks=30, max_seqs=3)
    prompts = [tokens_for(spec, n, 70 + n) for n in (9, 23, 4, 15, 2)]
    outs = eng.generate(prompts, SamplingParams(max_new_tokens=8), prefill_chunk=6)
    for p, o in zip(prompts, outs):
        seq = list(p)
        for t in o:
            margins = []
            lg = orc.forward(spec.to_config(), w, seq, margins)[0].numpy()
            if min(margins) < 1e-5:
                break                         # a router decision within rounding: the continuation may differ legitimately
            top2 = np.sort(lg[-1])[-2:]
            if top2[1] - top2[0] > 1e-3:      # a tie within rounding says nothing
                assert int(np.argmax(lg[-1])) == t
            seq.append(t)
    assert len(eng.blocks.free) == 30 and len(eng.states.free) == 3
    outs = eng.generate(prompts[:3], SamplingParams(temperature=0.9, top_k=20, top_p=0.9, max_new_tokens=5, seed=3))
    assert all(len(o) == 5 and all(0 <= t < spec.vocab for t in o) for o in outs)


def _write_checkpoint(tmp_path, spec, seed=0):
    import torch
    from safetensors.torch import save_file
    from vllm_rust_amd.fofinex import synthetic_weights
    ck = synthetic_weights(spec, seed)
    d = tmp_path / "model"
    d.mkdir()
    (d / "config.json").write_text(json.dumps(spec.to_config()))
    extra = {f"l{i}.{n}": torch.ones(spec.width, dtype=torch.bfloat16) for i, l in enumerate(spec.layers) if l.mlp is None for n in ("norm2", "norm2b")}   # skipped
    save_file({k: v.contiguous() for k, v in {**ck, **extra}.items()}, str(d / "model.safetensors"))
    return d, {k: v.double() for k, v in ck.items()}


def test_registry_and_command_line_tools(gpu, tmp_path):
    """A checkpoint directory written here: the registry picks the class from config.json; bin/trace_run replays a trace (a prompt,
    a portion, decode steps of two requests, an early finisher) in both modes; bin/generate continues greedily."""
    from vllm_rust_amd.engine import Engine
    from vllm_rust_amd.models import architecture_of, load_model
    spec = sure_routing(small_spec())        # one checkpoint for both modes
    d, w = _write_checkpoint(tmp_path, spec)
    assert architecture_of(d) == "Fofinex"
    model = load_model(d, dtype="float32", max_tokens=128, max_seqs=4, block_size=8)
    assert model.spec.to_config() == spec.to_config()
    ta, tb = tokens_for(spec, 30, 1), tokens_for(spec, 12, 2)
    wa, wb = {}, {}
    for dt in TOL:
        wa[dt], wb[dt] = Expected(spec, w, ta, dt), Expected(spec, w, tb, dt)
    lg, _, _ = Engine(model).step([("x", ta, [29])])
    wa["float32"].check(lg.cpu().numpy(), [29])
    model.close()
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": ta[:20], "want": [0, 19]}, {"id": "b", "tokens": tb[:10], "want": [9]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [ta[20]], "want": [0]}, {"id": "b", "tokens": [tb[10]], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": [ta[21]], "want": [0]}, {"id": "b", "tokens": [tb[11]], "want": [0]}], "end": ["b"]},
             {"step": 3, "entries": [{"id": "a", "tokens": ta[22:30], "want": [7]}], "end": ["a"]}]
    for dtype in ("float32", "bfloat16"):
        out = tmp_path / f"out_{dtype}"
        r = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--model", str(d), "--dtype", dtype, "--out", str(out), "--max-tokens", "64"],
                           input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
        assert r.returncode == 0, r.stderr
        assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
        rd = lambda i: np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, spec.vocab)   # noqa: E731
        wa[dtype].check(rd(0)[:2], [0, 19])
        wb[dtype].check(rd(0)[2:], [9])
        wa[dtype].check(rd(1), [20])
        wa[dtype].check(rd(2)[:1], [21])
        wb[dtype].check(rd(2)[1:], [11])
        wa[dtype].check(rd(3), [29])
    r = subprocess.run([sys.executable, str(ROOT / "bin" / "generate"), "--model", str(d), "--dtype", "float32", "--prompt", ",".join(map(str, ta[:9])),
                        "--max-new-tokens", "4"], capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr
    ids = [int(t) for t in r.stdout.strip().splitlines()[-1].split(",")]
    assert len(ids) == 4 and all(0 <= t < spec.vocab for t in ids)
