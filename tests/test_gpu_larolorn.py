"""Larolorn on the GPU against the float64 oracle (tests/larolorn_oracle.py): every mechanism alone (windowed latent attention and
chunked sink attention with needle keys at every edge, whole-row query / key preparation, the memory with constant decays fed in
portions through dirty state slots, the read-out of wide rows), then the executor through the engine's step function under different
cuttings of the same tokens (whole prompts, token-by-token decoding, portions down to two tokens, unequal batches, recycled cache
blocks and state slots), layers that share weights, rows of every width, other sizes, random models, and greedy generation through the
scheduler.  Small random models built here; float32 mode is held to 2e-4 of the logits' spread, bfloat16 mode to 4e-2 or three times
what rounding alone does."""
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


def rot(dims, base=500.0):
    from vllm_rust_amd.rotation import RotationSpec
    return RotationSpec(dims, base)


DENSE = dict(mlp="dense", ff=36, limit=0.9)      # a limit that many gate and up values pass on both sides


def att_layer(**kw):
    from vllm_rust_amd.larolorn import LarolornLayerSpec
    d = dict(mixer="latent_attention", heads=3, dim=10, rot_dim=6, vdim=14, kv_rank=20, scale=0.3, mask=7, rot=rot(6, 300.0), **DENSE)
    d.update(kw)
    return LarolornLayerSpec(**d)


def par_layer(**kw):
    from vllm_rust_amd.larolorn import LarolornLayerSpec
    d = dict(mixer="parallel", heads=6, kv_heads=2, dim=10, vdim=7, scale=0.4, mask=9, rot=rot(6, 200.0), r_heads=3, r_dim=9, r_vdim=11,
             decay=None, **DENSE)
    d.update(kw)
    if d["decay"] is None:                       # from fast forgetting to almost none
        d["decay"] = tuple(float(np.float32(1.0 - 0.5 ** (1 + 7 * i / max(d["r_heads"] - 1, 1)))) for i in range(d["r_heads"]))
    return LarolornLayerSpec(**d)


def small_spec(layers=None, **kw):
    from vllm_rust_amd.larolorn import LarolornSpec
    layers = layers or [att_layer(), par_layer(), att_layer(weights_of=0), par_layer(heads=4, kv_heads=4, dim=8, vdim=12, mask=5, rot=rot(8), r_heads=2, r_dim=14, r_vdim=5),
                        par_layer(weights_of=1), att_layer(heads=5, dim=7, vdim=9, kv_rank=33, rot_dim=10, rot=rot(10, 100.0), mask=16, mlp=None)]
    d = dict(vocab=67, width=40, layers=layers, norm_eps=1e-5, residual_mult=0.6, logit_scale=0.7)
    d.update(kw)
    return LarolornSpec(**d)


def build(spec, dtype="float32", seed=0, tweak=None, block_size=4, num_blocks=96, max_tokens=320, max_seqs=6):
    from vllm_rust_amd.engine import Engine
    from vllm_rust_amd.larolorn import LarolornForCausalLM, synthetic_weights
    ck = synthetic_weights(spec, seed)
    if tweak:
        tweak(ck)
    model = LarolornForCausalLM(spec, dtype=dtype, block_size=block_size, num_blocks=num_blocks, max_tokens=max_tokens, max_seqs=max_seqs)
    model.load_state(ck)
    return model, Engine(model), {k: v.double() for k, v in ck.items()}


def tokens_for(spec, n, seed):
    return np.random.default_rng(seed).integers(0, spec.vocab, n).tolist()


def row_errs(got, want):
    """Difference of two logits arrays per row, row means removed, relative to the spread of the expected row."""
    g, w = np.asarray(got, np.float64), np.asarray(want, np.float64)
    d = g - w
    d = d - d.mean(-1, keepdims=True)
    return np.sqrt((d ** 2).mean(-1)) / (w.std(-1) + 1e-12)


class Expected:
    """The oracle's logits and streams of a token sequence, and how far a run may be from them: float32 2e-4 in every row; bfloat16
    4e-2 in every row and 1.5e-2 in the mean, or three times what rounding the operands alone does to this model and these tokens
    (sublayer results are divided by their own size, so some rows amplify rounding a lot)."""

    def __init__(self, spec, weights, toks, dtype):
        from tests import larolorn_oracle as orc
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
    from tests import larolorn_oracle as orc
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

def _bf(t):
    import torch
    return t.to(torch.bfloat16).double()


def _scattered(torch, rows, bs, dtype, seed=1):
    """rows [T, n] in cache blocks scattered over a larger, NaN-filled cache: (cache, block table on the GPU)."""
    T, n = rows.shape
    nb = (T + bs - 1) // bs
    perm = np.random.default_rng(seed).permutation(nb + 5)[:nb].astype(np.int32)
    pos = np.arange(T)
    cache = torch.full(((nb + 5) * bs, n), float("nan"), dtype=torch.float32)
    cache[perm[pos // bs] * bs + pos % bs] = rows.float()
    return cache.to(torch.float32 if dtype == 0 else torch.bfloat16).cuda(), torch.from_numpy(perm[None]).cuda()


@pytest.mark.parametrize("H,R,rd,window", [(3, 24, 8, 40), (7, 112, 40, 65), (16, 64, 16, 64), (20, 16, 0, 17), (2, 33, 6, 96), (5, 256, 64, 1), (9, 40, 24, 130)])
@pytest.mark.parametrize("dtype,bs", [(0, 16), (1, 16), (1, 5), (0, 1)])
def test_windowed_latent_attention_with_needles(gpu, H, R, rd, window, dtype, bs):
    """Keys whose score stands out, asked for from distance window - 1 (the last row that sees them), window (the first that does not)
    and in between, in a prompt, in portions and as single decoded rows, with the first token of the sequence among them."""
    _, torch = gpu
    from vllm_rust_amd._lib import check, lib
    T = 330
    g = torch.Generator().manual_seed(R + H)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)   # noqa: E731
    q, row = 0.2 * rn(T, H, R + rd), 0.2 * rn(T, R + rd)
    needles = [0, 16, 31, 150]
    asked = {}
    for n in needles:
        d = rn(R + rd)
        row[n] = d * (5 / d.norm())
    for n in needles:
        for i in (n + window - 1, n + window, n + window // 2):
            if i < T and i not in needles:
                q[i], asked[i] = row[n] * 4, n       # score 50 against the needle, of order 1 against the rest
    q, row = _bf(q), _bf(row)
    s = torch.einsum("ihd,jd->hij", q, row) * 0.5
    i, j = torch.arange(T).unsqueeze(1), torch.arange(T).unsqueeze(0)
    s = s.masked_fill((j > i) | (i - j >= window), -math.inf)
    want = torch.einsum("hij,jr->ihr", torch.softmax(s, -1), row[:, :R])
    for i, n in asked.items():                       # by construction: there inside, gone outside
        near = float((want[i] - row[n, :R]).abs().max()) < 1e-3 * float(row[n].abs().max())
        assert near == (i - n < window) or window == 1
    cache, bt = _scattered(torch, row, bs, dtype)
    nb = bt.shape[1]
    tol = (3e-5 if dtype == 0 else 2e-2) * float(want.abs().max())
    for a, b in [(0, T), (290, T), (17, 19), (63, 130)] + [(i, i + 1) for i in asked]:
        n = b - a
        qa, qr = q[a:b, :, :R].float().contiguous().cuda(), q[a:b, :, R:].float().contiguous().cuda() if rd else torch.zeros(1, device="cuda")
        out = torch.empty(n, H, R, device="cuda")
        P, sid = torch.arange(a, b, dtype=torch.int32, device="cuda"), torch.zeros(n, dtype=torch.int32, device="cuda")
        ws = torch.empty(lib.vmx_latent_attention_workspace_bytes(n, H, R, window, nb, bs) // 4 + 1, device="cuda")
        check(lib.vmx_latent_attention(out.data_ptr(), qa.data_ptr(), qr.data_ptr(), cache.data_ptr(), dtype, bt.data_ptr(), nb, sid.data_ptr(), P.data_ptr(), None,
                                       0.5, window, n, H, R, rd, bs, ws.data_ptr(), ws.numel() * 4, None))
        torch.cuda.synchronize()
        assert float((out.cpu().double() - want[a:b]).abs().max()) < tol, (a, b)


FORMS = [(0, False), (1, False), (1, True), (1, "split")]   # (cache dtype, runs): f32 vector, bf16 vector, matrix cores, + key shares


def _attention_op(torch, q, k, v, scale, window, chunk, keep, bs, form, a, b, sink=None, talk=None):
    """vmx_window_attention_ex for rows a .. b - 1 of one sequence whose keys are all cached in scattered blocks."""
    from vllm_rust_amd._lib import WindowAttnExtras, check, lib
    dtype, runs = form
    T, H, D = q.shape
    G, V = k.shape[1], v.shape[2]
    kc, bt = _scattered(torch, k[:b].reshape(b, G * D), bs, dtype)
    vc, _ = _scattered(torch, v[:b].reshape(b, G * V), bs, dtype)
    n = b - a
    out = torch.empty((n, H * V), device="cuda")
    qd = q[a:b].reshape(n, H * D).float().contiguous().cuda()
    sid, P = torch.zeros(n, dtype=torch.int32, device="cuda"), torch.arange(a, b, dtype=torch.int32, device="cuda")
    st = torch.tensor([0, n], dtype=torch.int32, device="cuda")
    ws = torch.empty(lib.vmx_window_attention_workspace_bytes(n, H, V) // 4, device="cuda")
    kept = [None if t is None else t.to(torch.bfloat16).cuda() for t in (sink, talk)]
    ex = WindowAttnExtras(None if sink is None else kept[0].data_ptr(), None, None, None if talk is None else kept[1].data_ptr(), 0, chunk)
    check(lib.vmx_window_attention_ex(out.data_ptr(), 0, qd.data_ptr(), H * D, kc.data_ptr(), vc.data_ptr(), dtype, bt.data_ptr(), bt.shape[1], sid.data_ptr(),
                                      P.data_ptr(), None, None, 0, scale, 0.0, window, keep, n, H, G, D, V, bs, st.data_ptr() if runs else None, 1 if runs else 0,
                                      ws.data_ptr() if runs == "split" else None, ws.numel() * 4, C.byref(ex), None))
    torch.cuda.synchronize()
    return out.cpu().double().reshape(n, H, V)


def _attention_want(torch, q, k, v, scale, window, chunk, keep, sink=None, talk=None):
    """The same with one visibility matrix; rows of the oracle's own attention where no mixing or kept tokens are asked for."""
    T, H, _ = q.shape
    own = [h // (H // k.shape[1]) for h in range(H)]
    i, j = torch.arange(T).unsqueeze(1), torch.arange(T).unsqueeze(0)
    seen = (j <= i)
    far = torch.zeros_like(seen)
    if window:
        far = far | (i - j >= window)
    if chunk:
        far = far | (i // chunk != j // chunk)
    seen = seen & (~far | (j < keep))
    s = torch.einsum("ihd,jhd->hij", q, k[:, own]) * scale
    if talk is not None:
        s = torch.einsum("hg,gij->hij", talk, s)
    s = s.masked_fill(~seen, -math.inf)
    if sink is not None:
        s = torch.cat([s, sink.reshape(H, 1, 1).expand(H, T, 1)], -1)
    return torch.einsum("hij,jhv->ihv", torch.softmax(s, -1)[:, :, :T], v[:, own])


@pytest.mark.parametrize("form", FORMS)
@pytest.mark.parametrize("H,G,D,V,chunk,bs", [(4, 2, 16, 24, 9, 4), (6, 2, 8, 8, 1, 16), (3, 1, 11, 11, 50, 3), (8, 8, 64, 64, 40, 16), (12, 2, 40, 32, 70, 8), (1, 1, 40, 16, 2, 1),
                                             (16, 2, 128, 128, 100, 16), (4, 1, 24, 24, 64, 16), (2, 2, 32, 16, 400, 5)])
def test_chunked_sink_attention(gpu, form, H, G, D, V, chunk, bs):
    """All rows at once, a portion that starts inside a chunk, one that starts at a chunk's edge, and single rows at the edges."""
    _, torch = gpu
    from tests import larolorn_oracle as orc
    T = 210
    g = torch.Generator().manual_seed(H + chunk)
    q, k, v = (_bf(torch.randn(*s, generator=g, dtype=torch.float64)) for s in ((T, H, D), (T, G, D), (T, G, V)))
    sink = _bf(2 * torch.randn(H, generator=g, dtype=torch.float64))
    own = [h // (H // G) for h in range(H)]
    want = orc.softmax_attention(q, k[:, own], v[:, own], 0.3, lambda i: orc.chunk_start(i, chunk), sink)
    assert float((want - _attention_want(torch, q, k, v, 0.3, 0, chunk, 0, sink)).abs().max()) < 1e-9
    tol = 2e-5 if form[0] == 0 else 6e-3
    edge = min(chunk, T - 1)
    for a, b in [(0, T), (T - 37, T), (edge, T), (0, 1)] + [(i, i + 1) for i in (edge - 1, edge, edge + 1, T - 1) if i < T]:
        got = _attention_op(torch, q, k, v, 0.3, 0, chunk, 0, bs, form, a, b, sink=sink)
        assert float((got - want[a:b]).abs().max()) < tol * max(1.0, float(want.abs().max())), (a, b)


@pytest.mark.parametrize("form", FORMS)
@pytest.mark.parametrize("chunk,bs", [(40, 16), (64, 16), (65, 8), (17, 5), (128, 16), (3, 16)])
def test_needles_at_the_edges_of_chunks(gpu, form, chunk, bs):
    """Keys whose score stands out as the first and the last of their chunk: every later row of the chunk finds them, the first row
    of the next one does not, in a prompt and as single decoded rows; a chunk larger than the sequence loses nothing; the sink takes
    the weight of rows whose own scores are low."""
    _, torch = gpu
    H, G, D, V, T = 4, 2, 16, 24, 330
    g = torch.Generator().manual_seed(chunk)
    rn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)   # noqa: E731
    q, k, v = 0.2 * rn(T, H, D), 0.2 * rn(T, G, D), rn(T, G, V)
    d = rn(G, D).sign()
    first, last = 2 * chunk, 3 * chunk - 1
    if last + 1 >= T:
        first, last = chunk, 2 * chunk - 1
    k[first], k[last] = d, d                          # score 16 against a query along d
    rows = sorted({first, first + chunk // 2, last, last + 1, last + 2, T - 1})
    for i in rows:
        q[i] = d.repeat_interleave(H // G, dim=0)
    q, k, v = _bf(q), _bf(k), _bf(v)
    sink = _bf(torch.tensor([-3.0, 4.0, 0.0, 9.0], dtype=torch.float64))
    tol = 2e-5 if form[0] == 0 else 8e-3
    for size in (chunk, 0, 1000):
        want = _attention_want(torch, q, k, v, 1.0, 0, size, 0, sink)
        for a, b in [(0, T)] + [(i, i + 1) for i in rows] + [(first, last + 2), (last + 1, T)]:
            got = _attention_op(torch, q, k, v, 1.0, 0, size, 0, bs, form, a, b, sink=sink)
            assert float((got - want[a:b]).abs().max()) < tol * max(1.0, float(want.abs().max())), (size, a, b)
        if size == chunk:                             # head 0, whose sink is low: both needles inside, none outside
            assert chunk <= 3 or float((want[first + chunk // 2] - v[first, 0])[0].abs().max()) < 0.05
            assert float((want[last] - (v[first, 0] + v[last, 0]) / 2)[0].abs().max()) < 0.05
            for vn in (v[first, 0], v[last, 0], (v[first, 0] + v[last, 0]) / 2):
                assert float((want[last + 1] - vn)[0].abs().max()) > 0.2


@pytest.mark.parametrize("form", FORMS)
@pytest.mark.parametrize("mixed", [False, True])
@pytest.mark.parametrize("window,chunk,keep", [(20, 33, 0), (50, 33, 0), (20, 33, 3), (0, 33, 3), (33, 0, 2), (7, 7, 0)])
def test_chunks_beside_windows_kept_tokens_and_mixed_heads(gpu, form, mixed, window, chunk, keep):
    """Chunks are a parameter beside the window, the kept first tokens, the sink and the mixed heads of the same kernels."""
    _, torch = gpu
    H, G, D, T = 4, 2, 16, 150
    g = torch.Generator().manual_seed(window + chunk)
    rn = lambda *s: _bf(torch.randn(*s, generator=g, dtype=torch.float64))   # noqa: E731
    q, k, v, sink = rn(T, H, D), rn(T, G, D), rn(T, G, D), rn(H)
    talk = _bf(torch.eye(H, dtype=torch.float64) + 0.3 * torch.randn(H, H, generator=g, dtype=torch.float64)) if mixed else None
    want = _attention_want(torch, q, k, v, 0.3, window, chunk, keep, sink, talk)
    tol = 2e-5 if form[0] == 0 else 6e-3
    for a, b in [(0, T), (70, 120)] + [(i, i + 1) for i in (32, 33, 65, 66, T - 1)]:
        got = _attention_op(torch, q, k, v, 0.3, window, chunk, keep, 8, form, a, b, sink=sink, talk=talk)
        assert float((got - want[a:b]).abs().max()) < tol * max(1.0, float(want.abs().max())), (a, b)


@pytest.mark.parametrize("H,G,hd,rd,halves", [(4, 2, 12, 8, 1), (3, 1, 11, 10, 1), (8, 2, 64, 32, 1), (2, 2, 7, 0, 1), (5, 5, 130, 130, 1), (1, 1, 256, 256, 1), (32, 8, 128, 64, 1),
                                              (4, 2, 12, 8, 0), (8, 2, 64, 32, 0), (3, 3, 8, 0, 0), (5, 5, 130, 130, 0), (1, 1, 256, 256, 0)])
@pytest.mark.parametrize("dtype", [0, 1])
@pytest.mark.parametrize("cached", [True, False])
def test_whole_row_preparation(gpu, H, G, hd, rd, halves, dtype, cached):
    """Norms over all heads at once, then the rotation of each head, to the cache rows or to plain rows."""
    _, torch = gpu
    from tests import larolorn_oracle as orc
    from vllm_rust_amd._lib import QkPrepareOpts, check, lib
    T, V, base, eps = 9, 5, 777.0, 1e-2
    g = torch.Generator().manual_seed(H * hd)
    rn = lambda *s: torch.randn(*s, generator=g).float()   # noqa: E731
    q, k, v = rn(T, H * hd), rn(T, G * hd), rn(T, G * V)
    qn, kn = (1 + 0.2 * rn(H * hd)).to(torch.bfloat16), (1 + 0.2 * rn(G * hd)).to(torch.bfloat16)
    pos, slots = [0, 1, 2, 3, 50, 51, 1000, 1001, 5000], [5, 4, -1, 0, 1, 2, 11, 10, 7]
    fused = torch.cat([q, k, v, rn(T, 3)], 1).cuda()
    ld = fused.shape[1]
    i32 = lambda a: torch.tensor(a, dtype=torch.int32, device="cuda")   # noqa: E731
    P, S, qnd, knd = i32(pos), i32(slots), qn.cuda(), kn.cuda()
    steps = torch.tensor([base ** (-2.0 * i / rd) for i in range(rd // 2)], dtype=torch.float32, device="cuda") if rd else None
    cdt = torch.float32 if dtype == 0 else torch.bfloat16
    qo, kp = torch.empty(T, H * hd, device="cuda"), torch.full((T, G * hd + 2), 7.0, device="cuda")
    kc, vc = torch.full((13, G * hd), 7.0, dtype=cdt, device="cuda"), torch.full((13, G * V), 7.0, dtype=cdt, device="cuda")
    po = QkPrepareOpts(0, halves, 1.0, 0.5, 2.0, None if cached else kp.data_ptr(), G * hd + 2)
    at = lambda off: fused.data_ptr() + 4 * off   # noqa: E731
    check(lib.vmx_qk_prepare_ex(qo.data_ptr(), at(0), ld, H * hd, at(H * hd), ld, G * hd, at((H + G) * hd), ld, G * V, qnd.data_ptr(), knd.data_ptr(), eps,
                                None if steps is None else steps.data_ptr(), rd, hd, P.data_ptr(), S.data_ptr(), kc.data_ptr(), vc.data_ptr(), dtype, T, C.byref(po), None))
    torch.cuda.synchronize()
    turn = orc.rotate_halves if halves else orc.rotate_neighbours
    rotd = dict(dims=rd, base=base) if rd else None
    wq = turn(orc.rms_norm(q.double(), qn.double(), eps).reshape(T, H, hd), pos, rotd).reshape(T, H * hd) * 0.5
    wk = turn(orc.rms_norm(k.double(), kn.double(), eps).reshape(T, G, hd), pos, rotd).reshape(T, G * hd) * 2.0
    # angles are f32 products of a position and an f32 step: at position 5000 they carry an error of about 5000 * 2^-24
    tol, low = (1e-2 if rd else 1e-5), (0.06 if dtype == 1 else 0.0)
    assert float((qo.cpu().double() - wq).abs().max()) < tol
    if not cached:
        assert float((kp[:, :G * hd].cpu().double() - wk).abs().max()) < tol and bool((kp[:, G * hd:] == 7.0).all()) and bool((kc == 7.0).all()) and bool((vc == 7.0).all())
        return
    for t, s in enumerate(slots):
        if s >= 0:
            assert float((kc[s].cpu().double() - wk[t]).abs().max()) < tol + low
            assert float((vc[s].cpu().double() - v[t].double()).abs().max()) < 1e-6 + low
    for s in (3, 6, 8, 9, 12):
        assert bool((kc[s] == 7.0).all()) and bool((vc[s] == 7.0).all())


def _run_memory(torch, q, k, v, decay, portions, slot_of, chunks):
    """vmx_matrix_memory_recurrence_ex with constant decays over several sequences fed in unequal portions through NaN-filled slots."""
    from vllm_rust_amd._lib import MatrixMemoryOpts, check, lib
    H, D, V = k[0].shape[1], k[0].shape[2], v[0].shape[2]
    nslots = max(slot_of) + 2
    state = torch.full((lib.vmx_gated_delta_rule_state_bytes(nslots, H, D, V) // 4,), float("nan"), device="cuda")
    dec = torch.tensor(decay, dtype=torch.float32, device="cuda")
    lens = [x.shape[0] for x in q]
    got, fed = [[] for _ in lens], [0] * len(lens)
    i32 = lambda a: torch.tensor(a, dtype=torch.int32, device="cuda")   # noqa: E731
    for step in range(max(len(p) for p in portions)):
        parts, starts, slots, posn, owners = [], [0], [], [], []
        for s, n in enumerate(lens):
            if step < len(portions[s]) and fed[s] < n:
                c = min(portions[s][step], n - fed[s])
                a, b = fed[s], fed[s] + c
                parts.append(torch.cat([x[s][a:b].reshape(c, -1) for x in (q, k, v)], 1))
                posn += list(range(a, b))
                starts.append(starts[-1] + c)
                slots.append(slot_of[s])
                owners.append((s, c))
                fed[s] = b
        x = torch.cat(parts).float().cuda()
        T, ld = x.shape
        o = torch.empty(T, H * V, device="cuda")
        P, S, L = i32(posn), i32(starts), i32(slots)
        at = lambda off: x.data_ptr() + 4 * off   # noqa: E731
        mo = MatrixMemoryOpts(None, 0, None, 0, 1 if chunks else 0, T)
        check(lib.vmx_matrix_memory_recurrence_ex(o.data_ptr(), H * V, at(0), ld, 1.0, at(H * D), ld, at(2 * H * D), ld, dec.data_ptr(), 0, 1, None, 0, state.data_ptr(),
                                                  P.data_ptr(), S.data_ptr(), L.data_ptr(), len(slots), H, H, D, V, C.byref(mo), None))
        torch.cuda.synchronize()
        r, row = o.cpu().double().reshape(T, H, V), 0
        for s, c in owners:
            got[s].append(r[row:row + c])
            row += c
    assert fed == lens
    return [torch.cat(g) for g in got]


@pytest.mark.parametrize("H,D,V", [(2, 32, 32), (3, 5, 7), (4, 64, 47), (1, 130, 16), (2, 16, 1), (6, 40, 56)])
@pytest.mark.parametrize("chunks", [False, True])
def test_constant_decay_memory_in_portions_through_dirty_slots(gpu, H, D, V, chunks):
    """Both forms of the recurrence (q, k and v are bf16 numbers, so the chunked one is held to the same bounds; steps of few tokens
    take the other form, so the two hand the memory to each other) with decays from 0 to 1."""
    _, torch = gpu
    from tests import larolorn_oracle as orc
    gen = torch.Generator().manual_seed(H * D + V)
    lens = [331, 1, 70]
    bf = lambda *s: _bf(torch.randn(*s, generator=gen, dtype=torch.float64))   # noqa: E731
    q, k, v = [bf(n, H, D) for n in lens], [bf(n, H, D) for n in lens], [bf(n, H, V) for n in lens]
    decay = [float(np.float32(d)) for d in (1.0, 0.997, 0.4, 0.0, 0.95, 0.03)[:H]]
    got = _run_memory(torch, q, k, v, decay, [[90, 1, 1, 37, 2, 200], [1], [2, 3, 63, 1, 1]], [3, 0, 4], chunks)
    for s in range(3):
        want = orc.decayed_memory(q[s], k[s], v[s], decay)
        size = float(orc.decayed_memory(q[s].abs(), k[s].abs(), v[s].abs(), decay).max())
        assert float((got[s] - want).abs().max()) < 2e-6 * size, s


@pytest.mark.parametrize("chunks", [False, True])
def test_memory_keeps_a_far_key(gpu, chunks):
    """A key written at position 5 and asked for up to 290 tokens and four portions later: whole from a head with decay 1, faded by
    0.99^n from the next, gone from the last; before it there is nothing."""
    _, torch = gpu
    n, D, V = 300, 16, 8
    gen = torch.Generator().manual_seed(0)
    k = torch.zeros(n, 3, D, dtype=torch.float64)
    k[:, :, 1:] = _bf(torch.randn(n, 3, D - 1, generator=gen, dtype=torch.float64))
    k[5, :, 0] = 1.0
    v = _bf(torch.randn(n, 3, V, generator=gen, dtype=torch.float64))
    q = torch.zeros(n, 3, D, dtype=torch.float64)
    q[:, :, 0] = 1.0
    decay = [1.0, float(np.float32(0.99)), 0.5]
    got = _run_memory(torch, [q], [k], [v], decay, [[4, 100, 1, 150, 45]], [1], chunks)[0]
    assert float(got[:5].abs().max()) == 0
    for t in (5, 6, 63, 64, 104, 105, 295, 299):
        for h in range(3):
            assert float((got[t, h] - decay[h] ** (t - 5) * v[5, h]).abs().max()) < 2e-5


@pytest.mark.parametrize("H,V,pad", [(1, 257, 2), (1, 300, 0), (2, 1000, 4), (1, 1028, 2), (1, 2048, 0), (1, 4096, 4), (1, 4100, 0), (1, 9000, 0), (1, 9001, 4), (3, 64, 2)])
def test_read_out_of_wide_rows(gpu, H, V, pad):
    _, torch = gpu
    from tests import larolorn_oracle as orc
    from vllm_rust_amd._lib import ReadOutOpts, check, lib
    gen = torch.Generator().manual_seed(V)
    for per_head in (0, 1):
        for silu in (0, 1):
            for dtype in (0, 1):
                o, gate = torch.randn(5, H * V + pad, generator=gen).cuda() * 1e-2, torch.randn(5, H * V + 4, generator=gen).cuda()
                w = (1 + 0.2 * torch.randn(H * V if per_head else V, generator=gen)).to(torch.bfloat16).cuda()
                y = torch.empty(5, H * V, dtype=torch.bfloat16 if dtype else torch.float32, device="cuda")
                ro = ReadOutOpts(silu, per_head, None, 0, None, 0, 0.0)
                check(lib.vmx_head_read_out(y.data_ptr(), dtype, o.data_ptr(), H * V + pad, w.data_ptr(), gate.data_ptr(), H * V + 4, 1e-4, 5, H, V, C.byref(ro), None))
                torch.cuda.synchronize()
                ref = orc.rms_unit(o.cpu().double()[:, :H * V].reshape(5, H, V), 1e-4) * (w.cpu().double().reshape(H, V) if per_head else w.cpu().double())
                gz = gate.cpu().double()[:, :H * V]
                ref = ref.reshape(5, H * V) * torch.sigmoid(gz) * (gz if silu else 1.0)
                assert float((y.cpu().double() - ref).abs().max()) < (0.05 if dtype else 1e-5)


# ----------------------------------------------------------------------------- the executor through the engine

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_layers_and_logits_against_the_oracle(gpu, dtype):
    spec = small_spec()
    model, eng, w = build(spec, dtype)
    toks = tokens_for(spec, 41, 1)
    lg, _, tr = eng.step([("a", toks, list(range(len(toks))))], layer_trace=True)
    want = Expected(spec, w, toks, dtype)
    assert tr.shape[0] == len(spec.layers) == 6
    for r in range(tr.shape[0]):
        want.check_layer(r, tr[r].cpu().numpy())
    want.check(lg.cpu().numpy())


@pytest.mark.parametrize("kind", ["latent_attention", "parallel"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_every_layer_kind_alone(gpu, dtype, kind):
    """One layer of each kind with and without the feed-forward, with limits that cut almost everything, much and nothing."""
    make = att_layer if kind == "latent_attention" else par_layer
    for ff in (DENSE, dict(mlp=None), dict(DENSE, limit=0.05), dict(DENSE, limit=50.0, ff=1), dict(mask=0)):
        spec = small_spec(layers=[make(**ff)])
        model, eng, w = build(spec, dtype)
        toks = tokens_for(spec, 26, 2)
        lg, _, tr = eng.step([("a", toks, list(range(26)))], layer_trace=True)
        want = Expected(spec, w, toks, dtype)
        want.check_layer(0, tr[0].cpu().numpy())
        want.check(lg.cpu().numpy(), what=(kind, ff))
        model.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prompt_decode_and_portions_agree(gpu, dtype):
    spec = small_spec()
    model, eng, w = build(spec, dtype)
    toks = tokens_for(spec, 53, 2)
    want = Expected(spec, w, toks, dtype)
    for cuts in ([53], [1], [2], [3], [7, 16], [16, 1], [20, 2, 1], [9], [10, 8, 9]):
        want.check(feed(eng, "s", toks, cuts), what=f"cuts {cuts}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_batches_and_recycled_blocks_and_slots(gpu, dtype):
    """Three requests of unequal length in one batch, then decoded together while the short ones finish early; five generations of
    requests through 3 state slots and few blocks, freed blocks and slots handed out again in another order."""
    spec = small_spec()
    model, eng, w = build(spec, dtype, num_blocks=40, max_seqs=3)
    for gen in range(5):
        lens = [(29, 6), (3, 2), (14, 9)]
        reqs = {f"g{gen}r{i}": tokens_for(spec, n + d, 100 * gen + i) for i, (n, d) in enumerate(lens)}
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
            Expected(spec, w, reqs[k], dtype).check(np.concatenate(got[k]), what=k)
    assert len(eng.blocks.free) == 40 and len(eng.states.free) == 3


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_steps_of_portions_and_decoding(gpu, dtype):
    """Steps that hold a fresh prompt, a later portion and a decoding token of different requests at once."""
    spec = small_spec()
    model, eng, w = build(spec, dtype)
    reqs = {k: tokens_for(spec, n, 30 + n) for k, n in (("a", 31), ("b", 26), ("c", 18))}
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
@pytest.mark.parametrize("size,bs", [(1, 1), (2, 4), (3, 3), (4, 4), (5, 16), (8, 8), (16, 16), (17, 16)])
def test_small_windows_and_chunks_on_page_sizes(gpu, dtype, size, bs):
    """Windows and chunks of 1 .. 17 positions at, inside and across page borders, as prompts, portions and decoded rows; a window or
    chunk of one more position is another model."""
    spec = small_spec(layers=[att_layer(mask=size), par_layer(mask=size), att_layer(weights_of=0, mask=size, mlp="dense")])
    model, eng, w = build(spec, dtype, block_size=bs, num_blocks=200 // bs + 4)
    toks = tokens_for(spec, 44, size)
    want = Expected(spec, w, toks, dtype)
    for i in (0, 1):
        other = dataclasses.replace(spec, layers=[dataclasses.replace(l, mask=l.mask + 1) if (j == 1) == (i == 1) else l for j, l in enumerate(spec.layers)])
        assert row_errs(oracle(other, w, toks)[0], want.logits).max() > 0.1
    for cuts in ([44], [1], [2], [size + 1, size], [30, 1]):
        want.check(feed(eng, "a", toks, cuts), what=cuts)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_layers_that_share_weights(gpu, dtype):
    """Layers of both kinds that run with another layer's weights (an earlier one's, a later one's, through a chain), each with a cache
    and a memory of its own: the same tokens fed token by token find every layer's own past."""
    layers = [att_layer(weights_of=2), par_layer(), att_layer(), par_layer(weights_of=1), par_layer(weights_of=3), att_layer(weights_of=0)]
    spec = small_spec(layers=layers)
    assert [spec.weights_layer(i) for i in range(6)] == [2, 1, 2, 1, 1, 2] and not any(k.startswith(("l0.", "l3.", "l4.", "l5.")) for k in spec.tensor_shapes())
    model, eng, w = build(spec, dtype)
    toks = tokens_for(spec, 45, 7)
    want = Expected(spec, w, toks, dtype)
    for cuts in ([45], [20, 1], [2]):
        want.check(feed(eng, "a", toks, cuts))
    model.close()
    from vllm_rust_amd._lib import VmxError
    from vllm_rust_amd.larolorn import LarolornForCausalLM
    for bad in ([att_layer(weights_of=0)], [att_layer(weights_of=1)], [att_layer(weights_of=1), att_layer(weights_of=0)]):
        with pytest.raises(ValueError):
            LarolornForCausalLM(small_spec(layers=bad), dtype=dtype)
    for bad in ([att_layer(), par_layer(weights_of=0)], [att_layer(), att_layer(weights_of=0, mask=8)], [par_layer(), par_layer(weights_of=0, decay=(0.5, 0.5, 0.5))],
                [att_layer(), att_layer(weights_of=0, mlp=None)], [par_layer(), par_layer(weights_of=0, limit=1.0)], [att_layer(kv_rank=600)], [par_layer(dim=300)],
                [par_layer(r_dim=257)], [par_layer(kv_heads=4)], [att_layer(rot=rot(8))]):
        with pytest.raises(VmxError):
            LarolornForCausalLM(small_spec(layers=bad), dtype=dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width", [2, 40, 256, 257, 1000, 1500, 2600, 4100])
def test_rows_of_every_width(gpu, dtype, width):
    """From two columns up to rows wider than the norm kernels keep in registers."""
    spec = small_spec(layers=[att_layer(heads=2), par_layer(heads=2), par_layer(weights_of=1, heads=2)], width=width, vocab=31)
    model, eng, w = build(spec, dtype, max_tokens=32, num_blocks=16)
    toks = tokens_for(spec, 9, width)
    want = Expected(spec, w, toks, dtype)
    lg, _, tr = eng.step([("a", toks, list(range(9)))], layer_trace=True)
    if width > 2:
        want.check_layer(-1, tr[-1].cpu().numpy())
        want.check(lg.cpu().numpy())
    else:                                           # rows of two numbers: the spread of a row may be almost nothing
        scale = np.abs(want.trace[-1]).max()
        assert np.abs(tr[-1].cpu().numpy() - want.trace[-1]).max() < (1e-3 if dtype == "float32" else 0.3) * scale
    model.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_large_eps_shows_the_scales_that_norms_hide(gpu, dtype):
    """With eps of the order of the squares, the half in front of the two branches, the memory's scale and the latents' reach the
    logits instead of cancelling in the norm that follows them."""
    spec = small_spec(norm_eps=0.5)
    model, eng, w = build(spec, dtype)
    toks = tokens_for(spec, 48, 3)
    want = Expected(spec, w, toks, dtype)
    for cuts in ([48], [20, 1]):
        want.check(feed(eng, "a", toks, cuts))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", ["any", "eights"])
def test_sharp_attention_over_300_tokens_and_long_decoding(gpu, dtype, sizes):
    """Queries scaled up so that single keys decide rows, windows and chunks of tens of keys, memories that forget slowly; 220 tokens
    as a prompt and 80 decoded one by one (past every window and chunk edge), in portions, and whole."""
    def sharpen(ck):
        for k in ck:
            if k in ("l0.mix.q",) or k.endswith("left.q.norm"):
                ck[k] = (ck[k].float() * 2.5).to(ck[k].dtype)
    slow = dict(decay=(1.0, float(np.float32(0.999)), float(np.float32(0.98))))
    if sizes == "any":
        layers = [att_layer(mask=37), par_layer(mask=43, **slow), att_layer(weights_of=0, mask=37), par_layer(mask=0, mlp=None)]
    else:    # multiples of 8: the matrix-core forms in bfloat16
        layers = [att_layer(heads=8, dim=24, rot_dim=8, vdim=8, kv_rank=64, rot=rot(8, 1e4), mask=72), par_layer(heads=8, kv_heads=2, dim=24, vdim=16, rot=rot(16, 1e4), mask=88,
                  r_dim=32, r_vdim=24, **slow), att_layer(heads=8, dim=24, rot_dim=8, vdim=8, kv_rank=64, rot=rot(8, 1e4), mask=72, weights_of=0),
                  par_layer(heads=4, kv_heads=4, dim=16, vdim=32, rot=rot(16, 1e4), mask=0, r_heads=2, r_dim=64, r_vdim=32, mlp=None)]
    spec = small_spec(layers=layers)
    model, eng, w = build(spec, dtype, tweak=sharpen, block_size=16, num_blocks=64, max_tokens=512)
    toks = tokens_for(spec, 300, 9)
    want = Expected(spec, w, toks, dtype)
    want.check(feed(eng, "a", toks, [220, 1]))
    want.check(feed(eng, "b", toks, [300]))
    want.check(feed(eng, "c", toks, [90, 41, 8]))


OTHER_SIZES = {
    "one layer of each": dict(layers=[att_layer, par_layer]),
    "reverse order": dict(layers=[par_layer, att_layer]),
    "only two-sided": dict(layers=[par_layer, lambda: par_layer(r_heads=1, r_dim=1, r_vdim=33)]),
    "only latent attention": dict(layers=[att_layer, lambda: att_layer(mask=3)]),
    "one head": dict(layers=[lambda: att_layer(heads=1), lambda: par_layer(heads=1, kv_heads=1, r_heads=1)]),
    "many heads": dict(layers=[lambda: att_layer(heads=20, dim=8, rot_dim=8, rot=rot(8), vdim=8, kv_rank=32), lambda: par_layer(heads=24, kv_heads=2, dim=8, vdim=8, r_heads=9, r_dim=8, r_vdim=8)]),
    "one head per key head": dict(layers=[lambda: par_layer(heads=5, kv_heads=5)]),
    "sizes of 8s": dict(layers=[lambda: att_layer(heads=4, dim=16, rot_dim=16, rot=rot(16, 1e4), vdim=24, kv_rank=48, ff=64, mask=20),
                                lambda: par_layer(heads=8, kv_heads=2, dim=32, vdim=24, rot=rot(32), mask=24, r_heads=2, r_dim=24, r_vdim=40, ff=48)], width=64),
    "odd sizes": dict(layers=[lambda: att_layer(heads=3, dim=7, rot_dim=2, rot=rot(2), vdim=3, kv_rank=9, ff=11), lambda: par_layer(heads=3, kv_heads=1, dim=5, vdim=3, rot=rot(4), r_heads=3, r_dim=5,
                                                                                                                                    r_vdim=3, ff=7)], width=33, vocab=101),
    "no unrotated part": dict(layers=[lambda: att_layer(dim=0, rot_dim=16, rot=rot(16))]),
    "no rotated part": dict(layers=[lambda: att_layer(rot_dim=0, rot=rot(0)), lambda: par_layer(rot=rot(0))]),
    "partly rotated": dict(layers=[lambda: att_layer(rot_dim=12, rot=rot(4)), lambda: par_layer(rot=rot(2))]),
    "all rotated": dict(layers=[lambda: par_layer(dim=12, rot=rot(12))]),
    "no masks": dict(layers=[lambda: att_layer(mask=0), lambda: par_layer(mask=0)]),
    "masks longer than the sequence": dict(layers=[lambda: att_layer(mask=500), lambda: par_layer(mask=500)]),
    "wide latents": dict(layers=[lambda: att_layer(kv_rank=264, rot_dim=64, rot=rot(64, 1e4)), lambda: att_layer(kv_rank=512, rot_dim=64, rot=rot(64))]),
    "key sizes 130 and 200": dict(layers=[lambda: par_layer(r_heads=2, r_dim=130, r_vdim=8), lambda: par_layer(r_heads=1, r_dim=200, r_vdim=150, dim=136, vdim=130, rot=rot(136))]),
    "value sizes at a tile's edge": dict(layers=[lambda: par_layer(r_vdim=15), lambda: par_layer(r_vdim=16), lambda: par_layer(r_vdim=33), lambda: par_layer(r_vdim=1, vdim=1)]),
    "read-out of a wide row": dict(layers=[lambda: par_layer(r_heads=6, r_vdim=50)]),
    "decays of 1 and of 0": dict(layers=[lambda: par_layer(decay=(1.0, 1.0, 1.0)), lambda: par_layer(decay=(0.0, 0.5, 1.0))]),
    "unit constants": dict(layers=[lambda: att_layer(scale=1.0, limit=1.0), lambda: par_layer(scale=1.0, limit=1.0)], residual_mult=1.0, logit_scale=1.0),
    "small multiplier, negative scale": dict(layers=[att_layer, par_layer], residual_mult=0.05, logit_scale=-2.0),
    "no feed-forward anywhere": dict(layers=[lambda: att_layer(mlp=None), lambda: par_layer(mlp=None), lambda: att_layer(mlp=None, weights_of=0)]),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(OTHER_SIZES))
def test_other_sizes(gpu, dtype, name):
    kw = dict(OTHER_SIZES[name])
    kw["layers"] = [f() for f in kw["layers"]]
    spec = small_spec(**kw)
    model, eng, w = build(spec, dtype)
    toks = tokens_for(spec, 37, 4)
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
        own = [j for j, l in enumerate(layers) if l.weights_of is None]
        if own and rng.random() < 0.3:
            j = int(pick(*own))
            layers.append(dataclasses.replace(layers[j], weights_of=j))
            continue
        mult8 = rng.random() < 0.5
        size = lambda lo, hi: 8 * int(rng.integers(1, 6)) if mult8 else int(rng.integers(lo, hi))   # noqa: E731
        ff = dict(mlp="dense", ff=size(5, 70), limit=float(pick(0.3, 1.0, 7.0))) if rng.random() < 0.8 else dict(mlp=None)
        common = dict(scale=float(rng.uniform(0.1, 0.5)), mask=int(pick(0, 1, 5, 16, 23, 48)), **ff)
        if rng.random() < 0.5:
            rd = 8 * int(rng.integers(0, 4)) if mult8 else 2 * int(rng.integers(0, 12))
            layers.append(att_layer(heads=int(rng.integers(1, 20)), dim=size(2, 40), vdim=size(3, 40), kv_rank=size(6, 70), rot_dim=rd,
                                    rot=rot(rd, float(pick(100.0, 1e4, 1e6))) if rd else rot(0), **common))
        else:
            G, D, RH = int(rng.integers(1, 5)), size(3, 60), int(rng.integers(1, 6))
            rd = 2 * int(rng.integers(0, D // 2 + 1))
            layers.append(par_layer(heads=G * int(rng.integers(1, 6)), kv_heads=G, dim=D, vdim=size(3, 60), rot=rot(rd, float(pick(100.0, 1e4, 1e6))) if rd else rot(0), r_heads=RH,
                                    r_dim=size(3, 60), r_vdim=size(3, 50), decay=tuple(float(np.float32(rng.uniform(0.3, 1.0))) for _ in range(RH)), **common))
    return small_spec(layers=layers, width=8 * int(rng.integers(2, 12)) if rng.random() < 0.5 else int(rng.integers(12, 90)), vocab=int(rng.integers(20, 300)),
                      norm_eps=float(pick(1e-6, 1e-5)), residual_mult=float(pick(0.2, 0.5, 1.0)), logit_scale=float(pick(0.1, 1.0, 3.0)))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(14))
def test_random_models(gpu, dtype, seed):
    """Models drawn at random (layer order, shared weights, head counts, sizes, rotations, masks, decays) on random page sizes: two
    unequal requests decoding together, a third fed in portions."""
    rng = np.random.default_rng(seed)
    spec = random_spec(rng)
    bs = int(rng.choice([1, 3, 4, 8, 16]))
    model, eng, w = build(spec, dtype, seed=seed, block_size=bs, num_blocks=600 // bs + 8)
    ta, tb, tc = tokens_for(spec, 75, seed), tokens_for(spec, 33, seed + 50), tokens_for(spec, 60, seed + 99)
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
    spec = small_spec()
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
    from tests import larolorn_oracle as orc
    from vllm_rust_amd.engine import SamplingParams
    spec = small_spec()
    model, eng, w = build(spec, "float32", num_blocks=30, max_seqs=3)
    prompts = [tokens_for(spec, n, 70 + n) for n in (9, 23, 4, 15, 2)]
    outs = eng.generate(prompts, SamplingParams(max_new_tokens=8), prefill_chunk=6)
    sure = 0
    for p, o in zip(prompts, outs):
        seq = list(p)
        for t in o:
            lg = orc.forward(spec.to_config(), w, seq)[0].numpy()
            top2 = np.sort(lg[-1])[-2:]
            if top2[1] - top2[0] > 1e-3:      # a tie within rounding says nothing
                assert int(np.argmax(lg[-1])) == t
                sure += 1
            seq.append(t)
    assert sure > 30 and len(eng.blocks.free) == 30 and len(eng.states.free) == 3
    outs = eng.generate(prompts[:3], SamplingParams(temperature=0.9, top_k=20, top_p=0.9, max_new_tokens=5, seed=3))
    assert all(len(o) == 5 and all(0 <= t < spec.vocab for t in o) for o in outs)


def _write_checkpoint(tmp_path, spec, seed=0):
    import torch
    from safetensors.torch import save_file
    from vllm_rust_amd.larolorn import synthetic_weights
    ck = synthetic_weights(spec, seed)
    d = tmp_path / "model"
    d.mkdir()
    (d / "config.json").write_text(json.dumps(spec.to_config()))
    extra = {f"l{i}.norm2": torch.ones(spec.width, dtype=torch.bfloat16) for i, l in enumerate(spec.layers) if l.mlp is None}   # skipped
    save_file({k: v.contiguous() for k, v in {**ck, **extra}.items()}, str(d / "model.safetensors"))
    return d, {k: v.double() for k, v in ck.items()}


def test_registry_and_command_line_tools(gpu, tmp_path):
    """A checkpoint directory written here: the registry picks the class from config.json; bin/trace_run replays a trace (a prompt,
    a portion, decode steps of two requests, an early finisher) in both modes; bin/generate continues greedily."""
    from vllm_rust_amd.engine import Engine
    from vllm_rust_amd.models import architecture_of, load_model
    spec = small_spec()
    d, w = _write_checkpoint(tmp_path, spec)
    assert architecture_of(d) == "Larolorn"
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
