"""Plain, slow float64 restatement of the Larolorn design, one function per mechanism, for the tests only.

Nothing here is shared with the product path: it reads the configuration dictionary itself, recomputes whole sequences from
their first token (no cache, no carried state, no absorbed projections: every head's keys and values are formed) and loops over
heads and tokens.  Weights are dicts of float64 torch tensors under the checkpoint's names.

The sublayers read the stream as it is and only their results are normed: x <- x + m N1(mixer(x)), x <- x + m N2(ff(x)).  Mixers:
"latent_attention" (keys and values through one low-rank latent, one rotated key part for all heads, a sliding window, a sigmoid per
head on the output) and "parallel" (grouped-query attention inside chunks of positions, with a sink, beside a decayed matrix memory;
half the sum of the two normed results).  Feed-forward: a clamped gate, y = g sigmoid(1.702 g) (u + 1).  A layer may run with the
weights of an earlier one.
"""
import contextlib
import math

import torch

F = torch.float64
_rounding = None        # None, or a function that rounds what enters a product


@contextlib.contextmanager
def rounded_operands(fn=lambda t: t.to(torch.bfloat16).to(F)):
    """Inside, the activations that enter every linear map and what the caches keep go through `fn` first: how far rounding alone
    moves a model's results."""
    global _rounding
    _rounding = fn
    try:
        yield
    finally:
        _rounding = None


def rnd(t):
    return _rounding(t) if _rounding else t


def lin(h, w):
    return rnd(h) @ w.T


# ------------------------------------------------------------------------------------------------ small pieces
def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return rms_unit(x, eps) * w


def silu(z):
    return z * torch.sigmoid(z)


# ------------------------------------------------------------------------------------------------ rotation
def turn(u, v, positions, step):
    """The pair (u, v) [T, heads] turned by positions * step."""
    a = (torch.as_tensor(positions, dtype=F) * step).unsqueeze(-1)
    return u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a)


def rotate_neighbours(x, positions, rot):
    """x [T, heads, d]: coordinate 2i turns with 2i + 1, coordinates from dims on pass."""
    y = x.clone()
    dims = rot["dims"] if rot else 0
    for i in range(dims // 2):
        y[:, :, 2 * i], y[:, :, 2 * i + 1] = turn(x[:, :, 2 * i], x[:, :, 2 * i + 1], positions, rot["base"] ** (-2.0 * i / dims))
    return y


def rotate_halves(x, positions, rot):
    """x [T, heads, d]: coordinate i turns with i + dims / 2, coordinates from dims on pass."""
    y = x.clone()
    dims = rot["dims"] if rot else 0
    half = dims // 2
    for i in range(half):
        y[:, :, i], y[:, :, i + half] = turn(x[:, :, i], x[:, :, i + half], positions, rot["base"] ** (-2.0 * i / dims))
    return y


# ------------------------------------------------------------------------------------------------ attention
def window_start(i, size):
    """First position that position i sees through a sliding window (size 0: none)."""
    return max(0, i - size + 1) if size else 0


def chunk_start(i, size):
    """First position of the chunk that position i lies in, chunks counted from position 0 (size 0: one chunk)."""
    return i // size * size if size else 0


def softmax_attention(q, k, v, scale, start, sink=None):
    """q [T, H, D], k [T, H, D], v [T, H, V]: row i sees keys start(i) .. i; the denominator also holds exp(sink[h])."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=F)
    for h in range(H):
        for i in range(T):
            lo = start(i)
            s = (k[lo:i + 1, h] @ q[i, h]) * scale
            m = s.max() if sink is None else torch.maximum(s.max(), sink[h])
            e = torch.exp(s - m)
            den = e.sum() if sink is None else e.sum() + torch.exp(sink[h] - m)
            out[i, h] = (e / den) @ v[lo:i + 1, h]
    return out


def latent_attention(h, w, pre, m, eps):
    T = h.shape[0]
    H, D, RD, V, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = lin(h, w[pre + "q"]).reshape(T, H, D + RD)
    q = torch.cat([rnd(q[:, :, :D]), rotate_neighbours(q[:, :, D:], range(T), m.get("rot"))], -1)
    y = lin(h, w[pre + "dkv"])
    c = rnd(rms_norm(y[:, :R], w[pre + "dkv.norm"], eps))
    k_rot = rnd(rotate_neighbours(y[:, R:].unsqueeze(1), range(T), m.get("rot")))
    k = torch.cat([(c @ w[pre + "uk"].T).reshape(T, H, D), k_rot.expand(T, H, RD)], -1)
    v = (c @ w[pre + "uv"].T).reshape(T, H, V)
    size = (m.get("mask") or {}).get("size") or 0
    o = softmax_attention(q, k, v, m["scale"], lambda i: window_start(i, size))
    o = o * torch.sigmoid(lin(h, w[pre + "g"])).unsqueeze(-1)
    return lin(o.reshape(T, H * V), w[pre + "o"])


def chunked_attention(h, w, pre, m, eps):
    T = h.shape[0]
    H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(lin(h, w[pre + "q"]) + w[pre + "q.b"], w[pre + "q.norm"], eps).reshape(T, H, D)
    k = rms_norm(lin(h, w[pre + "k"]) + w[pre + "k.b"], w[pre + "k.norm"], eps).reshape(T, G, D)
    v = rnd((lin(h, w[pre + "v"]) + w[pre + "v.b"]).reshape(T, G, V))
    q, k = rnd(rotate_halves(q, range(T), m.get("rot"))), rnd(rotate_halves(k, range(T), m.get("rot")))
    owner = [i // (H // G) for i in range(H)]
    size = (m.get("mask") or {}).get("size") or 0
    o = softmax_attention(q, k[:, owner], v[:, owner], m["scale"], lambda i: chunk_start(i, size), w[pre + "sink"])
    return lin(o.reshape(T, H * V), w[pre + "o"]) + w[pre + "o.b"]


# ------------------------------------------------------------------------------------------------ decayed matrix memory
def decayed_memory(q, k, v, decay):
    """q, k [T, H, D], v [T, H, V]: per head, from zero, S <- decay S + k v^T; o = S^T q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F)
    g = torch.as_tensor(decay, dtype=F).reshape(H, 1, 1)
    out = []
    for t in range(T):
        S = g * S + k[t].unsqueeze(-1) * v[t].unsqueeze(-2)
        out.append((S * q[t].unsqueeze(-1)).sum(1))
    return torch.stack(out)


def lightning_attention(h, w, pre, m, eps):
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q, k = rnd(silu(lin(h, w[pre + "q"]))).reshape(T, H, D), rnd(silu(lin(h, w[pre + "k"]))).reshape(T, H, D)
    v = rnd(silu(lin(h, w[pre + "v"]))).reshape(T, H, V)
    o = decayed_memory(q, k, v, m["decay"]).reshape(T, H * V)
    return lin(rms_norm(o, w[pre + "norm"], eps) * torch.sigmoid(lin(h, w[pre + "g"])), w[pre + "o"])


def parallel(h, w, pre, m, eps):
    a = chunked_attention(h, w, pre + "left.", m["left"], eps)
    b = lightning_attention(h, w, pre + "right.", m["right"], eps)
    return 0.5 * (rms_norm(a, w[pre + "left.out"], eps) + rms_norm(b, w[pre + "right.out"], eps))


# ------------------------------------------------------------------------------------------------ feed-forward
def clamped_glu(g, u, limit):
    g, u = torch.clamp(g, max=limit), torch.clamp(u, min=-limit, max=limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def dense(h, w, pre, ff):
    return lin(clamped_glu(lin(h, w[pre + "gate"]), lin(h, w[pre + "up"]), ff["limit"]), w[pre + "down"])


# ------------------------------------------------------------------------------------------------ the model
def forward(cfg, w, tokens):
    """tokens: list of ids of ONE sequence.  Returns (logits [T, vocab], residual stream after every layer [layers, T, width])."""
    w = {k: v.to(F) for k, v in w.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    trace = []
    for i, e in enumerate(cfg["layers"]):
        j = i
        while cfg["layers"][j].get("weights_of") is not None:
            j = cfg["layers"][j]["weights_of"]
        pre = f"l{j}."
        mixer = latent_attention if e["type"] == "latent_attention" else parallel
        x = x + mult * rms_norm(mixer(x, w, pre + "mix.", e["mixer"], eps), w[pre + "norm1"], eps)
        if e.get("mlp"):
            x = x + mult * rms_norm(dense(x, w, pre + "mlp.", e["mlp"]), w[pre + "norm2"], eps)
        trace.append(x)
    return lin(rms_norm(x, w["final.norm"], eps), w["head"]) * cfg["logit_scale"], torch.stack(trace)
