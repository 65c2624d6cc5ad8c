"""Plain, slow float64 restatement of the Fofinex design, one function per mechanism, for the tests only.

Nothing here is shared with the product path: it reads the configuration dictionary itself, recomputes whole sequences from
their first token (no cache, no carried state, no absorbed projections: every head's keys and values are formed) and loops over
heads and tokens.  Weights are dicts of float64 torch tensors under the checkpoint's names.

A sublayer sits between two norms, x <- x + N_b(f(N_a(x))), with N a centred norm (layer norm with a gain, no bias); the embedding
is normed once more.  Mixers: "latent_attention" (queries and keys / values through low-rank latents, one rotated key part for all
heads with stretched rotation frequencies, a layer may read another layer's latents) and "mlstm" (matrix memory with exponential
input gate, forget gate, normaliser and running maximum).  Feed-forwards: biased tanh-GELU GLU; sigmoid-routed squared-ReLU experts
chosen by corrected scores inside the best groups, plus a gated shared expert.
"""
import contextlib
import math

import torch

F = torch.float64
_rounding = None        # None, or a function that rounds what enters a product


@contextlib.contextmanager
def rounded_operands(fn=lambda t: t.to(torch.bfloat16).to(F)):
    """Inside, the activations that enter every linear map and what the latent cache keeps go through `fn` first: how far rounding
    alone moves a model's results."""
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
def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def relu_squared(z):
    return torch.clamp(z, min=0.0) ** 2


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


# ------------------------------------------------------------------------------------------------ rotation
def rotation_steps(rot):
    """(angle step per coordinate pair, multiplier of cos and sin) of {base, dims[, scaling {factor, original, fast, slow}]}."""
    dims, base = rot["dims"], rot["base"]
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return plain, 1.0

    def index_of(turns):                # the pair that turns this often over the original length
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    first, last = max(math.floor(index_of(sc["fast"])), 0), min(math.ceil(index_of(sc["slow"])), dims - 1)
    steps = []
    for i, f in enumerate(plain):
        slow_share = min(max((i - first) / max(last - first, 0.001), 0.0), 1.0)
        steps.append(f / sc["factor"] * slow_share + f * (1.0 - slow_share))
    return steps, 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, positions, rot):
    """x [T, heads, d], one position per row: coordinate i turns with i + dims / 2, coordinates from dims on pass."""
    if not rot or not rot.get("dims"):
        return x.clone()
    steps, mul = rotation_steps(rot)
    half = rot["dims"] // 2
    y = x.clone()
    p = torch.as_tensor(positions, dtype=F)
    for i in range(half):
        c, s = (torch.cos(p * steps[i]) * mul).unsqueeze(-1), (torch.sin(p * steps[i]) * mul).unsqueeze(-1)
        u, v = x[:, :, i], x[:, :, i + half]
        y[:, :, i] = u * c - v * s
        y[:, :, i + half] = v * c + u * s
    return y


# ------------------------------------------------------------------------------------------------ latent attention
def causal_softmax_attention(q, k, v, scale):
    """q, k [T, H, D], v [T, H, V]: row i sees keys j <= i."""
    T, H, _ = q.shape
    out = torch.zeros(T, H, v.shape[2], dtype=F)
    for h in range(H):
        for i in range(T):
            p = torch.softmax((k[:i + 1, h] @ q[i, h]) * scale, 0)
            out[i, h] = p @ v[:i + 1, h]
    return out


def latents(h, w, pre, m, eps):
    """What a layer keeps per token: (normed latent [T, R], rotated key part [T, rot_dim])."""
    T, R = h.shape[0], m["kv_rank"]
    y = lin(h, w[pre + "dkv"])
    c = rms_unit(y[:, :R], eps) * w[pre + "dkv.norm"]
    return rnd(c), rnd(rotate(y[:, R:].unsqueeze(1), range(T), m.get("rot")).squeeze(1))


def latent_attention(h, w, pre, m, eps, kept):
    """kept: the (latent, rotated key part) this layer attends over, its own or another layer's."""
    T = h.shape[0]
    H, D, RD, V = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c_q = rms_unit(lin(h, w[pre + "dq"]), eps) * w[pre + "dq.norm"]
    q = lin(c_q, w[pre + "uq"]).reshape(T, H, D + RD)
    q = torch.cat([rnd(q[:, :, :D]), rotate(q[:, :, D:], range(T), m.get("rot"))], -1)
    c, k_rot = kept
    k = torch.cat([(c @ w[pre + "uk"].T).reshape(T, H, D), k_rot.unsqueeze(1).expand(T, H, RD)], -1)
    v = (c @ w[pre + "uv"].T).reshape(T, H, V)
    return lin(causal_softmax_attention(q, k, v, m["scale"]).reshape(T, H * V), w[pre + "o"])


# ------------------------------------------------------------------------------------------------ matrix memory with exponential gates
def exponential_gate_memory(q, k, v, log_i, log_f, parts=None):
    """q, k [T, H, D], v [T, H, V], log_i, log_f [T, H].  Per head, from zero memory, zero normaliser and maximum 0:
    m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T;  n <- e^(f + m - m') n + e^(i - m') k;
    o = S^T q / (max(|n . q|, e^(-m')) + 1e-6).  parts (a list): receives (S^T q, n . q, e^(-m'), sum |n_i q_i|) per token."""
    T, H, D = q.shape
    S, n, m = torch.zeros(H, D, v.shape[2], dtype=F), torch.zeros(H, D, dtype=F), torch.zeros(H, dtype=F)
    out = []
    for t in range(T):
        m_new = torch.maximum(log_f[t] + m, log_i[t])
        keep, add = torch.exp(log_f[t] + m - m_new), torch.exp(log_i[t] - m_new)
        S = keep.reshape(H, 1, 1) * S + add.reshape(H, 1, 1) * k[t].unsqueeze(-1) * v[t].unsqueeze(-2)
        n = keep.reshape(H, 1) * n + add.reshape(H, 1) * k[t]
        m = m_new
        top, nq = torch.einsum("hdv,hd->hv", S, q[t]), (n * q[t]).sum(-1)
        out.append(top / (torch.maximum(nq.abs(), torch.exp(-m)) + 1e-6).unsqueeze(-1))
        if parts is not None:
            parts.append((top, nq, torch.exp(-m), (n * q[t]).abs().sum(-1)))
    return torch.stack(out)


def log_gates(zi, zf, cap):
    return cap * torch.tanh(zi / cap), torch.nn.functional.logsigmoid(cap * torch.tanh(zf / cap))


def mlstm(h, w, pre, m, eps):
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = (lin(h, w[pre + "q"])).reshape(T, H, D) * D ** -0.5
    k = (lin(h, w[pre + "k"])).reshape(T, H, D)
    v = (lin(h, w[pre + "v"])).reshape(T, H, V)
    li, lf = log_gates(lin(h, w[pre + "i"]) + w[pre + "i.b"], lin(h, w[pre + "f"]) + w[pre + "f.b"], m["gate_cap"])
    o = rms_unit(exponential_gate_memory(q, k, v, li, lf), eps).reshape(T, H * V)
    return lin(o * w[pre + "norm"] * torch.sigmoid(lin(h, w[pre + "g"])), w[pre + "o"])


# ------------------------------------------------------------------------------------------------ feed-forward
def dense_glu(h, w, pre):
    g = gelu_tanh(lin(h, w[pre + "gate"]) + w[pre + "gate.b"])
    return lin(g * (lin(h, w[pre + "up"]) + w[pre + "up.b"]), w[pre + "down"]) + w[pre + "down.b"]


def expert(h, w, pre):
    return lin(relu_squared(lin(h, w[pre + "up"])), w[pre + "down"])


def choice_scores(z, correction, groups, keep):
    """Corrected sigmoid scores; experts outside the `keep` best groups (by the sum of a group's two best) are minus infinity."""
    c = torch.sigmoid(z) + correction
    T, E = c.shape
    if groups > 1:
        per = c.reshape(T, groups, E // groups)
        rank = torch.topk(per, min(2, E // groups), dim=-1).values.sum(-1)
        best = torch.sort(rank, dim=-1, descending=True, stable=True).indices[:, :keep]
        c = torch.full_like(per, -math.inf).scatter(1, best.unsqueeze(-1).expand(-1, -1, E // groups),
                                                     torch.gather(per, 1, best.unsqueeze(-1).expand(-1, -1, E // groups))).reshape(T, E)
    return c


def route(z, correction, top, groups, keep, scale):
    """(expert ids [T, top], weights): the largest choice scores win (ties to the smaller index); the weights are the plain
    scores times `scale`, not renormalised."""
    ids = torch.sort(choice_scores(z, correction, groups, keep), dim=-1, descending=True, stable=True).indices[:, :top]
    return ids, torch.gather(torch.sigmoid(z), 1, ids) * scale


def router_margin(z, correction, top, groups, keep):
    """Smallest gap of any decision the router takes on these rows (kept against dropped group, chosen against rejected expert):
    a gap near zero means that rounding may legitimately pick another expert."""
    out = math.inf
    c = torch.sigmoid(z) + correction
    T, E = c.shape
    if groups > 1 and keep < groups:
        rank = torch.sort(torch.topk(c.reshape(T, groups, E // groups), min(2, E // groups), dim=-1).values.sum(-1), -1, descending=True).values
        out = min(out, float((rank[:, keep - 1] - rank[:, keep]).min()))
    c = torch.sort(choice_scores(z, correction, groups, keep), -1, descending=True).values
    if top < E:
        out = min(out, float((c[:, top - 1] - c[:, top]).min()))
    return out


def mixture(h, w, pre, ff, margins=None):
    r = ff["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    z = lin(h, w[pre + "router"])
    ids, weight = route(z, w[pre + "correction"], r["top"], g["count"], g["keep"], r.get("scale", 1.0))
    if margins is not None:
        margins.append(router_margin(z, w[pre + "correction"], r["top"], g["count"], g["keep"]))
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(ids[t].tolist(), weight[t]):
            out[t] += s * expert(h[t:t + 1], w, f"{pre}e{e}.")[0]
    if ff.get("shared"):
        out = out + expert(h, w, pre + "shared.") * torch.sigmoid(lin(h, w[pre + "shared.sg"]))
    return out


def feed_forward(h, w, pre, ff, margins=None):
    return dense_glu(h, w, pre) if ff["kind"] == "dense" else mixture(h, w, pre, ff, margins)


# ------------------------------------------------------------------------------------------------ the model
def forward(cfg, w, tokens, margins=None):
    """tokens: list of ids of ONE sequence.  Returns (logits [T, vocab], residual stream after every layer [layers, T, width]).
    margins (a list): receives every routed layer's smallest router margin."""
    w = {k: v.to(F) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = layer_norm(w["embed"][torch.as_tensor(tokens, dtype=torch.long)], w["embed.norm"], eps)
    trace, kept = [], {}
    for i, e in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", e["mixer"]
        h = layer_norm(x, w[pre + "norm1"], eps)
        if e["type"] == "latent_attention":
            src = m.get("kv_from")
            if src is None:
                kept[i] = latents(h, w, pre + "mix.", m, eps)
            y = latent_attention(h, w, pre + "mix.", m, eps, kept[i if src is None else src])
        else:
            y = mlstm(h, w, pre + "mix.", m, eps)
        x = x + layer_norm(y, w[pre + "norm1b"], eps)
        if e.get("mlp"):
            y = feed_forward(layer_norm(x, w[pre + "norm2"], eps), w, pre + "mlp.", e["mlp"], margins)
            x = x + layer_norm(y, w[pre + "norm2b"], eps)
        trace.append(x)
    return lin(layer_norm(x, w["final.norm"], eps), w["embed"]), torch.stack(trace)
