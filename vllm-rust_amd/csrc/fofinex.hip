// Whole-step executor of the Fofinex decoder family: layers listed in the model's configuration whose sublayers sit between two
// layer norms,
//   x = N(embed[token]);   x <- x + N1b(mixer(N1(x)));   x <- x + N2b(ff(N2(x)));   logits = embed . N(x)
// with N a layer norm with a gain and no bias, and the embedding table as the output matrix.  Mixers (every size per layer):
//   VMX_MIXER_LATENT_ATTENTION  compressed keys / values in a paged cache (latent_attn.hip), queries through a normed latent of
//                               their own, rotation in halves with stretched steps; a layer may attend over an earlier layer's
//                               cache with its own up-projections and queries
//   VMX_MIXER_EXP_MEMORY        matrix memory with an exponential input gate and a forget gate (delta_rule.hip): a running maximum,
//                               the memory and its normaliser live in the sequence's state slot; the read-out is divided by the
//                               normaliser, RMS-normed per head and gated
// Feed-forwards: VMX_MLP_DENSE_GLU (biased tanh-GELU gate) and VMX_MLP_CORRECTED_MOE (sigmoid scores, choice by corrected scores
// inside the best groups, squared-ReLU experts run as token-grouped products, a shared expert times a sigmoid per token).
//
// Everything that reads a mixer's input is ONE product whose f32 row the other kernels address by column offset; the shared
// expert's gate is one more row of the router's exact product.  One kernel carries a sublayer's result through both norms into
// the next product's input (sandwich_norm_kernel); for a mixture it also forms the experts' weighted sum.  The stream, norms,
// router, positions and angles, scores, softmax, gates of the memory and its state are f32 in both modes; VMX_BF16 rounds the
// operands of the linears and the cache rows to bf16, VMX_F32 multiplies in true f32 everywhere.  The forward call allocates
// nothing, reads nothing back and is graph-capturable.
#include "executor_common.h"
#include <math.h>

namespace {

using Buf = VmxBuf;

struct Layer : VmxTensorTable {
    vmx_fofinex_layer_config c;
    Buf norm1, norm1b, norm2, norm2b, wfused, bias, wo;
    Buf dq_norm, wuq, dkv_norm, uk, uk_t, uv, rot_steps, cache;        // latent attention
    Buf head_norm, memory, maxima;                                      // matrix memory
    Buf wgu, bias_gu, wdown, bias_down;                                 // dense feed-forward
    Buf router, correction, eup, edown, sup, sdown;                     // mixture of experts
    float rot_mul = 1.f;
    int nf = 0, dq_off = 0, dkv_off = 0, q_off = 0, k_off = 0, v_off = 0, g_off = 0, i_off = 0, f_off = 0;
    int router_rows = 0;   // experts (+ 1: the shared expert's gate)
};

}  // namespace

struct vmx_fofinex {
    vmx_fofinex_config cfg;
    std::vector<Layer> layers;
    VmxTensorTable top;
    VmxExpertBlocks blocks;
    Buf embed, embed_norm, final_norm;
    Buf x, h, hsel, y, fused, cq, q, qabs, qrot, olat, attn, attn_ws, norm, floor, readout, rec, argmax_keys;
    Buf gu, dact, rlogits, act, ydown, sact, sout;
    bool f32() const { return cfg.dtype == VMX_F32; }
    size_t esz() const { return f32() ? 4 : 2; }
};

extern "C" int vmx_fofinex_create(const vmx_fofinex_config *cfg, const vmx_fofinex_layer_config *layer_cfgs, vmx_fofinex **out) {
    VMX_REQUIRE(cfg && layer_cfgs && out, "fofinex_create: null pointer");
    const vmx_fofinex_config &c = *cfg;
    VMX_REQUIRE(c.vocab >= 1 && c.width >= 1 && c.num_layers >= 1, "fofinex_create: bad sizes (vocab %d, width %d, layers %d)", c.vocab, c.width,
                c.num_layers);
    VMX_REQUIRE(c.dtype == VMX_F32 || c.dtype == VMX_BF16, "fofinex_create: dtype must be VMX_F32 or VMX_BF16");
    VMX_REQUIRE(c.block_size >= 1 && c.num_blocks >= 1 && c.max_tokens >= 1 && c.max_seqs >= 1 && c.state_slots >= 1,
                "fofinex_create: bad cache / batch geometry");
    vmx_fofinex *m = new vmx_fofinex();
    m->cfg = c;
    m->layers.resize(c.num_layers);
    const size_t T = c.max_tokens, W = c.width, rows = (size_t)c.num_blocks * c.block_size;
    size_t nf = 8, qr = 1, nq = 1, hr = 1, hrd = 1, hv = 1, maxr = 1, mh = 1, mhv = 1, gu = 1, dff = 1, ne = 1, eff = 1, sff = 1;
    int rc = VMX_OK;
#define GA(buf, n)                            \
    do {                                      \
        if (!rc) rc = vmx_alloc_zero(buf, n); \
    } while (0)
#define BAD(...)                    \
    {                               \
        vmx_set_error(__VA_ARGS__); \
        rc = VMX_EINVAL;            \
        break;                      \
    }
    for (int li = 0; li < c.num_layers && !rc; li++) {
        Layer &L = m->layers[li];
        const vmx_fofinex_layer_config &lc = L.c = layer_cfgs[li];
        if (lc.heads < 1 || lc.dim < 0 || lc.vdim < 1) BAD("fofinex_create: layer %d: bad head count or sizes (heads %d, dim %d, vdim %d)", li, lc.heads, lc.dim, lc.vdim);
        const size_t H = lc.heads, D = lc.dim, V = lc.vdim;
        int at = 0;
        auto seg = [&](size_t n) {
            const int o = at;
            at = vmx_pad8(at + (int)n);
            return o;
        };
        auto norm_pair = [&](const char *a, Buf &ba, const char *b, Buf &bb) {
            L.want(a, &ba, 0, W * 2);
            L.want(b, &bb, 0, W * 2);
            GA(ba, W * 2);
            GA(bb, W * 2);
        };
        norm_pair("norm1", L.norm1, "norm1b", L.norm1b);
        if (lc.mixer == VMX_MIXER_LATENT_ATTENTION) {
            if (lc.rot_dim < 0 || lc.dim + lc.rot_dim < 1 || lc.kv_rank < 1 || lc.kv_rank > 512 || lc.q_rank < 1)
                BAD("fofinex_create: layer %d: bad latent-attention sizes (dim %d, rot_dim %d, kv_rank %d, q_rank %d; kv_rank up to 512)", li, lc.dim,
                    lc.rot_dim, lc.kv_rank, lc.q_rank);
            if (!vmx_rotation_ok(lc.rot, lc.rot_dim)) BAD("fofinex_create: layer %d: bad rotation (%d of %d coordinates)", li, lc.rot.dims, lc.rot_dim);
            const size_t R = lc.kv_rank, RD = lc.rot_dim, Q = lc.q_rank, NQ = H * (D + RD);
            const bool own = lc.kv_from < 0;
            if (!own) {
                if (lc.kv_from >= li || m->layers[lc.kv_from].c.mixer != VMX_MIXER_LATENT_ATTENTION || m->layers[lc.kv_from].c.kv_from >= 0)
                    BAD("fofinex_create: layer %d: layer %d keeps no latents that it could use", li, lc.kv_from);
                const vmx_fofinex_layer_config &sc = m->layers[lc.kv_from].c;
                if (sc.kv_rank != lc.kv_rank || sc.rot_dim != lc.rot_dim)
                    BAD("fofinex_create: layer %d: latents of layer %d have other sizes (%d + %d, not %d + %d)", li, lc.kv_from, sc.kv_rank, sc.rot_dim, lc.kv_rank,
                        lc.rot_dim);
            }
            L.dq_off = seg(Q);
            if (own) L.dkv_off = seg(R + RD);
            L.nf = at;
            GA(L.wfused, (size_t)L.nf * W * 2);
            GA(L.dq_norm, Q * 2);
            GA(L.wuq, NQ * Q * 2);
            GA(L.uk, H * D * R * 2);
            GA(L.uk_t, H * D * R * 2);
            GA(L.uv, H * V * R * 2);
            GA(L.wo, W * H * V * 2);
            L.want("mix.dq", &L.wfused, (size_t)L.dq_off * W * 2, Q * W * 2);
            L.want("mix.dq.norm", &L.dq_norm, 0, Q * 2);
            L.want("mix.uq", &L.wuq, 0, NQ * Q * 2);
            if (own) {
                GA(L.dkv_norm, R * 2);
                GA(L.cache, rows * (R + RD) * m->esz());
                L.want("mix.dkv", &L.wfused, (size_t)L.dkv_off * W * 2, (R + RD) * W * 2);
                L.want("mix.dkv.norm", &L.dkv_norm, 0, R * 2);
            }
            L.want("mix.uk", &L.uk, 0, H * D * R * 2);
            L.want("mix.uv", &L.uv, 0, H * V * R * 2);
            L.want("mix.o", &L.wo, 0, W * H * V * 2);
            if (!rc) rc = vmx_upload_rotation(lc.rot, L.rot_steps, L.rot_mul);
            qr = std::max(qr, Q);
            nq = std::max(nq, NQ);
            hr = std::max(hr, H * R);
            hrd = std::max(hrd, H * RD);
            hv = std::max(hv, H * V);
            maxr = std::max(maxr, R);
        } else if (lc.mixer == VMX_MIXER_EXP_MEMORY) {
            if (lc.dim < 1 || lc.dim > 256 || !(lc.gate_cap > 0.f))
                BAD("fofinex_create: layer %d: bad matrix memory (key size %d outside 1..256, gate cap %g)", li, lc.dim, lc.gate_cap);
            L.q_off = seg(H * D);
            L.k_off = seg(H * D);
            L.v_off = seg(H * V);
            L.g_off = seg(H * V);
            L.i_off = seg(H);
            L.f_off = seg(H);
            L.nf = at;
            GA(L.wfused, (size_t)L.nf * W * 2);
            GA(L.bias, (size_t)L.nf * 2);
            GA(L.head_norm, H * V * 2);
            GA(L.wo, W * H * V * 2);
            GA(L.memory, vmx_gated_delta_rule_state_bytes(c.state_slots, lc.heads, lc.dim, lc.vdim + 1));   // + 1: the normaliser's column
            GA(L.maxima, (size_t)c.state_slots * H * 4);
            L.want("mix.q", &L.wfused, (size_t)L.q_off * W * 2, H * D * W * 2);
            L.want("mix.k", &L.wfused, (size_t)L.k_off * W * 2, H * D * W * 2);
            L.want("mix.v", &L.wfused, (size_t)L.v_off * W * 2, H * V * W * 2);
            L.want("mix.g", &L.wfused, (size_t)L.g_off * W * 2, H * V * W * 2);
            L.want("mix.i", &L.wfused, (size_t)L.i_off * W * 2, H * W * 2);
            L.want("mix.i.b", &L.bias, (size_t)L.i_off * 2, H * 2);
            L.want("mix.f", &L.wfused, (size_t)L.f_off * W * 2, H * W * 2);
            L.want("mix.f.b", &L.bias, (size_t)L.f_off * 2, H * 2);
            L.want("mix.norm", &L.head_norm, 0, H * V * 2);
            L.want("mix.o", &L.wo, 0, W * H * V * 2);
            mh = std::max(mh, H);
            mhv = std::max(mhv, H * V);
        } else {
            vmx_set_error("fofinex_create: layer %d: unknown mixer kind %d", li, lc.mixer);
            rc = VMX_EUNSUPPORTED;
            break;
        }
        nf = std::max(nf, (size_t)L.nf);
        if (lc.mlp == VMX_MLP_NONE) continue;
        norm_pair("norm2", L.norm2, "norm2b", L.norm2b);
        if (lc.mlp == VMX_MLP_DENSE_GLU) {
            if (lc.ff < 1) BAD("fofinex_create: layer %d: bad feed-forward width %d", li, lc.ff);
            const size_t F = lc.ff;
            GA(L.wgu, 2 * F * W * 2);   // gate rows, then up rows
            GA(L.bias_gu, 2 * F * 2);
            GA(L.wdown, W * F * 2);
            GA(L.bias_down, W * 2);
            L.want("mlp.gate", &L.wgu, 0, F * W * 2);
            L.want("mlp.gate.b", &L.bias_gu, 0, F * 2);
            L.want("mlp.up", &L.wgu, F * W * 2, F * W * 2);
            L.want("mlp.up.b", &L.bias_gu, F * 2, F * 2);
            L.want("mlp.down", &L.wdown, 0, W * F * 2);
            L.want("mlp.down.b", &L.bias_down, 0, W * 2);
            gu = std::max(gu, 2 * F);
            dff = std::max(dff, F);
        } else if (lc.mlp == VMX_MLP_CORRECTED_MOE) {
            if (lc.experts < 1 || lc.experts > 256 || lc.groups < 1 || lc.experts % lc.groups || lc.keep_groups < 1 || lc.keep_groups > lc.groups || lc.top < 1 ||
                lc.top > lc.keep_groups * (lc.experts / lc.groups) || lc.expert_ff < 1 || lc.shared_ff < 0)
                BAD("fofinex_create: layer %d: bad mixture-of-experts sizes (%d experts in %d groups, %d kept, top %d)", li, lc.experts, lc.groups,
                    lc.keep_groups, lc.top);
            const size_t E = lc.experts, one = (size_t)lc.expert_ff * W * 2, S = lc.shared_ff;
            L.router_rows = (int)E + (S ? 1 : 0);
            GA(L.router, (size_t)L.router_rows * W * 2);
            GA(L.correction, E * 2);
            GA(L.eup, E * one);
            GA(L.edown, E * one);
            L.want("mlp.router", &L.router, 0, E * W * 2);
            L.want("mlp.correction", &L.correction, 0, E * 2);
            for (int e = 0; e < lc.experts; e++) {
                const std::string p = "mlp.e" + std::to_string(e) + ".";
                L.want(p + "up", &L.eup, (size_t)e * one, one);
                L.want(p + "down", &L.edown, (size_t)e * one, one);
            }
            if (S) {
                GA(L.sup, S * W * 2);
                GA(L.sdown, S * W * 2);
                L.want("mlp.shared.up", &L.sup, 0, S * W * 2);
                L.want("mlp.shared.down", &L.sdown, 0, S * W * 2);
                L.want("mlp.shared.sg", &L.router, E * W * 2, W * 2);
            }
            m->blocks.reserve(T, lc.experts, lc.top);
            ne = std::max(ne, (size_t)L.router_rows);
            eff = std::max(eff, (size_t)lc.expert_ff);
            sff = std::max(sff, S);
        } else {
            vmx_set_error("fofinex_create: layer %d: unknown feed-forward kind %d", li, lc.mlp);
            rc = VMX_EUNSUPPORTED;
            break;
        }
    }
#undef BAD
    GA(m->embed, (size_t)c.vocab * W * 2);
    GA(m->embed_norm, W * 2);
    GA(m->final_norm, W * 2);
    m->top.want("embed", &m->embed, 0, (size_t)c.vocab * W * 2);
    m->top.want("embed.norm", &m->embed_norm, 0, W * 2);
    m->top.want("final.norm", &m->final_norm, 0, W * 2);
    const size_t cap = m->blocks.rows;
    GA(m->x, T * W * 4);
    GA(m->h, T * W * m->esz());
    GA(m->hsel, T * W * m->esz());
    GA(m->y, T * W * 4);
    GA(m->fused, T * std::max(nf, (size_t)c.vocab) * 4);   // also the logits of a greedy-only step
    GA(m->cq, T * qr * m->esz());
    GA(m->q, T * nq * 4);
    GA(m->qabs, T * hr * 4);
    GA(m->qrot, T * hrd * 4);
    GA(m->olat, T * hr * 4);
    GA(m->attn, T * hv * m->esz());
    GA(m->attn_ws, (size_t)24576 * (maxr + 2) * 4);   // key partitions of launches with few rows: tokens x heads x partitions < 24576
    GA(m->norm, T * mh * 4);
    GA(m->floor, T * mh * 4);
    GA(m->readout, T * mhv * 4);
    GA(m->rec, T * mhv * m->esz());
    GA(m->argmax_keys, T * ((size_t)c.vocab / VMX_ARGMAX_CHUNK + 1) * 8);
    GA(m->gu, T * gu * 4);
    GA(m->dact, T * dff * m->esz());
    GA(m->rlogits, T * ne * 4);
    GA(m->act, (cap + 1) * eff * m->esz());
    GA(m->ydown, (cap + 1) * W * 4);
    GA(m->sact, T * sff * m->esz());
    GA(m->sout, T * W * 4);
#undef GA
    if (!rc) rc = m->blocks.alloc();
    if (rc) {
        vmx_fofinex_destroy(m);
        return rc;
    }
    *out = m;
    return VMX_OK;
}

extern "C" void vmx_fofinex_destroy(vmx_fofinex *m) {
    if (!m) return;
    for (Layer &L : m->layers)
        for (Buf *b : {&L.norm1, &L.norm1b, &L.norm2, &L.norm2b, &L.wfused, &L.bias, &L.wo, &L.dq_norm, &L.wuq, &L.dkv_norm, &L.uk, &L.uk_t, &L.uv,
                       &L.rot_steps, &L.cache, &L.head_norm, &L.memory, &L.maxima, &L.wgu, &L.bias_gu, &L.wdown, &L.bias_down, &L.router, &L.correction,
                       &L.eup, &L.edown, &L.sup, &L.sdown})
            b->release();
    for (Buf *b : {&m->embed, &m->embed_norm, &m->final_norm, &m->x, &m->h, &m->hsel, &m->y, &m->fused, &m->cq, &m->q, &m->qabs, &m->qrot, &m->olat,
                   &m->attn, &m->attn_ws, &m->norm, &m->floor, &m->readout, &m->rec, &m->argmax_keys, &m->gu, &m->dact, &m->rlogits, &m->act, &m->ydown,
                   &m->sact, &m->sout})
        b->release();
    m->blocks.release();
    delete m;
}

extern "C" int vmx_fofinex_load_tensor(vmx_fofinex *m, const char *name, const void *data, size_t bytes, void *stream) {
    VMX_REQUIRE(m && name && (data || bytes == 0), "fofinex_load_tensor: null pointer");
    hipStream_t st = vmx_stream(stream);
    const std::string n(name);
    std::string key = n;
    VmxTensorTable *table = &m->top;
    Layer *L = nullptr;
    if (n.size() > 1 && n[0] == 'l' && isdigit((unsigned char)n[1])) {
        const size_t dot = n.find('.');
        VMX_REQUIRE(dot != std::string::npos, "fofinex_load_tensor: unknown tensor `%s`", name);
        const int li = atoi(n.substr(1, dot - 1).c_str());
        VMX_REQUIRE(li >= 0 && li < m->cfg.num_layers, "fofinex_load_tensor: `%s`: the model has %d layers", name, m->cfg.num_layers);
        L = &m->layers[li];
        table = L;
        key = n.substr(dot + 1);
    }
    const VmxTensorTable::Seg *dst = table->find(key);
    VMX_REQUIRE(dst, "fofinex_load_tensor: unknown tensor `%s`", name);
    VMX_REQUIRE(bytes == dst->bytes, "fofinex_load_tensor: `%s`: expected %zu bytes of bf16, got %zu", name, dst->bytes, bytes);
    if (bytes > 0) {
        if (int rc = vmx_upload(*dst->buf, dst->offset, data, bytes, st)) return rc;
        if (L && key == "mix.uk") {
            if (int rc = vmx_latent_transpose_heads(L->uk_t.as<uint16_t>(), L->uk.as<uint16_t>(), L->c.heads, L->c.dim, L->c.kv_rank, st)) return rc;
            VMX_CHECK_HIP(hipStreamSynchronize(st));
        }
    }
    table->loaded(key);
    return VMX_OK;
}

extern "C" int vmx_fofinex_missing_tensors(const vmx_fofinex *m) {
    if (!m) return -1;
    size_t n = m->top.missing.size();
    std::string first = n ? m->top.missing[0] : "";
    for (size_t li = 0; li < m->layers.size(); li++) {
        const Layer &L = m->layers[li];
        if (first.empty() && !L.missing.empty()) first = "l" + std::to_string(li) + "." + L.missing[0];
        n += L.missing.size();
    }
    if (n) vmx_set_error("fofinex: %zu tensors not loaded, first `%s`", n, first.c_str());
    return (int)n;
}

namespace {

// what a step's kernels are given besides their operands
struct Step {
    const int32_t *positions, *slots, *seq_ids, *block_tables, *seq_starts, *state_slots;
    int T, num_seqs, max_blocks;
    hipStream_t st;
};

// y = W a (+ bias): rows of K numbers (f32 or bf16, contiguous) times a checkpoint matrix [N, K]
VmxLinear product(const Buf &a, int a_f32, int K, const Buf &w, int N, void *c, int c_f32, int T, int exact) {
    VmxLinear p;
    p.A = a.p, p.a_f32 = a_f32, p.lda = K;
    p.W = w.as<uint16_t>(), p.w_sn = K, p.w_sk = 1;
    p.C = c, p.c_f32 = c_f32, p.ldc = N;
    p.M = T, p.N = N, p.K = K, p.exact = exact;
    return p;
}

// m->y = mixer(m->h)
int latent_attention(vmx_fofinex *m, Layer &L, const Step &s) {
    const vmx_fofinex_layer_config &lc = L.c;
    const int W = m->cfg.width, T = s.T, f32 = m->f32() ? 1 : 0, cdt = f32 ? VMX_F32 : VMX_BF16;
    const int H = lc.heads, D = lc.dim, RD = lc.rot_dim, R = lc.kv_rank, Q = lc.q_rank, V = lc.vdim, NQ = H * (D + RD);
    float *fused = m->fused.as<float>();
    Buf &cache = lc.kv_from < 0 ? L.cache : m->layers[lc.kv_from].cache;
    if (int rc = vmx_linear_launch(product(m->h, f32, W, L.wfused, L.nf, fused, 1, T, f32), s.st)) return rc;   // query latent | key/value latent, key part
    vmx_latent_prepare pk = {};   // both latents normed, the key part rotated, the cache row written
    pk.q_latent = fused + L.dq_off, pk.ldq_latent = L.nf, pk.q_rank = Q, pk.q_latent_norm_bf16 = L.dq_norm.as<uint16_t>();
    pk.eps = m->cfg.norm_eps;
    pk.kv_rank = R, pk.rot_dim = RD, pk.inv_freq = L.rot_steps.as<float>(), pk.rot_dims = lc.rot.dims, pk.rot_halves = 1, pk.rot_mul = L.rot_mul;
    if (lc.kv_from < 0) pk.kv = fused + L.dkv_off, pk.ldkv = L.nf, pk.latent_norm_bf16 = L.dkv_norm.as<uint16_t>();
    if (int rc = vmx_latent_prepare_rows(&pk, s.positions, s.slots, cache.p, cdt, m->cq.p, T, s.st)) return rc;
    if (int rc = vmx_linear_launch(product(m->cq, f32, Q, L.wuq, NQ, m->q.p, 1, T, f32), s.st)) return rc;
    if (RD > 0) {   // the heads' rotated query parts
        vmx_latent_prepare pq = {};
        pq.q = m->q.as<float>(), pq.ldq = NQ, pq.heads = H, pq.dim = D, pq.q_rot = m->qrot.as<float>();
        pq.kv_rank = R, pq.rot_dim = RD, pq.inv_freq = L.rot_steps.as<float>(), pq.rot_dims = lc.rot.dims, pq.rot_halves = 1, pq.rot_mul = L.rot_mul;
        if (int rc = vmx_latent_prepare_rows(&pq, s.positions, nullptr, nullptr, cdt, nullptr, T, s.st)) return rc;
    }
    if (D > 0) {    // qa_h = U_h^T q_h: per head, [T, D] x [D, R]
        VmxLinear a;
        a.A = m->q.p, a.a_f32 = 1, a.lda = NQ, a.a_bs = D + RD;
        a.W = L.uk_t.as<uint16_t>(), a.w_sn = D, a.w_sk = 1, a.w_bs = (int64_t)D * R;
        a.C = m->qabs.p, a.c_f32 = 1, a.ldc = (int64_t)H * R, a.c_bs = R;
        a.M = T, a.N = R, a.K = D, a.batch = H, a.exact = f32;
        if (int rc = vmx_linear_launch(a, s.st)) return rc;
    } else {
        if (int rc = vmx_zero_f32(m->qabs.as<float>(), (int64_t)T * H * R, s.st)) return rc;
    }
    if (int rc = vmx_latent_attention(m->olat.as<float>(), m->qabs.as<float>(), m->qrot.as<float>(), cache.p, cdt, s.block_tables, s.max_blocks, s.seq_ids,
                                      s.positions, nullptr, lc.scale, 0, T, H, R, RD, m->cfg.block_size, m->attn_ws.p, m->attn_ws.bytes, s.st))
        return rc;
    VmxLinear v;    // v_h = V_h o_h: per head, [T, R] x [V, R]^T
    v.A = m->olat.p, v.a_f32 = 1, v.lda = (int64_t)H * R, v.a_bs = R;
    v.W = L.uv.as<uint16_t>(), v.w_sn = R, v.w_sk = 1, v.w_bs = (int64_t)V * R;
    v.C = m->attn.p, v.c_f32 = f32, v.ldc = (int64_t)H * V, v.c_bs = V;
    v.M = T, v.N = V, v.K = R, v.batch = H, v.exact = f32;
    if (int rc = vmx_linear_launch(v, s.st)) return rc;
    return vmx_linear_launch(product(m->attn, f32, H * V, L.wo, W, m->y.p, 1, T, f32), s.st);
}

int exp_memory(vmx_fofinex *m, Layer &L, const Step &s) {
    const vmx_fofinex_layer_config &lc = L.c;
    const int W = m->cfg.width, T = s.T, f32 = m->f32() ? 1 : 0, cdt = f32 ? VMX_F32 : VMX_BF16, nf = L.nf;
    const int H = lc.heads, D = lc.dim, V = lc.vdim;
    float *fused = m->fused.as<float>(), *gain = fused + L.i_off, *decay = fused + L.f_off;
    VmxLinear p = product(m->h, f32, W, L.wfused, nf, fused, 1, T, f32);   // q | k | v | read-out gate | input gate | forget gate
    p.bias = L.bias.as<uint16_t>();
    if (int rc = vmx_linear_launch(p, s.st)) return rc;
    if (int rc = vmx_exp_gate_scan(gain, nf, decay, nf, m->floor.as<float>(), H, L.maxima.as<float>(), lc.gate_cap, s.positions, s.seq_starts,
                                   s.state_slots, s.num_seqs, H, s.st))
        return rc;
    const vmx_matrix_memory_opts mo = {gain, nf, m->norm.as<float>(), H, f32 ? 0 : 1, T};
    if (int rc = vmx_matrix_memory_recurrence_ex(m->readout.as<float>(), (int64_t)H * V, fused + L.q_off, nf, 1.0f / sqrtf((float)D), fused + L.k_off, nf,
                                                 fused + L.v_off, nf, decay, nf, 1, nullptr, 0, L.memory.as<float>(), s.positions, s.seq_starts,
                                                 s.state_slots, s.num_seqs, H, H, D, V, &mo, s.st))
        return rc;
    const vmx_read_out_opts ro = {0, 1, m->norm.as<float>(), H, m->floor.as<float>(), H, 1e-6f};
    if (int rc = vmx_head_read_out(m->rec.p, cdt, m->readout.as<float>(), (int64_t)H * V, L.head_norm.as<uint16_t>(), fused + L.g_off, nf,
                                   m->cfg.norm_eps, T, H, V, &ro, s.st))
        return rc;
    return vmx_linear_launch(product(m->rec, f32, H * V, L.wo, W, m->y.p, 1, T, f32), s.st);
}

// m->y = ff(m->h)
int dense_glu(vmx_fofinex *m, Layer &L, const Step &s) {
    const int W = m->cfg.width, F = L.c.ff, f32 = m->f32() ? 1 : 0;
    VmxLinear u = product(m->h, f32, W, L.wgu, 2 * F, m->gu.p, 1, s.T, f32);
    u.bias = L.bias_gu.as<uint16_t>();
    if (int rc = vmx_linear_launch(u, s.st)) return rc;
    if (int rc = vmx_glu_gelu_rows(m->dact.p, f32, m->gu.as<float>(), s.T, F, s.st)) return rc;
    VmxLinear d = product(m->dact, f32, F, L.wdown, W, m->y.p, 1, s.T, f32);
    d.bias = L.bias_down.as<uint16_t>();
    return vmx_linear_launch(d, s.st);
}

// the experts' results of every (token, slot) pair and the shared expert's; the norm kernel sums them
int corrected_moe(vmx_fofinex *m, Layer &L, const Step &s, VmxSandwich &sw) {
    const vmx_fofinex_layer_config &lc = L.c;
    const int W = m->cfg.width, f32 = m->f32() ? 1 : 0, E = lc.experts, k = lc.top, ff = lc.expert_ff, S = lc.shared_ff, pairs = s.T * k, NR = L.router_rows;
    VmxExpertBlocks &b = m->blocks;
    // router logits (and the shared expert's gate): always a true f32 product
    if (int rc = vmx_linear_launch(product(m->h, f32, W, L.router, NR, m->rlogits.p, 1, s.T, 1), s.st)) return rc;
    if (int rc = vmx_grouped_topk_sigmoid(m->rlogits.as<float>(), NR, L.correction.as<uint16_t>(), b.topw.as<float>(), b.topi.as<int32_t>(), s.T, E, k,
                                          lc.groups, lc.keep_groups, lc.router_scale, s.st))
        return rc;
    if (int rc = b.plan(pairs, E, s.st)) return rc;
    VmxLinear u = product(m->h, f32, W, L.eup, ff, m->act.p, f32, 0, f32);   // act = relu(W_up[e] h)^2 over the pairs' rows
    u.epilogue = VMX_EP_RELU2;
    b.first(u, pairs, k, (int64_t)ff * W);
    if (int rc = vmx_linear_launch(u, s.st)) return rc;
    VmxLinear d = product(m->act, f32, ff, L.edown, W, m->ydown.p, 1, 0, f32);
    b.second(d, (int64_t)ff * W);
    if (int rc = vmx_linear_launch(d, s.st)) return rc;
    sw.y = m->ydown.as<float>(), sw.pair_rows = b.pair_rows, sw.pair_w = b.topw.as<float>(), sw.top = k;
    if (!S) return VMX_OK;
    VmxLinear su = product(m->h, f32, W, L.sup, S, m->sact.p, f32, s.T, f32);
    su.epilogue = VMX_EP_RELU2;
    if (int rc = vmx_linear_launch(su, s.st)) return rc;
    if (int rc = vmx_linear_launch(product(m->sact, f32, S, L.sdown, W, m->sout.p, 1, s.T, f32), s.st)) return rc;
    sw.shared = m->sout.as<float>(), sw.shared_gate = m->rlogits.as<float>() + E, sw.ld_shared_gate = NR;
    return VMX_OK;
}

}  // namespace

extern "C" int vmx_fofinex_forward(vmx_fofinex *m, const int32_t *tokens, const int32_t *positions, const int32_t *slots, const int32_t *seq_ids,
                                   int num_tokens, const int32_t *block_tables, int num_seqs, int max_blocks_per_seq, const int32_t *seq_starts,
                                   const int32_t *state_slots, const int32_t *logit_rows, int num_logit_rows, float *logits, int32_t *greedy_ids,
                                   float *layer_trace, void *stream) {
    VMX_REQUIRE(m && tokens && positions && slots && seq_ids && block_tables && seq_starts && state_slots, "fofinex_forward: null pointer");
    const vmx_fofinex_config &c = m->cfg;
    VMX_REQUIRE(num_tokens >= 1 && num_tokens <= c.max_tokens, "fofinex_forward: %d tokens, the model was created for at most %d", num_tokens,
                c.max_tokens);
    VMX_REQUIRE(num_seqs >= 1 && num_seqs <= c.max_seqs && max_blocks_per_seq >= 1, "fofinex_forward: bad sequence count or block-table shape");
    VMX_REQUIRE(num_logit_rows >= 0 && num_logit_rows <= num_tokens && (num_logit_rows == 0 || (logit_rows && (logits || greedy_ids))),
                "fofinex_forward: bad logit rows");
    if (vmx_fofinex_missing_tensors(m) != 0) return VMX_EINVAL;
    const Step s{positions, slots, seq_ids, block_tables, seq_starts, state_slots, num_tokens, num_seqs, max_blocks_per_seq, vmx_stream(stream)};
    hipStream_t st = s.st;
    const int T = num_tokens, W = c.width, f32 = m->f32() ? 1 : 0;
    float *x = m->x.as<float>();
    VmxSandwich base;
    base.x = x, base.h = m->h.p, base.h_f32 = f32, base.width = W, base.eps = c.norm_eps, base.centered = 1;
    VmxSandwich in = base;    // x = N(embed[token]), and the first mixer's input
    in.embed = m->embed.as<uint16_t>(), in.tokens = tokens, in.vocab = c.vocab, in.accumulate = 0;
    in.w_post = m->embed_norm.as<uint16_t>(), in.w_next = m->layers[0].norm1.as<uint16_t>();
    if (int rc = vmx_sandwich_norm(in, T, st)) return rc;
    for (int li = 0; li < c.num_layers; li++) {
        Layer &L = m->layers[li];
        const uint16_t *next_layer = li + 1 < c.num_layers ? m->layers[li + 1].norm1.as<uint16_t>() : nullptr;
        const bool ff = L.c.mlp != VMX_MLP_NONE;
        if (int rc = L.c.mixer == VMX_MIXER_LATENT_ATTENTION ? latent_attention(m, L, s) : exp_memory(m, L, s)) return rc;
        VmxSandwich sw = base;
        sw.y = m->y.as<float>(), sw.w_post = L.norm1b.as<uint16_t>(), sw.w_next = ff ? L.norm2.as<uint16_t>() : next_layer;
        if (int rc = vmx_sandwich_norm(sw, T, st)) return rc;
        if (ff) {
            VmxSandwich sf = base;
            sf.y = m->y.as<float>(), sf.w_post = L.norm2b.as<uint16_t>(), sf.w_next = next_layer;
            if (int rc = L.c.mlp == VMX_MLP_DENSE_GLU ? dense_glu(m, L, s) : corrected_moe(m, L, s, sf)) return rc;
            if (int rc = vmx_sandwich_norm(sf, T, st)) return rc;
        }
        if (layer_trace)
            VMX_CHECK_HIP(hipMemcpyAsync(layer_trace + (size_t)li * T * W, x, (size_t)T * W * 4, hipMemcpyDeviceToDevice, st));
    }
    if (num_logit_rows > 0) {
        if (int rc = vmx_layer_norm_f32in(m->hsel.p, f32, x, logit_rows, m->final_norm.as<uint16_t>(), W, c.norm_eps, num_logit_rows, st)) return rc;
        float *lg = logits ? logits : m->fused.as<float>();   // greedy ids only: the logits live in a workspace
        if (int rc = vmx_linear_launch(product(m->hsel, f32, W, m->embed, c.vocab, lg, 1, num_logit_rows, f32), st)) return rc;
        if (greedy_ids)
            if (int rc = vmx_argmax_f32_rows(greedy_ids, m->argmax_keys.as<unsigned long long>(), lg, num_logit_rows, c.vocab, st)) return rc;
    }
    return VMX_OK;
}
