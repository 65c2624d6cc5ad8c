// Whole-step executor of the Larolorn decoder family: layers listed in the model's configuration whose sublayers read the residual
// stream as it is and whose results are normed before they are added,
//   x = embed[token];   x <- x + m N1(mixer(x));   x <- x + m N2(ff(x))  (ff may be absent);   logits = head . N(x) * logit_scale
// with N an RMS norm with a gain and one multiplier m for the model.  Mixers (every size and constant per layer):
//   VMX_MIXER_LATENT_ATTENTION    keys / values compressed to one latent and one rotated key part per token in a paged cache
//                                 (latent_attn.hip), queries straight from x, rotation of neighbours, a sliding window, a sigmoid per head
//                                 on the output
//   VMX_MIXER_CHUNKED_LIGHTNING   half the sum of two normed branches over the same x: grouped-query attention inside chunks of
//                                 positions (window_attn.hip: biased projections, RMS norms over the whole q and k rows, rotation in
//                                 halves, a sink per head, biased output product) and a matrix memory with one constant decay per head
//                                 (delta_rule.hip: SiLU on q, k and v; the read-out of all heads normed together and gated)
// Feed-forward VMX_MLP_CLAMPED_GLU: y = W_down (g sigmoid(1.702 g) (u + 1)), g = min(W_gate x, limit), u = W_up x clamped to +- limit.
// A layer may run with an earlier or later layer's weights (weights_of): it then owns nothing but its cache and its state.
//
// Everything that reads a mixer's input is ONE product whose f32 row the other kernels address by column offset; biases and the SiLU of
// the memory's columns happen in its epilogue.  The norm of a sublayer's result (for two branches all three norms), the residual sum
// and the next product's bf16 input row are one kernel (sandwich_norm_kernel).  The stream, norms, positions and angles, scores,
// softmax, decays, the memory and its read-out are f32 in both modes; VMX_BF16 rounds the operands of the linears and the cache rows
// to bf16, VMX_F32 multiplies in true f32 everywhere.  The forward call allocates nothing, reads nothing back and is graph-capturable.
#include "executor_common.h"
#include <string.h>

namespace {

using Buf = VmxBuf;

constexpr float GLU_SLOPE = 1.702f;

struct Layer : VmxTensorTable {
    vmx_larolorn_layer_config c;
    // weights (empty in a layer that runs with another one's)
    Buf norm1, norm2, wfused, bias, wo, rot_steps;
    Buf dkv_norm, uk, uk_t, uv;                                                              // latent attention
    Buf qnorm, knorm, sink, bias_o, left_out, right_out, wo_right, read_norm, decay;         // two-sided mixer
    Buf wgu, wdown;                                                                          // feed-forward
    float rot_mul = 1.f;
    int nf = 0, q_off = 0, dkv_off = 0, g_off = 0, k_off = 0, v_off = 0, rq_off = 0, rk_off = 0, rv_off = 0;
    // what every layer keeps of its own
    Buf cache, vcache, memory;
};

}  // namespace

struct vmx_larolorn {
    vmx_larolorn_config cfg;
    std::vector<Layer> layers;
    VmxTensorTable top;
    Buf embed, final_norm, head;
    Buf x, h, hsel, y, side, fused, q, qabs, olat, attn, attn_ws, readout, rec, act, argmax_keys;
    bool f32() const { return cfg.dtype == VMX_F32; }
    size_t esz() const { return f32() ? 4 : 2; }
    const Layer &weights(const Layer &L) const { return L.c.weights_of < 0 ? L : layers[L.c.weights_of]; }
    // what the products read: the stream itself in f32 mode, its bf16 copy otherwise
    const Buf &input() const { return f32() ? x : h; }
};

// Two layers that share weights must agree in everything that shapes them or that the kernels are given.
static bool same_layer(const vmx_larolorn_layer_config &a, const vmx_larolorn_layer_config &b) {
    if (a.mixer != b.mixer || a.mlp != b.mlp) return false;
    if (a.heads != b.heads || a.dim != b.dim || a.vdim != b.vdim || a.scale != b.scale || a.mask != b.mask) return false;
    const vmx_rotation &r = a.rot, &s = b.rot;
    if (r.dims != s.dims || r.base != s.base || r.factor != s.factor) return false;
    if (a.mlp != VMX_MLP_NONE && (a.ff != b.ff || a.limit != b.limit)) return false;
    if (a.mixer == VMX_MIXER_LATENT_ATTENTION) return a.rot_dim == b.rot_dim && a.kv_rank == b.kv_rank;
    if (a.kv_heads != b.kv_heads || a.r_heads != b.r_heads || a.r_dim != b.r_dim || a.r_vdim != b.r_vdim) return false;
    return a.decay && b.decay && memcmp(a.decay, b.decay, (size_t)a.r_heads * 4) == 0;
}

extern "C" int vmx_larolorn_create(const vmx_larolorn_config *cfg, const vmx_larolorn_layer_config *layer_cfgs, vmx_larolorn **out) {
    VMX_REQUIRE(cfg && layer_cfgs && out, "larolorn_create: null pointer");
    const vmx_larolorn_config &c = *cfg;
    VMX_REQUIRE(c.vocab >= 1 && c.width >= 1 && c.num_layers >= 1, "larolorn_create: bad sizes (vocab %d, width %d, layers %d)", c.vocab, c.width,
                c.num_layers);
    VMX_REQUIRE(c.dtype == VMX_F32 || c.dtype == VMX_BF16, "larolorn_create: dtype must be VMX_F32 or VMX_BF16");
    VMX_REQUIRE(c.block_size >= 1 && c.num_blocks >= 1 && c.max_tokens >= 1 && c.max_seqs >= 1 && c.state_slots >= 1,
                "larolorn_create: bad cache / batch geometry");
    vmx_larolorn *m = new vmx_larolorn();
    m->cfg = c;
    m->layers.resize(c.num_layers);
    const size_t T = c.max_tokens, W = c.width, rows = (size_t)c.num_blocks * c.block_size;
    size_t nf = 8, nq = 1, hr = 1, hv = 1, rhv = 1, dff = 1, ws = 16;
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
        L.c = layer_cfgs[li];
        L.c.decay = nullptr;   // host arrays of the caller are read here and not kept
        const vmx_larolorn_layer_config &lc = layer_cfgs[li];
        const bool own = lc.weights_of < 0;
        if (!own && (lc.weights_of >= c.num_layers || layer_cfgs[lc.weights_of].weights_of >= 0))
            BAD("larolorn_create: layer %d: layer %d has no weights of its own", li, lc.weights_of);
        if (!own && !same_layer(lc, layer_cfgs[lc.weights_of])) BAD("larolorn_create: layer %d differs from layer %d, whose weights it runs with", li, lc.weights_of);
        if (lc.heads < 1 || lc.dim < 0 || lc.vdim < 1 || lc.mask < 0)
            BAD("larolorn_create: layer %d: bad head count, sizes or mask (heads %d, dim %d, vdim %d, mask %d)", li, lc.heads, lc.dim, lc.vdim, lc.mask);
        const size_t H = lc.heads, D = lc.dim, V = lc.vdim;
        int at = 0;
        auto seg = [&](size_t n) {
            const int o = at;
            at = vmx_pad8(at + (int)n);
            return o;
        };
        if (lc.mixer == VMX_MIXER_LATENT_ATTENTION) {
            if (lc.rot_dim < 0 || lc.dim + lc.rot_dim < 1 || lc.kv_rank < 1 || lc.kv_rank > 512)
                BAD("larolorn_create: layer %d: bad latent-attention sizes (dim %d, rot_dim %d, kv_rank %d; kv_rank up to 512)", li, lc.dim, lc.rot_dim,
                    lc.kv_rank);
            if (!vmx_rotation_ok(lc.rot, lc.rot_dim)) BAD("larolorn_create: layer %d: bad rotation (%d of %d coordinates)", li, lc.rot.dims, lc.rot_dim);
            const size_t R = lc.kv_rank, RD = lc.rot_dim;
            GA(L.cache, rows * (R + RD) * m->esz());
            if (own) {
                L.q_off = seg(H * (D + RD));
                L.dkv_off = seg(R + RD);
                L.g_off = seg(H);
                L.nf = at;
                GA(L.wfused, (size_t)L.nf * W * 2);
                GA(L.dkv_norm, R * 2);
                GA(L.uk, H * D * R * 2);
                GA(L.uk_t, H * D * R * 2);
                GA(L.uv, H * V * R * 2);
                GA(L.wo, W * H * V * 2);
                L.want("mix.q", &L.wfused, (size_t)L.q_off * W * 2, H * (D + RD) * W * 2);
                L.want("mix.dkv", &L.wfused, (size_t)L.dkv_off * W * 2, (R + RD) * W * 2);
                L.want("mix.dkv.norm", &L.dkv_norm, 0, R * 2);
                L.want("mix.uk", &L.uk, 0, H * D * R * 2);
                L.want("mix.uv", &L.uv, 0, H * V * R * 2);
                L.want("mix.g", &L.wfused, (size_t)L.g_off * W * 2, H * W * 2);
                L.want("mix.o", &L.wo, 0, W * H * V * 2);
            }
            nq = std::max(nq, H * RD);
            hr = std::max(hr, H * R);
            ws = std::max(ws, (size_t)24576 * (R + 2) * 4);   // key partitions of launches with few rows: tokens x heads x partitions < 24576
        } else if (lc.mixer == VMX_MIXER_CHUNKED_LIGHTNING) {
            if (lc.kv_heads < 1 || lc.heads % lc.kv_heads || lc.dim < 1 || lc.dim > 256 || lc.vdim > 256)
                BAD("larolorn_create: layer %d: bad attention sizes (heads %d, kv_heads %d, dim %d, vdim %d; sizes up to 256)", li, lc.heads, lc.kv_heads, lc.dim,
                    lc.vdim);
            if (!vmx_rotation_ok(lc.rot, lc.dim)) BAD("larolorn_create: layer %d: bad rotation (%d of %d coordinates)", li, lc.rot.dims, lc.dim);
            if (lc.r_heads < 1 || lc.r_dim < 1 || lc.r_dim > 256 || lc.r_vdim < 1 || !lc.decay)
                BAD("larolorn_create: layer %d: bad memory (heads %d, key size %d outside 1..256, value size %d, or no decays)", li, lc.r_heads, lc.r_dim, lc.r_vdim);
            const size_t G = lc.kv_heads, RH = lc.r_heads, RD = lc.r_dim, RV = lc.r_vdim;
            GA(L.cache, rows * G * D * m->esz());
            GA(L.vcache, rows * G * V * m->esz());
            GA(L.memory, vmx_gated_delta_rule_state_bytes(c.state_slots, lc.r_heads, lc.r_dim, lc.r_vdim));
            if (own) {
                L.q_off = seg(H * D);
                L.k_off = seg(G * D);
                L.v_off = seg(G * V);
                L.rq_off = seg(RH * RD);
                L.rk_off = seg(RH * RD);
                L.rv_off = seg(RH * RV);
                L.g_off = seg(RH * RV);
                L.nf = at;
                GA(L.wfused, (size_t)L.nf * W * 2);
                GA(L.bias, (size_t)L.nf * 2);
                GA(L.qnorm, H * D * 2);
                GA(L.knorm, G * D * 2);
                GA(L.sink, H * 2);
                GA(L.wo, W * H * V * 2);
                GA(L.bias_o, W * 2);
                GA(L.left_out, W * 2);
                GA(L.right_out, W * 2);
                GA(L.wo_right, W * RH * RV * 2);
                GA(L.read_norm, RH * RV * 2);
                GA(L.decay, RH * 4);
                if (!rc && hipMemcpy(L.decay.p, lc.decay, RH * 4, hipMemcpyHostToDevice) != hipSuccess) BAD("larolorn_create: upload failed");
                L.want("mix.left.q", &L.wfused, (size_t)L.q_off * W * 2, H * D * W * 2);
                L.want("mix.left.q.b", &L.bias, (size_t)L.q_off * 2, H * D * 2);
                L.want("mix.left.k", &L.wfused, (size_t)L.k_off * W * 2, G * D * W * 2);
                L.want("mix.left.k.b", &L.bias, (size_t)L.k_off * 2, G * D * 2);
                L.want("mix.left.v", &L.wfused, (size_t)L.v_off * W * 2, G * V * W * 2);
                L.want("mix.left.v.b", &L.bias, (size_t)L.v_off * 2, G * V * 2);
                L.want("mix.left.q.norm", &L.qnorm, 0, H * D * 2);
                L.want("mix.left.k.norm", &L.knorm, 0, G * D * 2);
                L.want("mix.left.sink", &L.sink, 0, H * 2);
                L.want("mix.left.o", &L.wo, 0, W * H * V * 2);
                L.want("mix.left.o.b", &L.bias_o, 0, W * 2);
                L.want("mix.left.out", &L.left_out, 0, W * 2);
                L.want("mix.right.q", &L.wfused, (size_t)L.rq_off * W * 2, RH * RD * W * 2);
                L.want("mix.right.k", &L.wfused, (size_t)L.rk_off * W * 2, RH * RD * W * 2);
                L.want("mix.right.v", &L.wfused, (size_t)L.rv_off * W * 2, RH * RV * W * 2);
                L.want("mix.right.g", &L.wfused, (size_t)L.g_off * W * 2, RH * RV * W * 2);
                L.want("mix.right.o", &L.wo_right, 0, W * RH * RV * 2);
                L.want("mix.right.norm", &L.read_norm, 0, RH * RV * 2);
                L.want("mix.right.out", &L.right_out, 0, W * 2);
            }
            nq = std::max(nq, H * D);
            rhv = std::max(rhv, RH * RV);
            ws = std::max(ws, vmx_window_attention_workspace_bytes((int)T, lc.heads, lc.vdim));
        } else {
            vmx_set_error("larolorn_create: layer %d: unknown mixer kind %d", li, lc.mixer);
            rc = VMX_EUNSUPPORTED;
            break;
        }
        hv = std::max(hv, H * V);
        if (own) {
            if (!rc) rc = vmx_upload_rotation(lc.rot, L.rot_steps, L.rot_mul);
            GA(L.norm1, W * 2);
            L.want("norm1", &L.norm1, 0, W * 2);
        }
        nf = std::max(nf, (size_t)L.nf);
        if (lc.mlp == VMX_MLP_NONE) continue;
        if (lc.mlp != VMX_MLP_CLAMPED_GLU) {
            vmx_set_error("larolorn_create: layer %d: unknown feed-forward kind %d", li, lc.mlp);
            rc = VMX_EUNSUPPORTED;
            break;
        }
        if (lc.ff < 1 || !(lc.limit >= 0.f)) BAD("larolorn_create: layer %d: bad feed-forward (width %d, limit %g)", li, lc.ff, lc.limit);
        const size_t F = lc.ff;
        if (own) {
            GA(L.norm2, W * 2);
            GA(L.wgu, 2 * F * W * 2);   // gate rows, then up rows
            GA(L.wdown, W * F * 2);
            L.want("norm2", &L.norm2, 0, W * 2);
            L.want("mlp.gate", &L.wgu, 0, F * W * 2);
            L.want("mlp.up", &L.wgu, F * W * 2, F * W * 2);
            L.want("mlp.down", &L.wdown, 0, W * F * 2);
        }
        nf = std::max(nf, 2 * F);
        dff = std::max(dff, F);
    }
#undef BAD
    GA(m->embed, (size_t)c.vocab * W * 2);
    GA(m->final_norm, W * 2);
    GA(m->head, (size_t)c.vocab * W * 2);
    m->top.want("embed", &m->embed, 0, (size_t)c.vocab * W * 2);
    m->top.want("final.norm", &m->final_norm, 0, W * 2);
    m->top.want("head", &m->head, 0, (size_t)c.vocab * W * 2);
    GA(m->x, T * W * 4);
    GA(m->h, m->f32() ? 16 : T * W * 2);
    GA(m->hsel, T * W * m->esz());
    GA(m->y, T * W * 4);
    GA(m->side, T * W * 4);
    GA(m->fused, T * std::max(nf, (size_t)c.vocab) * 4);   // also gate | up of the feed-forward and the logits of a greedy-only step
    GA(m->q, T * nq * 4);
    GA(m->qabs, T * hr * 4);
    GA(m->olat, T * hr * 4);
    GA(m->attn, T * hv * m->esz());
    GA(m->attn_ws, ws);
    GA(m->readout, T * rhv * 4);
    GA(m->rec, T * rhv * m->esz());
    GA(m->act, T * dff * m->esz());
    GA(m->argmax_keys, T * ((size_t)c.vocab / VMX_ARGMAX_CHUNK + 1) * 8);
#undef GA
    if (rc) {
        vmx_larolorn_destroy(m);
        return rc;
    }
    *out = m;
    return VMX_OK;
}

extern "C" void vmx_larolorn_destroy(vmx_larolorn *m) {
    if (!m) return;
    for (Layer &L : m->layers)
        for (Buf *b : {&L.norm1, &L.norm2, &L.wfused, &L.bias, &L.wo, &L.rot_steps, &L.dkv_norm, &L.uk, &L.uk_t, &L.uv, &L.qnorm, &L.knorm, &L.sink, &L.bias_o,
                       &L.left_out, &L.right_out, &L.wo_right, &L.read_norm, &L.decay, &L.wgu, &L.wdown, &L.cache, &L.vcache, &L.memory})
            b->release();
    for (Buf *b : {&m->embed, &m->final_norm, &m->head, &m->x, &m->h, &m->hsel, &m->y, &m->side, &m->fused, &m->q, &m->qabs, &m->olat, &m->attn, &m->attn_ws,
                   &m->readout, &m->rec, &m->act, &m->argmax_keys})
        b->release();
    delete m;
}

extern "C" int vmx_larolorn_load_tensor(vmx_larolorn *m, const char *name, const void *data, size_t bytes, void *stream) {
    VMX_REQUIRE(m && name && (data || bytes == 0), "larolorn_load_tensor: null pointer");
    hipStream_t st = vmx_stream(stream);
    const std::string n(name);
    std::string key = n;
    VmxTensorTable *table = &m->top;
    Layer *L = nullptr;
    if (n.size() > 1 && n[0] == 'l' && isdigit((unsigned char)n[1])) {
        const size_t dot = n.find('.');
        VMX_REQUIRE(dot != std::string::npos, "larolorn_load_tensor: unknown tensor `%s`", name);
        const int li = atoi(n.substr(1, dot - 1).c_str());
        VMX_REQUIRE(li >= 0 && li < m->cfg.num_layers, "larolorn_load_tensor: `%s`: the model has %d layers", name, m->cfg.num_layers);
        L = &m->layers[li];
        table = L;
        key = n.substr(dot + 1);
    }
    const VmxTensorTable::Seg *dst = table->find(key);
    VMX_REQUIRE(dst, "larolorn_load_tensor: unknown tensor `%s`", name);
    VMX_REQUIRE(bytes == dst->bytes, "larolorn_load_tensor: `%s`: expected %zu bytes of bf16, got %zu", name, dst->bytes, bytes);
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

extern "C" int vmx_larolorn_missing_tensors(const vmx_larolorn *m) {
    if (!m) return -1;
    size_t n = m->top.missing.size();
    std::string first = n ? m->top.missing[0] : "";
    for (size_t li = 0; li < m->layers.size(); li++) {
        const Layer &L = m->layers[li];
        if (first.empty() && !L.missing.empty()) first = "l" + std::to_string(li) + "." + L.missing[0];
        n += L.missing.size();
    }
    if (n) vmx_set_error("larolorn: %zu tensors not loaded, first `%s`", n, first.c_str());
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

// m->y = mixer(x)
int latent_attention(vmx_larolorn *m, Layer &L, const Layer &w, const Step &s) {
    const vmx_larolorn_layer_config &lc = L.c;
    const int W = m->cfg.width, T = s.T, f32 = m->f32() ? 1 : 0, cdt = f32 ? VMX_F32 : VMX_BF16;
    const int H = lc.heads, D = lc.dim, RD = lc.rot_dim, R = lc.kv_rank, V = lc.vdim, nf = w.nf;
    float *fused = m->fused.as<float>();
    if (int rc = vmx_linear_launch(product(m->input(), f32, W, w.wfused, nf, fused, 1, T, f32), s.st)) return rc;   // q | latent, key part | head gates
    vmx_latent_prepare p = {};   // the latent normed, the key part rotated, the cache row written; the heads' rotated query parts
    p.kv = fused + w.dkv_off, p.ldkv = nf, p.latent_norm_bf16 = w.dkv_norm.as<uint16_t>(), p.eps = m->cfg.norm_eps;
    if (RD > 0) p.q = fused + w.q_off, p.ldq = nf, p.heads = H, p.dim = D, p.q_rot = m->q.as<float>();
    p.kv_rank = R, p.rot_dim = RD, p.inv_freq = w.rot_steps.as<float>(), p.rot_dims = lc.rot.dims, p.rot_mul = w.rot_mul;
    if (int rc = vmx_latent_prepare_rows(&p, s.positions, s.slots, L.cache.p, cdt, nullptr, T, s.st)) return rc;
    if (D > 0) {    // qa_h = U_h^T q_h: per head, [T, D] x [D, R]
        VmxLinear a;
        a.A = fused + w.q_off, a.a_f32 = 1, a.lda = nf, a.a_bs = D + RD;
        a.W = w.uk_t.as<uint16_t>(), a.w_sn = D, a.w_sk = 1, a.w_bs = (int64_t)D * R;
        a.C = m->qabs.p, a.c_f32 = 1, a.ldc = (int64_t)H * R, a.c_bs = R;
        a.M = T, a.N = R, a.K = D, a.batch = H, a.exact = f32;
        if (int rc = vmx_linear_launch(a, s.st)) return rc;
    } else {
        if (int rc = vmx_zero_f32(m->qabs.as<float>(), (int64_t)T * H * R, s.st)) return rc;
    }
    if (int rc = vmx_latent_attention(m->olat.as<float>(), m->qabs.as<float>(), m->q.as<float>(), L.cache.p, cdt, s.block_tables, s.max_blocks, s.seq_ids,
                                      s.positions, nullptr, lc.scale, lc.mask, T, H, R, RD, m->cfg.block_size, m->attn_ws.p, m->attn_ws.bytes, s.st))
        return rc;
    VmxLinear v;    // V_h o_h times the head's sigmoid: per head, [T, R] x [V, R]^T
    v.A = m->olat.p, v.a_f32 = 1, v.lda = (int64_t)H * R, v.a_bs = R;
    v.W = w.uv.as<uint16_t>(), v.w_sn = R, v.w_sk = 1, v.w_bs = (int64_t)V * R;
    v.C = m->attn.p, v.c_f32 = f32, v.ldc = (int64_t)H * V, v.c_bs = V;
    v.M = T, v.N = V, v.K = R, v.batch = H, v.exact = f32;
    v.epilogue = VMX_EP_MUL_SIGMOID, v.aux = fused + w.g_off, v.ldaux = nf, v.aux_sn = 0, v.aux_bs = 1;
    if (int rc = vmx_linear_launch(v, s.st)) return rc;
    return vmx_linear_launch(product(m->attn, f32, H * V, w.wo, W, m->y.p, 1, T, f32), s.st);
}

// m->y, m->side = the two branches ahead of their norms
int chunked_lightning(vmx_larolorn *m, Layer &L, const Layer &w, const Step &s) {
    const vmx_larolorn_layer_config &lc = L.c;
    const int W = m->cfg.width, T = s.T, f32 = m->f32() ? 1 : 0, cdt = f32 ? VMX_F32 : VMX_BF16, nf = w.nf;
    const int H = lc.heads, G = lc.kv_heads, D = lc.dim, V = lc.vdim, RH = lc.r_heads, RD = lc.r_dim, RV = lc.r_vdim;
    float *fused = m->fused.as<float>();
    VmxLinear p = product(m->input(), f32, W, w.wfused, nf, fused, 1, T, f32);   // q | k | v | SiLU of the memory's q | k | v | read-out gate
    p.bias = w.bias.as<uint16_t>();
    p.silu_begin = w.rq_off, p.silu_end = w.g_off;
    if (int rc = vmx_linear_launch(p, s.st)) return rc;
    // left: attention inside the chunk
    const vmx_qk_prepare_opts po = {0, 1, w.rot_mul, 1.0f, 1.0f, nullptr, 0};
    if (int rc = vmx_qk_prepare_ex(m->q.as<float>(), fused + w.q_off, nf, H * D, fused + w.k_off, nf, G * D, fused + w.v_off, nf, G * V,
                                   w.qnorm.as<uint16_t>(), w.knorm.as<uint16_t>(), m->cfg.norm_eps, w.rot_steps.as<float>(), lc.rot.dims, D, s.positions,
                                   s.slots, L.cache.p, L.vcache.p, cdt, T, &po, s.st))
        return rc;
    vmx_window_attn_extras ex = {};
    ex.sink_bf16 = w.sink.as<uint16_t>(), ex.chunk = lc.mask;
    if (int rc = vmx_window_attention_ex(m->attn.p, cdt, m->q.as<float>(), (int64_t)H * D, L.cache.p, L.vcache.p, cdt, s.block_tables, s.max_blocks,
                                         s.seq_ids, s.positions, nullptr, nullptr, 0, lc.scale, 0.f, 0, 0, T, H, G, D, V, m->cfg.block_size,
                                         s.seq_starts, s.num_seqs, m->attn_ws.p, m->attn_ws.bytes, &ex, s.st))
        return rc;
    VmxLinear o = product(m->attn, f32, H * V, w.wo, W, m->y.p, 1, T, f32);
    o.bias = w.bias_o.as<uint16_t>();
    if (int rc = vmx_linear_launch(o, s.st)) return rc;
    // right: S <- decay S + k v^T, o = S^T q
    const vmx_matrix_memory_opts mo = {nullptr, 0, nullptr, 0, f32 ? 0 : 1, T};
    if (int rc = vmx_matrix_memory_recurrence_ex(m->readout.as<float>(), (int64_t)RH * RV, fused + w.rq_off, nf, 1.0f, fused + w.rk_off, nf,
                                                 fused + w.rv_off, nf, w.decay.as<float>(), 0, 1, nullptr, 0, L.memory.as<float>(), s.positions,
                                                 s.seq_starts, s.state_slots, s.num_seqs, RH, RH, RD, RV, &mo, s.st))
        return rc;
    const vmx_read_out_opts ro = {};   // all heads of a token are one normed row
    if (int rc = vmx_head_read_out(m->rec.p, cdt, m->readout.as<float>(), (int64_t)RH * RV, w.read_norm.as<uint16_t>(), fused + w.g_off, nf,
                                   m->cfg.norm_eps, T, 1, RH * RV, &ro, s.st))
        return rc;
    return vmx_linear_launch(product(m->rec, f32, RH * RV, w.wo_right, W, m->side.p, 1, T, f32), s.st);
}

// m->y = ff(x)
int clamped_glu(vmx_larolorn *m, const Layer &w, const Step &s) {
    const int W = m->cfg.width, F = w.c.ff, f32 = m->f32() ? 1 : 0;
    if (int rc = vmx_linear_launch(product(m->input(), f32, W, w.wgu, 2 * F, m->fused.p, 1, s.T, f32), s.st)) return rc;
    if (int rc = vmx_glu_clamped_rows(m->act.p, f32, m->fused.as<float>(), s.T, F, GLU_SLOPE, w.c.limit, s.st)) return rc;
    return vmx_linear_launch(product(m->act, f32, F, w.wdown, W, m->y.p, 1, s.T, f32), s.st);
}

}  // namespace

extern "C" int vmx_larolorn_forward(vmx_larolorn *m, const int32_t *tokens, const int32_t *positions, const int32_t *slots, const int32_t *seq_ids,
                                    int num_tokens, const int32_t *block_tables, int num_seqs, int max_blocks_per_seq, const int32_t *seq_starts,
                                    const int32_t *state_slots, const int32_t *logit_rows, int num_logit_rows, float *logits, int32_t *greedy_ids,
                                    float *layer_trace, void *stream) {
    VMX_REQUIRE(m && tokens && positions && slots && seq_ids && block_tables && seq_starts && state_slots, "larolorn_forward: null pointer");
    const vmx_larolorn_config &c = m->cfg;
    VMX_REQUIRE(num_tokens >= 1 && num_tokens <= c.max_tokens, "larolorn_forward: %d tokens, the model was created for at most %d", num_tokens,
                c.max_tokens);
    VMX_REQUIRE(num_seqs >= 1 && num_seqs <= c.max_seqs && max_blocks_per_seq >= 1, "larolorn_forward: bad sequence count or block-table shape");
    VMX_REQUIRE(num_logit_rows >= 0 && num_logit_rows <= num_tokens && (num_logit_rows == 0 || (logit_rows && (logits || greedy_ids))),
                "larolorn_forward: bad logit rows");
    if (vmx_larolorn_missing_tensors(m) != 0) return VMX_EINVAL;
    const Step s{positions, slots, seq_ids, block_tables, seq_starts, state_slots, num_tokens, num_seqs, max_blocks_per_seq, vmx_stream(stream)};
    hipStream_t st = s.st;
    const int T = num_tokens, W = c.width, f32 = m->f32() ? 1 : 0;
    float *x = m->x.as<float>();
    VmxSandwich base;
    base.x = x, base.h = m->h.p, base.copy_h = !f32, base.width = W, base.eps = c.norm_eps, base.centered = 0;
    VmxSandwich in = base;    // x = embed[token]
    in.embed = m->embed.as<uint16_t>(), in.tokens = tokens, in.vocab = c.vocab, in.accumulate = 0;
    if (int rc = vmx_sandwich_norm(in, T, st)) return rc;
    base.y = m->y.as<float>(), base.post_mul = c.residual_mult;
    for (int li = 0; li < c.num_layers; li++) {
        Layer &L = m->layers[li];
        const Layer &w = m->weights(L);
        VmxSandwich sw = base;
        sw.w_post = w.norm1.as<uint16_t>();
        if (L.c.mixer == VMX_MIXER_LATENT_ATTENTION) {
            if (int rc = latent_attention(m, L, w, s)) return rc;
        } else {
            if (int rc = chunked_lightning(m, L, w, s)) return rc;
            sw.side = m->side.as<float>(), sw.w_y = w.left_out.as<uint16_t>(), sw.w_side = w.right_out.as<uint16_t>(), sw.side_mul = 0.5f;
        }
        if (int rc = vmx_sandwich_norm(sw, T, st)) return rc;
        if (L.c.mlp != VMX_MLP_NONE) {
            if (int rc = clamped_glu(m, w, s)) return rc;
            VmxSandwich sf = base;
            sf.w_post = w.norm2.as<uint16_t>();
            if (int rc = vmx_sandwich_norm(sf, T, st)) return rc;
        }
        if (layer_trace)
            VMX_CHECK_HIP(hipMemcpyAsync(layer_trace + (size_t)li * T * W, x, (size_t)T * W * 4, hipMemcpyDeviceToDevice, st));
    }
    if (num_logit_rows > 0) {
        if (int rc = vmx_rms_norm_f32in(m->hsel.p, f32, x, logit_rows, m->final_norm.as<uint16_t>(), 0, W, c.norm_eps, num_logit_rows, st)) return rc;
        float *lg = logits ? logits : m->fused.as<float>();   // greedy ids only: the logits live in a workspace
        VmxLinear hd = product(m->hsel, f32, W, m->head, c.vocab, lg, 1, num_logit_rows, f32);
        hd.out_scale = c.logit_scale;
        if (int rc = vmx_linear_launch(hd, st)) return rc;
        if (greedy_ids)
            if (int rc = vmx_argmax_f32_rows(greedy_ids, m->argmax_keys.as<unsigned long long>(), lg, num_logit_rows, c.vocab, st)) return rc;
    }
    return VMX_OK;
}
