// Linear recurrences over a matrix memory per head, as recurrent token mixers over packed steps (the gated delta rule with one
// decay per key channel or per head; the plain decayed outer-product memory of gated linear attention and retention), and the
// short causal convolution in front of the delta rule.  Both carry state from step to step in a SLOT per sequence (the caller's state-slot manager hands
// them out); a sequence whose step starts at position 0 starts from zeros whatever its slot held before.
//
// Short convolution (vmx_short_conv_silu): y[t, c] = silu(sum_s taps[c, n - 1 - s] * x[t - s, c]), zeros before the sequence's
// first token.  The last n - 1 inputs of every sequence are its state [slots, n - 1, channels] (f32); inputs older than the step
// come from there.  A group of channels (one head's query or key) may then be scaled to a unit vector, x / sqrt(sum x^2 + eps),
// times a constant.  vmx_short_conv_state_update moves the state on after all of a step's rows were read.
//
// Recurrence (vmx_gated_delta_rule), per head with a matrix memory S [dim, vdim] in f32:
//   S <- diag(g_t) S;   u = beta_t (v_t - S^T k_t);   S <- S + k_t u^T;   o_t = S^T q_t
// so a token reads the memory after its own write (computed as (g S)^T q + u (k . q), the same sum in another order).  The decay
// g_t is a number per key channel, or one per head (per token, or a constant of the head: row stride 0); without beta the write
// is the plain outer product, u = v_t (S <- diag(g_t) S + k_t v_t^T: gated linear attention, retention), optionally times a number
// per head and token (the write gain of a memory with an input gate).  A NORMALISER may ride along as one more value column that
// is 1 for every token: n <- g n + gain k, read out as n . q per head.  Query/key
// head of value head h: h / (heads / qk_heads).  A workgroup owns 16 value columns of one (sequence, head) and walks the
// sequence's tokens of the step in order; 16 threads share a column, each holding every 16th row of S in registers, and the
// column sums per token are 16-lane butterflies.  The state slot keeps S in the workgroup's own register order (the layout is
// private to this file), so that loading and storing it is coalesced.  Prompts of the plain memory with one decay per head have a
// chunked form on the matrix cores below, over the same state layout.
//
// Exponential gates (vmx_exp_gate_scan): a memory whose input gate is an exponential keeps the logarithm of its scale, a running
// maximum m_t = max(f_t + m_(t-1), i_t) per head (from 0), in its slot; what the recurrence needs are the decay
// exp(f_t + m_(t-1) - m_t), the write gain exp(i_t - m_t) and, for the read-out, exp(-m_t).  The maximum is a prefix scan over
// (sum of f, largest of "i plus the f after it") pairs: one workgroup per (sequence, head), 256 tokens a round.
#include "vmx_kernels.h"

namespace {

__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return z > 20.f ? z : log1pf(expf(z)); }

struct ConvArgs {
    const float *x;          // [tokens, ldx] inputs of the step, channels at column 0
    int64_t ldx;
    const uint16_t *taps;    // bf16 [channels, n]
    float *state;            // [slots, n - 1, channels]
    float *y;                // [tokens, ldy]
    int64_t ldy;
    const int32_t *positions, *seq_ids, *seq_starts, *state_slots;
    int tokens, channels, n;
    // unit-vector groups: channels [0, unit_groups * group) are groups of `group` channels; groups < scaled_groups also get `mul`
    int group, unit_groups, scaled_groups;
    float unit_eps, mul;
};

// one wave per (token, run of `group` channels); runs past the unit groups are plain 64-channel runs
__global__ __launch_bounds__(256) void short_conv_silu_kernel(const ConvArgs a) {
    const int t = blockIdx.x, lane = threadIdx.x & 63;   // tokens on x (no 65535 limit)
    const int run = blockIdx.y * 4 + (threadIdx.x >> 6);
    const int unit_ch = a.unit_groups * a.group;
    int c0, c1;
    bool unit = false;
    if (run < a.unit_groups) c0 = run * a.group, c1 = c0 + a.group, unit = true;
    else c0 = unit_ch + (run - a.unit_groups) * 64, c1 = min(c0 + 64, a.channels);
    if (c0 >= a.channels) return;
    const int pos = a.positions[t], seq = a.seq_ids[t];
    const int first = a.seq_starts[seq];             // packed row of the sequence's first token in this step
    const int start = pos - (t - first);             // position of that token
    const float *st = a.state + (int64_t)a.state_slots[seq] * (a.n - 1) * a.channels;
    auto conv_at = [&](int c) {
        float acc = 0.f;
        for (int s = a.n - 1; s >= 0; s--) {         // oldest input first
            const int q = pos - s;
            if (q < 0) continue;
            const float xv = q >= start ? a.x[(int64_t)(t - s) * a.ldx + c] : st[(int64_t)(q - start + a.n - 1) * a.channels + c];
            acc = fmaf(vmx_bf16_to_f32(a.taps[(int64_t)c * a.n + (a.n - 1 - s)]), xv, acc);
        }
        return silu_f(acc);
    };
    constexpr int HOLD = 4;                          // a lane's outputs of a run of up to 256 channels stay in registers
    float held[HOLD], ss = 0.f;
#pragma unroll
    for (int i = 0; i < HOLD; i++) {
        const int c = c0 + lane + 64 * i;
        held[i] = c < c1 ? conv_at(c) : 0.f;
        ss = fmaf(held[i], held[i], ss);
    }
    for (int c = c0 + lane + 64 * HOLD; c < c1; c += 64) {   // wider runs go through memory
        const float yv = conv_at(c);
        a.y[(int64_t)t * a.ldy + c] = yv;
        ss = fmaf(yv, yv, ss);
    }
    float f = 1.0f;
    if (unit) f = (run < a.scaled_groups ? a.mul : 1.0f) / sqrtf(vmx_wave_sum(ss) + a.unit_eps);
#pragma unroll
    for (int i = 0; i < HOLD; i++) {
        const int c = c0 + lane + 64 * i;
        if (c < c1) a.y[(int64_t)t * a.ldy + c] = held[i] * f;
    }
    if (unit)
        for (int c = c0 + lane + 64 * HOLD; c < c1; c += 64) a.y[(int64_t)t * a.ldy + c] *= f;   // each lane rescales what it wrote itself
}

// state[slot] <- the last n - 1 inputs of the sequence after this step.  A thread owns one (sequence, channel) and goes through
// the state rows in ascending order: row r takes the input of position end - (n - 1) + r, which is a row of the step or an OLDER
// state row r + count (not overwritten yet).
__global__ __launch_bounds__(256) void short_conv_state_kernel(const ConvArgs a, int num_seqs) {
    const int seq = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
    if (c >= a.channels) return;
    const int first = a.seq_starts[seq], count = a.seq_starts[seq + 1] - first;
    if (count <= 0) return;
    const int start = a.positions[first];
    float *st = a.state + (int64_t)a.state_slots[seq] * (a.n - 1) * a.channels;
    for (int r = 0; r < a.n - 1; r++) {
        const int q = start + count - (a.n - 1) + r;
        float v = 0.f;
        if (q >= start) v = a.x[(int64_t)(first + q - start) * a.ldx + c];
        else if (q >= 0) v = st[(int64_t)(r + count) * a.channels + c];
        st[(int64_t)r * a.channels + c] = v;
    }
}

// g[t, c] <- exp(-exp(A_log[c / dim]) * softplus(g[t, c] + dt_bias[c])) in place, and beta[t, h] <- sigmoid(beta[t, h]) in place
__global__ __launch_bounds__(256) void delta_gates_kernel(float *__restrict__ g, int64_t ldg, const uint16_t *__restrict__ a_log,
                                                           const uint16_t *__restrict__ dt_bias, float *__restrict__ beta, int64_t ldbeta,
                                                           int heads, int dim) {
    const int t = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
    if (c < heads * dim) {
        const float rate = expf(vmx_bf16_to_f32(a_log[c / dim]));
        const float dt = softplus_f(g[(int64_t)t * ldg + c] + vmx_bf16_to_f32(dt_bias[c]));
        g[(int64_t)t * ldg + c] = expf(-rate * dt);
    }
    if (c < heads) beta[(int64_t)t * ldbeta + c] = sigmoid_f(beta[(int64_t)t * ldbeta + c]);
}

// g[t, c] <- sigmoid(g[t, c])^(1 / tau) in place, through the logarithm: exp(-softplus(-z) / tau)
__global__ __launch_bounds__(256) void sigmoid_root_decay_kernel(float *__restrict__ g, int64_t ldg, int n, float inv_tau) {
    const int t = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
    if (c < n) g[(int64_t)t * ldg + c] = expf(-softplus_f(-g[(int64_t)t * ldg + c]) * inv_tau);
}

struct DeltaArgs {
    const float *q, *k, *v, *g, *beta;       // rows of the step: q, k [qk_heads * dim], v [heads * vdim], g [heads * dim], beta [heads]
    int64_t ldq, ldk, ldv, ldg, ldbeta;
    float *o;                                // [tokens, heads * vdim]
    int64_t ldo;
    float *state;                            // [slots, heads, tiles, DPT, 256]
    const int32_t *positions, *seq_starts, *state_slots;
    int heads, qk_heads, dim, vdim;
    int g_per_head;                          // g rows hold one decay per head (ldg 0: the same row for every token) instead of heads * dim
    int plain;                               // u = beta v (beta NULL: u = v) instead of beta (v - S^T k)
    float q_mul;                             // the queries are multiplied by this constant as they are read
    float *norm;                             // [tokens, ldnorm] n . q per head: value column vdim is 1 for every token (NULL: no such column)
    int64_t ldnorm;
};

constexpr int DR_RS = 16, DR_VT = 16;   // row splits per column, columns per workgroup

// Tokens are staged in rounds of CT through two LDS buffers: the next round is requested into registers before the current one
// is walked and stored afterwards, so one barrier per round remains and the walk never waits for memory.  q, k and g are stored
// in thread order ([row split r][u] for row r + 8 u), so a thread reads its rows as 16-byte vectors.
template <int DPT>
__global__ __launch_bounds__(256) void gated_delta_rule_kernel(const DeltaArgs a) {
    constexpr int DP = DPT * DR_RS;          // padded key dimension
    constexpr int LDP = DPT == 4 ? 4 : DPT + 4;   // floats between two row splits in LDS: the 16 splits of a read fall on different banks
    constexpr int CT = 128 / DPT;            // tokens per round: long enough for the next round's loads to land while this one is walked
    constexpr int NL = CT * DP / 256;        // q / k / g elements a thread stages per round
    constexpr int NV = (CT * DR_VT + 255) / 256;
    constexpr int ROW = DR_RS * LDP;         // floats of one token's q (k, g) in LDS
    extern __shared__ __align__(16) float delta_lds[];   // delta_lds_bytes(DPT): q | k | g [2][CT][ROW], v [2][CT][16], beta [2][CT]
    float *sq = delta_lds, *sk = sq + 2 * CT * ROW, *sg = sk + 2 * CT * ROW, *sv = sg + 2 * CT * ROW, *sb = sv + 2 * CT * DR_VT;
    const int seq = blockIdx.z, h = blockIdx.y, tile = blockIdx.x, tid = threadIdx.x;
    const int first = a.seq_starts[seq], count = a.seq_starts[seq + 1] - first;
    if (count <= 0) return;
    const int r = tid & (DR_RS - 1), cl = tid >> 4, c = tile * DR_VT + cl;
    const int qh = h / (a.heads / a.qk_heads);
    const int tiles = gridDim.x;
    float *sp = a.state + ((((int64_t)a.state_slots[seq] * a.heads + h) * tiles + tile) * DPT) * 256 + tid;
    float S[DPT];
    const bool fresh = a.positions[first] == 0;
#pragma unroll
    for (int u = 0; u < DPT; u++) S[u] = fresh ? 0.f : sp[(int64_t)u * 256];
    float rq[NL], rk[NL], rg[NL], rv[NV], rb = 0.f;
    auto request = [&](int t0) {
        const int ct = min(CT, count - t0);
#pragma unroll
        for (int j = 0; j < NL; j++) {
            const int i = tid + 256 * j, tt = i / DP, d = i % DP;
            const int64_t row = first + t0 + tt;
            const bool in = tt < ct && d < a.dim;
            rq[j] = in ? a.q[row * a.ldq + (int64_t)qh * a.dim + d] * a.q_mul : 0.f;
            rk[j] = in ? a.k[row * a.ldk + (int64_t)qh * a.dim + d] : 0.f;
            rg[j] = in ? a.g[row * a.ldg + (a.g_per_head ? (int64_t)h : (int64_t)h * a.dim + d)] : 1.f;
        }
#pragma unroll
        for (int j = 0; j < NV; j++) {
            const int i = tid + 256 * j, tt = i / DR_VT, cc = tile * DR_VT + i % DR_VT;
            rv[j] = (tt < ct && cc < a.vdim) ? a.v[(int64_t)(first + t0 + tt) * a.ldv + (int64_t)h * a.vdim + cc] : (cc == a.vdim && a.norm ? 1.f : 0.f);
        }
        rb = (tid < ct && a.beta) ? a.beta[(int64_t)(first + t0 + tid) * a.ldbeta + h] : 1.f;
    };
    auto stage = [&](int b) {
#pragma unroll
        for (int j = 0; j < NL; j++) {
            const int i = tid + 256 * j, tt = i / DP, d = i % DP, at = (d & (DR_RS - 1)) * LDP + (d >> 4);   // row d = r + 16 u -> [r][u]
            sq[(b * CT + tt) * ROW + at] = rq[j];
            sk[(b * CT + tt) * ROW + at] = rk[j];
            sg[(b * CT + tt) * ROW + at] = rg[j];
        }
#pragma unroll
        for (int j = 0; j < NV; j++) {
            const int i = tid + 256 * j;
            if (i < CT * DR_VT) sv[b * CT * DR_VT + i] = rv[j];
        }
        if (tid < CT) sb[b * CT + tid] = rb;
    };
    request(0);
    stage(0);
    __syncthreads();
    int b = 0;
    for (int t0 = 0; t0 < count; t0 += CT, b ^= 1) {
        const int ct = min(CT, count - t0);
        const bool more = t0 + CT < count;
        if (more) request(t0 + CT);
        // The read-out is taken from the decayed memory: o = (gS)^T q + u (k . q), so the three column sums of a token, (gS)^T k,
        // (gS)^T q and k . q, are independent chains and the write S += k u^T leaves the critical path.  The LDS reads of the next
        // token are issued before the current one is worked on (two register sets, A and B).
        auto ld = [&](int tt, float (&kk)[DPT], float (&gg)[DPT], float (&qq)[DPT], float &bv, float &vv) {
#pragma unroll
            for (int u = 0; u < DPT; u += 4) {
                const float4 k4 = *reinterpret_cast<const float4 *>(sk + (b * CT + tt) * ROW + r * LDP + u);
                const float4 g4 = *reinterpret_cast<const float4 *>(sg + (b * CT + tt) * ROW + r * LDP + u);
                const float4 q4 = *reinterpret_cast<const float4 *>(sq + (b * CT + tt) * ROW + r * LDP + u);
                kk[u] = k4.x, kk[u + 1] = k4.y, kk[u + 2] = k4.z, kk[u + 3] = k4.w;
                gg[u] = g4.x, gg[u + 1] = g4.y, gg[u + 2] = g4.z, gg[u + 3] = g4.w;
                qq[u] = q4.x, qq[u + 1] = q4.y, qq[u + 2] = q4.z, qq[u + 3] = q4.w;
            }
            bv = sb[b * CT + tt];
            vv = sv[(b * CT + tt) * DR_VT + cl];
        };
        auto step = [&](int tt, const float (&kk)[DPT], const float (&gg)[DPT], const float (&qq)[DPT], float bv, float vv) {
            float pk = 0.f, pq = 0.f, kq = 0.f;
#pragma unroll
            for (int u = 0; u < DPT; u++) {
                S[u] *= gg[u];
                pk = fmaf(S[u], kk[u], pk);
                pq = fmaf(S[u], qq[u], pq);
                kq = fmaf(kk[u], qq[u], kq);
            }
            pk += vmx_dpp<VMX_DPP_XOR1>(pk), pq += vmx_dpp<VMX_DPP_XOR1>(pq), kq += vmx_dpp<VMX_DPP_XOR1>(kq);
            pk += vmx_dpp<VMX_DPP_XOR2>(pk), pq += vmx_dpp<VMX_DPP_XOR2>(pq), kq += vmx_dpp<VMX_DPP_XOR2>(kq);
            pk += vmx_dpp<VMX_DPP_HALF_MIRROR>(pk), pq += vmx_dpp<VMX_DPP_HALF_MIRROR>(pq), kq += vmx_dpp<VMX_DPP_HALF_MIRROR>(kq);
            pk += vmx_dpp<VMX_DPP_ROR8>(pk), pq += vmx_dpp<VMX_DPP_ROR8>(pq), kq += vmx_dpp<VMX_DPP_ROR8>(kq);
            const float uu = bv * (a.plain ? vv : vv - pk);
            if (r == 0) {
                if (c < a.vdim) a.o[(int64_t)(first + t0 + tt) * a.ldo + (int64_t)h * a.vdim + c] = fmaf(uu, kq, pq);
                else if (c == a.vdim && a.norm) a.norm[(int64_t)(first + t0 + tt) * a.ldnorm + h] = fmaf(uu, kq, pq);
            }
#pragma unroll
            for (int u = 0; u < DPT; u++) S[u] = fmaf(kk[u], uu, S[u]);
        };
        float kA[DPT], gA[DPT], qA[DPT], kB[DPT], gB[DPT], qB[DPT], bA, vA, bB = 0.f, vB = 0.f;
        ld(0, kA, gA, qA, bA, vA);
        for (int tt = 0; tt < ct; tt += 2) {
            if (tt + 1 < ct) ld(tt + 1, kB, gB, qB, bB, vB);
            step(tt, kA, gA, qA, bA, vA);
            if (tt + 1 < ct) {
                if (tt + 2 < ct) ld(tt + 2, kA, gA, qA, bA, vA);
                step(tt + 1, kB, gB, qB, bB, vB);
            }
        }
        if (more) stage(b ^ 1);
        __syncthreads();
    }
#pragma unroll
    for (int u = 0; u < DPT; u++) sp[(int64_t)u * 256] = S[u];
}

// ---------------------------------------------------------------------------------------------------------------------------
// Chunked matrix-core form of the plain memory with one decay per head (S <- g_t S + a_t k_t v_t^T), for prompts.  A workgroup owns
// the same 16 value columns of one (sequence, head) as above and walks the sequence's tokens of the step 64 at a time; with
// L_t = sum of log g up to token t of the chunk and S the memory ahead of it,
//   o_t = e^(L_t) S^T q_t + sum_(s <= t) a_s e^(L_t - L_s) (q_t . k_s) v_s
//   S  <- e^(L_C) S + sum_s k_s (a_s e^(L_C - L_s) v_s)^T
// are four small products per chunk (v_mfma_f32_16x16x32_bf16).  q, k and v are rounded to bf16; everything else is f32: a number
// that is not a bf16 enters a product as the sum of three bf16 parts (24 bits), so the memory, the weighted scores and the weighted
// values keep f32 precision.  L is summed in double (a chunk may cross decays of e^-80, whose differences still count).
// Wave w takes tokens 16 w .. 16 w + 15 of the first two products and rows w, w + 4, ... of 16 of the memory in the last.
constexpr int MC_C = 64, MC_LD = MC_C + 8;

struct MemoryChunkLds {   // offsets in bytes
    int q, k, p, v, wv, s, gates, total, dp, ldq, ldk;
};
__host__ __device__ constexpr MemoryChunkLds memory_chunk_lds(int dt) {
    MemoryChunkLds l{};
    l.dp = 16 * dt, l.ldq = l.dp + 8, l.ldk = l.dp + 32;
    l.q = 0;
    l.k = l.q + MC_C * l.ldq * 2;
    l.p = l.k + MC_C * l.ldk * 2;
    l.v = l.p + 3 * MC_C * MC_LD * 2;
    l.wv = l.v + 16 * MC_LD * 2;
    l.s = l.wv + 3 * 16 * MC_LD * 2;
    l.gates = l.s + 3 * 16 * l.ldq * 2;
    l.total = l.gates + 2 * MC_C * (8 + 3 * 4) + 2 * 4;
    return l;
}
typedef short mc_s16x4 __attribute__((ext_vector_type(4)));
typedef short mc_s16x8 __attribute__((ext_vector_type(8)));

__device__ __forceinline__ void mc_split(float x, uint16_t (&p)[3]) {   // x = p0 + p1 + p2 to 24 bits
#pragma unroll
    for (int i = 0; i < 3; i++) {
        p[i] = vmx_f32_to_bf16(x);
        x -= vmx_bf16_to_f32(p[i]);
    }
}
__device__ __forceinline__ vmx_f32x4 mc_mfma(const uint4 a, const uint4 b, vmx_f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(vmx_bf16x8, a), __builtin_bit_cast(vmx_bf16x8, b), c, 0, 0, 0);
}

template <int DT> __global__ __launch_bounds__(256) void memory_chunk_kernel(const DeltaArgs a) {
    constexpr MemoryChunkLds l = memory_chunk_lds(DT);
    constexpr int DP = l.dp, NQ = MC_C * DP / 4 / 256, ST = DT / 4, KS = DP / 32;
    extern __shared__ __align__(16) unsigned char mc_lds[];
    uint16_t *Q = (uint16_t *)(mc_lds + l.q), *K = (uint16_t *)(mc_lds + l.k), *P = (uint16_t *)(mc_lds + l.p), *V = (uint16_t *)(mc_lds + l.v),
             *WV = (uint16_t *)(mc_lds + l.wv), *SS = (uint16_t *)(mc_lds + l.s);
    double *gl = (double *)(mc_lds + l.gates);                    // [2][C] L
    float *ga = (float *)(gl + 2 * MC_C), *gw = ga + 2 * MC_C, *gc = gw + 2 * MC_C, *gt = gc + 2 * MC_C;   // [2][C] a, a e^(L_C - L), e^L; [2] e^(L_C)
    const int seq = blockIdx.z, h = blockIdx.y, tile = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, fl = lane & 15, fg = lane >> 4;
    const int first = a.seq_starts[seq], count = a.seq_starts[seq + 1] - first;
    if (count <= 0) return;
    const int qh = h / (a.heads / a.qk_heads);
    const float *qp = a.q + (int64_t)first * a.ldq + (int64_t)qh * a.dim, *kp = a.k + (int64_t)first * a.ldk + (int64_t)qh * a.dim;
    const float *vp = a.v + (int64_t)first * a.ldv + (int64_t)h * a.vdim;
    const bool vec = (a.dim & 3) == 0 && (a.ldq & 3) == 0 && (a.ldk & 3) == 0 && (((uintptr_t)qp | (uintptr_t)kp) & 15) == 0;
    // ---- what a thread stages: NQ groups of four q / k channels, four value columns of one token, and (wave 0) a token's gates
    float4 rq[NQ], rk[NQ];
    float rv[4], g1 = 1.f, a1 = 0.f;
    const int vt = tid >> 2, vc = 4 * (tid & 3);
    auto four = [&](const float *p, int64_t ld, int t, int d) {
        if (t >= count || d >= a.dim) return make_float4(0.f, 0.f, 0.f, 0.f);
        p += (int64_t)t * ld + d;
        if (vec) return *reinterpret_cast<const float4 *>(p);
        return make_float4(p[0], d + 1 < a.dim ? p[1] : 0.f, d + 2 < a.dim ? p[2] : 0.f, d + 3 < a.dim ? p[3] : 0.f);
    };
    auto request = [&](int t0) {
#pragma unroll
        for (int j = 0; j < NQ; j++) {
            const int i = tid + 256 * j, t = t0 + i / (DP / 4), d = 4 * (i % (DP / 4));
            rq[j] = four(qp, a.ldq, t, d);
            rk[j] = four(kp, a.ldk, t, d);
        }
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int c = tile * DR_VT + vc + e;
            rv[e] = t0 + vt >= count ? 0.f : (c < a.vdim ? vp[(int64_t)(t0 + vt) * a.ldv + c] : (c == a.vdim && a.norm ? 1.f : 0.f));
        }
    };
    auto request_gates = [&](int t0) {   // wave 0
        const int t = t0 + lane;
        g1 = t < count ? a.g[(int64_t)(first + t) * a.ldg + h] : 1.f;
        a1 = t < count ? (a.beta ? a.beta[(int64_t)(first + t) * a.ldbeta + h] : 1.f) : 0.f;
    };
    auto scan_gates = [&](int b) {       // wave 0: L and what follows from it for the chunk whose gates it holds
        double L = log((double)fmaxf(g1, 1e-37f));
#pragma unroll
        for (int d = 1; d < 64; d <<= 1) {
            const double p = __shfl_up(L, d, 64);
            if (lane >= d) L += p;
        }
        const double end = __shfl(L, 63, 64);
        gl[b * MC_C + lane] = L;
        ga[b * MC_C + lane] = a1;
        gw[b * MC_C + lane] = a1 * expf((float)(end - L));
        gc[b * MC_C + lane] = expf((float)L) * a.q_mul;
        if (lane == 0) gt[b] = expf((float)end);
    };
    auto store4 = [](uint16_t *dst, const float4 f) {
        *reinterpret_cast<uint2 *>(dst) = make_uint2((uint32_t)vmx_f32_to_bf16(f.x) | ((uint32_t)vmx_f32_to_bf16(f.y) << 16),
                                                     (uint32_t)vmx_f32_to_bf16(f.z) | ((uint32_t)vmx_f32_to_bf16(f.w) << 16));
    };
    float vv[4];
    auto stage = [&]() {
#pragma unroll
        for (int j = 0; j < NQ; j++) {
            const int i = tid + 256 * j, t = i / (DP / 4), d = 4 * (i % (DP / 4));
            store4(Q + t * l.ldq + d, rq[j]);
            store4(K + t * l.ldk + d, rk[j]);
        }
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const uint16_t r = vmx_f32_to_bf16(rv[e]);
            V[(vc + e) * MC_LD + vt] = r;
            vv[e] = vmx_bf16_to_f32(r);
        }
    };
    // ---- the memory: rows 16 u + 4 fg + r (u = wave + 4 j), column fl, in registers; its three parts by column in LDS
    float *sp = a.state + ((((int64_t)a.state_slots[seq] * a.heads + h) * gridDim.x + tile) * DT) * 256 + fl * 16 + 4 * fg;
    const bool fresh = a.positions[first] == 0;
    vmx_f32x4 S[ST];
    auto split_memory = [&]() {
#pragma unroll
        for (int j = 0; j < ST; j++) {
            uint16_t p[4][3];
#pragma unroll
            for (int r = 0; r < 4; r++) mc_split(S[j][r], p[r]);
#pragma unroll
            for (int i = 0; i < 3; i++)
                *reinterpret_cast<uint2 *>(SS + (i * 16 + fl) * l.ldq + 16 * (wave + 4 * j) + 4 * fg) =
                    make_uint2((uint32_t)p[0][i] | ((uint32_t)p[1][i] << 16), (uint32_t)p[2][i] | ((uint32_t)p[3][i] << 16));
        }
    };
    request(0);
    if (wave == 0) request_gates(0);
#pragma unroll
    for (int j = 0; j < ST; j++) {
        const float4 f = fresh ? make_float4(0.f, 0.f, 0.f, 0.f) : *reinterpret_cast<const float4 *>(sp + (wave + 4 * j) * 256);
        S[j] = vmx_f32x4{f.x, f.y, f.z, f.w};
    }
    split_memory();
    for (int i = tid; i < 3 * MC_C * MC_LD / 4; i += 256) reinterpret_cast<uint2 *>(P)[i] = make_uint2(0, 0);   // scores after the diagonal block stay 0
    stage();
    if (wave == 0) {
        scan_gates(0);
        request_gates(MC_C);
    }
    for (int t0 = 0, b = 0; t0 < count; t0 += MC_C, b ^= 1) {
        __syncthreads();
        const bool more = t0 + MC_C < count;
        if (more) request(t0 + MC_C);
        if (wave == 0 && more) {
            scan_gates(b ^ 1);
            request_gates(t0 + 2 * MC_C);
        }
        // values times their weight at the chunk's end, in three parts
        {
            const float w = gw[b * MC_C + vt];
#pragma unroll
            for (int e = 0; e < 4; e++) {
                uint16_t p[3];
                mc_split(w * vv[e], p);
#pragma unroll
                for (int i = 0; i < 3; i++) WV[(i * 16 + vc + e) * MC_LD + vt] = p[i];
            }
        }
        // scores of this wave's tokens against the chunk's keys up to them, weighted, in three parts
        uint4 qf[KS];
#pragma unroll
        for (int ks = 0; ks < KS; ks++) qf[ks] = *reinterpret_cast<const uint4 *>(Q + (16 * wave + fl) * l.ldq + 32 * ks + 8 * fg);
        double Lt[4];
#pragma unroll
        for (int r = 0; r < 4; r++) Lt[r] = gl[b * MC_C + 16 * wave + 4 * fg + r];
        for (int j = 0; j <= wave; j++) {
            vmx_f32x4 sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < KS; ks++) sc = mc_mfma(qf[ks], *reinterpret_cast<const uint4 *>(K + (16 * j + fl) * l.ldk + 32 * ks + 8 * fg), sc);
            const int sidx = 16 * j + fl;
            const double Ls = gl[b * MC_C + sidx];
            const float as = ga[b * MC_C + sidx] * a.q_mul;
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int t = 16 * wave + 4 * fg + r;
                uint16_t p[3];
                mc_split(sidx <= t ? sc[r] * as * expf((float)(Lt[r] - Ls)) : 0.f, p);
#pragma unroll
                for (int i = 0; i < 3; i++) P[(i * MC_C + t) * MC_LD + sidx] = p[i];
            }
        }
        // o = e^L q . S (the memory ahead of the chunk) + weighted scores . v
        vmx_f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 2; i >= 0; i--)
#pragma unroll
            for (int ks = 0; ks < KS; ks++) o = mc_mfma(qf[ks], *reinterpret_cast<const uint4 *>(SS + (i * 16 + fl) * l.ldq + 32 * ks + 8 * fg), o);
#pragma unroll
        for (int r = 0; r < 4; r++) o[r] *= gc[b * MC_C + 16 * wave + 4 * fg + r];
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");   // the wave's own rows of P
        for (int ks = 0; ks < (wave >> 1) + 1; ks++) {
            const uint4 vf = *reinterpret_cast<const uint4 *>(V + fl * MC_LD + 32 * ks + 8 * fg);
#pragma unroll
            for (int i = 2; i >= 0; i--) o = mc_mfma(*reinterpret_cast<const uint4 *>(P + (i * MC_C + 16 * wave + fl) * MC_LD + 32 * ks + 8 * fg), vf, o);
        }
        const int c = tile * DR_VT + fl;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int t = t0 + 16 * wave + 4 * fg + r;
            if (t < count) {
                if (c < a.vdim) a.o[(int64_t)(first + t) * a.ldo + (int64_t)h * a.vdim + c] = o[r];
                else if (c == a.vdim && a.norm) a.norm[(int64_t)(first + t) * a.ldnorm + h] = o[r];
            }
        }
        __syncthreads();
        // the memory after the chunk
        const float gall = gt[b];
#pragma unroll
        for (int j = 0; j < ST; j++)
#pragma unroll
            for (int r = 0; r < 4; r++) S[j][r] *= gall;
#pragma unroll
        for (int ks = 0; ks < MC_C / 32; ks++) {
            uint4 wf[3];
#pragma unroll
            for (int i = 0; i < 3; i++) wf[i] = *reinterpret_cast<const uint4 *>(WV + (i * 16 + fl) * MC_LD + 32 * ks + 8 * fg);
#pragma unroll
            for (int j = 0; j < ST; j++) {
                // A operand = K^T: the transposing LDS read hands lane n channel 16 u + n of the four tokens its 16-lane group addressed
                const uint16_t *src = K + (32 * ks + 8 * fg + (fl >> 2)) * l.ldk + 16 * (wave + 4 * j) + 4 * (fl & 3);
                const mc_s16x4 c0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((mc_s16x4 __attribute__((address_space(3))) *)src);
                const mc_s16x4 c1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((mc_s16x4 __attribute__((address_space(3))) *)(src + 4 * l.ldk));
                const uint4 kf = __builtin_bit_cast(uint4, mc_s16x8{c0[0], c0[1], c0[2], c0[3], c1[0], c1[1], c1[2], c1[3]});
#pragma unroll
                for (int i = 2; i >= 0; i--) S[j] = mc_mfma(kf, wf[i], S[j]);
            }
        }
        if (more) split_memory();
        __syncthreads();
        if (more) stage();
    }
#pragma unroll
    for (int j = 0; j < ST; j++) *reinterpret_cast<float4 *>(sp + (wave + 4 * j) * 256) = make_float4(S[j][0], S[j][1], S[j][2], S[j][3]);
}

// In place, one workgroup per (sequence, head): i[t, h] <- exp(i_t - m_t), f[t, h] <- exp(f_t + m_(t-1) - m_t), floor[t, h] = exp(-m_t)
// with i_t = cap tanh(i / cap), f_t = log(sigmoid(cap tanh(f / cap))) and m the running maximum (the slot's; 0 at position 0).
__global__ __launch_bounds__(256) void exp_gate_scan_kernel(float *__restrict__ ig, int64_t ldi, float *__restrict__ fg, int64_t ldf,
                                                             float *__restrict__ floor, int64_t ldfloor, float *__restrict__ m_state, float cap,
                                                             const int32_t *__restrict__ positions, const int32_t *__restrict__ seq_starts,
                                                             const int32_t *__restrict__ state_slots, int heads) {
    __shared__ float tot[2][4][2];     // the waves' totals of a round, double-buffered
    const int h = blockIdx.x, seq = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int first = seq_starts[seq], count = seq_starts[seq + 1] - first;
    if (count <= 0) return;
    float *ms = m_state + (int64_t)state_slots[seq] * heads + h;
    float m0 = positions[first] == 0 ? 0.f : *ms;
    float zi = tid < count ? ig[(int64_t)(first + tid) * ldi + h] : 0.f, zf = tid < count ? fg[(int64_t)(first + tid) * ldf + h] : 0.f;
    for (int t0 = 0, b = 0; t0 < count; t0 += 256, b ^= 1) {
        const bool in = t0 + tid < count;
        const int64_t row = first + t0 + tid;
        const float li = in ? cap * tanhf(zi / cap) : -1e30f;
        const float lf = in ? -softplus_f(-cap * tanhf(zf / cap)) : 0.f;
        if (t0 + 256 + tid < count) zi = ig[(row + 256) * ldi + h], zf = fg[(row + 256) * ldf + h];   // the next round's, while this one is scanned
        float A = lf, B = li;      // over the wave's tokens up to this lane's: sum of f; largest i plus the f after it
#pragma unroll
        for (int d = 1; d < 64; d <<= 1) {
            const float pa = __shfl_up(A, d, 64), pb = __shfl_up(B, d, 64);
            if (lane >= d) {
                B = fmaxf(pb + A, B);
                A += pa;
            }
        }
        if (lane == 63) tot[b][wave][0] = A, tot[b][wave][1] = B;
        __syncthreads();
        float before = m0, end = m0;   // the maximum ahead of this wave's first token, and after the round
#pragma unroll
        for (int w = 0; w < 4; w++) {
            if (w == wave) before = end;
            end = fmaxf(end + tot[b][w][0], tot[b][w][1]);
        }
        const float m = fmaxf(before + A, B), up = __shfl_up(m, 1, 64), prev = lane == 0 ? before : up;
        if (in) {
            ig[row * ldi + h] = expf(li - m);
            fg[row * ldf + h] = expf(lf + prev - m);
            floor[row * ldfloor + h] = expf(-m);
        }
        m0 = end;
    }
    if (tid == 0) *ms = m0;
}

// y[t, h] = o[t, h] / sqrt(mean(o^2) + eps) * w * sigmoid(gate[t, h]) (gate_silu: * silu(gate[t, h])); one wave per (token, head);
// w bf16 [vdim] shared by heads or (w_per_head) [heads * vdim] (NULL: no gain).  norm != NULL: o is divided by
// max(|norm[t, h]|, floor[t, h]) + norm_eps first.
__global__ __launch_bounds__(256) void head_rms_gate_kernel(void *__restrict__ y, int y_f32, const float *__restrict__ o, int64_t ldo,
                                                             const uint16_t *__restrict__ w, const float *__restrict__ gate, int64_t ldgate,
                                                             float eps, int rows, int heads, int vdim, int gate_silu, int w_per_head,
                                                             const float *__restrict__ norm, int64_t ldnorm, const float *__restrict__ floor,
                                                             int64_t ldfloor, float norm_eps) {
    const int row = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (row >= rows) return;
    const int t = row / heads, h = row % heads;
    const float *src = o + (int64_t)t * ldo + (int64_t)h * vdim;
    if (w && w_per_head) w += (int64_t)h * vdim;
    const float div = norm ? 1.0f / (fmaxf(fabsf(norm[(int64_t)t * ldnorm + h]), floor[(int64_t)t * ldfloor + h]) + norm_eps) : 1.0f;
    float ss = 0.f;
    for (int i = lane; i < vdim; i += 64) {
        const float v = src[i] * div;
        ss = fmaf(v, v, ss);
    }
    ss = vmx_wave_sum(ss);
    const float inv = div / sqrtf(ss / (float)vdim + eps);
    for (int i = lane; i < vdim; i += 64) {
        float v = src[i] * inv;
        if (w) v *= vmx_bf16_to_f32(w[i]);
        if (gate) {
            const float z = gate[(int64_t)t * ldgate + (int64_t)h * vdim + i];
            v *= gate_silu ? silu_f(z) : sigmoid_f(z);
        }
        const int64_t at = ((int64_t)t * heads + h) * vdim + i;
        if (y_f32) ((float *)y)[at] = v;
        else ((uint16_t *)y)[at] = vmx_f32_to_bf16(v);
    }
}

// The same for wide heads (all of a token's heads normed together, say): a workgroup per (token, head).  A thread holds HELD groups of
// VEC neighbouring numbers, their gates and gains from the first read to the store; numbers past 256 HELD VEC are read twice.
template <int HELD, int VEC>
__global__ __launch_bounds__(256) void row_rms_gate_kernel(void *__restrict__ y, int y_f32, const float *__restrict__ o, int64_t ldo,
                                                            const uint16_t *__restrict__ w, const float *__restrict__ gate, int64_t ldgate,
                                                            float eps, int heads, int vdim, int gate_silu, int w_per_head) {
    __shared__ float red[4];
    const int t = blockIdx.x / heads, h = blockIdx.x % heads, tid = threadIdx.x;
    const float *src = o + (int64_t)t * ldo + (int64_t)h * vdim;
    const int64_t at = (int64_t)blockIdx.x * vdim;
    if (gate) gate += (int64_t)t * ldgate + (int64_t)h * vdim;
    if (w && w_per_head) w += (int64_t)h * vdim;
    float v[HELD][VEC], z[HELD][VEC], g[HELD][VEC], ss = 0.f;
#pragma unroll
    for (int u = 0; u < HELD; u++) {
        const int i = VEC * (tid + 256 * u);
#pragma unroll
        for (int e = 0; e < VEC; e++) v[u][e] = z[u][e] = 0.f, g[u][e] = 1.f;
        if (i >= vdim) continue;
        if constexpr (VEC == 4) {
            const float4 f = *reinterpret_cast<const float4 *>(src + i);
            v[u][0] = f.x, v[u][1] = f.y, v[u][2] = f.z, v[u][3] = f.w;
            if (gate) {
                const float4 q = *reinterpret_cast<const float4 *>(gate + i);
                z[u][0] = q.x, z[u][1] = q.y, z[u][2] = q.z, z[u][3] = q.w;
            }
            if (w) {
                const uint2 b = *reinterpret_cast<const uint2 *>(w + i);
                g[u][0] = vmx_bf16_to_f32((uint16_t)b.x), g[u][1] = vmx_bf16_to_f32((uint16_t)(b.x >> 16));
                g[u][2] = vmx_bf16_to_f32((uint16_t)b.y), g[u][3] = vmx_bf16_to_f32((uint16_t)(b.y >> 16));
            }
        } else {
            v[u][0] = src[i];
            if (gate) z[u][0] = gate[i];
            if (w) g[u][0] = vmx_bf16_to_f32(w[i]);
        }
    }
    constexpr int REST = 256 * HELD * VEC;
#pragma unroll
    for (int u = 0; u < HELD; u++)
#pragma unroll
        for (int e = 0; e < VEC; e++) ss = fmaf(v[u][e], v[u][e], ss);
    for (int i = tid + REST; i < vdim; i += 256) ss = fmaf(src[i], src[i], ss);
    const float inv = 1.0f / sqrtf(vmx_block_sum_256(ss, red) / (float)vdim + eps);
    auto gated = [&](float x, float gain, float zz) { return x * inv * gain * (gate ? (gate_silu ? silu_f(zz) : sigmoid_f(zz)) : 1.0f); };
#pragma unroll
    for (int u = 0; u < HELD; u++) {
        const int i = VEC * (tid + 256 * u);
        if (i >= vdim) continue;
        float r[VEC];
#pragma unroll
        for (int e = 0; e < VEC; e++) r[e] = gated(v[u][e], g[u][e], z[u][e]);
        if constexpr (VEC == 4) {
            if (y_f32) *reinterpret_cast<float4 *>((float *)y + at + i) = make_float4(r[0], r[1], r[2], r[3]);
            else
                *reinterpret_cast<uint2 *>((uint16_t *)y + at + i) = make_uint2((uint32_t)vmx_f32_to_bf16(r[0]) | ((uint32_t)vmx_f32_to_bf16(r[1]) << 16),
                                                                                (uint32_t)vmx_f32_to_bf16(r[2]) | ((uint32_t)vmx_f32_to_bf16(r[3]) << 16));
        } else {
            if (y_f32) ((float *)y)[at + i] = r[0];
            else ((uint16_t *)y)[at + i] = vmx_f32_to_bf16(r[0]);
        }
    }
    for (int i = tid + REST; i < vdim; i += 256) {
        const float r = gated(src[i], w ? vmx_bf16_to_f32(w[i]) : 1.0f, gate ? gate[i] : 0.f);
        if (y_f32) ((float *)y)[at + i] = r;
        else ((uint16_t *)y)[at + i] = vmx_f32_to_bf16(r);
    }
}

ConvArgs conv_args(const float *x, int64_t ldx, const uint16_t *taps, float *state, float *y, int64_t ldy, const int32_t *positions,
                   const int32_t *seq_ids, const int32_t *seq_starts, const int32_t *state_slots, int tokens, int channels, int n, int group,
                   int unit_groups, int scaled_groups, float unit_eps, float mul) {
    return ConvArgs{x, ldx, taps, state, y, ldy, positions, seq_ids, seq_starts, state_slots, tokens, channels, n, group, unit_groups,
                    scaled_groups, unit_eps, mul};
}

}  // namespace

extern "C" size_t vmx_short_conv_state_bytes(int slots, int channels, int taps) {
    return (size_t)slots * (size_t)(taps > 1 ? taps - 1 : 0) * channels * 4;
}

extern "C" int vmx_short_conv_silu(const float *x, int64_t ldx, const uint16_t *taps_bf16, float *state, float *y, int64_t ldy,
                                   const int32_t *positions, const int32_t *seq_ids, const int32_t *seq_starts, const int32_t *state_slots,
                                   int tokens, int channels, int taps, int unit_group, int unit_groups, int scaled_groups, float unit_eps,
                                   float scaled_mul, void *stream) {
    VMX_REQUIRE(x && taps_bf16 && y && positions && seq_ids && seq_starts && state_slots && (state || taps <= 1), "short_conv: null pointer");
    VMX_REQUIRE(channels >= 1 && taps >= 1 && ldx >= channels && ldy >= channels, "short_conv: bad sizes");
    VMX_REQUIRE(unit_groups >= 0 && scaled_groups >= 0 && scaled_groups <= unit_groups && (unit_groups == 0 || unit_group >= 1) &&
                    (int64_t)unit_groups * unit_group <= channels,
                "short_conv: bad unit-vector groups");
    if (tokens <= 0) return VMX_OK;
    const ConvArgs a = conv_args(x, ldx, taps_bf16, state, y, ldy, positions, seq_ids, seq_starts, state_slots, tokens, channels, taps, unit_group,
                                 unit_groups, scaled_groups, unit_eps, scaled_mul);
    const int runs = unit_groups + (channels - unit_groups * unit_group + 63) / 64;
    hipLaunchKernelGGL(short_conv_silu_kernel, dim3(tokens, (runs + 3) / 4), dim3(256), 0, vmx_stream(stream), a);
    VMX_CHECK_LAUNCH("short_conv_silu");
    return VMX_OK;
}

extern "C" int vmx_short_conv_state_update(const float *x, int64_t ldx, float *state, const int32_t *positions, const int32_t *seq_starts,
                                           const int32_t *state_slots, int num_seqs, int channels, int taps, void *stream) {
    VMX_REQUIRE(x && positions && seq_starts && state_slots && (state || taps <= 1), "short_conv_state_update: null pointer");
    if (num_seqs <= 0 || taps <= 1) return VMX_OK;
    const ConvArgs a = conv_args(x, ldx, nullptr, state, nullptr, 0, positions, nullptr, seq_starts, state_slots, 0, channels, taps, 1, 0, 0, 0.f, 1.f);
    hipLaunchKernelGGL(short_conv_state_kernel, dim3((channels + 255) / 256, num_seqs), dim3(256), 0, vmx_stream(stream), a, num_seqs);
    VMX_CHECK_LAUNCH("short_conv_state_update");
    return VMX_OK;
}

extern "C" int vmx_delta_rule_gates(float *g, int64_t ldg, const uint16_t *a_log_bf16, const uint16_t *dt_bias_bf16, float *beta,
                                    int64_t ldbeta, int tokens, int heads, int dim, void *stream) {
    VMX_REQUIRE(g && a_log_bf16 && dt_bias_bf16 && beta, "delta_rule_gates: null pointer");
    VMX_REQUIRE(heads >= 1 && dim >= 1 && ldg >= (int64_t)heads * dim && ldbeta >= heads, "delta_rule_gates: bad sizes");
    if (tokens <= 0) return VMX_OK;
    hipLaunchKernelGGL(delta_gates_kernel, dim3(tokens, (heads * dim + 255) / 256), dim3(256), 0, vmx_stream(stream), g, ldg, a_log_bf16,
                       dt_bias_bf16, beta, ldbeta, heads, dim);
    VMX_CHECK_LAUNCH("delta_rule_gates");
    return VMX_OK;
}

static int delta_dpt(int dim) { return dim <= 64 ? 4 : (dim <= 128 ? 8 : 16); }
static size_t delta_lds_bytes(int dpt) {
    const size_t ct = 128 / dpt, row = (size_t)DR_RS * (dpt == 4 ? 4 : dpt + 4);
    return (3 * 2 * ct * row + 2 * ct * DR_VT + 2 * ct) * 4;
}
template <int DT> static int memory_chunk_launch(const DeltaArgs &a, dim3 grid, hipStream_t st) {
    static bool sized = false;
    constexpr int lds = memory_chunk_lds(DT).total;
    if (!sized) {
        VMX_CHECK_HIP(hipFuncSetAttribute((const void *)memory_chunk_kernel<DT>, hipFuncAttributeMaxDynamicSharedMemorySize, lds));
        sized = true;
    }
    hipLaunchKernelGGL(memory_chunk_kernel<DT>, grid, dim3(256), lds, st, a);
    return VMX_OK;
}
template <int DPT> static int delta_launch(const DeltaArgs &a, dim3 grid, hipStream_t st) {
    static bool sized = false;   // more than 64 KiB of LDS has to be asked for once per kernel
    const size_t lds = delta_lds_bytes(DPT);
    if (!sized) {
        VMX_CHECK_HIP(hipFuncSetAttribute((const void *)gated_delta_rule_kernel<DPT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
        sized = true;
    }
    hipLaunchKernelGGL(gated_delta_rule_kernel<DPT>, grid, dim3(256), lds, st, a);
    return VMX_OK;
}

extern "C" size_t vmx_gated_delta_rule_state_bytes(int slots, int heads, int dim, int vdim) {
    const size_t tiles = (vdim + DR_VT - 1) / DR_VT;
    return (size_t)slots * heads * tiles * delta_dpt(dim) * 256 * 4;
}

extern "C" int vmx_gated_delta_rule(float *o, int64_t ldo, const float *q, int64_t ldq, const float *k, int64_t ldk, const float *v,
                                    int64_t ldv, const float *g, int64_t ldg, const float *beta, int64_t ldbeta, float *state,
                                    const int32_t *positions, const int32_t *seq_starts, const int32_t *state_slots, int num_seqs, int heads,
                                    int qk_heads, int dim, int vdim, void *stream) {
    VMX_REQUIRE(beta, "gated_delta_rule: null pointer");
    return vmx_matrix_memory_recurrence(o, ldo, q, ldq, 1.0f, k, ldk, v, ldv, g, ldg, 0, beta, ldbeta, state, positions, seq_starts, state_slots, num_seqs,
                                        heads, qk_heads, dim, vdim, stream);
}

extern "C" int vmx_sigmoid_root_decay(float *g, int64_t ldg, int tokens, int n, float tau, void *stream) {
    VMX_REQUIRE(g && n >= 1 && ldg >= n && tau > 0.f, "sigmoid_root_decay: bad arguments");
    if (tokens <= 0) return VMX_OK;
    hipLaunchKernelGGL(sigmoid_root_decay_kernel, dim3(tokens, (n + 255) / 256), dim3(256), 0, vmx_stream(stream), g, ldg, n, 1.0f / tau);
    VMX_CHECK_LAUNCH("sigmoid_root_decay");
    return VMX_OK;
}

extern "C" int vmx_matrix_memory_recurrence(float *o, int64_t ldo, const float *q, int64_t ldq, float q_mul, const float *k, int64_t ldk, const float *v,
                                            int64_t ldv, const float *g, int64_t ldg, int g_per_head, const float *beta, int64_t ldbeta,
                                            float *state, const int32_t *positions, const int32_t *seq_starts, const int32_t *state_slots,
                                            int num_seqs, int heads, int qk_heads, int dim, int vdim, void *stream) {
    return vmx_matrix_memory_recurrence_ex(o, ldo, q, ldq, q_mul, k, ldk, v, ldv, g, ldg, g_per_head, beta, ldbeta, state, positions, seq_starts,
                                           state_slots, num_seqs, heads, qk_heads, dim, vdim, nullptr, stream);
}

extern "C" int vmx_matrix_memory_recurrence_ex(float *o, int64_t ldo, const float *q, int64_t ldq, float q_mul, const float *k, int64_t ldk,
                                               const float *v, int64_t ldv, const float *g, int64_t ldg, int g_per_head, const float *beta,
                                               int64_t ldbeta, float *state, const int32_t *positions, const int32_t *seq_starts,
                                               const int32_t *state_slots, int num_seqs, int heads, int qk_heads, int dim, int vdim,
                                               const vmx_matrix_memory_opts *opts, void *stream) {
    VMX_REQUIRE(o && q && k && v && g && state && positions && seq_starts && state_slots, "matrix_memory_recurrence: null pointer");
    VMX_REQUIRE(heads >= 1 && qk_heads >= 1 && heads % qk_heads == 0, "matrix_memory_recurrence: %d heads do not share %d query/key heads evenly",
                heads, qk_heads);
    VMX_REQUIRE(dim >= 1 && dim <= 256 && vdim >= 1, "matrix_memory_recurrence: key size %d outside 1..256", dim);
    VMX_REQUIRE(ldg >= (g_per_head ? heads : (int64_t)heads * dim) || (g_per_head && ldg == 0), "matrix_memory_recurrence: bad decay row stride");
    if (num_seqs <= 0) return VMX_OK;
    const bool gain = opts && opts->write_gain, norm = opts && opts->norm_out;
    VMX_REQUIRE(!(gain && beta), "matrix_memory_recurrence: a write gain belongs to the plain write, beta to the delta rule");
    VMX_REQUIRE(!norm || opts->ldnorm >= heads, "matrix_memory_recurrence: bad row stride of the normaliser's read-out");
    const DeltaArgs a{q, k, v, g, gain ? opts->write_gain : beta, ldq, ldk, ldv, ldg, gain ? opts->ldgain : ldbeta, o, ldo, state, positions,
                      seq_starts, state_slots, heads, qk_heads, dim, vdim, g_per_head ? 1 : 0, beta ? 0 : 1, q_mul, norm ? opts->norm_out : nullptr,
                      norm ? opts->ldnorm : 0};
    const dim3 grid((vdim + (norm ? 1 : 0) + DR_VT - 1) / DR_VT, heads, num_seqs);
    hipStream_t st = vmx_stream(stream);
    int rc;
    // prompts: 64 tokens at a time on the matrix cores, where the caller takes q, k and v in bf16
    if (opts && opts->bf16_operands && !beta && g_per_head && opts->tokens >= 8 * num_seqs) {
        switch (delta_dpt(dim)) {
            case 4: rc = memory_chunk_launch<4>(a, grid, st); break;
            case 8: rc = memory_chunk_launch<8>(a, grid, st); break;
            default: rc = memory_chunk_launch<16>(a, grid, st); break;
        }
        if (rc) return rc;
        VMX_CHECK_LAUNCH("matrix_memory_recurrence (chunks)");
        return VMX_OK;
    }
    switch (delta_dpt(dim)) {
        case 4: rc = delta_launch<4>(a, grid, st); break;
        case 8: rc = delta_launch<8>(a, grid, st); break;
        default: rc = delta_launch<16>(a, grid, st); break;
    }
    if (rc) return rc;
    VMX_CHECK_LAUNCH("matrix_memory_recurrence");
    return VMX_OK;
}

extern "C" int vmx_head_rms_gate(void *y, int y_dtype, const float *o, int64_t ldo, const uint16_t *w_bf16, const float *gate, int64_t ldgate,
                                 float eps, int tokens, int heads, int vdim, void *stream) {
    VMX_REQUIRE(w_bf16, "head_rms_gate: null pointer");
    return vmx_head_rms_gate_ex(y, y_dtype, o, ldo, w_bf16, gate, ldgate, 0, eps, tokens, heads, vdim, stream);
}

extern "C" int vmx_head_rms_gate_ex(void *y, int y_dtype, const float *o, int64_t ldo, const uint16_t *w_bf16, const float *gate, int64_t ldgate,
                                       int gate_silu, float eps, int tokens, int heads, int vdim, void *stream) {
    const vmx_read_out_opts ro = {gate_silu, 0, nullptr, 0, nullptr, 0, 0.f};
    return vmx_head_read_out(y, y_dtype, o, ldo, w_bf16, gate, ldgate, eps, tokens, heads, vdim, &ro, stream);
}

extern "C" int vmx_exp_gate_scan(float *input_gate, int64_t ldi, float *forget_gate, int64_t ldf, float *floor, int64_t ldfloor, float *max_state,
                                 float cap, const int32_t *positions, const int32_t *seq_starts, const int32_t *state_slots, int num_seqs,
                                 int heads, void *stream) {
    VMX_REQUIRE(input_gate && forget_gate && floor && max_state && positions && seq_starts && state_slots, "exp_gate_scan: null pointer");
    VMX_REQUIRE(heads >= 1 && ldi >= heads && ldf >= heads && ldfloor >= heads && cap > 0.f, "exp_gate_scan: bad sizes or cap");
    if (num_seqs <= 0) return VMX_OK;
    hipLaunchKernelGGL(exp_gate_scan_kernel, dim3(heads, num_seqs), dim3(256), 0, vmx_stream(stream), input_gate, ldi, forget_gate, ldf, floor, ldfloor,
                       max_state, cap, positions, seq_starts, state_slots, heads);
    VMX_CHECK_LAUNCH("exp_gate_scan");
    return VMX_OK;
}

extern "C" int vmx_head_read_out(void *y, int y_dtype, const float *o, int64_t ldo, const uint16_t *w_bf16, const float *gate, int64_t ldgate,
                                 float eps, int tokens, int heads, int vdim, const vmx_read_out_opts *opts, void *stream) {
    VMX_REQUIRE(y && o && opts, "head_rms_gate: null pointer");
    VMX_REQUIRE(!opts->norm || opts->floor, "head_rms_gate: a normaliser comes with its floor");
    VMX_REQUIRE(y_dtype == VMX_F32 || y_dtype == VMX_BF16, "head_rms_gate: f32 or bf16 output");
    if (tokens <= 0) return VMX_OK;
    if (vdim > 256 && !opts->norm) {
        // whole groups of four numbers on 16-byte (f32) / 8-byte (bf16) boundaries
        const bool vec = vdim % 4 == 0 && ldo % 4 == 0 && ldgate % 4 == 0 && (((uintptr_t)o | (uintptr_t)gate | (uintptr_t)y) & 15) == 0 && ((uintptr_t)w_bf16 & 7) == 0;
#define RG(held, v)                                                                                                                                \
    hipLaunchKernelGGL((row_rms_gate_kernel<held, v>), dim3(tokens * heads), dim3(256), 0, vmx_stream(stream), y, y_dtype == VMX_F32, o, ldo, w_bf16, \
                       gate, ldgate, eps, heads, vdim, opts->gate_silu ? 1 : 0, opts->w_per_head ? 1 : 0)
        if (!vec) RG(8, 1);
        else if (vdim <= 1024) RG(1, 4);
        else if (vdim <= 2048) RG(2, 4);
        else RG(4, 4);
#undef RG
        VMX_CHECK_LAUNCH("head_rms_gate (wide)");
        return VMX_OK;
    }
    hipLaunchKernelGGL(head_rms_gate_kernel, dim3((tokens * heads + 3) / 4), dim3(256), 0, vmx_stream(stream), y, y_dtype == VMX_F32, o, ldo,
                       w_bf16, gate, ldgate, eps, tokens * heads, heads, vdim, opts->gate_silu ? 1 : 0, opts->w_per_head ? 1 : 0, opts->norm,
                       opts->ldnorm, opts->floor, opts->ldfloor, opts->norm_eps);
    VMX_CHECK_LAUNCH("head_rms_gate");
    return VMX_OK;
}
