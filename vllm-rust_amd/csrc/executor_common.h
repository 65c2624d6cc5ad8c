// Host-side pieces that packed-step executors share: where a checkpoint tensor lands, uploads, and the bookkeeping of a mixture of
// experts whose (token, slot) pairs run as expert blocks.
#pragma once
#include "vmx_kernels.h"
#include <algorithm>
#include <string>
#include <utility>
#include <vector>

inline int vmx_pad8(int n) { return (n + 7) & ~7; }

inline int vmx_upload(VmxBuf &b, size_t offset, const void *data, size_t bytes, hipStream_t st) {
    VMX_CHECK_HIP(hipMemcpyAsync((char *)b.p + offset, data, bytes, hipMemcpyDefault, st));
    VMX_CHECK_HIP(hipStreamSynchronize(st));
    return VMX_OK;
}

inline int vmx_alloc_zero(VmxBuf &b, size_t n) {
    if (int rc = b.alloc(n)) return rc;
    VMX_CHECK_HIP(hipMemset(b.p, 0, n ? n : 16));
    return VMX_OK;
}

inline bool vmx_rotation_ok(const vmx_rotation &r, int head_dim) {
    if (r.dims == 0) return true;
    if (r.dims < 0 || r.dims % 2 || r.dims > head_dim || !(r.base > 1.0)) return false;
    return r.factor == 0.0 || (r.factor > 0.0 && r.original > 0.0 && r.fast > 0.0 && r.slow > 0.0);
}

// angle steps of a rotation on the device and its cos / sin multiplier; dims 0: nothing
inline int vmx_upload_rotation(const vmx_rotation &r, VmxBuf &steps, float &mul) {
    mul = 1.f;
    if (r.dims <= 0) return VMX_OK;
    std::vector<float> f(r.dims / 2);
    if (int rc = vmx_rotation_steps(&r, f.data(), &mul)) return rc;
    if (int rc = steps.alloc(f.size() * 4)) return rc;
    VMX_CHECK_HIP(hipMemcpy(steps.p, f.data(), f.size() * 4, hipMemcpyHostToDevice));
    return VMX_OK;
}

inline void vmx_erase_name(std::vector<std::string> &v, const std::string &name) { v.erase(std::remove(v.begin(), v.end(), name), v.end()); }

// Checkpoint name -> destination (rows of a fused projection, or a buffer of its own), and which names are still to come.
struct VmxTensorTable {
    struct Seg {
        VmxBuf *buf = nullptr;
        size_t offset = 0, bytes = 0;
    };
    std::vector<std::pair<std::string, Seg>> tensors;
    std::vector<std::string> missing;
    void want(const std::string &name, VmxBuf *b, size_t off, size_t bytes) {
        tensors.push_back({name, Seg{b, off, bytes}});
        missing.push_back(name);
    }
    const Seg *find(const std::string &name) const {
        for (const auto &t : tensors)
            if (t.first == name) return &t.second;
        return nullptr;
    }
    void loaded(const std::string &name) { vmx_erase_name(missing, name); }
};

// Routing results of a step and the blocks its experts run as.  Up to VMX_MOE_FEW_PAIRS pairs: every pair is its own 16-row block
// (no sort; tables made once); more: sorted by expert into blocks of 16 or, from 32 pairs per expert on, 64 rows.
struct VmxExpertBlocks {
    VmxBuf few_pairs, topw, topi, sorted, blk_expert, total, inverse;
    size_t rows = (size_t)VMX_MOE_FEW_PAIRS * 16;   // most rows (padding included) of any layer's blocks
    size_t pairs = 0;
    // of the current step and layer
    int block_rows = 16, cap = 0;
    const int32_t *up_rows = nullptr, *down_rows = nullptr, *block_expert = nullptr, *total_rows = nullptr, *pair_rows = nullptr;

    void reserve(size_t tokens, int experts, int top) {
        pairs = std::max(pairs, tokens * top);
        rows = std::max(rows, tokens * top + (size_t)experts * 63);
    }
    int alloc() {
        const int FP = VMX_MOE_FEW_PAIRS;
        std::vector<int32_t> fp(2 * FP * 16 + FP + 1);
        for (int i = 0; i < FP * 16; i++) {
            fp[i] = i % 16 == 0 ? i / 16 : 0x7fffffff;           // gathered rows of the first product: pair index or padding
            fp[FP * 16 + i] = i % 16 == 0 ? i : 0x7fffffff;       // rows of the second product: themselves or padding
        }
        for (int p = 0; p < FP; p++) fp[2 * FP * 16 + p] = 16 * p;   // where pair p's result lies
        fp[2 * FP * 16 + FP] = 0x7fffffff;                        // "total rows": never cuts
        for (auto &b : {std::make_pair(&few_pairs, fp.size() * 4), std::make_pair(&topw, (pairs + 1) * 4), std::make_pair(&topi, (pairs + 1) * 4),
                        std::make_pair(&sorted, (rows + 1) * 4), std::make_pair(&blk_expert, (rows / 16 + 2) * 4), std::make_pair(&total, (size_t)16),
                        std::make_pair(&inverse, (pairs + 1) * 4)})
            if (int rc = vmx_alloc_zero(*b.first, b.second)) return rc;
        VMX_CHECK_HIP(hipMemcpy(few_pairs.p, fp.data(), fp.size() * 4, hipMemcpyHostToDevice));
        return VMX_OK;
    }
    void release() {
        for (VmxBuf *b : {&few_pairs, &topw, &topi, &sorted, &blk_expert, &total, &inverse}) b->release();
    }
    // block layout of `n` routed pairs (topi holds their experts)
    int plan(int n, int experts, hipStream_t st) {
        const int FP = VMX_MOE_FEW_PAIRS;
        const bool few = n <= FP;
        block_rows = few ? 16 : (n >= 32 * experts ? 64 : 16);
        cap = few ? n * 16 : n + experts * (block_rows - 1);
        const int32_t *fp = few_pairs.as<int32_t>();
        up_rows = few ? fp : sorted.as<int32_t>(), down_rows = few ? fp + FP * 16 : nullptr;
        block_expert = few ? topi.as<int32_t>() : blk_expert.as<int32_t>();
        total_rows = few ? fp + 2 * FP * 16 + FP : total.as<int32_t>();
        pair_rows = few ? fp + 2 * FP * 16 : inverse.as<int32_t>();
        if (few) return VMX_OK;
        if (int rc = vmx_moe_align_block_size(topi.as<int32_t>(), sorted.as<int32_t>(), blk_expert.as<int32_t>(), total.as<int32_t>(), n, experts,
                                              block_rows, cap, st))
            return rc;
        return vmx_moe_inverse(inverse.as<int32_t>(), sorted.as<int32_t>(), total.as<int32_t>(), n, cap, st);
    }
    // the two products of a layer's experts: rows gathered by token, `top` pairs a token; rows of the second are the pairs' blocks
    void first(VmxLinear &u, int n, int top, int64_t stride) const {
        u.M = cap, u.row_ids = up_rows, u.row_div = top, u.row_limit = n;
        u.block_expert = block_expert, u.expert_stride = stride, u.block_rows = block_rows, u.total_rows = total_rows;
    }
    void second(VmxLinear &d, int64_t stride) const {
        d.M = cap, d.row_ids = down_rows, d.row_div = 1, d.row_limit = cap;
        d.block_expert = block_expert, d.expert_stride = stride, d.block_rows = block_rows, d.total_rows = total_rows;
    }
};
