// Parameters of the extended paged attention (xattn.hip: entry points, plain kernels; xattn_mfma.hip: matrix-core kernels).
#pragma once
#include "md_common.h"

struct XattnParams {
    const void* q;            // normalised, padded queries [rows][H][DKp] (model dtype)
    const void* qkv;          // raw projection rows [rows][ld_qkv]: q | k | v (fused decode), else null
    int64_t ld_qkv;
    void* k_cache;            // [pages][KH][page_size][DKp]
    void* v_cache;            // [pages][KH][page_size][DVp]
    void* out;                // [rows][H][DV]
    const int32_t* qo_indptr;
    const int32_t* pos0;
    const int32_t* page_indices;
    const int32_t* page_indptr;
    const float* r1;          // distance bias per query head, or null
    const float* r2;
    float* ws;                // split-KV partials
    unsigned int* overflow;
    int B, n_max, H, KH, g, D, DV, DKp, DVp, page_size;
    int ldk, ldv;             // plain kernel: elements between rows of a page
    int chunk;                // > 0; 0x7fffffff: no chunk mask
    int sink, qk_norm, nsplit, n_qgroups, rows_cap;
    float eps, scale, scale_log2, ref_log2;   // ref_log2: the fixed softmax reference of the matrix-core kernels, log2 units
};

// the plain kernel of xattn.hip (16- or 32-bit pages): any head sizes up to 1024, online softmax in fp32
int md_internal_xattn_plain(const XattnParams& p, int dtype, hipStream_t st);

// one translation unit per padded query/key width; false: no kernel for (DKp, DVp)
#define MD_XATTN_DECL(DK)                                                                                       \
    int md_internal_xattn_decode_##DK(const XattnParams& p, int qt, bool fused, int grid, hipStream_t st);       \
    int md_internal_xattn_waves_##DK(int dv, int g, int rows);                                                    \
    int md_internal_xattn_prefill_##DK(const XattnParams& p, int nw, int grid, hipStream_t st);
MD_XATTN_DECL(32)
MD_XATTN_DECL(64)
MD_XATTN_DECL(96)
MD_XATTN_DECL(128)
MD_XATTN_DECL(192)
MD_XATTN_DECL(256)
#undef MD_XATTN_DECL
