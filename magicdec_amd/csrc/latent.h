// Parameters of the latent attention (latent.hip: entry points and small kernels; latent_mfma.hip: matrix-core kernels).
#pragma once
#include "md_common.h"

struct LatentParams {
    const void* z;            // projection rows [rows][ldz]: query latent (q_rank) | latent (kv_rank) | rotated key part (rot_dim)
    const void* dq_norm;      // [q_rank]
    const void* kv_norm;      // [kv_rank]
    void* cq;                 // normalised query latents [rows][q_rank]
    void* cache;              // [pages][page_size][W]: latent | rotated key part | zeros
    const float* cos_sin;     // [max_pos][rot_pairs][2], amplitude included
    const int32_t* qo_indptr;
    const int32_t* pos0;
    const int32_t* page_indices;
    const int32_t* page_indptr;
    const int32_t* ctx_indptr;   // first row of request b in the gathered / expanded context
    const void* q;            // absorbed form: [rows][H][W]; expanded form: raw query rows [rows][H][dim + rot_dim]
    const void* kv;           // expanded form: [context rows][H * dim | H * vdim]
    const void* gate;         // gate logits [rows][ld_gate], one per head, or null
    void* out;                // absorbed: [rows][H][kv_rank]; expanded: [rows][ldo], H * vdim used
    float* ws;                // kv split partials
    unsigned int* overflow;
    int64_t ldz, ldo, ld_gate;
    int B, n_max, H, dim, rot_dim, rot_pairs, vdim, q_rank, kv_rank, W, page_size, max_pos, append;
    int nsplit, n_groups;     // absorbed: kv splits, row groups per request; expanded: n_groups = row groups per (request, head)
    float eps, scale_log2;
};

// absorbed form; qt: 16-row tiles of (token, head) pairs per workgroup (1 or 2)
int md_internal_latent_absorbed(const LatentParams& p, int qt, hipStream_t st);
bool md_internal_latent_absorbed_ok(int kv_rank, int W, int qt);
// expanded form; DK: padded dim + rot_dim, one translation unit each
#define MD_LATENT_DECL(DK) int md_internal_latent_prefill_##DK(const LatentParams& p, int grid, hipStream_t st);
MD_LATENT_DECL(64)
MD_LATENT_DECL(128)
MD_LATENT_DECL(192)
MD_LATENT_DECL(256)
#undef MD_LATENT_DECL
constexpr int kLatentPrefillRows = 256;     // query rows (tokens) of one expanded workgroup
