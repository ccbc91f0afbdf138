// Expanded latent attention on the matrix cores (bf16, gfx950): prompts.  Keys are the context's expanded rows (dim numbers per
// head, dense) followed by the rotated part every head shares (straight from the cache pages); values are expanded rows.
// Compiled once per padded key width: -DMD_LATENT_DK=64 | 128 | 192 | 256; the value width is a template parameter.
//
// Eight wavefronts of 32 query rows share 64-key tiles through two LDS images, one barrier per tile.  S^T = K Q^T and
// O^T = V^T P^T on 32x32x16: a lane owns one query row, so the running maximum is a lane-local reduction plus one exchange.  It is
// followed lazily: sums are rescaled only when a tile's maximum exceeds the reference by 8 (weights up to 2^8 are harmless in
// fp32).  Queries are rotated as they are loaded; the output is multiplied by the head's gate.  Weights enter the product as a
// bf16 part and a bf16 rest.
#include "attn_common.h"
#include "latent.h"

#ifndef MD_LATENT_DK
#error "compile with -DMD_LATENT_DK=<padded key size>"
#endif

namespace {

typedef float f32x16 __attribute__((ext_vector_type(16)));
constexpr int DK = MD_LATENT_DK, KT = 64, NW = kLatentPrefillRows / 32, NT = 64 * NW;
constexpr int KROW = DK * 2 + 16;

template <int DV>
constexpr int stage_bytes() { return KT * KROW + (KT / 32) * (DV / 16) * kVSub; }

template <int DV>
__global__ __launch_bounds__(NT, 2) void latent_prefill_kernel(const LatentParams p) {
    constexpr int KS = DK / 16, NB = DV / 16, DB = DV / 32;
    constexpr int K_BYTES = KT * KROW, VG = NB * kVSub, STAGE = stage_bytes<DV>();
    constexpr int CK = KT * DK / 8, CV = KT * DV / 8, NK = CK / NT, NV = CV / NT;
    static_assert(CK % NT == 0 && CV % NT == 0, "a tile is a whole number of pieces per thread");
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];   // two tile images
    const int tid = threadIdx.x, lane = tid & 63, j = lane & 31, kh = lane >> 5;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    // blocks of one (request, head) differ by multiples of 8: same XCD; the long ones (late rows) first
    const int r0 = blockIdx.x >> 3;
    const int qg = p.n_groups - 1 - r0 % p.n_groups, pair = (r0 / p.n_groups) * 8 + (blockIdx.x & 7);
    if (pair >= p.B * p.H) return;
    const int b = pair / p.H, h = pair % p.H;
    const int q0 = p.qo_indptr[b], n_b = p.qo_indptr[b + 1] - q0;
    if (qg * kLatentPrefillRows >= n_b) return;                   // whole workgroup
    const int pos_b = p.pos0[b], pg0 = p.page_indptr[b], cap = (p.page_indptr[b + 1] - pg0) * p.page_size;
    const int c0 = p.ctx_indptr[b], ctx = min(p.ctx_indptr[b + 1] - c0, cap);
    const int wg_last = min(pos_b + min(qg * kLatentPrefillRows + kLatentPrefillRows, n_b) - 1, ctx - 1);
    if (wg_last < 0) return;
    const int qi = qg * kLatentPrefillRows + wave * 32 + j;
    const bool valid = qi < n_b;
    const int pos = pos_b + qi, lim = valid ? min(pos, ctx - 1) : 0;
    const int lim_lo = min(pos_b + qg * kLatentPrefillRows + wave * 32, ctx - 1);     // the wave's first row
    const int my_last = qg * kLatentPrefillRows + wave * 32 < n_b ? min(pos_b + min(qg * kLatentPrefillRows + wave * 32 + 32, n_b) - 1, ctx - 1) : -1;
    const int t1 = wg_last / KT, my1 = my_last >= 0 ? my_last / KT : -1;
    const int dq = p.dim + p.rot_dim;
    const float sl2 = fabsf(p.scale_log2);

    bf16x8 qf[KS];
    {
        const bf16_t* qp = reinterpret_cast<const bf16_t*>(p.q) + ((int64_t)(q0 + (valid ? qi : 0)) * p.H + h) * dq;
        const float* cs = p.cos_sin + (int64_t)min(max(pos, 0), p.max_pos - 1) * p.rot_pairs * 2;
        const bf16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
        const float sign = p.scale_log2 < 0.f ? -1.f : 1.f;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            const int d = ks * 16 + kh * 8;
            const bf16x8 raw = valid && d < dq ? *reinterpret_cast<const bf16x8*>(qp + d) : z;
            f32x8 v = __builtin_convertvector(raw, f32x8);
            if (d >= p.dim && d < dq) {
#pragma unroll
                for (int e = 0; e < 8; e += 2) {
                    const int i = (d - p.dim + e) >> 1;
                    if (i < p.rot_pairs) {
                        const float c = cs[2 * i], s = cs[2 * i + 1], a = v[e], w = v[e + 1];
                        v[e] = a * c - w * s;
                        v[e + 1] = w * c + a * s;
                    }
                }
            }
            qf[ks] = __builtin_convertvector(v * sign, bf16x8);
        }
    }
    f32x16 o[DB];
#pragma unroll
    for (int db = 0; db < DB; ++db)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[db][r] = 0.f;
    float m = -INFINITY, l = 0.f;

    u32x4 kreg[NK], vreg[NV];
    const u32x4 z4 = {0u, 0u, 0u, 0u};
    const int64_t ldkv = (int64_t)p.H * (p.dim + p.vdim);
    const bf16_t* kv = reinterpret_cast<const bf16_t*>(p.kv);
    const int hk = h * p.dim, hv = p.H * p.dim + h * p.vdim;
    auto issue = [&](int t) {
        const int kp0 = t * KT;
        const int64_t crow = (int64_t)p.page_indices[pg0 + kp0 / p.page_size] * p.page_size + kp0 % p.page_size;
        const bf16_t* rp = reinterpret_cast<const bf16_t*>(p.cache) + crow * p.W + p.kv_rank;
#pragma unroll
        for (int i = 0; i < NK; ++i) {
            const int c = i * NT + tid, row = c / (DK / 8), d = (c % (DK / 8)) * 8;
            kreg[i] = z4;
            if (kp0 + row < ctx && d < dq)
                kreg[i] = d < p.dim ? *reinterpret_cast<const u32x4*>(kv + (c0 + kp0 + row) * ldkv + hk + d)
                                    : *reinterpret_cast<const u32x4*>(rp + (int64_t)row * p.W + d - p.dim);
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = i * NT + tid, row = c / (DV / 8), d = (c % (DV / 8)) * 8;
            vreg[i] = kp0 + row < ctx && d < p.vdim ? *reinterpret_cast<const u32x4*>(kv + (c0 + kp0 + row) * ldkv + hv + d) : z4;
        }
    };
    auto stage = [&](unsigned char* img) {
#pragma unroll
        for (int i = 0; i < NK; ++i) {
            const int c = i * NT + tid;
            *reinterpret_cast<u32x4*>(img + (c / (DK / 8)) * KROW + (c % (DK / 8)) * 16) = kreg[i];
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = i * NT + tid, row = c / (DV / 8), ch = c % (DV / 8);
            *reinterpret_cast<u32x4*>(img + K_BYTES + (row >> 5) * VG + (ch >> 1) * kVSub + (row & 31) * 32 + (ch & 1) * 16) = vreg[i];
        }
    };
    const int kra0 = j * KROW + kh * 16, lq = lane & 15;
    const int vra0 = K_BYTES + ((lane >> 4) & 1) * (NB / 2) * kVSub + (kh * 4 + (lq >> 2)) * 32 + (lq & 3) * 8;
    auto compute = [&](int t, const unsigned char* img) {
        f32x16 sc[2];
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int r = 0; r < 16; ++r) sc[u][r] = 0.f;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
#pragma unroll
            for (int u = 0; u < 2; ++u)
                sc[u] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(lds_read_b128(img + kra0 + u * 32 * KROW + ks * 32), qf[ks], sc[u], 0, 0, 0);
        if (t * KT + KT - 1 > lim_lo) {                             // wave-uniform: the tile reaches past some row's position
#pragma unroll
            for (int u = 0; u < 2; ++u)
#pragma unroll
                for (int r = 0; r < 16; ++r)
                    if (t * KT + u * 32 + 4 * kh + (r & 3) + 8 * (r >> 2) > lim) sc[u][r] = -INFINITY;
        }
        float mx = sc[0][0];
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int r = 0; r < 16; ++r) mx = fmaxf(mx, sc[u][r]);
        mx = fmaxf(mx, __shfl_xor(mx, 32)) * sl2;
        if (__any(mx > m + 8.f)) {                                  // (the first tile holds key 0, which every row sees: m is finite)
            const float mn = fmaxf(m, mx), alpha = __builtin_amdgcn_exp2f(m - mn);
            l *= alpha;
#pragma unroll
            for (int db = 0; db < DB; ++db)
#pragma unroll
                for (int r = 0; r < 16; ++r) o[db][r] *= alpha;
            m = mn;
        }
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int s16 = 0; s16 < 2; ++s16) {
                f32x8 pv;
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    pv[e] = __builtin_amdgcn_exp2f(fmaf(sc[u][s16 * 8 + e], sl2, -m));
                    l += pv[e];
                }
                const bf16x8 ph = __builtin_convertvector(pv, bf16x8);
                const bf16x8 pl = __builtin_convertvector(pv - __builtin_convertvector(ph, f32x8), bf16x8);
#pragma unroll
                for (int db = 0; db < DB; ++db) {
                    const unsigned char* vb = img + u * VG + db * kVSub + vra0 + s16 * 16 * 32;
                    const bf16x4 v0 = lds_read_tr(vb), v1 = lds_read_tr(vb + 8 * 32);
                    const bf16x8 vf = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
                    o[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, ph, o[db], 0, 0, 0);
                    o[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pl, o[db], 0, 0, 0);
                }
            }
    };

    // tile t lies in image t & 1; it is overwritten two tiles later, after a barrier every wave reaches past its use
    issue(0);
    for (int t = 0; t <= t1; ++t) {
        unsigned char* img = smem + (t & 1) * STAGE;
        stage(img);
        if (t < t1) issue(t + 1);
        __syncthreads();
        if (t <= my1) compute(t, img);
    }

    l += __shfl_xor(l, 32);
    if (valid) {
        float inv = 1.0f / l;
        if (p.gate) inv /= 1.0f + expf(-(float)reinterpret_cast<const bf16_t*>(p.gate)[(q0 + qi) * p.ld_gate + h]);
        bf16_t* op = reinterpret_cast<bf16_t*>(p.out) + (q0 + qi) * p.ldo + h * p.vdim;
#pragma unroll
        for (int db = 0; db < DB; ++db)
#pragma unroll
            for (int rg = 0; rg < 4; ++rg) {
                const int d = (db + (rg >> 1) * (NB / 2)) * 16 + (rg & 1) * 8 + kh * 4;
                const f32x4 ov = {o[db][rg * 4] * inv, o[db][rg * 4 + 1] * inv, o[db][rg * 4 + 2] * inv, o[db][rg * 4 + 3] * inv};
                if (d < p.vdim) *reinterpret_cast<bf16x4*>(op + d) = __builtin_convertvector(ov, bf16x4);
            }
    }
}

template <int DV>
int launch(const LatentParams& p, int grid, hipStream_t st) {
    constexpr int lds = 2 * stage_bytes<DV>();
    static_assert(lds <= 160 * 1024, "the two tile images must fit the CU");
    auto k = latent_prefill_kernel<DV>;
    static MdPerDeviceOnce once;
    if (lds > 64 * 1024 && once.first() &&
        hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, lds) != hipSuccess) {
        once.undo();
        md_set_error("md_latent_prefill: hipFuncSetAttribute(%d B LDS) failed", lds);
        return MD_ERR_LAUNCH;
    }
    hipLaunchKernelGGL(k, dim3(grid), dim3(NT), lds, st, p);
    return MD_OK;
}

}  // namespace

#define MD_CAT_(a, b) a##b
#define MD_CAT(a, b) MD_CAT_(a, b)

int MD_CAT(md_internal_latent_prefill_, MD_LATENT_DK)(const LatentParams& p, int grid, hipStream_t st) {
    return p.vdim <= 64 ? launch<64>(p, grid, st) : p.vdim <= 128 ? launch<128>(p, grid, st)
         : p.vdim <= 192 ? launch<192>(p, grid, st) : launch<256>(p, grid, st);
}
