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

// weights -> upper 16 bits (truncated: bf16) and the rest rounded to bf16
__device__ __forceinline__ void split(const f32x8 w, bf16x8& hi, bf16x8& lo) {
    u32x4 h;
    f32x8 r;
#pragma unroll
    for (int e = 0; e < 8; e += 2) {
        const unsigned int a = __float_as_uint(w[e]), b = __float_as_uint(w[e + 1]);
        h[e / 2] = __builtin_amdgcn_perm(b, a, 0x07060302);
        r[e] = w[e] - __uint_as_float(a & 0xffff0000u);
        r[e + 1] = w[e + 1] - __uint_as_float(b & 0xffff0000u);
    }
    hi = *reinterpret_cast<const bf16x8*>(&h);
    lo = __builtin_convertvector(r, bf16x8);
}

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
    const int w0 = qg * kLatentPrefillRows + wave * 32, qi = w0 + j;            // the wave's first row, this lane's row
    const bool valid = qi < n_b;
    const int pos = pos_b + qi, lim = valid ? min(pos, ctx - 1) : 0;
    const int lim_lo = min(pos_b + w0, ctx - 1), my_last = w0 < n_b ? min(pos_b + min(w0 + 32, n_b) - 1, ctx - 1) : -1;
    const int t1 = wg_last / KT, my1 = my_last >= 0 ? my_last / KT : -1;
    const int dq = p.dim + p.rot_dim;
    const float sl2 = fabsf(p.scale_log2);

    bf16x8 qf[KS];
    {
        // rows past the last one read the first row's query; every load is requested before the first is used
        const bf16_t* qp = reinterpret_cast<const bf16_t*>(p.q) + ((int64_t)(q0 + (valid ? qi : 0)) * p.H + h) * dq;
        const float* cs = p.cos_sin + (int64_t)min(max(pos, 0), p.max_pos - 1) * p.rot_pairs * 2;
        const bf16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
        const float sign = p.scale_log2 < 0.f ? -1.f : 1.f;
        f32x4 ca[KS], cb[KS];                                       // (cos, sin) of the four pairs of an 8-element piece
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            const int d = ks * 16 + kh * 8, e = d - p.dim;
            qf[ks] = d < dq ? *reinterpret_cast<const bf16x8*>(qp + d) : z;
            ca[ks] = cb[ks] = f32x4{1.f, 0.f, 1.f, 0.f};
            if (p.rot_pairs % 4 == 0) {                             // uniform: pieces are rotated as a whole or not at all
                if (e >= 0 && e < 2 * p.rot_pairs) {
                    ca[ks] = *reinterpret_cast<const f32x4*>(cs + e);
                    cb[ks] = *reinterpret_cast<const f32x4*>(cs + e + 4);
                }
            } else if (e >= 0) {
#pragma unroll
                for (int u = 0; u < 4; ++u) {
                    if (e + u < 2 * p.rot_pairs) ca[ks][u] = cs[e + u];
                    if (e + 4 + u < 2 * p.rot_pairs) cb[ks][u] = cs[e + 4 + u];
                }
            }
        }
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            f32x8 v = __builtin_convertvector(qf[ks], f32x8);
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const float c = u < 2 ? ca[ks][u * 2] : cb[ks][u * 2 - 4], s = u < 2 ? ca[ks][u * 2 + 1] : cb[ks][u * 2 - 3];
                const float x = v[u * 2], y = v[u * 2 + 1];
                v[u * 2] = (x * c - y * s) * sign;
                v[u * 2 + 1] = (y * c + x * s) * sign;
            }
            qf[ks] = __builtin_convertvector(v, bf16x8);
        }
    }
    if (dq < DK) {                                                  // the images' columns behind a key stay zero
        for (int c = tid; c < 2 * KT * (DK - dq) / 8; c += NT) {
            const int row = c / ((DK - dq) / 8), d = dq + c % ((DK - dq) / 8) * 8;
            *reinterpret_cast<u32x4*>(smem + (row / KT) * STAGE + row % KT * KROW + d * 2) = u32x4{0u, 0u, 0u, 0u};
        }
    }
    f32x16 o[DB];
#pragma unroll
    for (int db = 0; db < DB; ++db)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[db][r] = 0.f;
    float m = -INFINITY, l = 0.f;

    u32x4 kreg[NK], vreg[NV];
    const int ldkv = p.H * (p.dim + p.vdim), hk = h * p.dim, hv = p.H * p.dim + h * p.vdim;
    auto issue = [&](int t) {
        const int kp0 = t * KT, rem = ctx - 1 - kp0;                // rows past the context repeat its last row: they are masked
        const bf16_t* kvb = reinterpret_cast<const bf16_t*>(p.kv) + (int64_t)(c0 + kp0) * ldkv;
        const bf16_t* rpb = reinterpret_cast<const bf16_t*>(p.cache) + p.kv_rank +
                            ((int64_t)p.page_indices[pg0 + kp0 / p.page_size] * p.page_size + kp0 % p.page_size) * p.W;
#pragma unroll
        for (int i = 0; i < NK; ++i) {
            const int c = i * NT + tid, row = min(c / (DK / 8), rem), d = (c % (DK / 8)) * 8;
            const bf16_t* src = d < p.dim ? kvb + (row * ldkv + hk + d) : rpb + (row * p.W + d - p.dim);
            if (d < dq) kreg[i] = *reinterpret_cast<const u32x4*>(src);
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = i * NT + tid, row = min(c / (DV / 8), rem), d = (c % (DV / 8)) * 8;
            if (d < p.vdim) vreg[i] = *reinterpret_cast<const u32x4*>(kvb + (row * ldkv + hv + d));
        }
    };
    auto stage = [&](unsigned char* img) {
#pragma unroll
        for (int i = 0; i < NK; ++i) {
            const int c = i * NT + tid;
            if ((c % (DK / 8)) * 8 < dq) *reinterpret_cast<u32x4*>(img + (c / (DK / 8)) * KROW + (c % (DK / 8)) * 16) = kreg[i];
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {                              // (columns behind a value reach only sums that are not stored)
            const int c = i * NT + tid, row = c / (DV / 8), ch = c % (DV / 8);
            if (ch * 8 < p.vdim)
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
                bf16x8 ph, pl;
                split(pv, ph, pl);
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
