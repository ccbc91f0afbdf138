// Absorbed latent attention on the matrix cores (bf16 pages, gfx950): queries of W numbers per (token, head) against cache rows
// every head shares; the value row is the first kv_rank numbers of the key row, so a key tile is staged once and read twice.
//
// A workgroup of 4 QT wavefronts owns 16 QT (token, head) rows of one request (token-major) and one range of 32-key tiles.  A
// tile passes through three steps, two of which overlap with a neighbour's, so that a tile costs two barriers:
//   * O^T += V^T P^T of tile t - 1: every wavefront takes its share of the kv_rank columns, V^T by transposing LDS reads -- beside
//     S^T = K Q^T of tile t: a wavefront takes 16 keys and 1 / (2 QT) of the depth for all rows; partial scores meet in LDS (fp32);
//   * weights of tile t: 16 lanes per row add the partial scores, mask, follow the maximum -- lazily: the reference moves only when
//     a tile exceeds it by 8 in the exponent -- and leave the weights in LDS as a bf16 part and a bf16 rest (error 2^-17), in
//     operand order -- beside the copy of tile t + 1, requested two tiles earlier (rows of a page are contiguous), into the image
//     that tile t - 1 has left.
// Splits leave sums, reference and weight per row.
#include "attn_common.h"
#include "latent.h"

#include <type_traits>

namespace {

constexpr int KT = 32;
constexpr int kSPitch = KT + 4;                     // floats per score row (the four behind it: the row's factor)
constexpr int kPPitch = KT * 2 + 16;                // bytes per weight row

__host__ __device__ constexpr int row_pitch(int W) { return W * 2 + 16; }

// over the 16 lanes of a row (rotations within it: no LDS)
template <int N>
__device__ __forceinline__ float row_ror(float v) {
    return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x120 + N, 0xf, 0xf, false));
}
__device__ __forceinline__ float row_max(float v) {
    v = fmaxf(v, row_ror<8>(v));
    v = fmaxf(v, row_ror<4>(v));
    v = fmaxf(v, row_ror<2>(v));
    return fmaxf(v, row_ror<1>(v));
}
__device__ __forceinline__ float row_sum(float v) {
    v += row_ror<8>(v);
    v += row_ror<4>(v);
    v += row_ror<2>(v);
    return v + row_ror<1>(v);
}

// QT: 16-row tiles; NBW: 16-column blocks of the latent per wavefront; KS: 32-deep steps of a score where known at compile time (a
// wavefront's queries then live in registers), 0: any
template <int QT, int NBW, int KS>
__global__ __launch_bounds__(256 * QT, 2) void latent_absorbed_kernel(const LatentParams p) {
    constexpr int ROWS = 16 * QT, NT = 256 * QT, PARTS = 2 * QT;                 // PARTS: of a score's depth
    constexpr int MAXP = KS ? (KS * 128 + NT - 1) / NT : NBW + 2;                // 16-byte pieces of a tile per thread
    constexpr int KH = (KS + PARTS - 1) / PARTS;
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    const int tid = threadIdx.x, lane = tid & 63, lq = lane & 15, lc = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int W = KS ? KS * 32 : p.W, pitch = row_pitch(W), R = p.kv_rank, image = KT * pitch;
    unsigned char* ldsQ = smem + 2 * image;
    // scores [part][row][key]; behind a row of part 0: the row's factor
    float* ldsS = reinterpret_cast<float*>(ldsQ + (KS ? 0 : ROWS * pitch));
    unsigned char* ldsP = reinterpret_cast<unsigned char*>(ldsS + PARTS * ROWS * kSPitch);   // weights: bf16 parts, then rests

    // request fastest: with a multiple of 8 requests one request's workgroups share an XCD (and its L2)
    const int b = blockIdx.x % p.B, sub = blockIdx.x / p.B, group = sub % p.n_groups, split = sub / p.n_groups;
    const int q0 = p.qo_indptr[b], n_b = p.qo_indptr[b + 1] - q0, nrows = n_b * p.H, row0 = group * ROWS;
    if (row0 >= nrows) return;                      // whole workgroup
    const int pos_b = p.pos0[b], pg0 = p.page_indptr[b], cap = (p.page_indptr[b + 1] - pg0) * p.page_size;
    const int written = min(pos_b + n_b - 1, cap - 1);              // last row of the cache that holds something
    const int last = min(pos_b + (min(row0 + ROWS, nrows) - 1) / p.H, cap - 1);
    const int ntiles = last >= 0 ? last / KT + 1 : 0;
    const int tps = (ntiles + p.nsplit - 1) / p.nsplit;
    const int t_begin = split * tps, t_end = min(ntiles, t_begin + tps);

    const int per_row = W / 8, pieces = KT * per_row;
    int at[MAXP];                                   // LDS byte of this thread's pieces
#pragma unroll
    for (int i = 0; i < MAXP; ++i) {
        const int c = i * NT + tid;
        at[i] = (c / per_row) * pitch + (c % per_row) * 16;
    }
    auto issue = [&](int t, u32x4 (&kr)[MAXP]) {
        const int pos = t * KT, page = p.page_indices[pg0 + pos / p.page_size];
        const u32x4* src = reinterpret_cast<const u32x4*>(reinterpret_cast<const bf16_t*>(p.cache) +
                                                          ((int64_t)page * p.page_size + pos % p.page_size) * W);
#pragma unroll
        for (int i = 0; i < MAXP; ++i)
            if ((KS > 0 && KS * 128 % NT == 0) || i * NT + tid < pieces) kr[i] = __builtin_nontemporal_load(src + i * NT + tid);
    };
    auto stage = [&](int t, unsigned char* img, u32x4 (&kr)[MAXP]) {
        if (t * KT + KT - 1 > written) {                            // rows not written yet may hold anything (NaN)
#pragma unroll
            for (int i = 0; i < MAXP; ++i)
                if (t * KT + (i * NT + tid) / per_row > written) kr[i] = u32x4{0u, 0u, 0u, 0u};
        }
#pragma unroll
        for (int i = 0; i < MAXP; ++i)
            if ((KS > 0 && KS * 128 % NT == 0) || i * NT + tid < pieces) *reinterpret_cast<u32x4*>(img + at[i]) = kr[i];
    };
    u32x4 kx[MAXP], ky[MAXP];
    if (t_begin < t_end) issue(t_begin, kx);
    if (t_begin + 1 < t_end) issue(t_begin + 1, ky);

    // score step: this wavefront's 16 keys and part of the depth
    const int ks = wave & 1, part = wave >> 1;
    const int steps = W / 32, k_begin = part * steps / PARTS, k_end = (part + 1) * steps / PARTS;
    const int ka = (ks * 16 + lq) * pitch + lc * 16 + k_begin * 64;
    const unsigned char* qa = ldsQ + lq * pitch + lc * 16 + k_begin * 64;
    float* s_out = ldsS + (part * ROWS + lq) * kSPitch + ks * 16 + lc * 4;
    bf16x8 qf[QT][KS ? KH : 1];
    if constexpr (KS > 0) {
        const bf16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) {
            const bf16_t* qp = reinterpret_cast<const bf16_t*>(p.q) + ((int64_t)q0 * p.H + min(row0 + qt * 16 + lq, nrows - 1)) * W +
                               k_begin * 32 + lc * 8;
#pragma unroll
            for (int k = 0; k < KH; ++k) qf[qt][k] = k_begin + k < k_end ? *reinterpret_cast<const bf16x8*>(qp + k * 32) : z;
        }
    } else {                                        // queries of the workgroup; rows past the last one are zero
        const u32x4* src = reinterpret_cast<const u32x4*>(reinterpret_cast<const bf16_t*>(p.q) + ((int64_t)q0 * p.H + row0) * W);
        const int have = min(ROWS, nrows - row0) * per_row;
        for (int c = tid; c < ROWS * per_row; c += NT)
            *reinterpret_cast<u32x4*>(ldsQ + (c / per_row) * pitch + (c % per_row) * 16) = c < have ? src[c] : u32x4{0u, 0u, 0u, 0u};
    }
    // weight step: this lane's row and two keys; key k of a tile stands at (k / 4 % 4) * 8 + k / 16 * 4 + k % 4
    const int wr = tid >> 4, wk = (tid & 15) * 2;
    const int lim = row0 + wr < nrows ? min(pos_b + (row0 + wr) / p.H, cap - 1) : -1;
    float* s_in = ldsS + wr * kSPitch;
    unsigned char* p_out = ldsP + wr * kPPitch + ((wk >> 2 & 3) * 8 + (wk >> 4) * 4 + (wk & 3)) * 2;
    const unsigned char* p_in = ldsP + lq * kPPitch + lc * 16;
    float m = -INFINITY, l = 0.f;

    f32x4 o[QT][NBW];
#pragma unroll
    for (int qt = 0; qt < QT; ++qt)
#pragma unroll
        for (int nb = 0; nb < NBW; ++nb) o[qt][nb] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int va = (lc * 4 + (lq >> 2)) * pitch + (lq & 3) * 8 + wave * NBW * 32;

    auto scores = [&](const unsigned char* img) {
        f32x4 s[QT];
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) s[qt] = f32x4{0.f, 0.f, 0.f, 0.f};
        if constexpr (KS > 0) {
#pragma unroll
            for (int k = 0; k < KH; ++k) {          // (a shorter part's last step multiplies by zeros)
                const bf16x8 kf = lds_read_b128(img + ka + (KS % PARTS == 0 || k_begin + k < k_end ? k : 0) * 64);
#pragma unroll
                for (int qt = 0; qt < QT; ++qt) s[qt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[qt][k], s[qt], 0, 0, 0);
            }
        } else {
            for (int k = 0; k < k_end - k_begin; ++k) {
                const bf16x8 kf = lds_read_b128(img + ka + k * 64);
#pragma unroll
                for (int qt = 0; qt < QT; ++qt)
                    s[qt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, lds_read_b128(qa + qt * 16 * pitch + k * 64), s[qt], 0, 0, 0);
            }
        }
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) *reinterpret_cast<f32x4*>(s_out + qt * 16 * kSPitch) = s[qt];
    };
    auto weights = [&](int t) {
        f32x2 s = {0.f, 0.f};
#pragma unroll
        for (int u = 0; u < PARTS; ++u) s += *reinterpret_cast<const f32x2*>(s_in + u * ROWS * kSPitch + wk);
        s *= p.scale_log2;
#pragma unroll
        for (int e = 0; e < 2; ++e)
            if (t * KT + wk + e > lim) s[e] = -INFINITY;
        const float mx = row_max(fmaxf(s[0], s[1]));
        float alpha = 1.f;
        if (mx > m + 8.f) {
            alpha = __builtin_amdgcn_exp2f(m - mx);
            m = mx;
        }
        const float ref = m == -INFINITY ? 0.f : m;                 // (nothing seen yet: the weights below are 0)
        const f32x2 w = {__builtin_amdgcn_exp2f(s[0] - ref), __builtin_amdgcn_exp2f(s[1] - ref)};
        l = l * alpha + (w[0] + w[1]);
        const bf16x2 hi = __builtin_convertvector(w, bf16x2);
        *reinterpret_cast<bf16x2*>(p_out) = hi;
        *reinterpret_cast<bf16x2*>(p_out + ROWS * kPPitch) = __builtin_convertvector(w - __builtin_convertvector(hi, f32x2), bf16x2);
        if (wk == 0) s_in[KT] = alpha;
    };
    auto values = [&](const unsigned char* img) {
        bf16x8 ph[QT], pl[QT];
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) {
            ph[qt] = lds_read_b128(p_in + qt * 16 * kPPitch);
            pl[qt] = lds_read_b128(p_in + (ROWS + qt * 16) * kPPitch);
            const float alpha = ldsS[(qt * 16 + lq) * kSPitch + KT];
            if (__any(alpha != 1.f)) {
#pragma unroll
                for (int nb = 0; nb < NBW; ++nb) o[qt][nb] *= alpha;
            }
        }
#pragma unroll
        for (int nb = 0; nb < NBW; ++nb)
            if (KS || (wave * NBW + nb) * 16 < R) { // wave-uniform
                const unsigned char* v = img + va + nb * 32;
                const bf16x4 v0 = lds_read_tr(v), v1 = lds_read_tr(v + 16 * pitch);
                const bf16x8 vf = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
                for (int qt = 0; qt < QT; ++qt) o[qt][nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph[qt], o[qt][nb], 0, 0, 0);
#pragma unroll
                for (int qt = 0; qt < QT; ++qt) o[qt][nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl[qt], o[qt][nb], 0, 0, 0);
            }
    };

    // tile t_begin + i lies in image i & 1 and is requested through kx (i even) or ky
    auto tile = [&](auto first, auto steady, int t, unsigned char* img, unsigned char* other, u32x4 (&kr)[MAXP]) {
        if constexpr (!decltype(first)::value) values(other);
        scores(img);
        __syncthreads();
        weights(t);
        if (decltype(steady)::value || t + 1 < t_end) stage(t + 1, other, kr);
        if (decltype(steady)::value || t + 3 < t_end) issue(t + 3, kr);
        __syncthreads();
    };
    unsigned char* img0 = smem;
    unsigned char* img1 = smem + image;
    if (t_begin < t_end) {
        stage(t_begin, img0, kx);
        if (t_begin + 2 < t_end) issue(t_begin + 2, kx);
        __syncthreads();
        tile(std::true_type{}, std::false_type{}, t_begin, img0, img1, ky);
        int t = t_begin + 1;
        for (; t + 4 < t_end; t += 2) {             // branch-free prefetch: the waits count only the tile being copied
            tile(std::false_type{}, std::true_type{}, t, img1, img0, kx);
            tile(std::false_type{}, std::true_type{}, t + 1, img0, img1, ky);
        }
        for (; t < t_end; t += 2) {
            tile(std::false_type{}, std::false_type{}, t, img1, img0, kx);
            if (t + 1 < t_end) tile(std::false_type{}, std::false_type{}, t + 1, img0, img1, ky);
        }
        values((t_end - 1 - t_begin) & 1 ? img1 : img0);
    }
    __syncthreads();

    // o[qt][nb][e] = O[row qt * 16 + lq][(wave * NBW + nb) * 16 + lc * 4 + e]
    const int Rp = (R + 15) / 16 * 16;
    const int64_t slot = ((int64_t)b * p.n_groups + group) * p.nsplit + split;
    l = row_sum(l);
    if (wk == 0) {
        s_in[KT] = l > 0.f ? 1.0f / l : 0.f;
        if (p.nsplit > 1) {
            float* ml = p.ws + (int64_t)p.B * p.n_groups * p.nsplit * ROWS * Rp + (slot * ROWS + wr) * 2;
            ml[0] = m;
            ml[1] = l;
        }
    }
    __syncthreads();
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        const int r = qt * 16 + lq;
        const float inv = ldsS[r * kSPitch + KT];
#pragma unroll
        for (int nb = 0; nb < NBW; ++nb) {
            const int c = (wave * NBW + nb) * 16 + lc * 4;
            if ((wave * NBW + nb) * 16 >= R) continue;
            if (p.nsplit > 1) {
                *reinterpret_cast<f32x4*>(p.ws + (slot * ROWS + r) * Rp + c) = o[qt][nb];
                continue;
            }
            if (row0 + r >= nrows) continue;
            bf16_t* op = reinterpret_cast<bf16_t*>(p.out) + ((int64_t)q0 * p.H + row0 + r) * R + c;
            if (R % 4 == 0) {
                if (c < R) *reinterpret_cast<bf16x4*>(op) = __builtin_convertvector(o[qt][nb] * inv, bf16x4);
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (c + e < R) op[e] = f32_to_bf16(o[qt][nb][e] * inv);
            }
        }
    }
}

int lds_bytes(int W, int qt, bool q_in_regs) {
    return (2 * KT + (q_in_regs ? 0 : 16 * qt)) * row_pitch(W) + 16 * qt * (2 * qt * kSPitch * 4 + 2 * kPPitch);
}

template <int QT, int NBW, int KS = 0>
int launch(const LatentParams& p, hipStream_t st) {
    auto k = latent_absorbed_kernel<QT, NBW, KS>;
    static MdPerDeviceOnce once;
    if (once.first() && hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize,
                                            160 * 1024) != hipSuccess) {
        once.undo();
        md_set_error("md_latent_attn: hipFuncSetAttribute(LDS) failed");
        return MD_ERR_LAUNCH;
    }
    const int64_t grid = (int64_t)p.B * p.n_groups * p.nsplit;
    MD_CHECK_ARG(grid < ((int64_t)1 << 31), "md_latent_attn: grid too large");
    hipLaunchKernelGGL(k, dim3((unsigned)grid), dim3(256 * QT), lds_bytes(p.W, QT, KS > 0), st, p);
    return MD_OK;
}

// column blocks per wavefront (a power of two) that cover kv_rank and whose MAXP pieces cover a tile of rows of W; 0: none
int blocks_per_wave(int kv_rank, int W, int qt) {
    for (int n = 1; n * qt <= 8; n *= 2)
        if (kv_rank <= 64 * n * qt && W <= 64 * n * qt + 128) return n;
    return 0;
}

}  // namespace

bool md_internal_latent_absorbed_ok(int kv_rank, int W, int qt) {
    return blocks_per_wave(kv_rank, W, qt) > 0 && lds_bytes(W, qt, false) <= 160 * 1024;
}

int md_internal_latent_absorbed(const LatentParams& p, int qt, hipStream_t st) {
    if (p.kv_rank == 512 && p.W == 576) return qt == 1 ? launch<1, 8, 18>(p, st) : launch<2, 4, 18>(p, st);   // usual for large models
    const int n = blocks_per_wave(p.kv_rank, p.W, qt);
    if (qt == 1) return n == 1 ? launch<1, 1>(p, st) : n == 2 ? launch<1, 2>(p, st) : n == 4 ? launch<1, 4>(p, st) : launch<1, 8>(p, st);
    return n == 1 ? launch<2, 1>(p, st) : n == 2 ? launch<2, 2>(p, st) : launch<2, 4>(p, st);
}
