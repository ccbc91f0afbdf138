// Absorbed latent attention on the matrix cores (bf16 pages, gfx950): queries of W numbers per (token, head) against cache rows
// every head shares; the value row is the first kv_rank numbers of the key row, so a key tile is staged once and read twice.
//
// A workgroup owns 16 QT (token, head) rows of one request (token-major) and one range of 64-key tiles.  Per tile
//   1. the tile, requested one iteration ahead (a linear copy: rows of a page are contiguous), goes from registers to LDS;
//   2. S^T = K Q^T on 16x16x32: a wavefront takes 16 keys of one 16-row tile, queries and keys both from LDS; the scaled, masked
//      scores of the whole tile meet in LDS (fp32);
//   3. every wavefront forms the same running maximum and weights for its rows (two 16-byte reads per 32 keys: the weights are
//      the PV operand as they are) and adds O^T += V^T P^T for its share of the kv_rank columns, V^T by transposing LDS reads.
// Weights enter the product as a bf16 part and a bf16 rest (error 2^-17).  Splits leave sums, maximum and weight per row.
#include "attn_common.h"
#include "latent.h"

namespace {

constexpr int KT = 64;
constexpr int kSPitch = KT + 4;                     // floats per score row

__host__ __device__ constexpr int row_pitch(int W) { return W * 2 + 16; }

// QT: 16-row tiles; NBW: 16-column blocks of the latent per wavefront
template <int QT, int NBW>
__global__ __launch_bounds__(256 * QT, 1) void latent_absorbed_kernel(const LatentParams p) {
    constexpr int NW = 4 * QT, NT = 64 * NW, ROWS = 16 * QT;
    constexpr int MAXP = 2 * NBW + 4;               // 16-byte pieces of a tile per thread (W <= 64 NBW QT + 128)
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    const int tid = threadIdx.x, lane = tid & 63, lq = lane & 15, lc = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int W = p.W, pitch = row_pitch(W), R = p.kv_rank;
    unsigned char* ldsK = smem;
    unsigned char* ldsQ = smem + KT * pitch;
    float* ldsS = reinterpret_cast<float*>(ldsQ + ROWS * pitch);

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
    {   // queries of the workgroup; rows past the last one are zero
        const u32x4* src = reinterpret_cast<const u32x4*>(reinterpret_cast<const bf16_t*>(p.q) + ((int64_t)q0 * p.H + row0) * W);
        const int have = min(ROWS, nrows - row0) * per_row;
        for (int c = tid; c < ROWS * per_row; c += NT)
            *reinterpret_cast<u32x4*>(ldsQ + (c / per_row) * pitch + (c % per_row) * 16) = c < have ? src[c] : u32x4{0u, 0u, 0u, 0u};
    }
    int at[MAXP];                                   // LDS byte of this thread's pieces
#pragma unroll
    for (int i = 0; i < MAXP; ++i) {
        const int c = i * NT + tid;
        at[i] = (c / per_row) * pitch + (c % per_row) * 16;
    }
    u32x4 kr[MAXP];
    auto issue = [&](int t) {
        const int pos = t * KT, page = p.page_indices[pg0 + pos / p.page_size];
        const u32x4* src = reinterpret_cast<const u32x4*>(reinterpret_cast<const bf16_t*>(p.cache) +
                                                          ((int64_t)page * p.page_size + pos % p.page_size) * W);
#pragma unroll
        for (int i = 0; i < MAXP; ++i)
            if (i * NT + tid < pieces) kr[i] = __builtin_nontemporal_load(src + i * NT + tid);
    };
    auto stage = [&](int t) {
        const bool tail = t * KT + KT - 1 > written;                // rows not written yet may hold anything (NaN)
#pragma unroll
        for (int i = 0; i < MAXP; ++i)
            if (i * NT + tid < pieces) {
                if (tail && t * KT + (i * NT + tid) / per_row > written) kr[i] = u32x4{0u, 0u, 0u, 0u};
                *reinterpret_cast<u32x4*>(ldsK + at[i]) = kr[i];
            }
    };

    // score step: this wavefront's 16 keys and 16-row tile
    const int ks = wave & 3, rt = wave >> 2;
    const int my_row = row0 + rt * 16 + lq;
    const int lim = my_row < nrows ? min(pos_b + my_row / p.H, cap - 1) : -1;
    const unsigned char* ka = ldsK + (ks * 16 + lq) * pitch + lc * 16;
    const unsigned char* qa = ldsQ + (rt * 16 + lq) * pitch + lc * 16;
    float* s_out = ldsS + (rt * 16 + lq) * kSPitch + ks * 16 + lc * 4;
    const int steps = W / 32;

    f32x4 o[QT][NBW];
    float m[QT], l[QT];
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        m[qt] = -INFINITY;
        l[qt] = 0.f;
#pragma unroll
        for (int nb = 0; nb < NBW; ++nb) o[qt][nb] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const int vra = (lc * 4 + (lq >> 2)) * pitch + (lq & 3) * 8;

    if (t_begin < t_end) issue(t_begin);
    for (int t = t_begin; t < t_end; ++t) {
        stage(t);
        if (t + 1 < t_end) issue(t + 1);
        __syncthreads();
        {
            f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = {0.f, 0.f, 0.f, 0.f};
            int k = 0;
            for (; k + 2 <= steps; k += 2) {
                s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lds_read_b128(ka + k * 64), lds_read_b128(qa + k * 64), s0, 0, 0, 0);
                s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lds_read_b128(ka + k * 64 + 64), lds_read_b128(qa + k * 64 + 64), s1, 0, 0, 0);
            }
            if (k < steps)
                s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lds_read_b128(ka + k * 64), lds_read_b128(qa + k * 64), s0, 0, 0, 0);
            const int kp = t * KT + ks * 16 + lc * 4;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                s0[e] = (s0[e] + s1[e]) * p.scale_log2;
                if (kp + e > lim) s0[e] = -INFINITY;
            }
            *reinterpret_cast<f32x4*>(s_out) = s0;
        }
        __syncthreads();
        bf16x8 ph[QT][2], pl[QT][2];
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) {
            const float* sr = ldsS + (qt * 16 + lq) * kSPitch + lc * 4;
            f32x4 s[4];
            float mx = -INFINITY;
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                s[u] = *reinterpret_cast<const f32x4*>(sr + u * 16);
                mx = fmaxf(mx, fmaxf(fmaxf(s[u][0], s[u][1]), fmaxf(s[u][2], s[u][3])));
            }
            mx = fmaxf(mx, __shfl_xor(mx, 16));
            mx = fmaxf(mx, __shfl_xor(mx, 32));
            const float mn = fmaxf(m[qt], mx), ref = mn == -INFINITY ? 0.f : mn;
            const float alpha = __builtin_amdgcn_exp2f(m[qt] - ref);
            float sum = 0.f;
#pragma unroll
            for (int kk = 0; kk < 2; ++kk) {
                f32x8 pv;
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    pv[e] = __builtin_amdgcn_exp2f(s[kk * 2 + (e >> 2)][e & 3] - ref);
                    sum += pv[e];
                }
                ph[qt][kk] = __builtin_convertvector(pv, bf16x8);
                pl[qt][kk] = __builtin_convertvector(pv - __builtin_convertvector(ph[qt][kk], f32x8), bf16x8);
            }
            l[qt] = l[qt] * alpha + sum;
            if (__any(mn != m[qt])) {
#pragma unroll
                for (int nb = 0; nb < NBW; ++nb) o[qt][nb] *= alpha;
            }
            m[qt] = mn;
        }
#pragma unroll
        for (int nb = 0; nb < NBW; ++nb) {
            const int col = (wave + nb * NW) * 16;
            if (col < R) {                          // wave-uniform
#pragma unroll
                for (int kk = 0; kk < 2; ++kk) {
                    const unsigned char* va = ldsK + vra + kk * 32 * pitch + col * 2;
                    const bf16x4 v0 = lds_read_tr(va), v1 = lds_read_tr(va + 16 * pitch);
                    const bf16x8 vf = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
                    for (int qt = 0; qt < QT; ++qt) {
                        o[qt][nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph[qt][kk], o[qt][nb], 0, 0, 0);
                        o[qt][nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl[qt][kk], o[qt][nb], 0, 0, 0);
                    }
                }
            }
        }
        __syncthreads();
    }

    // o[qt][nb][e] = O[row qt * 16 + lq][(wave + nb * NW) * 16 + lc * 4 + e]
    const int Rp = (R + 15) / 16 * 16;
    const int64_t slot = ((int64_t)b * p.n_groups + group) * p.nsplit + split;
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        l[qt] += __shfl_xor(l[qt], 16);
        l[qt] += __shfl_xor(l[qt], 32);
        const int r = qt * 16 + lq;
        const bool valid = row0 + r < nrows;
        const float inv = l[qt] > 0.f ? 1.0f / l[qt] : 0.f;
        if (p.nsplit > 1 && wave == 0 && lc == 0) {
            float* ml = p.ws + (int64_t)p.B * p.n_groups * p.nsplit * ROWS * Rp + (slot * ROWS + r) * 2;
            ml[0] = m[qt];
            ml[1] = l[qt];
        }
#pragma unroll
        for (int nb = 0; nb < NBW; ++nb) {
            const int c = (wave + nb * NW) * 16 + lc * 4;
            if ((wave + nb * NW) * 16 >= R) continue;
            if (p.nsplit > 1) {
                *reinterpret_cast<f32x4*>(p.ws + (slot * ROWS + r) * Rp + c) = o[qt][nb];
                continue;
            }
            if (!valid) continue;
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

int lds_bytes(int W, int qt) { return (KT + 16 * qt) * row_pitch(W) + 16 * qt * kSPitch * 4; }

template <int QT, int NBW>
int launch(const LatentParams& p, hipStream_t st) {
    auto k = latent_absorbed_kernel<QT, NBW>;
    static MdPerDeviceOnce once;
    if (once.first() && hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize,
                                            160 * 1024) != hipSuccess) {
        once.undo();
        md_set_error("md_latent_attn: hipFuncSetAttribute(LDS) failed");
        return MD_ERR_LAUNCH;
    }
    const int64_t grid = (int64_t)p.B * p.n_groups * p.nsplit;
    MD_CHECK_ARG(grid < ((int64_t)1 << 31), "md_latent_attn: grid too large");
    hipLaunchKernelGGL(k, dim3((unsigned)grid), dim3(256 * QT), lds_bytes(p.W, QT), st, p);
    return MD_OK;
}

// column blocks per wavefront (a power of two) that cover kv_rank and whose piece count covers W; 0: none
int blocks_per_wave(int kv_rank, int W, int qt) {
    for (int n = 1; n * qt <= 8; n *= 2)
        if (kv_rank <= 64 * n * qt && W <= 64 * n * qt + 128) return n;
    return 0;
}

}  // namespace

bool md_internal_latent_absorbed_ok(int kv_rank, int W, int qt) {
    return blocks_per_wave(kv_rank, W, qt) > 0 && lds_bytes(W, qt) <= 160 * 1024;
}

int md_internal_latent_absorbed(const LatentParams& p, int qt, hipStream_t st) {
    const int n = blocks_per_wave(p.kv_rank, p.W, qt);
    if (qt == 1) return n == 1 ? launch<1, 1>(p, st) : n == 2 ? launch<1, 2>(p, st) : n == 4 ? launch<1, 4>(p, st) : launch<1, 8>(p, st);
    return n == 1 ? launch<2, 1>(p, st) : n == 2 ? launch<2, 2>(p, st) : launch<2, 4>(p, st);
}
