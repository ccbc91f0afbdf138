// Matrix-core kernels of the extended paged attention (xattn.hip; bf16 pages).  Compiled once per padded query/key width:
// -DMD_XATTN_DK=32 | 64 | 96 | 128 | 192 | 256; the value width is a template parameter of the same set.
//
// No running maximum.  Query and key heads have unit RMS, so |q.k| <= dim and a score never exceeds
// dim * scale (plus what a negative bias coefficient can add): the host passes that bound, and softmax weights are taken
// against the FIXED reference max(0, bound - 60) instead of the row's maximum.  The sink (weight exp(-reference)) keeps the
// denominator away from 0, weights below exp(-87) of the reference are negligible next to it, and with the maximum gone
//   * there is no rescaling, no max reduction, and no second pass over a tile's scores: a 32-key block goes from its S
//     accumulator to P to the PV product at once, 16 + 16 registers instead of a whole tile's worth;
//   * partial sums of wavefronts and of kv splits simply add up.
// The distance bias is taken in the log2 domain (r1 ln(x) = (r1 log2 x) in the exp2 argument).  Decode evaluates it per score
// (fma + v_log_f32 + fma: 8 scores per lane and tile); prefill looks it up: a workgroup's rows and a key tile meet at only
// KT + tokens different distances, so the workgroup fills a small table per head and tile (a few logarithms per thread instead
// of one per score) and every score is one fma with a table entry.  Negative distances hold -inf: the causal mask is the table.
//
// P is kept to 16 significant bits: the bf16 weight and the bf16 rest of it feed two PV products, so that the attention
// weights reach the 32-bit accumulator with an error of 2^-17 instead of 2^-9.
//
// A key tile of one head is one contiguous block of its page (rows padded to DK / DV, heads outermost inside a page), whatever
// the row width: staging is a linear copy in 16-byte pieces.
#include "attn_common.h"
#include "xattn.h"

#ifndef MD_XATTN_DK
#error "compile with -DMD_XATTN_DK=<padded query/key head size>"
#endif

namespace {

typedef float f32x16 __attribute__((ext_vector_type(16)));
constexpr int DK = MD_XATTN_DK;
constexpr int KROW = DK * 2 + 16;        // K image row pitch

template <int DV>
constexpr int stage_bytes(int kt) { return kt * KROW + (kt / 32) * (DV / 16) * kVSub; }

// exp2 argument -> weight; bf16 part and bf16 rest
__device__ __forceinline__ void split_bf16(const f32x8 p, bf16x8& hi, bf16x8& lo) {
    hi = __builtin_convertvector(p, bf16x8);
    lo = __builtin_convertvector(p - __builtin_convertvector(hi, f32x8), bf16x8);
}

// ------------------------------------------------------------------------------------------------ decode / verify
template <int DV, int QT>
constexpr int decode_wave_lds() {
    const int stage = stage_bytes<DV>(32), merge = QT * 16 * DV * 4 + QT * 16 * 4;
    return ((stage > merge ? stage : merge) + 255) / 256 * 256;
}

// 16-byte loads in flight per wavefront: two tiles where the register budget allows it (256 registers at two workgroups per
// CU, 512 where the LDS images leave room for one anyway), else one
template <int DV, int QT>
constexpr int decode_wgs() { return 4 * decode_wave_lds<DV, QT>() > 80 * 1024 ? 1 : 2; }
template <int DV, int QT>
constexpr int decode_tiles_in_flight() {
    const int regs = 2 * (DK + DV) / 4 + QT * (DV / 4 + DK / 8);
    return regs <= (decode_wgs<DV, QT>() == 1 ? 400 : 176) ? 2 : 1;
}

// Four wavefronts share one (request, kv head, kv split); each owns a stream of 32-key tiles (two in flight in registers),
// no barrier in the loop.  S^T = K Q^T and O^T = V^T P^T on 16x16x32; the S accumulator is the PV operand.
// FUSED: q holds the RAW projection rows (q | k | v of the step's tokens): the q heads are normalised in registers, and the
// wavefront that owns the tile a new key falls into normalises it, puts it into its LDS image and appends it to the pages.
template <int DV, int QT, bool FUSED>
__global__ __launch_bounds__(256, (decode_wgs<DV, QT>())) void xattn_decode_kernel(const XattnParams p) {
    constexpr int KS = DK / 32, NB = DV / 16;
    constexpr int NK = DK / 16, NV = DV / 16;          // 16-byte pieces per lane of a 32-key K / V tile
    constexpr int WAVE_LDS = decode_wave_lds<DV, QT>();
    constexpr int NS = decode_tiles_in_flight<DV, QT>(), PF = 4 * NS;      // prefetch distance in tiles
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    const int tid = threadIdx.x, lane = tid & 63, lq = lane & 15, lc = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    // blocks of one (request, kv head) differ by multiples of 8: same XCD, shared L2
    const int r0 = blockIdx.x >> 3;
    const int split = r0 % p.nsplit, pair = (r0 / p.nsplit) * 8 + (blockIdx.x & 7);
    if (pair >= p.B * p.KH) return;
    const int b = pair / p.KH, kvh = pair % p.KH, g = p.g;
    const int q0 = p.qo_indptr[b], n_b = p.qo_indptr[b + 1] - q0;
    const int pos_b = p.pos0[b], pg0 = p.page_indptr[b];
    const int cap = (p.page_indptr[b + 1] - pg0) * p.page_size;
    const int nrows = n_b * g;
    const int last = min(pos_b + n_b - 1, cap - 1);
    const int t_first = ((pos_b / p.chunk) * p.chunk) >> 5;
    const int ntiles = n_b > 0 && last >= 0 ? (last >> 5) - t_first + 1 : 0;
    const int tps = (ntiles + p.nsplit - 1) / p.nsplit;
    const int t_begin = t_first + split * tps, t_end = min(t_first + ntiles, t_begin + tps);

    int lim[QT], low[QT];
    float r1[QT], r2[QT], qpos[QT];
    int lim_min = 0x7fffffff, low_max = -1;
    bf16x8 qf[QT][KS];
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        const int R = qt * 16 + lq;
        const bool valid = R < nrows;
        const int i = valid ? R / g : 0, r = valid ? R - i * g : 0, h = kvh * g + r;
        const int pos = pos_b + i;
        lim[qt] = valid ? min(pos, cap - 1) : -1;
        low[qt] = (pos / p.chunk) * p.chunk;
        if (valid) {
            lim_min = min(lim_min, lim[qt]);
            low_max = max(low_max, low[qt]);
        }
        qpos[qt] = (float)pos;
        r1[qt] = p.r1 ? p.r1[h] : 0.f;
        r2[qt] = p.r2 ? p.r2[h] : 0.f;
        const bf16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
        if constexpr (FUSED) {
            const bf16_t* qp = reinterpret_cast<const bf16_t*>(p.qkv) + (int64_t)(q0 + i) * p.ld_qkv + h * p.D;
            f32x8 v[KS];
            float ss = 0.f;
#pragma unroll
            for (int s = 0; s < KS; ++s) {
                const int d0 = s * 32 + lc * 8;
                v[s] = __builtin_convertvector(valid && d0 < p.D ? *reinterpret_cast<const bf16x8*>(qp + d0) : z, f32x8);
#pragma unroll
                for (int e = 0; e < 8; ++e) ss += v[s][e] * v[s][e];
            }
            ss += __shfl_xor(ss, 16);
            ss += __shfl_xor(ss, 32);
            const float rs = 1.0f / sqrtf(ss / (float)p.D + p.eps);
#pragma unroll
            for (int s = 0; s < KS; ++s) qf[qt][s] = __builtin_convertvector(v[s] * rs, bf16x8);
        } else {
            const bf16_t* qp = reinterpret_cast<const bf16_t*>(p.q) + ((int64_t)(q0 + i) * p.H + h) * DK;
#pragma unroll
            for (int s = 0; s < KS; ++s) qf[qt][s] = valid ? *reinterpret_cast<const bf16x8*>(qp + s * 32 + lc * 8) : z;
        }
    }
#pragma unroll
    for (int o = 1; o < 16; o <<= 1) {
        lim_min = min(lim_min, __shfl_xor(lim_min, o));
        low_max = max(low_max, __shfl_xor(low_max, o));
    }
    lim_min = __builtin_amdgcn_readfirstlane(lim_min);
    low_max = __builtin_amdgcn_readfirstlane(low_max);

    f32x4 o[QT][NB];
    float l[QT];
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        l[qt] = 0.f;
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) o[qt][nb] = f32x4{0.f, 0.f, 0.f, 0.f};
    }

    unsigned char* ldsK = smem + wave * WAVE_LDS;
    unsigned char* ldsV = ldsK + 32 * KROW;
    // piece c of a tile: row c / (D/8), 16-byte column c % (D/8)
    auto k_addr = [](int c) { return (c / (DK / 8)) * KROW + (c % (DK / 8)) * 16; };
    auto v_addr = [](int row, int ch) { return (ch >> 1) * kVSub + row * 32 + (ch & 1) * 16; };
    const int kra = lq * KROW + lc * 16;
    const int vra = (lc * 4 + (lq >> 2)) * 32 + (lq & 3) * 8;

    auto issue = [&](int t, u32x4 (&kr)[NK], u32x4 (&vr)[NV]) {
        const int pos = t * 32, page = pos / p.page_size, slot = pos - page * p.page_size;
        const int pid = __builtin_amdgcn_readfirstlane(p.page_indices[pg0 + page]);
        const int64_t row = ((int64_t)pid * p.KH + kvh) * p.page_size + slot;
        const u32x4* kp = reinterpret_cast<const u32x4*>(reinterpret_cast<const bf16_t*>(p.k_cache) + row * DK);
        const u32x4* vp = reinterpret_cast<const u32x4*>(reinterpret_cast<const bf16_t*>(p.v_cache) + row * DV);
#pragma unroll
        for (int i = 0; i < NK; ++i) kr[i] = __builtin_nontemporal_load(kp + i * 64 + lane);
#pragma unroll
        for (int i = 0; i < NV; ++i) vr[i] = __builtin_nontemporal_load(vp + i * 64 + lane);
    };
    auto process = [&](auto steady, int t, u32x4 (&kr)[NK], u32x4 (&vr)[NV]) {
        const int tail = t * 32 + 31;
        const bool masked = tail > lim_min || t * 32 < low_max;
        // rows past the last valid one may hold anything (even NaN): V becomes 0 there, so that 0 * V stays 0
#pragma unroll
        for (int i = 0; i < NK; ++i) *reinterpret_cast<u32x4*>(ldsK + k_addr(i * 64 + lane)) = kr[i];
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = i * 64 + lane, row = c / (DV / 8);
            if (tail > last && t * 32 + row > last) vr[i] = u32x4{0u, 0u, 0u, 0u};
            *reinterpret_cast<u32x4*>(ldsV + v_addr(row, c % (DV / 8))) = vr[i];
        }
        if constexpr (decltype(steady)::value) {
            issue(t + PF, kr, vr);
        } else {
            if (t + PF < t_end) issue(t + PF, kr, vr);
        }
        if constexpr (FUSED) {
            if (tail >= pos_b) {                    // wave-uniform: this tile takes (some of) the step's own keys
                for (int i = max(0, t * 32 - pos_b); i < n_b && pos_b + i <= min(tail, cap - 1); ++i) {
                    const bf16_t* src = reinterpret_cast<const bf16_t*>(p.qkv) + (int64_t)(q0 + i) * p.ld_qkv + p.H * p.D;
                    const int pos = pos_b + i, row = pos & 31;
                    const int pid = p.page_indices[pg0 + pos / p.page_size];
                    const int64_t crow = ((int64_t)pid * p.KH + kvh) * p.page_size + pos % p.page_size;
                    const bf16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
                    const bf16x8 kv = lane * 8 < p.D ? *reinterpret_cast<const bf16x8*>(src + kvh * p.D + lane * 8) : z;
                    const f32x8 kf = __builtin_convertvector(kv, f32x8);
                    float ss = 0.f;
#pragma unroll
                    for (int e = 0; e < 8; ++e) ss += kf[e] * kf[e];
                    const float rs = 1.0f / sqrtf(wave_reduce_sum(ss) / (float)p.D + p.eps);
                    if (lane < DK / 8) {
                        const bf16x8 kn = __builtin_convertvector(kf * rs, bf16x8);
                        *reinterpret_cast<bf16x8*>(ldsK + row * KROW + lane * 16) = kn;
                        *reinterpret_cast<bf16x8*>(reinterpret_cast<bf16_t*>(p.k_cache) + crow * DK + lane * 8) = kn;
                    }
                    if (lane < DV / 8) {
                        const bf16x8 vn = lane * 8 < p.DV
                            ? *reinterpret_cast<const bf16x8*>(src + p.KH * p.D + kvh * p.DV + lane * 8) : z;
                        *reinterpret_cast<bf16x8*>(ldsV + v_addr(row, lane)) = vn;
                        *reinterpret_cast<bf16x8*>(reinterpret_cast<bf16_t*>(p.v_cache) + crow * DV + lane * 8) = vn;
                    }
                }
            }
        }
        __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");      // same-wave LDS hand-off: LDS ops of a wave are in order
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");

        f32x4 s[QT][2];
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) s[qt][0] = s[qt][1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
#pragma unroll
            for (int kb = 0; kb < 2; ++kb) {
                const bf16x8 kf = lds_read_b128(ldsK + kra + kb * 16 * KROW + ks * 64);
#pragma unroll
                for (int qt = 0; qt < QT; ++qt)
                    s[qt][kb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[qt][ks], s[qt][kb], 0, 0, 0);
            }
        bf16x8 ph[QT], pl[QT];
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) {
            f32x8 pv;
#pragma unroll
            for (int kb = 0; kb < 2; ++kb)
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const int kpos = t * 32 + kb * 16 + lc * 4 + j;
                    const float dist = qpos[qt] - (float)kpos;
                    const float lg = __builtin_amdgcn_logf(fmaf(r2[qt], dist, 1.0f));
                    float e = fmaf(s[qt][kb][j], p.scale_log2, -p.ref_log2) - r1[qt] * lg;
                    if (masked && (kpos > lim[qt] || kpos < low[qt])) e = -INFINITY;
                    pv[kb * 4 + j] = __builtin_amdgcn_exp2f(e);
                    l[qt] += pv[kb * 4 + j];
                }
            split_bf16(pv, ph[qt], pl[qt]);
        }
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) {
            const bf16x4 v0 = lds_read_tr(ldsV + nb * kVSub + vra), v1 = lds_read_tr(ldsV + nb * kVSub + 512 + vra);
            const bf16x8 vf = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
            for (int qt = 0; qt < QT; ++qt) {
                o[qt][nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph[qt], o[qt][nb], 0, 0, 0);
                o[qt][nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl[qt], o[qt][nb], 0, 0, 0);
            }
        }
        __builtin_amdgcn_wave_barrier();
    };

    if constexpr (NS == 1) {
        u32x4 ka[NK], va[NV];
        int t = t_begin + wave;
        if (t < t_end) issue(t, ka, va);
        for (; t + 4 < t_end; t += 4) process(std::true_type{}, t, ka, va);
        if (t < t_end) process(std::false_type{}, t, ka, va);
    } else {
        u32x4 ka[NK], va[NV], kb[NK], vb[NV];
        int t = t_begin + wave;
        if (t < t_end) issue(t, ka, va);
        if (t + 4 < t_end) issue(t + 4, kb, vb);
        for (; t + 12 < t_end; t += 8) {             // branch-free prefetch: the waits count only the tile being consumed
            process(std::true_type{}, t, ka, va);
            process(std::true_type{}, t + 4, kb, vb);
        }
        for (; t < t_end; t += 8) {
            process(std::false_type{}, t, ka, va);
            if (t + 4 < t_end) process(std::false_type{}, t + 4, kb, vb);
        }
    }
    if constexpr (FUSED) {
        if (split == 0 && kvh == 0 && tid == 0 && n_b > 0 && pos_b + n_b > cap)
            atomicAdd(p.overflow, (unsigned int)(pos_b + n_b - max(cap, pos_b)));
    }

    // partial sums of the four wavefronts through LDS: o[qt][nb][j] = O[row qt*16 + lq][nb*16 + lc*4 + j]
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        l[qt] += __shfl_xor(l[qt], 16);
        l[qt] += __shfl_xor(l[qt], 32);
    }
    __syncthreads();
    float* ro = reinterpret_cast<float*>(ldsK);
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) *reinterpret_cast<f32x4*>(ro + (qt * 16 + lq) * DV + nb * 16 + lc * 4) = o[qt][nb];
        if (lc == 0) ro[QT * 16 * DV + qt * 16 + lq] = l[qt];
    }
    __syncthreads();
    const int64_t slot = (int64_t)pair * p.nsplit + split;
    for (int e = tid; e < nrows * (DV / 4); e += 256) {
        const int row = e / (DV / 4), d = (e - row * (DV / 4)) * 4;
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
        float ls = 0.f;
#pragma unroll
        for (int w = 0; w < 4; ++w) {
            const float* rw = reinterpret_cast<const float*>(smem + w * WAVE_LDS);
            acc += *reinterpret_cast<const f32x4*>(rw + row * DV + d);
            ls += rw[QT * 16 * DV + row];
        }
        if (p.nsplit > 1) {
            *reinterpret_cast<f32x4*>(p.ws + (slot * p.rows_cap + row) * DV + d) = acc;
            if (d == 0) p.ws[(int64_t)p.B * p.KH * p.nsplit * p.rows_cap * DV + slot * p.rows_cap + row] = ls;
            continue;
        }
        const float inv = 1.0f / (ls + __builtin_amdgcn_exp2f(-p.ref_log2));
        const int i = row / g, r = row - i * g;
        bf16_t* op = reinterpret_cast<bf16_t*>(p.out) + ((int64_t)(q0 + i) * p.H + kvh * g + r) * p.DV;
        if ((p.DV & 3) == 0) {
            if (d < p.DV) *reinterpret_cast<bf16x4*>(op + d) = __builtin_convertvector(acc * inv, bf16x4);
        } else {
#pragma unroll
            for (int u = 0; u < 4; ++u)
                if (d + u < p.DV) op[d + u] = f32_to_bf16(acc[u] * inv);
        }
    }
}

// ------------------------------------------------------------------------------------------------ prefill
// heads of at most 64: 64-key tiles and 128 registers put two eight-wave workgroups on a CU
template <int DV>
constexpr bool small_heads() { return DK <= 64 && DV <= 64; }

// NW wavefronts of 32 query rows (token-major: row = token * g + head of the group) share KT-key tiles through two LDS
// images, one barrier per tile.  A workgroup visits the tiles from its first row's chunk start to its last row's position.
template <int DV, int NW, int KT>
__global__ __launch_bounds__(64 * NW, NW == 8 ? (small_heads<DV>() ? 4 : 2) : 1) void xattn_prefill_kernel(const XattnParams p, const int W) {
    constexpr int KS = DK / 16, NB = DV / 16, DB = DV / 32;
    constexpr int K_BYTES = KT * KROW, VG = NB * kVSub, STAGE = stage_bytes<DV>(KT);
    constexpr int CK = KT * DK / 8, CV = KT * DV / 8;            // 16-byte pieces of a tile
    constexpr int NK = (CK + 64 * NW - 1) / (64 * NW), NV = (CV + 64 * NW - 1) / (64 * NW);
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];   // 2 x STAGE, int[2 NW], 2 x float[g W]
    int* s_rng = reinterpret_cast<int*>(smem + 2 * STAGE);
    float* s_bias = reinterpret_cast<float*>(smem + 2 * STAGE + 8 * NW);
    const int tid = threadIdx.x, lane = tid & 63, j = lane & 31, kh = lane >> 5;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int r0 = blockIdx.x >> 3;
    const int qg = r0 % p.n_qgroups, pair = (r0 / p.n_qgroups) * 8 + (blockIdx.x & 7);
    if (pair >= p.B * p.KH) return;
    const int b = pair / p.KH, kvh = pair % p.KH, g = p.g;
    const int q0 = p.qo_indptr[b], n_b = p.qo_indptr[b + 1] - q0;
    const int pos_b = p.pos0[b], pg0 = p.page_indptr[b];
    const int cap = (p.page_indptr[b + 1] - pg0) * p.page_size;
    const int nrows = n_b * g, last = min(pos_b + n_b - 1, cap - 1);
    if (qg * NW * 32 >= nrows || last < 0) return;                // whole workgroup
    const int R = (qg * NW + wave) * 32 + j;
    const bool valid = R < nrows;
    const int qi = valid ? R / g : 0, qr = valid ? R - qi * g : 0, h = kvh * g + qr;
    const int pos = pos_b + qi;
    const int lim = valid ? min(pos, cap - 1) : -1, low = valid ? (pos / p.chunk) * p.chunk : 0x7fffffff;
    int hi = lim, lo = low, low_max = valid ? low : -1;
#pragma unroll
    for (int o = 1; o < 32; o <<= 1) {
        hi = max(hi, __shfl_xor(hi, o));
        lo = min(lo, __shfl_xor(lo, o));
        low_max = max(low_max, __shfl_xor(low_max, o));
    }
    hi = __builtin_amdgcn_readfirstlane(hi);
    lo = __builtin_amdgcn_readfirstlane(lo);
    low_max = __builtin_amdgcn_readfirstlane(low_max);
    if (lane == 0) {
        s_rng[wave] = hi;
        s_rng[NW + wave] = lo;
    }
    __syncthreads();
    int hi_wg = -1, lo_wg = 0x7fffffff;
#pragma unroll
    for (int w = 0; w < NW; ++w) {
        hi_wg = max(hi_wg, s_rng[w]);
        lo_wg = min(lo_wg, s_rng[NW + w]);
    }
    const int t0 = lo_wg / KT, t1 = hi_wg / KT;                     // tiles of the workgroup, inclusive
    const int my0 = hi >= 0 ? lo / KT : 1, my1 = hi >= 0 ? hi / KT : 0;

    bf16x8 qf[KS];
    {
        const bf16_t* qp = reinterpret_cast<const bf16_t*>(p.q) + ((int64_t)(q0 + qi) * p.H + h) * DK;
        const bf16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) qf[ks] = valid ? *reinterpret_cast<const bf16x8*>(qp + ks * 16 + kh * 8) : z;
    }
    const float sl2 = p.scale_log2, mref = -p.ref_log2;
    // bias table of one tile: entry e of head r is the distance d = (position of the workgroup's first token) - (last key of
    // the tile) + e.  A lane's entries have the same indexes in every tile.
    const int tok0 = qg * NW * 32 / g, tsize = g * W;
    const float* my_bias = s_bias + (valid ? qr * W + qi - tok0 : 0) + 4 - 4 * kh;
    const int fill_r = tid / W, fill_e = tid - fill_r * W;
    auto fill = [&](int t, float* tab) {
        const int d0 = pos_b + tok0 - (t * KT + KT - 1);
        int r = fill_r, e = fill_e;
        for (int i = tid; i < tsize; i += 64 * NW) {
            const float a = p.r1 ? p.r1[kvh * g + r] : 0.f, c = p.r1 ? p.r2[kvh * g + r] : 0.f;
            const int d = d0 + e;
            tab[i] = d < 0 ? -INFINITY : fmaf(-a, __builtin_amdgcn_logf(fmaf(c, (float)d, 1.0f)), mref);
            e += 64 * NW;
            while (e >= W) {
                e -= W;
                ++r;
            }
        }
    };
    f32x16 o[DB];
#pragma unroll
    for (int db = 0; db < DB; ++db)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[db][r] = 0.f;
    float l = 0.f;

    u32x4 kreg[NK], vreg[NV];
    auto issue = [&](int t) {
        const int kp0 = t * KT, page = kp0 / p.page_size, slot = kp0 - page * p.page_size;
        const int pid = __builtin_amdgcn_readfirstlane(p.page_indices[pg0 + page]);
        const int64_t row = ((int64_t)pid * p.KH + kvh) * p.page_size + slot;
        const u32x4* kp = reinterpret_cast<const u32x4*>(reinterpret_cast<const bf16_t*>(p.k_cache) + row * DK);
        const u32x4* vp = reinterpret_cast<const u32x4*>(reinterpret_cast<const bf16_t*>(p.v_cache) + row * DV);
#pragma unroll
        for (int i = 0; i < NK; ++i)
            if (CK % (64 * NW) == 0 || i * 64 * NW + tid < CK) kreg[i] = kp[i * 64 * NW + tid];
#pragma unroll
        for (int i = 0; i < NV; ++i)
            if (CV % (64 * NW) == 0 || i * 64 * NW + tid < CV) vreg[i] = vp[i * 64 * NW + tid];
    };
    auto stage = [&](int t, unsigned char* img) {
#pragma unroll
        for (int i = 0; i < NK; ++i) {
            const int c = i * 64 * NW + tid, row = c / (DK / 8);
            if (CK % (64 * NW) == 0 || c < CK) {
                if (t * KT + row > last) kreg[i] = u32x4{0u, 0u, 0u, 0u};     // rows not written yet may hold anything (NaN)
                *reinterpret_cast<u32x4*>(img + row * KROW + (c % (DK / 8)) * 16) = kreg[i];
            }
        }
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int c = i * 64 * NW + tid, row = c / (DV / 8), ch = c % (DV / 8);
            if (CV % (64 * NW) == 0 || c < CV) {
                if (t * KT + row > last) vreg[i] = u32x4{0u, 0u, 0u, 0u};
                *reinterpret_cast<u32x4*>(img + K_BYTES + (row >> 5) * VG + (ch >> 1) * kVSub + (row & 31) * 32 + (ch & 1) * 16) =
                    vreg[i];
            }
        }
    };
    const int kra0 = j * KROW + kh * 16;
    const int lq = lane & 15;
    // the two 16-d sub-tiles one transpose read pairs lie NB / 2 apart (disjoint LDS banks at the usual widths)
    const int vra0 = K_BYTES + ((lane >> 4) & 1) * (NB / 2) * kVSub + (kh * 4 + (lq >> 2)) * 32 + (lq & 3) * 8;
    auto compute = [&](int t, const unsigned char* img, const float* bias, bool masked) {
        constexpr int KGU = NW == 8 && small_heads<DV>() ? 1 : 2;    // 32-key blocks whose S products run interleaved
#pragma unroll
        for (int kg0 = 0; kg0 < KT / 32; kg0 += KGU) {
            f32x16 sc[KGU];
#pragma unroll
            for (int u = 0; u < KGU; ++u)
#pragma unroll
                for (int r = 0; r < 16; ++r) sc[u][r] = 0.f;
#pragma unroll
            for (int ks = 0; ks < KS; ++ks)
#pragma unroll
                for (int u = 0; u < KGU; ++u) {
                    const bf16x8 kf = lds_read_b128(img + kra0 + (kg0 + u) * 32 * KROW + ks * 32);
                    sc[u] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[ks], sc[u], 0, 0, 0);
                }
#pragma unroll
            for (int u = 0; u < KGU; ++u) {
                const int kbase = t * KT + (kg0 + u) * 32 + 4 * kh;
#pragma unroll
                for (int r = 0; r < 16; ++r)
                    sc[u][r] = fmaf(sc[u][r], sl2, bias[(KT / 32 - 1 - kg0 - u) * 32 + 27 - (r & 3) - 8 * (r >> 2)]);
                if (masked) {                                       // keys of the previous chunk; a wave-uniform branch
#pragma unroll
                    for (int r = 0; r < 16; ++r) {
                        const int kp = kbase + (r & 3) + 8 * (r >> 2);
                        float v = sc[u][r];
                        if (kp < low) v = -INFINITY;
                        asm volatile("" : "+v"(v));                 // keeps the selects inside the branch
                        sc[u][r] = v;
                    }
                }
#pragma unroll
                for (int s16 = 0; s16 < 2; ++s16) {
                    f32x8 pv;
#pragma unroll
                    for (int e = 0; e < 8; ++e) {
                        pv[e] = __builtin_amdgcn_exp2f(sc[u][s16 * 8 + e]);
                        l += pv[e];
                    }
                    bf16x8 ph, pl;
                    split_bf16(pv, ph, pl);
#pragma unroll
                    for (int db = 0; db < DB; ++db) {
                        const unsigned char* vb = img + (kg0 + u) * VG + db * kVSub + vra0 + s16 * 16 * 32;
                        const bf16x4 v0 = lds_read_tr(vb), v1 = lds_read_tr(vb + 8 * 32);
                        const bf16x8 vf = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
                        o[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, ph, o[db], 0, 0, 0);
                        o[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pl, o[db], 0, 0, 0);
                    }
                }
            }
        }
    };

    // tile t lies in image t & 1; it is overwritten two tiles later, after a barrier every wave reaches past its use
    issue(t0);
    for (int t = t0; t <= t1; ++t) {
        unsigned char* img = smem + (t & 1) * STAGE;
        stage(t, img);
        fill(t, s_bias + (t & 1) * tsize);
        if (t < t1) issue(t + 1);
        __syncthreads();
        if (t >= my0 && t <= my1) compute(t, img, my_bias + (t & 1) * tsize, t * KT < low_max);
    }

    l += __shfl_xor(l, 32);
    if (valid) {
        const float inv = 1.0f / (l + __builtin_amdgcn_exp2f(mref));
        bf16_t* op = reinterpret_cast<bf16_t*>(p.out) + ((int64_t)(q0 + qi) * p.H + h) * p.DV;
#pragma unroll
        for (int db = 0; db < DB; ++db)
#pragma unroll
            for (int rg = 0; rg < 4; ++rg) {
                const int d = (db + (rg >> 1) * (NB / 2)) * 16 + (rg & 1) * 8 + kh * 4;
                const f32x4 ov = {o[db][rg * 4] * inv, o[db][rg * 4 + 1] * inv, o[db][rg * 4 + 2] * inv, o[db][rg * 4 + 3] * inv};
                if ((p.DV & 3) == 0) {
                    if (d < p.DV) *reinterpret_cast<bf16x4*>(op + d) = __builtin_convertvector(ov, bf16x4);
                } else {
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        if (d + e < p.DV) op[d + e] = f32_to_bf16(ov[e]);
                }
            }
    }
}

template <typename K>
int raise_lds(K k, int lds, MdPerDeviceOnce& once) {
    if (lds > 64 * 1024 && once.first() &&
        hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, lds) != hipSuccess) {
        once.undo();
        md_set_error("md_xattn: hipFuncSetAttribute(%d B LDS) failed", lds);
        return MD_ERR_LAUNCH;
    }
    return MD_OK;
}

template <int DV, int QT, bool FUSED>
int launch_decode(const XattnParams& p, int grid, hipStream_t st) {
    constexpr int lds = 4 * decode_wave_lds<DV, QT>();
    static_assert(lds <= 160 * 1024, "the waves' LDS images must fit the CU");
    static MdPerDeviceOnce once;
    auto k = xattn_decode_kernel<DV, QT, FUSED>;
    const int rc = raise_lds(k, lds, once);
    if (rc != MD_OK) return rc;
    hipLaunchKernelGGL(k, dim3(grid), dim3(256), lds, st, p);
    return MD_OK;
}

template <int DV>
int decode_dv(const XattnParams& p, int qt, bool fused, int grid, hipStream_t st) {
    if (qt == 1) return fused ? launch_decode<DV, 1, true>(p, grid, st) : launch_decode<DV, 1, false>(p, grid, st);
    return fused ? launch_decode<DV, 2, true>(p, grid, st) : launch_decode<DV, 2, false>(p, grid, st);
}

template <int DV, int NW>
constexpr int prefill_kt() { return NW == 8 && !small_heads<DV>() && 2 * stage_bytes<DV>(128) <= 144 * 1024 ? 128 : 64; }

// width of a bias table row: every distance between the workgroup's tokens and a tile's keys, the rows of the group's heads
// spread over the LDS banks
template <int DV, int NW>
int bias_width(int g) {
    int w = prefill_kt<DV, NW>() + (NW * 32 - 1) / g + 2;
    const int want = g < 64 ? 64 / g : 1;
    while (w % 64 != want % 64) ++w;
    return w;
}
template <int DV, int NW>
int prefill_lds(int g) { return 2 * stage_bytes<DV>(prefill_kt<DV, NW>()) + 8 * NW + 8 * g * bias_width<DV, NW>(g); }

template <int DV, int NW>
int launch_prefill(const XattnParams& p, int grid, hipStream_t st) {
    static_assert(2 * stage_bytes<DV>(prefill_kt<DV, NW>()) <= 150 * 1024, "the two tile images must fit the CU");
    static MdPerDeviceOnce once;
    auto k = xattn_prefill_kernel<DV, NW, prefill_kt<DV, NW>()>;
    const int rc = raise_lds(k, 160 * 1024, once);
    if (rc != MD_OK) return rc;
    const int lds = prefill_lds<DV, NW>(p.g), width = bias_width<DV, NW>(p.g);
    hipLaunchKernelGGL(k, dim3(grid), dim3(64 * NW), lds, st, p, width);
    return MD_OK;
}

// wavefronts per workgroup for this many rows: 8 where the rows fill them and the bias table fits beside the tiles; 0: none fits
template <int DV>
int prefill_waves(int g, int rows) {
    if (rows >= 256 && prefill_lds<DV, 8>(g) <= 160 * 1024) return 8;
    return prefill_lds<DV, 4>(g) <= 160 * 1024 ? 4 : 0;
}

template <int DV>
int prefill_dv(const XattnParams& p, int nw, int grid, hipStream_t st) {
    return nw == 8 ? launch_prefill<DV, 8>(p, grid, st) : launch_prefill<DV, 4>(p, grid, st);
}

}  // namespace

#define MD_CAT_(a, b) a##b
#define MD_CAT(a, b) MD_CAT_(a, b)

int MD_CAT(md_internal_xattn_decode_, MD_XATTN_DK)(const XattnParams& p, int qt, bool fused, int grid, hipStream_t st) {
    switch (p.DVp) {
    case 32: return decode_dv<32>(p, qt, fused, grid, st);
    case 64: return decode_dv<64>(p, qt, fused, grid, st);
    case 96: return decode_dv<96>(p, qt, fused, grid, st);
    case 128: return decode_dv<128>(p, qt, fused, grid, st);
    case 192: return decode_dv<192>(p, qt, fused, grid, st);
    default: return decode_dv<256>(p, qt, fused, grid, st);
    }
}

int MD_CAT(md_internal_xattn_waves_, MD_XATTN_DK)(int dv, int g, int rows) {
    switch (dv) {
    case 32: return prefill_waves<32>(g, rows);
    case 64: return prefill_waves<64>(g, rows);
    case 96: return prefill_waves<96>(g, rows);
    case 128: return prefill_waves<128>(g, rows);
    case 192: return prefill_waves<192>(g, rows);
    default: return prefill_waves<256>(g, rows);
    }
}

int MD_CAT(md_internal_xattn_prefill_, MD_XATTN_DK)(const XattnParams& p, int nw, int grid, hipStream_t st) {
    switch (p.DVp) {
    case 32: return prefill_dv<32>(p, nw, grid, st);
    case 64: return prefill_dv<64>(p, nw, grid, st);
    case 96: return prefill_dv<96>(p, nw, grid, st);
    case 128: return prefill_dv<128>(p, nw, grid, st);
    case 192: return prefill_dv<192>(p, nw, grid, st);
    default: return prefill_dv<256>(p, nw, grid, st);
    }
}
