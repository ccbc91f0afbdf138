// Paged attention for the MagicDec draft/verify decode path on gfx950 (MI355X).
//
// Replaces flashinfer's BatchPrefillWithPagedKVCacheWrapper.run as used by
// mylib::target_decode / draft_decode / target_prefill / draft_prefill
// (reference: Engine/SnapKV/backend.py:56-107, backend_draft.py:42-92,
//  StreamingLLM twins).  Semantics restated in oracle/flashinfer_ref.py.
//
// Design (decode is HBM-bound: every K/V byte is read exactly once):
//   * one wavefront owns a stream of 32-key tiles of one (request, kv head):
//     coalesced 16 B/lane global loads (whole 128/256-B rows) -> registers ->
//     wave-private LDS image -> MFMA fragments.  Waves never synchronise
//     inside the tile loop (no s_barrier); the next tile's global loads are
//     in flight while the current tile is computed.
//   * S^T = K.Q^T and O^T = V^T.P^T on v_mfma_f32_16x16x32_bf16, so the
//     softmax statistics of query row (lane&15) are lane-local and P never
//     moves between lanes: the S^T accumulator registers ARE the B operand of
//     the PV MFMA (after bf16 packing) with the key permutation
//     slot(c,t) -> key (t>>2)*16 + c*4 + (t&3).
//   * K image: row-major with a 16-B row pad (pitch D*2+16: consecutive rows
//     start 4 banks apart -> conflict-free ds_read_b128 fragment reads, and
//     every LDS address is lane base + immediate).  V image: [d/16][32 keys][16]
//     sub-tiles read with ds_read_b64_tr_b16 (hardware transpose).
//   * the tile loop has a branch-free steady state (unconditional prefetch of
//     tile t+NS) so that s_waitcnt vmcnt() only waits for the tile being
//     consumed; the ragged tail runs in a separate drain loop.
//   * g*(gamma+1) query rows share every K/V tile (16 rows for Llama-3.1-8B
//     at gamma=3 = exactly one MFMA M tile).
//   * verify/draft ("decode" variant): the 4 waves of a workgroup split the KV
//     range of one (request, kv head, kv-split) and merge (m,l,O) through
//     LDS; optional split-KV across workgroups + a small merge kernel.
//   * chunked prefill: prefill_attn_kernel below (a workgroup of 4 or 8 waves x 16/32 query rows shares every
//     K/V tile through LDS); workgroups sharing a (request, kv head) are placed on one XCD (block id mod 8).
#include <type_traits>

#include "attn_common.h"

#include <hip/hip_ext.h>

#include <vector>

namespace {

typedef float f32x16 __attribute__((ext_vector_type(16)));

struct AttnParams {
    const bf16_t* q;
    const void* cache;     // bf16 or OCP e4m3fn bytes (MD_KV_FP8_E4M3)
    bf16_t* out;
    const int32_t* qo_indptr;
    const int32_t* page_indices;
    const int32_t* page_indptr;
    const int32_t* last_page_len;
    float* ws_o;
    float* ws_ml;
    int64_t q_row_stride;  // elements
    int64_t page_stride;   // elements: 2*page_size*KH*D
    int64_t kv_half;       // elements: page_size*KH*D
    int slot_stride;       // elements between consecutive rows of a page: KH*D (NHD pages), D (HND pages)
    int head_stride;       // elements between kv heads inside a page half: D (NHD), page_size*D (HND)
    int B, H, KH, g, page_size, causal, nsplit, n_qgroups;
    float scale_log2;
    const float* k_scale;  // fp8 KV: per-kv-head dequant scales (K folded into the softmax scale, V into 1/l)
    const float* v_scale;
};


template <int D, int QT>
__host__ __device__ constexpr int attn_wave_lds() {
    int stage = 32 * (D * 2 + 16) + (D / 16) * kVSub;
    int merge = QT * D * 64 + QT * 128;
    int m = stage > merge ? stage : merge;
    return (m + 255) / 256 * 256;
}

template <int D, int KT = 32>
__host__ __device__ constexpr int prefill_stage_bytes() {
    return KT * (D * 2 + 16) + (KT / 32) * (D / 16) * kVSub;   // one shared KT-key K + V tile image (prefill kernel)
}

// decode/verify reads every K/V byte exactly once: non-temporal loads (+5 % of HBM peak measured); the prefill
// variant re-reads a (request, kv head) stream from L2 by several workgroups, where nt costs bandwidth
template <bool NT>
__device__ __forceinline__ u32x4 ldg_stream(const u32x4* p) {
    if constexpr (NT)
        return __builtin_nontemporal_load(p);
    else
        return *p;
}

// 16 e4m3fn bytes -> 16 bf16 (exact: e4m3 is a subset of bf16), v_cvt_scalef32_pk_bf16_fp8 with scale 1
__device__ __forceinline__ void cvt16_fp8_bf16(const u32x4 x, u32x4& lo, u32x4& hi) {
#pragma unroll
    for (int w = 0; w < 4; ++w) {
        const bf16x2 a = __builtin_amdgcn_cvt_scalef32_pk_bf16_fp8(x[w], 1.0f, false);
        const bf16x2 b = __builtin_amdgcn_cvt_scalef32_pk_bf16_fp8(x[w], 1.0f, true);
        const unsigned ua = *reinterpret_cast<const unsigned*>(&a), ub = *reinterpret_cast<const unsigned*>(&b);
        if (w < 2) {
            lo[2 * w] = ua;
            lo[2 * w + 1] = ub;
        } else {
            hi[2 * (w - 2)] = ua;
            hi[2 * (w - 2) + 1] = ub;
        }
    }
}

// NWV: wavefronts per workgroup, 4 or 8 (round 5).  A launch with <= 256 workgroups puts ONE on each CU; with four waves
// that is half the loads in flight of the two-workgroups-per-CU launches (B x KH_local = 512 pairs at TP1).  Eight waves
// share the workgroup's tile range round-robin and merge through LDS like four.  Measured (profiles/r05_attn_waves_ab.txt):
// it is NOT what holds the bf16 TP shards at 71-82 % (KH_local = 1 / 2 / 4 and B = 32: 8 waves equal or 1-3 % slower -- the
// deficit there is the fixed ~10 us of launch, tail and merge on an 85 us kernel), but the fp8 kernel with two M tiles
// (cfg5's shard: Qwen g = 5, B = 128 x 64 K keys, 2 splits) gains 7 %: 0.378 -> 0.352 ms = 71 -> 76 % of the HBM peak.
template <int D, int QT, bool FP8, int NWV>
__global__ __launch_bounds__(64 * NWV, NWV == 4 ? 2 : 1) void paged_attn_kernel(const AttnParams p) {
    constexpr int EB = FP8 ? 1 : 2;          // bytes per cache element
    constexpr int CH = D * EB / 16;          // 16-B chunks per K/V row in HBM
    constexpr int RPI = 64 / CH;             // rows per wave-wide load instruction
    constexpr int NL = 32 / RPI;             // load instructions per 32-key tile (K or V)
    constexpr int KS = D / 32;    // MFMA k-steps of QK^T
    constexpr int NB = D / 16;    // 16-wide d blocks of PV
    constexpr int KROW = D * 2 + 16;         // K image row pitch: +16 B pad instead of an XOR swizzle, so that every
                                             // LDS address is (per-lane base + compile-time immediate)
    constexpr int K_BYTES = 32 * KROW;
    // fp8, D=128: a lane's 16 bytes become two 16-B bf16 chunks; writing (lo,hi) to slots (2c,2c+1) makes 8
    // consecutive lanes hit 32-B-strided addresses (2-way bank conflict).  Lanes with c >= 4 therefore write
    // (lo,hi) to slots (2c+1,2c): this permutes d inside the K image (undone by loading Q with the same permutation)
    // and inside V sub-tiles 4..7 (undone when O is stored).
    constexpr bool FP8_SWAP = FP8 && D == 128;
    constexpr int WAVE_LDS = attn_wave_lds<D, QT>();
    constexpr int TSTEP = NWV;    // the waves of a workgroup take the KV tiles round-robin
    // two tiles of loads in flight per wave where the register budget allows it (256 VGPRs at 2 waves/SIMD)
    // register staging depth: tiles of this wave whose loads are in flight while one tile is consumed.  Two where
    // the register budget allows it (256 VGPRs at 2 waves/SIMD; QT=2 at D=128 needs them for O and Q).  Deeper
    // staging was measured and does not help: with exact wait counts two tiles already cover the HBM latency.
    // two M tiles at D=128 (g*(gamma+1) in 17..32: Qwen2.5-32B g=5, Llama-70B g=8) are register-bound; measured best:
    // fp8: both tiles in flight + batched fragment reads, plain loop (60-63 % of peak vs 57-59 % for the other
    // combinations); bf16: one tile in flight, steady loop (70-78 %; batching / plain loop measured equal, two tiles spill)
    constexpr bool Q2F8 = FP8 && QT == 2 && D == 128;
    constexpr int NS = Q2F8 ? 2 : (QT == 2 && D == 128) ? 1 : 2;
    // fp8 with two M tiles (e.g. Qwen2.5-32B: g=5, gamma+1=4 -> 20 rows) has no registers left for the duplicated
    // steady-state body; it keeps both tiles in flight with the plain (conditional-prefetch) loop
    constexpr bool STEADY = !Q2F8;
    constexpr bool BATCH = Q2F8 || ((FP8 || D == 64) && QT == 1);
    constexpr int PF = NS * TSTEP;   // prefetch distance in tiles of this wave

    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    const int tid = threadIdx.x;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int lane = tid & 63;
    const int lq = lane & 15, lc = lane >> 4;

    // block -> ((request, kv head), (q group, kv split)); blocks of one pair
    // differ by multiples of 8 in block id (same XCD -> shared L2).
    const int bid = blockIdx.x;
    const int nsub = p.n_qgroups * p.nsplit;
    const int xcd = bid & 7;
    const int r0 = bid >> 3;
    const int sub = r0 % nsub;
    const int pair = (r0 / nsub) * 8 + xcd;
    if (pair >= p.B * p.KH) return;
    const int qg = sub / p.nsplit, split = sub % p.nsplit;
    const int b = pair / p.KH, kvh = pair % p.KH;
    const int g = p.g;

    const int q0 = p.qo_indptr[b];
    const int n_b = p.qo_indptr[b + 1] - q0;
    const int pg0 = p.page_indptr[b];
    const int npages = p.page_indptr[b + 1] - pg0;
    // clamped to the mapped pages: an over-long last_page_len must not walk past the request's page list
    const int kv_len = npages > 0 ? min((npages - 1) * p.page_size + p.last_page_len[b], npages * p.page_size) : 0;
    const int nrows = n_b * g;
    const int tile_base = qg * QT;

    // per-lane query row (column lq of S^T) and its causal limit
    int lim[QT];
    int hi = -1, lo = 0x7fffffff;
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        const int R = (tile_base + qt) * 16 + lq;
        const bool valid = R < nrows;
        const int i = R / g;
        lim[qt] = valid ? (p.causal ? kv_len - n_b + i : kv_len - 1) : -1;
        hi = max(hi, lim[qt]);
        if (valid) lo = min(lo, lim[qt]);
    }
#pragma unroll
    for (int o = 1; o < 16; o <<= 1) {
        hi = max(hi, __shfl_xor(hi, o));
        lo = min(lo, __shfl_xor(lo, o));
    }
    hi = __builtin_amdgcn_readfirstlane(hi);
    lo = __builtin_amdgcn_readfirstlane(lo);

    const int kv_end = min(hi + 1, kv_len);
    const int ntiles = kv_end > 0 ? (kv_end + 31) >> 5 : 0;
    const int tps = (ntiles + p.nsplit - 1) / p.nsplit;
    const int t_begin = split * tps;
    const int t_end = min(ntiles, t_begin + tps);

    // Q fragments (B operand of S^T = K.Q^T): lane (lq,lc) holds Q[row lq][s*32+lc*8 .. +8]
    bf16x8 qf[QT][KS];
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        const int R = (tile_base + qt) * 16 + lq;
        const bool valid = R < nrows;
        const int i = R / g, r = R - i * g;
        const bf16_t* qp = p.q + (int64_t)(q0 + i) * p.q_row_stride + (kvh * g + r) * D;
#pragma unroll
        for (int s = 0; s < KS; ++s) {
            bf16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
            int slot = s * 4 + lc;                       // 8-element d group held by K-image chunk slot `slot`
            if (FP8_SWAP && s >= 2) slot ^= 1;
            qf[qt][s] = valid ? *reinterpret_cast<const bf16x8*>(qp + slot * 8) : z;
        }
    }

    // fp8 KV: K's per-head scale is folded into the softmax scale, V's into the final 1/l
    const float sl2 = FP8 ? p.scale_log2 * p.k_scale[kvh] : p.scale_log2;
    const float vsc = FP8 ? p.v_scale[kvh] : 1.0f;
    f32x4 o[QT][NB];
    float m[QT], l[QT];
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        m[qt] = -1e30f;
        l[qt] = 0.f;
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) o[qt][nb] = f32x4{0.f, 0.f, 0.f, 0.f};
    }

    unsigned char* ldsK = smem + wave * WAVE_LDS;
    unsigned char* ldsV = ldsK + K_BYTES;

    // staging (write) side: lane -> (row wrow + j*RPI, 16-B HBM chunk wch).  bf16 cache: one 16-B LDS chunk;
    // fp8 cache: the 16 bytes expand to two adjacent bf16 chunks (2*wch, 2*wch+1) = one V sub-tile row
    const int wrow = lane / CH, wch = lane % CH;
    const bool swp = FP8_SWAP && wch >= 4;
    int kw[NL], kw2[NL], vw[NL], vw2[NL];
#pragma unroll
    for (int j = 0; j < NL; ++j) {
        const int row = wrow + j * RPI;
        if constexpr (FP8) {
            kw[j] = row * KROW + ((2 * wch + (swp ? 1 : 0)) << 4);
            kw2[j] = row * KROW + ((2 * wch + (swp ? 0 : 1)) << 4);
            vw[j] = wch * kVSub + row * 32 + (swp ? 16 : 0);
            vw2[j] = wch * kVSub + row * 32 + (swp ? 0 : 16);
        } else {
            kw[j] = row * KROW + (wch << 4);
            kw2[j] = 0;
            vw[j] = (wch >> 1) * kVSub + row * 32 + (wch & 1) * 16;
            vw2[j] = 0;
        }
    }
    // fragment (read) side
    int kra[2][KS];
#pragma unroll
    for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int s = 0; s < KS; ++s) {
            const int row = kb * 16 + lq, ch = s * 4 + lc;
            kra[kb][s] = row * KROW + (ch << 4);
        }
    const int vra = (lc * 4 + (lq >> 2)) * 32 + (lq & 3) * 8;  // + nb*kVSub + kb*512
    const unsigned goff = (unsigned)((wrow * p.slot_stride + kvh * p.head_stride) * EB + wch * 16);  // bytes, per lane

    // two tiles in flight per wavefront: register sets A and B alternate (2 x 16 KiB of loads outstanding while a
    // tile is computed -- the loop is latency x bandwidth bound, not compute bound)
    u32x4 kR[NS][NL], vR[NS][NL];
    auto issue = [&](int tt, u32x4 (&kreg)[NL], u32x4 (&vreg)[NL]) {
        const int pos0 = tt * 32;
        const int page = pos0 / p.page_size;
        const int slot0 = pos0 - page * p.page_size;
        const int pid = __builtin_amdgcn_readfirstlane(p.page_indices[pg0 + page]);
        // wave-uniform 64-bit base (SGPRs) + one shared 32-bit per-lane offset: the 2*NL loads of a tile then need
        // no per-load address VGPRs (global_load ... v_off, s[base:base+1])
        const unsigned char* kb_ = reinterpret_cast<const unsigned char*>(p.cache) +
                                   ((int64_t)pid * p.page_stride + (int64_t)slot0 * p.slot_stride) * EB;
        const unsigned char* vb_ = kb_ + p.kv_half * EB;
        const int64_t jstep = (int64_t)RPI * p.slot_stride * EB;
#pragma unroll
        for (int j = 0; j < NL; ++j)
            kreg[j] = ldg_stream<true>(reinterpret_cast<const u32x4*>(kb_ + j * jstep + goff));
#pragma unroll
        for (int j = 0; j < NL; ++j)
            vreg[j] = ldg_stream<true>(reinterpret_cast<const u32x4*>(vb_ + j * jstep + goff));
    };

    // `always_prefetch` (a std::bool_constant): the steady-state loop issues the next tile's loads unconditionally, so
    // the loop body is straight-line code and the compiler's s_waitcnt vmcnt() values are exact (only this tile's loads
    // are waited for; the other NS-1 tiles stay in flight).  With a conditional prefetch the wait-count analysis
    // merges the "issued" and "not issued" states at every join and degrades to vmcnt(0): every tile then drains the
    // whole queue and a wavefront processes one tile per HBM round trip.
    auto process = [&](auto always_prefetch, int t, u32x4 (&kreg)[NL], u32x4 (&vreg)[NL]) {
#ifdef MD_ATTN_LOADS_ONLY   // experiment: memory-side ceiling of this access pattern (results are garbage)
        {
            u32x4 acc = {0u, 0u, 0u, 0u};
#pragma unroll
            for (int j = 0; j < NL; ++j) acc = acc ^ kreg[j] ^ vreg[j];
            o[0][0][0] += __uint_as_float((acc[0] ^ acc[1] ^ acc[2] ^ acc[3]) & 0x007fffffu);
            if constexpr (decltype(always_prefetch)::value) {
                issue(t + PF, kreg, vreg);
            } else {
                if (t + PF < t_end) issue(t + PF, kreg, vreg);
            }
            return;
        }
#endif
        const bool need_mask = (t * 32 + 31) > lo;
        if (need_mask) {
            // rows past the request's length may hold anything (even NaN): zero V so 0*V stays 0
#pragma unroll
            for (int j = 0; j < NL; ++j)
                if (t * 32 + wrow + j * RPI >= kv_len) vreg[j] = u32x4{0u, 0u, 0u, 0u};
        }
        if constexpr (FP8) {
#pragma unroll
            for (int j = 0; j < NL; ++j) {
                u32x4 lo, hi;
                cvt16_fp8_bf16(kreg[j], lo, hi);
                *reinterpret_cast<u32x4*>(ldsK + kw[j]) = lo;
                *reinterpret_cast<u32x4*>(ldsK + kw2[j]) = hi;
            }
#pragma unroll
            for (int j = 0; j < NL; ++j) {
                u32x4 lo, hi;
                cvt16_fp8_bf16(vreg[j], lo, hi);
                *reinterpret_cast<u32x4*>(ldsV + vw[j]) = lo;
                *reinterpret_cast<u32x4*>(ldsV + vw2[j]) = hi;
            }
        } else {
#pragma unroll
            for (int j = 0; j < NL; ++j) *reinterpret_cast<u32x4*>(ldsK + kw[j]) = kreg[j];
#pragma unroll
            for (int j = 0; j < NL; ++j) *reinterpret_cast<u32x4*>(ldsV + vw[j]) = vreg[j];
        }
        if constexpr (decltype(always_prefetch)::value) {
            issue(t + PF, kreg, vreg);
        } else {
            if (t + PF < t_end) issue(t + PF, kreg, vreg);
        }
        // same-wave LDS hand-off: LDS ops of one wave execute in order
        __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");

        // ---- S^T = K.Q^T : s[qt][kb][j] = score(key kb*16+lc*4+j, query lq)
        f32x4 s[QT][2];
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) {
            s[qt][0] = f32x4{0.f, 0.f, 0.f, 0.f};
            s[qt][1] = f32x4{0.f, 0.f, 0.f, 0.f};
        }
        // BATCH (fp8 / D=64 variants: half the staging registers, so VGPRs are free and the per-key work is what
        // bounds them): all K fragments of the tile are requested before the first MFMA -- one LDS round trip
        // instead of 2*KS dependent ones.  The bf16 D=128 variants are HBM-bound and keep the register-lean order.
        if constexpr (BATCH) {
            bf16x8 kf[2][KS];
#pragma unroll
            for (int kb = 0; kb < 2; ++kb)
#pragma unroll
                for (int ks = 0; ks < KS; ++ks) kf[kb][ks] = lds_read_b128(ldsK + kra[kb][ks]);
            __builtin_amdgcn_sched_barrier(0);   // keep the reads clustered (the scheduler would re-serialise them)
#pragma unroll
            for (int ks = 0; ks < KS; ++ks)
#pragma unroll
                for (int kb = 0; kb < 2; ++kb)
#pragma unroll
                    for (int qt = 0; qt < QT; ++qt)
                        s[qt][kb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[kb][ks], qf[qt][ks], s[qt][kb], 0, 0, 0);
        } else {
#pragma unroll
            for (int kb = 0; kb < 2; ++kb)
#pragma unroll
                for (int ks = 0; ks < KS; ++ks) {
                    const bf16x8 kf = lds_read_b128(ldsK + kra[kb][ks]);
#pragma unroll
                    for (int qt = 0; qt < QT; ++qt)
                        s[qt][kb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[qt][ks], s[qt][kb], 0, 0, 0);
                }
        }

        // ---- online softmax (log2 domain), statistics are per lane (query lq)
        bf16x8 pf[QT];
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) {
            float v[8];
#pragma unroll
            for (int kb = 0; kb < 2; ++kb)
#pragma unroll
                for (int j = 0; j < 4; ++j) v[kb * 4 + j] = s[qt][kb][j] * sl2;
            if (need_mask) {
#pragma unroll
                for (int kb = 0; kb < 2; ++kb)
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        const int pos = t * 32 + kb * 16 + lc * 4 + j;
                        if (pos > lim[qt]) v[kb * 4 + j] = -INFINITY;
                    }
            }
            float mx = v[0];
#pragma unroll
            for (int e = 1; e < 8; ++e) mx = fmaxf(mx, v[e]);
            mx = fmaxf(mx, __shfl_xor(mx, 16));
            mx = fmaxf(mx, __shfl_xor(mx, 32));
            const float mnew = fmaxf(m[qt], mx);
            const float alpha = __builtin_amdgcn_exp2f(m[qt] - mnew);
            m[qt] = mnew;
            float ps = 0.f;
            f32x8 pv;
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const float pe = __builtin_amdgcn_exp2f(v[e] - mnew);
                pv[e] = pe;
                ps += pe;
            }
            l[qt] = l[qt] * alpha + ps;
#pragma unroll
            for (int nb = 0; nb < NB; ++nb) o[qt][nb] *= alpha;
            pf[qt] = __builtin_convertvector(pv, bf16x8);
        }

        // ---- O^T += V^T.P^T : A = V fragment (d x key slots) via transpose read
        constexpr int VG = BATCH ? 4 : 1;   // V fragments requested per LDS round trip
#pragma unroll
        for (int nb0 = 0; nb0 < NB; nb0 += VG) {
            bf16x8 vf[VG];
#pragma unroll
            for (int u = 0; u < VG; ++u) {
                const bf16x4 v0 = lds_read_tr(ldsV + (nb0 + u) * kVSub + vra);
                const bf16x4 v1 = lds_read_tr(ldsV + (nb0 + u) * kVSub + 512 + vra);
                vf[u] = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
            }
            if constexpr (BATCH) __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int u = 0; u < VG; ++u)
#pragma unroll
                for (int qt = 0; qt < QT; ++qt)
                    o[qt][nb0 + u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[u], pf[qt], o[qt][nb0 + u], 0, 0, 0);
        }
        __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
        __builtin_amdgcn_wave_barrier();
    };

    int t = t_begin + wave;
    if (STEADY && t + (2 * NS - 1) * TSTEP < t_end) {
        // steady state: NS tiles in flight, every processed tile re-arms its register set with tile t + PF
#pragma unroll
        for (int st = 0; st < NS; ++st) issue(t + st * TSTEP, kR[st], vR[st]);
        do {
#pragma unroll
            for (int st = 0; st < NS; ++st) process(std::true_type{}, t + st * TSTEP, kR[st], vR[st]);
            t += NS * TSTEP;
        } while (t + (2 * NS - 1) * TSTEP < t_end);
        // here tiles t + st*TSTEP (st < NS) are valid and in flight: the drain loop below finishes them
    } else {
#pragma unroll
        for (int st = 0; st < NS; ++st)
            if (t + st * TSTEP < t_end) issue(t + st * TSTEP, kR[st], vR[st]);
    }
    for (; t < t_end; t += NS * TSTEP) {
#pragma unroll
        for (int st = 0; st < NS; ++st)
            if (t + st * TSTEP < t_end) process(std::false_type{}, t + st * TSTEP, kR[st], vR[st]);
    }

    // row sums live as per-lane partials over the 4 lane groups of a query
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        l[qt] += __shfl_xor(l[qt], 16);
        l[qt] += __shfl_xor(l[qt], 32);
    }

    {
        // merge the waves' (m, l, O) through LDS
        __syncthreads();
        float* mo = reinterpret_cast<float*>(smem + wave * WAVE_LDS);
        float* mst = mo + QT * D * 16;
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) {
#pragma unroll
            for (int nb = 0; nb < NB; ++nb)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int dd = nb * 16 + ((FP8_SWAP && nb >= 4) ? (lc ^ 2) : lc) * 4 + r;
                    mo[(qt * D + dd) * 16 + lq] = o[qt][nb][r];
                }
            if (lc == 0) {
                mst[(qt * 16 + lq) * 2 + 0] = m[qt];
                mst[(qt * 16 + lq) * 2 + 1] = l[qt];
            }
        }
        __syncthreads();
        constexpr int ROWS = QT * 16;
        const int item = pair * p.n_qgroups + qg;
        for (int e = tid; e < ROWS * D; e += 64 * NWV) {
            const int Rl = e / D, d = e - Rl * D;  // local row (qt*16+q), d
            const int R = qg * ROWS + Rl;
            if (R >= nrows) continue;
            const int qt = Rl >> 4, qq = Rl & 15;
            float M = -1e30f;
#pragma unroll
            for (int w = 0; w < NWV; ++w) {
                const float* st = reinterpret_cast<const float*>(smem + w * WAVE_LDS) + QT * D * 16;
                M = fmaxf(M, st[(qt * 16 + qq) * 2]);
            }
            float L = 0.f, acc = 0.f;
#pragma unroll
            for (int w = 0; w < NWV; ++w) {
                const float* ow = reinterpret_cast<const float*>(smem + w * WAVE_LDS);
                const float* st = ow + QT * D * 16;
                const float sc = __builtin_amdgcn_exp2f(st[(qt * 16 + qq) * 2] - M);
                L += st[(qt * 16 + qq) * 2 + 1] * sc;
                acc += ow[(qt * D + d) * 16 + qq] * sc;
            }
            if (p.nsplit == 1) {
                const int i = R / g, r = R - i * g;
                const float val = L > 0.f ? acc * vsc / L : 0.f;
                p.out[((int64_t)(q0 + i) * p.H + kvh * g + r) * D + d] = f32_to_bf16(val);
            } else {
                const int64_t slot = ((int64_t)item * p.nsplit + split) * ROWS + Rl;
                p.ws_o[slot * D + d] = acc;
                if (d == 0) {
                    p.ws_ml[slot * 2 + 0] = M;
                    p.ws_ml[slot * 2 + 1] = L;
                }
            }
        }
    }
}

// combine split-KV partials: one thread per 4 consecutive d of one (item, row)
template <int D>
__global__ __launch_bounds__(256) void attn_merge_kernel(const AttnParams p, int rows_cap) {
    constexpr int VPR = D / 4;                         // float4 vectors per row
    const int64_t gid = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int64_t total = (int64_t)p.B * p.KH * p.n_qgroups * rows_cap * VPR;
    if (gid >= total) return;
    const int v = (int)(gid % VPR);
    const int64_t rowid = gid / VPR;
    const int Rl = (int)(rowid % rows_cap);
    const int item = (int)(rowid / rows_cap);          // pair * n_qgroups + qg  (n_qgroups == 1 in decode mode)
    const int pair = item / p.n_qgroups, qg = item % p.n_qgroups;
    const int b = pair / p.KH, kvh = pair % p.KH;
    const int q0 = p.qo_indptr[b];
    const int n_b = p.qo_indptr[b + 1] - q0;
    const int R = qg * rows_cap + Rl;
    if (R >= n_b * p.g) return;
    float M = -1e30f;
    for (int s = 0; s < p.nsplit; ++s) M = fmaxf(M, p.ws_ml[(((int64_t)item * p.nsplit + s) * rows_cap + Rl) * 2]);
    float L = 0.f;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < p.nsplit; ++s) {
        const int64_t slot = ((int64_t)item * p.nsplit + s) * rows_cap + Rl;
        const float sc = __builtin_amdgcn_exp2f(p.ws_ml[slot * 2] - M);
        L += p.ws_ml[slot * 2 + 1] * sc;
        acc += *reinterpret_cast<const f32x4*>(p.ws_o + slot * D + v * 4) * sc;
    }
    const int i = R / p.g, r = R - i * p.g;
    const float inv = L > 0.f ? (p.v_scale ? p.v_scale[kvh] : 1.f) / L : 0.f;
    *reinterpret_cast<bf16x4*>(p.out + ((int64_t)(q0 + i) * p.H + kvh * p.g + r) * D + v * 4) =
        __builtin_convertvector(acc * inv, bf16x4);
}

// ---------------------------------------------------------------------------------------------------------------
// K3: chunked prefill (mylib::target_prefill / draft_prefill, Engine/SnapKV/backend.py:66-80,96-107).
// 128 query tokens x g heads per (request, kv head) = hundreds of query rows against the whole causal KV range:
// MFMA / on-chip-bandwidth bound, not HBM bound.  A workgroup owns 4 x QT M-tiles of query rows (one set per wave)
// and ALL FOUR WAVES SHARE every 32-key K/V tile: the tile is fetched once per workgroup (each wave issues a
// quarter of the 16-B/lane loads), staged once into a double-buffered LDS image (same K / V images as the decode
// kernel) and consumed by the four waves after one s_barrier per tile.  Versus the wave-private staging of the
// decode kernel this divides the L2->CU traffic and the LDS writes by 4.  Causal: a wave stops computing at its own
// last needed tile but keeps staging until the workgroup's last tile.
// KT = keys per shared tile (32 or 64).  64 halves the per-tile fixed cost a wave pays between its MFMAs -- one barrier,
// one pair of cross-lane max reductions and one rescale test per query tile, the loop and staging bookkeeping -- while
// the MFMA work per key is unchanged (the round-2 kernel spent ~190 VALU per 32 MFMAs: VALU-bound).
template <int D, int QT, bool FP8, int NW, int KT>
__global__ __launch_bounds__(64 * NW, 2) void prefill_attn_kernel(const AttnParams p) {
    constexpr bool TMASK = D == 128;       // causal mask as a compile-time property of the tile body (see `compute`)
    constexpr int KG = KT / 32;            // 32-key groups per tile (V sub-tile images, PV MFMA k-groups)
    constexpr int KBN = KT / 16;           // 16-key MFMA blocks per tile
    constexpr int EB = FP8 ? 1 : 2;
    constexpr int CH = D * EB / 16;
    constexpr int RPI = 64 / CH;
    constexpr int NL = KT / RPI;           // wave-wide load instructions per KT-key tile (K or V) ...
    constexpr int NLW = (NL + NW - 1) / NW;   // ... of which wave w issues j = w, w+NW, ... (< NL)
    constexpr int KS = D / 32;
    constexpr int NB = D / 16;
    constexpr int KROW = D * 2 + 16;
    constexpr int K_BYTES = KT * KROW;
    constexpr int VG = NB * kVSub;         // bytes of one 32-key V group image
    constexpr int STAGE = prefill_stage_bytes<D, KT>();
    constexpr bool FP8_SWAP = FP8 && D == 128;

    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];   // 2 x STAGE, then int[NW]
    int* s_end = reinterpret_cast<int*>(smem + 2 * STAGE);
    const int tid = threadIdx.x;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int lane = tid & 63;
    const int lq = lane & 15, lc = lane >> 4;

    const int bid = blockIdx.x;
    const int xcd = bid & 7;
    const int r0 = bid >> 3;
    const int qg = r0 % p.n_qgroups;
    const int pair = (r0 / p.n_qgroups) * 8 + xcd;
    if (pair >= p.B * p.KH) return;
    const int b = pair / p.KH, kvh = pair % p.KH;
    const int g = p.g;
    const int q0 = p.qo_indptr[b];
    const int n_b = p.qo_indptr[b + 1] - q0;
    const int pg0 = p.page_indptr[b];
    const int npages = p.page_indptr[b + 1] - pg0;
    // clamped to the mapped pages: an over-long last_page_len must not walk past the request's page list
    const int kv_len = npages > 0 ? min((npages - 1) * p.page_size + p.last_page_len[b], npages * p.page_size) : 0;
    const int nrows = n_b * g;
    const int tile_base = (qg * NW + wave) * QT;

    int lim[QT];
    int hi = -1, lo = 0x7fffffff;
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        const int R = (tile_base + qt) * 16 + lq;
        const bool valid = R < nrows;
        const int i = R / g;
        lim[qt] = valid ? (p.causal ? kv_len - n_b + i : kv_len - 1) : -1;
        hi = max(hi, lim[qt]);
        if (valid) lo = min(lo, lim[qt]);
    }
#pragma unroll
    for (int o = 1; o < 16; o <<= 1) {
        hi = max(hi, __shfl_xor(hi, o));
        lo = min(lo, __shfl_xor(lo, o));
    }
    hi = __builtin_amdgcn_readfirstlane(hi);
    lo = __builtin_amdgcn_readfirstlane(lo);
    const int kv_end = min(hi + 1, kv_len);
    if (lane == 0) s_end[wave] = kv_end;
    __syncthreads();
    int kv_end_wg = 0;
#pragma unroll
    for (int w = 0; w < NW; ++w) kv_end_wg = max(kv_end_wg, s_end[w]);
    const int ntiles_wg = kv_end_wg > 0 ? (kv_end_wg + KT - 1) / KT : 0;
    const int my_ntiles = kv_end > 0 ? (kv_end + KT - 1) / KT : 0;

    bf16x8 qf[QT][KS];
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        const int R = (tile_base + qt) * 16 + lq;
        const bool valid = R < nrows;
        const int i = R / g, r = R - i * g;
        const bf16_t* qp = p.q + (int64_t)(q0 + i) * p.q_row_stride + (kvh * g + r) * D;
#pragma unroll
        for (int s = 0; s < KS; ++s) {
            bf16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
            int slot = s * 4 + lc;
            if (FP8_SWAP && s >= 2) slot ^= 1;
            qf[qt][s] = valid ? *reinterpret_cast<const bf16x8*>(qp + slot * 8) : z;
        }
    }
    const float sl2 = FP8 ? p.scale_log2 * p.k_scale[kvh] : p.scale_log2;
    const float vsc = FP8 ? p.v_scale[kvh] : 1.0f;
    f32x4 o[QT][NB];
    float m[QT], l[QT];
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        m[qt] = -1e30f;
        l[qt] = 0.f;
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) o[qt][nb] = f32x4{0.f, 0.f, 0.f, 0.f};
    }

    // staging: this wave's share of the tile = load instructions j = wave + 4*s
    const int wrow = lane / CH, wch = lane % CH;
    const bool swp = FP8_SWAP && wch >= 4;
    int kw[NLW], kw2[NLW], vw[NLW], vw2[NLW];
#pragma unroll
    for (int s = 0; s < NLW; ++s) {
        const int row = wrow + (wave + NW * s) * RPI;      // key row of the tile, 0 .. KT-1
        const int vrow = K_BYTES + (row >> 5) * VG + (row & 31) * 32;
        if constexpr (FP8) {
            kw[s] = row * KROW + ((2 * wch + (swp ? 1 : 0)) << 4);
            kw2[s] = row * KROW + ((2 * wch + (swp ? 0 : 1)) << 4);
            vw[s] = vrow + wch * kVSub + (swp ? 16 : 0);
            vw2[s] = vrow + wch * kVSub + (swp ? 0 : 16);
        } else {
            kw[s] = row * KROW + (wch << 4);
            kw2[s] = 0;
            vw[s] = vrow + (wch >> 1) * kVSub + (wch & 1) * 16;
            vw2[s] = 0;
        }
    }
    const int kra0 = lq * KROW + (lc << 4);       // K fragment (kb, ks) at kra0 + kb * 16 * KROW + ks * 64: immediates
    const int vra = K_BYTES + (lc * 4 + (lq >> 2)) * 32 + (lq & 3) * 8;
    const unsigned goff = (unsigned)((wrow * p.slot_stride + kvh * p.head_stride) * EB + wch * 16);

    u32x4 kreg[NLW], vreg[NLW];
    auto issue = [&](int tt) {
        const int pos0 = tt * KT;
        const int page = pos0 / p.page_size;
        const int slot0 = pos0 - page * p.page_size;
        const int pid = __builtin_amdgcn_readfirstlane(p.page_indices[pg0 + page]);
        const unsigned char* kb_ = reinterpret_cast<const unsigned char*>(p.cache) +
                                   ((int64_t)pid * p.page_stride + (int64_t)slot0 * p.slot_stride) * EB;
        const unsigned char* vb_ = kb_ + p.kv_half * EB;
        const int64_t jstep = (int64_t)RPI * p.slot_stride * EB;
#pragma unroll
        for (int s = 0; s < NLW; ++s)
            if (wave + NW * s < NL) {
                kreg[s] = *reinterpret_cast<const u32x4*>(kb_ + (wave + NW * s) * jstep + goff);
                vreg[s] = *reinterpret_cast<const u32x4*>(vb_ + (wave + NW * s) * jstep + goff);
            }
    };
    auto stage = [&](int t, unsigned char* img) {
#pragma unroll
        for (int s = 0; s < NLW; ++s)
            if (wave + NW * s < NL) {
                // rows past the request's length may hold anything (even NaN): zero V so 0*V stays 0
                if (t * KT + wrow + (wave + NW * s) * RPI >= kv_len) vreg[s] = u32x4{0u, 0u, 0u, 0u};
                if constexpr (FP8) {
                    u32x4 a, c;
                    cvt16_fp8_bf16(kreg[s], a, c);
                    *reinterpret_cast<u32x4*>(img + kw[s]) = a;
                    *reinterpret_cast<u32x4*>(img + kw2[s]) = c;
                    cvt16_fp8_bf16(vreg[s], a, c);
                    *reinterpret_cast<u32x4*>(img + vw[s]) = a;
                    *reinterpret_cast<u32x4*>(img + vw2[s]) = c;
                } else {
                    *reinterpret_cast<u32x4*>(img + kw[s]) = kreg[s];
                    *reinterpret_cast<u32x4*>(img + vw[s]) = vreg[s];
                }
            }
    };
    // MASK is a compile-time property of the call: only the last few tiles of a causal chunk reach past the smallest
    // limit of the wave's rows; every tile before them runs a body without a single compare / select
    // At D = 128 the two bodies cost nothing (one workgroup per CU either way); at D = 64 the duplicated body pushes the
    // kernel from 117 to 167 VGPRs = from two workgroups per CU to one (measured: 1.62 -> 2.38 ms at 16K keys), so
    // there the mask stays a run-time, wave-uniform branch (TMASK = false).
    auto compute = [&](int t, const unsigned char* img, auto mask_c) {
        bool need_mask;
        if constexpr (std::is_same_v<decltype(mask_c), bool>)
            need_mask = mask_c;
        else
            need_mask = decltype(mask_c)::value;
        f32x4 s[QT][KBN];
#pragma unroll
        for (int qt = 0; qt < QT; ++qt)
#pragma unroll
            for (int kb = 0; kb < KBN; ++kb) s[qt][kb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kb = 0; kb < KBN; ++kb)
#pragma unroll
            for (int ks = 0; ks < KS; ++ks) {
                const bf16x8 kf = lds_read_b128(img + kra0 + kb * 16 * KROW + ks * 64);
#pragma unroll
                for (int qt = 0; qt < QT; ++qt)
                    s[qt][kb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[qt][ks], s[qt][kb], 0, 0, 0);
            }
        bf16x8 pf[QT][KG];
#pragma unroll
        for (int qt = 0; qt < QT; ++qt) {
            float v[KBN * 4];                      // raw scores q.k (the softmax scale is folded into the exp2 below)
#pragma unroll
            for (int kb = 0; kb < KBN; ++kb)
#pragma unroll
                for (int j = 0; j < 4; ++j) v[kb * 4 + j] = s[qt][kb][j];
            if (need_mask) {
#pragma unroll
                for (int kb = 0; kb < KBN; ++kb)
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        const int pos = t * KT + kb * 16 + lc * 4 + j;
                        if (pos > lim[qt]) v[kb * 4 + j] = -INFINITY;
                    }
            }
            float mx = v[0];
#pragma unroll
            for (int e = 1; e < KBN * 4; ++e) mx = fmaxf(mx, v[e]);
            mx = fmaxf(mx, __shfl_xor(mx, 16));
            mx = fmaxf(mx, __shfl_xor(mx, 32));
            mx *= sl2;                             // sl2 > 0: max(v) * sl2 == max(v * sl2)
            // lazy rescale: after the first tiles the running maxima rarely move; when no query of the wave raised
            // its maximum (wave-uniform test) the D/4 accumulator multiplies per lane are skipped (alpha == 1)
            if (__builtin_amdgcn_ballot_w64(mx > m[qt]) != 0) {
                const float mnew = fmaxf(m[qt], mx);
                const float alpha = __builtin_amdgcn_exp2f(m[qt] - mnew);
                m[qt] = mnew;
                l[qt] *= alpha;
#pragma unroll
                for (int nb = 0; nb < NB; ++nb) o[qt][nb] *= alpha;
            }
            float ps = 0.f;
            const float mneg = -m[qt];
#pragma unroll
            for (int kg = 0; kg < KG; ++kg) {
                f32x8 pv;
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    const float pe = __builtin_amdgcn_exp2f(fmaf(v[kg * 8 + e], sl2, mneg));   // one v_fma + v_exp
                    pv[e] = pe;
                    ps += pe;
                }
                pf[qt][kg] = __builtin_convertvector(pv, bf16x8);
            }
            l[qt] += ps;
        }
#pragma unroll
        for (int nb = 0; nb < NB; ++nb)
#pragma unroll
            for (int kg = 0; kg < KG; ++kg) {
                const bf16x4 v0 = lds_read_tr(img + kg * VG + nb * kVSub + vra);
                const bf16x4 v1 = lds_read_tr(img + kg * VG + nb * kVSub + 512 + vra);
                const bf16x8 vf = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
                for (int qt = 0; qt < QT; ++qt)
                    o[qt][nb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[qt][kg], o[qt][nb], 0, 0, 0);
            }
    };

    // tile t is staged into image t&1; iteration t+2 overwrites it only after every wave has passed the barrier of
    // iteration t+1, i.e. after it finished computing on tile t -> one barrier per tile
    if (ntiles_wg > 0) issue(0);
    for (int t = 0; t < ntiles_wg; ++t) {
        unsigned char* img = smem + (t & 1) * STAGE;
        stage(t, img);
        if (t + 1 < ntiles_wg) issue(t + 1);
        __syncthreads();
        if (t < my_ntiles) {
            const bool masked = (t * KT + KT - 1) > lo;
            if constexpr (TMASK) {
                if (masked)
                    compute(t, img, std::true_type{});
                else
                    compute(t, img, std::false_type{});
            } else {
                compute(t, img, masked);
            }
        }
    }

#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        l[qt] += __shfl_xor(l[qt], 16);
        l[qt] += __shfl_xor(l[qt], 32);
    }
#pragma unroll
    for (int qt = 0; qt < QT; ++qt) {
        const int R = (tile_base + qt) * 16 + lq;
        if (R < nrows) {
            const int i = R / g, r = R - i * g;
            const float inv = l[qt] > 0.f ? vsc / l[qt] : 0.f;
            bf16_t* op = p.out + ((int64_t)(q0 + i) * p.H + kvh * g + r) * D;
#pragma unroll
            for (int nb = 0; nb < NB; ++nb) {
                const f32x4 ov = o[qt][nb] * inv;
                const int dd = nb * 16 + ((FP8_SWAP && nb >= 4) ? (lc ^ 2) : lc) * 4;
                *reinterpret_cast<bf16x4*>(op + dd) = __builtin_convertvector(ov, bf16x4);
            }
        }
    }
}

// ---------------------------------------------------------------------------------------------------------------
// K3, round 3: the same shared-tile prefill structure on v_mfma_f32_32x32x16_bf16 (bf16 pages).  A wave owns ONE 32-row
// query tile instead of two 16-row tiles; per 32 keys it issues 16 MFMAs of 32 cycles instead of 32 of 16 -- the same
// matrix time -- but every K and V fragment read from LDS now feeds twice the flops (8 + 8 KiB of fragment reads per 32
// keys instead of 16 + 16), the softmax statistics of a query live in TWO lanes (lane, lane ^ 32) instead of four, and
// the per-tile bookkeeping (max reduction, rescale test) is paid once per wave, not once per M tile.
//   S^T = K Q^T   A = K fragment (lane (j, kh): key row j, d = 16 ks + 8 kh ..), B = Q fragment (q row j, same d): the
//                 accumulator register r of lane (j, kh) is S[key (r&3) + 8 (r>>2) + 4 kh][query j];
//   O^T = V^T P^T A = V^T fragment via ds_read_b64_tr_b16 from the same [d/16][32 keys][16] sub-tile images (a 16-lane
//                 group reads a [4 keys][16 d] block: keys 16 s + 4 kh + {0..3} and + 8), B = P^T: registers
//                 8 s .. 8 s + 7 of the S accumulator ARE the k-slots of 16-key step s -- no cross-lane movement.
// Staging, double buffering, the one barrier per tile and the causal bookkeeping are those of prefill_attn_kernel.
// Round 4, measured and NOT kept (profiles/r04_prefill_pipelined_rejected.txt): the tile loop software-pipelined inside a
// wave -- softmax of tile t between the MFMAs of S(t+1), ring of three K/V images, sched_group_barrier-pinned: 589-605
// TFLOP/s at 64 keys (40 registers spilled: the Q fragments come back from scratch inside the loop), 661 at 32 keys against
// 667-685 for the un-pipelined 32-key form and 883-929 for this kernel at 128 keys.
// Measured and NOT kept (same box, profiles/r03_prefill_mfma32_ab.txt): s_setprio(1) around the MFMA clusters (808 vs 820
// TFLOP/s), the causal mask as a compile-time property of the tile body (two bodies: 480 -- the register file again), the
// MFMAs of one accumulator issued back to back instead of alternating accumulators (795 vs 817).
template <int D, int NW, int KT, bool VP = true>
__global__ __launch_bounds__(64 * NW, 2) void prefill32_attn_kernel(const AttnParams p) {
    constexpr int KG = KT / 32;            // 32-key blocks per tile
    constexpr int CH = D * 2 / 16;
    constexpr int RPI = 64 / CH;
    constexpr int NL = KT / RPI;
    constexpr int NLW = (NL + NW - 1) / NW;
    constexpr int KS = D / 16;             // 16-deep k-steps of QK^T
    constexpr int NB = D / 16;             // 16-d V sub-tiles
    constexpr int DB = D / 32;             // 32-d output blocks
    constexpr int KROW = D * 2 + 16;
    constexpr int K_BYTES = KT * KROW;
    constexpr int VG = NB * kVSub;
    constexpr int STAGE = prefill_stage_bytes<D, KT>();

    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];   // 2 x STAGE, then int[NW]
    int* s_end = reinterpret_cast<int*>(smem + 2 * STAGE);
    const int tid = threadIdx.x;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int lane = tid & 63;
    const int j = lane & 31, kh = lane >> 5;

    const int bid = blockIdx.x;
    const int xcd = bid & 7;
    const int r0 = bid >> 3;
    const int qg = r0 % p.n_qgroups;
    const int pair = (r0 / p.n_qgroups) * 8 + xcd;
    if (pair >= p.B * p.KH) return;
    const int b = pair / p.KH, kvh = pair % p.KH;
    const int g = p.g;
    const int q0 = p.qo_indptr[b];
    const int n_b = p.qo_indptr[b + 1] - q0;
    const int pg0 = p.page_indptr[b];
    const int npages = p.page_indptr[b + 1] - pg0;
    const int kv_len = npages > 0 ? min((npages - 1) * p.page_size + p.last_page_len[b], npages * p.page_size) : 0;
    const int nrows = n_b * g;
    const int R = (qg * NW + wave) * 32 + j;           // this lane's query row (both kh halves hold the same query)
    const bool valid = R < nrows;
    const int qi = R / g, qr = R - qi * g;
    const int lim = valid ? (p.causal ? kv_len - n_b + qi : kv_len - 1) : -1;
    int hi = lim, lo = valid ? lim : 0x7fffffff;
#pragma unroll
    for (int o = 1; o < 32; o <<= 1) {
        hi = max(hi, __shfl_xor(hi, o));
        lo = min(lo, __shfl_xor(lo, o));
    }
    hi = __builtin_amdgcn_readfirstlane(hi);
    lo = __builtin_amdgcn_readfirstlane(lo);
    const int kv_end = min(hi + 1, kv_len);
    if (lane == 0) s_end[wave] = kv_end;
    __syncthreads();
    int kv_end_wg = 0;
#pragma unroll
    for (int w = 0; w < NW; ++w) kv_end_wg = max(kv_end_wg, s_end[w]);
    const int ntiles_wg = kv_end_wg > 0 ? (kv_end_wg + KT - 1) / KT : 0;
    const int my_ntiles = kv_end > 0 ? (kv_end + KT - 1) / KT : 0;

    bf16x8 qf[KS];
    {
        const bf16_t* qp = p.q + (int64_t)(q0 + qi) * p.q_row_stride + (kvh * g + qr) * D;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            const bf16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
            qf[ks] = valid ? *reinterpret_cast<const bf16x8*>(qp + ks * 16 + kh * 8) : z;
        }
    }
    const float sl2 = p.scale_log2;
    f32x16 o[DB];
#pragma unroll
    for (int db = 0; db < DB; ++db)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[db][r] = 0.f;
    float m = -1e30f, l = 0.f;

    // staging (identical to prefill_attn_kernel, bf16)
    const int wrow = lane / CH, wch = lane % CH;
    int kw[NLW], vw[NLW];
#pragma unroll
    for (int s = 0; s < NLW; ++s) {
        const int row = wrow + (wave + NW * s) * RPI;
        kw[s] = row * KROW + (wch << 4);
        vw[s] = K_BYTES + (row >> 5) * VG + (row & 31) * 32 + (wch >> 1) * kVSub + (wch & 1) * 16;
    }
    const unsigned goff = (unsigned)((wrow * p.slot_stride + kvh * p.head_stride) * 2 + wch * 16);
    u32x4 kreg[NLW], vreg[NLW];
    auto issue = [&](int tt) {
        const int pos0 = tt * KT;
        const int page = pos0 / p.page_size;
        const int slot0 = pos0 - page * p.page_size;
        const int pid = __builtin_amdgcn_readfirstlane(p.page_indices[pg0 + page]);
        const unsigned char* kb_ = reinterpret_cast<const unsigned char*>(p.cache) +
                                   ((int64_t)pid * p.page_stride + (int64_t)slot0 * p.slot_stride) * 2;
        const unsigned char* vb_ = kb_ + p.kv_half * 2;
        const int64_t jstep = (int64_t)RPI * p.slot_stride * 2;
#pragma unroll
        for (int s = 0; s < NLW; ++s)
            if (wave + NW * s < NL) {
                kreg[s] = *reinterpret_cast<const u32x4*>(kb_ + (wave + NW * s) * jstep + goff);
                vreg[s] = *reinterpret_cast<const u32x4*>(vb_ + (wave + NW * s) * jstep + goff);
            }
    };
    auto stage = [&](int t, unsigned char* img) {
#pragma unroll
        for (int s = 0; s < NLW; ++s)
            if (wave + NW * s < NL) {
                if (t * KT + wrow + (wave + NW * s) * RPI >= kv_len) vreg[s] = u32x4{0u, 0u, 0u, 0u};
                *reinterpret_cast<u32x4*>(img + kw[s]) = kreg[s];
                *reinterpret_cast<u32x4*>(img + vw[s]) = vreg[s];
            }
    };
    // fragment addresses: K (lane (j, kh)): row j, 16-B piece 2 ks + kh; V tr-read (16-lane group = (kh, j >> 4)):
    // sub-tile ((lane >> 4) & 1) of the 32-d block, key row 4 kh + (lq >> 2) (+ 16 s, + 8), d group lq & 3
    const int kra0 = j * KROW + (kh << 4);
    const int lq = lane & 15;
    // the two 16-d sub-tiles one tr-read pairs (lanes 0-15 | 16-31 of a 32-lane group): sub-tiles db and db + NB/2, whose
    // images lie 4 x 1056 B = 128 B (mod 256) apart at D = 128 -- disjoint halves of the 64 LDS banks.  Adjacent sub-tiles
    // (32 B mod 256 apart: VP = false, the first version) overlap on 24 banks: every ds_read_b64_tr_b16 took 4 LDS cycles
    // instead of 2 (SQ_LDS_BANK_CONFLICT = 2 per MFMA, 28 % of SQ_LDS_IDX_ACTIVE; profiles/r03_prefill_pmc_call22.txt)
    constexpr int VPS = VP ? NB / 2 : 1;        // sub-tile distance inside a pair
    constexpr int VDS = VP ? 1 : 2;             // sub-tile distance between output blocks
    const int vra0 = K_BYTES + ((lane >> 4) & 1) * VPS * kVSub + (kh * 4 + (lq >> 2)) * 32 + (lq & 3) * 8;

    auto compute = [&](int t, const unsigned char* img, bool need_mask) {
        f32x16 sc[KG];
#pragma unroll
        for (int kg = 0; kg < KG; ++kg)
#pragma unroll
            for (int r = 0; r < 16; ++r) sc[kg][r] = 0.f;
        // ks outer, key block inner: consecutive MFMAs accumulate into different registers
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
#pragma unroll
            for (int kg = 0; kg < KG; ++kg) {
                const bf16x8 kf = lds_read_b128(img + kra0 + kg * 32 * KROW + ks * 32);
                sc[kg] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[ks], sc[kg], 0, 0, 0);
            }
        bf16x8 pf[KG][2];
        if (need_mask) {
            // a real (wave-uniform) branch: only the last tiles of a causal chunk take it; the empty volatile asm keeps
            // the compiler from if-converting it into 32 compare/select pairs executed on every tile
#pragma unroll
            for (int kg = 0; kg < KG; ++kg)
#pragma unroll
                for (int r = 0; r < 16; ++r) {
                    const int pos = t * KT + kg * 32 + (r & 3) + 8 * (r >> 2) + 4 * kh;
                    float v = sc[kg][r];
                    if (pos > lim) v = -INFINITY;
                    asm volatile("" : "+v"(v));          // volatile: cannot be hoisted out of the branch
                    sc[kg][r] = v;
                }
        }
        float mx = sc[0][0];
#pragma unroll
        for (int kg = 0; kg < KG; ++kg)
#pragma unroll
            for (int r = 0; r < 16; ++r) mx = fmaxf(mx, sc[kg][r]);
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        mx *= sl2;
        if (__builtin_amdgcn_ballot_w64(mx > m) != 0) {       // lazy rescale, wave-uniform
            const float mnew = fmaxf(m, mx);
            const float alpha = __builtin_amdgcn_exp2f(m - mnew);
            m = mnew;
            l *= alpha;
#pragma unroll
            for (int db = 0; db < DB; ++db)
#pragma unroll
                for (int r = 0; r < 16; ++r) o[db][r] *= alpha;
        }
        const float mneg = -m;
        float ps = 0.f;
#pragma unroll
        for (int kg = 0; kg < KG; ++kg)
#pragma unroll
            for (int s16 = 0; s16 < 2; ++s16) {
                f32x8 pv;
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    const float pe = __builtin_amdgcn_exp2f(fmaf(sc[kg][s16 * 8 + e], sl2, mneg));
                    pv[e] = pe;
                    ps += pe;
                }
                pf[kg][s16] = __builtin_convertvector(pv, bf16x8);
            }
        l += ps;
        auto pv = [&](int db, int kg, int s16) {
            const unsigned char* vb = img + kg * VG + (VDS * db) * kVSub + vra0 + s16 * 16 * 32;
            const bf16x4 v0 = lds_read_tr(vb);
            const bf16x4 v1 = lds_read_tr(vb + 8 * 32);
            const bf16x8 vf = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
            o[db] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pf[kg][s16], o[db], 0, 0, 0);
        };
        // 16-key step outer, d block inner: consecutive MFMAs accumulate into different O blocks
#pragma unroll
        for (int kg = 0; kg < KG; ++kg)
#pragma unroll
            for (int s16 = 0; s16 < 2; ++s16)
#pragma unroll
                for (int db = 0; db < DB; ++db) pv(db, kg, s16);
    };

    if (ntiles_wg > 0) issue(0);
    for (int t = 0; t < ntiles_wg; ++t) {
        unsigned char* img = smem + (t & 1) * STAGE;
        stage(t, img);
        if (t + 1 < ntiles_wg) issue(t + 1);
        __syncthreads();
        if (t < my_ntiles) compute(t, img, (t * KT + KT - 1) > lo);
    }

    l += __shfl_xor(l, 32);
    if (valid) {
        const float inv = l > 0.f ? 1.0f / l : 0.f;
        bf16_t* op = p.out + ((int64_t)(q0 + qi) * p.H + kvh * g + qr) * D;
#pragma unroll
        for (int db = 0; db < DB; ++db)
#pragma unroll
            for (int rg = 0; rg < 4; ++rg) {
                const f32x4 ov = {o[db][rg * 4] * inv, o[db][rg * 4 + 1] * inv, o[db][rg * 4 + 2] * inv,
                                  o[db][rg * 4 + 3] * inv};
                const int dd = VP ? (db + (rg >> 1) * (NB / 2)) * 16 + (rg & 1) * 8 : db * 32 + rg * 8;
                *reinterpret_cast<bf16x4*>(op + dd + kh * 4) = __builtin_convertvector(ov, bf16x4);
            }
    }
}

struct AttnPlan {
    bool splitq;
    int nw;   // prefill: waves per workgroup sharing each K/V tile (4 or 8); decode / verify: waves splitting the tiles
    int qt;
    int n_qgroups;
    int nsplit;
    int rows_cap;  // rows per item in the workspace (decode mode)
};

// split-KV target: one 4-wave workgroup per CU measured best on MI355X for every TP shard shape of the verify
// step (B=64, 16K: 81 % / 80 % / 75 % / 70 % of HBM peak at KH_local = 8 / 4 / 2 / 1 vs 77 / 77 / 72 / 47 % at 1024);
// per-workgroup prologue/epilogue and the partial-result round trip dominate once a wave owns < ~30 tiles
int g_target_wgs = 256;  // dev knob: md_debug_set_attn_target_wgs
int g_decode_nw = 0;     // dev knob (md_debug_set_attn_waves): 0 = the rule in make_plan, 4 / 8 = forced
int g_prefill_nw = 0;     // dev knob (md_debug_set_prefill_kt): 0 = the measured rule below, 4 / 8 = forced

// measurement mode of the decode / verify kernel (bench.py's roofline): see md_debug_attn_timing
struct TimedLaunch { hipEvent_t e0, e1; };
constexpr size_t kMaxTimed = 4096;
bool g_time_launches = false;
int g_time_rows = 0;
bool g_time_this = false;  // set by md_paged_attn for the launch it is about to make
std::vector<TimedLaunch> g_timed;

AttnPlan make_plan(int B, int n_max, int H, int KH, int max_pages, int page_size, bool fp8) {
    AttnPlan pl;
    pl.nw = 4;
    const int g = H / KH;
    const int rows = n_max * g;
    if (rows <= 32) {
        pl.splitq = false;
        pl.qt = rows <= 16 ? 1 : 2;
        pl.n_qgroups = 1;
        const long max_tiles = (long)max_pages * page_size / 32;
        long want = (g_target_wgs + (long)B * KH - 1) / ((long)B * KH);
        long cap = max_tiles / 16;  // >= 16 tiles (4 per wave) per workgroup
        if (cap < 1) cap = 1;
        if (want > cap) want = cap;
        if (want > 64) want = 64;
        if (want < 1) want = 1;
        pl.nsplit = (int)want;
        pl.rows_cap = pl.qt * 16;
        // eight waves where measured faster: the fp8 two-M-tile kernel when the launch leaves one workgroup per CU and
        // every wave still owns a stream of tiles (>= 8 each); see the kernel's header
        const long wgs = (long)B * KH * pl.nsplit, tiles_per_wg = max_tiles / pl.nsplit;
        pl.nw = (fp8 && pl.qt == 2 && wgs <= 256 && tiles_per_wg >= 64) ? 8 : 4;
        if (g_decode_nw == 4 || g_decode_nw == 8) pl.nw = g_decode_nw;
    } else {
        pl.splitq = true;
        pl.qt = rows >= 128 ? 2 : 1;
        // 8 waves (256 query rows) per workgroup halve the number of times a (request, kv head) stream is pulled
        // through L2: +21 % at the 8B TP1 shape and still +10 % at the TP8 shard shape where the grid no longer
        // fills the chip (128 workgroups); fp8 staging (4 load instructions per tile, plus the conversion) is
        // better spread over 4-wave workgroups (measured: 2.9 vs 3.3 ms)
        pl.nw = (!fp8 && rows >= 16 * pl.qt * 8) ? 8 : 4;
        if (g_prefill_nw == 4 || (g_prefill_nw == 8 && rows >= 16 * pl.qt * 8)) pl.nw = g_prefill_nw;   // dev knob
        const int wg_rows = 16 * pl.qt * pl.nw;
        pl.n_qgroups = (rows + wg_rows - 1) / wg_rows;
        pl.nsplit = 1;
        pl.rows_cap = 0;
    }
    return pl;
}

template <int D, int QT, bool FP8, int NWV>
int launch_attn_nw(const AttnParams& p, int grid, hipStream_t st) {
    constexpr int lds = NWV * attn_wave_lds<D, QT>();
    static_assert(lds <= 160 * 1024, "the waves' LDS images must fit the CU");
    static MdPerDeviceOnce attr_once;
    if (attr_once.first()) {
        hipError_t e = hipFuncSetAttribute(
            reinterpret_cast<const void*>(&paged_attn_kernel<D, QT, FP8, NWV>),
            hipFuncAttributeMaxDynamicSharedMemorySize, lds);
        if (e != hipSuccess) {
            md_set_error("md_paged_attn: hipFuncSetAttribute(%d B LDS) failed: %s", lds, hipGetErrorString(e));
            return MD_ERR_LAUNCH;
        }
    }
    hipStreamCaptureStatus cap = hipStreamCaptureStatusNone;
    if (g_time_this && g_timed.size() < kMaxTimed &&
        (hipStreamIsCapturing(st, &cap) != hipSuccess || cap == hipStreamCaptureStatusNone)) {
        // measurement mode (md_debug_attn_timing): the kernel's own begin / end timestamps -- what a rocprofv3 kernel
        // trace reports -- instead of stream events around the launch, which also see the dispatch overhead
        hipEvent_t e0, e1;
        if (hipEventCreate(&e0) == hipSuccess && hipEventCreate(&e1) == hipSuccess) {
            hipExtLaunchKernelGGL((paged_attn_kernel<D, QT, FP8, NWV>), dim3(grid), dim3(64 * NWV), lds, st, e0, e1, 0, p);
            g_timed.push_back({e0, e1});
            MD_CHECK_LAUNCH("md_paged_attn");
            return MD_OK;
        }
    }
    hipLaunchKernelGGL((paged_attn_kernel<D, QT, FP8, NWV>), dim3(grid), dim3(64 * NWV), lds, st, p);
    MD_CHECK_LAUNCH("md_paged_attn");
    return MD_OK;
}

template <int D, int QT, bool FP8>
int launch_attn(const AttnParams& p, int grid, int nw, hipStream_t st) {
    return nw == 8 ? launch_attn_nw<D, QT, FP8, 8>(p, grid, st) : launch_attn_nw<D, QT, FP8, 4>(p, grid, st);
}

int g_prefill_kt = 64;    // dev knob (md_debug_set_prefill_kt): keys per shared tile of the bf16 prefill kernel (D = 64)

template <int D, int QT, bool FP8, int NW, int KT>
int launch_prefill_kt(const AttnParams& p, int grid, hipStream_t st) {
    constexpr int lds = 2 * prefill_stage_bytes<D, KT>() + 32;
    auto k = prefill_attn_kernel<D, QT, FP8, NW, KT>;
    if (lds > 64 * 1024) {
        static MdPerDeviceOnce once;
        if (once.first()) {
            if (hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, lds) !=
                hipSuccess) {
                once.undo();
                md_set_error("md_paged_attn(prefill): hipFuncSetAttribute(%d B LDS) failed", lds);
                return MD_ERR_LAUNCH;
            }
        }
    }
    hipLaunchKernelGGL(k, dim3(grid), dim3(64 * NW), lds, st, p);
    MD_CHECK_LAUNCH("md_paged_attn(prefill)");
    return MD_OK;
}

// The 32x32x16-MFMA kernel serves the two-M-tile bf16 prefill shapes.  Keys per shared tile: 128 at D = 128 (242 VGPRs, no
// spills, 137 KB LDS), 64 at D = 64 (118 VGPRs: two workgroups per CU; 128 keys would cost the second one) -- measured,
// same box (profiles/r03_prefill_mfma32_ab.txt; B = 64, 128 tokens x 32 heads vs 16 K keys, TFLOP/s): D = 128: 668 (16x16
// kernel, 32 keys) -> 778 (32) -> 805 (64) -> 874 (128); D = 64: 712 -> 729 (64), 667 (128).
// Dev knob (md_debug_set_prefill_mfma32 / MAGICDEC_PREFILL_MFMA32): -1 = this rule, 0 = the 16x16x32 kernel, 32 | 64 | 128 forced
// (halved until it divides the page size), 129 = first V pairing.  (The two timing ablations of docs/DESIGN_r1_r5_lab_notes.md 3.5 -- no
// softmax / no P.V, wrong results by construction -- were removed after the measurement.)
int g_prefill_mfma32 = -1;

template <int D, int NW, int KT, bool VP = true>
int launch_prefill32_kt(const AttnParams& p, int grid, hipStream_t st) {
    constexpr int lds = 2 * prefill_stage_bytes<D, KT>() + 32;
    auto k = prefill32_attn_kernel<D, NW, KT, VP>;
    if (lds > 64 * 1024) {
        static MdPerDeviceOnce once;
        if (once.first()) {
            if (hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, lds) !=
                hipSuccess) {
                once.undo();
                md_set_error("md_paged_attn(prefill32): hipFuncSetAttribute(%d B LDS) failed", lds);
                return MD_ERR_LAUNCH;
            }
        }
    }
    hipLaunchKernelGGL(k, dim3(grid), dim3(64 * NW), lds, st, p);
    MD_CHECK_LAUNCH("md_paged_attn(prefill32)");
    return MD_OK;
}

template <int D, int QT, bool FP8>
int launch_prefill(const AttnParams& p, int grid, int nw, hipStream_t st) {
    // a shared tile never crosses a page: keys per tile must divide the page size (32 always does, md_paged_attn checks)
    const auto fits = [&](int kt) { return p.page_size % kt == 0; };
    if constexpr (!FP8 && QT == 2) {
        if constexpr (D == 128)
            if (nw == 8 && fits(128)) {      // dev variants of the 128-key kernel (md_debug_set_prefill_mfma32)
                if (g_prefill_mfma32 == 129) return launch_prefill32_kt<D, 8, 128, false>(p, grid, st);    // first V pairing
            }
        int kt32 = g_prefill_mfma32 < 0 ? (D == 128 ? 128 : 64) : g_prefill_mfma32;
        while (kt32 > 32 && !fits(kt32)) kt32 >>= 1;
        // 128-key tiles only with 8 waves: the 4-wave instantiation stages twice the rows per wave and spills 11 registers
        //  -- 4-wave workgroups take 64-key tiles
        if (kt32 == 128 && nw == 8) return launch_prefill32_kt<D, 8, 128>(p, grid, st);
        if (kt32 == 128) kt32 = 64;
        if (kt32 == 64)
            return nw == 8 ? launch_prefill32_kt<D, 8, 64>(p, grid, st) : launch_prefill32_kt<D, 4, 64>(p, grid, st);
        if (kt32 == 32)
            return nw == 8 ? launch_prefill32_kt<D, 8, 32>(p, grid, st) : launch_prefill32_kt<D, 4, 32>(p, grid, st);
    }
    if constexpr (!FP8 && D == 64) {
        // 64-key shared tiles where the registers allow it: D = 64, bf16 pages, run-time mask (124 VGPRs: two workgroups
        // per CU) -- 714 vs 663 TFLOP/s at the 1B draft model's prefill shape, +6..15 % at shorter contexts
        // (profiles/r03_prefill_ab.txt).  At D = 128 the 64-key body needs 256 VGPRs + 43 spilled (o 64 + q 32 + s 32 +
        // p 16 ...) and LOSES (587 vs 663 TFLOP/s); the fp8 staging path (two conversions per load) was not
        // generalised (the D = 128 instantiations of that body, 43-63 spilled registers, are gone).
        if (g_prefill_kt == 64 && fits(64))
            return nw == 8 ? launch_prefill_kt<D, QT, FP8, 8, 64>(p, grid, st)
                           : launch_prefill_kt<D, QT, FP8, 4, 64>(p, grid, st);
    }
    return nw == 8 ? launch_prefill_kt<D, QT, FP8, 8, 32>(p, grid, st) : launch_prefill_kt<D, QT, FP8, 4, 32>(p, grid, st);
}

}  // namespace

#ifdef MD_DEV_KNOBS   // include/magicdec_hip_dev.h: tuning knobs, not part of the drop-in boundary
extern "C" void md_debug_set_attn_target_wgs(int n) { g_target_wgs = n > 0 ? n : 256; }
extern "C" void md_debug_set_attn_waves(int nw) { g_decode_nw = (nw == 4 || nw == 8) ? nw : 0; }
extern "C" void md_debug_set_prefill_mfma32(int kt) {
    // < 0: the rule, 0: the 16x16 kernel, 32 | 64 | 128: keys per tile; 129: 128 keys with the first version's V pairing
    g_prefill_mfma32 = (kt == 32 || kt == 64 || kt == 128 || kt == 129 || kt < 0) ? kt : 0;
}

extern "C" void md_debug_set_prefill_kt(int kt, int nw) {
    g_prefill_kt = kt == 32 ? 32 : 64;
    g_prefill_nw = (nw == 4 || nw == 8) ? nw : 0;
}
#endif

extern "C" void md_debug_attn_timing(int enable, int n_rows) {
    g_time_launches = enable != 0;
    g_time_rows = n_rows;
}

extern "C" int md_debug_attn_timing_read(float* ms_out, int cap) {
    (void)hipDeviceSynchronize();
    int n = 0;
    for (auto& t : g_timed) {
        float ms = 0.f;
        if (hipEventElapsedTime(&ms, t.e0, t.e1) == hipSuccess && ms_out && n < cap) ms_out[n++] = ms;
        (void)hipEventDestroy(t.e0);
        (void)hipEventDestroy(t.e1);
    }
    g_timed.clear();
    return n;
}

extern "C" size_t md_paged_attn_workspace_bytes(int B, int n_max, int H, int KH, int D,
                                                int max_pages_per_req, int page_size) {
    if (B <= 0 || KH <= 0 || H % KH != 0) return 0;
    const AttnPlan pl = make_plan(B, n_max, H, KH, max_pages_per_req, page_size, false);
    if (pl.splitq || pl.nsplit == 1) return 256;
    const size_t slots = (size_t)B * KH * pl.nsplit * pl.rows_cap;
    return slots * (size_t)D * 4 + slots * 8 + 256;
}

extern "C" int md_paged_attn(const void* q, int64_t q_row_stride, const void* cache, void* out,
                             const int32_t* qo_indptr, const int32_t* page_indices,
                             const int32_t* page_indptr, const int32_t* last_page_len, int B,
                             int n_max, int H, int KH, int D, int page_size, int causal,
                             float sm_scale, int max_pages_per_req, int kv_dtype, const float* k_scale,
                             const float* v_scale, void* workspace, size_t workspace_bytes,
                             md_stream_t stream) {
    MD_CHECK_ARG(q && cache && out && qo_indptr && page_indices && page_indptr && last_page_len,
                 "md_paged_attn: null pointer argument");
    MD_CHECK_ARG(B > 0 && n_max > 0 && H > 0 && KH > 0 && H % KH == 0,
                 "md_paged_attn: bad shape B=%d n_max=%d H=%d KH=%d", B, n_max, H, KH);
    if (D != 64 && D != 128) {
        md_set_error("md_paged_attn: head_dim %d unsupported (64 or 128)", D);
        return MD_ERR_UNSUPPORTED;
    }
    MD_CHECK_ARG(page_size > 0 && page_size % 32 == 0, "md_paged_attn: page_size %d must be a multiple of 32", page_size);
    MD_CHECK_ARG(q_row_stride % 8 == 0 && ((uintptr_t)q & 15) == 0 && ((uintptr_t)cache & 15) == 0 &&
                     ((uintptr_t)out & 7) == 0,
                 "md_paged_attn: q/cache must be 16-byte aligned with a row stride multiple of 8");
    MD_CHECK_ARG(max_pages_per_req > 0, "md_paged_attn: max_pages_per_req must be > 0");
    MD_CHECK_ARG((kv_dtype & ~(MD_KV_DTYPE_MASK | MD_KV_LAYOUT_HND)) == 0, "md_paged_attn: unknown kv_dtype flags");
    const bool hnd = (kv_dtype & MD_KV_LAYOUT_HND) != 0;
    kv_dtype &= MD_KV_DTYPE_MASK;
    MD_CHECK_ARG(kv_dtype == MD_KV_BF16 || (kv_dtype == MD_KV_FP8_E4M3 && k_scale && v_scale),
                 "md_paged_attn: kv_dtype must be MD_KV_BF16 or MD_KV_FP8_E4M3 (with per-head scales)");
    const bool fp8 = kv_dtype == MD_KV_FP8_E4M3;

    const AttnPlan pl = make_plan(B, n_max, H, KH, max_pages_per_req, page_size, fp8);
    AttnParams p;
    p.q = (const bf16_t*)q;
    p.cache = cache;
    p.k_scale = fp8 ? k_scale : nullptr;
    p.v_scale = fp8 ? v_scale : nullptr;
    p.out = (bf16_t*)out;
    p.qo_indptr = qo_indptr;
    p.page_indices = page_indices;
    p.page_indptr = page_indptr;
    p.last_page_len = last_page_len;
    p.q_row_stride = q_row_stride;
    p.slot_stride = hnd ? D : KH * D;
    p.head_stride = hnd ? page_size * D : D;
    p.kv_half = (int64_t)page_size * KH * D;
    p.page_stride = 2 * p.kv_half;
    p.B = B;
    p.H = H;
    p.KH = KH;
    p.g = H / KH;
    p.page_size = page_size;
    p.causal = causal ? 1 : 0;
    p.nsplit = pl.nsplit;
    p.n_qgroups = pl.n_qgroups;
    p.scale_log2 = sm_scale * 1.4426950408889634f;
    p.ws_o = nullptr;
    p.ws_ml = nullptr;
    if (!pl.splitq && pl.nsplit > 1) {
        const size_t slots = (size_t)B * KH * pl.nsplit * pl.rows_cap;
        const size_t need = slots * (size_t)D * 4 + slots * 8;
        if (!workspace || workspace_bytes < need || ((uintptr_t)workspace & 15)) {
            md_set_error("md_paged_attn: workspace too small or misaligned (%zu < %zu)", workspace_bytes, need);
            return MD_ERR_WORKSPACE;
        }
        p.ws_o = (float*)workspace;
        p.ws_ml = p.ws_o + slots * (size_t)D;
    }
    hipStream_t st = (hipStream_t)stream;
    const int npairs8 = (B * KH + 7) / 8 * 8;
    const int grid = npairs8 * pl.n_qgroups * pl.nsplit;
    g_time_this = g_time_launches && n_max == g_time_rows;
    int rc;
#define MD_ATTN_DISPATCH(DD, FP)                                                                                  \
    (pl.splitq ? (pl.qt == 2 ? launch_prefill<DD, 2, FP>(p, grid, pl.nw, st)                                         \
                             : launch_prefill<DD, 1, FP>(p, grid, pl.nw, st))                                       \
               : (pl.qt == 2 ? launch_attn<DD, 2, FP>(p, grid, pl.nw, st) : launch_attn<DD, 1, FP>(p, grid, pl.nw, st)))
    if (D == 128)
        rc = fp8 ? MD_ATTN_DISPATCH(128, true) : MD_ATTN_DISPATCH(128, false);
    else
        rc = fp8 ? MD_ATTN_DISPATCH(64, true) : MD_ATTN_DISPATCH(64, false);
#undef MD_ATTN_DISPATCH
    if (rc != MD_OK) return rc;
    if (!pl.splitq && pl.nsplit > 1) {
        const int64_t threads = (int64_t)B * KH * pl.n_qgroups * pl.rows_cap * (D / 4);
        const unsigned mgrid = (unsigned)((threads + 255) / 256);
        if (D == 128)
            hipLaunchKernelGGL((attn_merge_kernel<128>), dim3(mgrid), dim3(256), 0, st, p, pl.rows_cap);
        else
            hipLaunchKernelGGL((attn_merge_kernel<64>), dim3(mgrid), dim3(256), 0, st, p, pl.rows_cap);
        MD_CHECK_LAUNCH("md_paged_attn(merge)");
    }
    return MD_OK;
}
