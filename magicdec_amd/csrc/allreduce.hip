// C1: sum-all-reduce of the per-layer bf16 partials over peer-mapped buffers (xGMI), for the tensor-parallel decode
// path -- one-shot and two-shot, optionally fused with the residual add + RMSNorm that follows it.
//
// Replaces the two `dist.all_reduce` per layer of the reference (Engine/SnapKV/model.py:334-335,453-454 and twins;
// NCCL there, with ENABLE_INTRA_NODE_COMM one-/two-shot kernels per README.md:59) plus, in the fused form, the
// `h = x + y ; norm(h)` that consumes the result (model.py:260-278).  The messages are small and latency-bound --
// [B*(gamma+1), dim] bf16 = 2 MiB for the 8B verify step, 256 KiB for a 1B draft step -- and xGMI is point-to-point:
// a ring pays 2(N-1) link latencies.
//
//   one-shot  every rank publishes its partial in an IPC-mapped buffer, raises a flag at every peer, then reads all
//             N partials and sums them itself: one hop, (N-1) x message inbound per rank.  Right for <= 256 KiB.
//   two-shot  rank r owns the rows r, r+N, ...: it sums only those over the N published partials (reduce-scatter),
//             publishes the reduced rows in a second registered buffer, raises a second flag, and copies the other
//             ranks' reduced rows (all-gather): two hops, 2(N-1)/N x message inbound.  Right for the 2 MiB verify
//             message at N = 8 (3.5 MiB instead of 14 MiB per rank).
//
// Determinism: a row is summed by exactly one piece of code in rank order 0..N-1 with fp32
// accumulation and one rounding -- in the one-shot form by every rank identically, in the two-shot form by its
// owner only -- so all ranks obtain bit-identical results (the replicated argmax / page tables need that).
//
// Fused epilogue (md_allreduce_add_rmsnorm): the unit of work is a ROW of the [rows, dim] message and a wavefront
// handles a whole row, so the consumer of the reduced row can finish the layer's next two ops in registers:
// h = bf16(x + sum) and y = bf16(bf16(h * rsqrt(mean(h^2) + eps)) * w) -- the reference's rounding points
// (Engine/SnapKV/model.py:464-469) -- saving one kernel launch and one round trip of h per all-reduce.
//
// Protocol, per call k = 1, 2, ... (k lives in device memory so that a captured hipGraph replays correctly; every
// block of a call reads the same k because the counter is advanced only once ALL blocks of the call have read it:
// round 5, see "call counter" below) and per block b of a grid that is sized to the message:
//   1. copy the rows of block b from `in` into my data buffer half (k & 1);
//   2. release; store k into start[b][me] of every peer; spin until start[b][p] >= k for every p; acquire;
//   3. one-shot: sum the rows of block b over all ranks -> out.           two-shot: sum MY rows of block b -> my
//      result buffer half (k & 1) (and out); release; store k into start2[b][me] of every peer; spin until
//      start2[b][p] >= k; acquire; copy the other owners' rows of block b from their result buffers -> out.
//   Rows are dealt to blocks by (row / N) % grid, so the producer of anything block b reads is the peer's block b.
//   Two halves per buffer make a closing barrier unnecessary and the message-size-dependent grid safe: I overwrite
//   half (k & 1) in call k+2, after ALL my blocks finished call k+1; one of them (block 0 exists in every call) waited
//   for every peer's call-(k+1) flag, so every peer had entered call k+1, i.e. finished reading in call k (kernels
//   of one stream run in order).  tests/test_allreduce_protocol_model.py runs the protocol under random schedules.
// Signals live in uncached (fine-grained) memory; data buffers are ordinary device memory -- the system-scope
// release / acquire pair performs the L2 write-back / invalidate the AMDGPU memory model prescribes.
// Spins are bounded: on a time-out the kernel does NOT continue silently -- it records the error in the status word
// and POISONS its output rows with NaN, and the host raises at the next status check (Engine/oneshot.py).
#include "md_common.h"

namespace {

constexpr int kMaxRanks = 8;
constexpr int kMaxBlocks = 64;
constexpr int kThreads = 512;                 // 8 wavefronts: 8 rows in flight per block
constexpr int kRowVecs = 512;                 // plain (unfused) calls: a "row" is 512 vectors of 8 bf16 = 8 KiB
constexpr int kMaxVecPerLane = 16;            // fused rows: dim <= 64 * 16 * 8 = 8192
constexpr unsigned long long kSpinTimeoutTicks = 200ull * 1000 * 1000;   // wall_clock64() ticks at 100 MHz: 2 s

struct Signal {
    uint32_t start[kMaxBlocks][kMaxRanks];    // written by peers (system-scope release), read by the owner
    uint32_t start2[kMaxBlocks][kMaxRanks];   // second hop of the two-shot form
    uint32_t status;                          // owner only: 0 ok, 1 = a spin timed out (output poisoned)
};

// Call counter (round 5).  Owner-only state in ORDINARY (cached) device memory: ctrl[0] = number of calls whose counter
// has been handed on, ctrl[1] = blocks of the running call that have read it.  Rounds 2-4 kept both in the uncached signal
// area and let the LAST block to FINISH advance the counter: an uncached read at the head of every launch (everything
// else waits for k) and a returning atomic on uncached memory at its tail -- ~3 us of a 9 us launch with one rank
// (tools/ar_bench.py).  All the protocol needs is that no block of call k reads the counter after it was advanced, so the
// last block to have READ it advances it: thread 0 reads ctrl[0] (behind the waves' prefetch loads; its value returns
// before the block's first barrier), after the barrier lane 0 of the last wave adds 1 to ctrl[1] -- at once if that wave
// has no row in this call (usual: nobody waits for the round trip), after its rows otherwise -- and the block that drew
// G - 1 resets ctrl[1] and stores k.  The next launch on the
// stream reads it behind a kernel boundary.  (tests/test_allreduce_protocol_model.py models exactly this.)
struct ArDev {
    bf16_t* data[kMaxRanks];   // peer buffers: [data half 0][data half 1][result half 0][result half 1]
    Signal* sig[kMaxRanks];
    uint32_t* ctrl;            // owner only, cached: [0] call counter, [1] blocks of the running call that have read it
    int rank, world;
    size_t buf_elems;          // elements per half buffer
    int publish_fence;         // MD_AR_PUBLISH_FENCE: a system-scope release fence behind the write-through stores
};

struct ArArgs {
    const bf16_t* in;          // [rows][row_elems] contiguous
    bf16_t* out;               // sum (plain) or h = x + sum (fused)
    const bf16_t* resid;       // fused: x
    const bf16_t* weight;      // fused: RMSNorm weight [row_elems]
    bf16_t* out_y;             // fused: normalised rows
    float eps;
    int rows, row_vecs;        // row_vecs = vectors of 8 bf16 per row (the last row of a plain call may be shorter)
    size_t n_vec;              // total vectors
};

// Publishing (round 4).  Rounds 2-3 wrote the registered buffers with plain stores and made them
// visible with a system-scope RELEASE FENCE (buffer_wbl2 sc0 sc1: a write-back sweep of the XCD's L2, 1.7-6.5 us by
// MI355X_MICROARCH.md), polled the flags with ACQUIRE loads (an L1/L2 invalidate per poll) and closed every call with
// two __threadfence(): ~18 us per launch before a byte had crossed a link.  Now the payload is stored WRITE-THROUGH
// at system scope (16-byte `sc0 sc1` stores: the data is in memory when the store retires), every wave drains its own
// stores (s_waitcnt vmcnt(0), inline asm: the compiler cannot drop it), the flags are polled with RELAXED loads and ONE
// acquire fence per hop follows the poll (the guide's R1 hand-off in its cross-device form); the call counter needs no
// fence at all -- its only reader is the next launch on the same stream.
// INVARIANT: every store into a registered buffer that a PEER reads -- data[] (the published partials) and the
// result halves (`myres`) -- must go through store_wt and be followed by drain_stores() before the flag is raised; a plain
// store would sit in this XCD's L2 behind a relaxed flag.  finish_row's plain stores write the caller's OUTPUT tensors, which
// no peer reads.  The correctness of the hand-off rests on vmcnt retiring a write-through store only once it is visible
// at system scope; it has been validated between processes sharing one GPU (tests/test_gpu_allreduce.py: thousands of
// calls, bit-exact) and NOT yet over xGMI links -- bench.py's child-process report is what decides
// whether a multi-GPU run uses it.
__device__ __forceinline__ void store_wt(bf16_t* base, size_t vec_index, const u32x4 v) {
    u32x4* p = reinterpret_cast<u32x4*>(base) + vec_index;
    asm volatile("global_store_dwordx4 %0, %1, off sc0 sc1\n\ts_nop 1" ::"v"(p), "v"(v) : "memory");
}
__device__ __forceinline__ void drain_stores() { asm volatile("s_waitcnt vmcnt(0)" ::: "memory"); }

// MD_AR_PUBLISH_FENCE (round 6): the write-through publish above rests on ONE hardware
// property that no single-GPU test can probe -- that vmcnt retires an `sc0 sc1` store only once a PEER can see it.  In
// this mode the flag-raising lanes additionally execute the system-scope RELEASE fence of rounds 2-3 (buffer_wbl2 sc0 sc1
// + s_waitcnt: the AMDGPU memory model's own release sequence, which writes back whatever this XCD's L2 still holds)
// between the block barrier that follows every wave's drain and the flag stores.  It costs the L2 write-back sweep
// (1.7-6.5 us per hop by MI355X_MICROARCH.md) and assumes nothing beyond the documented memory model: if the
// write-through arm fails its bit-exact stress on real links, a run degrades to THIS xGMI path, not all the way to RCCL.
__device__ __forceinline__ void release_fence_system() {
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "");
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");          // the compiler may drop the fence's own wait (guide: hazard)
}

__device__ __forceinline__ bool spin_ge(const uint32_t* p, uint32_t want) {
    const unsigned long long t0 = wall_clock64();
    while ((int32_t)(__hip_atomic_load(p, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_SYSTEM) - want) < 0) {
        __builtin_amdgcn_s_sleep(2);
        if (wall_clock64() - t0 > kSpinTimeoutTicks) return false;
    }
    return true;
}

__device__ __forceinline__ void unpack8(const u32x4 v, float (&f)[8]) {
#pragma unroll
    for (int w = 0; w < 4; ++w) {
        f[2 * w] = __uint_as_float(v[w] << 16);
        f[2 * w + 1] = __uint_as_float(v[w] & 0xffff0000u);
    }
}
__device__ __forceinline__ u32x4 pack8(const float (&f)[8]) {
    bf16x8 o;
#pragma unroll
    for (int e = 0; e < 8; ++e) o[e] = f32_to_bf16(f[e]);
    return *reinterpret_cast<u32x4*>(&o);
}

constexpr int kPF = 8;    // vectors per lane a wave may hold ahead of the hand-shake: rows of <= 64 * 8 * 8 = 4096 bf16

// A wavefront finishes one row whose reduced value it holds as vectors s[0..nv) (lane-strided: vector lane + 64*i).
// Plain: store.  Fused: h = bf16(x + s) -> out, y = rmsnorm(h) * w -> out_y.  poisoned: NaN everywhere.
// PF (rows of <= 4096 elements): the RMSNorm weights are already in registers (`wpf`, loaded once per wave BEFORE the
// hand-shake), and for the wave's first row so is the residual row (`xpf`, when x_ready).
template <bool FUSED, bool PF>
__device__ __forceinline__ void finish_row(const ArArgs& a, int row, int lane, int nvec_row, u32x4 (&s)[kMaxVecPerLane],
                                           bool poisoned, const u32x4 (&wpf)[kPF], const u32x4 (&xpf)[kPF], bool x_ready) {
    const size_t base = (size_t)row * a.row_vecs;
    u32x4* o = reinterpret_cast<u32x4*>(a.out) + base;
    if (poisoned) {
        const u32x4 nan = {0x7fc07fc0u, 0x7fc07fc0u, 0x7fc07fc0u, 0x7fc07fc0u};
        for (int i = 0; lane + 64 * i < nvec_row; ++i) {
            o[lane + 64 * i] = nan;
            if constexpr (FUSED) (reinterpret_cast<u32x4*>(a.out_y) + base)[lane + 64 * i] = nan;
        }
        return;
    }
    constexpr int NV = PF ? kPF : kMaxVecPerLane;
    if constexpr (!FUSED) {
#pragma unroll
        for (int i = 0; i < NV; ++i)
            if (lane + 64 * i < nvec_row) o[lane + 64 * i] = s[i];
    } else {
        const u32x4* x = reinterpret_cast<const u32x4*>(a.resid) + base;
        u32x4 xv[NV];
        if (PF && x_ready) {                                       // wave-uniform
#pragma unroll
            for (int i = 0; i < NV; ++i) xv[i] = xpf[i < kPF ? i : 0];
        } else {
#pragma unroll
            for (int i = 0; i < NV; ++i)
                if (lane + 64 * i < nvec_row) xv[i] = x[lane + 64 * i];
        }
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            if (lane + 64 * i < nvec_row) {
                float fs[8], fx[8], fh[8];
                unpack8(s[i], fs);
                unpack8(xv[i], fx);
#pragma unroll
                for (int e = 0; e < 8; ++e) fh[e] = bf16_to_f32(f32_to_bf16(fx[e] + fs[e]));   // h = x + y in bf16
                s[i] = pack8(fh);
                o[lane + 64 * i] = s[i];
#pragma unroll
                for (int e = 0; e < 8; ++e) ss += fh[e] * fh[e];
            }
        }
        ss = wave_reduce_sum(ss);
        const float rstd = rsqrtf(ss / (float)(a.row_vecs * 8) + a.eps);
        const u32x4* w = reinterpret_cast<const u32x4*>(a.weight);
        u32x4* y = reinterpret_cast<u32x4*>(a.out_y) + base;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            if (lane + 64 * i < nvec_row) {
                float fh[8], fw[8], fy[8];
                unpack8(s[i], fh);
                unpack8(PF ? wpf[i < kPF ? i : 0] : w[lane + 64 * i], fw);
#pragma unroll
                for (int e = 0; e < 8; ++e) fy[e] = bf16_to_f32(f32_to_bf16(fh[e] * rstd)) * fw[e];   // (x*rstd).type_as(x) * w
                y[lane + 64 * i] = pack8(fy);
            }
        }
    }
}

// PF: rows of <= 4096 elements (every plain call: 512 vectors per row; the fused rows of the 1B / 8B / 32B models).
// Everything a wave needs for its FIRST row that does not come from a peer -- its own partial, the residual row, the norm
// weights -- is requested BEFORE the block waits for the call counter and for the peers' flags, so those round trips
// overlap instead of queueing behind each other (round 5: 9.3 -> see tools/ar_bench.py).
template <int NR, bool TWOSHOT, bool FUSED, bool PF>
__global__ __launch_bounds__(kThreads) void allreduce_kernel(const ArDev c, const ArArgs a) {
    const int b = blockIdx.x, G = gridDim.x, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    __shared__ uint32_t s_k;
    __shared__ int s_bad;
    Signal* self = c.sig[c.rank];

    // rows of this block: row -> owner = row % NR, idx = row / NR, block = idx % G
    auto row_vecs_of = [&](int row) -> int {
        const size_t v0 = (size_t)row * a.row_vecs;
        const size_t left = a.n_vec - v0;
        return left < (size_t)a.row_vecs ? (int)left : a.row_vecs;
    };

    // the wave's first row (one-shot: rows of the block dealt to the 8 waves; two-shot: the rows this rank owns)
    int row0;
    bool have0;
    if constexpr (!TWOSHOT) {
        const int idx0 = b + (wave / NR) * G;
        row0 = idx0 * NR + wave % NR;
        have0 = idx0 * NR < a.rows && row0 < a.rows;
    } else {
        row0 = (b + wave * G) * NR + c.rank;
        have0 = row0 < a.rows;
    }
    u32x4 own0[kPF], x0[kPF], wpf[kPF];
    if constexpr (PF) {
        const int nv0 = have0 ? row_vecs_of(row0) : 0;
        const size_t base0 = (size_t)row0 * a.row_vecs;
#pragma unroll
        for (int i = 0; i < kPF; ++i) {
            if (lane + 64 * i < nv0) {
                own0[i] = reinterpret_cast<const u32x4*>(a.in)[base0 + lane + 64 * i];
                if constexpr (FUSED) x0[i] = reinterpret_cast<const u32x4*>(a.resid)[base0 + lane + 64 * i];
            }
            if constexpr (FUSED)
                if (lane + 64 * i < a.row_vecs) wpf[i] = reinterpret_cast<const u32x4*>(a.weight)[lane + 64 * i];
        }
    }
    if (tid == 0) {
        // BEHIND the wave's prefetch in program order, so that the two round trips overlap.  A plain (cacheable) load:
        // nobody writes the counter while a block of this call may still read it (that is the protocol), and the
        // previous call's store is behind a kernel boundary
        s_k = c.ctrl[0] + 1;
        s_bad = 0;
    }
    __syncthreads();
    const uint32_t k = s_k;
    const size_t half = (k & 1u) ? c.buf_elems : 0;
    // This block has read the counter: count it.  The ticket is drawn by lane 0 of the LAST wave -- at once if that wave has
    // no row in this call (the usual case: a block's rows go to its first waves), so that the atomic's round trip costs
    // nobody anything; after its rows otherwise.  The result is used at the very end of the kernel only.
    const bool drawer = tid == kThreads - 64;
    const bool draw_early = !have0;                  // wave-uniform
    uint32_t drawn = 0;
    if (drawer && draw_early)
        drawn = __hip_atomic_fetch_add(&c.ctrl[1], 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);

    // 1. publish: copy every row of block b into my data buffer, write-through (a lone rank has nobody to publish to)
    if constexpr (NR > 1) {
        bf16_t* mine = c.data[c.rank] + half;
        const u32x4* src = reinterpret_cast<const u32x4*>(a.in);
        for (int idx = b; idx * NR < a.rows; idx += G) {
            const int r0 = idx * NR;
            const int r1 = r0 + NR < a.rows ? r0 + NR : a.rows;            // NR consecutive rows (one per owner)
            const size_t v0 = (size_t)r0 * a.row_vecs;
            size_t v1 = (size_t)r1 * a.row_vecs;
            if (v1 > a.n_vec) v1 = a.n_vec;
            for (size_t i = v0 + tid; i < v1; i += kThreads) store_wt(mine, i, src[i]);
        }
        drain_stores();                             // every wave: its copies are in memory before the flag is raised
        __syncthreads();
        // 2. first hop
        if (tid < NR) {
            if (c.publish_fence) release_fence_system();
            __hip_atomic_store(&c.sig[tid]->start[b][c.rank], k, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_SYSTEM);
            if (!spin_ge(&self->start[b][tid], k)) s_bad = 1;
        }
        __syncthreads();
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "");   // every wave, once: no stale peer data from two calls ago
    }
    bool bad = s_bad != 0;

    // my own partial is read where it is (`in`, L2-hot), the peers' from their registered buffers
    const u32x4* peer[NR];
#pragma unroll
    for (int r = 0; r < NR; ++r) peer[r] = reinterpret_cast<const u32x4*>(c.data[r] + half);
    peer[c.rank] = reinterpret_cast<const u32x4*>(a.in);

    constexpr int NV = PF ? kPF : kMaxVecPerLane;
    // sum of one row over the ranks, in rank order, fp32 accumulate, one rounding (own_ready: this rank's vectors of the
    // row are already in own0)
    auto reduce_row = [&](int row, int nv, u32x4 (&s)[kMaxVecPerLane], bool own_ready) {
        const size_t base = (size_t)row * a.row_vecs;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            if (lane + 64 * i < nv) {
                float acc[8];
#pragma unroll
                for (int e = 0; e < 8; ++e) acc[e] = 0.f;
#pragma unroll
                for (int r = 0; r < NR; ++r) {
                    float f[8];
                    u32x4 v;
                    if (r == c.rank)
                        v = (PF && own_ready) ? own0[i < kPF ? i : 0] : peer[r][base + lane + 64 * i];
                    else
                        v = __builtin_nontemporal_load(peer[r] + base + lane + 64 * i);
                    unpack8(v, f);
#pragma unroll
                    for (int e = 0; e < 8; ++e) acc[e] += f[e];
                }
                s[i] = pack8(acc);
            }
        }
    };

    if constexpr (!TWOSHOT) {
        // 3. every rank sums every row of block b itself (rows of the block dealt to the 8 waves)
        for (int t = wave;; t += kThreads / 64) {
            const int idx = b + (t / NR) * G, row = idx * NR + t % NR;
            if (idx * NR >= a.rows) break;
            if (row >= a.rows) continue;
            const int nv = row_vecs_of(row);
            const bool first = t == wave;
            u32x4 s[kMaxVecPerLane];
            if (!bad) reduce_row(row, nv, s, first);
            finish_row<FUSED, PF>(a, row, lane, nv, s, bad, wpf, x0, first);
        }
    } else {
        // 3a. reduce-scatter: my rows of block b -> my result buffer (+ finished locally)
        bf16_t* myres = c.data[c.rank] + 2 * c.buf_elems + half;
        for (int idx = b + wave * G; idx * NR + c.rank < a.rows; idx += G * (kThreads / 64)) {
            const int row = idx * NR + c.rank;
            const int nv = row_vecs_of(row);
            const bool first = idx == b + wave * G;
            u32x4 s[kMaxVecPerLane];
            if (!bad) {
                reduce_row(row, nv, s, first);
            } else {
                // a peer's partial never arrived: the rows this rank owns are NaN for EVERYONE -- the peers gather
                // them from `myres` in step 3c, and must not find the rows of two calls ago there
                const u32x4 nan = {0x7fc07fc0u, 0x7fc07fc0u, 0x7fc07fc0u, 0x7fc07fc0u};
#pragma unroll
                for (int i = 0; i < NV; ++i) s[i] = nan;
            }
            {
                const size_t base = (size_t)row * a.row_vecs;
#pragma unroll
                for (int i = 0; i < NV; ++i)
                    if (lane + 64 * i < nv) store_wt(myres, base + lane + 64 * i, s[i]);
            }
            finish_row<FUSED, PF>(a, row, lane, nv, s, bad, wpf, x0, first);
        }
        drain_stores();
        __syncthreads();
        // 3b. second hop
        if (tid < NR) {
            if (c.publish_fence) release_fence_system();
            __hip_atomic_store(&c.sig[tid]->start2[b][c.rank], k, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_SYSTEM);
            if (!spin_ge(&self->start2[b][tid], k)) s_bad = 1;
        }
        __syncthreads();
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "");
        bad = s_bad != 0;
        // 3c. all-gather: the other owners' rows of block b from their result buffers
        for (int t = wave;; t += kThreads / 64) {
            const int idx = b + (t / NR) * G, o = t % NR, row = idx * NR + o;
            if (idx * NR >= a.rows) break;
            if (row >= a.rows || o == c.rank) continue;
            const int nv = row_vecs_of(row);
            const u32x4* src = reinterpret_cast<const u32x4*>(c.data[o] + 2 * c.buf_elems + half) +
                               (size_t)row * a.row_vecs;
            u32x4 s[kMaxVecPerLane];
            if (!bad) {
#pragma unroll
                for (int i = 0; i < NV; ++i)
                    if (lane + 64 * i < nv) s[i] = __builtin_nontemporal_load(src + lane + 64 * i);
            }
            finish_row<FUSED, PF>(a, row, lane, nv, s, bad, wpf, x0, false);
        }
    }

    // the block that drew the last ticket hands the call counter on (every block of this call has read it; the next
    // launch on the stream reads it behind a kernel boundary); `status` is read by the host behind one, too
    if (drawer && !draw_early)
        drawn = __hip_atomic_fetch_add(&c.ctrl[1], 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    if (drawer && drawn == (uint32_t)G - 1) {
        __hip_atomic_store(&c.ctrl[1], 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        __hip_atomic_store(&c.ctrl[0], k, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    if (tid == 0 && (bad || s_bad)) self->status = 1;
}

}  // namespace

struct md_ar_comm {
    ArDev dev;
    void* my_data;
    void* my_sig;
    void* my_ctrl;
    void* opened[2 * kMaxRanks];
    int n_opened;
    size_t max_bytes;
};

extern "C" int md_ar_create(int rank, int world, size_t max_bytes, md_ar_comm** comm_out) {
    MD_CHECK_ARG(comm_out && world >= 1 && world <= kMaxRanks && rank >= 0 && rank < world,
                 "md_ar_create: need 1 <= world <= %d and 0 <= rank < world", kMaxRanks);
    MD_CHECK_ARG(max_bytes >= 16 && max_bytes % 16 == 0, "md_ar_create: max_bytes must be a positive multiple of 16");
    md_ar_comm* c = new md_ar_comm();
    c->n_opened = 0;
    c->max_bytes = max_bytes;
    // one registered allocation: data halves 0/1 (published partials), result halves 0/1 (two-shot reduced rows)
    c->my_data = c->my_sig = c->my_ctrl = nullptr;
    if (hipMalloc(&c->my_data, 4 * max_bytes) != hipSuccess || hipMalloc(&c->my_ctrl, 256) != hipSuccess ||
        hipExtMallocWithFlags(&c->my_sig, sizeof(Signal), hipDeviceMallocUncached) != hipSuccess) {
        md_set_error("md_ar_create: device allocation failed: %s", hipGetErrorString(hipGetLastError()));
        delete c;
        return MD_ERR_WORKSPACE;
    }
    if (hipMemset(c->my_sig, 0, sizeof(Signal)) != hipSuccess || hipMemset(c->my_data, 0, 4 * max_bytes) != hipSuccess ||
        hipMemset(c->my_ctrl, 0, 256) != hipSuccess || hipDeviceSynchronize() != hipSuccess) {
        md_set_error("md_ar_create: clearing the buffers failed: %s", hipGetErrorString(hipGetLastError()));
        (void)hipFree(c->my_data);
        (void)hipFree(c->my_sig);
        (void)hipFree(c->my_ctrl);
        delete c;
        return MD_ERR_WORKSPACE;
    }
    for (int r = 0; r < kMaxRanks; ++r) {
        c->dev.data[r] = nullptr;
        c->dev.sig[r] = nullptr;
    }
    c->dev.rank = rank;
    c->dev.world = world;
    c->dev.buf_elems = max_bytes / 2;
    c->dev.publish_fence = 0;
    c->dev.data[rank] = (bf16_t*)c->my_data;
    c->dev.sig[rank] = (Signal*)c->my_sig;
    c->dev.ctrl = (uint32_t*)c->my_ctrl;
    *comm_out = c;
    return MD_OK;
}

extern "C" int md_ar_get_handles(md_ar_comm* c, void* handles_host) {
    MD_CHECK_ARG(c && handles_host, "md_ar_get_handles: null argument");
    static_assert(sizeof(hipIpcMemHandle_t) == MD_AR_HANDLE_BYTES, "IPC handle size");
    hipIpcMemHandle_t* h = (hipIpcMemHandle_t*)handles_host;
    if (hipIpcGetMemHandle(&h[0], c->my_data) != hipSuccess || hipIpcGetMemHandle(&h[1], c->my_sig) != hipSuccess) {
        md_set_error("md_ar_get_handles: hipIpcGetMemHandle failed: %s (is HSA_ENABLE_IPC_MODE_LEGACY=0 set?)",
                     hipGetErrorString(hipGetLastError()));
        return MD_ERR_LAUNCH;
    }
    return MD_OK;
}

extern "C" int md_ar_open_peers(md_ar_comm* c, const void* all_handles_host) {
    MD_CHECK_ARG(c && all_handles_host, "md_ar_open_peers: null argument");
    const hipIpcMemHandle_t* h = (const hipIpcMemHandle_t*)all_handles_host;
    for (int r = 0; r < c->dev.world; ++r) {
        if (r == c->dev.rank) continue;
        void *d = nullptr, *s = nullptr;
        if (hipIpcOpenMemHandle(&d, h[2 * r], hipIpcMemLazyEnablePeerAccess) != hipSuccess ||
            hipIpcOpenMemHandle(&s, h[2 * r + 1], hipIpcMemLazyEnablePeerAccess) != hipSuccess) {
            md_set_error("md_ar_open_peers: hipIpcOpenMemHandle(rank %d) failed: %s", r,
                         hipGetErrorString(hipGetLastError()));
            return MD_ERR_LAUNCH;
        }
        c->opened[c->n_opened++] = d;
        c->opened[c->n_opened++] = s;
        c->dev.data[r] = (bf16_t*)d;
        c->dev.sig[r] = (Signal*)s;
    }
    return MD_OK;
}

namespace {

template <bool TWOSHOT, bool FUSED>
void launch_world(const md_ar_comm* c, const ArArgs& a, int grid, hipStream_t st) {
    const bool pf = a.row_vecs <= 64 * kPF;
#define MD_AR_LAUNCH(N)                                                                                         \
    case N:                                                                                                     \
        if (pf)                                                                                                 \
            hipLaunchKernelGGL((allreduce_kernel<N, TWOSHOT, FUSED, true>), dim3(grid), dim3(kThreads), 0, st, c->dev, a); \
        else                                                                                                    \
            hipLaunchKernelGGL((allreduce_kernel<N, TWOSHOT, FUSED, false>), dim3(grid), dim3(kThreads), 0, st, c->dev, a); \
        break;
    switch (c->dev.world) {
        MD_AR_LAUNCH(1)
        MD_AR_LAUNCH(2)
        MD_AR_LAUNCH(3)
        MD_AR_LAUNCH(4)
        MD_AR_LAUNCH(5)
        MD_AR_LAUNCH(6)
        MD_AR_LAUNCH(7)
        MD_AR_LAUNCH(8)
    }
#undef MD_AR_LAUNCH
}

int run(md_ar_comm* c, ArArgs a, int algo, bool fused, hipStream_t st, const char* who) {
    for (int r = 0; r < c->dev.world; ++r)
        MD_CHECK_ARG(c->dev.data[r] && c->dev.sig[r], "%s: peer %d not opened (md_ar_open_peers)", who, r);
    MD_CHECK_ARG(algo == MD_AR_ALGO_AUTO || algo == MD_AR_ALGO_ONESHOT || algo == MD_AR_ALGO_TWOSHOT,
                 "%s: unknown algorithm %d", who, algo);
    const size_t bytes = a.n_vec * 16;
    bool two = algo == MD_AR_ALGO_TWOSHOT;
    if (algo == MD_AR_ALGO_AUTO)   // one-shot pulls (N-1) x the message into every rank, two-shot 2(N-1)/N x in two hops
        two = c->dev.world >= 4 && bytes > (size_t)512 * 1024;
    if (c->dev.world == 1) two = false;
    // grid sized to the message: one block per group of N rows (a block's 8 waves take a row each), at least one
    // (block 0 carries the call-level hand-shake), at most kMaxBlocks
    const int groups = (a.rows + c->dev.world - 1) / c->dev.world;
    const int grid = groups < 1 ? 1 : (groups > kMaxBlocks ? kMaxBlocks : groups);
    if (two) {
        if (fused) launch_world<true, true>(c, a, grid, st); else launch_world<true, false>(c, a, grid, st);
    } else {
        if (fused) launch_world<false, true>(c, a, grid, st); else launch_world<false, false>(c, a, grid, st);
    }
    return MD_OK;
}

}  // namespace

extern "C" int md_allreduce(md_ar_comm* c, const void* in, void* out, size_t count, int algo, md_stream_t stream) {
    MD_CHECK_ARG(c && in && out, "md_allreduce: null argument");
    MD_CHECK_ARG(count % 8 == 0 && count * 2 <= c->max_bytes,
                 "md_allreduce: count must be a multiple of 8 bf16 and fit the registered buffer (%zu bytes)",
                 c->max_bytes);
    MD_CHECK_ARG(((uintptr_t)in | (uintptr_t)out) % 16 == 0, "md_allreduce: in/out must be 16-byte aligned");
    if (count == 0) return MD_OK;
    ArArgs a = {};
    a.in = (const bf16_t*)in;
    a.out = (bf16_t*)out;
    a.n_vec = count / 8;
    a.row_vecs = kRowVecs;
    a.rows = (int)((a.n_vec + kRowVecs - 1) / kRowVecs);
    const int rc = run(c, a, algo, false, (hipStream_t)stream, "md_allreduce");
    if (rc != MD_OK) return rc;
    MD_CHECK_LAUNCH("md_allreduce");
    return MD_OK;
}

extern "C" int md_allreduce_oneshot(md_ar_comm* c, const void* in, void* out, size_t count, md_stream_t stream) {
    return md_allreduce(c, in, out, count, MD_AR_ALGO_ONESHOT, stream);
}

extern "C" int md_allreduce_add_rmsnorm(md_ar_comm* c, const void* partial, const void* resid, const void* weight,
                                        void* out_h, void* out_y, int rows, int dim, float eps, int algo,
                                        md_stream_t stream) {
    MD_CHECK_ARG(c && partial && resid && weight && out_h && out_y, "md_allreduce_add_rmsnorm: null argument");
    MD_CHECK_ARG(rows > 0 && dim > 0 && dim % 8 == 0 && dim <= 64 * kMaxVecPerLane * 8,
                 "md_allreduce_add_rmsnorm: need rows > 0 and dim %% 8 == 0, dim <= %d", 64 * kMaxVecPerLane * 8);
    MD_CHECK_ARG((size_t)rows * dim * 2 <= c->max_bytes,
                 "md_allreduce_add_rmsnorm: message does not fit the registered buffer (%zu bytes)", c->max_bytes);
    MD_CHECK_ARG(((uintptr_t)partial | (uintptr_t)resid | (uintptr_t)weight | (uintptr_t)out_h | (uintptr_t)out_y) % 16 == 0,
                 "md_allreduce_add_rmsnorm: pointers must be 16-byte aligned");
    ArArgs a = {};
    a.in = (const bf16_t*)partial;
    a.out = (bf16_t*)out_h;
    a.resid = (const bf16_t*)resid;
    a.weight = (const bf16_t*)weight;
    a.out_y = (bf16_t*)out_y;
    a.eps = eps;
    a.rows = rows;
    a.row_vecs = dim / 8;
    a.n_vec = (size_t)rows * (dim / 8);
    const int rc = run(c, a, algo, true, (hipStream_t)stream, "md_allreduce_add_rmsnorm");
    if (rc != MD_OK) return rc;
    MD_CHECK_LAUNCH("md_allreduce_add_rmsnorm");
    return MD_OK;
}

extern "C" int md_ar_set_publish(md_ar_comm* c, int mode) {
    MD_CHECK_ARG(c, "md_ar_set_publish: null communicator");
    MD_CHECK_ARG(mode == MD_AR_PUBLISH_WRITE_THROUGH || mode == MD_AR_PUBLISH_FENCE,
                 "md_ar_set_publish: mode must be MD_AR_PUBLISH_WRITE_THROUGH (0) or MD_AR_PUBLISH_FENCE (1), got %d", mode);
    c->dev.publish_fence = mode == MD_AR_PUBLISH_FENCE ? 1 : 0;     // read by the next launch (passed by value)
    return MD_OK;
}

extern "C" int md_ar_status(md_ar_comm* c, int* status_host) {
    MD_CHECK_ARG(c && status_host, "md_ar_status: null argument");
    uint32_t s = 0;
    if (hipMemcpy(&s, &((Signal*)c->my_sig)->status, sizeof(s), hipMemcpyDeviceToHost) != hipSuccess) {
        md_set_error("md_ar_status: copy failed: %s", hipGetErrorString(hipGetLastError()));
        return MD_ERR_LAUNCH;
    }
    *status_host = (int)s;
    return MD_OK;
}

extern "C" int md_ar_status_async(md_ar_comm* c, int* status_host_pinned, md_stream_t stream) {
    MD_CHECK_ARG(c && status_host_pinned, "md_ar_status_async: null argument");
    if (hipMemcpyAsync(status_host_pinned, &((Signal*)c->my_sig)->status, sizeof(uint32_t), hipMemcpyDeviceToHost,
                       (hipStream_t)stream) != hipSuccess) {
        md_set_error("md_ar_status_async: copy failed: %s", hipGetErrorString(hipGetLastError()));
        return MD_ERR_LAUNCH;
    }
    return MD_OK;
}

extern "C" int md_ar_destroy(md_ar_comm* c) {
    if (!c) return MD_OK;
    (void)hipDeviceSynchronize();
    for (int i = 0; i < c->n_opened; ++i) (void)hipIpcCloseMemHandle(c->opened[i]);
    (void)hipFree(c->my_data);
    // my_sig is uncached device memory that kernels have read: it stays allocated until the process ends (allocations made
    // after such a free have been seen to hold wrong values)
    (void)hipFree(c->my_ctrl);
    delete c;
    return MD_OK;
}
