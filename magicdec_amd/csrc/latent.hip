// Latent attention (gfx950): keys and values of every head are linear maps of one small latent row per token, and one rotated
// key part is shared by all heads, so a cache row is  latent (kv_rank) | rotated key part (rot_dim) | zeros up to W.
//   score(t, s, h) = (qn_th . K_h c_s + rot(qr_th) . r_s) * scale,   o_th = sum_s p_ts (V_h c_s)
// Two forms of the same sums:
//   absorbed   K_h moves to the query, V_h behind the sum: scores are (K_h^T qn | rot(qr)) . (c | r), one query of W numbers per
//              (token, head) against rows every head shares -- a multi-query attention whose value row is a prefix of its key row.
//              A cached row is read once for all heads: decoding.
//   expanded   keys and values of the context are computed (one library product over the gathered latents) and attended per
//              head with dim + rot_dim and vdim numbers: several times fewer operations per (query, key): prompts.
//
//   md_latent_append     query latent -> weighted RMS norm; latent -> weighted RMS norm, key part -> rotation, both -> cache
//   md_head_linear       y[row][h] = W_h x[row][h]: the absorbed queries (+ their rotated part) and the way out of the latent
//                        (* sigmoid of the head's gate)
//   md_latent_attn       the absorbed form over the cache; 32-bit and unusual sizes run the plain attention kernel of xattn.hip
//   md_latent_gather     latents of a paged context as dense rows
//   md_latent_prefill    the expanded form
// Positions, angles, norms, scores, softmax weights and gates are fp32.
#include "latent.h"
#include "xattn.h"

unsigned int* md_page_overflow_counter_device();   // kvops.hip

namespace {

constexpr int kMaxRow = 1024;

// ------------------------------------------------------------------------------------------------ norms, rotation, append
template <typename T, int VEC>
__device__ __forceinline__ void ld_piece(const T* p, float (&f)[VEC]) {
    typedef T vec __attribute__((ext_vector_type(VEC)));
    if constexpr (VEC == 1) {
        f[0] = (float)p[0];
    } else {
        const vec v = *reinterpret_cast<const vec*>(p);
#pragma unroll
        for (int e = 0; e < VEC; ++e) f[e] = (float)v[e];
    }
}
template <typename T, int VEC>
__device__ __forceinline__ void st_piece(T* p, const float (&f)[VEC]) {
    typedef T vec __attribute__((ext_vector_type(VEC)));
    if constexpr (VEC == 1) {
        p[0] = (T)f[0];
    } else {
        vec v;
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] = (T)f[e];
        *reinterpret_cast<vec*>(p) = v;
    }
}

// dst = src / sqrt(mean(src^2) + eps) * w by one wavefront
template <typename T, int VEC>
__device__ __forceinline__ void norm_row(const T* src, const T* w, T* dst, int n, float eps, int lane) {
    float ss = 0.f, f[VEC], g[VEC];
    for (int d = lane * VEC; d < n; d += 64 * VEC) {
        ld_piece<T, VEC>(src + d, f);
#pragma unroll
        for (int e = 0; e < VEC; ++e) ss += f[e] * f[e];
    }
    const float rs = 1.0f / sqrtf(wave_reduce_sum(ss) / (float)n + eps);
    for (int d = lane * VEC; d < n; d += 64 * VEC) {
        ld_piece<T, VEC>(src + d, f);
        ld_piece<T, VEC>(w + d, g);
#pragma unroll
        for (int e = 0; e < VEC; ++e) f[e] = (f[e] * rs) * g[e];
        st_piece<T, VEC>(dst + d, f);
    }
}

// element d of a rotated vector (neighbouring pairs of the first 2 * pairs elements turn, the rest pass)
template <typename T>
__device__ __forceinline__ float rotated(const T* x, int d, int pairs, const float* cs) {
    const float a = (float)x[d];
    if (d >= 2 * pairs) return a;
    const float b = (float)x[d ^ 1], c = cs[d & ~1], s = cs[d | 1];      // cs = (cos, sin) of every pair
    return d & 1 ? a * c + b * s : a * c - b * s;
}

// two wavefronts per row: one normalises the query latent, the other the latent and rotates the key part
template <typename T, int VEC>
__global__ __launch_bounds__(256) void latent_append_kernel(const LatentParams p) {
    const int b = blockIdx.y, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int q0 = p.qo_indptr[b], j = blockIdx.x * 2 + (wave >> 1);
    if (j >= p.qo_indptr[b + 1] - q0) return;
    const T* row = reinterpret_cast<const T*>(p.z) + (int64_t)(q0 + j) * p.ldz;
    if ((wave & 1) == 0) {
        norm_row<T, VEC>(row, reinterpret_cast<const T*>(p.dq_norm), reinterpret_cast<T*>(p.cq) + (int64_t)(q0 + j) * p.q_rank,
                         p.q_rank, p.eps, lane);
        return;
    }
    if (!p.append) return;
    const int pos = p.pos0[b] + j, pg0 = p.page_indptr[b];
    if (pos < 0 || pos >= (p.page_indptr[b + 1] - pg0) * p.page_size || pos >= p.max_pos) {
        if (lane == 0) atomicAdd(p.overflow, 1u);
        return;
    }
    T* dst = reinterpret_cast<T*>(p.cache) +
             ((int64_t)p.page_indices[pg0 + pos / p.page_size] * p.page_size + pos % p.page_size) * p.W;
    const T* src = row + p.q_rank;
    norm_row<T, VEC>(src, reinterpret_cast<const T*>(p.kv_norm), dst, p.kv_rank, p.eps, lane);
    const float* cs = p.cos_sin + (int64_t)pos * p.rot_pairs * 2;
    for (int d = lane; d < p.W - p.kv_rank; d += 64)
        dst[p.kv_rank + d] = d < p.rot_dim ? (T)rotated(src + p.kv_rank, d, p.rot_pairs, cs) : (T)0.f;
}

// ------------------------------------------------------------------------------------------------ per-head linear
struct HeadLinearParams {
    const void* x;
    const void* w;            // [H][N][K]
    void* out;
    const void* gate;         // [M][ld_gate] or null: y *= sigmoid(gate[row][h])
    // a rotated tail behind the N outputs of a head: out[row][h][N + d] = rotated(tail[row][h])[d], zeros up to tail_pad
    const void* tail;
    const float* cos_sin;
    const int32_t* qo_indptr;
    const int32_t* pos0;
    int64_t ldx, hx, ldo, ho, ld_gate, ldt, ht;
    int M, H, N, K, B, tail_dim, tail_pad, rot_pairs, max_pos;
};

__device__ __forceinline__ float sigmoid(float v) { return 1.0f / (1.0f + expf(-v)); }

template <typename T>
__device__ __forceinline__ void head_tail(const HeadLinearParams& p, int h, int row0, int nrow) {
    // the column blocks of a row tile share its tail: this block's rows are row0 + blockIdx.x, + gridDim.x, ...
    __shared__ int s_pos[64];
    if (threadIdx.x < nrow) {
        const int row = min(row0 + (int)threadIdx.x, p.M - 1);
        int lo = 0, hi = p.B;                                       // request of the row: qo_indptr[lo] <= row < qo_indptr[lo + 1]
        while (hi - lo > 1) {
            const int mid = (lo + hi) >> 1;
            if (p.qo_indptr[mid] <= row) lo = mid; else hi = mid;
        }
        s_pos[threadIdx.x] = min(max(p.pos0[lo] + row - p.qo_indptr[lo], 0), p.max_pos - 1);
    }
    __syncthreads();
    const int mine = (nrow - (int)blockIdx.x + (int)gridDim.x - 1) / (int)gridDim.x;
    for (int i = threadIdx.x; i < mine * p.tail_pad; i += 256) {
        const int r = blockIdx.x + i / p.tail_pad * gridDim.x, d = i % p.tail_pad, row = row0 + r;
        if (row >= p.M) break;
        const float v = d < p.tail_dim ? rotated(reinterpret_cast<const T*>(p.tail) + row * p.ldt + h * p.ht, d, p.rot_pairs,
                                                 p.cos_sin + (int64_t)s_pos[r] * p.rot_pairs * 2) : 0.f;
        (reinterpret_cast<T*>(p.out) + row * p.ldo + h * p.ho)[p.N + d] = (T)v;
    }
}

// 16-bit: 64 columns x 16 RT rows of one head per workgroup, 16 columns per wavefront, operands straight from memory
template <int RT, bool VEC>
__global__ __launch_bounds__(256) void head_linear_mfma_kernel(const HeadLinearParams p) {
    const int lane = threadIdx.x & 63, lq = lane & 15, lc = lane >> 4, wave = threadIdx.x >> 6;
    const int h = blockIdx.z, row0 = blockIdx.y * 16 * RT, n0 = blockIdx.x * 64 + wave * 16;
    if (p.tail) head_tail<bf16_t>(p, h, row0, 16 * RT);
    const bf16x8 z8 = {0, 0, 0, 0, 0, 0, 0, 0};
    auto piece = [&](const bf16_t* src, int k, bool ok) {
        if (VEC) return ok && k < p.K ? *reinterpret_cast<const bf16x8*>(src + k) : z8;
        bf16x8 v = z8;
#pragma unroll
        for (int e = 0; e < 8; ++e)
            if (ok && k + e < p.K) v[e] = src[k + e];
        return v;
    };
    if (n0 < p.N) {
        const int n = n0 + lq;
        const bool n_ok = n < p.N;
        const bf16_t* wp = reinterpret_cast<const bf16_t*>(p.w) + ((int64_t)h * p.N + (n_ok ? n : 0)) * p.K;
        const bf16_t* xp[RT];
        bool r_ok[RT];
        f32x4 acc[RT];
#pragma unroll
        for (int r = 0; r < RT; ++r) {
            const int row = row0 + r * 16 + lq;
            r_ok[r] = row < p.M;
            xp[r] = reinterpret_cast<const bf16_t*>(p.x) + (int64_t)(r_ok[r] ? row : 0) * p.ldx + h * p.hx;
            acc[r] = f32x4{0.f, 0.f, 0.f, 0.f};
        }
        for (int kb = 0; kb < p.K; kb += 128) {                     // four steps requested together (zeros past K)
            bf16x8 wf[4], xf[4][RT];
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                wf[u] = piece(wp, kb + u * 32 + lc * 8, n_ok);
#pragma unroll
                for (int r = 0; r < RT; ++r) xf[u][r] = piece(xp[r], kb + u * 32 + lc * 8, r_ok[r]);
            }
#pragma unroll
            for (int u = 0; u < 4; ++u)
#pragma unroll
                for (int r = 0; r < RT; ++r) acc[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[u], xf[u][r], acc[r], 0, 0, 0);
        }
        // acc[r][e] = y[row0 + r * 16 + lq][n0 + lc * 4 + e]
#pragma unroll
        for (int r = 0; r < RT; ++r) {
            const int row = row0 + r * 16 + lq, c = n0 + lc * 4;
            if (row >= p.M) continue;
            const float s = p.gate ? sigmoid((float)reinterpret_cast<const bf16_t*>(p.gate)[row * p.ld_gate + h]) : 1.f;
            bf16_t* o = reinterpret_cast<bf16_t*>(p.out) + row * p.ldo + h * p.ho + c;
            if (VEC && c + 4 <= p.N) {
                *reinterpret_cast<bf16x4*>(o) = __builtin_convertvector(acc[r] * s, bf16x4);
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (c + e < p.N) o[e] = (bf16_t)(acc[r][e] * s);
            }
        }
    }
}

// 32-bit: a thread per output
__global__ __launch_bounds__(256) void head_linear_f32_kernel(const HeadLinearParams p) {
    const int h = blockIdx.z, row0 = blockIdx.y * 16, n = blockIdx.x * 16 + (threadIdx.x & 15), row = row0 + (threadIdx.x >> 4);
    if (n < p.N && row < p.M) {
        const float* w = reinterpret_cast<const float*>(p.w) + ((int64_t)h * p.N + n) * p.K;
        const float* x = reinterpret_cast<const float*>(p.x) + (int64_t)row * p.ldx + h * p.hx;
        float s = 0.f;
        for (int k = 0; k < p.K; ++k) s = fmaf(w[k], x[k], s);
        if (p.gate) s *= sigmoid(reinterpret_cast<const float*>(p.gate)[row * p.ld_gate + h]);
        (reinterpret_cast<float*>(p.out) + row * p.ldo + h * p.ho)[n] = s;
    }
    if (p.tail) head_tail<float>(p, h, row0, 16);
}

// ------------------------------------------------------------------------------------------------ merge, gather
// partials of the kv splits: ws = sums [slot][rows_wg][Rp], then (reference, weight) [slot][rows_wg][2]; slot =
// (b * groups + g) * nsplit + s.  Lane s knows split s's factor; Q wavefronts share 256 columns of one row, each adds every Q-th split
// (four requested together), and their sums meet in LDS in order
template <int Q>
__global__ __launch_bounds__(256) void latent_merge_kernel(const LatentParams p, int rows_wg, int Rp) {
    __shared__ f32x4 part[4][64];
    const int lane = threadIdx.x & 63, all = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), wave = Q == 4 ? all : 0;
    const int b = blockIdx.z, row = Q == 4 ? blockIdx.x : blockIdx.x * 4 + all, q0 = p.qo_indptr[b];
    if (row >= (p.qo_indptr[b + 1] - q0) * p.H) return;               // (Q == 4: whole workgroup)
    const int g = row / rows_wg, r = row - g * rows_wg, d = (blockIdx.y * 64 + lane) * 4;
    const int64_t slot0 = ((int64_t)b * p.n_groups + g) * p.nsplit;
    const float* ml = p.ws + (int64_t)p.B * p.n_groups * p.nsplit * rows_wg * Rp;
    f32x2 t = {-INFINITY, 0.f};
    if (lane < p.nsplit) t = *reinterpret_cast<const f32x2*>(ml + ((slot0 + lane) * rows_wg + r) * 2);
    const float m = wave_reduce_max(t[0]), w = t[0] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(t[0] - m);
    const float l = wave_reduce_sum(t[1] * w);
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
    for (int s0 = wave; s0 < p.nsplit; s0 += 4 * Q) {
        f32x4 v[4];
#pragma unroll
        for (int u = 0; u < 4; ++u)
            if (s0 + Q * u < p.nsplit && d < Rp) v[u] = *reinterpret_cast<const f32x4*>(p.ws + ((slot0 + s0 + Q * u) * rows_wg + r) * Rp + d);
#pragma unroll
        for (int u = 0; u < 4; ++u)
            if (s0 + Q * u < p.nsplit) {                              // uniform
                const float f = __shfl(w, s0 + Q * u);
                if (d < Rp) o += v[u] * f;
            }
    }
    if constexpr (Q == 4) {
        part[wave][lane] = o;
        __syncthreads();
        if (wave > 0) return;
        o = (part[0][lane] + part[1][lane]) + (part[2][lane] + part[3][lane]);
    }
    if (d >= Rp) return;
    const float inv = l > 0.f ? 1.0f / l : 0.f;
    bf16_t* op = reinterpret_cast<bf16_t*>(p.out) + ((int64_t)q0 * p.H + row) * p.kv_rank + d;
    if (p.kv_rank % 4 == 0) {
        if (d < p.kv_rank) *reinterpret_cast<bf16x4*>(op) = __builtin_convertvector(o * inv, bf16x4);
    } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (d + e < p.kv_rank) op[e] = (bf16_t)(o[e] * inv);
    }
}

// one wavefront per context row
__global__ __launch_bounds__(256) void latent_gather_kernel(const LatentParams p, bf16_t* __restrict__ dst) {
    const int b = blockIdx.y, pos = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    const int c0 = p.ctx_indptr[b];
    if (pos >= p.ctx_indptr[b + 1] - c0) return;
    const int pg0 = p.page_indptr[b];
    const bool fits = pos < (p.page_indptr[b + 1] - pg0) * p.page_size;
    const bf16_t* src = reinterpret_cast<const bf16_t*>(p.cache) +
                        (fits ? ((int64_t)p.page_indices[pg0 + pos / p.page_size] * p.page_size + pos % p.page_size) * p.W : 0);
    const u32x4 z = {0u, 0u, 0u, 0u};
    for (int d = lane * 8; d < p.kv_rank; d += 512)
        *reinterpret_cast<u32x4*>(dst + (int64_t)(c0 + pos) * p.kv_rank + d) = fits ? *reinterpret_cast<const u32x4*>(src + d) : z;
}

bool aligned(const void* q, int n) { return ((uintptr_t)q & (n - 1)) == 0; }
int row_width(int kv_rank, int rot_dim) { return (kv_rank + rot_dim + 31) / 32 * 32; }
int row_tiles(const md_latent_args* a) { return (long)a->n_max * a->H <= 16 ? 1 : 2; }
int row_groups(const md_latent_args* a) { return (int)(((long)a->n_max * a->H + 16 * row_tiles(a) - 1) / (16 * row_tiles(a))); }

bool mfma_ok(const md_latent_args* a) {
    return a->dtype == MD_T_BF16 && !a->force_plain && a->page_size % 64 == 0 &&
           md_internal_latent_absorbed_ok(a->kv_rank, row_width(a->kv_rank, a->rot_dim), row_tiles(a));
}

constexpr int kTargetWgs = 512;              // 16-row workgroups: two per CU (of 32 rows: one)

int kv_splits(const md_latent_args* a) {
    const long tiles = ((long)a->max_pages * a->page_size + 31) / 32, groups = (long)a->B * row_groups(a);
    const long target = kTargetWgs / row_tiles(a);
    long want = (target + groups - 1) / groups;
    const long cap = tiles / 8 > 1 ? tiles / 8 : 1;                  // >= 256 keys per workgroup
    if (want > cap) want = cap;
    return (int)(want < 1 ? 1 : want > 64 ? 64 : want);            // (the merge holds a split per lane)
}

int check_args(const char* who, const md_latent_args* a) {
    MD_CHECK_ARG(a && a->cache && a->qo_indptr && a->pos0 && a->page_indices && a->page_indptr, "%s: null pointer argument", who);
    MD_CHECK_ARG(a->B > 0 && a->B <= 65535 && a->n_max > 0 && a->H > 0 && a->H <= 65535, "%s: bad shape B=%d n_max=%d H=%d", who,
                 a->B, a->n_max, a->H);
    MD_CHECK_ARG(a->kv_rank > 0 && a->rot_dim > 0 && a->rot_pairs >= 0 && 2 * a->rot_pairs <= a->rot_dim &&
                     row_width(a->kv_rank, a->rot_dim) <= kMaxRow, "%s: kv_rank %d + rot_dim %d (<= %d)", who, a->kv_rank,
                 a->rot_dim, kMaxRow);
    MD_CHECK_ARG(a->page_size > 0 && a->page_size % 32 == 0 && a->max_pages > 0, "%s: page_size %d must be a multiple of 32", who,
                 a->page_size);
    MD_CHECK_ARG(a->dtype == MD_T_BF16 || a->dtype == MD_T_F32, "%s: dtype must be MD_T_BF16 or MD_T_F32", who);
    MD_CHECK_ARG(aligned(a->cache, 16), "%s: the cache must be 16-byte aligned", who);
    return MD_OK;
}

LatentParams make_params(const md_latent_args* a) {
    LatentParams p = {};
    p.z = a->z;
    p.dq_norm = a->dq_norm;
    p.kv_norm = a->kv_norm;
    p.cq = a->cq;
    p.cache = a->cache;
    p.cos_sin = a->cos_sin;
    p.qo_indptr = a->qo_indptr;
    p.pos0 = a->pos0;
    p.page_indices = a->page_indices;
    p.page_indptr = a->page_indptr;
    p.ctx_indptr = a->ctx_indptr;
    p.q = a->q;
    p.kv = a->kv;
    p.gate = a->gate;
    p.out = a->out;
    p.ldz = a->ldz;
    p.ldo = a->ldo;
    p.ld_gate = a->ld_gate;
    p.B = a->B;
    p.n_max = a->n_max;
    p.H = a->H;
    p.dim = a->dim;
    p.rot_dim = a->rot_dim;
    p.rot_pairs = a->rot_pairs;
    p.vdim = a->vdim;
    p.q_rank = a->q_rank;
    p.kv_rank = a->kv_rank;
    p.W = row_width(a->kv_rank, a->rot_dim);
    p.page_size = a->page_size;
    p.max_pos = a->max_pos;
    p.append = a->append;
    p.eps = a->eps;
    p.scale_log2 = a->scale * 1.4426950408889634f;
    p.overflow = md_page_overflow_counter_device();
    return p;
}

int prefill_dk(int n) { return n <= 64 ? 64 : n <= 128 ? 128 : n <= 192 ? 192 : n <= 256 ? 256 : 0; }

}  // namespace

extern "C" int md_latent_row_width(int kv_rank, int rot_dim) {
    return kv_rank > 0 && rot_dim > 0 && row_width(kv_rank, rot_dim) <= kMaxRow ? row_width(kv_rank, rot_dim) : 0;
}

extern "C" int md_latent_append(const md_latent_args* a, md_stream_t stream) {
    const int rc = check_args("md_latent_append", a);
    if (rc != MD_OK) return rc;
    MD_CHECK_ARG(a->z && a->dq_norm && a->cq && a->q_rank > 0, "md_latent_append: null pointer argument");
    MD_CHECK_ARG(!a->append || (a->kv_norm && a->cos_sin && a->max_pos > 0), "md_latent_append: the append needs kv_norm and the angle table");
    MD_CHECK_ARG(a->ldz >= a->q_rank + (a->append ? a->kv_rank + a->rot_dim : 0), "md_latent_append: rows of %lld elements are too short",
                 (long long)a->ldz);
    const LatentParams p = make_params(a);
    MD_CHECK_ARG(p.overflow, "md_latent_append: cannot resolve the page-overflow counter");
    const dim3 grid((a->n_max + 1) / 2, a->B);
    const bool vec = a->q_rank % 8 == 0 && a->kv_rank % 8 == 0 && a->ldz % 8 == 0 && aligned(a->z, 32) && aligned(a->cq, 32) &&
                     aligned(a->cache, 32) && aligned(a->dq_norm, 32) && (!a->append || aligned(a->kv_norm, 32));
    hipStream_t st = (hipStream_t)stream;
    if (a->dtype == MD_T_F32) {
        if (vec) hipLaunchKernelGGL((latent_append_kernel<float, 8>), grid, dim3(256), 0, st, p);
        else hipLaunchKernelGGL((latent_append_kernel<float, 1>), grid, dim3(256), 0, st, p);
    } else {
        if (vec) hipLaunchKernelGGL((latent_append_kernel<bf16_t, 8>), grid, dim3(256), 0, st, p);
        else hipLaunchKernelGGL((latent_append_kernel<bf16_t, 1>), grid, dim3(256), 0, st, p);
    }
    MD_CHECK_LAUNCH("md_latent_append");
    return MD_OK;
}

extern "C" int md_head_linear(const md_head_linear_args* a, md_stream_t stream) {
    MD_CHECK_ARG(a && a->x && a->w && a->out, "md_head_linear: null pointer argument");
    MD_CHECK_ARG(a->M > 0 && a->H > 0 && a->H <= 65535 && a->N > 0 && a->K > 0, "md_head_linear: bad shape M=%d H=%d N=%d K=%d", a->M,
                 a->H, a->N, a->K);
    MD_CHECK_ARG(a->dtype == MD_T_BF16 || a->dtype == MD_T_F32, "md_head_linear: dtype must be MD_T_BF16 or MD_T_F32");
    MD_CHECK_ARG(!a->tail || (a->cos_sin && a->qo_indptr && a->pos0 && a->B > 0 && a->tail_pad >= a->tail_dim && a->tail_dim > 0 &&
                              2 * a->rot_pairs <= a->tail_dim && a->rot_pairs >= 0 && a->max_pos > 0),
                 "md_head_linear: the rotated tail needs positions and the angle table");
    HeadLinearParams p = {};
    p.x = a->x;
    p.w = a->w;
    p.out = a->out;
    p.gate = a->gate;
    p.tail = a->tail;
    p.cos_sin = a->cos_sin;
    p.qo_indptr = a->qo_indptr;
    p.pos0 = a->pos0;
    p.ldx = a->ldx;
    p.hx = a->hx;
    p.ldo = a->ldo;
    p.ho = a->ho;
    p.ld_gate = a->ld_gate;
    p.ldt = a->ldt;
    p.ht = a->ht;
    p.M = a->M;
    p.H = a->H;
    p.N = a->N;
    p.K = a->K;
    p.B = a->B;
    p.tail_dim = a->tail_dim;
    p.tail_pad = a->tail_pad;
    p.rot_pairs = a->rot_pairs;
    p.max_pos = a->max_pos;
    hipStream_t st = (hipStream_t)stream;
    if (a->dtype == MD_T_F32) {
        MD_CHECK_ARG((a->M + 15) / 16 <= 65535, "md_head_linear: %d rows", a->M);
        hipLaunchKernelGGL(head_linear_f32_kernel, dim3((a->N + 15) / 16, (a->M + 15) / 16, a->H), dim3(256), 0, st, p);
        MD_CHECK_LAUNCH("md_head_linear");
        return MD_OK;
    }
    const bool vec = a->K % 8 == 0 && a->ldx % 8 == 0 && a->hx % 8 == 0 && a->ldo % 4 == 0 && a->ho % 4 == 0 && aligned(a->x, 16) &&
                     aligned(a->w, 16) && aligned(a->out, 8);
    const int nb = (a->N + 63) / 64;
    const int rt = (long)nb * a->H * ((a->M + 63) / 64) >= 256 ? 4 : (long)nb * a->H * ((a->M + 31) / 32) >= 256 ? 2 : 1;
    const dim3 grid(nb, (a->M + 16 * rt - 1) / (16 * rt), a->H);
    MD_CHECK_ARG(grid.y <= 65535, "md_head_linear: %d rows", a->M);
#define MD_HL(RT)                                                                                               \
    do {                                                                                                        \
        if (vec) hipLaunchKernelGGL((head_linear_mfma_kernel<RT, true>), grid, dim3(256), 0, st, p);            \
        else hipLaunchKernelGGL((head_linear_mfma_kernel<RT, false>), grid, dim3(256), 0, st, p);               \
    } while (0)
    if (rt == 4) MD_HL(4);
    else if (rt == 2) MD_HL(2);
    else MD_HL(1);
#undef MD_HL
    MD_CHECK_LAUNCH("md_head_linear");
    return MD_OK;
}

extern "C" size_t md_latent_workspace_bytes(const md_latent_args* a) {
    if (!a || !mfma_ok(a)) return 0;
    const int ns = kv_splits(a);
    if (ns == 1) return 0;
    const size_t Rp = (a->kv_rank + 15) / 16 * 16;
    return (size_t)a->B * row_groups(a) * ns * 16 * row_tiles(a) * (Rp + 2) * 4;
}

extern "C" int md_latent_attn(const md_latent_args* a, md_stream_t stream) {
    int rc = check_args("md_latent_attn", a);
    if (rc != MD_OK) return rc;
    MD_CHECK_ARG(a->q && a->out && aligned(a->q, 16) && aligned(a->out, 8), "md_latent_attn: q and out (16-byte aligned) are needed");
    hipStream_t st = (hipStream_t)stream;
    LatentParams p = make_params(a);
    if (!mfma_ok(a)) {
        // the same sums as a one-kv-head attention whose values are the first kv_rank elements of its keys
        XattnParams x = {};
        x.q = a->q;
        x.k_cache = a->cache;
        x.v_cache = a->cache;
        x.out = a->out;
        x.qo_indptr = a->qo_indptr;
        x.pos0 = a->pos0;
        x.page_indices = a->page_indices;
        x.page_indptr = a->page_indptr;
        x.B = a->B;
        x.n_max = a->n_max;
        x.H = x.g = a->H;
        x.KH = 1;
        x.D = x.DKp = x.ldk = x.ldv = p.W;
        x.DV = x.DVp = a->kv_rank;
        x.page_size = a->page_size;
        x.chunk = 0x7fffffff;
        x.scale = a->scale;
        return md_internal_xattn_plain(x, a->dtype, st);
    }
    const int qt = row_tiles(a);
    p.n_groups = row_groups(a);
    p.nsplit = kv_splits(a);
    if (p.nsplit > 1) {
        MD_CHECK_ARG(a->workspace && a->workspace_bytes >= md_latent_workspace_bytes(a) && aligned(a->workspace, 16),
                     "md_latent_attn: workspace of %zu bytes needed, got %zu", md_latent_workspace_bytes(a), a->workspace_bytes);
        p.ws = (float*)a->workspace;
    }
    rc = md_internal_latent_absorbed(p, qt, st);
    if (rc != MD_OK) return rc;
    if (p.nsplit > 1) {
        const int Rp = (a->kv_rank + 15) / 16 * 16;
        const int rows = a->n_max * a->H, cols = (Rp + 255) / 256;
        if (p.nsplit > 8) hipLaunchKernelGGL((latent_merge_kernel<4>), dim3(rows, cols, a->B), dim3(256), 0, st, p, 16 * qt, Rp);
        else hipLaunchKernelGGL((latent_merge_kernel<1>), dim3((rows + 3) / 4, cols, a->B), dim3(256), 0, st, p, 16 * qt, Rp);
    }
    MD_CHECK_LAUNCH("md_latent_attn");
    return MD_OK;
}

extern "C" int md_latent_gather(const md_latent_args* a, int ctx_max, void* dst, md_stream_t stream) {
    const int rc = check_args("md_latent_gather", a);
    if (rc != MD_OK) return rc;
    MD_CHECK_ARG(a->ctx_indptr && dst && aligned(dst, 16) && ctx_max > 0 && a->kv_rank % 8 == 0 && a->dtype == MD_T_BF16,
                 "md_latent_gather: needs context lengths, bf16 and kv_rank %% 8 == 0");
    const LatentParams p = make_params(a);
    hipLaunchKernelGGL(latent_gather_kernel, dim3((ctx_max + 3) / 4, a->B), dim3(256), 0, (hipStream_t)stream, p, (bf16_t*)dst);
    MD_CHECK_LAUNCH("md_latent_gather");
    return MD_OK;
}

extern "C" int md_latent_prefill_supported(const md_latent_args* a) {
    return a && a->dtype == MD_T_BF16 && a->dim > 0 && a->dim % 8 == 0 && a->rot_dim % 8 == 0 && a->vdim > 0 && a->vdim % 8 == 0 &&
           a->kv_rank % 8 == 0 && prefill_dk(a->dim + a->rot_dim) && prefill_dk(a->vdim) && a->page_size % 64 == 0 ? 1 : 0;
}

extern "C" int md_latent_prefill(const md_latent_args* a, md_stream_t stream) {
    const int rc0 = check_args("md_latent_prefill", a);
    if (rc0 != MD_OK) return rc0;
    MD_CHECK_ARG(md_latent_prefill_supported(a), "md_latent_prefill: unsupported sizes (md_latent_prefill_supported)");
    MD_CHECK_ARG(a->q && a->kv && a->ctx_indptr && a->cos_sin && a->out && a->max_pos > 0 && aligned(a->q, 16) && aligned(a->kv, 16) &&
                     aligned(a->out, 8) && a->ldo % 4 == 0 && a->ldo >= (int64_t)a->H * a->vdim,
                 "md_latent_prefill: null or misaligned argument");
    LatentParams p = make_params(a);
    p.n_groups = (a->n_max + kLatentPrefillRows - 1) / kLatentPrefillRows;
    const int64_t grid = ((int64_t)a->B * a->H + 7) / 8 * 8 * p.n_groups;
    MD_CHECK_ARG(grid < ((int64_t)1 << 31), "md_latent_prefill: grid too large");
    int rc;
    switch (prefill_dk(a->dim + a->rot_dim)) {
    case 64: rc = md_internal_latent_prefill_64(p, (int)grid, (hipStream_t)stream); break;
    case 128: rc = md_internal_latent_prefill_128(p, (int)grid, (hipStream_t)stream); break;
    case 192: rc = md_internal_latent_prefill_192(p, (int)grid, (hipStream_t)stream); break;
    default: rc = md_internal_latent_prefill_256(p, (int)grid, (hipStream_t)stream);
    }
    if (rc != MD_OK) return rc;
    MD_CHECK_LAUNCH("md_latent_prefill");
    return MD_OK;
}
