// The fp32 residual stream of the layered decoder designs (gfx950): embedding with learned positions, and the residual add +
// weighted RMS norm + token shift between two sub-layers, in one launch.
//
//   md_embed_pos        x = float(E[token]) * scale + float(P[pos])                                     (fp32 rows)
//   md_embed_bigram     x = rms(float(E[token]) + float(G[(a * before + b * token) % n])) * w            (fp32 rows)
//   md_resid_norm       x += delta;  h = x / sqrt(mean(x^2) + eps) * w  (fp32);  y = h * out_scale  (rounded to the model dtype)
//   md_resid_norm_shift the same with the token shift  y = h_t + (h_{t-1} - h_t) * mu  in front of the rounding
//
// `delta` is the output of the sub-layer's projection: model-dtype rows, or the S fp32 partial planes [S][rows][width] a
// split-K GEMM left in its workspace (the add and the norm then ARE that GEMM's combine launch, and the projection reaches
// the fp32 residual without a 16-bit rounding in between).
//
// Bigram embedding.  The token before a row is the step's own previous row, or -- first row of a portion -- comes from a token
// history that is paged like a KV cache: position p of a sequence lies in its page p / page_size.  A row writes its own entry
// only, so a step may be repeated, rolled back or continued in any portions without further state.
//
// Token shift.  h_{t-1} of a row is the previous row's own h: the workgroup recomputes it from x + delta of that row (x_out is
// a different buffer from x, so no workgroup sees a half-updated residual), except for the first row of a portion, whose
// predecessor was processed by an earlier step.  That one comes from a per-sequence RING of the last `ring` unshifted rows,
// indexed by position: row p reads slot (p - 1) % ring and leaves its own h in slot p % ring.  Because the slot follows from
// the position,
//   * running a step again (warm-up and capture of a graph) reads and writes the same values, and
//   * a sequence may be rolled back by up to ring - 2 positions (rejected draft tokens) without saving anything.
// A launch of at most ring - 1 rows per sequence writes the ring itself (its slots are distinct from the one row 0 reads);
// longer portions leave it to a second launch over their last ring - 1 rows (state_only).
//
// One workgroup of 256 threads per `rows_per_wg` consecutive rows of one sequence; a row lives in registers (width <= 8192,
// 8 elements per thread and trip, or 1 where the width is no multiple of 8).
#include "md_common.h"

namespace {

template <int VEC>
__device__ __forceinline__ void ld_vec(const float* p, float (&f)[VEC]) {
    if constexpr (VEC == 8) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(p), b = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            f[e] = a[e];
            f[4 + e] = b[e];
        }
    } else {
        f[0] = p[0];
    }
}
template <int VEC>
__device__ __forceinline__ void ld_vec(const bf16_t* p, float (&f)[VEC]) {
    if constexpr (VEC == 8) {
        const f32x8 a = __builtin_convertvector(*reinterpret_cast<const bf16x8*>(p), f32x8);
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] = a[e];
    } else {
        f[0] = (float)p[0];
    }
}
template <int VEC>
__device__ __forceinline__ void st_vec(float* p, const float (&f)[VEC]) {
    if constexpr (VEC == 8) {
        *reinterpret_cast<f32x4*>(p) = f32x4{f[0], f[1], f[2], f[3]};
        *reinterpret_cast<f32x4*>(p + 4) = f32x4{f[4], f[5], f[6], f[7]};
    } else {
        p[0] = f[0];
    }
}
template <int VEC>
__device__ __forceinline__ void st_vec(bf16_t* p, const float (&f)[VEC]) {
    if constexpr (VEC == 8) {
        f32x8 a;
#pragma unroll
        for (int e = 0; e < 8; ++e) a[e] = f[e];
        *reinterpret_cast<bf16x8*>(p) = __builtin_convertvector(a, bf16x8);
    } else {
        p[0] = (bf16_t)f[0];
    }
}

struct ResidParams {
    const float* x;          // [rows][width]
    const void* delta;       // model dtype [rows][width], or null
    const float* planes;     // [S][rows][width] fp32, or null
    int S;
    int64_t plane_stride;
    float* x_out;            // null: the residual is unchanged (no delta)
    const void* w;           // norm weight, model dtype
    const void* mu;          // token shift, model dtype, or null
    void* y;                 // [rows][width] model dtype
    float eps, out_scale;
    int width, rows, rows_per_wg;
    // token shift
    const int32_t* qo_indptr;
    const int32_t* pos0;
    const int32_t* slots;    // ring row of request b (null: b)
    float* ring;             // [slots][ring_len][width]
    int ring_len, write_ring, state_only;
};

__device__ __forceinline__ float block_sum(float v, float* red) {
    v = wave_reduce_sum(v);
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, nw = blockDim.x >> 6;
    if (lane == 0) red[wave] = v;
    __syncthreads();
    float t = 0.f;
    for (int w = 0; w < nw; ++w) t += red[w];
    __syncthreads();
    return t;
}

template <typename T, int VEC, int MAXV, bool SHIFT>
__global__ __launch_bounds__(256) void resid_norm_kernel(const ResidParams p) {
    __shared__ float red[8];
    const int nvec = p.width / VEC;
    int row0, nrow, j0 = 0, n_b = 0, pos_b = 0;
    float* ring = nullptr;
    if constexpr (SHIFT) {
        const int b = blockIdx.y;
        const int q0 = p.qo_indptr[b];
        n_b = p.qo_indptr[b + 1] - q0;
        pos_b = p.pos0[b];
        const int first = p.state_only ? max(0, n_b - (p.ring_len - 1)) : 0;
        j0 = first + blockIdx.x * p.rows_per_wg;
        if (j0 >= n_b) return;
        nrow = min(p.rows_per_wg, n_b - j0);
        row0 = q0 + j0;
        ring = p.ring + (int64_t)(p.slots ? p.slots[b] : b) * p.ring_len * p.width;
    } else {
        row0 = blockIdx.x * p.rows_per_wg;
        nrow = min(p.rows_per_wg, p.rows - row0);
    }
    float h[MAXV][VEC], hp[SHIFT ? MAXV : 1][VEC];

    // h of one row: x + delta (optionally stored), the weighted RMS norm, all in fp32
    auto load_row = [&](int row, bool store) {
        float ss = 0.f;
#pragma unroll
        for (int it = 0; it < MAXV; ++it) {
            const int i = threadIdx.x + it * 256;
            if (i < nvec) {
                const int64_t off = (int64_t)row * p.width + i * VEC;
                ld_vec<VEC>(p.x + off, h[it]);
                if (p.planes) {
                    float d[VEC];
#pragma unroll
                    for (int e = 0; e < VEC; ++e) d[e] = 0.f;
                    for (int s0 = 0; s0 < p.S; s0 += 4) {            // four slices requested together, added in order
                        float t[4][VEC];
#pragma unroll
                        for (int u = 0; u < 4; ++u)
                            if (s0 + u < p.S) ld_vec<VEC>(p.planes + (s0 + u) * p.plane_stride + off, t[u]);
#pragma unroll
                        for (int u = 0; u < 4; ++u)
                            if (s0 + u < p.S) {
#pragma unroll
                                for (int e = 0; e < VEC; ++e) d[e] += t[u][e];
                            }
                    }
#pragma unroll
                    for (int e = 0; e < VEC; ++e) h[it][e] += d[e];
                } else if (p.delta) {
                    float d[VEC];
                    ld_vec<VEC>(reinterpret_cast<const T*>(p.delta) + off, d);
#pragma unroll
                    for (int e = 0; e < VEC; ++e) h[it][e] += d[e];
                }
                if (store && p.x_out) st_vec<VEC>(p.x_out + off, h[it]);
#pragma unroll
                for (int e = 0; e < VEC; ++e) ss += h[it][e] * h[it][e];
            }
        }
        const float rs = 1.0f / sqrtf(block_sum(ss, red) / (float)p.width + p.eps);
#pragma unroll
        for (int it = 0; it < MAXV; ++it) {
            const int i = threadIdx.x + it * 256;
            if (i < nvec) {
                float w[VEC];
                ld_vec<VEC>(reinterpret_cast<const T*>(p.w) + i * VEC, w);
#pragma unroll
                for (int e = 0; e < VEC; ++e) h[it][e] = (h[it][e] * rs) * w[e];
            }
        }
    };

    if constexpr (SHIFT) {
        if (!p.state_only) {
            if (j0 > 0) {
                load_row(row0 - 1, false);
#pragma unroll
                for (int it = 0; it < MAXV; ++it)
#pragma unroll
                    for (int e = 0; e < VEC; ++e) hp[it][e] = h[it][e];
            } else {
#pragma unroll
                for (int it = 0; it < MAXV; ++it) {
                    const int i = threadIdx.x + it * 256;
#pragma unroll
                    for (int e = 0; e < VEC; ++e) hp[it][e] = 0.f;
                    if (pos_b > 0 && i < nvec)
                        ld_vec<VEC>(ring + (int64_t)((pos_b - 1) % p.ring_len) * p.width + i * VEC, hp[it]);
                }
            }
        }
    }
    for (int r = 0; r < nrow; ++r) {
        load_row(row0 + r, !p.state_only);
        if constexpr (SHIFT) {
            const int pos = pos_b + j0 + r;
#pragma unroll
            for (int it = 0; it < MAXV; ++it) {
                const int i = threadIdx.x + it * 256;
                if (i >= nvec) continue;
                if (p.write_ring) st_vec<VEC>(ring + (int64_t)(pos % p.ring_len) * p.width + i * VEC, h[it]);
                if (p.state_only) continue;
                float mu[VEC], y[VEC];
                ld_vec<VEC>(reinterpret_cast<const T*>(p.mu) + i * VEC, mu);
#pragma unroll
                for (int e = 0; e < VEC; ++e) {
                    y[e] = (h[it][e] + (hp[it][e] - h[it][e]) * mu[e]) * p.out_scale;
                    hp[it][e] = h[it][e];
                }
                st_vec<VEC>(reinterpret_cast<T*>(p.y) + (int64_t)(row0 + r) * p.width + i * VEC, y);
            }
        } else {
#pragma unroll
            for (int it = 0; it < MAXV; ++it) {
                const int i = threadIdx.x + it * 256;
                if (i >= nvec) continue;
                float y[VEC];
#pragma unroll
                for (int e = 0; e < VEC; ++e) y[e] = h[it][e] * p.out_scale;
                st_vec<VEC>(reinterpret_cast<T*>(p.y) + (int64_t)(row0 + r) * p.width + i * VEC, y);
            }
        }
    }
}

template <typename T, int VEC, bool SHIFT>
void launch_resid_v(const ResidParams& p, dim3 grid, hipStream_t st) {
    const int trips = (p.width / VEC + 255) / 256;
    if constexpr (VEC == 8) {
        if (trips <= 1) hipLaunchKernelGGL((resid_norm_kernel<T, 8, 1, SHIFT>), grid, dim3(256), 0, st, p);
        else if (trips <= 2) hipLaunchKernelGGL((resid_norm_kernel<T, 8, 2, SHIFT>), grid, dim3(256), 0, st, p);
        else hipLaunchKernelGGL((resid_norm_kernel<T, 8, 4, SHIFT>), grid, dim3(256), 0, st, p);
    } else {
        if (trips <= 4) hipLaunchKernelGGL((resid_norm_kernel<T, 1, 4, SHIFT>), grid, dim3(256), 0, st, p);
        else hipLaunchKernelGGL((resid_norm_kernel<T, 1, 32, SHIFT>), grid, dim3(256), 0, st, p);
    }
}

template <bool SHIFT>
void launch_resid(const ResidParams& p, int dtype, bool vec, dim3 grid, hipStream_t st) {
    if (dtype == MD_T_F32) {
        vec ? launch_resid_v<float, 8, SHIFT>(p, grid, st) : launch_resid_v<float, 1, SHIFT>(p, grid, st);
    } else {
        vec ? launch_resid_v<bf16_t, 8, SHIFT>(p, grid, st) : launch_resid_v<bf16_t, 1, SHIFT>(p, grid, st);
    }
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void embed_pos_kernel(const int64_t* __restrict__ tokens, const T* __restrict__ table,
                                                        const T* __restrict__ pos_table, const int32_t* __restrict__ qo_indptr,
                                                        const int32_t* __restrict__ pos0, int width, int vocab, int max_pos,
                                                        float scale, float* __restrict__ out) {
    const int b = blockIdx.y, j = blockIdx.x;
    const int q0 = qo_indptr[b];
    if (j >= qo_indptr[b + 1] - q0) return;
    int64_t tok = tokens[q0 + j];
    tok = tok < 0 ? 0 : (tok >= vocab ? vocab - 1 : tok);            // the host refuses such ids; never index past the table
    int pos = pos0[b] + j;
    pos = pos < 0 ? 0 : (pos >= max_pos ? max_pos - 1 : pos);
    for (int i = threadIdx.x; i < width / VEC; i += 256) {
        float v[VEC], q[VEC];
        ld_vec<VEC>(table + tok * width + i * VEC, v);
        if (pos_table) ld_vec<VEC>(pos_table + (int64_t)pos * width + i * VEC, q);
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
            v[e] *= scale;
            if (pos_table) v[e] += q[e];
        }
        st_vec<VEC>(out + (int64_t)(q0 + j) * width + i * VEC, v);
    }
}

template <typename T, int VEC>
void launch_embed(const int64_t* tokens, const void* table, const void* pos_table, const int32_t* qo_indptr, const int32_t* pos0,
                  dim3 grid, int width, int vocab, int max_pos, float scale, float* out, hipStream_t st) {
    hipLaunchKernelGGL((embed_pos_kernel<T, VEC>), grid, dim3(256), 0, st, tokens, (const T*)table, (const T*)pos_table,
                       qo_indptr, pos0, width, vocab, max_pos, scale, out);
}

struct BigramParams {
    const int64_t* tokens;
    const void* table;       // [vocab][width]
    const void* pairs;       // [buckets + 1][width]; row `buckets`: a sequence's first token
    const void* w;           // norm weight
    const int32_t* qo_indptr;
    const int32_t* pos0;
    const int32_t* page_indices;
    const int32_t* page_indptr;
    int32_t* history;        // [pages][page_size]
    float* out;
    int64_t mul_before, mul_token;
    int width, vocab, buckets, page_size;
    float eps;
};

__device__ __forceinline__ int64_t clamp_token(int64_t t, int vocab) {   // the host refuses such ids; never index past the table
    return t < 0 ? 0 : (t >= vocab ? vocab - 1 : t);
}

template <typename T, int VEC, int MAXV>
__global__ __launch_bounds__(256) void embed_bigram_kernel(const BigramParams p) {
    __shared__ float red[8];
    const int b = blockIdx.y, j = blockIdx.x;
    const int q0 = p.qo_indptr[b];
    if (j >= p.qo_indptr[b + 1] - q0) return;
    const int pos = p.pos0[b] + j, pg0 = p.page_indptr[b], cap = (p.page_indptr[b + 1] - pg0) * p.page_size;
    const int64_t tok = clamp_token(p.tokens[q0 + j], p.vocab);
    auto entry = [&](int at) { return p.history + (int64_t)p.page_indices[pg0 + at / p.page_size] * p.page_size + at % p.page_size; };
    int64_t before = 0;
    if (j > 0) before = clamp_token(p.tokens[q0 + j - 1], p.vocab);
    else if (pos > 0 && pos - 1 < cap) before = *entry(pos - 1);
    if (threadIdx.x == 0 && pos >= 0 && pos < cap) *entry(pos) = (int32_t)tok;
    int64_t pair = pos <= 0 ? p.buckets : (before * p.mul_before + tok * p.mul_token) % p.buckets;
    if (pair < 0) pair += p.buckets;
    const int nvec = p.width / VEC;
    float h[MAXV][VEC], ss = 0.f;
#pragma unroll
    for (int it = 0; it < MAXV; ++it) {
        const int i = threadIdx.x + it * 256;
        if (i < nvec) {
            float g[VEC];
            ld_vec<VEC>(reinterpret_cast<const T*>(p.table) + tok * p.width + i * VEC, h[it]);
            ld_vec<VEC>(reinterpret_cast<const T*>(p.pairs) + pair * p.width + i * VEC, g);
#pragma unroll
            for (int e = 0; e < VEC; ++e) {
                h[it][e] += g[e];
                ss += h[it][e] * h[it][e];
            }
        }
    }
    const float rs = 1.0f / sqrtf(block_sum(ss, red) / (float)p.width + p.eps);
#pragma unroll
    for (int it = 0; it < MAXV; ++it) {
        const int i = threadIdx.x + it * 256;
        if (i < nvec) {
            float w[VEC];
            ld_vec<VEC>(reinterpret_cast<const T*>(p.w) + i * VEC, w);
#pragma unroll
            for (int e = 0; e < VEC; ++e) h[it][e] = (h[it][e] * rs) * w[e];
            st_vec<VEC>(p.out + (int64_t)(q0 + j) * p.width + i * VEC, h[it]);
        }
    }
}

template <typename T>
void launch_bigram(const BigramParams& p, bool vec, dim3 grid, hipStream_t st) {
    const int trips = (p.width / (vec ? 8 : 1) + 255) / 256;
    if (vec) {
        if (trips <= 1) hipLaunchKernelGGL((embed_bigram_kernel<T, 8, 1>), grid, dim3(256), 0, st, p);
        else if (trips <= 2) hipLaunchKernelGGL((embed_bigram_kernel<T, 8, 2>), grid, dim3(256), 0, st, p);
        else hipLaunchKernelGGL((embed_bigram_kernel<T, 8, 4>), grid, dim3(256), 0, st, p);
    } else {
        if (trips <= 4) hipLaunchKernelGGL((embed_bigram_kernel<T, 1, 4>), grid, dim3(256), 0, st, p);
        else hipLaunchKernelGGL((embed_bigram_kernel<T, 1, 32>), grid, dim3(256), 0, st, p);
    }
}

bool aligned16(const void* q) { return ((uintptr_t)q & 15) == 0; }

int resid_check(const char* who, const md_resid_norm_args* a) {
    MD_CHECK_ARG(a && a->x && a->weight && a->y, "%s: null pointer argument", who);
    MD_CHECK_ARG(a->rows > 0 && a->width > 0 && a->width <= 8192, "%s: bad shape rows=%d width=%d (width <= 8192)", who, a->rows,
                 a->width);
    MD_CHECK_ARG(a->dtype == MD_T_BF16 || a->dtype == MD_T_F32, "%s: dtype must be MD_T_BF16 or MD_T_F32", who);
    MD_CHECK_ARG(!(a->delta && a->planes), "%s: delta and planes are alternatives", who);
    MD_CHECK_ARG(!a->planes || a->n_planes > 0, "%s: planes need n_planes", who);
    MD_CHECK_ARG(!(a->delta || a->planes) || (a->x_out && a->x_out != a->x),
                 "%s: the updated residual needs a buffer of its own", who);
    return MD_OK;
}

ResidParams resid_params(const md_resid_norm_args* a) {
    ResidParams p = {};
    p.x = a->x;
    p.delta = a->delta;
    p.planes = a->planes;
    p.S = a->n_planes;
    p.plane_stride = (int64_t)a->rows * a->width;
    p.x_out = (a->delta || a->planes) ? a->x_out : nullptr;
    p.w = a->weight;
    p.y = a->y;
    p.eps = a->eps;
    p.out_scale = a->out_scale;
    p.width = a->width;
    p.rows = a->rows;
    return p;
}

bool resid_vec(const md_resid_norm_args* a) {
    return a->width % 8 == 0 && aligned16(a->x) && aligned16(a->delta) && aligned16(a->planes) && aligned16(a->x_out) &&
           aligned16(a->weight) && aligned16(a->y) && aligned16(a->shift) && aligned16(a->ring);
}

}  // namespace

// the split-K GEMMs (gemm.hip, tilegemm.hip, blockgemm.hip) up to their partial planes
#define MD_PLANES_DECL(kind)                                                                                              \
    int md_internal_planes_##kind##_count(int M, int N, int K);                                                            \
    int md_internal_planes_##kind(const void* x, int64_t ldx, const void* w, int M, int N, int K, void* ws, size_t ws_bytes, \
                                  int* S, hipStream_t st);
MD_PLANES_DECL(skinny)
MD_PLANES_DECL(tile)
MD_PLANES_DECL(block)
#undef MD_PLANES_DECL

extern "C" int md_linear_planes_count(int kind, int M, int N, int K) {
    return kind == MD_PLANES_SKINNY ? md_internal_planes_skinny_count(M, N, K)
         : kind == MD_PLANES_TILE   ? md_internal_planes_tile_count(M, N, K)
         : kind == MD_PLANES_BLOCK  ? md_internal_planes_block_count(M, N, K) : 0;
}

extern "C" int md_linear_planes(int kind, const void* x, int64_t ldx, const void* w_packed, int M, int N, int K, float* planes,
                                size_t planes_bytes, md_stream_t stream) {
    MD_CHECK_ARG(md_linear_planes_count(kind, M, N, K) > 0, "md_linear_planes: unsupported shape kind=%d M=%d N=%d K=%d", kind, M,
                 N, K);
    int S = 0, rc;
    hipStream_t st = (hipStream_t)stream;
    if (kind == MD_PLANES_SKINNY) rc = md_internal_planes_skinny(x, ldx, w_packed, M, N, K, planes, planes_bytes, &S, st);
    else if (kind == MD_PLANES_TILE) rc = md_internal_planes_tile(x, ldx, w_packed, M, N, K, planes, planes_bytes, &S, st);
    else rc = md_internal_planes_block(x, ldx, w_packed, M, N, K, planes, planes_bytes, &S, st);
    if (rc != MD_OK) return rc;
    MD_CHECK_LAUNCH("md_linear_planes");
    return MD_OK;
}

extern "C" int md_embed_pos(const int64_t* tokens, const void* table, const void* pos_table, int dtype,
                            const int32_t* qo_indptr, const int32_t* pos0, int B, int n_max, int width, int vocab, int max_pos,
                            float scale, float* out, md_stream_t stream) {
    MD_CHECK_ARG(tokens && table && qo_indptr && pos0 && out, "md_embed_pos: null pointer argument");
    MD_CHECK_ARG(B > 0 && B <= 65535 && n_max > 0 && width > 0 && vocab > 0 && max_pos > 0,
                 "md_embed_pos: bad shape B=%d n_max=%d width=%d", B, n_max, width);
    MD_CHECK_ARG(dtype == MD_T_BF16 || dtype == MD_T_F32, "md_embed_pos: dtype must be MD_T_BF16 or MD_T_F32");
    const bool vec = width % 8 == 0 && aligned16(table) && aligned16(pos_table) && aligned16(out);
    auto k = dtype == MD_T_F32 ? (vec ? launch_embed<float, 8> : launch_embed<float, 1>)
                               : (vec ? launch_embed<bf16_t, 8> : launch_embed<bf16_t, 1>);
    k(tokens, table, pos_table, qo_indptr, pos0, dim3(n_max, B), width, vocab, max_pos, scale, out, (hipStream_t)stream);
    MD_CHECK_LAUNCH("md_embed_pos");
    return MD_OK;
}

extern "C" int md_embed_bigram(const int64_t* tokens, const void* table, const void* pairs, const void* norm_weight, int dtype,
                               const int32_t* qo_indptr, const int32_t* pos0, int B, int n_max, int width, int vocab, int buckets,
                               int64_t mul_before, int64_t mul_token, int32_t* history, const int32_t* page_indices,
                               const int32_t* page_indptr, int page_size, float eps, float* out, md_stream_t stream) {
    MD_CHECK_ARG(tokens && table && pairs && norm_weight && qo_indptr && pos0 && history && page_indices && page_indptr && out,
                 "md_embed_bigram: null pointer argument");
    MD_CHECK_ARG(B > 0 && B <= 65535 && n_max > 0 && width > 0 && width <= 8192 && vocab > 0 && buckets > 0 && page_size > 0,
                 "md_embed_bigram: bad shape B=%d n_max=%d width=%d (<= 8192) buckets=%d", B, n_max, width, buckets);
    MD_CHECK_ARG(dtype == MD_T_BF16 || dtype == MD_T_F32, "md_embed_bigram: dtype must be MD_T_BF16 or MD_T_F32");
    BigramParams p = {tokens, table, pairs, norm_weight, qo_indptr, pos0, page_indices, page_indptr, history, out,
                      mul_before, mul_token, width, vocab, buckets, page_size, eps};
    const bool vec = width % 8 == 0 && aligned16(table) && aligned16(pairs) && aligned16(norm_weight) && aligned16(out);
    if (dtype == MD_T_F32) launch_bigram<float>(p, vec, dim3(n_max, B), (hipStream_t)stream);
    else launch_bigram<bf16_t>(p, vec, dim3(n_max, B), (hipStream_t)stream);
    MD_CHECK_LAUNCH("md_embed_bigram");
    return MD_OK;
}

extern "C" int md_resid_norm(const md_resid_norm_args* a, md_stream_t stream) {
    const int rc = resid_check("md_resid_norm", a);
    if (rc != MD_OK) return rc;
    MD_CHECK_ARG(!a->shift, "md_resid_norm: the token shift is md_resid_norm_shift");
    ResidParams p = resid_params(a);
    p.rows_per_wg = 1;
    launch_resid<false>(p, a->dtype, resid_vec(a), dim3(a->rows), (hipStream_t)stream);
    MD_CHECK_LAUNCH("md_resid_norm");
    return MD_OK;
}

extern "C" int md_resid_norm_shift(const md_resid_norm_args* a, md_stream_t stream) {
    const int rc = resid_check("md_resid_norm_shift", a);
    if (rc != MD_OK) return rc;
    MD_CHECK_ARG(a->shift && a->ring && a->qo_indptr && a->pos0, "md_resid_norm_shift: null pointer argument");
    MD_CHECK_ARG(a->B > 0 && a->B <= 65535 && a->n_max > 0 && a->ring_len >= 2,
                 "md_resid_norm_shift: bad shape B=%d n_max=%d ring=%d", a->B, a->n_max, a->ring_len);
    ResidParams p = resid_params(a);
    p.mu = a->shift;
    p.qo_indptr = a->qo_indptr;
    p.pos0 = a->pos0;
    p.slots = a->slots;
    p.ring = a->ring;
    p.ring_len = a->ring_len;
    hipStream_t st = (hipStream_t)stream;
    // rows per workgroup: enough workgroups to fill the chip first, then fewer rows computed twice
    p.rows_per_wg = a->rows >= 16384 ? 8 : a->rows >= 8192 ? 4 : a->rows >= 4096 ? 2 : 1;
    const bool short_step = a->n_max <= a->ring_len - 1;
    p.write_ring = short_step ? 1 : 0;
    const bool vec = resid_vec(a);
    launch_resid<true>(p, a->dtype, vec, dim3((a->n_max + p.rows_per_wg - 1) / p.rows_per_wg, a->B), st);
    MD_CHECK_LAUNCH("md_resid_norm_shift");
    if (!short_step) {
        // the last ring - 1 rows of every portion, from the updated residual (their h is the one computed above)
        p.state_only = 1;
        p.write_ring = 1;
        if (p.x_out) p.x = p.x_out;
        p.delta = nullptr;
        p.planes = nullptr;
        p.x_out = nullptr;
        p.rows_per_wg = 1;
        launch_resid<true>(p, a->dtype, vec, dim3(a->ring_len - 1, a->B), st);
        MD_CHECK_LAUNCH("md_resid_norm_shift(state)");
    }
    return MD_OK;
}
