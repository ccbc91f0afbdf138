// Extended paged attention (gfx950): the softmax attention of the layered decoder designs, every feature a parameter --
//   * query/key and value head sizes of their own (K and V pages are separate slabs, rows padded to the kernels' widths);
//   * unit-RMS query and key heads (scaled in fp32, no weights; keys once, at the append);
//   * a distance penalty per query head, -a ln(1 + c d) at distance d (r1 = a, r2 = c);
//   * block-diagonal causality: a row at position t sees the positions from (t / chunk) * chunk up to t;
//   * a softmax sink: the denominator is 1 + (sum of the exponentials).
// Positions come from pos0[b] + row, and a request's page list maps EVERY position it may reach (position p lies in its page
// p / page_size), so that neither the append nor the attention needs a last-page length: decoding crosses pages, a step may
// be run again, and a rolled-back sequence just writes its rows anew.
//
//   md_qk_norm_append   q -> normalised padded rows; k -> normalised, v -> the cache
//   md_xattn            attention over the cache.  bf16 with a bounded score: the matrix-core kernels of xattn_mfma.hip --
//                       given the RAW projection rows, a decode step's normalisation and append happen inside the attention
//                       launch --; otherwise (32-bit, unusual sizes, unbounded scores) the plain kernel below.
#include "xattn.h"

unsigned int* md_page_overflow_counter_device();   // kvops.hip

namespace {

constexpr int kMaxHead = 1024;          // plain kernel: largest padded head size

// ------------------------------------------------------------------------------------------------ normalise + append
// one wavefront per head vector of a row: q heads, k heads, v heads
template <typename T>
__global__ __launch_bounds__(256) void qk_norm_append_kernel(const XattnParams p, T* __restrict__ q_out) {
    const int b = blockIdx.y, j = blockIdx.x;
    const int q0 = p.qo_indptr[b];
    if (j >= p.qo_indptr[b + 1] - q0) return;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int pos = p.pos0[b] + j;
    const int pg0 = p.page_indptr[b], np = p.page_indptr[b + 1] - pg0;
    const bool fits = pos >= 0 && pos < np * p.page_size;
    if (!fits && threadIdx.x == 0) atomicAdd(p.overflow, 1u);
    const int page = fits ? p.page_indices[pg0 + pos / p.page_size] : 0, slot = pos % p.page_size;
    const T* row = reinterpret_cast<const T*>(p.qkv) + (int64_t)(q0 + j) * p.ld_qkv;
    for (int hv = wave; hv < p.H + 2 * p.KH; hv += 4) {
        const bool is_q = hv < p.H, is_v = hv >= p.H + p.KH;
        const int h = is_q ? hv : is_v ? hv - p.H - p.KH : hv - p.H;
        const int n = is_v ? p.DV : p.D, np_ = is_v ? p.DVp : p.DKp;
        const T* src = row + (is_q ? h * p.D : is_v ? (p.H + p.KH) * p.D + h * p.DV : p.H * p.D + h * p.D);
        float rs = 1.f;
        if (!is_v && p.qk_norm) {
            float ss = 0.f;
            for (int d = lane; d < n; d += 64) {
                const float v = (float)src[d];
                ss += v * v;
            }
            rs = 1.0f / sqrtf(wave_reduce_sum(ss) / (float)n + p.eps);
        }
        T* dst;
        if (is_q) {
            dst = q_out + ((int64_t)(q0 + j) * p.H + h) * p.DKp;
        } else {
            if (!fits) continue;
            dst = reinterpret_cast<T*>(is_v ? p.v_cache : p.k_cache) + (((int64_t)page * p.KH + h) * p.page_size + slot) * np_;
        }
        for (int d = lane; d < np_; d += 64) dst[d] = d < n ? (T)((float)src[d] * rs) : (T)0.f;
    }
}

// the same with 8-element pieces (head sizes and rows that are multiples of 8): `lanes` = lanes per head vector (a power of two
// that covers its padded width), several heads per wavefront; the sum of squares is a butterfly over them
template <typename T>
__global__ __launch_bounds__(256) void qk_norm_append_vec_kernel(const XattnParams p, T* __restrict__ q_out, int lanes_log2,
                                                                 int vlanes_log2) {
    typedef T vec8 __attribute__((ext_vector_type(8)));
    const int b = blockIdx.y, j = blockIdx.x;
    const int q0 = p.qo_indptr[b];
    if (j >= p.qo_indptr[b + 1] - q0) return;
    const int pos = p.pos0[b] + j;
    const int pg0 = p.page_indptr[b], np = p.page_indptr[b + 1] - pg0;
    const bool fits = pos >= 0 && pos < np * p.page_size;
    if (!fits && threadIdx.x == 0) atomicAdd(p.overflow, 1u);
    const int page = fits ? p.page_indices[pg0 + pos / p.page_size] : 0, slot = pos % p.page_size;
    const T* row = reinterpret_cast<const T*>(p.qkv) + (int64_t)(q0 + j) * p.ld_qkv;
    const int nqk = (p.H + p.KH) << lanes_log2, total = nqk + (p.KH << vlanes_log2);
    for (int i = threadIdx.x; i < total; i += 256) {          // a head's lanes are aligned neighbours: active together
        if (i < nqk) {
            const int hv = i >> lanes_log2, d = (i - (hv << lanes_log2)) * 8;
            f32x8 v = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            if (d < p.D) v = __builtin_convertvector(*reinterpret_cast<const vec8*>(row + hv * p.D + d), f32x8);
            float ss = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) ss += v[e] * v[e];
            for (int o = 1; o < (1 << lanes_log2); o <<= 1) ss += __shfl_xor(ss, o);
            const float rs = p.qk_norm ? 1.0f / sqrtf(ss / (float)p.D + p.eps) : 1.f;
            if (d >= p.DKp || (hv >= p.H && !fits)) continue;
            T* dst = hv < p.H ? q_out + ((int64_t)(q0 + j) * p.H + hv) * p.DKp
                              : reinterpret_cast<T*>(p.k_cache) + (((int64_t)page * p.KH + hv - p.H) * p.page_size + slot) * p.DKp;
            *reinterpret_cast<vec8*>(dst + d) = __builtin_convertvector(v * rs, vec8);
        } else {
            const int h = (i - nqk) >> vlanes_log2, d = (i - nqk - (h << vlanes_log2)) * 8;
            if (d >= p.DVp || !fits) continue;
            vec8 v = {};
            if (d < p.DV) v = *reinterpret_cast<const vec8*>(row + (p.H + p.KH) * p.D + h * p.DV + d);
            *reinterpret_cast<vec8*>(reinterpret_cast<T*>(p.v_cache) + (((int64_t)page * p.KH + h) * p.page_size + slot) * p.DVp + d) = v;
        }
    }
}

int lanes_log2_of(int padded) {           // lanes of 8 elements each
    int n = 0;
    while ((8 << n) < padded) ++n;
    return n;
}

// ------------------------------------------------------------------------------------------------ plain attention
template <typename T>
__device__ __forceinline__ float dot_row(const T* k, const float* q, int n);
template <>
__device__ __forceinline__ float dot_row<float>(const float* k, const float* q, int n) {
    float s = 0.f;
    for (int d = 0; d < n; d += 4) {
        const f32x4 v = *reinterpret_cast<const f32x4*>(k + d);
#pragma unroll
        for (int e = 0; e < 4; ++e) s = fmaf(v[e], q[d + e], s);
    }
    return s;
}
template <>
__device__ __forceinline__ float dot_row<bf16_t>(const bf16_t* k, const float* q, int n) {
    float s = 0.f;
    for (int d = 0; d < n; d += 8) {
        const f32x8 v = __builtin_convertvector(*reinterpret_cast<const bf16x8*>(k + d), f32x8);
#pragma unroll
        for (int e = 0; e < 8; ++e) s = fmaf(v[e], q[d + e], s);
    }
    return s;
}

// one workgroup per (row, query head); online softmax over 256-key blocks, everything in fp32
template <typename T>
__global__ __launch_bounds__(256) void xattn_plain_kernel(const XattnParams p) {
    __shared__ float sq[kMaxHead];
    __shared__ float sp[256];
    __shared__ float red[4];
    const int b = blockIdx.z, h = blockIdx.y, j = blockIdx.x, tid = threadIdx.x;
    const int q0 = p.qo_indptr[b];
    if (j >= p.qo_indptr[b + 1] - q0) return;
    const int pos = p.pos0[b] + j;
    const int pg0 = p.page_indptr[b], cap = (p.page_indptr[b + 1] - pg0) * p.page_size;
    const int hi = min(pos, cap - 1), lo = (pos / p.chunk) * p.chunk;
    const int kvh = h / p.g;
    const T* q = reinterpret_cast<const T*>(p.q) + ((int64_t)(q0 + j) * p.H + h) * p.DKp;
    for (int d = tid; d < p.DKp; d += 256) sq[d] = (float)q[d];
    const float r1 = p.r1 ? p.r1[h] : 0.f, r2 = p.r2 ? p.r2[h] : 0.f;
    float m = p.sink ? 0.f : -INFINITY, l = p.sink ? 1.f : 0.f;
    float acc[kMaxHead / 256] = {};
    const int parts = p.DVp < 256 ? 256 / p.DVp : 1;
    const int vd = p.DVp < 256 ? tid % p.DVp : tid, part = p.DVp < 256 ? tid / p.DVp : 0;
    __syncthreads();
    for (int base = lo; base <= hi; base += 256) {
        const int kp = base + tid;
        float s = -INFINITY;
        if (kp <= hi) {
            const int page = p.page_indices[pg0 + kp / p.page_size];
            const T* k = reinterpret_cast<const T*>(p.k_cache) +
                         (((int64_t)page * p.KH + kvh) * p.page_size + kp % p.page_size) * p.ldk;
            s = dot_row<T>(k, sq, p.DKp) * p.scale;
            if (p.r1) s -= r1 * logf(1.0f + r2 * (float)(pos - kp));
        }
        float mx = wave_reduce_max(s);
        if ((tid & 63) == 0) red[tid >> 6] = mx;
        __syncthreads();
        const float mnew = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
        const float pe = kp <= hi ? expf(s - mnew) : 0.f;
        const float alpha = expf(m - mnew);
        m = mnew;
        sp[tid] = pe;
        const float ps = wave_reduce_sum(pe);
        __syncthreads();
        if ((tid & 63) == 0) red[tid >> 6] = ps;
        __syncthreads();
        l = l * alpha + ((red[0] + red[1]) + (red[2] + red[3]));
#pragma unroll
        for (int v = 0; v < kMaxHead / 256; ++v) acc[v] *= alpha;
        const int nk = min(256, hi - base + 1);
        for (int k = part; k < nk && part < parts; k += parts) {
            const int kq = base + k;
            const int page = p.page_indices[pg0 + kq / p.page_size];
            const T* vr = reinterpret_cast<const T*>(p.v_cache) +
                          (((int64_t)page * p.KH + kvh) * p.page_size + kq % p.page_size) * p.ldv;
            const float pk = sp[k];
            if (p.DVp < 256) {
                acc[0] = fmaf(pk, (float)vr[vd], acc[0]);
            } else {
#pragma unroll
                for (int v = 0; v < kMaxHead / 256; ++v)
                    if (vd + v * 256 < p.DVp) acc[v] = fmaf(pk, (float)vr[vd + v * 256], acc[v]);
            }
        }
        __syncthreads();
    }
    const float inv = l > 0.f ? 1.0f / l : 0.f;
    T* o = reinterpret_cast<T*>(p.out) + ((int64_t)(q0 + j) * p.H + h) * p.DV;
    if (p.DVp < 256) {
        sp[tid] = part < parts ? acc[0] : 0.f;
        __syncthreads();
        if (tid < p.DV) {
            float t = 0.f;
            for (int u = 0; u < parts; ++u) t += sp[u * p.DVp + tid];
            o[tid] = (T)(t * inv);
        }
    } else {
#pragma unroll
        for (int v = 0; v < kMaxHead / 256; ++v)
            if (vd + v * 256 < p.DV) o[vd + v * 256] = (T)(acc[v] * inv);
    }
}

// sums the kv splits of a decode launch: partials [slot][rows_cap][DVp] + weights [slot][rows_cap], slot = pair * nsplit + split
__global__ __launch_bounds__(256) void xattn_merge_kernel(const XattnParams p) {
    const int d4 = p.DVp / 4;
    const int64_t id = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int64_t R = id / d4;                              // (pair, row)
    const int d = (int)(id - R * d4) * 4;
    const int pair = (int)(R / p.rows_cap), row = (int)(R - (int64_t)pair * p.rows_cap);
    if (pair >= p.B * p.KH) return;
    const int b = pair / p.KH, kvh = pair % p.KH;
    const int q0 = p.qo_indptr[b], n_b = p.qo_indptr[b + 1] - q0;
    if (row >= n_b * p.g) return;
    const int64_t slots = (int64_t)p.B * p.KH * p.nsplit;
    const float* wl = p.ws + slots * p.rows_cap * p.DVp;
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
    float l = __builtin_amdgcn_exp2f(-p.ref_log2);
    for (int s = 0; s < p.nsplit; ++s) {
        const int64_t slot = ((int64_t)pair * p.nsplit + s) * p.rows_cap + row;
        o += *reinterpret_cast<const f32x4*>(p.ws + slot * p.DVp + d);
        l += wl[slot];
    }
    const float inv = 1.0f / l;
    const int i = row / p.g, r = row - i * p.g;
    bf16_t* op = reinterpret_cast<bf16_t*>(p.out) + ((int64_t)(q0 + i) * p.H + kvh * p.g + r) * p.DV;
#pragma unroll
    for (int e = 0; e < 4; ++e)
        if (d + e < p.DV) op[d + e] = f32_to_bf16(o[e] * inv);
}

int bucket(int n) {
    static const int w[] = {32, 64, 96, 128, 192, 256};
    for (int b : w)
        if (n <= b) return b;
    return (n + 31) / 32 * 32;
}

bool mfma_ok(const md_xattn_args* a) {
    // fixed softmax reference: every score lies below score_bound, the sink's weight exp(-ref) must not vanish
    return a->dtype == MD_T_BF16 && a->qk_norm && a->sink && a->score_bound > 0.f && a->score_bound <= 100.f &&
           bucket(a->D) <= 256 && bucket(a->DV) <= 256 && a->page_size % 128 == 0;
}

int decode_rows(const md_xattn_args* a) { return a->n_max * (a->H / a->KH); }

int g_target_wgs = 256;

int decode_splits(const md_xattn_args* a) {
    // keys one request can see in a step: its chunk (plus the step's own rows), or its whole page list
    long keys = (long)a->max_pages * a->page_size;
    if (a->chunk > 0 && a->chunk + a->n_max < keys) keys = a->chunk + a->n_max;
    const long tiles = (keys + 31) / 32 + 1, pairs = (long)a->B * a->KH;
    long want = (g_target_wgs + pairs - 1) / pairs;
    const long cap = tiles / 16 > 1 ? tiles / 16 : 1;        // >= 16 tiles (4 per wavefront) per workgroup
    if (want > cap) want = cap;
    return (int)(want < 1 ? 1 : want > 64 ? 64 : want);
}

XattnParams make_params(const md_xattn_args* a) {
    XattnParams p = {};
    p.q = a->q;
    p.qkv = a->qkv;
    p.ld_qkv = a->ld_qkv;
    p.k_cache = a->k_cache;
    p.v_cache = a->v_cache;
    p.out = a->out;
    p.qo_indptr = a->qo_indptr;
    p.pos0 = a->pos0;
    p.page_indices = a->page_indices;
    p.page_indptr = a->page_indptr;
    p.r1 = a->r1;
    p.r2 = a->r2;
    p.B = a->B;
    p.n_max = a->n_max;
    p.H = a->H;
    p.KH = a->KH;
    p.g = a->H / a->KH;
    p.D = a->D;
    p.DV = a->DV;
    p.DKp = bucket(a->D);
    p.DVp = bucket(a->DV);
    p.ldk = p.DKp;
    p.ldv = p.DVp;
    p.page_size = a->page_size;
    p.chunk = a->chunk > 0 ? a->chunk : 0x7fffffff;
    p.sink = a->sink;
    p.qk_norm = a->qk_norm;
    p.eps = a->eps;
    p.scale = a->scale;
    p.scale_log2 = a->scale * 1.4426950408889634f;
    p.ref_log2 = (a->score_bound > 60.f ? a->score_bound - 60.f : 0.f) * 1.4426950408889634f;
    p.overflow = md_page_overflow_counter_device();
    return p;
}

int check_args(const char* who, const md_xattn_args* a) {
    MD_CHECK_ARG(a && a->k_cache && a->v_cache && a->qo_indptr && a->pos0 && a->page_indices && a->page_indptr,
                 "%s: null pointer argument", who);
    MD_CHECK_ARG(a->B > 0 && a->B <= 65535 && a->n_max > 0 && a->H > 0 && a->H <= 65535 && a->KH > 0 && a->H % a->KH == 0,
                 "%s: bad shape B=%d n_max=%d H=%d KH=%d", who, a->B, a->n_max, a->H, a->KH);
    MD_CHECK_ARG(a->D > 0 && a->DV > 0 && bucket(a->D) <= kMaxHead && bucket(a->DV) <= kMaxHead,
                 "%s: head sizes %d / %d (<= %d)", who, a->D, a->DV, kMaxHead);
    MD_CHECK_ARG(a->page_size > 0 && a->page_size % 32 == 0 && a->max_pages > 0, "%s: page_size %d must be a multiple of 32",
                 who, a->page_size);
    MD_CHECK_ARG(a->dtype == MD_T_BF16 || a->dtype == MD_T_F32, "%s: dtype must be MD_T_BF16 or MD_T_F32", who);
    MD_CHECK_ARG((((uintptr_t)a->k_cache | (uintptr_t)a->v_cache | (uintptr_t)a->q) & 15) == 0,
                 "%s: q and the caches must be 16-byte aligned", who);
    MD_CHECK_ARG(!a->r1 == !a->r2, "%s: the distance bias needs r1 and r2", who);
    return MD_OK;
}

}  // namespace

int md_internal_xattn_plain(const XattnParams& p, int dtype, hipStream_t st) {
    const dim3 grid(p.n_max, p.H, p.B);
    if (dtype == MD_T_F32)
        hipLaunchKernelGGL((xattn_plain_kernel<float>), grid, dim3(256), 0, st, p);
    else
        hipLaunchKernelGGL((xattn_plain_kernel<bf16_t>), grid, dim3(256), 0, st, p);
    MD_CHECK_LAUNCH("attention(plain)");
    return MD_OK;
}

extern "C" int md_xattn_head_pad(int head_size) { return head_size > 0 && bucket(head_size) <= kMaxHead ? bucket(head_size) : 0; }

extern "C" int md_xattn_fused_supported(const md_xattn_args* a) {
    return a && mfma_ok(a) && decode_rows(a) <= 32 && a->D % 8 == 0 && a->DV % 8 == 0 ? 1 : 0;
}

extern "C" size_t md_xattn_workspace_bytes(const md_xattn_args* a) {
    if (!a || !mfma_ok(a) || decode_rows(a) > 32) return 0;
    const int ns = decode_splits(a);
    if (ns == 1) return 0;
    const size_t cap = decode_rows(a) <= 16 ? 16 : 32;
    return (size_t)a->B * a->KH * ns * cap * (bucket(a->DV) + 1) * 4;
}

extern "C" int md_qk_norm_append(const md_xattn_args* a, void* q_out, md_stream_t stream) {
    const int rc = check_args("md_qk_norm_append", a);
    if (rc != MD_OK) return rc;
    MD_CHECK_ARG(a->qkv && q_out && a->ld_qkv >= (int64_t)(a->H + a->KH) * a->D + (int64_t)a->KH * a->DV,
                 "md_qk_norm_append: needs the projection rows and q_out");
    const XattnParams p = make_params(a);
    MD_CHECK_ARG(p.overflow, "md_qk_norm_append: cannot resolve the page-overflow counter");
    const dim3 grid(a->n_max, a->B);
    const int ll = lanes_log2_of(p.DKp), lv = lanes_log2_of(p.DVp);
    if (a->D % 8 == 0 && a->DV % 8 == 0 && a->ld_qkv % 8 == 0 && ll <= 6 && lv <= 6 &&
        (((uintptr_t)a->qkv | (uintptr_t)q_out) & 31) == 0) {
        if (a->dtype == MD_T_F32)
            hipLaunchKernelGGL((qk_norm_append_vec_kernel<float>), grid, dim3(256), 0, (hipStream_t)stream, p, (float*)q_out, ll, lv);
        else
            hipLaunchKernelGGL((qk_norm_append_vec_kernel<bf16_t>), grid, dim3(256), 0, (hipStream_t)stream, p, (bf16_t*)q_out, ll, lv);
        MD_CHECK_LAUNCH("md_qk_norm_append");
        return MD_OK;
    }
    if (a->dtype == MD_T_F32)
        hipLaunchKernelGGL((qk_norm_append_kernel<float>), grid, dim3(256), 0, (hipStream_t)stream, p, (float*)q_out);
    else
        hipLaunchKernelGGL((qk_norm_append_kernel<bf16_t>), grid, dim3(256), 0, (hipStream_t)stream, p, (bf16_t*)q_out);
    MD_CHECK_LAUNCH("md_qk_norm_append");
    return MD_OK;
}

extern "C" int md_xattn(const md_xattn_args* a, md_stream_t stream) {
    const int rc0 = check_args("md_xattn", a);
    if (rc0 != MD_OK) return rc0;
    MD_CHECK_ARG(a->out && (a->q || a->qkv), "md_xattn: null pointer argument");
    hipStream_t st = (hipStream_t)stream;
    XattnParams p = make_params(a);
    const bool fused = !a->q;
    MD_CHECK_ARG(!fused || md_xattn_fused_supported(a), "md_xattn: normalise + append inside the attention is not supported "
                 "for this shape (md_xattn_fused_supported)");
    if (fused) {
        MD_CHECK_ARG(((uintptr_t)a->qkv & 15) == 0 && a->ld_qkv % 8 == 0 && p.overflow,
                     "md_xattn: projection rows must be 16-byte aligned");
    }
    const int rows = decode_rows(a), pairs8 = (a->B * a->KH + 7) / 8 * 8;
    int nw = 0;                                   // prefill: wavefronts per workgroup (0: its bias table does not fit)
    if (mfma_ok(a) && rows > 32) {
#define MD_XW(DK) case DK: nw = md_internal_xattn_waves_##DK(p.DVp, p.g, rows); break;
        switch (p.DKp) { MD_XW(32) MD_XW(64) MD_XW(96) MD_XW(128) MD_XW(192) default: nw = md_internal_xattn_waves_256(p.DVp, p.g, rows); }
#undef MD_XW
    }
    if (!mfma_ok(a) || a->force_plain || (rows > 32 && nw == 0)) {
        MD_CHECK_ARG(!fused, "md_xattn: the plain kernel takes normalised queries");
        return md_internal_xattn_plain(p, a->dtype, st);
    }
    int rc;
    if (rows <= 32) {
        p.nsplit = decode_splits(a);
        p.rows_cap = rows <= 16 ? 16 : 32;
        if (p.nsplit > 1) {
            MD_CHECK_ARG(a->workspace && a->workspace_bytes >= md_xattn_workspace_bytes(a) && ((uintptr_t)a->workspace & 15) == 0,
                         "md_xattn: workspace of %zu bytes needed, got %zu", md_xattn_workspace_bytes(a), a->workspace_bytes);
            p.ws = (float*)a->workspace;
        }
        const int qt = rows <= 16 ? 1 : 2, grid = pairs8 * p.nsplit;
#define MD_XD(DK) case DK: rc = md_internal_xattn_decode_##DK(p, qt, fused, grid, st); break;
        switch (p.DKp) { MD_XD(32) MD_XD(64) MD_XD(96) MD_XD(128) MD_XD(192) default: rc = md_internal_xattn_decode_256(p, qt, fused, grid, st); }
#undef MD_XD
        if (rc != MD_OK) return rc;
        if (p.nsplit > 1) {
            const int64_t threads = (int64_t)a->B * a->KH * p.rows_cap * (p.DVp / 4);
            hipLaunchKernelGGL(xattn_merge_kernel, dim3((unsigned)((threads + 255) / 256)), dim3(256), 0, st, p);
        }
    } else {
        p.n_qgroups = (rows + 32 * nw - 1) / (32 * nw);
        const int grid = pairs8 * p.n_qgroups;
#define MD_XP(DK) case DK: rc = md_internal_xattn_prefill_##DK(p, nw, grid, st); break;
        switch (p.DKp) { MD_XP(32) MD_XP(64) MD_XP(96) MD_XP(128) MD_XP(192) default: rc = md_internal_xattn_prefill_256(p, nw, grid, st); }
#undef MD_XP
        if (rc != MD_OK) return rc;
    }
    MD_CHECK_LAUNCH("md_xattn");
    return MD_OK;
}
