// Kernels of latent.h.
#include <algorithm>

#include "bf16.hip.h"
#include "latent.h"
#include "partials.hip.h"

namespace {

struct LArgs {
    LatentShape l;
    const float* x;
    uint64_t ld;
    uint32_t n, start, kp, rank_p, dim_p, row, rot_p;
    void *cache, *q, *qn;
    bool whole;               // query heads start 16-byte aligned and their unrotated part is in whole eights
    const __bf16* w;          // step: per-head matrices
    uint32_t slices, rows;    // step: workgroups and rows per head
    SAttnPartials parts;
    void* out;
};

// entry c of a rotated part at `pos`
__device__ __forceinline__ float rotated(const LatentShape& l, const float* x, uint32_t c, uint32_t pos) {
    if (c >= l.rot_dims) return x[c];
    const float* const cs = l.rot_table + static_cast<uint64_t>(pos) * l.rot_dims + (c & ~1u);
    const float u = x[c & ~1u], v = x[c | 1u];
    return c & 1 ? v * cs[0] + u * cs[1] : u * cs[0] - v * cs[1];
}
// by one wavefront: the cache row of a token
template <typename T> __device__ __forceinline__ void latent_append(const LArgs& a, const float* down, uint32_t pos, uint32_t lane) {
    const LatentShape& l = a.l;
    T* const dst = static_cast<T*>(a.cache) + static_cast<uint64_t>(pos) * a.row;
    float ss = 0.0f;
    for (uint32_t c = lane; c < l.rank; c += 64) ss = fmaf(down[c], down[c], ss);
    const float inv = 1.0f / sqrtf(wave_sum(ss) / static_cast<float>(l.rank) + l.eps);
    for (uint32_t c = lane; c < a.rank_p; c += 64) dst[c] = ElemOps<T>::from(c < l.rank ? down[c] * inv * l.c_norm[c] : 0.0f);
    for (uint32_t c = lane; c < a.row - a.rank_p; c += 64)
        dst[a.rank_p + c] = ElemOps<T>::from(c < l.rot_dim ? rotated(l, down + l.rank, c, pos) : 0.0f);
}

// sixteen lanes per query head, eight entries each at a time, and a wavefront for the cache row
template <typename T> __global__ __launch_bounds__(256) void latent_prep_kernel(LArgs a) {
    const LatentShape& l = a.l;
    const uint32_t lane = threadIdx.x & 63, l8 = (lane & 15) * 8, item = blockIdx.x * 16 + (threadIdx.x >> 4), tok = blockIdx.y, pos = a.start + tok;
    const float* const row = a.x + tok * a.ld;
    if (blockIdx.x == gridDim.x - 1) {
        if (threadIdx.x < 64) latent_append<T>(a, row + l.heads * (l.dim + l.rot_dim), pos, lane);
        return;
    }
    if (item >= l.heads) return;
    const float* const x = row + item * (l.dim + l.rot_dim);
    T* const q = static_cast<T*>(a.q) + (static_cast<uint64_t>(tok) * l.heads + item) * a.kp;
    float v[8];
    // unrotated entries: whole eights, but in front of the rotated ones the last few one by one
    T* const un = a.qn ? static_cast<T*>(a.qn) + (static_cast<uint64_t>(tok) * l.heads + item) * a.dim_p : q;
    for (uint32_t c = l8; c < (a.qn ? a.dim_p : l.dim); c += 128) {
        load8(x, c, l.dim, a.whole, v);
        if (a.qn || c + 8 <= l.dim) ElemOps<T>::store8(un + c, v);
        else
            for (uint32_t i = 0; c + i < l.dim; ++i) un[c + i] = ElemOps<T>::from(x[c + i]);
    }
    const uint32_t at = a.qn ? a.rank_p : l.dim;
    for (uint32_t c = lane & 15; at + c < a.kp; c += 16) q[at + c] = ElemOps<T>::from(c < l.rot_dim ? rotated(l, x + l.dim, c, pos) : 0.0f);
}

// What the products leave open of the expanded rows, eight columns per thread: from `dim` (c0 eights) to the values, from
// the values' end (c1 eights) to the row's end, and whole rows behind the last position.
struct SpreadArgs {
    const void* cache;
    void* rows;
    uint32_t cache_row, rank_p, rot_dim, dim, vdim, v_off, row, total, to, cap;
    uint32_t c0, c1, open;    // open: eights per live row
    bool whole;               // dim and rot_dim come in whole eights
};
template <typename T> __global__ __launch_bounds__(256) void latent_spread_kernel(SpreadArgs a) {
    const uint32_t i = blockIdx.x * 256 + threadIdx.x, live = a.total * a.open, eights = a.row / 8;
    uint32_t pos, c;
    if (i < live) {
        pos = i / a.open;
        const uint32_t e = i - pos * a.open, front = a.v_off / 8 - a.c0;
        c = (e < front ? a.c0 + e : a.c1 + e - front) * 8;
    } else {
        pos = a.total + (i - live) / eights;
        c = (i - live) % eights * 8;
    }
    if (pos >= a.to) return;
    T* const dst = static_cast<T*>(a.rows) + (static_cast<uint64_t>(blockIdx.y) * a.cap + pos) * a.row + c;
    const T* const kr = static_cast<const T*>(a.cache) + static_cast<uint64_t>(pos) * a.cache_row + a.rank_p;
    float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (i < live && a.whole && c < a.dim + a.rot_dim) {
        typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
        const u32x4* const from = reinterpret_cast<const u32x4*>(kr + (c - a.dim));
#pragma unroll
        for (uint32_t k = 0; k < sizeof(T) / 2; ++k) reinterpret_cast<u32x4*>(dst)[k] = from[k];
    } else if (i < live && (c < a.dim + a.rot_dim || (c >= a.v_off && c < a.v_off + a.vdim))) {   // beside or among the products' columns
        for (uint32_t k = c; k < c + 8; ++k)
            if (k >= a.dim && (k < a.v_off || k >= a.v_off + a.vdim)) dst[k - c] = k < a.dim + a.rot_dim ? kr[k - a.dim] : ElemOps<T>::from(0.0f);
    } else {
        ElemOps<T>::store8(dst, v);
    }
}

// y[r] = w[r] . xs for rows r0 + 4 j + (lane / 16) of a matrix with k columns (a multiple of 64): sixteen lanes per row
template <typename T> __device__ __forceinline__ float head_row_dot(const __bf16* w, uint64_t row, uint32_t k, const T* xs, uint32_t l16) {
    const __bf16* const p = w + row * k;
    float acc = 0.0f;
#pragma unroll 4
    for (uint32_t c = l16 * 8; c < k; c += 128) acc = ElemOps<T>::dot8(*reinterpret_cast<const uint4*>(p + c), ElemOps<T>::ld8(xs + c), acc);
    return wave_row_sum(acc);
}

// workgroups (head, slice of the rank); the last one appends
template <typename T> __global__ __launch_bounds__(256) void latent_step_kernel(LArgs a) {
    extern __shared__ __align__(16) unsigned char smem[];
    T* const xs = reinterpret_cast<T*>(smem);
    const LatentShape& l = a.l;
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    if (blockIdx.x == l.heads * a.slices) {
        if (wave == 0) latent_append<T>(a, a.x + l.heads * (l.dim + l.rot_dim), a.start, lane);
        return;
    }
    const uint32_t head = blockIdx.x / a.slices, slice = blockIdx.x % a.slices;
    const float* const x = a.x + head * (l.dim + l.rot_dim);
    T* const q = static_cast<T*>(a.q) + static_cast<uint64_t>(head) * a.kp;
    for (uint32_t c = threadIdx.x; c < a.dim_p; c += 256) xs[c] = ElemOps<T>::from(c < l.dim ? x[c] : 0.0f);
    if (slice == 0)
        for (uint32_t c = threadIdx.x; a.rank_p + c < a.kp; c += 256)
            q[a.rank_p + c] = ElemOps<T>::from(c < l.rot_dim ? rotated(l, x + l.dim, c, a.start) : 0.0f);
    __syncthreads();
    const uint32_t r0 = slice * a.rows, r1 = min(r0 + a.rows, a.rank_p);
    for (uint32_t r = r0 + wave * 4 + (lane >> 4); r < r1; r += 16) {   // row counts are multiples of 4: the lanes of a row stay together
        const float y = head_row_dot<T>(a.w, static_cast<uint64_t>(head) * a.rank_p + r, a.dim_p, xs, lane & 15);
        if ((lane & 15) == 0) q[r] = ElemOps<T>::from(y);
    }
}

// workgroups (head, slice of its values)
template <typename T> __global__ __launch_bounds__(256) void latent_values_kernel(LArgs a) {
    extern __shared__ __align__(16) unsigned char smem[];
    T* const xs = reinterpret_cast<T*>(smem);
    const LatentShape& l = a.l;
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6, head = blockIdx.x / a.slices, slice = blockIdx.x % a.slices;
    if (a.parts.part) {
        __shared__ float wz[LATENT_PARTS];
        partials_weights(a.parts, head, 1, threadIdx.x, 256, wz);
        __syncthreads();
        for (uint32_t c = threadIdx.x * 4; c < a.rank_p; c += 1024) {
            const f32x4 s = partials_sum4(a.parts, wz, head, c);
            ElemOps<T>::store4(xs + c, s.x, s.y, s.z, s.w);
        }
    } else {
        const T* const x = static_cast<const T*>(a.q) + static_cast<uint64_t>(head) * a.rank_p;
        for (uint32_t c = threadIdx.x; c < a.rank_p; c += 256) xs[c] = x[c];
    }
    __syncthreads();
    const uint32_t r0 = slice * a.rows, r1 = min(r0 + a.rows, l.vdim);
    for (uint32_t rb = r0 + wave * 4; rb < r1; rb += 16) {
        const uint32_t r = rb + (lane >> 4);
        const float y = head_row_dot<T>(a.w, static_cast<uint64_t>(head) * l.vdim + min(r, l.vdim - 1), a.rank_p, xs, lane & 15);
        if ((lane & 15) == 0 && r < r1) static_cast<T*>(a.out)[head * l.vdim + r] = ElemOps<T>::from(y);
    }
}

LArgs fill(const LatentShape& l, const FAttnShape& s) {
    LArgs a{};
    a.l = l;
    a.rank_p = l.rank_p(); a.dim_p = l.dim_p(); a.row = s.row; a.kp = s.kp;
    return a;
}
// rows per workgroup so that the heads' products spread over about two workgroups per CU
void slice_rows(cera_hip_ctx* ctx, LArgs& a, uint32_t heads, uint32_t rows) {
    const uint32_t want = std::max(1u, 2 * ctx->n_cu / heads);
    a.rows = std::max(16u, fattn_pad((rows + want - 1) / want, 16));
    a.slices = (rows + a.rows - 1) / a.rows;
}

}  // namespace

cera_hip_status cera_launch_latent_prep(cera_hip_ctx* ctx, const LatentShape& l, const FAttnShape& absorbed, const float* x, uint64_t ld, uint32_t n,
                                        uint32_t start, void* cache, void* q, uint32_t kp, void* qn, bool f32) {
    LArgs a = fill(l, absorbed);
    a.x = x; a.ld = ld; a.n = n; a.start = start; a.cache = cache; a.q = q; a.qn = qn; a.kp = kp;
    a.whole = l.dim % 8 == 0 && l.rot_dim % 4 == 0 && ld % 4 == 0;
    const dim3 grid((l.heads + 15) / 16 + 1, n);
    if (f32) hipLaunchKernelGGL(latent_prep_kernel<float>, grid, dim3(256), 0, ctx->stream, a);
    else hipLaunchKernelGGL(latent_prep_kernel<__bf16>, grid, dim3(256), 0, ctx->stream, a);
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}

cera_hip_status cera_launch_latent_spread(cera_hip_ctx* ctx, const LatentShape& l, const FAttnShape& absorbed, const FAttnShape& expanded,
                                          const void* cache, uint32_t total, void* rows, uint32_t cap, bool f32) {
    const uint32_t to = fattn_pad(total, FATTN_CAP_STEP);
    if (to > cap) return cera_fail(ctx, CERA_HIP_ERR_POSITION, "latent attention: positions beyond the expanded rows");
    SpreadArgs a{};
    a.cache = cache; a.rows = rows; a.cache_row = absorbed.row; a.rank_p = l.rank_p(); a.rot_dim = l.rot_dim; a.dim = l.dim; a.vdim = l.vdim;
    a.v_off = expanded.v_off; a.row = expanded.row; a.total = total; a.to = to; a.cap = cap;
    a.c0 = l.dim / 8; a.c1 = (expanded.v_off + l.vdim) / 8; a.open = expanded.v_off / 8 - a.c0 + expanded.row / 8 - a.c1;
    a.whole = l.dim % 8 == 0 && l.rot_dim % 8 == 0;
    const uint64_t threads = static_cast<uint64_t>(total) * a.open + static_cast<uint64_t>(to - total) * (a.row / 8);
    if (threads > UINT32_MAX - 256) return cera_fail(ctx, CERA_HIP_ERR_POSITION, "latent attention: too many positions to expand");
    const dim3 grid(static_cast<uint32_t>((threads + 255) / 256), l.heads);
    auto go = [&](auto tag) { hipLaunchKernelGGL(latent_spread_kernel<decltype(tag)>, grid, dim3(256), 0, ctx->stream, a); };
    if (f32) go(float{});
    else go(static_cast<__bf16>(0.0f));
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}

cera_hip_status cera_launch_latent_step(cera_hip_ctx* ctx, const LatentShape& l, const FAttnShape& absorbed, const DenseMat& wk, const float* x,
                                        uint32_t pos, void* cache, void* q, bool f32) {
    LArgs a = fill(l, absorbed);
    a.x = x; a.start = pos; a.cache = cache; a.q = q; a.w = static_cast<const __bf16*>(wk.w);
    if (wk.rows != l.heads * a.rank_p || wk.kp != a.dim_p) return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "latent step: key matrix shape");
    slice_rows(ctx, a, l.heads, a.rank_p);
    const dim3 grid(l.heads * a.slices + 1);
    if (f32) hipLaunchKernelGGL(latent_step_kernel<float>, grid, dim3(256), a.dim_p * 4, ctx->stream, a);
    else hipLaunchKernelGGL(latent_step_kernel<__bf16>, grid, dim3(256), a.dim_p * 2, ctx->stream, a);
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}

cera_hip_status cera_launch_latent_values(cera_hip_ctx* ctx, const LatentShape& l, const DenseMat& wv, const SAttnPartials& parts, const void* merged,
                                          void* out, bool f32) {
    LArgs a{};
    a.l = l; a.rank_p = l.rank_p(); a.parts = parts; a.q = const_cast<void*>(merged); a.out = out; a.w = static_cast<const __bf16*>(wv.w);
    if (wv.rows != l.heads * l.vdim || wv.kp != a.rank_p ||
        (parts.part ? parts.vdim_p != a.rank_p || parts.heads != l.heads || parts.splits > LATENT_PARTS : !merged))
        return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "latent values: matrix or partial results do not fit");
    slice_rows(ctx, a, l.heads, l.vdim);
    const dim3 grid(l.heads * a.slices);
    if (f32) hipLaunchKernelGGL(latent_values_kernel<float>, grid, dim3(256), a.rank_p * 4, ctx->stream, a);
    else hipLaunchKernelGGL(latent_values_kernel<__bf16>, grid, dim3(256), a.rank_p * 2, ctx->stream, a);
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}
