// Matrix products on bfloat16 weights (dense.h).
//
// GEMM: tiles of weight rows x tokens, K in steps of 64 through two LDS buffers filled by direct
// global-to-LDS loads (a 16-byte chunk c of row r sits in slot c ^ (r & 7) of its row, so the
// fragment reads spread over the banks), v_mfma_f32_16x16x32_bf16 with the weight rows as the A
// operand: a lane then holds four consecutive output rows of one token, which the epilogue stores
// as one vector.  The f32 variant stages both operands as f32 and runs on v_mfma_f32_16x16x4_f32.
//
// GEMV: a wavefront streams up to four rows at a time, 16 bytes per lane per row and step, against the
// activation vector in LDS; the workgroup prepares that vector itself (row norm, convolution of the
// current token, concatenation), so those need no launch of their own.
#include <algorithm>

#include "bf16.hip.h"
#include "dense.h"
#include "partials.hip.h"

namespace {

struct GemmDArgs {
    const __bf16* w;
    const void* x;
    uint64_t ldx;
    uint32_t m, n, kp, k_chunk;
    uint32_t tiles_m, tiles_n;
    int epi;
    void* out;
    uint64_t ldo;
    const float* bias;
    float mult;
    uint32_t out_rows;
    float* part;           // split K: [split][n][m] f32
    uint32_t groups;
    uint64_t gw, gx, go;   // between the groups: elements of their matrices and inputs, bytes of their outputs
    bool vec;              // four outputs of a token in a row may be stored as one vector
    float* u;
    DenseStreams st;
};

// four consecutive channels of every stream (n < 4: the first n of them).  S: the number of streams, 0: any, at run time
template <int SN> __device__ __forceinline__ void dense_streams4(const DenseStreams& st, float* x, float* u, bool vec, int n, const float (&y)[4]) {
    constexpr int S = SN ? SN : static_cast<int>(DENSE_MAX_STREAMS);
    float o[S][4];
#pragma unroll
    for (int s = 0; s < S; ++s)
        if (SN || s < static_cast<int>(st.count)) {
            float* const p = x + s * st.stride;
            if (vec) {
                const float4 v = *reinterpret_cast<const float4*>(p);
                o[s][0] = v.x; o[s][1] = v.y; o[s][2] = v.z; o[s][3] = v.w;
            } else {
#pragma unroll
                for (int i = 0; i < 4; ++i) o[s][i] = i < n ? p[i] : 0.0f;
            }
        }
    float sum[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < S; ++t)
        if (SN || t < static_cast<int>(st.count)) {
            float v[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                v[i] = st.out[t] * y[i];
#pragma unroll
                for (int s = 0; s < S; ++s)
                    if (SN || s < static_cast<int>(st.count)) v[i] = fmaf(st.mix[s][t], o[s][i], v[i]);
                sum[i] = fmaf(st.next[t], v[i], sum[i]);
            }
            float* const p = x + t * st.stride;
            if (vec) *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
            else
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (i < n) p[i] = v[i];
        }
    if (vec) *reinterpret_cast<float4*>(u) = make_float4(sum[0], sum[1], sum[2], sum[3]);
    else
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (i < n) u[i] = sum[i];
}
// one channel of every stream
template <int SN> __device__ __forceinline__ void dense_streams1(const DenseStreams& st, float* x, float* u, float y) {
    constexpr int S = SN ? SN : static_cast<int>(DENSE_MAX_STREAMS);
    float o[S], sum = 0.0f;
#pragma unroll
    for (int s = 0; s < S; ++s)
        if (SN || s < static_cast<int>(st.count)) o[s] = x[s * st.stride];
#pragma unroll
    for (int t = 0; t < S; ++t)
        if (SN || t < static_cast<int>(st.count)) {
            float v = st.out[t] * y;
#pragma unroll
            for (int s = 0; s < S; ++s)
                if (SN || s < static_cast<int>(st.count)) v = fmaf(st.mix[s][t], o[s], v);
            x[t * st.stride] = v;
            sum = fmaf(st.next[t], v, sum);
        }
    *u = sum;
}
__device__ __forceinline__ float dense_relu2(float y) {
    const float r = fmaxf(y, 0.0f);
    return r * r;
}

// ---- epilogues on four consecutive rows m .. m+3 of one token -----------------------------------
// EPI: a DenseEpilogue; SN: of DENSE_STREAMS
template <typename T, int EPI, int SN> __device__ __forceinline__ void dense_store4(const GemmDArgs& a, uint32_t row, uint32_t tok, f32x4 v) {
    const uint64_t at = static_cast<uint64_t>(tok) * a.ldo + row;
    if constexpr (EPI == DENSE_STORE) {
        float* o = static_cast<float*>(a.out) + at;
        if (row + 4 <= a.m && a.vec) {
            if (a.bias) {
                const float4 b = *reinterpret_cast<const float4*>(a.bias + row);
                v.x += b.x; v.y += b.y; v.z += b.z; v.w += b.w;
            }
            *reinterpret_cast<float4*>(o) = make_float4(v.x, v.y, v.z, v.w);
        } else {
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (row + i < a.m) o[i] = a.bias ? v[i] + a.bias[row + i] : v[i];
        }
    } else if constexpr (EPI == DENSE_CAST || EPI == DENSE_RELU2) {
        T* o = static_cast<T*>(a.out) + at;
        if (EPI == DENSE_RELU2) { v.x = dense_relu2(v.x); v.y = dense_relu2(v.y); v.z = dense_relu2(v.z); v.w = dense_relu2(v.w); }
        if (row + 4 <= a.m && a.vec) {
            ElemOps<T>::store4(o, v.x, v.y, v.z, v.w);
        } else {
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (row + i < a.m) o[i] = ElemOps<T>::from(v[i]);
        }
    } else if constexpr (EPI == DENSE_STREAMS) {
        const float y[4] = {v.x, v.y, v.z, v.w};
        float* const x = static_cast<float*>(a.out) + at;
        const int n = static_cast<int>(min(4u, a.m - row));
        dense_streams4<SN>(a.st, x, a.u + at, n == 4 && a.vec, n, y);
    } else {
        float* o = static_cast<float*>(a.out) + at;
        if (row + 4 <= a.m && a.vec) {
            float4 r = *reinterpret_cast<const float4*>(o);
            r.x = fmaf(a.mult, v.x, r.x); r.y = fmaf(a.mult, v.y, r.y);
            r.z = fmaf(a.mult, v.z, r.z); r.w = fmaf(a.mult, v.w, r.w);
            *reinterpret_cast<float4*>(o) = r;
        } else {
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (row + i < a.m) o[i] = fmaf(a.mult, v[i], o[i]);
        }
    }
}
__device__ __forceinline__ float dense_silu_mul(float g, float u) { return g * sigmoid_f32(g) * u; }
// rows grow .. grow+3 of a gate group; i0 = their index among the outputs
template <typename T>
__device__ __forceinline__ void dense_swiglu4(const GemmDArgs& a, uint32_t i0, uint32_t tok, f32x4 g, f32x4 u) {
    T* o = static_cast<T*>(a.out) + static_cast<uint64_t>(tok) * a.ldo + i0;
    const float r0 = dense_silu_mul(g.x, u.x), r1 = dense_silu_mul(g.y, u.y), r2 = dense_silu_mul(g.z, u.z), r3 = dense_silu_mul(g.w, u.w);
    if (i0 + 4 <= a.out_rows && (a.ldo & 3) == 0) {
        ElemOps<T>::store4(o, r0, r1, r2, r3);
    } else {
        const float r[4] = {r0, r1, r2, r3};
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (i0 + i < a.out_rows) o[i] = ElemOps<T>::from(r[i]);
    }
}
// one wavefront's tile: acc[mi][ni], rows m0 + 16 mi + 4 (lane / 16) + i, token n0 + 16 ni + lane % 16
template <typename T, int EPI, int SN, int MI, int NI>
__device__ __forceinline__ void dense_epilogue(const GemmDArgs& a, uint32_t m0, uint32_t n0, uint32_t lane, uint32_t z,
                                               f32x4 (&acc)[MI][NI]) {
    const uint32_t g4 = (lane >> 4) * 4;
#pragma unroll
    for (int ni = 0; ni < NI; ++ni) {
        const uint32_t tok = n0 + 16 * ni + (lane & 15);
        if (tok >= a.n) continue;
        if (a.part) {
            float* p = a.part + (static_cast<uint64_t>(z) * a.n + tok) * a.m;
#pragma unroll
            for (int mi = 0; mi < MI; ++mi) {
                const uint32_t row = m0 + 16 * mi + g4;
                if (row + 4 <= a.m && (a.m & 3) == 0) *reinterpret_cast<f32x4*>(p + row) = acc[mi][ni];
                else
#pragma unroll
                    for (int i = 0; i < 4; ++i)
                        if (row + i < a.m) p[row + i] = acc[mi][ni][i];
            }
        } else if constexpr (EPI == DENSE_SWIGLU) {
            static_assert(MI % 2 == 0, "a wavefront holds gate rows with their up rows");
#pragma unroll
            for (int mi = 0; mi < MI; mi += 2) {
                const uint32_t row = m0 + 16 * mi;
                if (row < a.m) dense_swiglu4<T>(a, row / 2 + g4, tok, acc[mi][ni], acc[mi + 1][ni]);
            }
        } else {
#pragma unroll
            for (int mi = 0; mi < MI; ++mi) {
                const uint32_t row = m0 + 16 * mi + g4;
                if (row < a.m) dense_store4<T, EPI, SN>(a, row, tok, acc[mi][ni]);
            }
        }
    }
}

// Workgroups go to the eight XCDs round robin in launch order; the token tiles of one weight tile (of one group)
// take indices 8 apart, so one XCD's L2 reads that weight tile for all of them.
__device__ __forceinline__ bool dense_tile(const GemmDArgs& a, uint32_t& tm, uint32_t& tn, uint32_t& group) {
    const uint32_t b = blockIdx.x, xcd = b & 7, t = b >> 3;
    tn = t % a.tiles_n;
    const uint32_t i = (t / a.tiles_n) * 8 + xcd;
    group = a.groups > 1 ? i / a.tiles_m : 0;
    tm = i - group * a.tiles_m;
    return i < a.tiles_m * a.groups;
}

// BM x BN tile, four wavefronts as WM x WN
template <int EPI, int SN, int BM, int BN, int WM, int WN>
__global__ __launch_bounds__(256) void dense_gemm_bf16_kernel(GemmDArgs a) {
    constexpr int BK = 64, TM = BM / WM, TN = BN / WN, MI = TM / 16, NI = TN / 16;
    constexpr int SEGS = (BM + BN) / 8;   // 1 KB pieces: eight rows of one K step
    static_assert(WM * WN == 4 && SEGS % 4 == 0 && MI >= 1 && NI >= 1, "tile shape");
    __shared__ __align__(1024) __bf16 lds[2][(BM + BN) * BK];
    uint32_t tm, tn, group;
    if (!dense_tile(a, tm, tn, group)) return;
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const uint32_t k0 = blockIdx.y * a.k_chunk, k1 = min(a.kp, k0 + a.k_chunk);
    const __bf16* const w = a.w + group * a.gw;
    const __bf16* const x = static_cast<const __bf16*>(a.x) + group * a.gx;
    // this lane's source address per 1 KB piece; rows past the matrix / batch re-read the last one
    const uint32_t sub = lane >> 3, slot = lane & 7, chunk = (slot ^ sub) * 8;
    const __bf16* src[SEGS / 4];
#pragma unroll
    for (int s = 0; s < SEGS / 4; ++s) {
        const uint32_t r = (wave * (SEGS / 4) + s) * 8 + sub;
        src[s] = r < BM ? w + static_cast<uint64_t>(min(tm * BM + r, a.m - 1)) * a.kp + chunk
                        : x + static_cast<uint64_t>(min(tn * BN + (r - BM), a.n - 1)) * a.ldx + chunk;
    }
    auto stage = [&](uint32_t k, int buf) {
#pragma unroll
        for (int s = 0; s < SEGS / 4; ++s) {
            __bf16* dst = &lds[buf][(wave * (SEGS / 4) + s) * 8 * BK];   // wavefront-uniform; lane i lands 16 i bytes on
            __builtin_amdgcn_global_load_lds(reinterpret_cast<const __attribute__((address_space(1))) void*>(reinterpret_cast<uintptr_t>(src[s] + k)),
                                             (__attribute__((address_space(3))) void*)dst, 16, 0, 0);
        }
    };
    f32x4 acc[MI][NI];
#pragma unroll
    for (int mi = 0; mi < MI; ++mi)
#pragma unroll
        for (int ni = 0; ni < NI; ++ni) acc[mi][ni] = f32x4{0.f, 0.f, 0.f, 0.f};
    const uint32_t wm = wave / WN, wn = wave % WN, fr = lane & 15, fg = lane >> 4;
    stage(k0, 0);
    int buf = 0;
    for (uint32_t k = k0; k < k1; k += BK, buf ^= 1) {
        // this step's pieces are in, and every wavefront is past its reads of the other buffer
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
        if (k + BK < k1) stage(k + BK, buf ^ 1);
        const __bf16* const aw = &lds[buf][(wm * TM + fr) * BK];
        const __bf16* const bx = &lds[buf][(BM + wn * TN + fr) * BK];
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
            const uint32_t off = ((kk * 4 + fg) ^ (fr & 7)) * 8;
            bf16x8 fa[MI], fb[NI];
#pragma unroll
            for (int mi = 0; mi < MI; ++mi) fa[mi] = *reinterpret_cast<const bf16x8*>(aw + mi * 16 * BK + off);
#pragma unroll
            for (int ni = 0; ni < NI; ++ni) fb[ni] = *reinterpret_cast<const bf16x8*>(bx + ni * 16 * BK + off);
#pragma unroll
            for (int mi = 0; mi < MI; ++mi)
#pragma unroll
                for (int ni = 0; ni < NI; ++ni)
                    acc[mi][ni] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fa[mi], fb[ni], acc[mi][ni], 0, 0, 0);
        }
    }
    a.out = static_cast<char*>(a.out) + group * a.go;
    dense_epilogue<__bf16, EPI, SN, MI, NI>(a, tm * BM + wm * TM, tn * BN + wn * TN, lane, blockIdx.y, acc);
}

// 64 x 64 tile in true f32: weights widened on their way into LDS, K in steps of 32.  A lane's four
// consecutive k of a 16-wide block feed four MFMA steps (the same k order in both operands).
template <int EPI, int SN> __global__ __launch_bounds__(256) void dense_gemm_f32_kernel(GemmDArgs a) {
    constexpr int BM = 64, BN = 64, BK = 32, LD = BK + 4;
    __shared__ __align__(16) float lw[BM * LD], lx[BN * LD];
    uint32_t tm, tn, group;
    if (!dense_tile(a, tm, tn, group)) return;
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const uint32_t k0 = blockIdx.y * a.k_chunk, k1 = min(a.kp, k0 + a.k_chunk);
    const __bf16* const w0 = a.w + group * a.gw;
    const float* const x = static_cast<const float*>(a.x) + group * a.gx;
    const uint32_t r = threadIdx.x >> 2, c = (threadIdx.x & 3) * 8;   // eight k of one row per thread
    const __bf16* const ws = w0 + static_cast<uint64_t>(min(tm * BM + r, a.m - 1)) * a.kp + c;
    const float* const xs = x + static_cast<uint64_t>(min(tn * BN + r, a.n - 1)) * a.ldx + c;
    f32x4 acc[2][2];
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    const uint32_t wm = wave >> 1, wn = wave & 1, fr = lane & 15, fg = lane >> 4;
    for (uint32_t k = k0; k < k1; k += BK) {
        const uint4 w = *reinterpret_cast<const uint4*>(ws + k);
        const float4 xa = *reinterpret_cast<const float4*>(xs + k), xb = *reinterpret_cast<const float4*>(xs + k + 4);
        __syncthreads();
        *reinterpret_cast<float4*>(lw + r * LD + c) = make_float4(bf16_lo(w.x), bf16_hi(w.x), bf16_lo(w.y), bf16_hi(w.y));
        *reinterpret_cast<float4*>(lw + r * LD + c + 4) = make_float4(bf16_lo(w.z), bf16_hi(w.z), bf16_lo(w.w), bf16_hi(w.w));
        *reinterpret_cast<float4*>(lx + r * LD + c) = xa;
        *reinterpret_cast<float4*>(lx + r * LD + c + 4) = xb;
        __syncthreads();
#pragma unroll
        for (int kb = 0; kb < BK; kb += 16) {
            f32x4 fa[2], fb[2];
#pragma unroll
            for (int i = 0; i < 2; ++i) {
                fa[i] = *reinterpret_cast<const f32x4*>(lw + (wm * 32 + i * 16 + fr) * LD + kb + fg * 4);
                fb[i] = *reinterpret_cast<const f32x4*>(lx + (wn * 32 + i * 16 + fr) * LD + kb + fg * 4);
            }
#pragma unroll
            for (int s = 0; s < 4; ++s)
#pragma unroll
                for (int i = 0; i < 2; ++i)
#pragma unroll
                    for (int j = 0; j < 2; ++j)
                        acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(fa[i][s], fb[j][s], acc[i][j], 0, 0, 0);
        }
    }
    a.out = static_cast<char*>(a.out) + group * a.go;
    dense_epilogue<float, EPI, SN, 2, 2>(a, tm * BM + wm * 32, tn * BN + wn * 32, lane, blockIdx.y, acc);
}

// split K: adds the partial sums in split order, then the epilogue.  One thread per four rows of a token
// (SWIGLU: per four outputs).
template <typename T, int EPI, int SN>
__global__ __launch_bounds__(256) void dense_reduce_kernel(GemmDArgs a, uint32_t split) {
    const uint32_t quads = EPI == DENSE_SWIGLU ? (a.m / 2 + 3) / 4 : (a.m + 3) / 4;
    const uint64_t t = static_cast<uint64_t>(blockIdx.x) * 256 + threadIdx.x;
    if (t >= static_cast<uint64_t>(quads) * a.n) return;
    const uint32_t tok = static_cast<uint32_t>(t / quads), q = static_cast<uint32_t>(t % quads) * 4;
    const uint64_t slice = static_cast<uint64_t>(a.n) * a.m;
    const float* p = a.part + static_cast<uint64_t>(tok) * a.m;
    auto sum4 = [&](uint32_t row) {
        f32x4 v{0.f, 0.f, 0.f, 0.f};
        if ((a.m & 3) == 0) {
#pragma unroll 4
            for (uint32_t z = 0; z < split; ++z) v += *reinterpret_cast<const f32x4*>(p + z * slice + row);
            return v;
        }
        for (uint32_t z = 0; z < split; ++z) {
            const float* s = p + z * slice + row;
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (row + i < a.m) v[i] += s[i];
        }
        return v;
    };
    if constexpr (EPI == DENSE_SWIGLU) {
        const uint32_t row = (q >> 4) * 32 + (q & 15);
        dense_swiglu4<T>(a, q, tok, sum4(row), sum4(row + 16));
    } else {
        dense_store4<T, EPI, SN>(a, q, tok, sum4(q));
    }
}

// ---------------------------------------------------------------------------
struct GemvDArgs {
    DenseIn in;
    const __bf16 *wa, *wb;
    uint32_t rows_a, rows_b, kp, stage_len;   // stage_len: LDS elements, kp rounded up to a whole step of the wavefront
    uint32_t blocks_a, groups_a, groups_b, blocks_b;   // groups of R rows
    DenseOut oa, ob;
    DenseStreams st;
};

constexpr int GEMV_WAVES = 8;
// A wavefront has R rows in flight, U steps of 64 16-byte chunks each: 8 KB per wavefront either way.
template <int R> constexpr int GEMV_U = 8 / R;
template <int R> constexpr uint32_t GEMV_STEP = 64 * 8 * GEMV_U<R>;

// Fills the workgroup's activation vector xs[0, stage_len).
template <typename T, int KIND>
__device__ __forceinline__ void gemv_stage(const GemvDArgs& a, bool second, bool store_h, T* xs, float* red, float* wz) {
    const DenseIn& in = a.in;
    if (KIND == DenseIn::RAW) {
        const T* x = static_cast<const T*>(in.x);
        constexpr uint32_t V = 16 / sizeof(T);
#pragma unroll 4
        for (uint32_t i = threadIdx.x * V; i < a.stage_len; i += GEMV_WAVES * 64 * V)
            *reinterpret_cast<uint4*>(xs + i) = i < a.kp ? *reinterpret_cast<const uint4*>(x + i) : make_uint4(0, 0, 0, 0);
    } else if (KIND == DenseIn::MERGE) {
        const T* x = static_cast<const T*>(in.x);
        const SAttnPartials& m = in.merge;
        const uint32_t cols = m.heads * m.vdim, cols_p = (cols + DENSE_PAD - 1) / DENSE_PAD * DENSE_PAD;
        partials_weights(m, 0, m.heads, threadIdx.x, GEMV_WAVES * 64, wz);
        constexpr uint32_t V = 16 / sizeof(T);
#pragma unroll 4
        for (uint32_t i = cols_p + threadIdx.x * V; i < a.stage_len; i += GEMV_WAVES * 64 * V)
            *reinterpret_cast<uint4*>(xs + i) = i < a.kp ? *reinterpret_cast<const uint4*>(x + i) : make_uint4(0, 0, 0, 0);
        lds_barrier();
#pragma unroll 2
        for (uint32_t i = threadIdx.x * 4; i < cols_p; i += GEMV_WAVES * 256) {
            if (i + 4 <= cols && m.vdim % 4 == 0) {
                const uint32_t h = i / m.vdim;
                const f32x4 s = partials_sum4(m, wz + h * m.splits, h, i - h * m.vdim);
                ElemOps<T>::store4(xs + i, s.x, s.y, s.z, s.w);
            } else {
#pragma unroll
                for (uint32_t e = i; e < i + 4; ++e) {
                    const float s = e < cols ? partials_sum(m, wz + e / m.vdim * m.splits, e / m.vdim, e % m.vdim) : 0.0f;
                    xs[e] = ElemOps<T>::from(s);
                }
            }
        }
    } else if (KIND == DenseIn::CONCAT) {
        const float* x = static_cast<const float*>(in.x);
        const uint32_t half = a.kp / 2;
        for (uint32_t i = threadIdx.x * 4; i < a.stage_len; i += GEMV_WAVES * 256) {
            float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
            if (i < a.kp) v = *reinterpret_cast<const float4*>(i < half ? x + i : in.x2 + (i - half));
            ElemOps<T>::store4(xs + i, v.x, v.y, v.z, v.w);
        }
    } else {
        const float* x = static_cast<const float*>(in.x);
        const float *sc = second ? in.scale_b : in.scale_a, *ad = second ? in.add_b : in.add_a;
        float ss = 0.0f;
        for (uint32_t i = threadIdx.x * 4; i < a.kp; i += GEMV_WAVES * 256) {
            const float4 v = *reinterpret_cast<const float4*>(x + i);
            ss = fmaf(v.x, v.x, ss); ss = fmaf(v.y, v.y, ss); ss = fmaf(v.z, v.z, ss); ss = fmaf(v.w, v.w, ss);
        }
        ss = wave_sum(ss);
        if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
        lds_barrier();
        float tot = 0.0f;
#pragma unroll
        for (int i = 0; i < GEMV_WAVES; ++i) tot += red[i];
        const float inv = 1.0f / sqrtf(tot / static_cast<float>(in.n_mean) + in.eps);
        for (uint32_t i = threadIdx.x * 4; i < a.stage_len; i += GEMV_WAVES * 256) {
            float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
            if (i < a.kp) {
                const float4 v = *reinterpret_cast<const float4*>(x + i), s = *reinterpret_cast<const float4*>(sc + i);
                if (ad) o = *reinterpret_cast<const float4*>(ad + i);
                o.x = fmaf(v.x * inv, s.x, o.x); o.y = fmaf(v.y * inv, s.y, o.y);
                o.z = fmaf(v.z * inv, s.z, o.z); o.w = fmaf(v.w * inv, s.w, o.w);
                if (store_h) {
                    const float4 p = *reinterpret_cast<const float4*>(in.plain + i);
                    *reinterpret_cast<float4*>(in.h_out + i) = make_float4(v.x * inv * p.x, v.y * inv * p.y, v.z * inv * p.z, v.w * inv * p.w);
                }
            }
            ElemOps<T>::store4(xs + i, o.x, o.y, o.z, o.w);
        }
    }
    lds_barrier();
}

// One wavefront's walk over its groups of R rows (g, g + GEMV_WAVES, ... below g1) of one matrix, a step of
// U * 64 16-byte chunks at a time; SWIGLU: a group is R / 2 gate rows and their up rows.  Two step buffers
// alternate, the next step's loads -- of the next group too -- going out before the current one is multiplied.
// SN: streams of the epilogue (0: any number, -1: it is another one)
template <typename T, int R, int SN> struct GemvWalk {
    static constexpr int U = GEMV_U<R>, H = R > 1 ? R / 2 : 1;
    typedef uint4 Buf[U][R];
    const __bf16* w;
    uint32_t rows, kp, stage_len, g1, lane, last;
    bool swiglu;
    uint32_t lg, lk;            // group and step the next load takes
    const __bf16* p[R];
    float acc[R];

    __device__ __forceinline__ void set_rows() {
#pragma unroll
        for (int r = 0; r < R; ++r) {
            uint32_t row = lg * R + r;
            if (swiglu) {
                const uint32_t i = lg * H + r % H;
                row = (i >> 4) * 32 + (i & 15) + (r >= H && R > 1 ? 16 : 0);
            }
            p[r] = w + static_cast<uint64_t>(min(row, rows - 1)) * kp;
        }
    }
    __device__ __forceinline__ void begin(const __bf16* w_, uint32_t rows_, uint32_t kp_, uint32_t stage_len_, bool swiglu_, uint32_t g, uint32_t g1_) {
        w = w_; rows = rows_; kp = kp_; stage_len = stage_len_; swiglu = R > 1 && swiglu_; g1 = g1_;
        lane = threadIdx.x & 63; last = kp / 8 - 1;
        lg = g; lk = 0;
        if (lg < g1) set_rows();
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r] = 0.0f;
    }
    __device__ __forceinline__ bool load(Buf& b) {
        if (lg >= g1) return false;
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int r = 0; r < R; ++r)   // past the row's end: its last chunk again, against zeros
                b[u][r] = ld_u128_nt(p[r] + min(lk / 8 + u * 64 + lane, last) * 8);
        lk += GEMV_STEP<R>;
        if (lk >= stage_len) {
            lk = 0;
            lg += GEMV_WAVES;
            if (lg < g1) set_rows();
        }
        return true;
    }
    // multiplies a step of group g at k; at the group's last step reduces and stores, and moves on
    __device__ __forceinline__ void use(const Buf& b, uint32_t& g, uint32_t& k, const T* xs, const DenseOut& o, const DenseStreams& st) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const typename ElemOps<T>::X8 xv = ElemOps<T>::ld8(xs + k + (u * 64 + lane) * 8);
#pragma unroll
            for (int r = 0; r < R; ++r) acc[r] = ElemOps<T>::dot8(b[u][r], xv, acc[r]);
        }
        k += GEMV_STEP<R>;
        if (k < stage_len) return;
        k = 0;
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r] = wave_sum(acc[r]);
        if (swiglu) {
            const uint32_t i = g * H + lane;
            float gt = acc[0], up = acc[R > 1 ? H : 0];
#pragma unroll
            for (int r = 1; r < H; ++r)
                if (lane == static_cast<uint32_t>(r)) { gt = acc[r]; up = acc[H + r]; }
            if (lane < static_cast<uint32_t>(H) && i < o.rows) static_cast<T*>(o.out)[i] = ElemOps<T>::from(dense_silu_mul(gt, up));
        } else {
            const uint32_t i = g * R + lane;
            float y = acc[0];
#pragma unroll
            for (int r = 1; r < R; ++r)
                if (lane == static_cast<uint32_t>(r)) y = acc[r];
            if (lane < static_cast<uint32_t>(R) && i < rows) {
                float* out = static_cast<float*>(o.out) + i;
                if constexpr (SN >= 0) dense_streams1<SN>(st, out, o.u + i, y);
                else if (o.epi == DENSE_ADD) *out = fmaf(o.mult, y, *out);
                else if (o.epi == DENSE_STORE) *out = o.bias ? y + o.bias[i] : y;
                else static_cast<T*>(o.out)[i] = ElemOps<T>::from(o.epi == DENSE_RELU2 ? dense_relu2(y) : y);
            }
        }
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r] = 0.0f;
        g += GEMV_WAVES;
    }
};

template <typename T, int KIND, int R, int SN>
__global__ __launch_bounds__(GEMV_WAVES * 64) void dense_gemv_kernel(GemvDArgs a) {
    extern __shared__ __align__(16) unsigned char smem[];
    __shared__ float red[GEMV_WAVES], wz[KIND == DenseIn::MERGE ? PARTIALS_MAX : 1];
    T* const xs = reinterpret_cast<T*>(smem);
    const bool second = blockIdx.x >= a.blocks_a;
    const uint32_t groups = second ? a.groups_b : a.groups_a, blocks = second ? a.blocks_b : a.blocks_a;
    const uint32_t b = second ? blockIdx.x - a.blocks_a : blockIdx.x;
    // the first `groups % blocks` workgroups take one group more
    const uint32_t each = groups / blocks, more = groups % blocks;
    const uint32_t g0 = b * each + min(b, more), g1 = g0 + each + (b < more ? 1 : 0);
    const DenseOut& o = second ? a.ob : a.oa;
    GemvWalk<T, R, SN> walk;
    typename GemvWalk<T, R, SN>::Buf w0, w1;
    uint32_t g = g0 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), k = 0;
    walk.begin(second ? a.wb : a.wa, second ? a.rows_b : a.rows_a, a.kp, a.stage_len, o.epi == DENSE_SWIGLU, g, g1);
    // the first weights are on their way while the activation vector is prepared
    bool more0 = walk.load(w0);
    gemv_stage<T, KIND>(a, second, KIND == DenseIn::NORM && a.in.h_out && blockIdx.x == 0, xs, red, wz);
    while (more0) {
        const bool more1 = walk.load(w1);
        walk.use(w0, g, k, xs, o, a.st);
        if (!more1) break;
        more0 = walk.load(w0);
        walk.use(w1, g, k, xs, o, a.st);
    }
}

constexpr uint64_t GEMV_LDS_MAX = 60 * 1024;

}  // namespace

static bool streams_ok(const DenseOut& o) { return o.streams && o.u && o.streams->count >= 1 && o.streams->count <= DENSE_MAX_STREAMS && o.streams->stride % 4 == 0; }
static uint64_t gemv_stage_len(uint64_t kp, int r) {
    const uint64_t step = 64ull * 8 * (8 / r);
    return (kp + step - 1) / step * step;
}
bool cera_dense_gemv_fits(uint64_t kp, bool f32) { return gemv_stage_len(kp, 1) * (f32 ? 4 : 2) <= GEMV_LDS_MAX; }

cera_hip_status cera_launch_dense_gemm(cera_hip_ctx* ctx, const DenseMat& w, const void* x, uint64_t ldx, uint32_t n,
                                       const DenseOut& o, bool f32, const DenseGroups& groups) {
    if (n == 0 || w.rows == 0 || groups.count == 0 || w.rows % groups.count || w.kp == 0 || w.kp % DENSE_PAD || ldx < w.kp || ldx % 8)
        return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "dense_gemm: bad shape");
    if (o.epi == DENSE_SWIGLU && w.rows % 32) return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "dense_gemm: gate | up rows come in groups of 32");
    if (o.epi == DENSE_STREAMS && (!streams_ok(o) || groups.count != 1)) return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "dense_gemm: streams");
    GemmDArgs a{};
    a.w = static_cast<const __bf16*>(w.w); a.x = x; a.ldx = ldx; a.m = w.rows / groups.count; a.n = n; a.kp = w.kp;
    a.gw = static_cast<uint64_t>(a.m) * w.kp; a.groups = groups.count; a.gx = groups.x_stride;
    a.go = groups.out_stride * (f32 || (o.epi != DENSE_CAST && o.epi != DENSE_RELU2 && o.epi != DENSE_SWIGLU) ? 4 : 2);
    a.vec = (o.ld & 3) == 0 && (groups.out_stride & 3) == 0;
    a.u = o.u;
    if (o.streams) a.st = *o.streams;
    a.epi = o.epi; a.out = o.out; a.ldo = o.ld; a.bias = o.bias; a.mult = o.mult; a.out_rows = o.rows;
    // tile: large where it fills the chip, else smaller, else K is split
    int shape = 2;
    uint32_t bm = 64, bn = 32;
    auto count = [&](uint32_t tm, uint32_t tn) { return static_cast<uint64_t>((a.m + tm - 1) / tm) * ((n + tn - 1) / tn) * groups.count; };
    if (f32) { bm = bn = 64; }
    else if (n > 64 && (count(128, 128) >= ctx->n_cu || (a.kp >= 8192 && count(128, 128) * 4 >= ctx->n_cu))) { shape = 0; bm = bn = 128; }
    else if (n > 32) { shape = 1; bm = bn = 64; }
    a.tiles_m = (a.m + bm - 1) / bm;
    a.tiles_n = (n + bn - 1) / bn;
    const uint64_t wgs = count(bm, bn);
    const uint32_t steps = a.kp / DENSE_PAD;
    uint32_t split = 1;
    const uint32_t want_wgs = 2 * ctx->n_cu;
    if (wgs < want_wgs && groups.count == 1) split = static_cast<uint32_t>(std::min<uint64_t>({(want_wgs + wgs - 1) / wgs, steps / 4, 16}));
    if (split < 1) split = 1;
    const uint32_t per = (steps + split - 1) / split;
    split = (steps + per - 1) / per;
    a.k_chunk = per * DENSE_PAD;
    // any number of streams but four: through the reduction, whose threads hold little else
    const bool apart = o.epi == DENSE_STREAMS && o.streams->count != 4;
    if (split > 1 || apart) {
        void* part;
        CERA_TRY(cera_scratch(ctx, 9, static_cast<uint64_t>(split) * n * a.m * sizeof(float), &part));
        a.part = static_cast<float*>(part);
    }
    const dim3 grid((a.tiles_m * groups.count + 7) / 8 * 8 * a.tiles_n, split);
    const uint64_t quads = (a.epi == DENSE_SWIGLU ? (a.m / 2 + 3) / 4 : (a.m + 3) / 4) * static_cast<uint64_t>(n);
    const dim3 rg(static_cast<uint32_t>((quads + 255) / 256)), block(256);
    auto go = [&](auto epi, auto streams) {
        constexpr int E = decltype(epi)::value, SN = decltype(streams)::value;
        constexpr int EG = E == DENSE_STREAMS && SN == 0 ? DENSE_STORE : E;   // leaves partial sums, whatever it is
        if (f32) hipLaunchKernelGGL((dense_gemm_f32_kernel<EG, SN>), grid, block, 0, ctx->stream, a);
        else if (shape == 0) hipLaunchKernelGGL((dense_gemm_bf16_kernel<EG, SN, 128, 128, 2, 2>), grid, block, 0, ctx->stream, a);
        else if (shape == 1) hipLaunchKernelGGL((dense_gemm_bf16_kernel<EG, SN, 64, 64, 2, 2>), grid, block, 0, ctx->stream, a);
        else hipLaunchKernelGGL((dense_gemm_bf16_kernel<EG, SN, 64, 32, 2, 2>), grid, block, 0, ctx->stream, a);
        if (!a.part) return;
        if (f32) hipLaunchKernelGGL((dense_reduce_kernel<float, E, SN>), rg, block, 0, ctx->stream, a, split);
        else hipLaunchKernelGGL((dense_reduce_kernel<__bf16, E, SN>), rg, block, 0, ctx->stream, a, split);
    };
    const std::integral_constant<int, 0> any{};
    switch (a.epi) {
        case DENSE_STORE: go(std::integral_constant<int, DENSE_STORE>{}, any); break;
        case DENSE_ADD: go(std::integral_constant<int, DENSE_ADD>{}, any); break;
        case DENSE_SWIGLU: go(std::integral_constant<int, DENSE_SWIGLU>{}, any); break;
        case DENSE_CAST: go(std::integral_constant<int, DENSE_CAST>{}, any); break;
        case DENSE_RELU2: go(std::integral_constant<int, DENSE_RELU2>{}, any); break;
        default:
            if (a.st.count == 4) go(std::integral_constant<int, DENSE_STREAMS>{}, std::integral_constant<int, 4>{});
            else go(std::integral_constant<int, DENSE_STREAMS>{}, any);
    }
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}

cera_hip_status cera_launch_dense_gemv(cera_hip_ctx* ctx, const DenseIn& in, const DenseMat& wa, const DenseOut& oa,
                                       const DenseMat* wb, const DenseOut* ob, bool f32, bool* launched) {
    *launched = false;
    if (wa.rows == 0 || wa.kp == 0 || wa.kp % DENSE_PAD || (wb && wb->kp != wa.kp))
        return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "dense_gemv: bad shape");
    if (oa.epi == DENSE_STREAMS && (!streams_ok(oa) || wb || (in.kind != DenseIn::RAW && in.kind != DenseIn::MERGE)))
        return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "dense_gemv: streams take one matrix and a finished or partial input");
    if (in.kind == DenseIn::MERGE && (!in.merge.part || in.merge.heads * in.merge.splits > PARTIALS_MAX))
        return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "dense_gemv: partial results of too many heads and key ranges");
    GemvDArgs a{};
    if (oa.streams) a.st = *oa.streams;
    a.in = in;
    a.wa = static_cast<const __bf16*>(wa.w); a.rows_a = wa.rows; a.kp = wa.kp; a.oa = oa;
    if (!cera_dense_gemv_fits(wa.kp, f32)) return CERA_HIP_OK;
    // fewer rows per wavefront (and a longer run of each) where four would leave CUs without work
    const bool pairs = oa.epi == DENSE_SWIGLU || (wb && ob->epi == DENSE_SWIGLU);
    const uint64_t all_rows = static_cast<uint64_t>(wa.rows) + (wb ? wb->rows : 0);
    int r = 4;
    if (all_rows < 8ull * GEMV_WAVES * ctx->n_cu && wa.kp >= 1024) r = 2;
    if (all_rows < 4ull * GEMV_WAVES * ctx->n_cu && wa.kp >= 2048 && !pairs) r = 1;
    a.stage_len = static_cast<uint32_t>(gemv_stage_len(wa.kp, r));
    const uint64_t lds = a.stage_len * (f32 ? 4ull : 2ull);
    a.groups_a = oa.epi == DENSE_SWIGLU ? wa.rows / r : (wa.rows + r - 1) / r;
    if (wb) {
        a.wb = static_cast<const __bf16*>(wb->w); a.rows_b = wb->rows; a.ob = *ob;
        a.groups_b = ob->epi == DENSE_SWIGLU ? wb->rows / r : (wb->rows + r - 1) / r;
    }
    // about two workgroups per CU, shared between the matrices by their rows; no workgroup without a group
    const uint32_t total = a.groups_a + a.groups_b;
    const uint32_t want = std::max(2u, std::min(2 * ctx->n_cu, (total + GEMV_WAVES - 1) / GEMV_WAVES));
    a.blocks_a = std::max(1u, std::min(a.groups_a, wb ? static_cast<uint32_t>(static_cast<uint64_t>(want) * a.groups_a / total) : want));
    a.blocks_b = wb ? std::max(1u, std::min(a.groups_b, want > a.blocks_a ? want - a.blocks_a : 1u)) : 0;
    const dim3 grid(a.blocks_a + a.blocks_b), block(GEMV_WAVES * 64);
    auto go = [&](auto tag, auto rows) {
        using T = decltype(tag);
        constexpr int R = decltype(rows)::value;
        auto kind = [&](auto streams) {
            constexpr int SN = decltype(streams)::value;
            if (in.kind == DenseIn::RAW) hipLaunchKernelGGL((dense_gemv_kernel<T, DenseIn::RAW, R, SN>), grid, block, lds, ctx->stream, a);
            else if (in.kind == DenseIn::MERGE) hipLaunchKernelGGL((dense_gemv_kernel<T, DenseIn::MERGE, R, SN>), grid, block, lds, ctx->stream, a);
            else if constexpr (SN < 0) {
                if (in.kind == DenseIn::NORM) hipLaunchKernelGGL((dense_gemv_kernel<T, DenseIn::NORM, R, SN>), grid, block, lds, ctx->stream, a);
                else hipLaunchKernelGGL((dense_gemv_kernel<T, DenseIn::CONCAT, R, SN>), grid, block, lds, ctx->stream, a);
            }
        };
        if (oa.epi != DENSE_STREAMS) kind(std::integral_constant<int, -1>{});
        else if (a.st.count == 4) kind(std::integral_constant<int, 4>{});
        else kind(std::integral_constant<int, 0>{});
    };
    auto by_rows = [&](auto tag) {
        if (r == 4) go(tag, std::integral_constant<int, 4>{});
        else if (r == 2) go(tag, std::integral_constant<int, 2>{});
        else go(tag, std::integral_constant<int, 1>{});
    };
    if (f32) by_rows(float{});
    else by_rows(static_cast<__bf16>(0.0f));
    HIP_TRY(ctx, hipGetLastError());
    *launched = true;
    return CERA_HIP_OK;
}
