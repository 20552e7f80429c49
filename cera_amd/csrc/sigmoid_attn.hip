// Kernels of sigmoid_attn.h.
//
// A wavefront works on 16 * CT columns, a column being one (query, query head of the kv head) pair,
// and walks the keys in blocks of 32.  Scores are K . q on the matrix cores with the keys as rows:
// a lane then holds, for its one column, the scores of exactly the keys whose V entries it must
// supply for the second product (V^T . weights) -- for bf16 the two 16-key score tiles take keys
// 8 (r / 4) + r % 4 and that plus 4 as their row r, which leaves lane group g with keys 8 g .. 8 g + 7,
// the operand layout of v_mfma_f32_16x16x32_bf16.  The weights never move between lanes.  Sigmoid
// weights need no running maximum and no normaliser: partial results over key ranges just add.
//
// In bf16 the weights enter the second product as a high and a low bf16 part, so they carry 16
// significant bits against V's eight.
#include <algorithm>

#include "bf16.hip.h"
#include "sigmoid_attn.h"

namespace {

struct AArgs {
    const void* q;          // rotated queries [n][heads][dim_p] (not the fused step)
    const float* qkvg;
    uint64_t ld;
    const void *kc, *vc;
    uint32_t cap, n, start;
    uint32_t heads, kv_heads, per, dim, vdim, dim_p, vdim_p, chunk;
    float scale;
    const float* bias;
    const float* rot_row;   // fused step: (cos, sin) of the position
    uint32_t rot_dims;
    void* out;
    uint64_t out_ld;
    float* part;            // [split][n][heads][vdim_p], splits > 1
    uint32_t splits;
    uint32_t attn_blocks;   // fused step: workgroups past these add up the convolution history
    ConvRing ring;
    ConvHist hist;
};

// first and last visible position of the query at `pos`
__device__ __forceinline__ uint32_t first_visible(uint32_t pos, uint32_t chunk) { return chunk ? pos - pos % chunk : 0u; }

// ---- the two matrix products over one block of 32 keys ------------------------------------------
// DK: 32-wide steps of the head size, VT: 16-wide tiles of the value size; 0 = up to 8 / 16, at run time.
template <typename T, int DK, int VT, int CT> struct Tile;

template <int DK, int VT, int CT> struct Tile<__bf16, DK, VT, CT> {
    static constexpr int MK = DK ? DK : 8, MV = VT ? VT : 16;
    bf16x8 q[CT][MK];
    f32x4 o[CT][MV];

    __device__ __forceinline__ void load_q(int ct, const __bf16* row, bool live, uint32_t nk, uint32_t lane) {
        const uint32_t g = lane >> 4;
#pragma unroll
        for (int kd = 0; kd < MK; ++kd) {
            q[ct][kd] = bf16x8{};
            if ((DK || kd < static_cast<int>(nk)) && live) q[ct][kd] = *reinterpret_cast<const bf16x8*>(row + kd * 32 + g * 8);
        }
    }
    // A block's K rows go into registers ahead of its turn.
    bf16x8 ka[MK], kc[MK];
    __device__ __forceinline__ void load_k(const __bf16* kbase, uint32_t kb, uint32_t nk, uint32_t dim_p, uint32_t lane) {
        const uint32_t r = lane & 15, g = lane >> 4;
        const __bf16* const k0 = kbase + static_cast<uint64_t>(kb + (r >> 2) * 8 + (r & 3)) * dim_p + g * 8;
        const __bf16* const k1 = k0 + 4 * static_cast<uint64_t>(dim_p);
#pragma unroll
        for (int kd = 0; kd < MK; ++kd)
            if (DK || kd < static_cast<int>(nk)) {
                ka[kd] = *reinterpret_cast<const bf16x8*>(k0 + kd * 32);
                kc[kd] = *reinterpret_cast<const bf16x8*>(k1 + kd * 32);
            }
    }
    // kb: first key of the block, its K rows loaded; next: the block whose K rows are loaded meanwhile (UINT32_MAX:
    // none); lo / hi: the visible range of this lane's column; inside: the whole block is visible to every column
    // of the wavefront
    __device__ __forceinline__ void block(const __bf16* kbase, const __bf16* vbase, uint32_t cap, uint32_t kb, uint32_t next, uint32_t nk,
                                          uint32_t nv, uint32_t dim_p, const uint32_t (&lo)[CT], const uint32_t (&hi)[CT],
                                          bool inside, float scale, const float (&bias)[CT], uint32_t lane) {
        const uint32_t r = lane & 15, g = lane >> 4;
        const __bf16* const v0 = vbase + static_cast<uint64_t>(r) * cap + kb + g * 8;
        bf16x8 va[MV];
        if (VT) {
#pragma unroll
            for (int vt = 0; vt < MV; ++vt) va[vt] = *reinterpret_cast<const bf16x8*>(v0 + static_cast<uint64_t>(vt * 16) * cap);
        }
        f32x4 s0[CT], s1[CT];
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) {
            s0[ct] = s1[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kd = 0; kd < MK; ++kd)
                if (DK || kd < static_cast<int>(nk)) {
                    s0[ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka[kd], q[ct][kd], s0[ct], 0, 0, 0);
                    s1[ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kc[kd], q[ct][kd], s1[ct], 0, 0, 0);
                }
        }
        if (next != UINT32_MAX) load_k(kbase, next, nk, dim_p, lane);
        bf16x8 ph[CT], pl[CT];
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) {
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                const float s = i < 4 ? s0[ct][i & 3] : s1[ct][i & 3];
                float p = sigmoid_fast(fmaf(s, scale, bias[ct]));
                if (!inside) {
                    const uint32_t key = kb + g * 8 + i;
                    p = key >= lo[ct] && key <= hi[ct] ? p : 0.0f;
                }
                const __bf16 h = static_cast<__bf16>(p);
                ph[ct][i] = h;
                pl[ct][i] = static_cast<__bf16>(p - static_cast<float>(h));
            }
        }
#pragma unroll
        for (int vt = 0; vt < MV; ++vt)
            if (VT || vt < static_cast<int>(nv)) {
                const bf16x8 v = VT ? va[vt] : *reinterpret_cast<const bf16x8*>(v0 + static_cast<uint64_t>(vt * 16) * cap);
#pragma unroll
                for (int ct = 0; ct < CT; ++ct) {
                    o[ct][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, ph[ct], o[ct][vt], 0, 0, 0);
                    o[ct][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pl[ct], o[ct][vt], 0, 0, 0);
                }
            }
    }
};

// true f32: the same walk in two blocks of 16 keys on v_mfma_f32_16x16x4_f32; a lane's four consecutive
// entries of a 16-wide run feed four steps of the product
template <int DK, int VT, int CT> struct Tile<float, DK, VT, CT> {
    static constexpr int MK = DK ? DK : 8, MV = VT ? VT : 16;
    f32x4 q[CT][2 * MK];
    f32x4 o[CT][MV];

    __device__ __forceinline__ void load_q(int ct, const float* row, bool live, uint32_t nk, uint32_t lane) {
        const uint32_t g = lane >> 4;
#pragma unroll
        for (int kd = 0; kd < 2 * MK; ++kd) {
            q[ct][kd] = f32x4{0.f, 0.f, 0.f, 0.f};
            if ((DK || kd < static_cast<int>(2 * nk)) && live) q[ct][kd] = *reinterpret_cast<const f32x4*>(row + kd * 16 + g * 4);
        }
    }
    __device__ __forceinline__ void load_k(const float*, uint32_t, uint32_t, uint32_t, uint32_t) {}   // read where they are used
    __device__ __forceinline__ void block(const float* kbase, const float* vbase, uint32_t cap, uint32_t kb0, uint32_t, uint32_t nk,
                                          uint32_t nv, uint32_t dim_p, const uint32_t (&lo)[CT], const uint32_t (&hi)[CT],
                                          bool inside, float scale, const float (&bias)[CT], uint32_t lane) {
        const uint32_t r = lane & 15, g = lane >> 4;
        for (uint32_t kb = kb0; kb < kb0 + 32; kb += 16) {
            const float* const k0 = kbase + static_cast<uint64_t>(kb + r) * dim_p + g * 4;
            const float* const v0 = vbase + static_cast<uint64_t>(r) * cap + kb + g * 4;
            f32x4 s[CT];
#pragma unroll
            for (int ct = 0; ct < CT; ++ct) s[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kd = 0; kd < 2 * MK; ++kd)
                if (DK || kd < static_cast<int>(2 * nk)) {
                    const f32x4 ka = *reinterpret_cast<const f32x4*>(k0 + kd * 16);
#pragma unroll
                    for (int st = 0; st < 4; ++st)
#pragma unroll
                        for (int ct = 0; ct < CT; ++ct) s[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[st], q[ct][kd][st], s[ct], 0, 0, 0);
                }
#pragma unroll
            for (int ct = 0; ct < CT; ++ct)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const float p = sigmoid_f32(fmaf(s[ct][i], scale, bias[ct]));
                    const uint32_t key = kb + g * 4 + i;
                    s[ct][i] = inside || (key >= lo[ct] && key <= hi[ct]) ? p : 0.0f;
                }
#pragma unroll
            for (int vt = 0; vt < MV; ++vt)
                if (VT || vt < static_cast<int>(nv)) {
                    const f32x4 v = *reinterpret_cast<const f32x4*>(v0 + static_cast<uint64_t>(vt * 16) * cap);
#pragma unroll
                    for (int st = 0; st < 4; ++st)
#pragma unroll
                        for (int ct = 0; ct < CT; ++ct) o[ct][vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(v[st], s[ct][st], o[ct][vt], 0, 0, 0);
                }
        }
    }
};

// Four consecutive value columns v .. v+3 of (query, head): gated, into the output row.
template <typename T>
__device__ __forceinline__ void finish4(const AArgs& a, uint32_t query, uint32_t head, uint32_t v, f32x4 o) {
    const float gate = sigmoid_f32(a.qkvg[query * a.ld + a.heads * a.dim + a.kv_heads * (a.dim + a.vdim) + head]);
    T* dst = static_cast<T*>(a.out) + query * a.out_ld + head * a.vdim + v;
    if (v + 4 <= a.vdim && a.vdim % 4 == 0) {
        ElemOps<T>::store4(dst, o.x * gate, o.y * gate, o.z * gate, o.w * gate);
    } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (v + i < a.vdim) dst[i] = ElemOps<T>::from(o[i] * gate);
    }
}

// One wavefront's columns: 16 * CT from c0 on of the n * per columns of its kv head.
template <typename T, int DK, int VT, int CT>
struct Columns {
    uint32_t query[CT], head[CT], lo[CT], hi[CT];
    float bias[CT];
    bool live[CT];
    uint32_t lo_min, lo_max, hi_min, hi_max;   // over the wavefront's live columns
    __device__ __forceinline__ void set(const AArgs& a, uint32_t c0, uint32_t kvh, uint32_t lane) {
        const uint32_t cols = a.n * a.per;
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) {
            const uint32_t c = c0 + ct * 16 + (lane & 15), cc = min(c, cols - 1);
            live[ct] = c < cols;
            query[ct] = cc / a.per;
            head[ct] = kvh * a.per + cc % a.per;
            hi[ct] = a.start + query[ct];
            lo[ct] = first_visible(hi[ct], a.chunk);
            bias[ct] = a.bias[head[ct]];
        }
        // columns ascend with the query: the ends of the range are the first and the last live column
        const uint32_t ql = c0 / a.per, qh = min(c0 + 16 * CT - 1, cols - 1) / a.per;
        hi_min = a.start + ql;
        hi_max = a.start + qh;
        lo_min = first_visible(hi_min, a.chunk);
        lo_max = first_visible(hi_max, a.chunk);
    }
};

// ---- many queries: every wavefront its own columns -----------------------------------------------
template <typename T, int DK, int VT, int CT>
__global__ __launch_bounds__(256) void sattn_rows_kernel(AArgs a) {
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6, kvh = blockIdx.y;
    const uint32_t tile = (gridDim.x - 1 - blockIdx.x) * 4 + wave;   // the longest key ranges start first
    const uint32_t c0 = tile * 16 * CT;
    if (c0 >= a.n * a.per) return;
    const uint32_t nk = a.dim_p / 32, nv = a.vdim_p / 16;
    Columns<T, DK, VT, CT> col;
    col.set(a, c0, kvh, lane);
    Tile<T, DK, VT, CT> t;
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
        t.load_q(ct, static_cast<const T*>(a.q) + (static_cast<uint64_t>(col.query[ct]) * a.heads + col.head[ct]) * a.dim_p, col.live[ct], nk, lane);
#pragma unroll
        for (int vt = 0; vt < t.MV; ++vt) t.o[ct][vt] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const T* const kb_ = static_cast<const T*>(a.kc) + static_cast<uint64_t>(kvh) * a.cap * a.dim_p;
    const T* const vb_ = static_cast<const T*>(a.vc) + static_cast<uint64_t>(kvh) * a.vdim_p * a.cap;
    t.load_k(kb_, col.lo_min & ~31u, nk, a.dim_p, lane);
    for (uint32_t kb = col.lo_min & ~31u; kb <= col.hi_max; kb += 32)
        t.block(kb_, vb_, a.cap, kb, kb + 32 <= col.hi_max ? kb + 32 : UINT32_MAX, nk, nv, a.dim_p, col.lo, col.hi,
                kb >= col.lo_max && kb + 31 <= col.hi_min, a.scale, col.bias, lane);
#pragma unroll
    for (int ct = 0; ct < CT; ++ct)
        if (col.live[ct]) {
#pragma unroll
            for (int vt = 0; vt < t.MV; ++vt)
                if (VT || vt < static_cast<int>(nv)) finish4<T>(a, col.query[ct], col.head[ct], vt * 16 + (lane >> 4) * 4, t.o[ct][vt]);
        }
}

// ---- few queries: the wavefronts of a workgroup (and `splits` workgroups) share the keys ---------
constexpr int SPLIT_WAVES = 8;

__device__ __forceinline__ void conv_hist_body(const ConvRing& ring, const ConvHist& h, uint32_t pos, uint32_t i) {
    // history of the token at `pos`: taps 0 .. taps-2 against rows pos - taps + 1 .. pos - 1
    const float* const w = i < ring.width ? h.wa : h.wb;
    const uint32_t c = i < ring.width ? i : i - ring.width;
    if (!w || c >= ring.width) return;
    float s = 0.0f;
    for (uint32_t j = 0; j + 1 < h.taps; ++j) {
        const uint32_t back = h.taps - 1 - j;
        if (back <= pos) s = fmaf(w[static_cast<uint64_t>(j) * ring.width + c], ring.rows[static_cast<uint64_t>((pos - back) & (ring.depth - 1)) * ring.ld + c], s);
    }
    (i < ring.width ? h.a : h.b)[c] = s;
}

// FUSED: the decode step (n == 1, per <= 16): q, k, v come straight from the projections.  Every workgroup
// rotates the queries of its kv head; all of a kv head's workgroups but one read a cache that the new
// position is not part of yet, and the one whose range ends with it appends it first.
template <typename T, int DK, int VT, bool FUSED>
__global__ __launch_bounds__(SPLIT_WAVES * 64) void sattn_split_kernel(AArgs a) {
    constexpr int MV = VT ? VT : 16, MKD = (DK ? DK : 8) * 32;
    __shared__ __align__(16) float red[SPLIT_WAVES / 2][MV * 16 * 16];
    __shared__ __align__(16) T qs[FUSED ? 16 * MKD : 16];
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    if (FUSED && blockIdx.x >= a.attn_blocks) {
        conv_hist_body(a.ring, a.hist, a.start + 1, (blockIdx.x - a.attn_blocks) * SPLIT_WAVES * 64 + threadIdx.x);
        return;
    }
    // launch index: column tiles of a kv head, kv heads, splits
    const uint32_t cols = a.n * a.per, tiles = (cols + 15) / 16;
    const uint32_t tile = blockIdx.x % tiles, kvh = blockIdx.x / tiles % a.kv_heads, split = blockIdx.x / tiles / a.kv_heads;
    const uint32_t c0 = tile * 16, nk = a.dim_p / 32, nv = a.vdim_p / 16;
    Columns<T, DK, VT, 1> col;
    col.set(a, c0, kvh, lane);
    // this workgroup's share of the key blocks
    const uint32_t b0 = col.lo_min / 32, nb = col.hi_max / 32 + 1 - b0, per_split = (nb + a.splits - 1) / a.splits;
    const uint32_t first = b0 + split * per_split, last = min(b0 + nb, first + per_split);
    Tile<T, DK, VT, 1> t;
    const T* const kb_ = static_cast<const T*>(a.kc) + static_cast<uint64_t>(kvh) * a.cap * a.dim_p;
    const T* const vb_ = static_cast<const T*>(a.vc) + static_cast<uint64_t>(kvh) * a.vdim_p * a.cap;
    // the first block's K rows are on their way while the queries are prepared, unless the block holds the new key
    uint32_t b = first + wave;
    const bool early = b < last && !(FUSED && b == b0 + nb - 1);
    if (early) t.load_k(kb_, b * 32, nk, a.dim_p, lane);
    if (FUSED) {
        const float* const row = a.qkvg;
        const float* const kn = row + a.heads * a.dim + kvh * a.dim;
        for (uint32_t i = threadIdx.x; i < 16 * a.dim_p / 2; i += SPLIT_WAVES * 64) {
            const uint32_t h = i / (a.dim_p / 2), e = (i % (a.dim_p / 2)) * 2;
            float u = 0.0f, v = 0.0f;
            if (h < a.per) {
                const float* const qr = row + (kvh * a.per + h) * a.dim;
                if (e < a.dim) u = qr[e];
                if (e + 1 < a.dim) v = qr[e + 1];
                if (e < a.rot_dims) {
                    const float c = a.rot_row[e], s = a.rot_row[e + 1], x = u;
                    u = x * c - v * s;
                    v = v * c + x * s;
                }
            }
            qs[h * a.dim_p + e] = ElemOps<T>::from(u);
            qs[h * a.dim_p + e + 1] = ElemOps<T>::from(v);
        }
        if (last == b0 + nb && first < last) {
            T* const kd = const_cast<T*>(static_cast<const T*>(a.kc)) + (static_cast<uint64_t>(kvh) * a.cap + a.start) * a.dim_p;
            T* const vd = const_cast<T*>(static_cast<const T*>(a.vc)) + static_cast<uint64_t>(kvh) * a.vdim_p * a.cap + a.start;
            const float* const vn = row + (a.heads + a.kv_heads) * a.dim + kvh * a.vdim;
            for (uint32_t i = threadIdx.x; i < a.dim; i += SPLIT_WAVES * 64) {
                float x = kn[i];
                if (i < a.rot_dims) {
                    const uint32_t e = i & ~1u;
                    const float c = a.rot_row[e], s = a.rot_row[e + 1];
                    x = (i & 1) ? kn[i] * c + kn[e] * s : kn[i] * c - kn[i + 1] * s;
                }
                kd[i] = ElemOps<T>::from(x);
            }
            for (uint32_t i = threadIdx.x; i < a.vdim; i += SPLIT_WAVES * 64) vd[static_cast<uint64_t>(i) * a.cap] = ElemOps<T>::from(vn[i]);
        }
        __syncthreads();
        t.load_q(0, qs + (lane & 15) * a.dim_p, true, nk, lane);
    } else {
        t.load_q(0, static_cast<const T*>(a.q) + (static_cast<uint64_t>(col.query[0]) * a.heads + col.head[0]) * a.dim_p, col.live[0], nk, lane);
    }
#pragma unroll
    for (int vt = 0; vt < MV; ++vt) t.o[0][vt] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (b < last && !early) t.load_k(kb_, b * 32, nk, a.dim_p, lane);
    for (; b < last; b += SPLIT_WAVES) {
        const uint32_t kb = b * 32;
        t.block(kb_, vb_, a.cap, kb, b + SPLIT_WAVES < last ? kb + 32 * SPLIT_WAVES : UINT32_MAX, nk, nv, a.dim_p, col.lo, col.hi,
                kb >= col.lo_max && kb + 31 <= col.hi_min, a.scale, col.bias, lane);
    }
    // add the wavefronts up: the upper half hands its tile to the lower half, three times
#pragma unroll
    for (int half = SPLIT_WAVES / 2; half >= 1; half /= 2) {
        if (wave >= static_cast<uint32_t>(half) && wave < 2u * half) {
#pragma unroll
            for (int vt = 0; vt < MV; ++vt)
                if (VT || vt < static_cast<int>(nv)) *reinterpret_cast<f32x4*>(&red[wave - half][(vt * 64 + lane) * 4]) = t.o[0][vt];
        }
        __syncthreads();
        if (wave < static_cast<uint32_t>(half)) {
#pragma unroll
            for (int vt = 0; vt < MV; ++vt)
                if (VT || vt < static_cast<int>(nv)) t.o[0][vt] += *reinterpret_cast<const f32x4*>(&red[wave][(vt * 64 + lane) * 4]);
        }
        __syncthreads();
    }
    if (wave || !col.live[0]) return;
#pragma unroll
    for (int vt = 0; vt < MV; ++vt)
        if (VT || vt < static_cast<int>(nv)) {
            const uint32_t v = vt * 16 + (lane >> 4) * 4;
            if (a.part)
                *reinterpret_cast<f32x4*>(a.part + ((static_cast<uint64_t>(split) * a.n + col.query[0]) * a.heads + col.head[0]) * a.vdim_p + v) = t.o[0][vt];
            else
                finish4<T>(a, col.query[0], col.head[0], v, t.o[0][vt]);
        }
}

// One workgroup per (query, head): a thread holds four value columns of every `groups`-th partial result.
template <typename T>
__global__ __launch_bounds__(256) void sattn_merge_kernel(AArgs a) {
    __shared__ __align__(16) f32x4 red[256];
    const uint32_t quads = a.vdim_p / 4, groups = 256 / quads, q = threadIdx.x % quads, grp = threadIdx.x / quads;
    const uint32_t query = blockIdx.x / a.heads, head = blockIdx.x % a.heads;
    const uint64_t slice = static_cast<uint64_t>(a.n) * a.heads * a.vdim_p;
    const float* p = a.part + (static_cast<uint64_t>(query) * a.heads + head) * a.vdim_p + q * 4;
    f32x4 s{0.f, 0.f, 0.f, 0.f};
    if (grp < groups) {
#pragma unroll 4
        for (uint32_t z = grp; z < a.splits; z += groups) s += *reinterpret_cast<const f32x4*>(p + z * slice);
    }
    red[threadIdx.x] = s;
    __syncthreads();
    if (grp != 0) return;
    for (uint32_t i = 1; i < groups; ++i) s += red[i * quads + q];
    if (q * 4 < a.vdim) finish4<T>(a, query, head, q * 4, s);
}

// ---- append ---------------------------------------------------------------------------------------
struct AppendArgs {
    AArgs a;
    const float* rot_table;
    void* q;
    uint32_t v_blocks_x;     // 64-position tiles of the transposed V write
    uint32_t n_qk, n_v, n_ring, ring_rows;
    const float *x, *inv, *w;
    uint64_t x_ld;
};
template <typename T>
__global__ __launch_bounds__(256) void sattn_append_kernel(AppendArgs p) {
    __shared__ float tr[32][65];
    const AArgs& a = p.a;
    uint32_t b = blockIdx.x;
    if (b < p.n_qk) {   // one token: its q and k heads
        const uint32_t tok = b, pos = a.start + tok, pairs = a.dim_p / 2;
        const float* const row = a.qkvg + tok * a.ld;
        const float* const cs = p.rot_table + static_cast<uint64_t>(pos) * a.rot_dims;
        for (uint32_t i = threadIdx.x; i < (a.heads + a.kv_heads) * pairs; i += 256) {
            const uint32_t h = i / pairs, e = (i % pairs) * 2;
            float u = e < a.dim ? row[h * a.dim + e] : 0.0f, v = e + 1 < a.dim ? row[h * a.dim + e + 1] : 0.0f;
            if (e < a.rot_dims) {
                const float c = cs[e], s = cs[e + 1], x = u;
                u = x * c - v * s;
                v = v * c + x * s;
            }
            T* dst = h < a.heads ? static_cast<T*>(p.q) + (static_cast<uint64_t>(tok) * a.heads + h) * a.dim_p + e
                                 : const_cast<T*>(static_cast<const T*>(a.kc)) + (static_cast<uint64_t>(h - a.heads) * a.cap + pos) * a.dim_p + e;
            dst[0] = ElemOps<T>::from(u);
            dst[1] = ElemOps<T>::from(v);
        }
        return;
    }
    b -= p.n_qk;
    if (b < p.n_v) {    // 64 tokens x 32 value columns of one kv head, through LDS
        const uint32_t tx = b % p.v_blocks_x, vy = b / p.v_blocks_x % (a.vdim_p / 32), kvh = b / p.v_blocks_x / (a.vdim_p / 32);
        const float* const src = a.qkvg + (a.heads + a.kv_heads) * a.dim + kvh * a.vdim;
        for (uint32_t i = threadIdx.x; i < 64 * 32; i += 256) {
            const uint32_t tok = tx * 64 + i / 32, c = vy * 32 + i % 32;
            tr[i % 32][i / 32] = tok < a.n && c < a.vdim ? src[tok * a.ld + c] : 0.0f;
        }
        __syncthreads();
        T* const dst = const_cast<T*>(static_cast<const T*>(a.vc)) + static_cast<uint64_t>(kvh) * a.vdim_p * a.cap + a.start;
        for (uint32_t i = threadIdx.x; i < 64 * 32; i += 256) {
            const uint32_t tok = tx * 64 + i % 64, c = vy * 32 + i / 64;
            if (tok < a.n && c < a.vdim) dst[static_cast<uint64_t>(c) * a.cap + tok] = ElemOps<T>::from(tr[i / 64][i % 64]);
        }
        return;
    }
    b -= p.n_v;         // one of the pass's last normalised rows
    const uint32_t tok = a.n - p.ring_rows + b, pos = a.start + tok;
    const float s = p.inv[tok];
    float* const dst = a.ring.rows + static_cast<uint64_t>(pos & (a.ring.depth - 1)) * a.ring.ld;
    for (uint32_t c = threadIdx.x; c < a.ring.width; c += 256) dst[c] = p.x[tok * p.x_ld + c] * s * p.w[c];
}

__global__ __launch_bounds__(256) void conv_hist_kernel(ConvRing ring, ConvHist hist, uint32_t pos) {
    conv_hist_body(ring, hist, pos, blockIdx.x * 256 + threadIdx.x);
}

// ---- host -----------------------------------------------------------------------------------------
cera_hip_status fill(cera_hip_ctx* ctx, const SAttnShape& s, const SAttnPass& p, AArgs* a) {
    if (!s.heads || !s.kv_heads || s.heads % s.kv_heads || !s.dim || !s.vdim || s.dim > 256 || s.vdim > 256 || s.rot_dims > s.dim ||
        s.rot_dims % 2)
        return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "sigmoid attention: head sizes up to 256, heads a multiple of kv_heads");
    if (!p.n || p.cap % SATTN_CAP_STEP || static_cast<uint64_t>(p.start) + p.n > p.cap)
        return cera_fail(ctx, CERA_HIP_ERR_POSITION, "sigmoid attention: positions beyond the cache");
    *a = AArgs{};
    a->q = p.q; a->qkvg = p.qkvg; a->ld = p.ld; a->kc = p.kc; a->vc = p.vc; a->cap = p.cap; a->n = p.n; a->start = p.start;
    a->heads = s.heads; a->kv_heads = s.kv_heads; a->per = s.heads / s.kv_heads;
    a->dim = s.dim; a->vdim = s.vdim; a->dim_p = sattn_pad32(s.dim); a->vdim_p = sattn_pad32(s.vdim);
    a->chunk = s.chunk; a->scale = s.scale; a->bias = s.bias; a->rot_dims = s.rot_dims;
    a->rot_row = s.rot_dims ? s.rot_table + static_cast<uint64_t>(p.start) * s.rot_dims : nullptr;
    a->out = p.out; a->out_ld = p.out_ld; a->splits = 1;
    return CERA_HIP_OK;
}

// calls f(DK, VT) with the compile-time head sizes where there is an instance, else (0, 0)
template <int V> using Int = std::integral_constant<int, V>;
template <class F> void by_size(const AArgs& a, bool f32, F&& f) {
    if (!f32 && a.dim_p == a.vdim_p) {
        if (a.dim_p == 64) return f(Int<2>{}, Int<4>{});
        if (a.dim_p == 96) return f(Int<3>{}, Int<6>{});
        if (a.dim_p == 128) return f(Int<4>{}, Int<8>{});
    }
    f(Int<0>{}, Int<0>{});
}

// longest key range of the pass, in blocks of 32
uint32_t max_blocks(const AArgs& a) {
    const uint32_t end = a.start + a.n, reach = a.chunk ? std::min(a.chunk + 31, end) : end;
    return (reach + 31) / 32 + 1;
}
// merge (nullable, fused only): where to leave the partial results for the consumer instead of merging them here
cera_hip_status run_split(cera_hip_ctx* ctx, AArgs& a, bool f32, bool fused, SAttnPartials* merge) {
    const uint32_t tiles = (a.n * a.per + 15) / 16, wgs = tiles * a.kv_heads;
    const uint32_t nb = fused ? a.start / 32 + 1 - (a.chunk ? a.start - a.start % a.chunk : 0) / 32 : max_blocks(a);
    // two blocks per wavefront before a second workgroup takes a share; one round of the chip at most
    a.splits = std::max(1u, std::min({(nb + 2 * SPLIT_WAVES - 1) / (2 * SPLIT_WAVES), std::max(1u, 2 * ctx->n_cu / wgs), 64u}));
    if (merge) {
        *merge = SAttnPartials{};
        const uint32_t fine = std::min((nb + SPLIT_WAVES - 1) / SPLIT_WAVES, SATTN_MERGE_SPLITS);
        if (nb <= SATTN_MERGE_SPLITS * SPLIT_WAVES * 2 && a.heads * fine <= PARTIALS_MAX) a.splits = fine;   // one block per wavefront, two at the most
        else merge = nullptr;
    }
    if (a.splits > 1 || merge) {
        void* part;
        CERA_TRY(cera_scratch(ctx, 10, static_cast<uint64_t>(a.splits) * a.n * a.heads * a.vdim_p * sizeof(float), &part));
        a.part = static_cast<float*>(part);
    }
    a.attn_blocks = wgs * a.splits;
    const uint32_t extra = fused && a.ring.rows ? (2 * a.ring.width + SPLIT_WAVES * 64 - 1) / (SPLIT_WAVES * 64) : 0;
    const dim3 grid(a.attn_blocks + extra), block(SPLIT_WAVES * 64);
    by_size(a, f32, [&](auto dk, auto vt) {
        constexpr int DK = decltype(dk)::value, VT = decltype(vt)::value;
        if (f32) {
            if (fused) hipLaunchKernelGGL((sattn_split_kernel<float, 0, 0, true>), grid, block, 0, ctx->stream, a);
            else hipLaunchKernelGGL((sattn_split_kernel<float, 0, 0, false>), grid, block, 0, ctx->stream, a);
        } else {
            if (fused) hipLaunchKernelGGL((sattn_split_kernel<__bf16, DK, VT, true>), grid, block, 0, ctx->stream, a);
            else hipLaunchKernelGGL((sattn_split_kernel<__bf16, DK, VT, false>), grid, block, 0, ctx->stream, a);
        }
    });
    HIP_TRY(ctx, hipGetLastError());
    if (merge) {
        merge->part = a.part; merge->splits = a.splits; merge->heads = a.heads; merge->vdim = a.vdim; merge->vdim_p = a.vdim_p;
        merge->gate = a.qkvg + a.heads * a.dim + a.kv_heads * (a.dim + a.vdim);
    } else if (a.splits > 1) {
        const dim3 mg(a.n * a.heads);
        if (f32) hipLaunchKernelGGL(sattn_merge_kernel<float>, mg, dim3(256), 0, ctx->stream, a);
        else hipLaunchKernelGGL(sattn_merge_kernel<__bf16>, mg, dim3(256), 0, ctx->stream, a);
        HIP_TRY(ctx, hipGetLastError());
    }
    return CERA_HIP_OK;
}

}  // namespace

cera_hip_status cera_launch_sattn_append(cera_hip_ctx* ctx, const SAttnShape& s, const SAttnPass& p, const ConvRing& ring,
                                         const float* x, uint64_t x_ld, const float* inv, const float* w, bool f32) {
    AppendArgs g{};
    CERA_TRY(fill(ctx, s, p, &g.a));
    g.a.ring = ring;
    g.rot_table = s.rot_table; g.q = p.q; g.x = x; g.x_ld = x_ld; g.inv = inv; g.w = w;
    g.v_blocks_x = (p.n + 63) / 64;
    g.n_qk = p.n;
    g.n_v = g.v_blocks_x * (g.a.vdim_p / 32) * s.kv_heads;
    g.ring_rows = x && ring.rows ? std::min(p.n, ring.depth) : 0;
    const dim3 grid(g.n_qk + g.n_v + g.ring_rows);
    if (f32) hipLaunchKernelGGL(sattn_append_kernel<float>, grid, dim3(256), 0, ctx->stream, g);
    else hipLaunchKernelGGL(sattn_append_kernel<__bf16>, grid, dim3(256), 0, ctx->stream, g);
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}

cera_hip_status cera_launch_sattn(cera_hip_ctx* ctx, const SAttnShape& s, const SAttnPass& p, bool f32) {
    AArgs a;
    CERA_TRY(fill(ctx, s, p, &a));
    const uint32_t cols = p.n * a.per;
    // too few columns to fill the chip with a wavefront each: share the keys out instead
    if (static_cast<uint64_t>(cols) / 16 * s.kv_heads < 2 * ctx->n_cu) return run_split(ctx, a, f32, false, nullptr);
    const bool wide = static_cast<uint64_t>(cols) / 32 * s.kv_heads >= 4 * ctx->n_cu;
    by_size(a, f32, [&](auto dk, auto vt) {
        constexpr int DK = decltype(dk)::value, VT = decltype(vt)::value;
        const uint32_t per_wg = 64 * (wide && VT ? 2 : 1);
        const dim3 grid((cols + per_wg - 1) / per_wg, s.kv_heads);
        if (f32) hipLaunchKernelGGL((sattn_rows_kernel<float, 0, 0, 1>), grid, dim3(256), 0, ctx->stream, a);
        else if (VT && wide) hipLaunchKernelGGL((sattn_rows_kernel<__bf16, DK, VT, VT ? 2 : 1>), grid, dim3(256), 0, ctx->stream, a);
        else hipLaunchKernelGGL((sattn_rows_kernel<__bf16, DK, VT, 1>), grid, dim3(256), 0, ctx->stream, a);
    });
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}

cera_hip_status cera_launch_sattn_step(cera_hip_ctx* ctx, const SAttnShape& s, const SAttnPass& p, const ConvRing& ring,
                                       const ConvHist& hist, SAttnPartials* merge, bool f32) {
    if (merge) *merge = SAttnPartials{};
    AArgs a;
    CERA_TRY(fill(ctx, s, p, &a));
    if (p.n != 1) return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "sigmoid attention step: one token");
    if (a.per > 16) {   // more query heads per kv head than one tile of columns: separate append
        CERA_TRY(cera_launch_sattn_append(ctx, s, p, ConvRing{}, nullptr, 0, nullptr, nullptr, f32));
        if (ring.rows) CERA_TRY(cera_launch_conv_hist(ctx, ring, hist, p.start + 1));
        return run_split(ctx, a, f32, false, nullptr);
    }
    a.ring = ring;
    a.hist = hist;
    return run_split(ctx, a, f32, true, merge);
}

cera_hip_status cera_launch_conv_hist(cera_hip_ctx* ctx, const ConvRing& ring, const ConvHist& hist, uint32_t pos) {
    hipLaunchKernelGGL(conv_hist_kernel, dim3((2 * ring.width + 255) / 256), dim3(256), 0, ctx->stream, ring, hist, pos);
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}
