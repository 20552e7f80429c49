// Kernels of softmax_attn.h.
//
// A workgroup of four wavefronts walks the keys in blocks of 32 rows that it stages in LDS by direct
// global-to-LDS loads (16-byte chunk c of row k sits in slot c ^ swz(k) of its group of eight).  Wavefronts are
// `cg` column groups times `kg` key groups times VG value groups: a column is one (query, query head of the kv head)
// pair, 16 * CT of them per wavefront; key groups take blocks in turn and add up through LDS at the end; value groups
// compute the same scores and a share of the value columns each.  Scores are K . q with the
// keys as matrix rows; a lane then holds, for its one column, the scores of exactly the keys whose values it must
// supply for the second product -- for bf16 the two 16-key tiles take keys 8 (r / 4) + r % 4 and that plus 4 as
// their row r, which leaves lane group g with keys 8 g .. 8 g + 7, the operand layout of
// v_mfma_f32_16x16x32_bf16.  The values come out of the same rows by transposing LDS reads.
//
// The running maximum of a column starts at its sink, so it is always finite; the sink's own share of the
// denominator is added where the column ends.  Everything is in powers of two.  Accumulators are rescaled only
// when a score exceeds the maximum by 2^8.  In bf16 the weights enter the second product as a high and a low part.
#include <algorithm>

#include "bf16.hip.h"
#include "softmax_attn.h"

namespace {

constexpr int FW = 4;                // wavefronts of a workgroup
constexpr int FATTN_LDS_MAX = 150 * 1024;
constexpr float LOG2E = 1.44269504088896340736f;
constexpr float RESCALE_AT = 8.0f;

struct FArgs {
    const void* q;
    const void* kv;
    uint64_t head_stride;
    uint32_t row, row_magic;         // row_magic: ceil(2^20 / 16-byte chunks of a row)
    uint32_t n, start, heads, kv_heads, per, kp, vp, vdim, v_off;
    float scale2;                    // scale * log2(e)
    const float* sink;
    void* out;
    uint64_t out_ld;
    uint32_t out_head;
    float *part, *ml;                // [split][n][heads][vp], [split][n][heads][2]; splits > 1 or merged by the consumer
    uint32_t splits, tiles, cg, kg, stages;
};

__device__ __forceinline__ uint32_t swz(uint32_t key) { return (key & 3) | ((((key >> 3) ^ (key >> 2)) & 1) << 2); }

// over the four 16-lane rows of the wavefront, lane by lane
__device__ __forceinline__ float rows_max(float v) {
    auto a = __builtin_amdgcn_permlane32_swap(__builtin_bit_cast(uint32_t, v), __builtin_bit_cast(uint32_t, v), false, false);
    v = fmaxf(__builtin_bit_cast(float, static_cast<uint32_t>(a[0])), __builtin_bit_cast(float, static_cast<uint32_t>(a[1])));
    auto b = __builtin_amdgcn_permlane16_swap(__builtin_bit_cast(uint32_t, v), __builtin_bit_cast(uint32_t, v), false, false);
    return fmaxf(__builtin_bit_cast(float, static_cast<uint32_t>(b[0])), __builtin_bit_cast(float, static_cast<uint32_t>(b[1])));
}
__device__ __forceinline__ float rows_sum(float v) {
    auto a = __builtin_amdgcn_permlane32_swap(__builtin_bit_cast(uint32_t, v), __builtin_bit_cast(uint32_t, v), false, false);
    v = __builtin_bit_cast(float, static_cast<uint32_t>(a[0])) + __builtin_bit_cast(float, static_cast<uint32_t>(a[1]));
    auto b = __builtin_amdgcn_permlane16_swap(__builtin_bit_cast(uint32_t, v), __builtin_bit_cast(uint32_t, v), false, false);
    return __builtin_bit_cast(float, static_cast<uint32_t>(b[0])) + __builtin_bit_cast(float, static_cast<uint32_t>(b[1]));
}

// ---- one block of 32 keys ----------------------------------------------------------------------------
// MK: 32-wide steps of the key columns, MV: 16-wide tiles of the value columns; at most that many, counted at run
// time, unless EXACT
template <int MV> struct Column {    // one lane's column: running maximum, its lane group's share of the sum, values
    float m, l;
    f32x4 o[MV];
    // scores of the block in powers of two (masked: -inf) -> weights
    template <int N> __device__ __forceinline__ void weigh(float (&s)[N], int nv) {
        float mx = s[0];
#pragma unroll
        for (int i = 1; i < N; ++i) mx = fmaxf(mx, s[i]);
        mx = rows_max(mx);
        if (__any(mx > m + RESCALE_AT)) {
            const float mn = fmaxf(m, mx), c = __builtin_amdgcn_exp2f(m - mn);
            m = mn;
            l *= c;
#pragma unroll
            for (int vt = 0; vt < MV; ++vt)
                if (vt < nv) { o[vt].x *= c; o[vt].y *= c; o[vt].z *= c; o[vt].w *= c; }
        }
#pragma unroll
        for (int i = 0; i < N; ++i) {
            s[i] = __builtin_amdgcn_exp2f(s[i] - m);
            l += s[i];
        }
    }
};

template <typename T, int MK, int MV, int CT, bool EXACT> struct Block;

template <int MK, int MV, int CT, bool EXACT> struct Block<__bf16, MK, MV, CT, EXACT> {
    bf16x8 q[CT][MK];
    __device__ __forceinline__ void load_q(int ct, const __bf16* row, bool live, int nk, uint32_t lane) {
        const uint32_t g = lane >> 4;
#pragma unroll
        for (int kd = 0; kd < MK; ++kd) {
            q[ct][kd] = bf16x8{};
            if ((EXACT || kd < nk) && live) q[ct][kd] = *reinterpret_cast<const bf16x8*>(row + kd * 32 + g * 8);
        }
    }
    // lds: the block's rows; hi: last visible key of the lane's column; inside: every key is visible to every column
    __device__ __forceinline__ void run(const __bf16* lds, uint32_t row, uint32_t v_off, uint32_t kb, int nk, int nv, const uint32_t (&hi)[CT],
                                        bool inside, float scale2, Column<MV> (&col)[CT], uint32_t lane) {
        const uint32_t r = lane & 15, g = lane >> 4;
        const char* const base = reinterpret_cast<const char*>(lds);
        const uint32_t ka = (r >> 2) * 8 + (r & 3), e = (g ^ swz(ka)) * 16;
        const char* const k0 = base + ka * row * 2;
        const char* const k1 = k0 + 8 * row;
        f32x4 s0[CT], s1[CT];
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) s0[ct] = s1[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kd = 0; kd < MK; ++kd)
            if (EXACT || kd < nk) {
                const uint32_t off = (kd >> 1) * 128, el = kd & 1 ? e ^ 64 : e;
                const bf16x8 fa = *reinterpret_cast<const bf16x8*>(k0 + off + el), fb = *reinterpret_cast<const bf16x8*>(k1 + off + (el ^ 64));
#pragma unroll
                for (int ct = 0; ct < CT; ++ct) {
                    s0[ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fa, q[ct][kd], s0[ct], 0, 0, 0);
                    s1[ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fb, q[ct][kd], s1[ct], 0, 0, 0);
                }
            }
        bf16x8 ph[CT], pl[CT];
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) {
            float s[8];
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                s[i] = (i < 4 ? s0[ct][i & 3] : s1[ct][i & 3]) * scale2;
                if (!inside) s[i] = kb + g * 8 + i <= hi[ct] ? s[i] : -__builtin_inff();
            }
            col[ct].weigh(s, nv);
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                const __bf16 h = static_cast<__bf16>(s[i]);
                ph[ct][i] = h;
                pl[ct][i] = static_cast<__bf16>(s[i] - static_cast<float>(h));
            }
        }
        // values: lane i of a 16-lane group supplies the address of four columns of row i / 4 and receives column i of
        // four rows
        const uint32_t kv = g * 8 + (r >> 2), ev = (((r & 3) >> 1) ^ swz(kv)) * 16 + (r & 1) * 8;
        const char* const v0 = base + kv * row * 2 + v_off * 2;
        const char* const v1 = v0 + 8 * row;
        typedef short s16x4 __attribute__((ext_vector_type(4)));
        typedef __attribute__((address_space(3))) s16x4* lds_s16x4;
#pragma unroll
        for (int vt = 0; vt < MV; ++vt)
            if (EXACT || vt < nv) {
                const uint32_t off = (vt >> 2) * 128, el = ev ^ ((vt & 3) << 5);
                const bf16x4 lo = __builtin_bit_cast(bf16x4, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4)(v0 + off + el)));
                const bf16x4 up = __builtin_bit_cast(bf16x4, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4)(v1 + off + (el ^ 64))));
                const bf16x8 v = __builtin_shufflevector(lo, up, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
                for (int ct = 0; ct < CT; ++ct) {
                    col[ct].o[vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, ph[ct], col[ct].o[vt], 0, 0, 0);
                    col[ct].o[vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pl[ct], col[ct].o[vt], 0, 0, 0);
                }
            }
    }
};

// true f32: two runs of 16 keys on v_mfma_f32_16x16x4_f32; a lane's four consecutive entries of a 16-wide run feed
// four steps of the product
template <int MK, int MV, int CT, bool EXACT> struct Block<float, MK, MV, CT, EXACT> {
    f32x4 q[CT][2 * MK];
    __device__ __forceinline__ void load_q(int ct, const float* row, bool live, int nk, uint32_t lane) {
        const uint32_t g = lane >> 4;
#pragma unroll
        for (int kd = 0; kd < 2 * MK; ++kd) {
            q[ct][kd] = f32x4{0.f, 0.f, 0.f, 0.f};
            if (kd < 2 * nk && live) q[ct][kd] = *reinterpret_cast<const f32x4*>(row + kd * 16 + g * 4);
        }
    }
    __device__ __forceinline__ void run(const float* lds, uint32_t row, uint32_t v_off, uint32_t kb, int nk, int nv, const uint32_t (&hi)[CT],
                                        bool inside, float scale2, Column<MV> (&col)[CT], uint32_t lane) {
        const uint32_t r = lane & 15, g = lane >> 4;
        for (uint32_t h = 0; h < 32; h += 16) {
            const float* const k0 = lds + (h + r) * row;
            const uint32_t z = swz(h + r);
            f32x4 sc[CT];
#pragma unroll
            for (int ct = 0; ct < CT; ++ct) sc[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kd = 0; kd < 2 * MK; ++kd)
                if (kd < 2 * nk) {
                    const f32x4 fa = *reinterpret_cast<const f32x4*>(k0 + ((kd * 4 + g) ^ z) * 4);
#pragma unroll
                    for (int st = 0; st < 4; ++st)
#pragma unroll
                        for (int ct = 0; ct < CT; ++ct) sc[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(fa[st], q[ct][kd][st], sc[ct], 0, 0, 0);
                }
            float p[CT][4];
#pragma unroll
            for (int ct = 0; ct < CT; ++ct) {
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    p[ct][i] = sc[ct][i] * scale2;
                    if (!inside) p[ct][i] = kb + h + g * 4 + i <= hi[ct] ? p[ct][i] : -__builtin_inff();
                }
                col[ct].weigh(p[ct], nv);
            }
#pragma unroll
            for (int st = 0; st < 4; ++st) {
                const uint32_t key = h + g * 4 + st, zv = swz(key);
                const float* const v0 = lds + key * row + (r & 3);
#pragma unroll
                for (int vt = 0; vt < MV; ++vt)
                    if (vt < nv) {
                        const float v = v0[((v_off / 4 + vt * 4 + (r >> 2)) ^ zv) * 4];
#pragma unroll
                        for (int ct = 0; ct < CT; ++ct) col[ct].o[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(v, p[ct][st], col[ct].o[vt], 0, 0, 0);
                    }
            }
        }
    }
};

// Four consecutive value columns of (query, head), already divided by the denominator.
template <typename T> __device__ __forceinline__ void finish4(const FArgs& a, uint32_t query, uint32_t head, uint32_t v, f32x4 o) {
    T* dst = static_cast<T*>(a.out) + query * a.out_ld + head * a.out_head + v;
    if (v + 4 <= a.vdim && a.out_head % 4 == 0 && a.out_ld % 4 == 0) {
        ElemOps<T>::store4(dst, o.x, o.y, o.z, o.w);
    } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (v + i < a.vdim) dst[i] = ElemOps<T>::from(o[i]);
    }
}

template <typename T, int MK, int MV, int CT, int VG, bool EXACT, int WPE>
__global__ __launch_bounds__(FW * 64, WPE) void fattn_kernel(FArgs a) {
    static_assert(VG == 1 || (EXACT && MV / VG % 4 == 0), "value groups start at whole 64 columns");
    constexpr int MW = MV / VG;
    extern __shared__ __align__(16) unsigned char smem[];
    const uint32_t lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const uint32_t cgi = wave % a.cg, kgi = wave / a.cg % a.kg, vgi = VG > 1 ? wave / a.cg / a.kg : 0;
    // launch index: kv heads (consecutive ones on different XCDs), column tiles with the longest key ranges first, splits
    const uint32_t kvh = blockIdx.x % a.kv_heads, tile = a.tiles - 1 - blockIdx.x / a.kv_heads % a.tiles, split = blockIdx.x / a.kv_heads / a.tiles;
    const uint32_t cols = a.n * a.per, wg_c0 = tile * a.cg * 16 * CT, wg_c1 = min(wg_c0 + a.cg * 16 * CT, cols);
    const int nk = EXACT ? MK : static_cast<int>(a.kp / 32), nv = EXACT ? MW : static_cast<int>(a.vp / 16);
    // this workgroup's key blocks
    const uint32_t nb = (a.start + (wg_c1 - 1) / a.per) / 32 + 1;
    const uint32_t share = ((nb + a.splits - 1) / a.splits + a.kg - 1) / a.kg * a.kg;
    const uint32_t first = min(nb, split * share), last = min(nb, first + share);
    // this wavefront's columns
    const uint32_t c0 = wg_c0 + cgi * 16 * CT;
    const bool wave_live = c0 < cols;
    uint32_t query[CT], head[CT], hi[CT];
    bool live[CT];
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
        const uint32_t c = c0 + ct * 16 + (lane & 15), cc = min(c, cols - 1);
        live[ct] = c < cols;
        query[ct] = cc / a.per;
        head[ct] = kvh * a.per + cc % a.per;
        hi[ct] = a.start + query[ct];
    }
    const uint32_t hi_min = a.start + min(c0, cols - 1) / a.per, hi_max = a.start + min(c0 + 16 * CT - 1, cols - 1) / a.per;
    // staging
    constexpr uint32_t E = 16 / sizeof(T);
    const uint32_t cpr = a.row / E, segs = 32 * cpr / 64;
    const uint32_t block_bytes = 32 * a.row * sizeof(T);
    const T* const kv = static_cast<const T*>(a.kv) + kvh * a.head_stride;
    auto stage = [&](uint32_t b, uint32_t buf) {
        unsigned char* const dst = smem + (buf * a.kg + kgi) * block_bytes;
        const T* const src = kv + static_cast<uint64_t>(b) * 32 * a.row;
        for (uint32_t s = cgi + vgi * a.cg; s < segs; s += a.cg * VG) {
            const uint32_t i = s * 64 + lane, key = (i * a.row_magic) >> 20, slot = i - key * cpr;
            __builtin_amdgcn_global_load_lds(
                reinterpret_cast<const __attribute__((address_space(1))) void*>(reinterpret_cast<uintptr_t>(src + key * a.row + (slot ^ swz(key)) * E)),
                (__attribute__((address_space(3))) void*)(dst + s * 1024), 16, 0, 0);
        }
    };
    uint32_t b = first + kgi;
    if (b < last) stage(b, 0);
    Block<T, MK, MW, CT, EXACT> t;
    Column<MW> col[CT];
    const uint32_t vc0 = vgi * MW * 16;   // this wavefront's first value column
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
        t.load_q(ct, static_cast<const T*>(a.q) + (static_cast<uint64_t>(query[ct]) * a.heads + head[ct]) * a.kp, live[ct], nk, lane);
        col[ct].m = a.sink[head[ct]] * LOG2E;
        col[ct].l = 0.0f;
#pragma unroll
        for (int vt = 0; vt < MW; ++vt) col[ct].o[vt] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    uint32_t buf = 0;
    for (uint32_t b0 = first; b0 < last; b0 += a.kg, b += a.kg) {
        // this step's rows are in, and every wavefront is past its reads of the other buffer
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
        if (a.stages == 2 && b + a.kg < last) stage(b + a.kg, buf ^ 1);
        if (b < last && wave_live && b * 32 <= hi_max)
            t.run(reinterpret_cast<const T*>(smem + (buf * a.kg + kgi) * block_bytes), a.row, a.v_off + vc0, b * 32, nk, nv, hi, b * 32 + 31 <= hi_min,
                  a.scale2, col, lane);
        if (a.stages == 2) {
            buf ^= 1;
        } else {
            __syncthreads();
            if (b + a.kg < last) stage(b + a.kg, 0);
        }
    }
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) col[ct].l = rows_sum(col[ct].l);
    // key groups: the upper ones hand their columns to the first through LDS, one after the other
    for (uint32_t k = 1; k < a.kg; ++k) {
        float* const red = reinterpret_cast<float*>(smem) + (cgi + vgi * a.cg) * (CT * (MW * 256 + 128));
        __syncthreads();
        if (kgi == k) {
#pragma unroll
            for (int ct = 0; ct < CT; ++ct) {
                float* const p = red + ct * (MW * 256 + 128);
                p[lane] = col[ct].m;
                p[64 + lane] = col[ct].l;
#pragma unroll
                for (int vt = 0; vt < MW; ++vt)
                    if (vt < nv) *reinterpret_cast<f32x4*>(p + 128 + (vt * 64 + lane) * 4) = col[ct].o[vt];
            }
        }
        __syncthreads();
        if (kgi == 0) {
#pragma unroll
            for (int ct = 0; ct < CT; ++ct) {
                const float* const p = red + ct * (MW * 256 + 128);
                const float m2 = p[lane], mn = fmaxf(col[ct].m, m2), c1 = __builtin_amdgcn_exp2f(col[ct].m - mn), c2 = __builtin_amdgcn_exp2f(m2 - mn);
                col[ct].m = mn;
                col[ct].l = col[ct].l * c1 + p[64 + lane] * c2;
#pragma unroll
                for (int vt = 0; vt < MW; ++vt)
                    if (vt < nv) {
                        const f32x4 o2 = *reinterpret_cast<const f32x4*>(p + 128 + (vt * 64 + lane) * 4);
#pragma unroll
                        for (int i = 0; i < 4; ++i) col[ct].o[vt][i] = col[ct].o[vt][i] * c1 + o2[i] * c2;
                    }
            }
        }
    }
    if (kgi != 0) return;
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
        if (!live[ct]) continue;
        const uint64_t at = (static_cast<uint64_t>(split) * a.n + query[ct]) * a.heads + head[ct];
        if (a.part) {
            if (vgi == 0 && lane < 16) {
                a.ml[at * 2] = col[ct].m;
                a.ml[at * 2 + 1] = col[ct].l;
            }
        } else {
            const float inv = 1.0f / (col[ct].l + __builtin_amdgcn_exp2f(a.sink[head[ct]] * LOG2E - col[ct].m));
#pragma unroll
            for (int vt = 0; vt < MW; ++vt) { col[ct].o[vt].x *= inv; col[ct].o[vt].y *= inv; col[ct].o[vt].z *= inv; col[ct].o[vt].w *= inv; }
        }
#pragma unroll
        for (int vt = 0; vt < MW; ++vt)
            if (vt < nv) {
                const uint32_t v = vc0 + vt * 16 + (lane >> 4) * 4;
                if (a.part) *reinterpret_cast<f32x4*>(a.part + at * a.vp + v) = col[ct].o[vt];
                else finish4<T>(a, query[ct], head[ct], v, col[ct].o[vt]);
            }
    }
}

// Many pairs with few parts: a.vp / 4 threads per (query, head), four value columns each.
template <typename T> __global__ __launch_bounds__(256) void fattn_merge_kernel(FArgs a) {
    const uint32_t threads = a.vp / 4, q = threadIdx.x % threads, slot = threadIdx.x / threads;
    const uint64_t rows = static_cast<uint64_t>(a.n) * a.heads, at = static_cast<uint64_t>(blockIdx.x) * (256 / threads) + slot;
    if (slot >= 256 / threads || at >= rows || q * 4 >= a.vdim) return;
    const uint32_t query = static_cast<uint32_t>(at / a.heads), head = static_cast<uint32_t>(at % a.heads);
    const float2* const ml = reinterpret_cast<const float2*>(a.ml) + at;
    const float sink2 = a.sink[head] * LOG2E;
    float m = sink2;
#pragma unroll 8
    for (uint32_t z = 0; z < a.splits; ++z) m = fmaxf(m, ml[z * rows].x);
    float l = __builtin_amdgcn_exp2f(sink2 - m);
    f32x4 s{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (uint32_t z = 0; z < a.splits; ++z) {
        const float2 e = ml[z * rows];
        const f32x4 v = *reinterpret_cast<const f32x4*>(a.part + (at + z * rows) * a.vp + q * 4);
        const float w = __builtin_amdgcn_exp2f(e.x - m);
        l = fmaf(e.y, w, l);
#pragma unroll
        for (int i = 0; i < 4; ++i) s[i] = fmaf(v[i], w, s[i]);
    }
    const float inv = 1.0f / l;
    s.x *= inv; s.y *= inv; s.z *= inv; s.w *= inv;
    finish4<T>(a, query, head, q * 4, s);
}
// Few pairs with many parts (at most 256): a workgroup per (query, head) and 32 value columns, the parts shared out
// over 32 groups of eight threads.
template <typename T> __global__ __launch_bounds__(256) void fattn_merge_few_kernel(FArgs a) {
    __shared__ float wz[256], red[8];
    __shared__ __align__(16) f32x4 sums[4][8];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, slices = a.vp / 32, q = blockIdx.x % slices * 8 + (tid & 7), grp = tid >> 3;
    const uint32_t pair = blockIdx.x / slices, query = pair / a.heads, head = pair % a.heads;
    const uint64_t rows = static_cast<uint64_t>(a.n) * a.heads;
    const float sink2 = a.sink[head] * LOG2E;
    const float2 e = tid < a.splits ? reinterpret_cast<const float2*>(a.ml)[pair + tid * rows] : make_float2(sink2, 0.0f);
    float m = wave_max(e.x);
    if (lane == 0) red[wave] = m;
    __syncthreads();
    m = fmaxf(fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])), sink2);
    const float w = __builtin_amdgcn_exp2f(e.x - m), part = wave_sum(e.y * w);
    wz[tid] = w;
    if (lane == 0) red[4 + wave] = part;
    __syncthreads();
    const float inv = 1.0f / (red[4] + red[5] + red[6] + red[7] + __builtin_amdgcn_exp2f(sink2 - m));
    f32x4 s{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (uint32_t z = grp; z < a.splits; z += 32) {
        const f32x4 v = *reinterpret_cast<const f32x4*>(a.part + (pair + z * rows) * a.vp + q * 4);
#pragma unroll
        for (int i = 0; i < 4; ++i) s[i] = fmaf(v[i], wz[z], s[i]);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int d = 8; d <= 32; d <<= 1) s[i] += __shfl_xor(s[i], d);
    if (lane < 8) sums[wave][lane] = s;
    __syncthreads();
    if (tid >= 8 || q * 4 >= a.vdim) return;
    s = sums[0][tid] + sums[1][tid] + sums[2][tid] + sums[3][tid];
    s.x *= inv; s.y *= inv; s.z *= inv; s.w *= inv;
    finish4<T>(a, query, head, q * 4, s);
}

// ---- preparation: sixteen lanes per head of q, k or v, eight entries each at a time -------------------
struct PrepArgs {
    FAttnPrep p;
    uint32_t n, start, heads, kv_heads, kp, v_off, vp, vdim, row;
    uint64_t head_stride;
    void *q, *kv;
    bool whole_k, whole_v;   // heads start 16-byte aligned and come in whole eights
};
template <typename T> __global__ __launch_bounds__(256) void fattn_prep_kernel(PrepArgs a) {
    const uint32_t l8 = (threadIdx.x & 15) * 8, item = blockIdx.x * 16 + (threadIdx.x >> 4), tok = blockIdx.y, dim = a.p.dim;
    if (item >= a.heads + 2 * a.kv_heads) return;
    const uint32_t pos = a.start + tok;
    const float* const src = a.p.qkv + tok * a.p.ld;
    float v[8];
    if (item < a.heads + a.kv_heads) {   // q | k heads stand back to back
        const bool is_q = item < a.heads;
        const float* const x = src + item * dim;
        const float* const w = is_q ? a.p.q_norm : a.p.k_norm;
        float ss = 0.0f;
        for (uint32_t c = l8; c < dim; c += 128) {
            load8(x, c, dim, a.whole_k, v);
#pragma unroll
            for (int i = 0; i < 8; ++i) ss = fmaf(v[i], v[i], ss);
        }
        const float f = 1.0f / sqrtf(wave_row_sum(ss) / static_cast<float>(dim) + a.p.eps);
        const float temp = is_q && a.p.q_mult ? a.p.q_mult[pos] : 1.0f;
        T* const dst = is_q ? static_cast<T*>(a.q) + (static_cast<uint64_t>(tok) * a.heads + item) * a.kp
                            : static_cast<T*>(a.kv) + (item - a.heads) * a.head_stride + static_cast<uint64_t>(pos) * a.row;
        for (uint32_t c = l8; c < a.kp; c += 128) {   // the pads become zero
            float wv[8];
            load8(x, c, dim, a.whole_k, v);
            load8(w, c, dim, a.whole_k, wv);
#pragma unroll
            for (int i = 0; i < 8; ++i) v[i] = v[i] * f * wv[i] * temp;
            ElemOps<T>::store8(dst + c, v);
        }
        return;
    }
    const uint32_t h = item - a.heads - a.kv_heads;
    const float* const x = src + (a.heads + a.kv_heads) * dim + h * a.vdim;
    T* const dst = static_cast<T*>(a.kv) + h * a.head_stride + static_cast<uint64_t>(pos) * a.row + a.v_off;
    float* const first = a.p.v_first ? a.p.v_first + (static_cast<uint64_t>(tok) * a.kv_heads + h) * a.vdim : nullptr;
    for (uint32_t c = l8; c < a.vp; c += 128) {
        load8(x, c, a.vdim, a.whole_v, v);
        if (first && a.p.v_store) {
            if (a.whole_v && c < a.vdim) ElemOps<float>::store8(first + c, v);
            else
#pragma unroll
                for (int i = 0; i < 8; ++i)
                    if (c + i < a.vdim) first[c + i] = v[i];
        } else if (first) {
            float u[8];
            load8(first, c, a.vdim, a.whole_v, u);
#pragma unroll
            for (int i = 0; i < 8; ++i) v[i] = (1.0f - a.p.v_lambda) * v[i] + a.p.v_lambda * u[i];
        }
        ElemOps<T>::store8(dst + c, v);
    }
}

// ---- host --------------------------------------------------------------------------------------------
template <int V> using Int = std::integral_constant<int, V>;
// calls f(MK, MV, exact) with the instance for the shape
template <class F> void by_size(const FArgs& a, bool f32, F&& f) {
    const uint32_t nk = a.kp / 32, nv = a.vp / 16;
    if (!f32) {
        if (nk == 2 && nv == 4) return f(Int<2>{}, Int<4>{}, std::true_type{});
        if (nk == 4 && nv == 8) return f(Int<4>{}, Int<8>{}, std::true_type{});
        if (nk == 6 && nv == 8) return f(Int<6>{}, Int<8>{}, std::true_type{});
        if (nk == 18 && nv == 32) return f(Int<18>{}, Int<32>{}, std::true_type{});
    }
    if (nk <= 4 && nv <= 8) return f(Int<4>{}, Int<8>{}, std::false_type{});
    if (nk <= 8 && nv <= 16) return f(Int<8>{}, Int<16>{}, std::false_type{});
    return f(Int<18>{}, Int<32>{}, std::false_type{});
}

constexpr int wavefronts_per_simd(int mk) { return mk <= 6 ? 2 : 1; }   // what the registers leave room for
template <typename T, int MK, int MV, int CT, int VG, bool EXACT>
cera_hip_status launch(cera_hip_ctx* ctx, const FArgs& a, uint32_t grid, uint64_t lds) {
    auto* const fn = fattn_kernel<T, MK, MV, CT, VG, EXACT, wavefronts_per_simd(MK)>;
    if (lds > 64 * 1024) {
        static const hipError_t allowed = hipFuncSetAttribute(reinterpret_cast<const void*>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, FATTN_LDS_MAX);
        HIP_TRY(ctx, allowed);
    }
    hipLaunchKernelGGL(fn, dim3(grid), dim3(FW * 64), lds, ctx->stream, a);
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}

}  // namespace

bool cera_fattn_fits(const FAttnShape& s) { return s.kp <= FATTN_MAX_KEY && s.vp <= FATTN_MAX_VALUE && s.row <= FATTN_MAX_ROW; }

static cera_hip_status fattn_check(cera_hip_ctx* ctx, const FAttnShape& s, const FAttnPass& p) {
    if (!s.heads || !s.kv_heads || s.heads % s.kv_heads || !s.kp || !s.vp || s.kp % 32 || s.vp % 32 || s.v_off % 64 || s.row % 64 || s.kp > s.row ||
        s.v_off + s.vp > s.row || s.vdim > s.vp || !cera_fattn_fits(s))
        return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "softmax attention: head sizes beyond the kernels' limits");
    if (!p.n || p.cap % FATTN_CAP_STEP || static_cast<uint64_t>(p.start) + p.n > p.cap)
        return cera_fail(ctx, CERA_HIP_ERR_POSITION, "softmax attention: positions beyond the cache");
    return CERA_HIP_OK;
}

cera_hip_status cera_launch_fattn(cera_hip_ctx* ctx, const FAttnShape& s, const FAttnPass& p, SAttnPartials* merge, uint32_t most, bool f32) {
    if (merge) *merge = SAttnPartials{};
    CERA_TRY(fattn_check(ctx, s, p));
    if (merge && p.n != 1) return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "softmax attention: partial results are for one token");
    const uint32_t esz = f32 ? 4 : 2;
    FArgs a{};
    a.q = p.q; a.kv = p.kv; a.head_stride = static_cast<uint64_t>(p.cap) * s.row; a.row = s.row;
    const uint32_t cpr = s.row * esz / 16;
    a.row_magic = ((1u << 20) + cpr - 1) / cpr;
    a.n = p.n; a.start = p.start; a.heads = s.heads; a.kv_heads = s.kv_heads; a.per = s.heads / s.kv_heads;
    a.kp = s.kp; a.vp = s.vp; a.vdim = s.vdim; a.v_off = s.v_off; a.scale2 = s.scale * LOG2E; a.sink = s.sink;
    a.out = p.out; a.out_ld = p.out_ld; a.out_head = p.out_head;
    const uint32_t cols = p.n * a.per, col_tiles = (cols + 15) / 16, nb = (p.start + p.n + 31) / 32;
    cera_hip_status st = CERA_HIP_OK;
    by_size(a, f32, [&](auto mk, auto mv, auto exact) {
        constexpr int MK = decltype(mk)::value, MV = decltype(mv)::value;
        constexpr bool EX = decltype(exact)::value;
        constexpr bool CAN2 = EX && MK <= 6;
        // two column tiles per wavefront where that still fills the chip
        const bool two = CAN2 && !f32 && static_cast<uint64_t>(col_tiles + 7) / 8 * s.kv_heads >= ctx->n_cu;
        const uint32_t tiles = two ? (col_tiles + 1) / 2 : col_tiles;
        // a row so large that two blocks of it take all LDS: two wavefronts share a column instead of the keys
        constexpr bool CAN_SHARE = EX && MK > 8 && MV % 8 == 0;
        const bool share = CAN_SHARE && tiles <= 2;
        a.cg = share ? 2 : tiles >= 3 ? 4 : tiles;
        a.kg = share ? 1 : FW / a.cg;
        a.tiles = (tiles + a.cg - 1) / a.cg;
        const uint64_t block = 32ull * s.row * esz, red = a.kg > 1 ? static_cast<uint64_t>(a.cg) * (two ? 2 : 1) * (MV * 256 + 128) * 4 : 0;
        while (a.kg > 1 && a.kg * block > FATTN_LDS_MAX) a.kg /= 2;
        if (!share && a.cg * a.kg != FW) {   // wavefronts without a key group take columns that do not exist: they only help staging
            a.cg = FW / a.kg;
            a.tiles = (tiles + a.cg - 1) / a.cg;
        }
        a.stages = 2 * a.kg * block <= (wavefronts_per_simd(MK) == 1 ? FATTN_LDS_MAX : 64 * 1024) ? 2 : 1;
        // share the keys out where the column tiles do not fill the chip: at least two steps of a workgroup each,
        // one for a single token (its launch is all latency)
        const uint32_t wgs = a.tiles * s.kv_heads, steps = (nb + a.kg - 1) / a.kg, least = p.n == 1 ? 1 : 2;
        a.splits = std::max(1u, std::min({std::max(1u, 2 * ctx->n_cu / wgs), steps / least, p.n == 1 ? 256u : 16u}));
        if (merge) {
            most = std::min(most, PARTIALS_MAX / s.heads);
            if (a.splits > most && steps <= 2 * most) a.splits = most;   // two steps cost less than a launch
            if (a.splits > most) merge = nullptr;
        }
        if (a.splits > 1 || merge) {
            void* part;
            const uint64_t rows = static_cast<uint64_t>(a.splits) * a.n * a.heads;
            st = cera_scratch(ctx, 10, rows * (a.vp + 2) * sizeof(float), &part);
            if (st != CERA_HIP_OK) return;
            a.part = static_cast<float*>(part);
            a.ml = a.part + rows * a.vp;
        }
        const uint32_t grid = wgs * a.splits;
        const uint64_t lds = std::max(a.stages * a.kg * block, red);
        if constexpr (!EX) {
            st = f32 ? launch<float, MK, MV, 1, 1, EX>(ctx, a, grid, lds) : launch<__bf16, MK, MV, 1, 1, EX>(ctx, a, grid, lds);
        } else {
            st = CERA_HIP_ERR_SHAPE;
            if constexpr (CAN2) { if (two) st = launch<__bf16, MK, MV, 2, 1, EX>(ctx, a, grid, lds); }
            if constexpr (CAN_SHARE) { if (share) st = launch<__bf16, MK, MV, 1, 2, EX>(ctx, a, grid, lds); }
            if (!two && !share) st = launch<__bf16, MK, MV, 1, 1, EX>(ctx, a, grid, lds);
        }
    });
    CERA_TRY(st);
    if (merge) {
        merge->part = a.part; merge->ml = a.ml; merge->sink = s.sink; merge->splits = a.splits; merge->heads = s.heads;
        merge->vdim = s.vdim; merge->vdim_p = s.vp;
    } else if (a.splits > 1) {
        const uint32_t quads = s.vp / 4, pairs = p.n * s.heads;
        const bool few = pairs < 4 * ctx->n_cu;
        const dim3 grid(few ? pairs * (s.vp / 32) : (pairs + 256 / quads - 1) / (256 / quads));
        auto go = [&](auto* fn) { hipLaunchKernelGGL(fn, grid, dim3(256), 0, ctx->stream, a); };
        if (few) go(f32 ? fattn_merge_few_kernel<float> : fattn_merge_few_kernel<__bf16>);
        else go(f32 ? fattn_merge_kernel<float> : fattn_merge_kernel<__bf16>);
        HIP_TRY(ctx, hipGetLastError());
    }
    return CERA_HIP_OK;
}

cera_hip_status cera_launch_fattn_prep(cera_hip_ctx* ctx, const FAttnShape& s, const FAttnPass& p, const FAttnPrep& prep, bool f32) {
    CERA_TRY(fattn_check(ctx, s, p));
    PrepArgs a{};
    a.p = prep;
    a.n = p.n; a.start = p.start; a.heads = s.heads; a.kv_heads = s.kv_heads; a.kp = s.kp; a.v_off = s.v_off; a.vp = s.vp; a.vdim = s.vdim; a.row = s.row;
    a.whole_k = prep.dim % 8 == 0 && (p.n == 1 || prep.ld % 4 == 0);
    a.whole_v = a.whole_k && s.vdim % 8 == 0;
    a.head_stride = static_cast<uint64_t>(p.cap) * s.row;
    a.q = const_cast<void*>(p.q); a.kv = p.kv;
    const dim3 grid((s.heads + 2 * s.kv_heads + 15) / 16, p.n);
    if (f32) hipLaunchKernelGGL(fattn_prep_kernel<float>, grid, dim3(256), 0, ctx->stream, a);
    else hipLaunchKernelGGL(fattn_prep_kernel<__bf16>, grid, dim3(256), 0, ctx->stream, a);
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}
