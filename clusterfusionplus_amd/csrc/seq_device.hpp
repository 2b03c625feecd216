// Device-side building blocks of the sequence models (prefill in portions + decode) for gfx950.
//
// Everything is written in units of 16 bytes, so that one body serves both element types: 8 bf16 values (one
// v_mfma_f32_16x16x32_bf16 per unit and lane) or 4 fp32 values (four v_mfma_f32_16x16x4_f32, true fp32).  The order of k
// inside a product is free as long as both operands use the same one.
//
// Matrix products put the weight rows (attention: keys, value columns) on the MFMA's row operand and the tokens (attention:
// query columns) on its column operand: a lane then holds four consecutive rows of one token, which makes the stores wide,
// puts the interleaved gate and up rows of one output into the same lane, and leaves the softmax of a query in the lanes
// of one column.
#pragma once
#include "cfpp_device.hpp"

namespace cfpp {

typedef __bf16 bf16_t;
typedef __bf16 bf16x2_t __attribute__((ext_vector_type(2)));
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x2 __attribute__((ext_vector_type(2)));

constexpr int kRowBytes = 128;                    // matrix rows are padded to this
constexpr int kSeqThreads = 256;                  // threads of every sequence kernel: four waves
constexpr int kSeqWaves = kSeqThreads / kWave;
constexpr float kLog2e = 1.4426950408889634f;
constexpr float kMasked = -3.0e38f;               // score of a key that is not seen: its exp2 is zero next to any other, and next
                                                  // to kNegBig, where a column has seen nothing yet

template <typename T> struct Unit;                // elements in 16 bytes
template <> struct Unit<bf16_t> { static constexpr int n = 8; };
template <> struct Unit<float> { static constexpr int n = 4; };

__device__ __forceinline__ float to_f32(bf16_t v) { return (float)v; }
__device__ __forceinline__ float to_f32(float v) { return v; }
template <typename T> __device__ __forceinline__ T from_f32(float v) { return (T)v; }

__device__ __forceinline__ uint32_t pack_bf16(float a, float b) {
    bf16x2_t v = {(bf16_t)a, (bf16_t)b};
    return __builtin_bit_cast(uint32_t, v);
}

template <typename T> __device__ __forceinline__ f32x4 mma16(u32x4 a, u32x4 b, f32x4 c);
template <> __device__ __forceinline__ f32x4 mma16<bf16_t>(u32x4 a, u32x4 b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, a), __builtin_bit_cast(bf16x8_t, b), c, 0, 0, 0);
}
template <> __device__ __forceinline__ f32x4 mma16<float>(u32x4 a, u32x4 b, f32x4 c) {
    const f32x4 fa = __builtin_bit_cast(f32x4, a), fb = __builtin_bit_cast(f32x4, b);
#pragma unroll
    for (int j = 0; j < 4; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(fa[j], fb[j], c, 0, 0, 0);
    return c;
}

// dot product of two 16-byte units, accumulated in fp32
template <typename T> __device__ __forceinline__ float dot16(u32x4 w, u32x4 x, float acc);
template <> __device__ __forceinline__ float dot16<bf16_t>(u32x4 w, u32x4 x, float acc) {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const uint32_t wj = w[j], xj = x[j];             // (a bit cast of a vector's element itself reads element 0)
        acc = __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(bf16x2_t, wj), __builtin_bit_cast(bf16x2_t, xj), acc, false);
    }
    return acc;
}
template <> __device__ __forceinline__ float dot16<float>(u32x4 w, u32x4 x, float acc) {
    const f32x4 fw = __builtin_bit_cast(f32x4, w), fx = __builtin_bit_cast(f32x4, x);
#pragma unroll
    for (int j = 0; j < 4; ++j) acc = fmadd(fw[j], fx[j], acc);
    return acc;
}

// the elements of a 16-byte unit
template <typename T> __device__ __forceinline__ void unpack16(u32x4 b, float (&v)[Unit<T>::n]);
template <> __device__ __forceinline__ void unpack16<bf16_t>(u32x4 b, float (&v)[8]) {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        v[2 * j] = __uint_as_float(b[j] << 16);
        v[2 * j + 1] = __uint_as_float(b[j] & 0xffff0000u);
    }
}
template <> __device__ __forceinline__ void unpack16<float>(u32x4 b, float (&v)[4]) {
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = __uint_as_float(b[j]);
}

// 64 lanes copy 64 units from memory straight to LDS; the lanes' units land next to each other from `lds` (wave-uniform) on
__device__ __forceinline__ void copy_to_lds16(const void* g, void* lds) {
    __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(uintptr_t)g,
                                     (__attribute__((address_space(3))) void*)(uintptr_t)lds, 16, 0, 0);
}

// waits until at most N of the wave's vector memory operations are still on their way
template <int N> __device__ __forceinline__ void wait_vm() { asm volatile("s_waitcnt vmcnt(%0)" ::"n"(N) : "memory"); }

// A barrier of the workgroup behind its LDS accesses only.  Written out: __syncthreads(), and a fence over LDS as well, would
// also wait for the loads in flight, those that go straight to LDS among them.
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
    for (int m = 1; m < kWave; m <<= 1) v = fmaxf(v, xor_shfl(v, m));
    return v;
}

// sum over the workgroup, in every thread, in a fixed order; `red` holds kSeqWaves values
__device__ __forceinline__ float block_sum(float v, float* red) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return (red[0] + red[1]) + (red[2] + red[3]);
}

__device__ __forceinline__ float2 block_sum2(float a, float b, float2* red) {
    a = wave_sum(a);
    b = wave_sum(b);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = make_float2(a, b);
    __syncthreads();
    return make_float2((red[0].x + red[1].x) + (red[2].x + red[3].x), (red[0].y + red[1].y) + (red[2].y + red[3].y));
}

__device__ __forceinline__ float inv_rms(float sum_sq, int n, float eps) { return 1.0f / sqrtf(sum_sq / (float)n + eps); }
__device__ __forceinline__ float sigmoid(float v) { return 1.0f / (1.0f + fast_exp2(-v * kLog2e)); }
__device__ __forceinline__ float relu2(float v) { v = fmaxf(v, 0.0f); return v * v; }
__device__ __forceinline__ float soft_cap(float v, float cap) { return cap > 0.0f ? cap * tanhf(v / cap) : v; }

// sum of squares of n floats over the workgroup's threads (each thread's share)
__device__ __forceinline__ float share_sq(const float* __restrict__ v, int n, int tid) {
    float s = 0.0f;
    int i0 = 0;
    if (((uintptr_t)v & 15) == 0) {
        i0 = n & ~3;
        for (int i = tid; i < n / 4; i += 4 * kSeqThreads) {         // four loads in one round trip
            f32x4 x[4];
#pragma unroll
            for (int b = 0; b < 4; ++b) x[b] = reinterpret_cast<const f32x4*>(v)[min(i + b * kSeqThreads, n / 4 - 1)];
#pragma unroll
            for (int b = 0; b < 4; ++b)
                if (i + b * kSeqThreads < n / 4) {
#pragma unroll
                    for (int j = 0; j < 4; ++j) s = fmadd(x[b][j], x[b][j], s);
                }
        }
    }
    for (int i = i0 + tid; i < n; i += kSeqThreads) s = fmadd(v[i], v[i], s);
    return s;
}

// four values to T, 16 or 8 bytes (p aligned to that)
template <typename T> __device__ __forceinline__ void store4(void* p, f32x4 v) {
    if constexpr (sizeof(T) == 4) {
        *reinterpret_cast<f32x4*>(p) = v;
    } else {
        *reinterpret_cast<u32x2*>(p) = u32x2{pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3])};
    }
}
// N = 4: one access of 16 (T: 8) bytes; N = 1: one element
template <int N> __device__ __forceinline__ void add_n(float (&s)[N], const float* __restrict__ p) {
    if constexpr (N == 4) {
        const f32x4 v = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
        for (int j = 0; j < 4; ++j) s[j] += v[j];
    } else {
        s[0] += *p;
    }
}
template <typename T, int N> __device__ __forceinline__ void put_n(T* p, const float (&v)[N]) {
    if constexpr (N == 4) store4<T>(p, f32x4{v[0], v[1], v[2], v[3]});
    else *p = from_f32<T>(v[0]);
}

// Element d of head h of a run of heads (D elements each) after the norm over the whole projection and the rotation: the
// element and its partner with their norm weights, and (cos, sin) of the pair.  `row` is the run in the projection, `w` in
// the norm weight, `cs` the pairs of the position.
struct RotIn { float a, b, c, s; };
__device__ __forceinline__ RotIn rotate_request(const float* __restrict__ row, const float* __restrict__ w, int h, int d, int D, int rot,
                                                const float2* __restrict__ cs) {
    const int e = h * D + d;
    RotIn r = {row[e] * w[e], 0.0f, 1.0f, 0.0f};
    if (d < rot) {
        const int o = e + ((d & 1) ? -1 : 1);
        const float2 t = cs[d >> 1];
        r.b = row[o] * w[o];
        r.c = t.x;
        r.s = (d & 1) ? t.y : -t.y;
    }
    return r;
}
__device__ __forceinline__ float rotate_finish(const RotIn& r, float inv) { return (r.a * inv) * r.c + (r.b * inv) * r.s; }

// First position of position p's chunk (chunk 0: the whole past).
__device__ __forceinline__ int chunk_start(int p, int chunk) { return chunk > 0 ? (p / chunk) * chunk : 0; }

// ------------------------------------------------------------------------------------------------
// attention
// ------------------------------------------------------------------------------------------------
// A wave works on 16 query columns; lane l belongs to column l & 15 and to row group g = l >> 4.  Scores of a 16-key tile
// are one MFMA result: the lane holds keys 4g .. 4g + 3 of its column.  Those registers are the column operand of the
// second product as they are: its k slots are taken in the order in which the lanes hold the keys, and the transposed value
// tile in LDS (V^T, one row of keys per value column) is read in the same order.
//
// Attention weights stay in 32 bits.  With bf16 matrices they are split into a high and a low bf16 part, which carry 16
// bits of the weight into the product, and both parts are multiplied.
template <typename T, int KT> struct VtTile {
    static constexpr int pitch = KT * (int)sizeof(T) + 16;      // bytes; 16 more than the keys: rows start in different banks
};

// 4 keys x one unit of value columns per step, transposed on the way into LDS.  `rowp(key)` is the address of a key's
// value row, for keys 0 .. KT - 1 of the tile; threads tid of NTHREADS share the tile.  Steps [FIRST, FIRST + N) of
// VtSteps: request puts them into registers, store writes them out.
template <typename T, int KT, int NT, int NTHREADS> struct VtSteps {
    static constexpr int n = (KT / 4 * (NT / Unit<T>::n) + NTHREADS - 1) / NTHREADS;
};
template <typename T, int KT, int NTHREADS, int FIRST, int N, typename RowPtr>
__device__ __forceinline__ void vt_request(u32x4 (&r)[N][4], int vunits, int tid, RowPtr rowp) {
    constexpr int KG = KT / 4;
#pragma unroll
    for (int b = 0; b < N; ++b) {
        const int idx = tid + (FIRST + b) * NTHREADS, kg = idx % KG, vc = min(idx / KG, vunits - 1);
#pragma unroll
        for (int j = 0; j < 4; ++j) r[b][j] = ld16(rowp(kg * 4 + j) + (size_t)vc * 16);
    }
}
template <typename T, int KT, int NTHREADS, int FIRST, int N>
__device__ __forceinline__ void vt_store(const u32x4 (&r)[N][4], char* vt, int vunits, int tid) {
    constexpr int KG = KT / 4;
#pragma unroll
    for (int b = 0; b < N; ++b) {
        const int idx = tid + (FIRST + b) * NTHREADS, kg = idx % KG, vc = idx / KG;
        if (vc < vunits) {
            if constexpr (sizeof(T) == 2) {
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    // halfword e & 1 of word e >> 1 of the four keys
                    constexpr uint32_t kLow = 0x05040100u, kHigh = 0x07060302u;
                    const uint32_t sel = (e & 1) ? kHigh : kLow;
                    u32x2 v = {__builtin_amdgcn_perm(r[b][1][e >> 1], r[b][0][e >> 1], sel), __builtin_amdgcn_perm(r[b][3][e >> 1], r[b][2][e >> 1], sel)};
                    *reinterpret_cast<u32x2*>(vt + (vc * 8 + e) * VtTile<T, KT>::pitch + kg * 8) = v;
                }
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    u32x4 v = {r[b][0][e], r[b][1][e], r[b][2][e], r[b][3][e]};
                    *reinterpret_cast<u32x4*>(vt + (vc * 4 + e) * VtTile<T, KT>::pitch + kg * 16) = v;
                }
            }
        }
    }
}

template <int NT> struct AttnState {              // of one column tile
    float m, l;                                   // running maximum (log2 domain) and denominator, the same in every row group
    f32x4 acc[NT / 16];                           // value columns 16 i + 4 g + r of the lane's column
};

template <int NT>
__device__ __forceinline__ void attn_reset(AttnState<NT>& st) {
    st.m = kNegBig;
    st.l = 0.0f;
#pragma unroll
    for (int i = 0; i < NT / 16; ++i) st.acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
}

// s[kt][r]: scores (already times scale * log2 e; kMasked: not seen) of keys 16 kt + 4 g + r.  Turns them into
// weights relative to the new maximum and rescales the state.
template <int NT, int NKT>
__device__ __forceinline__ void attn_softmax(AttnState<NT>& st, f32x4 (&s)[NKT], int vtiles) {
    float mx = kNegBig;
#pragma unroll
    for (int kt = 0; kt < NKT; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) mx = fmaxf(mx, s[kt][r]);
    mx = fmaxf(mx, xor_shfl(mx, 16));
    mx = fmaxf(mx, xor_shfl(mx, 32));
    const float m = fmaxf(st.m, mx);
    const float c = fast_exp2(st.m - m);
    float sum = 0.0f;
#pragma unroll
    for (int kt = 0; kt < NKT; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float p = fast_exp2(s[kt][r] - m);
            s[kt][r] = p;
            sum += p;
        }
    sum += xor_shfl(sum, 16);
    sum += xor_shfl(sum, 32);
    st.l = st.l * c + sum;
    st.m = m;
#pragma unroll
    for (int i = 0; i < NT / 16; ++i)
        if (i < vtiles) st.acc[i] *= c;
}

// acc += V^T p for the keys of one tile and CT column tiles, which share the reads of V^T
template <typename T, int NT, int KT, int CT>
__device__ __forceinline__ void attn_pv(AttnState<NT>* st, const f32x4 (*p)[KT / 16], const char* vt, int vtiles, int lane) {
    const int col = lane & 15, g = lane >> 4;
    if constexpr (sizeof(T) == 2) {
        u32x4 hi[CT][KT / 32], lo[CT][KT / 32];
#pragma unroll
        for (int ct = 0; ct < CT; ++ct)
#pragma unroll
            for (int s = 0; s < KT / 32; ++s)
#pragma unroll
                for (int h = 0; h < 2; ++h) {
                    const f32x4 v = p[ct][2 * s + h];
                    f32x4 rest;
#pragma unroll
                    for (int r = 0; r < 4; ++r) rest[r] = v[r] - (float)(bf16_t)v[r];
                    hi[ct][s][2 * h] = pack_bf16(v[0], v[1]);
                    hi[ct][s][2 * h + 1] = pack_bf16(v[2], v[3]);
                    lo[ct][s][2 * h] = pack_bf16(rest[0], rest[1]);
                    lo[ct][s][2 * h + 1] = pack_bf16(rest[2], rest[3]);
                }
#pragma unroll
        for (int i = 0; i < NT / 16; ++i)
            if (i < vtiles) {
                const char* row = vt + (i * 16 + col) * VtTile<T, KT>::pitch + g * 8;
#pragma unroll
                for (int s = 0; s < KT / 32; ++s) {
                    const u32x2 a = *reinterpret_cast<const u32x2*>(row + s * 64), b = *reinterpret_cast<const u32x2*>(row + s * 64 + 32);
                    const u32x4 f = {a.x, a.y, b.x, b.y};
#pragma unroll
                    for (int ct = 0; ct < CT; ++ct) {
                        st[ct].acc[i] = mma16<T>(f, hi[ct][s], st[ct].acc[i]);
                        st[ct].acc[i] = mma16<T>(f, lo[ct][s], st[ct].acc[i]);
                    }
                }
            }
    } else {
#pragma unroll
        for (int i = 0; i < NT / 16; ++i)
            if (i < vtiles) {
                const char* row = vt + (i * 16 + col) * VtTile<T, KT>::pitch + g * 16;
#pragma unroll
                for (int s = 0; s < KT / 16; ++s) {
                    const u32x4 f = *reinterpret_cast<const u32x4*>(row + s * 64);
#pragma unroll
                    for (int ct = 0; ct < CT; ++ct) st[ct].acc[i] = mma16<T>(f, __builtin_bit_cast(u32x4, p[ct][s]), st[ct].acc[i]);
                }
            }
    }
}

}  // namespace cfpp
