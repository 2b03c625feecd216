// Latent attention and residual streams of the sequence models (device code; included by seq_kernels.hip).
//
// A latent mixer caches one row per position: the normed latent c (kv_rank values, padded to whole weight rows) and, behind
// it, the rotated key part that all heads share.
//   Portions: the plain keys and the values of all heads are made from the cached latents by one matrix product
//   (kEpiHeads) and attention runs over them head by head; the rotated part is read from the cache rows as it is.
//   Decode: the query is taken into the latent space instead, q' = W_uk^T q (k_seq_latent_q), all heads attend to the cache
//   rows themselves, as keys and as values (k_seq_latent_attn), and W_uv turns the weighted latents into the heads' outputs
//   (k_seq_latent_out, which also merges the splits).  A step reads the cache once instead of making keys and values.
#pragma once
#include <type_traits>

#include "seq_device.hpp"

namespace cfpp {

// (cos, sin) of pair j of a position; the pair is (j, j + R/2) or (2j, 2j + 1)
__device__ __forceinline__ int pair_first(int j, int R, int half) { return half ? j : 2 * j; }
__device__ __forceinline__ int pair_second(int j, int R, int half) { return half ? j + R / 2 : 2 * j + 1; }

// R rotated values of `row` to `out`, zeros up to `end` bytes; the workgroup's threads from `tid` on, `n` of them
template <typename T>
__device__ __forceinline__ void rotate_row(const float* __restrict__ row, char* out, int R, int end, int half, const float2* __restrict__ cs, int tid, int n) {
    T* o = reinterpret_cast<T*>(out);
    for (int j = tid; j < R / 2; j += n) {
        const float2 t = cs[j];
        const float u = row[pair_first(j, R, half)], v = row[pair_second(j, R, half)];
        o[pair_first(j, R, half)] = from_f32<T>(u * t.x - v * t.y);
        o[pair_second(j, R, half)] = from_f32<T>(v * t.x + u * t.y);
    }
    for (int j = R + tid; j < end / (int)sizeof(T); j += n) o[j] = from_f32<T>(0.0f);
}

// The latent row of one position: norm over the first `rank` values, rotation of the other R.
struct LatentRow {
    const float* w;          // [rank]
    int rank, R, rot_off, crow, half;
    float eps;
};
template <typename T>
__device__ __forceinline__ void latent_row(const LatentRow& a, const float* __restrict__ z, char* row, const float2* __restrict__ cs, float* red) {
    const float inv = inv_rms(block_sum(share_sq(z, a.rank, threadIdx.x), red), a.rank, a.eps);
    for (int i = threadIdx.x; i < a.rank; i += kSeqThreads) reinterpret_cast<T*>(row)[i] = from_f32<T>(z[i] * inv * a.w[i]);
    rotate_row<T>(z + a.rank, row + a.rot_off, a.R, a.crow - a.rot_off, a.half, cs, threadIdx.x, kSeqThreads);
}

// ---- portions ----------------------------------------------------------------------------------
// One workgroup per token: raw projection (fp32) -> queries [token][head][plain | rotated | zeros] and the cache row.
struct SeqLatentFinish {
    const float* z;
    int ld, own;             // own: the layer makes cache rows
    LatentRow kv;
    const float2* cs;        // [positions][R / 2]
    int H, D, R, pos0, rot_at, qrow;      // rot_at: bytes in front of the rotated part of a query
    char *q, *kc;            // kc: cache row of position 0
};
template <typename T>
__global__ __launch_bounds__(kSeqThreads) void k_seq_latent_finish(SeqLatentFinish a) {
    __shared__ float red[kSeqWaves];
    const int t = blockIdx.x, n = a.D + a.R;
    const float* z = a.z + (size_t)t * a.ld;
    const float2* cs = a.cs + (size_t)(a.pos0 + t) * (a.R / 2);
    char* q = a.q + (size_t)t * a.H * a.qrow;
    if (a.own) latent_row<T>(a.kv, z + a.H * n, a.kc + (size_t)(a.pos0 + t) * a.kv.crow, cs, red);
    const int p4 = a.rot_at / (int)sizeof(T) / 4;        // groups of four plain values, padding included
    for (int i = threadIdx.x; i < a.H * p4; i += kSeqThreads) {
        const int h = i / p4, d = (i - h * p4) * 4;
        const float* row = z + h * n + d;
        f32x4 x;
#pragma unroll
        for (int j = 0; j < 4; ++j) x[j] = d + j < a.D ? row[j] : 0.0f;
        store4<T>(q + (size_t)h * a.qrow + d * sizeof(T), x);
    }
    const int end = a.qrow - a.rot_at, per = max(a.R / 2, end / (int)sizeof(T) - a.R);     // threads per head: pairs, zeros behind them
    for (int i = threadIdx.x; i < a.H * per; i += kSeqThreads) {
        const int h = i / per;
        rotate_row<T>(z + h * n + a.D, q + (size_t)h * a.qrow + a.rot_at, a.R, end, a.kv.half, cs, i - h * per, per);
    }
}

// ---- one token ---------------------------------------------------------------------------------
// Workgroup (head, 128 bytes of latent columns): those columns of W_uk^T q, summed in fp32 over the head's plain dimensions.
// A thread owns one 16-byte unit of the columns and every 32nd dimension.  The first workgroup of a head also rotates the
// rest of its query; one more workgroup makes the position's cache row.
struct SeqLatentQ {
    const float* z;
    const int* state;
    const float2* cs;
    const char* w_uk;        // T [H * D][pitch bytes]
    int pitch, H, D, R, nrb, own;
    LatentRow kv;
    char* q;                 // T [H][kv.crow bytes]: q' padded to `pitch` bytes, then the rotated part
    char* kc;                // caches, slot 0
    size_t slot_bytes;
};
template <typename T>
__global__ __launch_bounds__(kSeqThreads) void k_seq_latent_q(SeqLatentQ a) {
    constexpr int U = Unit<T>::n, G = kSeqThreads / 8;   // elements per unit, dimension groups
    constexpr int kLoads = 4;
    __shared__ float red[kSeqWaves];
    __shared__ float part[kSeqWaves][8 * U];
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, h = blockIdx.x / a.nrb, rb = blockIdx.x - h * a.nrb;
    const int pos = a.state[1];
    const float2* cs = a.cs + (size_t)pos * (a.R / 2);
    if (h == a.H) {
        latent_row<T>(a.kv, a.z + a.H * (a.D + a.R), a.kc + a.state[3] * a.slot_bytes + (size_t)pos * a.kv.crow, cs, red);
        return;
    }
    const float* z = a.z + h * (a.D + a.R);
    const char* w = a.w_uk + (size_t)h * a.D * a.pitch + rb * 128 + (tid & 7) * 16;
    float acc[U];
#pragma unroll
    for (int e = 0; e < U; ++e) acc[e] = 0.0f;
    for (int d0 = tid >> 3; d0 < a.D; d0 += G * kLoads) {
        u32x4 b[kLoads];
        float x[kLoads];
#pragma unroll
        for (int i = 0; i < kLoads; ++i) {
            const int d = min(d0 + i * G, a.D - 1);
            b[i] = ld16(w + (size_t)d * a.pitch);
            x[i] = d0 + i * G < a.D ? z[d] : 0.0f;
        }
#pragma unroll
        for (int i = 0; i < kLoads; ++i) {
            float v[U];
            unpack16<T>(b[i], v);
#pragma unroll
            for (int e = 0; e < U; ++e) acc[e] = fmadd(v[e], x[i], acc[e]);
        }
    }
#pragma unroll
    for (int e = 0; e < U; ++e) {                        // lanes of the same unit
        acc[e] += xor_shfl(acc[e], 8);
        acc[e] += xor_shfl(acc[e], 16);
        acc[e] += xor_shfl(acc[e], 32);
    }
    if (lane < 8) {
#pragma unroll
        for (int e = 0; e < U; ++e) part[wave][lane * U + e] = acc[e];
    }
    __syncthreads();
    char* q = a.q + (size_t)h * a.kv.crow;
    if (tid < 8 * U) reinterpret_cast<T*>(q + rb * 128)[tid] = from_f32<T>((part[0][tid] + part[1][tid]) + (part[2][tid] + part[3][tid]));
    if (rb == 0) rotate_row<T>(z + a.D, q + a.kv.rot_off, a.R, a.kv.crow - a.kv.rot_off, a.kv.half, cs, tid, kSeqThreads);
}

// Tiles of keys of a decode step, and how many workgroups share them: a few tiles each while that keeps the number of partial
// results, which every workgroup of k_seq_latent_out reads for its head, small.
template <typename T> struct LatentTile { static constexpr int keys = sizeof(T) == 2 ? 32 : 16; };
template <typename T> __device__ __forceinline__ int latent_tiles(int pos) { return (pos + LatentTile<T>::keys) / LatentTile<T>::keys; }
__device__ __forceinline__ int latent_splits(int tiles, int most, int least) { return min(most, (tiles + least - 1) / least); }

// Column fragments of c^T for the second product, for eight (or two) sets of 16 latent columns: keys 4g .. 4g + 3 (x) and 16 + 4g .. (y) of
// column lane & 15, from a tile of cache rows in LDS; `p`, `q`: the lane's place in the rows of the one and the other.  The reads
// and their wait are written out: behind its own transposed reads the compiler would also wait for the copies to the other buffers.
struct TrCols { u32x2 x, y; };
__device__ __forceinline__ void tr_read8(TrCols (&f)[8], uint32_t p, uint32_t q) {
    asm volatile(
        "ds_read_b64_tr_b16 %0, %16\n\tds_read_b64_tr_b16 %1, %17\n\t"
        "ds_read_b64_tr_b16 %2, %16 offset:32\n\tds_read_b64_tr_b16 %3, %17 offset:32\n\t"
        "ds_read_b64_tr_b16 %4, %16 offset:64\n\tds_read_b64_tr_b16 %5, %17 offset:64\n\t"
        "ds_read_b64_tr_b16 %6, %16 offset:96\n\tds_read_b64_tr_b16 %7, %17 offset:96\n\t"
        "ds_read_b64_tr_b16 %8, %16 offset:128\n\tds_read_b64_tr_b16 %9, %17 offset:128\n\t"
        "ds_read_b64_tr_b16 %10, %16 offset:160\n\tds_read_b64_tr_b16 %11, %17 offset:160\n\t"
        "ds_read_b64_tr_b16 %12, %16 offset:192\n\tds_read_b64_tr_b16 %13, %17 offset:192\n\t"
        "ds_read_b64_tr_b16 %14, %16 offset:224\n\tds_read_b64_tr_b16 %15, %17 offset:224\n\t"
        "s_waitcnt lgkmcnt(0)"
        : "=&v"(f[0].x), "=&v"(f[0].y), "=&v"(f[1].x), "=&v"(f[1].y), "=&v"(f[2].x), "=&v"(f[2].y), "=&v"(f[3].x), "=&v"(f[3].y), "=&v"(f[4].x),
          "=&v"(f[4].y), "=&v"(f[5].x), "=&v"(f[5].y), "=&v"(f[6].x), "=&v"(f[6].y), "=&v"(f[7].x), "=&v"(f[7].y)
        : "v"(p), "v"(q)
        : "memory");
}
__device__ __forceinline__ void tr_read2(TrCols (&f)[2], uint32_t p, uint32_t q) {
    asm volatile(
        "ds_read_b64_tr_b16 %0, %4\n\tds_read_b64_tr_b16 %1, %5\n\t"
        "ds_read_b64_tr_b16 %2, %4 offset:32\n\tds_read_b64_tr_b16 %3, %5 offset:32\n\t"
        "s_waitcnt lgkmcnt(0)"
        : "=&v"(f[0].x), "=&v"(f[0].y), "=&v"(f[1].x), "=&v"(f[1].y)
        : "v"(p), "v"(q)
        : "memory");
}

// Workgroup (split, group of heads).  Four waves: RW of them share 16 heads, each with its part of the scores' dimensions (the
// parts are added through LDS, in the same order by all of them) and of the output's latent columns; 4 / RW sets of 16 heads.
// Tiles of cache rows go through buffers in LDS, two ahead, and
// serve as keys (row fragments) and as values (transposed reads).  A row in LDS has room for NR latents and 128 rotated values
// and an odd number of 16-byte units; past the end of the cache row its last unit is repeated, which meets zeros in the query
// and columns that are not stored.
struct SeqLatentAttn {
    const char* q;           // T [H][crow bytes]
    const char* kc;          // caches, slot 0
    size_t slot_bytes;
    const int* state;
    float *acc, *ml;         // [ns][H][rp], [ns][H][2]
    float scale_log2;
    int H, crow, ns, least, rp;      // least: tiles of a split
};
template <typename T, int NR> struct LatentLds {
    static constexpr int ksteps = (NR + 128) * (int)sizeof(T) / 64, up = ksteps * 4 + 1;
    static constexpr int copies = (LatentTile<T>::keys * up + 255) / 256;            // 1 KB copies per wave and tile
    static constexpr int tile = copies * kSeqWaves * 1024, buffers = 3;
};

// 64 units of the tile per copy, the waves in turn
template <typename T, int NR>
__device__ __forceinline__ void latent_stage(char* __restrict__ tile, const char* __restrict__ kc, int crow, int kb, int last, int wave, int lane) {
    using L = LatentLds<T, NR>;
    const int units = crow / 16;
#pragma unroll
    for (int i = 0; i < L::copies; ++i) {
        const int c = i * kSeqWaves + wave, l = c * 64 + lane, r = l / L::up, u = l - r * L::up;
        copy_to_lds16(kc + (size_t)min(kb + r, last) * crow + min(u, units - 1) * 16, tile + c * 1024);
    }
}

// One tile: the copies of a later one, scores, softmax, second product.  `parts`: [wave][KF][lane].
template <typename T, int NR, int RW>
__device__ __forceinline__ void latent_tile(AttnState<NR / RW>& st, const u32x4 (&qf)[LatentLds<T, NR>::ksteps / RW], const char* __restrict__ tile,
                                            char* __restrict__ next, bool more, f32x4* __restrict__ parts, const char* __restrict__ kc, int crow, int kb, int kn,
                                            int k1, float scale_log2, int rw, int wave, int lane) {
    using L = LatentLds<T, NR>;
    constexpr int KT = LatentTile<T>::keys, KF = KT / 16, NW = NR / RW, KS = L::ksteps / RW;
    static_assert(L::ksteps % RW == 0, "");
    const int col = lane & 15, g = lane >> 4;
    if (more) latent_stage<T, NR>(next, kc, crow, kn, k1 - 1, wave, lane);
    f32x4 s[KF];
    u32x4 kf[KS][KF];
#pragma unroll
    for (int d = 0; d < KS; ++d)
#pragma unroll
        for (int kt = 0; kt < KF; ++kt) kf[d][kt] = *reinterpret_cast<const u32x4*>(tile + ((kt * 16 + col) * L::up + (rw * KS + d) * 4 + g) * 16);
    __builtin_amdgcn_sched_barrier(0);                   // (all reads are requested before the first product waits for one)
#pragma unroll
    for (int kt = 0; kt < KF; ++kt) {
        s[kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int d = 0; d < KS; ++d) s[kt] = mma16<T>(kf[d][kt], qf[d], s[kt]);
    }
#pragma unroll
    for (int kt = 0; kt < KF; ++kt) parts[(wave * KF + kt) * kWave + lane] = s[kt];
    lds_barrier();
#pragma unroll
    for (int kt = 0; kt < KF; ++kt) {
        f32x4 p[RW];
#pragma unroll
        for (int w = 0; w < RW; ++w) p[w] = parts[((wave - rw + w) * KF + kt) * kWave + lane];
        s[kt] = p[0];
#pragma unroll
        for (int w = 1; w < RW; ++w) s[kt] += p[w];
    }
#pragma unroll
    for (int kt = 0; kt < KF; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) s[kt][r] = kb + kt * 16 + g * 4 + r < k1 ? s[kt][r] * scale_log2 : kMasked;
    attn_softmax<NW, KF>(st, s, NW / 16);
    if constexpr (sizeof(T) == 2) {
        u32x4 hi, lo;
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) {
            f32x4 rest;
#pragma unroll
            for (int r = 0; r < 4; ++r) rest[r] = s[kt][r] - (float)(bf16_t)s[kt][r];
            hi[2 * kt] = pack_bf16(s[kt][0], s[kt][1]);
            hi[2 * kt + 1] = pack_bf16(s[kt][2], s[kt][3]);
            lo[2 * kt] = pack_bf16(rest[0], rest[1]);
            lo[2 * kt + 1] = pack_bf16(rest[2], rest[3]);
        }
        constexpr int B = NW >= 128 ? 8 : 2;             // sets of 16 columns read together
        const uint32_t v = (uint32_t)(uintptr_t)(tile + (4 * g + (col >> 2)) * L::up * 16 + rw * NW * 2 + (col & 3) * 8);
#pragma unroll
        for (int i = 0; i < NW / 16; i += B) {
            TrCols c[B];
            if constexpr (B == 8) tr_read8(c, v + i * 32, v + i * 32 + 16 * L::up * 16);
            else tr_read2(c, v + i * 32, v + i * 32 + 16 * L::up * 16);
#pragma unroll
            for (int j = 0; j < B; ++j) {
                const u32x4 f = {c[j].x.x, c[j].x.y, c[j].y.x, c[j].y.y};
                st.acc[i + j] = mma16<T>(f, hi, st.acc[i + j]);
                st.acc[i + j] = mma16<T>(f, lo, st.acc[i + j]);
            }
        }
    } else {
        const char* v = tile + 4 * g * L::up * 16 + (rw * NW + col) * 4;
#pragma unroll
        for (int i = 0; i < NW / 16; ++i) {
            f32x4 f;
#pragma unroll
            for (int j = 0; j < 4; ++j) f[j] = *reinterpret_cast<const float*>(v + j * L::up * 16 + i * 64);
            st.acc[i] = mma16<T>(__builtin_bit_cast(u32x4, f), __builtin_bit_cast(u32x4, s[0]), st.acc[i]);
        }
    }
}

template <typename T, int NR, int RW>
__global__ __launch_bounds__(kSeqThreads, 1) void k_seq_latent_attn(SeqLatentAttn a) {
    using L = LatentLds<T, NR>;
    constexpr int KT = LatentTile<T>::keys, NW = NR / RW, KS = L::ksteps / RW;
    extern __shared__ __align__(1024) char tiles[];
    __shared__ f32x4 parts[kSeqWaves * (KT / 16) * kWave];
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, col = lane & 15, g = lane >> 4;
    const int rw = wave % RW, h0 = ((int)blockIdx.y * (kSeqWaves / RW) + wave / RW) * 16;
    const int pos = a.state[1], ntiles = latent_tiles<T>(pos), nsplit = latent_splits(ntiles, a.ns, a.least), sp = blockIdx.x;
    if (sp >= nsplit) return;
    const int k0 = mul_div(ntiles, sp, nsplit) * KT, k1 = min(mul_div(ntiles, sp + 1, nsplit) * KT, pos + 1);
    const char* kc = a.kc + a.state[3] * a.slot_bytes;
    const int ksteps = a.crow / 64;
    const char* qr = a.q + (size_t)min(h0 + col, a.H - 1) * a.crow + g * 16;
    u32x4 qf[KS];
#pragma unroll
    for (int s = 0; s < KS; ++s) {
        qf[s] = ld16(qr + min(rw * KS + s, ksteps - 1) * 64);
        if (rw * KS + s >= ksteps) qf[s] = u32x4{0, 0, 0, 0};
    }
    latent_stage<T, NR>(tiles, kc, a.crow, k0, k1 - 1, wave, lane);
    if (k0 + KT < k1) latent_stage<T, NR>(tiles + L::tile, kc, a.crow, k0 + KT, k1 - 1, wave, lane);
    AttnState<NW> st;
    attn_reset(st);
    int buf = 0;
    for (int kb = k0; kb < k1; kb += KT) {
        // this wave's copies of the tile have arrived (the next tile's may be on their way), then everybody's; and nobody reads
        // the buffer of the tile before any more
        if (kb + KT < k1) wait_vm<L::copies>();
        else wait_vm<0>();
        lds_barrier();
        const int ahead = buf == 0 ? 2 : buf - 1;        // (buf + 2) % 3
        latent_tile<T, NR, RW>(st, qf, tiles + buf * L::tile, tiles + ahead * L::tile, kb + 2 * KT < k1, parts, kc, a.crow, kb, kb + 2 * KT, k1, a.scale_log2, rw,
                               wave, lane);
        buf = buf == 2 ? 0 : buf + 1;
    }
    if (h0 + col >= a.H) return;
    const size_t row = (size_t)sp * a.H + h0 + col;
    if (rw == 0 && g == 0) *reinterpret_cast<float2*>(a.ml + row * 2) = make_float2(st.m, st.l);
#pragma unroll
    for (int i = 0; i < NW / 16; ++i)
        if (rw * NW + i * 16 < a.rp) *reinterpret_cast<f32x4*>(a.acc + row * a.rp + rw * NW + i * 16 + g * 4) = st.acc[i];
}

// Workgroup (head, kLatentOut of its outputs; the head runs fastest, which keeps the workgroups of one head, who read the same
// partial results, on few XCDs): merges the splits of the head, then its rows of W_uv, four per wave, in fp32, and
// the output gate.
constexpr int kLatentOut = 16;
constexpr int kLatentSplits = kSeqThreads;
struct SeqLatentOut {
    const float *acc, *ml;
    const int* state;
    const float* sink;       // nullable
    const float* gate;       // nullable: [H * V] before the sigmoid
    const char* w_uv;        // T [H * V][pitch bytes]
    char* out;               // T [H * V]
    int H, V, pitch, ns, least, rp;
};
template <typename T>
__global__ __launch_bounds__(kSeqThreads) void k_seq_latent_out(SeqLatentOut a) {
    constexpr int U = Unit<T>::n, RPW = kLatentOut / kSeqWaves, NC = sizeof(T) == 2 ? 1 : 2;     // rows per wave, 1 KB loads per row
    __shared__ float f[kLatentSplits], red[kSeqWaves];
    __shared__ __align__(16) float sum[kSeqThreads * 4];
    __shared__ __align__(16) float lat[NC * 64 * U];
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, h = blockIdx.x, v0 = blockIdx.y * kLatentOut;
    u32x4 b[RPW][NC];
#pragma unroll
    for (int i = 0; i < RPW; ++i) {
        const int v = min(v0 + wave * RPW + i, a.V - 1);
#pragma unroll
        for (int c = 0; c < NC; ++c) b[i][c] = ld16(a.w_uv + ((size_t)h * a.V + v) * a.pitch + min(c * 1024 + lane * 16, a.pitch - 16));
    }
    const int nsplit = latent_splits(latent_tiles<T>(a.state[1]), a.ns, a.least);
    // a thread sums four latent columns over every nsg-th split; the first kM of these are requested before their weights
    // are known
    constexpr int kM = 16;
    const int r4 = a.rp / 4, nsg = kSeqThreads / r4, sg = tid / r4, x = tid - sg * r4;
    const float* p = a.acc + (size_t)h * a.rp + x * 4;
    const size_t split_stride = (size_t)a.H * a.rp;
    f32x4 t[kM];
    auto request = [&](int s0) {
#pragma unroll
        for (int j = 0; j < kM; ++j) t[j] = *reinterpret_cast<const f32x4*>(p + min(s0 + j * nsg, nsplit - 1) * split_stride);
    };
    request(sg);
    {                                                    // (at most one split per thread)
        const float2 ml = tid < nsplit ? *reinterpret_cast<const float2*>(a.ml + ((size_t)tid * a.H + h) * 2) : make_float2(kNegBig, 0.0f);
        const float snk = a.sink != nullptr ? a.sink[h] * kLog2e : kNegBig;
        const float wm = wave_max(ml.x);
        if (lane == 0) red[wave] = wm;
        __syncthreads();
        const float m = fmaxf(fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])), snk), e = fast_exp2(ml.x - m);
        const float l = block_sum(ml.y * e, red) + (a.sink != nullptr ? fast_exp2(snk - m) : 0.0f);
        f[tid] = e / l;
    }
    for (int i = tid; i < NC * 64 * U; i += kSeqThreads) lat[i] = 0.0f;
    __syncthreads();
    if (sg < nsg) {
        f32x4 s = {0.f, 0.f, 0.f, 0.f};
        for (int s0 = sg; s0 < nsplit; s0 += nsg * kM) {
            if (s0 != sg) request(s0);
#pragma unroll
            for (int j = 0; j < kM; ++j)
                if (s0 + j * nsg < nsplit) {
                    const float w = f[s0 + j * nsg];
#pragma unroll
                    for (int e = 0; e < 4; ++e) s[e] = fmadd(t[j][e], w, s[e]);
                }
        }
        *reinterpret_cast<f32x4*>(sum + sg * a.rp + x * 4) = s;
    }
    __syncthreads();
    for (int i = tid; i < a.rp; i += kSeqThreads) {
        float s = 0.0f;
        for (int j = 0; j < nsg; ++j) s += sum[j * a.rp + i];
        lat[i] = s;
    }
    __syncthreads();
    float acc[RPW];
#pragma unroll
    for (int i = 0; i < RPW; ++i) acc[i] = 0.0f;
#pragma unroll
    for (int c = 0; c < NC; ++c) {
        float y[U];
        const bool in = c * 1024 + lane * 16 < a.pitch;
#pragma unroll
        for (int e = 0; e < U; ++e) y[e] = in ? lat[(c * 64 + lane) * U + e] : 0.0f;
#pragma unroll
        for (int i = 0; i < RPW; ++i) {
            float w[U];
            unpack16<T>(b[i][c], w);
#pragma unroll
            for (int e = 0; e < U; ++e) acc[i] = fmadd(w[e], y[e], acc[i]);
        }
    }
#pragma unroll
    for (int i = 0; i < RPW; ++i) acc[i] = wave_sum(acc[i]);
    if (lane < RPW) {
        float o = 0.0f;
#pragma unroll
        for (int i = 0; i < RPW; ++i) o = lane == i ? acc[i] : o;
        const int v = v0 + wave * RPW + lane;
        if (v < a.V) {
            if (a.gate != nullptr) o *= sigmoid(a.gate[h * a.V + v]);
            reinterpret_cast<T*>(a.out)[h * a.V + v] = from_f32<T>(o);
        }
    }
}

// ---- residual streams --------------------------------------------------------------------------
// One workgroup per token: the streams after a sublayer (or at the start: all equal to the embedding, or at the end: as they
// are), and the next sublayer's input norm(sum_t in[t] x_t).
struct SeqStreams {
    float* x;                // [tokens][streams][width]
    const float* y;          // the sublayer's output, nullable
    const float* ys;         // nullable: [tokens][top][width], outputs of the chosen experts
    int top;
    float slot_weight;
    const float *mix, *out;  // null: the streams stay as they are
    const float* in;         // null: all one
    const float* w;          // norm weight; null: no next input
    float noff, eps;
    int streams, width;
    char* xb;
    int pitch;
    float* copy;             // nullable: receives the sum of the streams
    const int* rows;         // nullable: take token rows[t], write input t
    // the start
    const int* tokens;       // null: not the start
    const int* state;        // not null: one token, its position from here instead of pos0 + t
    const char *embed, *pos;
    int embed_pitch, pos0;
};
template <typename T, int S>
__global__ __launch_bounds__(kSeqThreads) void k_seq_streams(SeqStreams a) {
    __shared__ float red[kSeqWaves];
    extern __shared__ __align__(16) float us[];
    const int t = a.rows != nullptr ? a.rows[blockIdx.x] : (int)blockIdx.x;
    float* x = a.x + (size_t)t * a.streams * a.width;
    float mix[S][S], out[S], in[S];
#pragma unroll
    for (int s = 0; s < S; ++s) {
        const bool live = s < a.streams;
        in[s] = !live ? 0.0f : a.in != nullptr ? a.in[s] : 1.0f;
        out[s] = live && a.mix != nullptr ? a.out[s] : 0.0f;
#pragma unroll
        for (int j = 0; j < S; ++j) mix[s][j] = live && j < a.streams && a.mix != nullptr ? a.mix[s * a.streams + j] : 0.0f;
    }
    const T *e = nullptr, *ep = nullptr;
    if (a.tokens != nullptr) {
        e = reinterpret_cast<const T*>(a.embed + (size_t)a.tokens[t] * a.embed_pitch);
        if (a.pos != nullptr) ep = reinterpret_cast<const T*>(a.pos + (size_t)(a.state != nullptr ? a.state[1] : a.pos0 + t) * a.embed_pitch);
    }
    float ss = 0.0f;
    // N elements at a time (4 where the rows allow it); every thread reads back only what it has written
    auto sum = [&](auto n, int i) {
        constexpr int N = decltype(n)::value;
        float v[S][N];
        if (e != nullptr) {
#pragma unroll
            for (int j = 0; j < N; ++j) {
                const float z = to_f32(e[i + j]) + (ep != nullptr ? to_f32(ep[i + j]) : 0.0f);
#pragma unroll
                for (int s = 0; s < S; ++s) v[s][j] = z;
            }
        } else {
            float o[S][N], y[N];
#pragma unroll
            for (int s = 0; s < S; ++s) {
#pragma unroll
                for (int j = 0; j < N; ++j) o[s][j] = 0.0f;
                if (s < a.streams) add_n<N>(o[s], x + (size_t)s * a.width + i);
            }
#pragma unroll
            for (int j = 0; j < N; ++j) y[j] = 0.0f;
            if (a.ys != nullptr) {
                const float* ys = a.ys + (size_t)t * a.top * a.width + i;
                for (int k = 0; k < a.top; ++k) add_n<N>(y, ys + (size_t)k * a.width);
#pragma unroll
                for (int j = 0; j < N; ++j) y[j] *= a.slot_weight;
            }
            if (a.y != nullptr) add_n<N>(y, a.y + (size_t)t * a.width + i);
#pragma unroll
            for (int s = 0; s < S; ++s)
#pragma unroll
                for (int j = 0; j < N; ++j) {
                    if (a.mix == nullptr) {
                        v[s][j] = o[s][j];
                    } else {
                        v[s][j] = out[s] * y[j];
#pragma unroll
                        for (int k = 0; k < S; ++k) v[s][j] = fmadd(mix[k][s], o[k][j], v[s][j]);
                    }
                }
        }
        if (a.rows == nullptr) {
#pragma unroll
            for (int s = 0; s < S; ++s)
                if (s < a.streams) put_n<float, N>(x + (size_t)s * a.width + i, v[s]);
        }
        float u[N], all[N];
#pragma unroll
        for (int j = 0; j < N; ++j) {
            u[j] = all[j] = 0.0f;
#pragma unroll
            for (int s = 0; s < S; ++s) {
                u[j] = fmadd(in[s], v[s][j], u[j]);
                all[j] += s < a.streams ? v[s][j] : 0.0f;
            }
            us[i + j] = u[j];
            ss = fmadd(u[j], u[j], ss);
        }
        if (a.copy != nullptr) put_n<float, N>(a.copy + (size_t)t * a.width + i, all);
    };
    const int w4 = (a.width & 3) ? 0 : a.width;
    for (int i = threadIdx.x * 4; i < w4; i += kSeqThreads * 4) sum(std::integral_constant<int, 4>{}, i);
    for (int i = w4 + threadIdx.x; i < a.width; i += kSeqThreads) sum(std::integral_constant<int, 1>{}, i);
    if (a.w == nullptr) return;
    const float inv = inv_rms(block_sum(ss, red), a.width, a.eps);
    T* xb = reinterpret_cast<T*>(a.xb + (size_t)blockIdx.x * a.pitch);
    auto put = [&](auto n, int i) {
        constexpr int N = decltype(n)::value;
        float w[N], v[N];
#pragma unroll
        for (int j = 0; j < N; ++j) w[j] = a.noff;
        add_n<N>(w, a.w + i);
#pragma unroll
        for (int j = 0; j < N; ++j) v[j] = us[i + j] * inv * w[j];
        put_n<T, N>(xb + i, v);
    };
    for (int i = threadIdx.x * 4; i < w4; i += kSeqThreads * 4) put(std::integral_constant<int, 4>{}, i);
    for (int i = w4 + threadIdx.x; i < a.width; i += kSeqThreads) put(std::integral_constant<int, 1>{}, i);
}

}  // namespace cfpp
