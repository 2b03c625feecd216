// Kernels and host side of the sequence models (include/cfpp_seq.h).
//
// Prefill (a portion of T tokens): per layer
//   k_seq_gemm (q, k, v rows + bias) -> k_seq_qkv_finish (norms over the projections, rotation, value mixing) -> k_seq_attn ->
//   k_seq_append (what later portions can see goes into the cache) -> k_seq_gemm (output rows) -> k_seq_postnorm ->
//   k_seq_gemm (up rows with the activation) -> k_seq_gemm (down rows) -> k_seq_postnorm;
//   table experts: the same two products over tiles of tokens sorted by expert (k_seq_route), plus the shared expert's.
// Decode (one token): five launches per layer, each with its neighbours' work fused in:
//   k_seq_gemv (residual sum + norm of the sublayer before | q, k, v rows + bias)
//   k_seq_attn_decode (norms, rotation, value mixing, cache append, split-KV attention, merge)
//   k_seq_gemv (output rows)
//   k_seq_gemv (residual sum + norm | up rows of the chosen and the shared experts | activation)
//   k_seq_gemv (down rows of all of them, weighted and summed)
// then k_seq_gemv over the vocabulary (both last norms | head rows | soft cap | best logit per workgroup) and k_seq_pick.
// Latent mixers (seq_latent.hpp): in portions k_seq_latent_finish and a product that makes the keys and values of all heads come
// before k_seq_attn, and nothing is appended after it; in decode k_seq_latent_q, k_seq_latent_attn and k_seq_latent_out take the
// place of k_seq_attn_decode.  Residual streams: k_seq_streams instead of k_seq_postnorm; in decode the launches of the output
// and down rows update the streams themselves.
#include <hip/hip_runtime.h>
#include <math.h>
#include <stdint.h>
#include <string.h>

#include <algorithm>
#include <map>
#include <new>
#include <tuple>
#include <type_traits>
#include <utility>
#include <vector>

#include "cfpp_seq.h"
#include "seq_device.hpp"
#include "seq_latent.hpp"

using namespace cfpp;

namespace {

enum : int { kStToken = 0, kStPos = 1, kStSteps = 2, kStSlot = 3 };
constexpr int kAttnCols = 16;          // query columns of a decode item (one MFMA column tile)
constexpr int kMaxSeqSplit = 64;       // KV splits of a decode step
constexpr int kAttnWgs = 1;            // ... sized for this many workgroups per compute unit

// ------------------------------------------------------------------------------------------------
// small kernels
// ------------------------------------------------------------------------------------------------
__global__ void k_seq_set_state(int* state, int slot, int token, int pos, int steps) {
    if (threadIdx.x == 0) {
        state[kStToken] = token;
        state[kStPos] = pos;
        state[kStSlot] = slot;
        if (steps >= 0) state[kStSteps] = steps;
    }
}

__global__ void k_seq_fill_zero(u32x4* p, size_t n) {
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x) p[i] = u32x4{0, 0, 0, 0};
}

// One workgroup per token: embedding row -> residual stream (fp32) and product input (T).
template <typename T>
__global__ __launch_bounds__(kSeqThreads) void k_seq_embed(const int* __restrict__ tokens, const char* __restrict__ embed, int pitch, int width,
                                                           float* __restrict__ x, char* __restrict__ xb) {
    const int t = blockIdx.x;
    const T* e = reinterpret_cast<const T*>(embed + (size_t)tokens[t] * pitch);
    T* o = reinterpret_cast<T*>(xb + (size_t)t * pitch);
    for (int i = threadIdx.x; i < width; i += kSeqThreads) {
        x[(size_t)t * width + i] = to_f32(e[i]);
        o[i] = e[i];
    }
}

// x <- norm(alpha x + y + slot_weight * sum_j ys[t, j]); one workgroup per token.  `rows`: take the token rows[t] instead of
// t and only write xb (the last norm, on the rows whose logits are wanted).
struct SeqPostNorm {
    const float* x;
    float* x_out;            // may be x
    const float* y;          // nullable
    const float* ys;         // nullable: [T][top][width], outputs of the chosen experts
    int top;
    float slot_weight;
    const float* w;
    float alpha, eps, noff;  // noff: the norm weight is noff + w
    int width;
    char* xb;
    int pitch;
    const int* rows;
    float* copy;             // nullable: receives the new residual row too
};
template <typename T>
__global__ __launch_bounds__(kSeqThreads) void k_seq_postnorm(SeqPostNorm a) {
    __shared__ float red[kSeqWaves];
    extern __shared__ __align__(16) float ts[];
    const int t = a.rows != nullptr ? a.rows[blockIdx.x] : (int)blockIdx.x;
    const float* x = a.x + (size_t)t * a.width;
    char* xb = a.xb + (size_t)blockIdx.x * a.pitch;
    float ss = 0.0f;
    // N elements at a time (4 where the rows allow it); every thread reads back only what it has written
    auto sum = [&](auto n, int i) {
        constexpr int N = decltype(n)::value;
        float s[N];
#pragma unroll
        for (int j = 0; j < N; ++j) s[j] = 0.0f;
        if (a.ys != nullptr) {
            const float* ys = a.ys + (size_t)t * a.top * a.width + i;
            for (int e = 0; e < a.top; ++e) add_n<N>(s, ys + (size_t)e * a.width);
#pragma unroll
            for (int j = 0; j < N; ++j) s[j] *= a.slot_weight;
        }
        if (a.y != nullptr) add_n<N>(s, a.y + (size_t)t * a.width + i);
        float v[N];
#pragma unroll
        for (int j = 0; j < N; ++j) v[j] = 0.0f;
        add_n<N>(v, x + i);
#pragma unroll
        for (int j = 0; j < N; ++j) {
            if (a.rows == nullptr) v[j] = fmadd(a.alpha, v[j], s[j]);
            ts[i + j] = v[j];
            ss = fmadd(v[j], v[j], ss);
        }
    };
    auto out = [&](auto n, int i, float inv) {
        constexpr int N = decltype(n)::value;
        float w[N], v[N];
#pragma unroll
        for (int j = 0; j < N; ++j) w[j] = a.noff;
        add_n<N>(w, a.w + i);
#pragma unroll
        for (int j = 0; j < N; ++j) v[j] = ts[i + j] * inv * w[j];
        if (a.rows == nullptr) {
            put_n<float, N>(a.x_out + (size_t)t * a.width + i, v);
            if (a.copy != nullptr) put_n<float, N>(a.copy + (size_t)t * a.width + i, v);
        }
        put_n<T, N>(reinterpret_cast<T*>(xb) + i, v);
    };
    const int w4 = (a.width & 3) ? 0 : a.width;
    for (int i = threadIdx.x * 4; i < w4; i += kSeqThreads * 4) sum(std::integral_constant<int, 4>{}, i);
    for (int i = w4 + threadIdx.x; i < a.width; i += kSeqThreads) sum(std::integral_constant<int, 1>{}, i);
    const float inv = inv_rms(block_sum(ss, red), a.width, a.eps);
    for (int i = threadIdx.x * 4; i < w4; i += kSeqThreads * 4) out(std::integral_constant<int, 4>{}, i, inv);
    for (int i = w4 + threadIdx.x; i < a.width; i += kSeqThreads) out(std::integral_constant<int, 1>{}, i, inv);
}

// One workgroup per token: raw q | k | v rows (fp32, biases included) -> norm over all of q and all of k, rotation, value
// mixing -> q [T][H][Dp], portion k [G][cap][Dp] and v [G][cap][Vp].
struct SeqQkv {
    const float* qkv;
    int ld;
    const float *qn, *kn;
    const float2* cs;        // [positions][rot / 2]
    float eps, lambda;
    int H, G, D, Dp, V, Vp, rot, pos0, cap;
    int v_role;              // 0: plain, 1: this layer's values are the ones later layers mix in, 2: mix
    float* v_first;          // [T][G * V]
    char *q, *k, *v;
};
template <typename T>
__global__ __launch_bounds__(kSeqThreads) void k_seq_qkv_finish(SeqQkv a) {
    __shared__ float2 red[kSeqWaves];
    const int t = blockIdx.x, nq = a.H * a.D, nk = a.G * a.D, nv = a.G * a.V;
    const float* q = a.qkv + (size_t)t * a.ld;
    const float *k = q + nq, *v = k + nk;
    const float2 sums = block_sum2(share_sq(q, nq, threadIdx.x), share_sq(k, nk, threadIdx.x), red);
    const float iq = inv_rms(sums.x, nq, a.eps), ik = inv_rms(sums.y, nk, a.eps);
    const float2* cs = a.cs + (size_t)(a.pos0 + t) * (a.rot / 2);
    char* qo = a.q + (size_t)t * a.H * a.Dp * sizeof(T);
    char* ko = a.k + (size_t)t * a.Dp * sizeof(T);
    char* vo = a.v + (size_t)t * a.Vp * sizeof(T);
    const size_t khead = (size_t)a.cap * a.Dp * sizeof(T), vhead = (size_t)a.cap * a.Vp * sizeof(T);
    // four elements at a time: head `h`, elements d .. d + 3 of its padded row (zeros past the end: the padding is written
    // too, since layers of other sizes share these buffers)
    auto rotated = [&](const float* row, const float* w, float inv, int d) {
        f32x4 x, y;
        const bool whole = d + 3 < a.D && ((uintptr_t)(row + d) & 15) == 0 && ((uintptr_t)(w + d) & 15) == 0;
        if (whole) {
            const f32x4 xr = *reinterpret_cast<const f32x4*>(row + d), wr = *reinterpret_cast<const f32x4*>(w + d);
#pragma unroll
            for (int j = 0; j < 4; ++j) x[j] = xr[j] * wr[j];
        } else {
#pragma unroll
            for (int j = 0; j < 4; ++j) x[j] = d + j < a.D ? row[d + j] * w[d + j] : 0.0f;
        }
#pragma unroll
        for (int j = 0; j < 4; j += 2) {
            const bool r = d + j < a.rot;
            const float2 cc = r ? cs[(d + j) / 2] : make_float2(1.0f, 0.0f);
            y[j] = rotate_finish(RotIn{x[j], x[j + 1], cc.x, -cc.y}, inv);
            y[j + 1] = rotate_finish(RotIn{x[j + 1], x[j], cc.x, cc.y}, inv);
        }
        return y;
    };
    const int q4 = a.Dp / 4, v4 = a.Vp / 4;
    for (int i = threadIdx.x; i < a.H * q4; i += kSeqThreads) {
        const int h = i / q4, d = (i - h * q4) * 4;
        store4<T>(qo + ((size_t)h * a.Dp + d) * sizeof(T), rotated(q + h * a.D, a.qn + h * a.D, iq, d));
    }
    for (int i = threadIdx.x; i < a.G * q4; i += kSeqThreads) {
        const int g = i / q4, d = (i - g * q4) * 4;
        store4<T>(ko + g * khead + d * sizeof(T), rotated(k + g * a.D, a.kn + g * a.D, ik, d));
    }
    for (int i = threadIdx.x; i < a.G * v4; i += kSeqThreads) {
        const int g = i / v4, d = (i - g * v4) * 4;
        f32x4 x;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            x[j] = 0.0f;
            if (d + j < a.V) {
                float* first = a.v_first + (size_t)t * nv + g * a.V + d + j;
                x[j] = v[g * a.V + d + j];
                if (a.v_role == 1) *first = x[j];
                if (a.v_role == 2) x[j] = (1.0f - a.lambda) * x[j] + a.lambda * *first;
            }
        }
        store4<T>(vo + g * vhead + d * sizeof(T), x);
    }
}

// Portion rows -> cache rows: one workgroup per kept position.
struct SeqAppend { const char *k, *v; char *kc, *vc; int G, krow, vrow, cap, rows, first, row0; };
__global__ __launch_bounds__(kSeqThreads) void k_seq_append(SeqAppend a) {
    const int t = a.first + blockIdx.x, r = a.row0 + blockIdx.x;
    const int ku = a.krow / 16, vu = a.vrow / 16;
    for (int i = threadIdx.x; i < a.G * (ku + vu); i += kSeqThreads) {
        const int g = i / (ku + vu), u = i - g * (ku + vu);
        if (u < ku)
            *reinterpret_cast<u32x4*>(a.kc + ((size_t)g * a.rows + r) * a.krow + u * 16) = ld16(a.k + ((size_t)g * a.cap + t) * a.krow + u * 16);
        else
            *reinterpret_cast<u32x4*>(a.vc + ((size_t)g * a.rows + r) * a.vrow + (u - ku) * 16) = ld16(a.v + ((size_t)g * a.cap + t) * a.vrow + (u - ku) * 16);
    }
}

// ------------------------------------------------------------------------------------------------
// matrix products of a portion: out[token][row] = W[row] . a[token]
// ------------------------------------------------------------------------------------------------
// kEpiHeads: rows of keys of all heads, then rows of values of all heads, each head's rows [position] in a buffer of its own.
// kEpiStreams (one token): the output row goes into the residual streams.
enum : int { kEpiF32 = 0, kEpiRelu2 = 1, kEpiGated = 2, kEpiHead = 3, kEpiHeads = 4, kEpiStreams = 5 };
struct SeqGemm {
    const char* w;           // [n rows][kbytes]
    const char* a;           // [tokens][lda bytes]
    int n, m, kbytes, lda;
    const float* bias;       // nullable (kEpiF32, kEpiGated)
    float* yf;               // kEpiF32 / kEpiHead: [tokens][ldy]
    int ldy;
    char* yt;                // kEpiRelu2 / kEpiGated: T, [tokens][ldyt bytes]; kEpiHeads: keys
    int ldyt;
    float mul, cap;          // kEpiHead
    char* yv;                // kEpiHeads: values; key rows of kd elements, kp bytes apart, heads kh bytes apart; values alike
    int nk, kd, kp, vd, vp;  // ... nk: rows of keys
    size_t kh, vh;
    // tiles of tokens sorted by expert (tile_off null: a plain product)
    const int* tile_off;     // [experts + 1] prefix sums of tiles
    const int* row_off;      // [experts + 1] prefix sums of sorted slots
    const int* slots;        // sorted slots: token * top + j
    int experts, slot_div;   // input row of slot s: s / slot_div
    size_t w_stride;
};

// rows of 128 bytes: units of row r are stored at unit ^ swz(r), which spreads 16 consecutive rows over all banks
__device__ __forceinline__ int swz128(int row) { return (row >> 1) & 7; }

template <typename T, int BW, int BT, int EPI>
__global__ __launch_bounds__(kSeqThreads, 2) void k_seq_gemm(SeqGemm p) {
    constexpr int MI = BW / 32, NI = BT / 32;            // 16 x 16 tiles of a wave; waves are 2 (rows) x 2 (tokens)
    constexpr int WI = BW / 32, AI = BT / 32;            // 1 KB copies per wave and k step
    __shared__ __align__(1024) char lds[2][(BW + BT) * kRowBytes];
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63;
    const int wr = wave >> 1, wc = wave & 1;

    const int tiles_w = (p.n + BW - 1) / BW;
    int tw, tt, m = p.m, row0 = 0;
    const char* w = p.w;
    {
        // every XCD works on a contiguous range of tiles; inside it tiles go through groups of up to 8 token tiles
        const int total = gridDim.x, per = total / 8, rem = total % 8, xcd = blockIdx.x % 8, i = blockIdx.x / 8;
        const int id = xcd * per + min(xcd, rem) + i;
        if (p.tile_off != nullptr) {
            tt = id / tiles_w;
            tw = id - tt * tiles_w;
            if (tt >= p.tile_off[p.experts]) return;
            int lo = 0, hi = p.experts;                  // last expert whose first tile is <= tt
            while (hi - lo > 1) {
                const int mid = (lo + hi) >> 1;
                if (p.tile_off[mid] <= tt) lo = mid; else hi = mid;
            }
            // (experts without tokens have no tiles: skip to the one that owns the tile)
            while (p.tile_off[lo + 1] <= tt) ++lo;
            w += (size_t)lo * p.w_stride;
            row0 = p.row_off[lo] + (tt - p.tile_off[lo]) * BT;
            m = p.row_off[lo + 1] - row0;
            tt = 0;
        } else {
            const int tiles_t = (p.m + BT - 1) / BT, group = 8 * tiles_w, gi = id / group, first = gi * 8;
            const int gs = min(8, tiles_t - first), r = id - gi * group;
            tt = first + r % gs;
            tw = r / gs;
        }
    }
    const char* src_w[WI];
    const char* src_a[AI];
#pragma unroll
    for (int i = 0; i < WI; ++i) {
        const int r = wave * (BW / 4) + i * 8 + (lane >> 3);
        src_w[i] = w + (size_t)min(tw * BW + r, p.n - 1) * p.kbytes + ((lane & 7) ^ swz128(r)) * 16;
    }
#pragma unroll
    for (int i = 0; i < AI; ++i) {
        const int r = wave * (BT / 4) + i * 8 + (lane >> 3);
        int tok = min(tt * BT + r, m - 1);
        if (p.tile_off != nullptr) tok = p.slots[row0 + tok] / p.slot_div;
        src_a[i] = p.a + (size_t)tok * p.lda + ((lane & 7) ^ swz128(r)) * 16;
    }
    auto stage = [&](int buf, int k) {
        char* base = lds[buf];
#pragma unroll
        for (int i = 0; i < WI; ++i) copy_to_lds16(src_w[i] + k, base + (wave * (BW / 4) + i * 8) * kRowBytes);
#pragma unroll
        for (int i = 0; i < AI; ++i) copy_to_lds16(src_a[i] + k, base + BW * kRowBytes + (wave * (BT / 4) + i * 8) * kRowBytes);
    };
    f32x4 acc[MI][NI];
#pragma unroll
    for (int i = 0; i < MI; ++i)
#pragma unroll
        for (int j = 0; j < NI; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};

    const int col = lane & 15, g = lane >> 4, nk = p.kbytes / kRowBytes;
    stage(0, 0);
    for (int k = 0; k < nk; ++k) {
        __syncthreads();                                 // this step's tile has arrived; the other buffer is free
        if (k + 1 < nk) stage((k + 1) & 1, (k + 1) * kRowBytes);
        const char* lw = lds[k & 1];
        const char* la = lw + BW * kRowBytes;
#pragma unroll
        for (int s = 0; s < 2; ++s) {
            u32x4 fw[MI], fa[NI];
#pragma unroll
            for (int i = 0; i < MI; ++i) {
                const int r = wr * (BW / 2) + i * 16 + col;
                fw[i] = *reinterpret_cast<const u32x4*>(lw + r * kRowBytes + ((s * 4 + g) ^ swz128(r)) * 16);
            }
#pragma unroll
            for (int j = 0; j < NI; ++j) {
                const int r = wc * (BT / 2) + j * 16 + col;
                fa[j] = *reinterpret_cast<const u32x4*>(la + r * kRowBytes + ((s * 4 + g) ^ swz128(r)) * 16);
            }
#pragma unroll
            for (int i = 0; i < MI; ++i)
#pragma unroll
                for (int j = 0; j < NI; ++j) acc[i][j] = mma16<T>(fw[i], fa[j], acc[i][j]);
        }
    }
    // kEpiHeads: where row n goes at position 0, and the bytes from one position to the next; `whole`: rows n0 .. n0 + 3 lie together
    auto head_row = [&](int n, int& rp) {
        const bool k = n < p.nk;
        const int d = k ? p.kd : p.vd, m = k ? n : n - p.nk, h = m / d;
        rp = k ? p.kp : p.vp;
        return (k ? p.yt + h * p.kh : p.yv + h * p.vh) + (m - h * d) * (int)sizeof(T);
    };
    char* dst[MI];
    int pitch[MI];
    bool whole[MI];
    if constexpr (EPI == kEpiHeads) {
#pragma unroll
        for (int i = 0; i < MI; ++i) {
            const int n0 = min(tw * BW + wr * (BW / 2) + i * 16 + g * 4, p.n - 1);
            dst[i] = head_row(n0, pitch[i]);
            whole[i] = ((p.kd | p.vd) & 3) == 0 && n0 + 3 < p.n;       // (n0, the keys' rows and the heads' rows are multiples of four)
        }
    }
#pragma unroll
    for (int j = 0; j < NI; ++j) {
        const int tl = tt * BT + wc * (BT / 2) + j * 16 + col;
        if (tl >= m) continue;
        const int row = p.tile_off != nullptr ? p.slots[row0 + tl] : tl;
#pragma unroll
        for (int i = 0; i < MI; ++i) {
            const int n0 = tw * BW + wr * (BW / 2) + i * 16 + g * 4;
            const f32x4 v = acc[i][j];
            if constexpr (EPI == kEpiF32 || EPI == kEpiHead) {
                float* y = p.yf + (size_t)row * p.ldy + n0;
                f32x4 o = v;
                if (EPI == kEpiF32 && p.bias != nullptr) {
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        if (n0 + r < p.n) o[r] += p.bias[n0 + r];
                }
                if (EPI == kEpiHead) {
#pragma unroll
                    for (int r = 0; r < 4; ++r) o[r] = soft_cap(o[r] * p.mul, p.cap);
                }
                if (n0 + 3 < p.n && (p.ldy & 3) == 0) {
                    *reinterpret_cast<f32x4*>(y) = o;
                } else {
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        if (n0 + r < p.n) y[r] = o[r];
                }
            } else if constexpr (EPI == kEpiRelu2) {
                T* y = reinterpret_cast<T*>(p.yt + (size_t)row * p.ldyt) + n0;
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (n0 + r < p.n) y[r] = from_f32<T>(relu2(v[r]));
            } else if constexpr (EPI == kEpiHeads) {
                if (whole[i]) {
                    store4<T>(dst[i] + (size_t)row * pitch[i], v);
                } else {
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        if (n0 + r < p.n) {
                            int rp;
                            char* b = head_row(n0 + r, rp);
                            *reinterpret_cast<T*>(b + (size_t)row * rp) = from_f32<T>(v[r]);
                        }
                }
            } else {
                T* y = reinterpret_cast<T*>(p.yt + (size_t)row * p.ldyt) + n0 / 2;
#pragma unroll
                for (int r = 0; r < 4; r += 2)
                    if (n0 + r < p.n) {
                        const float bg = p.bias != nullptr ? p.bias[n0 + r] : 0.0f, bu = p.bias != nullptr ? p.bias[n0 + r + 1] : 0.0f;
                        y[r / 2] = from_f32<T>(silu(v[r] + bg) * (v[r + 1] + bu));
                    }
            }
        }
    }
}

// Slots (token * top + j) sorted by expert, per layer with table experts: one workgroup per such layer.
struct SeqRoute { const int* table; int* tile_off; int* row_off; int* slots; int experts, top; };
__global__ __launch_bounds__(1024) void k_seq_route(const SeqRoute* layers, const int* __restrict__ tokens, int T, int bt) {
    extern __shared__ int sh[];
    const SeqRoute a = layers[blockIdx.x];
    int *cnt = sh, *next = sh + a.experts;
    for (int e = threadIdx.x; e < a.experts; e += blockDim.x) cnt[e] = 0;
    __syncthreads();
    const int n = T * a.top;
    for (int s = threadIdx.x; s < n; s += blockDim.x) {
        const int t = s / a.top;
        atomicAdd(&cnt[a.table[(size_t)tokens[t] * a.top + (s - t * a.top)]], 1);
    }
    __syncthreads();
    if (threadIdx.x == 0) {
        int rows = 0, tiles = 0;
        for (int e = 0; e < a.experts; ++e) {
            const int c = cnt[e];
            a.row_off[e] = rows;
            a.tile_off[e] = tiles;
            next[e] = rows;
            rows += c;
            tiles += (c + bt - 1) / bt;
        }
        a.row_off[a.experts] = rows;
        a.tile_off[a.experts] = tiles;
    }
    __syncthreads();
    for (int s = threadIdx.x; s < n; s += blockDim.x) {
        const int t = s / a.top;
        a.slots[atomicAdd(&next[a.table[(size_t)tokens[t] * a.top + (s - t * a.top)]], 1)] = s;
    }
}

// ------------------------------------------------------------------------------------------------
// attention of a portion
// ------------------------------------------------------------------------------------------------
// The query columns of one key / value head are (token, head of the group), head fastest; a workgroup takes 64 CT of them
// and walks the keys its tokens can see, first the cached ones (positions before k_split), then those in the buffer.  Behind a
// key's own row comes the part that all heads share, if there is one.  The softmax is online, the sink is added to the
// denominator at the end.
struct SeqAttn {
    const char *q, *k, *v, *kc, *vc;
    const char* kr;          // rows of the shared part, of position 0 on
    char* out;
    const float* sink;       // nullable
    const float* gate;       // nullable: [T][ldg], the outputs are multiplied by its sigmoid
    int T, H, R, dsteps, qrow, krow, vrow, V, vtiles, pos0, chunk, cap, rows, ldo, k_split, runits, rrow, ldg;
    float scale_log2;
};
template <int UN> __device__ __forceinline__ int swz_key(int row) { return UN % 16 ? (row >> 1) & 7 : row & 15; }

// (the next tile's keys go straight to the other LDS buffer and its values into registers while this one is worked on)
// (NK: elements of a key row in LDS, NT: value columns.  The products run over all of them, without branches between the reads
// of LDS: past the end of the query there are zeros, and of the columns past the end of a value nothing is stored)
template <typename T, int NK, int NT, int CT>
__global__ __launch_bounds__(kSeqThreads, (NT <= 128 ? 2 : 1)) void k_seq_attn(SeqAttn a) {
    constexpr int KT = sizeof(T) == 2 ? 64 : 32;
    constexpr int NB = NK * (int)sizeof(T), UN = NB / 16;                    // bytes and units of a key row in LDS
    constexpr int VS = VtSteps<T, KT, NT, kSeqThreads>::n;
    __shared__ __align__(1024) char ks[2][KT * NB];
    __shared__ __align__(16) char vt[NT * VtTile<T, KT>::pitch];
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, col = lane & 15, g = lane >> 4;
    // the longest walks first; every second group of eight runs backwards, so that each XCD (workgroups go round them) gets as
    // many long ones as the others
    const int gq = blockIdx.y, ncols = a.T * a.R, gx = gridDim.x;
    int bx = blockIdx.x;
    if (((bx >> 3) & 1) && (bx | 7) < gx) bx ^= 7;
    const int c0 = (gx - 1 - bx) * 64 * CT;

    int pq[CT], first[CT], tok[CT], head[CT];
    u32x4 qf[CT][NB / 64];
    AttnState<NT> st[CT];
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
        const int cc = min(c0 + (wave * CT + ct) * 16 + col, ncols - 1);
        tok[ct] = cc / a.R;
        head[ct] = gq * a.R + (cc - tok[ct] * a.R);
        pq[ct] = a.pos0 + tok[ct];
        first[ct] = chunk_start(pq[ct], a.chunk);
        const char* qr = a.q + ((size_t)tok[ct] * a.H + head[ct]) * a.qrow + g * 16;
#pragma unroll
        for (int s = 0; s < NB / 64; ++s) {
            qf[ct][s] = ld16(qr + min(s, a.dsteps - 1) * 64);
            if (s >= a.dsteps) qf[ct][s] = u32x4{0, 0, 0, 0};
        }
        attn_reset(st[ct]);
    }
    // keys the workgroup needs, and those every column of this wave sees / any column sees
    const int t_first = c0 / a.R, t_last = min(a.T - 1, (c0 + 64 * CT - 1) / a.R);
    const int k_first = chunk_start(a.pos0 + t_first, a.chunk), k_end = a.pos0 + t_last + 1;
    const int w_first = min(c0 + wave * CT * 16, ncols - 1) / a.R, w_last = min(c0 + (wave + 1) * CT * 16 - 1, ncols - 1) / a.R;
    const int all_lo = chunk_start(a.pos0 + w_last, a.chunk), all_hi = a.pos0 + w_first;
    const int any_lo = chunk_start(a.pos0 + w_first, a.chunk), any_hi = a.pos0 + w_last;
    const int dunits = a.krow / 16, vunits = a.vrow / 16;

    // tiles: [k_first, k_split) in the cache, then [k_split, k_end) in the buffer
    struct Tile { int k0, hi; const char *k, *v; };      // first key, end of its part, row of position 0
    auto tile_at = [&](int k0) {
        const bool cached = k0 < a.k_split;
        const size_t row0 = (size_t)gq * (cached ? a.rows : a.cap) - (cached ? chunk_start(a.pos0, a.chunk) : a.k_split);
        return Tile{k0, cached ? min(k_end, a.k_split) : k_end, (cached ? a.kc : a.k) + (ptrdiff_t)row0 * a.krow, (cached ? a.vc : a.v) + (ptrdiff_t)row0 * a.vrow};
    };
    u32x4 vr[VS][4];
    auto fetch = [&](const Tile& t, int buf) {
        for (int i = wave; i < KT * NB / 1024; i += kSeqWaves) {
            const int r = (i * 64 + lane) / UN, u = ((i * 64 + lane) % UN) ^ swz_key<UN>(r), key = min(t.k0 + r, t.hi - 1);
            const char* src = t.k + (ptrdiff_t)key * a.krow + (u < dunits ? u : 0) * 16;
            if (u >= dunits && u < dunits + a.runits) src = a.kr + (ptrdiff_t)key * a.rrow + (u - dunits) * 16;
            copy_to_lds16(src, ks[buf] + i * 1024);
        }
        vt_request<T, KT, kSeqThreads, 0, VS>(vr, vunits, tid, [&](int key) { return t.v + (ptrdiff_t)min(t.k0 + key, t.hi - 1) * a.vrow; });
    };
    Tile t = tile_at(k_first);
    fetch(t, 0);
    for (int buf = 0;; buf ^= 1) {
        __syncthreads();                                 // the tile's keys are there; nobody reads the last tile's values any more
        vt_store<T, KT, kSeqThreads, 0, VS>(vr, vt, vunits, tid);
        const int next = min(t.k0 + KT, t.hi);
        Tile tn = t;
        if (next < k_end) {
            tn = tile_at(next);
            fetch(tn, buf ^ 1);
        }
        lds_barrier();                                   // (waits for the stores to LDS, not for the next tile)
        if (t.k0 <= any_hi && next > any_lo) {
            // the fragments of the next 16 keys are read while these are multiplied
            f32x4 s[CT][KT / 16];
            u32x4 kf[2][NB / 64];
            auto read = [&](int kt) __attribute__((always_inline)) {
                const int r = kt * 16 + col;
#pragma unroll
                for (int d = 0; d < NB / 64; ++d)
                    kf[kt & 1][d] = *reinterpret_cast<const u32x4*>(ks[buf] + r * NB + ((d * 4 + g) ^ swz_key<UN>(r)) * 16);
            };
            read(0);
#pragma unroll
            for (int kt = 0; kt < KT / 16; ++kt) {
                if (kt + 1 < KT / 16) read(kt + 1);
                __builtin_amdgcn_sched_barrier(0);
#pragma unroll
                for (int ct = 0; ct < CT; ++ct) {
                    s[ct][kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                    for (int d = 0; d < NB / 64; ++d) s[ct][kt] = mma16<T>(kf[kt & 1][d], qf[ct][d], s[ct][kt]);
                }
            }
            __builtin_amdgcn_sched_barrier(0);
            const bool full = t.k0 + KT <= t.hi && t.k0 >= all_lo && t.k0 + KT - 1 <= all_hi;
#pragma unroll
            for (int ct = 0; ct < CT; ++ct) {
#pragma unroll
                for (int kt = 0; kt < KT / 16; ++kt)
#pragma unroll
                    for (int r = 0; r < 4; ++r) s[ct][kt][r] *= a.scale_log2;
                if (!full) {
#pragma unroll
                    for (int kt = 0; kt < KT / 16; ++kt)
#pragma unroll
                        for (int r = 0; r < 4; ++r) {
                            const int key = t.k0 + kt * 16 + g * 4 + r;
                            if (key >= t.hi || key > pq[ct] || key < first[ct]) s[ct][kt][r] = kMasked;
                        }
                }
                attn_softmax<NT, KT / 16>(st[ct], s[ct], NT / 16);
            }
            __builtin_amdgcn_sched_barrier(0);           // (values read ahead of the softmax would take its registers)
            attn_pv<T, NT, KT, CT>(st, s, vt, NT / 16, lane);
        }
        if (next >= k_end) break;
        t = tn;
    }
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) {
        if (c0 + (wave * CT + ct) * 16 + col >= ncols) continue;
        const float snk = a.sink != nullptr ? a.sink[head[ct]] * kLog2e : kNegBig, m = fmaxf(st[ct].m, snk), c = fast_exp2(st[ct].m - m);
        const float f = c / (st[ct].l * c + fast_exp2(snk - m));       // (no sink: the last term is zero)
        T* o = reinterpret_cast<T*>(a.out + (size_t)tok[ct] * a.ldo) + head[ct] * a.V;
        const float* gate = a.gate + (size_t)tok[ct] * a.ldg + head[ct] * a.V;
#pragma unroll
        for (int i = 0; i < NT / 16; ++i)
            if (i < a.vtiles) {
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const int v = i * 16 + g * 4 + r;
                    if (v < a.V) o[v] = from_f32<T>(a.gate != nullptr ? st[ct].acc[i][r] * f * sigmoid(gate[v]) : st[ct].acc[i][r] * f);
                }
            }
    }
}

// ------------------------------------------------------------------------------------------------
// attention of one token
// ------------------------------------------------------------------------------------------------
// Workgroup (split, key / value head x group of 16 query heads).  Its prologue makes q from the raw projection; the split
// that holds the newest position also makes that position's k and v rows and appends them.  Every wave takes every fourth
// tile of the split's keys; the waves merge in LDS, the splits through memory, by the workgroup that arrives last.
struct SeqAttnDec {
    const float* qkv;
    const float *qn, *kn, *sink;
    const float2* cs;
    const int* state;
    char *kc, *vc;           // this layer's caches, slot 0
    size_t k_slot, v_slot;   // bytes per slot
    float* v_first;
    char* out;               // T [H * V]
    float* part;             // [items][ns][16][Vp + 2]
    int* cnt;                // [items][kHeadCntStride], self-resetting
    float eps, lambda, scale_log2;
    int v_role, H, G, R, nct, D, V, rot, chunk, krow, vrow, dsteps, vtiles, rows, ns;
};
template <typename T, int NT> struct DecTile { static constexpr int kt = sizeof(T) == 2 ? 32 : (NT <= 128 ? 32 : 16); };

template <typename T, int NT>
__global__ __launch_bounds__(kSeqThreads) void k_seq_attn_decode(SeqAttnDec a) {
    constexpr int KT = DecTile<T, NT>::kt, NB = NT * (int)sizeof(T);
    constexpr int VB = NT * VtTile<T, KT>::pitch, MB = kAttnCols * NT * 4;
    constexpr int VS = VtSteps<T, KT, NT, kWave>::n, KF = KT / 16;
    __shared__ __align__(16) char buf[kSeqWaves * (VB > MB ? VB : MB)];
    __shared__ __align__(16) char qs[kAttnCols * NB];
    __shared__ float2 red2[kSeqWaves];
    __shared__ float wm[kSeqWaves][kAttnCols], wl[kSeqWaves][kAttnCols];
    __shared__ float sm[kMaxSeqSplit][kAttnCols], sl[kMaxSeqSplit][kAttnCols];
    __shared__ int last;
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, col = lane & 15, g = lane >> 4;
    const int item = blockIdx.y, gq = item / a.nct, cols0 = (item - gq * a.nct) * kAttnCols, ncols = min(kAttnCols, a.R - cols0);
    const int pos = a.state[kStPos], slot = a.state[kStSlot];
    // tiles of KT keys are shared evenly among the splits, no more of them than give every wave a tile
    const int k_first = chunk_start(pos, a.chunk), ntiles = (pos - k_first + KT) / KT;
    const int nsplit = min(a.ns, (ntiles + kSeqWaves - 1) / kSeqWaves), sp = blockIdx.x;
    if (sp >= nsplit) return;
    const int k0 = k_first + mul_div(ntiles, sp, nsplit) * KT, k1 = min(k_first + mul_div(ntiles, sp + 1, nsplit) * KT, pos + 1);
    char* kc = a.kc + slot * a.k_slot + (size_t)gq * a.rows * a.krow;
    char* vc = a.vc + slot * a.v_slot + (size_t)gq * a.rows * a.vrow;
    const int vunits = a.vrow / 16;

    u32x4 kf[KF][NB / 64], vr[VS][4];
    auto fetch = [&](int kb) {
#pragma unroll
        for (int kt = 0; kt < KF; ++kt) {
            const char* kr = kc + (size_t)(min(kb + kt * 16 + col, k1 - 1) - k_first) * a.krow + g * 16;
#pragma unroll
            for (int d = 0; d < NB / 64; ++d)
                if (d < a.dsteps) kf[kt][d] = ld16(kr + d * 64);
        }
        vt_request<T, KT, kWave, 0, VS>(vr, vunits, lane, [&](int key) { return vc + (size_t)(min(kb + key, k1 - 1) - k_first) * a.vrow; });
    };
    // everything the prologue reads is requested up front: one round trip instead of one per use
    const int nq = a.H * a.D, nk = a.G * a.D;
    const float *q = a.qkv, *k = q + nq, *v = k + nk;
    const float2* cs = a.cs + (size_t)pos * (a.rot / 2);
    const bool newest = k1 == pos + 1;                   // this split makes and appends the newest position's rows
    // NT threads per head; the first kQ passes are held in registers, more query heads go through a loop
    constexpr int kQ = 2, kHeads = kSeqThreads / NT;
    const int own0 = (gq * a.R + cols0) * a.D, qd = tid % NT, qc = tid / NT;
    RotIn rq[kQ], rk;
    float vn = 0.0f, vm = 0.0f;
#pragma unroll
    for (int i = 0; i < kQ; ++i)
        if (qc + i * kHeads < ncols && qd < a.D) rq[i] = rotate_request(q + own0, a.qn + own0, qc + i * kHeads, qd, a.D, a.rot, cs);
    if (newest && tid < a.D) rk = rotate_request(k, a.kn, gq, tid, a.D, a.rot, cs);
    if (newest && tid < a.V) {
        vn = v[gq * a.V + tid];
        if (a.v_role == 2) vm = a.v_first[gq * a.V + tid];
    }
    const float sq = share_sq(q, nq, tid), sk = newest ? share_sq(k, nk, tid) : 0.0f;
    // the wave's first tile, unless the newest position, which is not in the cache yet, is in it
    int kb = k0 + wave * KT;
    const bool early = kb + KT <= pos && kb < k1;
    if (early) fetch(kb);

    for (int i = tid; i < kAttnCols * NB / 16; i += kSeqThreads) reinterpret_cast<u32x4*>(qs)[i] = u32x4{0, 0, 0, 0};
    const float2 sums = block_sum2(sq, sk, red2);        // (its barriers also separate the zeros from what follows)
    const float iq = inv_rms(sums.x, nq, a.eps);
    T* qt = reinterpret_cast<T*>(qs);
#pragma unroll
    for (int i = 0; i < kQ; ++i)
        if (qc + i * kHeads < ncols && qd < a.D) qt[(qc + i * kHeads) * NT + qd] = from_f32<T>(rotate_finish(rq[i], iq));
#pragma unroll 1
    for (int c = qc + kQ * kHeads; c < ncols; c += kHeads)
        if (qd < a.D) qt[c * NT + qd] = from_f32<T>(rotate_finish(rotate_request(q + own0, a.qn + own0, c, qd, a.D, a.rot, cs), iq));
    if (newest) {
        const float ik = inv_rms(sums.y, nk, a.eps);
        if (tid < a.D) reinterpret_cast<T*>(kc + (size_t)(pos - k_first) * a.krow)[tid] = from_f32<T>(rotate_finish(rk, ik));
        if (tid < a.V) {
            if (a.v_role == 1) a.v_first[gq * a.V + tid] = vn;
            if (a.v_role == 2) vn = (1.0f - a.lambda) * vn + a.lambda * vm;
            reinterpret_cast<T*>(vc + (size_t)(pos - k_first) * a.vrow)[tid] = from_f32<T>(vn);
        }
    }
    __syncthreads();
    u32x4 qf[NB / 64];
#pragma unroll
    for (int s = 0; s < NB / 64; ++s)
        if (s < a.dsteps) qf[s] = *reinterpret_cast<const u32x4*>(qs + col * NB + s * 64 + g * 16);

    AttnState<NT> st;
    attn_reset(st);
    char* vt = buf + wave * VB;
    if (!early && kb < k1) fetch(kb);
    for (; kb < k1; kb += KT * kSeqWaves) {
        f32x4 s[KF];
#pragma unroll
        for (int kt = 0; kt < KF; ++kt) {
            s[kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int d = 0; d < NB / 64; ++d)
                if (d < a.dsteps) s[kt] = mma16<T>(kf[kt][d], qf[d], s[kt]);
        }
        vt_store<T, KT, kWave, 0, VS>(vr, vt, vunits, lane);
        if (kb + KT * kSeqWaves < k1) fetch(kb + KT * kSeqWaves);
#pragma unroll
        for (int kt = 0; kt < KF; ++kt)
#pragma unroll
            for (int r = 0; r < 4; ++r) s[kt][r] = kb + kt * 16 + g * 4 + r < k1 ? s[kt][r] * a.scale_log2 : kMasked;
        attn_softmax<NT, KF>(st, s, a.vtiles);
        __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
        __builtin_amdgcn_wave_barrier();                 // the tile in LDS belongs to this wave alone
        attn_pv<T, NT, KT, 1>(&st, &s, vt, a.vtiles, lane);
        __builtin_amdgcn_wave_barrier();
    }
    // waves of the workgroup
    __syncthreads();
    float* wacc = reinterpret_cast<float*>(buf);         // [wave][column][NT]
    if (g == 0) {
        wm[wave][col] = st.m;
        wl[wave][col] = st.l;
    }
#pragma unroll
    for (int i = 0; i < NT / 16; ++i)
        if (i < a.vtiles) *reinterpret_cast<f32x4*>(wacc + (wave * kAttnCols + col) * NT + i * 16 + g * 4) = st.acc[i];
    __syncthreads();
    const int vp = a.vtiles * 16, stride = vp + 2;
    float* part = a.part + (size_t)item * a.ns * kAttnCols * stride;
    for (int i = tid; i < ncols * vp; i += kSeqThreads) {
        const int c = i / vp, x = i - c * vp;
        const float m = fmaxf(fmaxf(wm[0][c], wm[1][c]), fmaxf(wm[2][c], wm[3][c]));
        float acc = 0.0f, l = 0.0f;
#pragma unroll
        for (int w = 0; w < kSeqWaves; ++w) {
            const float f = fast_exp2(wm[w][c] - m);
            acc = fmadd(wacc[(w * kAttnCols + c) * NT + x], f, acc);
            l = fmadd(wl[w][c], f, l);
        }
        if (nsplit == 1) {
            const int h = gq * a.R + cols0 + c;
            const float snk = a.sink[h] * kLog2e, mm = fmaxf(m, snk), f = fast_exp2(m - mm);
            if (x < a.V) reinterpret_cast<T*>(a.out)[(size_t)h * a.V + x] = from_f32<T>(acc * f / (l * f + fast_exp2(snk - mm)));
        } else {
            float* pr = part + ((size_t)sp * kAttnCols + c) * stride;
            st_agent(pr + 2 + x, acc);
            if (x == 0) {
                st_agent(pr, m);
                st_agent(pr + 1, l);
            }
        }
    }
    if (nsplit == 1) return;
    drain_memory_ops();
    __syncthreads();
    if (tid == 0) {
        int* ctr = a.cnt + item * kHeadCntStride;
        const int done = __hip_atomic_fetch_add(ctr, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == nsplit - 1;
        if (done) __hip_atomic_store(ctr, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        last = done;
    }
    __syncthreads();
    if (!last) return;
    // pairs of value columns, kM splits at a time; the first ones travel together with the maxima
    constexpr int kM = 8;
    const int half = vp / 2, pairs = ncols * half, split_stride = kAttnCols * stride;
    float2 pv[kM];
    auto request = [&](const float* p0, int s0) {
#pragma unroll
        for (int j = 0; j < kM; ++j) ld_agent2(p0 + (size_t)min(s0 + j, nsplit - 1) * split_stride, pv[j].x, pv[j].y);
    };
    for (int i = tid; i < nsplit * ncols; i += kSeqThreads) {
        const int s = i / ncols, c = i - s * ncols;
        ld_agent2(part + (size_t)s * split_stride + c * stride, sm[s][c], sl[s][c]);
    }
    int i = tid, c = i / half, x = (i - c * half) * 2;
    if (i < pairs) request(part + c * stride + 2 + x, 0);
    __syncthreads();
#pragma unroll 1
    while (i < pairs) {
        const int h = gq * a.R + cols0 + c;
        const float snk = a.sink[h] * kLog2e;
        float m = snk;
        for (int s = 0; s < nsplit; ++s) m = fmaxf(m, sm[s][c]);
        float ax = 0.0f, ay = 0.0f, l = fast_exp2(snk - m);
#pragma unroll 1
        for (int s0 = 0;;) {
#pragma unroll
            for (int j = 0; j < kM; ++j)
                if (s0 + j < nsplit) {
                    const float f = fast_exp2(sm[s0 + j][c] - m);
                    ax = fmadd(pv[j].x, f, ax);
                    ay = fmadd(pv[j].y, f, ay);
                    l = fmadd(sl[s0 + j][c], f, l);
                }
            s0 += kM;
            if (s0 >= nsplit) break;
            request(part + c * stride + 2 + x, s0);
        }
        T* o = reinterpret_cast<T*>(a.out) + (size_t)h * a.V + x;
        if (x < a.V) o[0] = from_f32<T>(ax / l);
        if (x + 1 < a.V) o[1] = from_f32<T>(ay / l);
        i += kSeqThreads;
        c = i / half;
        x = (i - c * half) * 2;
        if (i < pairs) request(part + c * stride + 2 + x, 0);
    }
}

// ------------------------------------------------------------------------------------------------
// matrix-vector products of one token
// ------------------------------------------------------------------------------------------------
// A wave streams its weight rows as one sequence of 1 KB chunks (one wave-wide load each), four per step, two steps in
// flight, the first two requested before the prologue.  The input sits in LDS.  Rows go to waves in equal contiguous shares.
//
// ROWS: the outputs are the rows of up to `top` chosen matrices and of one that is always there, one after the other.
// KCAT: every output is the sum of the products with the rows of these matrices (the chosen ones weighted 1 / top); the
// inputs lie one after the other in LDS.  top == 0: a plain matrix.
enum : int { kInVector = 0, kInNorm = 1, kInEmbed = 2 };
struct SeqGemv {
    int input;
    const float *x, *y;      // kInNorm: the residual row and the sublayer's output that is still to be added (nullable)
    float* x_out;            // ... where the new residual row goes (not x); nullable
    float* copy;             // nullable: a second copy
    const float *nw, *nw2;   // norm weights; nw2 (nullable): a second norm follows
    float alpha, eps, noff;  // noff: the norms' weights are noff + nw
    int width;
    const char* embed;
    int embed_pitch;
    const int* state;
    const char* xin;         // kInVector: the T inputs; chosen ones at multiples of seg_e bytes, the other at top * seg_e
    int seg_e;
    // matrices
    const char *w_e, *w_s;   // chosen (matrix stride e_stride) and always-on rows
    size_t e_stride;
    int pitch_e, pitch_s;    // row bytes
    const int* table;
    int top, units_e, units_s;   // ROWS: output units per chosen matrix and of the other; KCAT: units_s outputs
    // outputs
    const float* bias;
    float* yf;
    char* yt;                // T; ROWS: a chosen matrix' outputs at multiples of seg_y bytes
    int seg_y;
    float mul, cap;          // kEpiHead
    float* xs;               // kEpiStreams: the streams [streams][width], updated in place
    const float *mix, *out, *in;          // ... in: of the next sublayer, null: all one
    int streams;
    float *u, *sum;          // ... its input before the norm; the sum of the streams (nullable)
    float* best_v;           // kEpiHead: best logit of every workgroup and its row
    int* best_i;
    int park, park_n;        // LDS: offset of the finished outputs, outputs per wave at most
};
constexpr int kGemvChunk = 1024;      // bytes of a row per wave-wide load
constexpr int kGemvLoads = 4;         // loads per step
constexpr int kGemvWgs = 4;           // workgroups per compute unit

template <typename T, int EPI, bool KCAT>
__global__ __launch_bounds__(kSeqThreads, 2) void k_seq_gemv(SeqGemv p) {
    constexpr int UR = EPI == kEpiGated ? 2 : 1;         // rows per output
    extern __shared__ __align__(16) char smem[];
    __shared__ float red[kSeqWaves];
    __shared__ float bv[kSeqWaves];
    __shared__ int bi[kSeqWaves];
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63;

    const int nch_e = (p.pitch_e + kGemvChunk - 1) / kGemvChunk, nch_s = (p.pitch_s + kGemvChunk - 1) / kGemvChunk;
    const int nch_all_e = KCAT ? p.top * nch_e : 0;      // chunks of the chosen part of a row
    const int nch = KCAT ? nch_all_e + nch_s : nch_s;    // chunks of a whole row
    const int outputs = KCAT ? p.units_s : p.top * p.units_e + p.units_s;
    const int nw = gridDim.x * kSeqWaves, gw = blockIdx.x * kSeqWaves + wave;
    const int u0 = mul_div(outputs, gw, nw), u1 = mul_div(outputs, gw + 1, nw);
    int expert = 0;                                      // lane j: the j-th chosen matrix
    if (p.top > 0) {
        const int tok = p.state[kStToken];
        if (lane < p.top) expert = p.table[(size_t)tok * p.top + lane];
    }

    // ---- the wave's chunks, one after the other.  Requests are never conditional (past the end they repeat the last
    // chunk), so that the number of loads in flight is known and a step waits for its own loads only.
    const char* ask_row = nullptr;                       // row (KCAT: of the segment) being requested
    int ask_lim = 0, ask_n = 0, ask_c = 0;               // offset of its last 16 bytes, its chunks, the next chunk
    int ask_u = 0, ask_seg = 0;                          // output; matrix: the seg-th chosen one, or p.top: the one that is always there
    int ask_j = 0, ask_r = 0;                            // ROWS: output inside the matrix, row of the output
    auto open_row = [&]() __attribute__((always_inline)) {
        // (both alternatives are read before one is chosen: a choice between two members' addresses would keep the
        // parameters in memory)
        const bool e = ask_seg < p.top;
        const char *we = p.w_e + (size_t)__builtin_amdgcn_readlane(expert, e ? ask_seg : 0) * p.e_stride, *ws = p.w_s;
        const int pe = p.pitch_e, ps = p.pitch_s, pitch = e ? pe : ps;
        ask_row = (e ? we : ws) + (size_t)(KCAT ? ask_u : ask_j * UR + ask_r) * pitch;
        ask_lim = pitch - 16;
        ask_n = e ? nch_e : nch_s;
    };
    auto next_chunk = [&]() __attribute__((always_inline)) {
        if (ask_c + 1 < ask_n) {
            ask_c = ask_c + 1;
            return;
        }
        const bool same = KCAT ? ask_seg + 1 < p.top + (nch_s > 0 ? 1 : 0) : ask_r + 1 < UR;    // the output has another row
        if (!same && ask_u + 1 >= u1) return;
        ask_c = 0;
        const int du = same ? 0 : 1;
        ask_u = ask_u + du;
        if constexpr (KCAT) {
            ask_seg = same ? ask_seg + 1 : 0;
        } else {
            ask_r = same ? ask_r + 1 : 0;
            const int j = ask_j + du;
            const bool hop = j == p.units_e && ask_seg < p.top;
            ask_j = hop ? 0 : j;
            ask_seg = ask_seg + (hop ? 1 : 0);
        }
        open_row();
    };
    auto request = [&](u32x4 (&b)[kGemvLoads]) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < kGemvLoads; ++i) {
            b[i] = ld_stream16(ask_row + min(ask_c * kGemvChunk + lane * 16, ask_lim));
            next_chunk();
        }
    };
    ask_u = min(u0, outputs - 1);                        // (a wave without rows asks for a valid one and uses nothing)
    ask_r = ask_c = 0;
    ask_seg = KCAT || p.top == 0 ? 0 : min(ask_u / p.units_e, p.top);
    ask_j = ask_u - ask_seg * p.units_e;
    open_row();

    // ---- prologue: the input into LDS, zeros up to whole chunks.  What it reads is requested before the first weights
    // (loads return in order), in registers up to kPre units per thread, the rest afterwards.
    constexpr int kPre = KCAT ? 8 : 4;
    T* xs = reinterpret_cast<T*>(smem);
    const int nunits = nch * (kGemvChunk / 16);          // units of the input in LDS
    auto input_unit = [&](int i) -> u32x4 {
        const int c = i / (kGemvChunk / 16), o = i - c * (kGemvChunk / 16);
        const bool e = c < nch_all_e;
        const int seg = e ? c / nch_e : p.top, off = (e ? c - seg * nch_e : c - nch_all_e) * kGemvChunk + o * 16;
        const int pe = p.pitch_e, ps = p.pitch_s;
        u32x4 v = {0, 0, 0, 0};
        if (off < (e ? pe : ps)) v = ld16(p.xin + (size_t)seg * p.seg_e + off);
        return v;
    };
    const f32x4 *x4 = reinterpret_cast<const f32x4*>(p.x), *y4 = reinterpret_cast<const f32x4*>(p.y), *n4 = reinterpret_cast<const f32x4*>(p.nw);
    const int w4 = (p.width & 3) ? 0 : p.width / 4;
    u32x4 pv[kPre];
    f32x4 px[kPre], py[kPre], pn[kPre];
    if constexpr (KCAT) {
#pragma unroll
        for (int i = 0; i < kPre; ++i)
            if (tid + i * kSeqThreads < nunits) pv[i] = input_unit(tid + i * kSeqThreads);
    } else if (p.input == kInNorm) {
#pragma unroll
        for (int i = 0; i < kPre; ++i) {
            const int k = min(tid + i * kSeqThreads, w4 - 1);
            if (w4 > 0) {
                px[i] = x4[k];
                py[i] = p.y != nullptr ? y4[k] : f32x4{0.f, 0.f, 0.f, 0.f};
                pn[i] = n4[k];
            }
        }
    }
    // kEpiStreams: lane (output, stream); the first outputs' streams and the connections
    constexpr int kS = CFPP_SEQ_MAX_STREAMS;
    const int st_t = lane % kS, st_o = lane / kS;
    float so[kS], sm[kS], s_out = 0.0f, s_in = 0.0f, s_bias = 0.0f;
    auto streams_of = [&](int u) __attribute__((always_inline)) {
#pragma unroll
        for (int s = 0; s < kS; ++s) so[s] = p.xs[(size_t)min(s, p.streams - 1) * p.width + u];
        s_bias = p.bias != nullptr ? p.bias[u] : 0.0f;
    };
    if constexpr (EPI == kEpiStreams) {
        const int t = min(st_t, p.streams - 1);
#pragma unroll
        for (int s = 0; s < kS; ++s) sm[s] = s < p.streams ? p.mix[s * p.streams + t] : 0.0f;
        s_out = p.out[t];
        s_in = st_t >= p.streams ? 0.0f : p.in != nullptr ? p.in[t] : 1.0f;
        streams_of(min(u0 + st_o, outputs - 1));
    }
    __builtin_amdgcn_sched_barrier(0);
    u32x4 b0[kGemvLoads], b1[kGemvLoads];
    request(b0);
    request(b1);
    __builtin_amdgcn_sched_barrier(0);

    if constexpr (KCAT) {
#pragma unroll
        for (int i = 0; i < kPre; ++i)
            if (tid + i * kSeqThreads < nunits) reinterpret_cast<u32x4*>(smem)[tid + i * kSeqThreads] = pv[i];
        for (int i = tid + kPre * kSeqThreads; i < nunits; i += kSeqThreads) reinterpret_cast<u32x4*>(smem)[i] = input_unit(i);
    } else {
        for (int i = p.width + tid; i < nch * kGemvChunk / (int)sizeof(T); i += kSeqThreads) xs[i] = from_f32<T>(0.0f);
        const bool keep = blockIdx.x == 0 && p.x_out != nullptr;
        if (p.input == kInEmbed) {
            const T* e = reinterpret_cast<const T*>(p.embed + (size_t)p.state[kStToken] * p.embed_pitch);
            for (int i = tid; i < p.width; i += kSeqThreads) {
                xs[i] = e[i];
                if (keep) p.x_out[i] = to_f32(e[i]);
            }
        } else {
            float* ts = reinterpret_cast<float*>(smem + nch * kGemvChunk);
            float ss = 0.0f;
            // (every thread reads back only what it has written)
            auto sum4 = [&](int i, f32x4 x, f32x4 y) {
                f32x4 t;
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    t[j] = fmadd(p.alpha, x[j], y[j]);
                    ss = fmadd(t[j], t[j], ss);
                }
                reinterpret_cast<f32x4*>(ts)[i] = t;
            };
#pragma unroll
            for (int i = 0; i < kPre; ++i)
                if (tid + i * kSeqThreads < w4) sum4(tid + i * kSeqThreads, px[i], py[i]);
            for (int i = tid + kPre * kSeqThreads; i < w4; i += kSeqThreads) sum4(i, x4[i], p.y != nullptr ? y4[i] : f32x4{0.f, 0.f, 0.f, 0.f});
            for (int i = w4 * 4 + tid; i < p.width; i += kSeqThreads) {
                const float t = fmadd(p.alpha, p.x[i], p.y != nullptr ? p.y[i] : 0.0f);
                ss = fmadd(t, t, ss);
                ts[i] = t;
            }
            float inv = inv_rms(block_sum(ss, red), p.width, p.eps);
            ss = 0.0f;
            auto out1 = [&](int i, float v) {
                ss = fmadd(v, v, ss);
                if (keep) {
                    p.x_out[i] = v;
                    if (p.copy != nullptr) p.copy[i] = v;
                }
                if (p.nw2 != nullptr) ts[i] = v; else xs[i] = from_f32<T>(v);
            };
            auto out4 = [&](int i, f32x4 w) {
                const f32x4 t = reinterpret_cast<const f32x4*>(ts)[i];
#pragma unroll
                for (int j = 0; j < 4; ++j) out1(i * 4 + j, t[j] * inv * (p.noff + w[j]));
            };
#pragma unroll
            for (int i = 0; i < kPre; ++i)
                if (tid + i * kSeqThreads < w4) out4(tid + i * kSeqThreads, pn[i]);
            for (int i = tid + kPre * kSeqThreads; i < w4; i += kSeqThreads) out4(i, n4[i]);
            for (int i = w4 * 4 + tid; i < p.width; i += kSeqThreads) out1(i, ts[i] * inv * (p.noff + p.nw[i]));
            if (p.nw2 != nullptr) {
                __syncthreads();
                inv = inv_rms(block_sum(ss, red), p.width, p.eps);
                for (int i = tid; i < p.width; i += kSeqThreads) xs[i] = from_f32<T>(ts[i] * inv * (p.noff + p.nw2[i]));
            }
        }
    }
    __syncthreads();

    // ---- the rows; finished outputs are parked in LDS and stored together at the end
    const int n_out = u1 - u0;
    float* park = reinterpret_cast<float*>(smem + p.park) + wave * p.park_n * UR;
    float acc = 0.0f;
    int c_use = 0, r_use = 0, done = 0;                  // chunk and row of the output in work, outputs finished
    const float we = p.top > 0 ? 1.0f / (float)p.top : 1.0f;
    auto consume = [&](const u32x4 (&b)[kGemvLoads]) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < kGemvLoads; ++i)
            if (done < n_out) {
                const u32x4 x = *reinterpret_cast<const u32x4*>(smem + c_use * kGemvChunk + lane * 16);
                if constexpr (KCAT)
                    acc = fmadd(c_use < nch_all_e ? we : 1.0f, dot16<T>(b[i], x, 0.0f), acc);
                else
                    acc = dot16<T>(b[i], x, acc);
                if (++c_use == nch) {
                    c_use = 0;
                    const float v = wave_sum(acc);
                    acc = 0.0f;
                    if (lane == 0) park[done * UR + r_use] = v;
                    if (UR == 2 && r_use == 0) {
                        r_use = 1;
                    } else {
                        r_use = 0;
                        ++done;
                    }
                }
            }
    };
    const int steps = (n_out * UR * nch + kGemvLoads - 1) / kGemvLoads;
    for (int s = 2; s < steps; s += 2) {                 // the steps before the last two
        consume(b0);
        request(b0);
        consume(b1);
        request(b1);
    }
    consume(b0);
    consume(b1);
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
    float top_v = -INFINITY;
    int top_i = 0;
    if constexpr (EPI == kEpiStreams) {
        for (int i0 = 0; i0 < n_out; i0 += kWave / kS) {
            const int i = min(i0 + st_o, n_out - 1), u = u0 + i;
            if (i0 > 0) streams_of(u);
            float z = s_out * (park[i] + s_bias);
#pragma unroll
            for (int s = 0; s < kS; ++s) z = fmadd(sm[s], so[s], z);
            const bool live = st_t < p.streams && i0 + st_o < n_out;
            if (live) p.xs[(size_t)st_t * p.width + u] = z;
            float next = s_in * z, all = st_t < p.streams ? z : 0.0f;
#pragma unroll
            for (int m = 1; m < kS; m <<= 1) {
                next += xor_shfl(next, m);
                all += xor_shfl(all, m);
            }
            if (live && st_t == 0) {
                p.u[u] = next;
                if (p.sum != nullptr) p.sum[u] = all;
            }
        }
        return;
    }
    for (int i = lane; i < n_out; i += kWave) {
        const float v = park[i * UR];
        const int u = u0 + i;
        if constexpr (EPI == kEpiF32) {
            p.yf[u] = p.bias != nullptr ? v + p.bias[u] : v;
        } else if constexpr (EPI == kEpiHead) {
            const float z = soft_cap(v * p.mul, p.cap);
            p.yf[u] = z;
            if (z > top_v) {
                top_v = z;
                top_i = u;
            }
        } else if constexpr (EPI == kEpiRelu2) {
            reinterpret_cast<T*>(p.yt)[u] = from_f32<T>(relu2(v));
        } else {
            const int b = u < p.top * p.units_e ? u / p.units_e : p.top;
            const float bg = p.bias != nullptr ? p.bias[2 * u] : 0.0f, bu = p.bias != nullptr ? p.bias[2 * u + 1] : 0.0f;
            reinterpret_cast<T*>(p.yt + (size_t)b * p.seg_y)[u - b * p.units_e] = from_f32<T>(silu(v + bg) * (park[i * UR + 1] + bu));
        }
    }
    if constexpr (EPI == kEpiHead) {
        for (int m = 1; m < kWave; m <<= 1) {            // the wave's best; the lowest row on ties
            const float ov = __shfl_xor(top_v, m, kWave);
            const int oi = __shfl_xor(top_i, m, kWave);
            if (ov > top_v || (ov == top_v && oi < top_i)) {
                top_v = ov;
                top_i = oi;
            }
        }
        if (lane == 0) {
            bv[wave] = top_v;
            bi[wave] = top_i;
        }
        __syncthreads();
        if (tid == 0) {
            for (int w = 1; w < kSeqWaves; ++w)
                if (bv[w] > bv[0]) {
                    bv[0] = bv[w];
                    bi[0] = bi[w];
                }
            p.best_v[blockIdx.x] = bv[0];
            p.best_i[blockIdx.x] = bi[0];
        }
    }
}

// The largest logit (lowest row on ties) becomes the next step's token.
__global__ __launch_bounds__(kSeqThreads) void k_seq_pick(const float* best_v, const int* best_i, int n, int* state, int* history, int history_cap) {
    __shared__ float v[kSeqThreads];
    __shared__ int r[kSeqThreads];
    float bv = -INFINITY;
    int bi = 0x7fffffff;
    for (int i = threadIdx.x; i < n; i += kSeqThreads)
        if (best_v[i] > bv || (best_v[i] == bv && best_i[i] < bi)) {
            bv = best_v[i];
            bi = best_i[i];
        }
    v[threadIdx.x] = bv;
    r[threadIdx.x] = bi;
    for (int h = kSeqThreads / 2; h > 0; h /= 2) {
        __syncthreads();
        if ((int)threadIdx.x < h) {
            const int o = threadIdx.x + h;
            if (v[o] > v[threadIdx.x] || (v[o] == v[threadIdx.x] && r[o] < r[threadIdx.x])) {
                v[threadIdx.x] = v[o];
                r[threadIdx.x] = r[o];
            }
        }
    }
    if (threadIdx.x == 0) {
        const int tok = r[0] == 0x7fffffff ? 0 : r[0];     // (no finite logit: any row will do, but it must be one)
        if (state[kStSteps] < history_cap) history[state[kStSteps]] = tok;
        state[kStToken] = tok;
        state[kStPos] += 1;
        state[kStSteps] += 1;
    }
}

// angle = position * frequency, evaluated in double; cos and sin times `mul`, rounded once
__global__ void k_seq_rope_table(float2* t, const double* freq, double mul, int half, int positions) {
    const size_t n = (size_t)positions * half;
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x) {
        const double a = (double)(i / half) * freq[i % half];
        t[i] = make_float2((float)(mul * cos(a)), (float)(mul * sin(a)));
    }
}

// ================================================================================================
// host side
// ================================================================================================
int up_to(int a, int b) { return (a + b - 1) / b * b; }
int ceil_div(int a, int b) { return (a + b - 1) / b; }
size_t pitch_of(int K, int esize) { return (size_t)up_to(K * esize, kRowBytes); }

struct LayerPlan {
    cfpp_seq_layer d;
    int R, nct, Dp, Vp, krow, vrow, rows, n_qkv, v_role, NT;
    float2* cs;
    char *kc, *vc;
    int ns;
    // latent mixers: the cache rows are kc's, in bytes
    bool latent, own;
    int lpitch, crow;        // latent part (a padded weight row), whole cache row
    int plain, shared, qrow; // plain and rotated part of a key, whole query row
    int least;               // tiles of a split of a decode step at least
    int rp;                  // latent columns of the partial results of a decode step
    int gate_at;             // first gate row of the projection
    int route;               // index among the layers with table experts, -1: none
};

}  // namespace

struct cfpp_seq {
    cfpp_seq_desc d;
    std::vector<LayerPlan> layers;
    int esize, cus, portion, device, xpitch;
    std::vector<void*> owned;
    size_t bytes = 0;
    bool failed = false;
    // portion buffers
    int *tokens, *want;
    float *x, *qkv, *y, *ys, *v_first;
    char *xb, *q, *k, *v, *o, *h, *hs, *wb;
    int ld_qkv;
    SeqRoute* routes;
    std::vector<SeqRoute> host_routes;
    int max_experts = 0;
    // decode buffers
    int* state;
    int *history, *cnt, *best_i;
    float *dx[2], *dy, *dres, *logits, *part, *best_v;
    float *du;               // residual streams: the next sublayer's input before its norm
    int history_cap, pos = 0, launches = 0, head_grid = 0;
    hipGraphExec_t graph = nullptr;
    hipStream_t capture = nullptr;

    template <typename P> P* alloc(size_t n) {
        void* p = nullptr;
        const size_t b = (std::max<size_t>(n, 1) * sizeof(P) + 255) / 256 * 256;
        if (failed || hipMalloc(&p, b) != hipSuccess) {
            failed = true;
            return nullptr;
        }
        owned.push_back(p);
        bytes += b;
        hipLaunchKernelGGL(k_seq_fill_zero, dim3((unsigned)std::min<size_t>((b / 16 + 255) / 256, 4096)), dim3(256), 0, nullptr,
                           reinterpret_cast<u32x4*>(p), b / 16);
        return reinterpret_cast<P*>(p);
    }
};

namespace {

int last_error() {
    const hipError_t e = hipGetLastError();
    return e == hipSuccess ? CFPP_OK : (int)e;
}

// dynamic LDS beyond the default limit has to be asked for, once per kernel
template <typename K>
void allow_lds(K kernel, size_t bytes) {
    if (bytes > 65536) (void)hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
}

// ---- portions ----------------------------------------------------------------------------------
// max_tiles: upper bound of the expert products' token tiles (their number is known on the device only)
template <typename T, int EPI>
void launch_gemm(const SeqGemm& g, int max_tiles, bool big, hipStream_t st) {
    const int tile = big ? 128 : 64, tw = ceil_div(g.n, tile), tt = g.tile_off != nullptr ? max_tiles : ceil_div(g.m, tile);
    if (big) hipLaunchKernelGGL((k_seq_gemm<T, 128, 128, EPI>), dim3(tw * tt), dim3(kSeqThreads), 0, st, g);
    else hipLaunchKernelGGL((k_seq_gemm<T, 64, 64, EPI>), dim3(tw * tt), dim3(kSeqThreads), 0, st, g);
}

// large tiles where they still give every compute unit one
template <typename T, int EPI>
void gemm(const cfpp_seq* s, const SeqGemm& g, hipStream_t st) {
    launch_gemm<T, EPI>(g, 0, ceil_div(g.n, 128) * ceil_div(g.m, 128) >= s->cus, st);
}

// tokens per tile of the expert products
int expert_tile(const LayerPlan& L, int n) { return (long long)n * L.d.top >= 96LL * L.d.experts ? 128 : 64; }

template <typename T, int EPI>
void expert_gemm(const cfpp_seq* s, const LayerPlan& L, SeqGemm g, int n, hipStream_t st) {
    const SeqRoute& r = s->host_routes[L.route];
    const int bt = expert_tile(L, n), slots = n * L.d.top;
    g.m = slots;
    g.tile_off = r.tile_off;
    g.row_off = r.row_off;
    g.slots = r.slots;
    g.experts = L.d.experts;
    launch_gemm<T, EPI>(g, slots / bt + std::min(L.d.experts, slots), bt == 128, st);
}

template <typename T, int NK, int NT>
void launch_attn(const SeqAttn& a, int G, int cus, hipStream_t st) {
    const int cols = a.T * a.R;
    if constexpr (sizeof(T) == 2) {                      // (fp32: two column tiles do not fit the registers)
        if (ceil_div(cols, 128) * G >= 2 * cus) {
            hipLaunchKernelGGL((k_seq_attn<T, NK, NT, 2>), dim3(ceil_div(cols, 128), G), dim3(kSeqThreads), 0, st, a);
            return;
        }
    }
    hipLaunchKernelGGL((k_seq_attn<T, NK, NT, 1>), dim3(ceil_div(cols, 64), G), dim3(kSeqThreads), 0, st, a);
}

template <typename T>
void attn(const cfpp_seq* s, const SeqAttn& a, int G, hipStream_t st) {
    const int nk = a.qrow / (int)sizeof(T), nv = a.vtiles * 16;
    if (nk <= 64 && nv <= 64) launch_attn<T, 64, 64>(a, G, s->cus, st);
    else if (nk <= 128 && nv <= 128) launch_attn<T, 128, 128>(a, G, s->cus, st);
    else if (nk <= 192 && nv <= 128) launch_attn<T, 192, 128>(a, G, s->cus, st);
    else launch_attn<T, 256, 256>(a, G, s->cus, st);
}

template <typename T>
void postnorm(const cfpp_seq* s, const SeqPostNorm& n, int rows, hipStream_t st) {
    const size_t lds = (size_t)s->d.width * 4;
    allow_lds(k_seq_postnorm<T>, lds);
    hipLaunchKernelGGL(k_seq_postnorm<T>, dim3(rows), dim3(kSeqThreads), lds, st, n);
}

template <typename T>
void streams(const cfpp_seq* s, SeqStreams a, int rows, hipStream_t st) {
    const size_t lds = (size_t)s->d.width * 4;
    a.streams = s->d.streams;
    a.width = s->d.width;
    a.pitch = s->xpitch;
    a.eps = s->d.eps;
    a.noff = s->d.norm_offset;
    auto go = [&](auto n) {
        constexpr int S = decltype(n)::value;
        allow_lds(k_seq_streams<T, S>, lds);
        hipLaunchKernelGGL((k_seq_streams<T, S>), dim3(rows), dim3(kSeqThreads), lds, st, a);
    };
    if (a.streams == 1) go(std::integral_constant<int, 1>{});
    else if (a.streams == 2) go(std::integral_constant<int, 2>{});
    else if (a.streams <= 4) go(std::integral_constant<int, 4>{});
    else go(std::integral_constant<int, CFPP_SEQ_MAX_STREAMS>{});
}

// What reads the sum after sublayer `q` (0: mixer, 1: feed-forward) of layer `li`; both null after the last one.
struct NextInput { const float *norm, *in; };
NextInput next_input(const cfpp_seq* s, size_t li, int q) {
    const cfpp_seq_layer& d = s->layers[li].d;
    if (q == 0 && d.ff_kind != CFPP_SEQ_FF_NONE) return {d.norm2, d.hc2.in};
    if (li + 1 < s->layers.size()) return {s->layers[li + 1].d.norm1, s->layers[li + 1].d.hc1.in};
    return {nullptr, nullptr};
}

// The mixer of a portion, from s->xb to s->y.
template <typename T>
void portion_grouped(cfpp_seq* s, const LayerPlan& L, int slot, int n, int pos, hipStream_t st) {
    const cfpp_seq_layer& d = L.d;
    const int cap = s->portion;
    SeqQkv f{s->qkv, s->ld_qkv, d.q_norm, d.k_norm, L.cs, s->d.eps, d.v_lambda, d.heads, d.kv_heads, d.dim, L.Dp, d.vdim, L.Vp,
             d.rot_dims, pos, cap, L.v_role, s->v_first, s->q, s->k, s->v};
    hipLaunchKernelGGL(k_seq_qkv_finish<T>, dim3(n), dim3(kSeqThreads), 0, st, f);

    char* kc = L.kc + (size_t)slot * d.kv_heads * L.rows * L.krow;
    char* vc = L.vc + (size_t)slot * d.kv_heads * L.rows * L.vrow;
    SeqAttn a{};
    a.q = s->q;
    a.k = s->k;
    a.v = s->v;
    a.kc = kc;
    a.vc = vc;
    a.out = s->o;
    a.sink = d.sink;
    a.T = n;
    a.H = d.heads;
    a.R = L.R;
    a.dsteps = L.krow / 64;
    a.qrow = a.krow = L.krow;
    a.vrow = L.vrow;
    a.V = d.vdim;
    a.vtiles = L.Vp / 16;
    a.pos0 = a.k_split = pos;
    a.chunk = d.chunk;
    a.cap = cap;
    a.rows = L.rows;
    a.ldo = (int)pitch_of(d.heads * d.vdim, s->esize);
    a.scale_log2 = d.scale * kLog2e;
    attn<T>(s, a, d.kv_heads, st);

    const int last = pos + n - 1, cs0 = d.chunk > 0 ? last / d.chunk * d.chunk : 0, first = std::max(pos, cs0) - pos;
    SeqAppend ap{s->k, s->v, kc, vc, d.kv_heads, L.krow, L.vrow, cap, L.rows, first, pos + first - cs0};
    hipLaunchKernelGGL(k_seq_append, dim3(n - first), dim3(kSeqThreads), 0, st, ap);
}

template <typename T>
LatentRow latent_row_of(const cfpp_seq* s, const LayerPlan& L) {
    return LatentRow{L.d.kv_norm, L.d.kv_rank, L.d.rot_dims, L.lpitch, L.crow, L.d.rot_half, s->d.eps};
}

template <typename T>
void portion_latent(cfpp_seq* s, const LayerPlan& L, int slot, int n, int pos, hipStream_t st) {
    const cfpp_seq_layer& d = L.d;
    char* kc = L.kc + (size_t)slot * s->d.capacity * L.crow;
    SeqLatentFinish f{s->qkv, s->ld_qkv, L.own, latent_row_of<T>(s, L), L.cs, d.heads, d.dim, d.rot_dims, pos, L.plain, L.qrow, s->q, kc};
    hipLaunchKernelGGL(k_seq_latent_finish<T>, dim3(n), dim3(kSeqThreads), 0, st, f);

    const int ctx = pos + n, cap = s->d.capacity;
    SeqGemm g{};
    g.w = (const char*)d.w_ukv;
    g.a = kc;
    g.n = d.heads * (d.dim + d.vdim);
    g.m = ctx;
    g.kbytes = L.lpitch;
    g.lda = L.crow;
    g.yt = s->k;
    g.yv = s->v;
    g.nk = d.heads * d.dim;
    g.kd = d.dim;
    g.kp = L.plain;
    g.kh = (size_t)cap * L.plain;
    g.vd = d.vdim;
    g.vp = L.vrow;
    g.vh = (size_t)cap * L.vrow;
    gemm<T, kEpiHeads>(s, g, st);

    SeqAttn a{};
    a.q = s->q;
    a.k = s->k;
    a.v = s->v;
    a.kr = kc + L.lpitch;
    a.out = s->o;
    a.sink = d.sink;
    a.gate = d.gated ? s->qkv + L.gate_at : nullptr;
    a.ldg = s->ld_qkv;
    a.T = n;
    a.H = d.heads;
    a.R = 1;
    a.dsteps = L.qrow / 64;
    a.qrow = L.qrow;
    a.krow = L.plain;
    a.runits = L.shared / 16;
    a.rrow = L.crow;
    a.vrow = L.vrow;
    a.V = d.vdim;
    a.vtiles = L.Vp / 16;
    a.pos0 = pos;
    a.cap = cap;
    a.ldo = (int)pitch_of(d.heads * d.vdim, s->esize);
    a.scale_log2 = d.scale * kLog2e;
    attn<T>(s, a, d.heads, st);
}

// One portion: n tokens (device, s->tokens) at positions pos .. pos + n - 1.  want: device places (n_want of them), logits rows.
template <typename T>
int run_portion(cfpp_seq* s, int slot, int n, int pos, int n_want, float* logits, float* residuals, size_t residual_stride, hipStream_t st) {
    const int width = s->d.width, xp = s->xpitch;
    if (s->d.streams > 0) {
        SeqStreams e{};
        e.x = s->x;
        e.in = s->layers[0].d.hc1.in;
        e.w = s->layers[0].d.norm1;
        e.xb = s->xb;
        e.tokens = s->tokens;
        e.embed = (const char*)s->d.embed;
        e.pos = (const char*)s->d.pos;
        e.embed_pitch = xp;
        e.pos0 = pos;
        streams<T>(s, e, n, st);
    } else {
        hipLaunchKernelGGL(k_seq_embed<T>, dim3(n), dim3(kSeqThreads), 0, st, s->tokens, (const char*)s->d.embed, xp, width, s->x, s->xb);
    }
    if (!s->host_routes.empty()) {
        // (one tile size for every layer of the launch: the layers share it when they share top and the expert count)
        for (size_t i = 0; i < s->layers.size(); ++i) {
            const LayerPlan& L = s->layers[i];
            if (L.route < 0) continue;
            size_t j = i + 1, count = 1;
            for (; j < s->layers.size(); ++j) {
                const LayerPlan& M = s->layers[j];
                if (M.route < 0) continue;
                if (expert_tile(M, n) != expert_tile(L, n)) break;
                ++count;
            }
            const size_t lds = (size_t)s->max_experts * 8;
            allow_lds(k_seq_route, lds);
            hipLaunchKernelGGL(k_seq_route, dim3((unsigned)count), dim3(1024), lds, st, s->routes + L.route, s->tokens, n, expert_tile(L, n));
            i = j - 1;
        }
    }
    for (size_t li = 0; li < s->layers.size(); ++li) {
        const LayerPlan& L = s->layers[li];
        const cfpp_seq_layer& d = L.d;
        float* copy = residuals != nullptr ? residuals + li * residual_stride : nullptr;
        SeqGemm g{};
        g.w = (const char*)d.w_qkv;
        g.a = s->xb;
        g.n = L.n_qkv;
        g.m = n;
        g.kbytes = g.lda = xp;
        g.bias = d.b_qkv;
        g.yf = s->qkv;
        g.ldy = s->ld_qkv;
        gemm<T, kEpiF32>(s, g, st);

        if (L.latent) portion_latent<T>(s, L, slot, n, pos, st);
        else portion_grouped<T>(s, L, slot, n, pos, st);

        g = SeqGemm{};
        g.w = (const char*)d.w_o;
        g.a = s->o;
        g.n = width;
        g.m = n;
        g.kbytes = g.lda = (int)pitch_of(d.heads * d.vdim, s->esize);
        g.yf = s->y;
        g.ldy = width;
        gemm<T, kEpiF32>(s, g, st);
        // the residual sum of a sublayer: y (nullable) and the chosen experts' outputs (`top` 0: none)
        auto close = [&](int q, const float* y, int top) {
            float* c = q == 1 || d.ff_kind == CFPP_SEQ_FF_NONE ? copy : nullptr;
            const float* ys = top > 0 ? s->ys : nullptr;
            const float share = top > 0 ? 1.0f / (float)top : 0.0f;
            if (s->d.streams > 0) {
                const cfpp_seq_streams& hc = q == 0 ? d.hc1 : d.hc2;
                const NextInput next = next_input(s, li, q);
                SeqStreams a{};
                a.x = s->x;
                a.y = y;
                a.ys = ys;
                a.top = top;
                a.slot_weight = share;
                a.mix = hc.mix;
                a.out = hc.out;
                a.in = next.in;
                a.w = next.norm;
                a.xb = s->xb;
                a.copy = c;
                streams<T>(s, a, n, st);
            } else {
                SeqPostNorm pn{};
                pn.x = pn.x_out = s->x;
                pn.y = y;
                pn.ys = ys;
                pn.top = top;
                pn.slot_weight = share;
                pn.w = q == 0 ? d.norm1 : d.norm2;
                pn.alpha = s->d.alpha;
                pn.eps = s->d.eps;
                pn.noff = s->d.norm_offset;
                pn.width = width;
                pn.xb = s->xb;
                pn.pitch = xp;
                pn.copy = c;
                postnorm<T>(s, pn, n, st);
            }
        };
        close(0, s->y, 0);
        if (d.ff_kind == CFPP_SEQ_FF_NONE) continue;

        if (d.ff_kind != CFPP_SEQ_FF_TABLE_EXPERTS) {
            const int hp = (int)pitch_of(d.ff, s->esize);
            g = SeqGemm{};
            g.w = (const char*)d.w_up;
            g.a = s->xb;
            g.m = n;
            g.kbytes = g.lda = xp;
            g.yt = s->h;
            g.ldyt = hp;
            if (d.ff_kind == CFPP_SEQ_FF_RELU2) {
                g.n = d.ff;
                gemm<T, kEpiRelu2>(s, g, st);
            } else {
                g.n = 2 * d.ff;
                g.bias = d.b_up;
                gemm<T, kEpiGated>(s, g, st);
            }
            g = SeqGemm{};
            g.w = (const char*)d.w_down;
            g.a = s->h;
            g.n = width;
            g.m = n;
            g.kbytes = g.lda = hp;
            g.bias = d.b_down;
            g.yf = s->y;
            g.ldy = width;
            gemm<T, kEpiF32>(s, g, st);
            close(1, s->y, 0);
        } else {
            const int hp = (int)pitch_of(d.ff, s->esize);
            g = SeqGemm{};
            g.w = (const char*)d.w_up;
            g.w_stride = (size_t)2 * d.ff * xp;
            g.a = s->xb;
            g.n = 2 * d.ff;
            g.kbytes = g.lda = xp;
            g.yt = s->h;
            g.ldyt = hp;
            g.slot_div = d.top;
            expert_gemm<T, kEpiGated>(s, L, g, n, st);
            g = SeqGemm{};
            g.w = (const char*)d.w_down;
            g.w_stride = (size_t)width * hp;
            g.a = s->h;
            g.n = width;
            g.kbytes = g.lda = hp;
            g.yf = s->ys;
            g.ldy = width;
            g.slot_div = 1;
            expert_gemm<T, kEpiF32>(s, L, g, n, st);
            if (d.shared_ff > 0) {
                const int sp = (int)pitch_of(d.shared_ff, s->esize);
                g = SeqGemm{};
                g.w = (const char*)d.w_shared_up;
                g.a = s->xb;
                g.n = 2 * d.shared_ff;
                g.m = n;
                g.kbytes = g.lda = xp;
                g.yt = s->hs;
                g.ldyt = sp;
                gemm<T, kEpiGated>(s, g, st);
                g = SeqGemm{};
                g.w = (const char*)d.w_shared_down;
                g.a = s->hs;
                g.n = width;
                g.m = n;
                g.kbytes = g.lda = sp;
                g.yf = s->y;
                g.ldy = width;
                gemm<T, kEpiF32>(s, g, st);
            }
            close(1, d.shared_ff > 0 ? s->y : nullptr, d.top);
        }
    }
    if (n_want > 0) {
        if (s->d.streams > 0) {
            SeqStreams a{};
            a.x = s->x;
            a.w = s->d.final_norm;
            a.xb = s->wb;
            a.rows = s->want;
            streams<T>(s, a, n_want, st);
        } else {
            SeqPostNorm pn{};
            pn.x = s->x;
            pn.w = s->d.final_norm;
            pn.eps = s->d.eps;
            pn.noff = s->d.norm_offset;
            pn.width = width;
            pn.xb = s->wb;
            pn.pitch = xp;
            pn.rows = s->want;
            postnorm<T>(s, pn, n_want, st);
        }
        SeqGemm g{};
        g.w = (const char*)s->d.head;
        g.a = s->wb;
        g.n = s->d.vocab;
        g.m = n_want;
        g.kbytes = g.lda = xp;
        g.yf = logits;
        g.ldy = s->d.vocab;
        g.mul = s->d.logit_scale;
        g.cap = s->d.softcap;
        gemm<T, kEpiHead>(s, g, st);
    }
    return last_error();
}

// ---- one token ---------------------------------------------------------------------------------
template <typename T, int EPI, bool KCAT>
int gemv(const cfpp_seq* s, SeqGemv p, hipStream_t st) {
    const int nch_e = ceil_div(p.pitch_e, kGemvChunk), nch_s = ceil_div(p.pitch_s, kGemvChunk);
    const int nch = KCAT ? p.top * nch_e + nch_s : nch_s;
    const int total = KCAT ? p.units_s : p.top * p.units_e + p.units_s;
    const int grid = std::max(1, std::min(kGemvWgs * s->cus, ceil_div(total, kSeqWaves)));
    p.park = nch * kGemvChunk + (p.input == kInNorm ? up_to(p.width * 4, 16) : 0);
    p.park_n = ceil_div(total, grid * kSeqWaves);
    const size_t lds = (size_t)p.park + (size_t)p.park_n * (EPI == kEpiGated ? 2 : 1) * kSeqWaves * 4;
    allow_lds(k_seq_gemv<T, EPI, KCAT>, lds);
    hipLaunchKernelGGL((k_seq_gemv<T, EPI, KCAT>), dim3(grid), dim3(kSeqThreads), lds, st, p);
    return grid;
}

template <typename T, int NT>
void launch_attn_decode(const SeqAttnDec& a, hipStream_t st) {
    hipLaunchKernelGGL((k_seq_attn_decode<T, NT>), dim3(a.ns, a.G * a.nct), dim3(kSeqThreads), 0, st, a);
}

// The mixer of one token between its projection (s->qkv) and its output rows (s->o); the number of launches.
template <typename T>
int step_grouped(cfpp_seq* s, const LayerPlan& L, hipStream_t st) {
    const cfpp_seq_layer& d = L.d;
    SeqAttnDec a{s->qkv, d.q_norm, d.k_norm, d.sink, L.cs, s->state, L.kc, L.vc, (size_t)d.kv_heads * L.rows * L.krow,
                 (size_t)d.kv_heads * L.rows * L.vrow, s->v_first, s->o, s->part, s->cnt, s->d.eps, d.v_lambda, d.scale * kLog2e, L.v_role,
                 d.heads, d.kv_heads, L.R, L.nct, d.dim, d.vdim, d.rot_dims, d.chunk, L.krow, L.vrow, L.krow / 64, L.Vp / 16, L.rows, L.ns};
    if (L.NT == 64) launch_attn_decode<T, 64>(a, st);
    else if (L.NT == 128) launch_attn_decode<T, 128>(a, st);
    else launch_attn_decode<T, 256>(a, st);
    return 1;
}

// sets of 16 heads of a workgroup of k_seq_latent_attn
int latent_sets(int heads) { return heads <= 32 ? 1 : 2; }

template <typename T, int NR>
void launch_latent_attn(const SeqLatentAttn& a, hipStream_t st) {
    const int sets = latent_sets(a.H);
    const size_t lds = (size_t)LatentLds<T, NR>::buffers * LatentLds<T, NR>::tile;
    const dim3 grid(a.ns, ceil_div(a.H, 16 * sets));
    auto go = [&](auto n) {
        constexpr int RW = decltype(n)::value;
        allow_lds(k_seq_latent_attn<T, NR, RW>, lds);
        hipLaunchKernelGGL((k_seq_latent_attn<T, NR, RW>), grid, dim3(kSeqThreads), lds, st, a);
    };
    if (sets == 1) go(std::integral_constant<int, 4>{});
    else go(std::integral_constant<int, 2>{});
}

template <typename T>
int step_latent(cfpp_seq* s, const LayerPlan& L, hipStream_t st) {
    const cfpp_seq_layer& d = L.d;
    const size_t slot = (size_t)s->d.capacity * L.crow;
    SeqLatentQ q{s->qkv, s->state, L.cs, (const char*)d.w_ukv, L.lpitch, d.heads, d.dim, d.rot_dims, L.lpitch / 128, L.own, latent_row_of<T>(s, L),
                 s->q, L.kc, slot};
    hipLaunchKernelGGL(k_seq_latent_q<T>, dim3(d.heads * q.nrb + (L.own ? 1 : 0)), dim3(kSeqThreads), 0, st, q);

    float* ml = s->part + (size_t)L.ns * d.heads * L.rp;
    SeqLatentAttn a{s->q, L.kc, slot, s->state, s->part, ml, d.scale * kLog2e, d.heads, L.crow, L.ns, L.least, L.rp};
    if (L.rp <= 128) launch_latent_attn<T, 128>(a, st);
    else launch_latent_attn<T, 512>(a, st);

    SeqLatentOut o{s->part, ml, s->state, d.sink, d.gated ? s->qkv + L.gate_at : nullptr, (const char*)d.w_ukv + (size_t)d.heads * d.dim * L.lpitch, s->o,
                   d.heads, d.vdim, L.lpitch, L.ns, L.least, L.rp};
    hipLaunchKernelGGL(k_seq_latent_out<T>, dim3(d.heads, ceil_div(d.vdim, kLatentOut)), dim3(kSeqThreads), 0, st, o);
    return 3;
}

// Enqueues one step for the device-side state.  pick: also choose the next token.
template <typename T>
int run_step(cfpp_seq* s, bool head, bool pick, float* residuals, hipStream_t st) {
    const int width = s->d.width, xp = s->xpitch;
    const bool multi = s->d.streams > 0;
    int cur = 0, launches = 0;             // dx[cur]: the residual row before the sum that is still pending
    const float* pending = nullptr;        // norm weight of that sum
    float* pending_copy = nullptr;
    // The input of a sublayer: the streams' weighted sum and its norm, or the pending residual sum and its norm.
    auto input = [&](SeqGemv& p, const float* norm) {
        p.state = s->state;
        p.width = width;
        p.eps = s->d.eps;
        p.noff = s->d.norm_offset;
        if (multi) {
            p.input = kInNorm;
            p.x = s->du;
            p.alpha = 1.0f;
            p.nw = norm;
            return;
        }
        p.alpha = s->d.alpha;
        if (pending == nullptr) {
            p.input = kInEmbed;
            p.embed = (const char*)s->d.embed;
            p.embed_pitch = xp;
            p.x_out = s->dx[cur];
        } else {
            p.input = kInNorm;
            p.x = s->dx[cur];
            p.y = s->dy;
            p.x_out = s->dx[cur ^ 1];
            p.copy = pending_copy;
            p.nw = pending;
            cur ^= 1;
        }
        pending_copy = nullptr;
    };
    // The rows that end sublayer `q`: into the streams, or to dy for the sum that the next launch makes.
    auto output = [&](SeqGemv& p, size_t li, int q, float* copy) {
        const cfpp_seq_layer& d = s->layers[li].d;
        p.units_s = width;
        if (multi) {
            const cfpp_seq_streams& hc = q == 0 ? d.hc1 : d.hc2;
            p.width = width;
            p.xs = s->dx[0];
            p.mix = hc.mix;
            p.out = hc.out;
            p.in = next_input(s, li, q).in;
            p.streams = s->d.streams;
            p.u = s->du;
            p.sum = copy;
            gemv<T, kEpiStreams, true>(s, p, st);
        } else {
            p.yf = s->dy;
            gemv<T, kEpiF32, true>(s, p, st);
            pending = q == 0 ? d.norm1 : d.norm2;
            pending_copy = copy;
        }
    };
    if (multi) {
        SeqStreams e{};
        e.x = s->dx[0];
        e.in = s->layers[0].d.hc1.in;
        e.w = s->layers[0].d.norm1;
        e.xb = s->xb;
        e.tokens = s->state + kStToken;
        e.state = s->state;
        e.embed = (const char*)s->d.embed;
        e.pos = (const char*)s->d.pos;
        e.embed_pitch = xp;
        streams<T>(s, e, 1, st);
        ++launches;
    }
    for (size_t li = 0; li < s->layers.size(); ++li) {
        const LayerPlan& L = s->layers[li];
        const cfpp_seq_layer& d = L.d;
        float* copy = residuals != nullptr ? residuals + li * width : nullptr;
        SeqGemv p{};
        p.w_s = (const char*)d.w_qkv;
        p.pitch_s = xp;
        p.units_s = L.n_qkv;
        p.bias = d.b_qkv;
        p.yf = s->qkv;
        if (multi && li == 0) {
            p.input = kInVector;
            p.xin = s->xb;
            gemv<T, kEpiF32, true>(s, p, st);
        } else {
            input(p, d.norm1);
            gemv<T, kEpiF32, false>(s, p, st);
        }
        launches += L.latent ? step_latent<T>(s, L, st) : step_grouped<T>(s, L, st);

        p = SeqGemv{};
        p.input = kInVector;
        p.xin = s->o;
        p.w_s = (const char*)d.w_o;
        p.pitch_s = (int)pitch_of(d.heads * d.vdim, s->esize);
        output(p, li, 0, d.ff_kind == CFPP_SEQ_FF_NONE ? copy : nullptr);
        launches += 2;
        if (d.ff_kind == CFPP_SEQ_FF_NONE) continue;
        const bool moe = d.ff_kind == CFPP_SEQ_FF_TABLE_EXPERTS;
        const int hp = (int)pitch_of(d.ff, s->esize), sp = moe ? (int)pitch_of(d.shared_ff, s->esize) : hp;
        p = SeqGemv{};
        input(p, d.norm2);
        p.yt = s->h;
        p.seg_y = hp;
        p.pitch_s = xp;
        if (moe) {
            p.table = d.table;
            p.top = d.top;
            p.w_e = (const char*)d.w_up;
            p.pitch_e = xp;
            p.e_stride = (size_t)2 * d.ff * xp;
            p.units_e = d.ff;
            p.w_s = (const char*)d.w_shared_up;
            p.units_s = d.shared_ff;
            gemv<T, kEpiGated, false>(s, p, st);
        } else {
            p.w_s = (const char*)d.w_up;
            p.units_s = d.ff;
            p.bias = d.b_up;
            if (d.ff_kind == CFPP_SEQ_FF_GATED) gemv<T, kEpiGated, false>(s, p, st);
            else gemv<T, kEpiRelu2, false>(s, p, st);
        }
        p = SeqGemv{};
        p.input = kInVector;
        p.state = s->state;
        p.xin = s->h;
        p.seg_e = hp;
        if (moe) {
            p.table = d.table;
            p.top = d.top;
            p.w_e = (const char*)d.w_down;
            p.pitch_e = hp;
            p.e_stride = (size_t)width * hp;
            p.w_s = (const char*)d.w_shared_down;
            p.pitch_s = d.shared_ff > 0 ? sp : 0;
        } else {
            p.w_s = (const char*)d.w_down;
            p.pitch_s = hp;
            p.bias = d.b_down;
        }
        output(p, li, 1, copy);
        launches += 2;
    }
    if (head || (residuals != nullptr && !multi)) {
        SeqGemv p{};
        input(p, s->d.final_norm);
        if (!multi) p.nw2 = s->d.final_norm;
        p.w_s = (const char*)s->d.head;
        p.pitch_s = xp;
        p.units_s = s->d.vocab;
        p.yf = s->logits;
        p.mul = s->d.logit_scale;
        p.cap = s->d.softcap;
        p.best_v = s->best_v;
        p.best_i = s->best_i;
        s->head_grid = gemv<T, kEpiHead, false>(s, p, st);
        ++launches;
        if (pick) {
            hipLaunchKernelGGL(k_seq_pick, dim3(1), dim3(kSeqThreads), 0, st, s->best_v, s->best_i, s->head_grid, s->state, s->history, s->history_cap);
            ++launches;
        }
    }
    if (pick) s->launches = launches;
    return last_error();
}

int step(cfpp_seq* s, bool head, bool pick, float* residuals, hipStream_t st) {
    return s->d.dtype == CFPP_SEQ_BF16 ? run_step<bf16_t>(s, head, pick, residuals, st) : run_step<float>(s, head, pick, residuals, st);
}

bool connected(const cfpp_seq_streams& c) { return c.in != nullptr && c.mix != nullptr && c.out != nullptr; }

int check_mixer(const cfpp_seq_desc& D, int li, int esize) {
    const cfpp_seq_layer& d = D.layers[li];
    if (d.heads < 1 || d.dim < 1 || d.vdim < 1 || d.dim > 256 || d.vdim > 256 || d.rot_dims < 0 || d.rot_dims % 2) return CFPP_ERR_DIMS;
    if (d.rot_factor != 0.0 && !(d.rot_factor > 0.0 && d.rot_original > 0.0 && d.rot_fast > 0.0 && d.rot_slow > 0.0 && d.rot_base > 1.0)) return CFPP_ERR_DIMS;
    if (d.rot_dims > 0 && !(d.rot_base > 0.0)) return CFPP_ERR_DIMS;
    if (d.w_qkv == nullptr || d.w_o == nullptr || d.norm1 == nullptr) return CFPP_ERR_NULL;
    if (D.streams > 0 && !connected(d.hc1)) return CFPP_ERR_NULL;
    if (d.mixer == CFPP_SEQ_MIX_GROUPED) {
        if (d.kv_heads < 1 || d.heads % d.kv_heads || d.chunk < 0 || d.rot_dims > d.dim) return CFPP_ERR_DIMS;
        if (d.rot_half || d.gated) return CFPP_ERR_MODE;
        if (d.b_qkv == nullptr || d.q_norm == nullptr || d.k_norm == nullptr || d.sink == nullptr) return CFPP_ERR_NULL;
        return CFPP_OK;
    }
    if (d.mixer != CFPP_SEQ_MIX_LATENT || d.v_mix || d.chunk != 0) return CFPP_ERR_MODE;
    if (d.heads > 4096 || d.kv_rank < 1 || d.kv_rank > 512 || d.rot_dims > 128 || up_to(d.dim * esize, 16) + up_to(d.rot_dims * esize, 16) > 256 * esize) return CFPP_ERR_DIMS;
    if (d.w_ukv == nullptr) return CFPP_ERR_NULL;
    if (d.kv_from < 0) return d.kv_norm != nullptr ? CFPP_OK : CFPP_ERR_NULL;
    if (d.kv_from >= li) return CFPP_ERR_DIMS;
    const cfpp_seq_layer& o = D.layers[d.kv_from];
    return o.mixer == CFPP_SEQ_MIX_LATENT && o.kv_from < 0 && o.kv_rank == d.kv_rank && o.rot_dims == d.rot_dims ? CFPP_OK : CFPP_ERR_DIMS;
}

int check_layer(const cfpp_seq_desc& D, int li, int esize) {
    const cfpp_seq_layer& d = D.layers[li];
    const int rc = check_mixer(D, li, esize);
    if (rc) return rc;
    if (d.ff_kind < CFPP_SEQ_FF_NONE || d.ff_kind > CFPP_SEQ_FF_GATED) return CFPP_ERR_MODE;
    size_t lds = std::max(pitch_of(D.width, esize) + 1024 + (size_t)D.width * 4, pitch_of(d.heads * d.vdim, esize) + 1024);
    if (d.ff_kind != CFPP_SEQ_FF_NONE) {
        if (d.ff < 1 || d.w_up == nullptr || d.w_down == nullptr || d.norm2 == nullptr) return CFPP_ERR_NULL;
        if (D.streams > 0 && !connected(d.hc2)) return CFPP_ERR_NULL;
        const size_t one = pitch_of(d.ff, esize) + 1024;
        if (d.ff_kind == CFPP_SEQ_FF_TABLE_EXPERTS) {
            if (d.experts < 1 || d.experts > 8192 || d.top < 1 || d.top > kWave || d.top > d.experts || d.shared_ff < 0) return CFPP_ERR_DIMS;
            if (d.table == nullptr || (d.shared_ff > 0 && (d.w_shared_up == nullptr || d.w_shared_down == nullptr))) return CFPP_ERR_NULL;
            lds = std::max(lds, d.top * one + (d.shared_ff > 0 ? pitch_of(d.shared_ff, esize) + 1024 : 0));
        } else {
            lds = std::max(lds, one);
        }
    }
    // the input of a matrix-vector product sits in LDS
    return lds > 150 * 1024 ? CFPP_ERR_DIMS : CFPP_OK;
}

// Angles per position of the layer's rotary pairs; the factor on cos and sin.  With scaling, pairs that make more than
// rot_fast turns over rot_original positions keep their angle, those with fewer than rot_slow have it divided by rot_factor,
// and the ones between are blended linearly in the pair index.
double angles(const cfpp_seq_layer& d, double* freq) {
    const int half = d.rot_dims / 2;
    const double base = d.rot_base;
    for (int j = 0; j < half; ++j) freq[j] = pow(base, -2.0 * j / d.rot_dims);
    if (!(d.rot_factor > 0.0)) return 1.0;
    const double two_pi = 6.283185307179586476925, factor = d.rot_factor;
    auto index_of = [&](double turns) { return d.rot_dims * log(d.rot_original / (two_pi * turns)) / (2.0 * log(base)); };
    const double lo = std::max(floor(index_of(d.rot_fast)), 0.0), hi = std::min(ceil(index_of(d.rot_slow)), (double)(d.rot_dims - 1));
    for (int j = 0; j < half; ++j) {
        const double r = std::min(std::max((j - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
        freq[j] = freq[j] / factor * r + freq[j] * (1.0 - r);
    }
    return 0.1 * log(factor) + 1.0;
}

}  // namespace

extern "C" {

size_t cfpp_seq_row_pitch(int32_t K, int32_t dtype) { return pitch_of(K, dtype == CFPP_SEQ_F32 ? 4 : 2); }
const char* cfpp_seq_version(void) { return "cfpp_seq 0.1 (gfx950)"; }

int cfpp_seq_create(const cfpp_seq_desc* desc, cfpp_seq** out) {
    if (desc == nullptr || out == nullptr) return CFPP_ERR_NULL;
    *out = nullptr;
    const cfpp_seq_desc& D = *desc;
    if (D.layers == nullptr || D.embed == nullptr || D.final_norm == nullptr || D.head == nullptr) return CFPP_ERR_NULL;
    if (D.dtype != CFPP_SEQ_BF16 && D.dtype != CFPP_SEQ_F32) return CFPP_ERR_MODE;
    if (D.n_layers < 1 || D.width < 1 || D.width > 16384 || D.vocab < 1 || D.vocab > 524288 || D.slots < 1 || D.capacity < 1 || D.max_portion < 1)
        return CFPP_ERR_DIMS;
    if (D.streams < 0 || D.streams > CFPP_SEQ_MAX_STREAMS || (D.pos != nullptr && (D.streams == 0 || D.positions < D.capacity))) return CFPP_ERR_DIMS;
    const int esize = D.dtype == CFPP_SEQ_BF16 ? 2 : 4;
    int first_mix = -1;
    for (int i = 0; i < D.n_layers; ++i) {
        const int rc = check_layer(D, i, esize);
        if (rc) return rc;
        if (D.layers[i].v_mix) {
            if (first_mix < 0) first_mix = i;
            // the mixed values are those of the first such layer, element by element
            else if (D.layers[i].kv_heads * D.layers[i].vdim != D.layers[first_mix].kv_heads * D.layers[first_mix].vdim) return CFPP_ERR_DIMS;
        }
    }
    cfpp_seq* s = new (std::nothrow) cfpp_seq();
    if (s == nullptr) return CFPP_ERR_NULL;
    s->d = D;
    s->esize = esize;
    s->xpitch = (int)pitch_of(D.width, esize);
    s->portion = std::min(D.max_portion, D.capacity);
    (void)hipGetDevice(&s->device);
    if (hipDeviceGetAttribute(&s->cus, hipDeviceAttributeMultiprocessorCount, s->device) != hipSuccess || s->cus < 1) s->cus = 256;
    const size_t P = (size_t)s->portion, C = (size_t)D.capacity;
    size_t n_qkv = 0, o_bytes = 0, h_bytes = 0, hs_bytes = 0, q_bytes = 0, k_bytes = 0, v_bytes = 0, vf = 0, ys = 0, part = 0, items = 0, dec_h = 0;
    std::map<std::tuple<double, int, double, double, double, double>, float2*> tables;
    for (int i = 0; i < D.n_layers; ++i) {
        LayerPlan L{};
        L.d = D.layers[i];
        const cfpp_seq_layer& d = L.d;
        L.latent = d.mixer == CFPP_SEQ_MIX_LATENT;
        if (L.latent) {
            L.own = d.kv_from < 0;
            L.Vp = up_to(d.vdim, 16);
            L.vrow = L.Vp * esize;
            L.rp = up_to(d.kv_rank, 16);
            L.lpitch = (int)pitch_of(d.kv_rank, esize);
            L.plain = up_to(d.dim * esize, 16);
            L.shared = up_to(d.rot_dims * esize, 16);
            L.crow = up_to(L.lpitch + L.shared, 64);
            L.qrow = up_to(L.plain + L.shared, 64);
            L.n_qkv = d.heads * (d.dim + d.rot_dims);
            if (L.own) L.n_qkv += d.kv_rank + d.rot_dims;
            L.gate_at = L.n_qkv;
            if (d.gated) L.n_qkv += d.heads * d.vdim;
            const int groups = ceil_div(d.heads, 16 * latent_sets(d.heads)), keys = esize == 2 ? LatentTile<bf16_t>::keys : LatentTile<float>::keys;
            L.least = 2;
            L.ns = std::max(1, std::min({kLatentSplits, ceil_div(s->cus, groups), ceil_div(D.capacity, keys * L.least)}));
            L.kc = L.own ? s->alloc<char>((size_t)D.slots * C * L.crow) : s->layers[d.kv_from].kc;
            q_bytes = std::max({q_bytes, P * d.heads * L.qrow, (size_t)d.heads * L.crow});
            k_bytes = std::max(k_bytes, C * d.heads * L.plain);
            v_bytes = std::max(v_bytes, C * d.heads * L.vrow);
            part = std::max(part, (size_t)L.ns * d.heads * (L.rp + 2));
        } else {
            L.R = d.heads / d.kv_heads;
            L.nct = ceil_div(L.R, kAttnCols);
            L.Dp = up_to(d.dim, 64 / esize);
            L.Vp = up_to(d.vdim, 16);
            L.krow = L.Dp * esize;
            L.vrow = L.Vp * esize;
            L.NT = std::max(L.Dp, L.Vp) <= 64 ? 64 : std::max(L.Dp, L.Vp) <= 128 ? 128 : 256;
            L.rows = d.chunk > 0 ? std::min(d.chunk, D.capacity) : D.capacity;
            L.n_qkv = d.heads * d.dim + d.kv_heads * (d.dim + d.vdim);
            L.v_role = !d.v_mix ? 0 : i == first_mix ? 1 : 2;
            const int kt = esize == 2 ? 32 : (L.NT <= 128 ? 32 : 16);
            L.ns = std::max(1, std::min({kMaxSeqSplit, ceil_div(kAttnWgs * s->cus, d.kv_heads * L.nct), ceil_div(L.rows, kt * kSeqWaves)}));
            L.kc = s->alloc<char>((size_t)D.slots * d.kv_heads * L.rows * L.krow);
            L.vc = s->alloc<char>((size_t)D.slots * d.kv_heads * L.rows * L.vrow);
            q_bytes = std::max(q_bytes, P * d.heads * L.krow);
            k_bytes = std::max(k_bytes, P * d.kv_heads * L.krow);
            v_bytes = std::max(v_bytes, P * d.kv_heads * L.vrow);
            if (d.v_mix) vf = std::max(vf, (size_t)d.kv_heads * d.vdim);
            items = std::max(items, (size_t)d.kv_heads * L.nct);
            part = std::max(part, (size_t)d.kv_heads * L.nct * L.ns * kAttnCols * (L.Vp + 2));
        }
        L.cs = nullptr;
        if (d.rot_dims > 0) {
            const double f = d.rot_factor;
            float2*& t = tables[{d.rot_base, d.rot_dims, f, f > 0 ? d.rot_original : 0.0, f > 0 ? d.rot_fast : 0.0, f > 0 ? d.rot_slow : 0.0}];
            if (t == nullptr) {
                const int half = d.rot_dims / 2;
                t = s->alloc<float2>((size_t)D.capacity * half);
                std::vector<double> freq(half);
                const double mul = angles(d, freq.data());
                double* df = s->alloc<double>(half);
                if (!s->failed) {
                    (void)hipDeviceSynchronize();        // the zero fill of the table comes before its copy
                    if (hipMemcpy(df, freq.data(), half * sizeof(double), hipMemcpyHostToDevice) != hipSuccess) s->failed = true;
                    hipLaunchKernelGGL(k_seq_rope_table, dim3(1024), dim3(256), 0, nullptr, t, df, mul, half, D.capacity);
                }
            }
            L.cs = t;
        }
        n_qkv = std::max(n_qkv, (size_t)L.n_qkv);
        o_bytes = std::max(o_bytes, pitch_of(d.heads * d.vdim, esize));
        L.route = -1;
        if (d.ff_kind == CFPP_SEQ_FF_RELU2 || d.ff_kind == CFPP_SEQ_FF_GATED) {
            h_bytes = std::max(h_bytes, pitch_of(d.ff, esize));
        } else if (d.ff_kind == CFPP_SEQ_FF_TABLE_EXPERTS) {
            h_bytes = std::max(h_bytes, d.top * pitch_of(d.ff, esize));
            hs_bytes = std::max(hs_bytes, pitch_of(d.shared_ff, esize));
            ys = std::max(ys, (size_t)d.top * D.width);
            dec_h = std::max(dec_h, d.top * pitch_of(d.ff, esize) + pitch_of(d.shared_ff, esize));
            SeqRoute r{d.table, s->alloc<int>(d.experts + 1), s->alloc<int>(d.experts + 1), s->alloc<int>(P * d.top), d.experts, d.top};
            L.route = (int)s->host_routes.size();
            s->host_routes.push_back(r);
            s->max_experts = std::max(s->max_experts, d.experts);
        }
        s->layers.push_back(L);
    }
    s->ld_qkv = up_to((int)n_qkv, 4);
    s->tokens = s->alloc<int>(2 * P);
    s->want = s->tokens != nullptr ? s->tokens + P : nullptr;
    const size_t rows_of_x = std::max(1, D.streams);
    s->x = s->alloc<float>(P * rows_of_x * D.width);
    s->y = s->alloc<float>(P * D.width);
    s->ys = s->alloc<float>(P * ys);
    s->qkv = s->alloc<float>(P * s->ld_qkv);
    s->v_first = s->alloc<float>(P * vf);
    s->xb = s->alloc<char>(P * s->xpitch);
    s->wb = s->alloc<char>(P * s->xpitch);
    s->q = s->alloc<char>(q_bytes);
    s->k = s->alloc<char>(k_bytes);
    s->v = s->alloc<char>(v_bytes);
    s->o = s->alloc<char>(P * o_bytes);
    s->h = s->alloc<char>(std::max(P * h_bytes, dec_h));
    s->hs = s->alloc<char>(P * hs_bytes);
    s->routes = s->alloc<SeqRoute>(s->host_routes.size());
    s->state = s->alloc<int>(4);
    s->history_cap = D.capacity;
    s->history = s->alloc<int>(s->history_cap);
    s->cnt = s->alloc<int>(items * kHeadCntStride);
    s->part = s->alloc<float>(part);
    s->dx[0] = s->alloc<float>(rows_of_x * D.width);
    s->du = s->alloc<float>(D.width);
    s->dx[1] = s->alloc<float>(D.width);
    s->dy = s->alloc<float>(D.width);
    s->dres = s->alloc<float>((size_t)D.n_layers * D.width);
    s->logits = s->alloc<float>(D.vocab);
    s->best_v = s->alloc<float>(kGemvWgs * s->cus);
    s->best_i = s->alloc<int>(kGemvWgs * s->cus);
    if (!s->failed && hipDeviceSynchronize() != hipSuccess) s->failed = true;
    if (!s->failed && !s->host_routes.empty() &&
        hipMemcpy(s->routes, s->host_routes.data(), s->host_routes.size() * sizeof(SeqRoute), hipMemcpyHostToDevice) != hipSuccess)
        s->failed = true;
    if (s->failed) {
        const int e = (int)hipGetLastError();
        cfpp_seq_destroy(s);
        return e > 0 ? e : (int)hipErrorOutOfMemory;
    }
    *out = s;
    return CFPP_OK;
}

int cfpp_seq_destroy(cfpp_seq* s) {
    if (s == nullptr) return CFPP_OK;
    (void)hipDeviceSynchronize();
    if (s->graph != nullptr) (void)hipGraphExecDestroy(s->graph);
    if (s->capture != nullptr) (void)hipStreamDestroy(s->capture);
    for (void* p : s->owned) (void)hipFree(p);
    delete s;
    return CFPP_OK;
}

size_t cfpp_seq_bytes(const cfpp_seq* s) { return s != nullptr ? s->bytes : 0; }

int cfpp_seq_forward(cfpp_seq* s, int32_t slot, const int32_t* tokens, int32_t n, int32_t pos, const int32_t* want, int32_t n_want,
                     float* logits, float* residuals, void* stream) {
    if (s == nullptr || tokens == nullptr || n_want < 0 || (n_want > 0 && (want == nullptr || logits == nullptr))) return CFPP_ERR_NULL;
    if (slot < 0 || slot >= s->d.slots) return CFPP_ERR_CONTEXT;
    if (n < 1 || pos < 0 || n > s->d.capacity - pos) return CFPP_ERR_SEQ;
    for (int i = 0; i < n; ++i)
        if (tokens[i] < 0 || tokens[i] >= s->d.vocab) return CFPP_ERR_DIMS;
    for (int i = 0; i < n_want; ++i)
        if (want[i] < 0 || want[i] >= n || (i > 0 && want[i] <= want[i - 1])) return CFPP_ERR_DIMS;
    hipStream_t st = (hipStream_t)stream;
    const int width = s->d.width, V = s->d.vocab;
    int w = 0;
    for (int off = 0; off < n;) {
        const int T = std::min(n - off, s->portion);
        int w1 = w;
        while (w1 < n_want && want[w1] < off + T) ++w1;
        const int nw = w1 - w;
        int rc;
        if (T == 1) {
            hipLaunchKernelGGL(k_seq_set_state, dim3(1), dim3(64), 0, st, s->state, slot, tokens[off], pos + off, -1);
            // (a single token's residual rows are written one layer after the other; with other tokens they lie n rows apart)
            float* res = residuals == nullptr || n == 1 ? residuals : s->dres;
            rc = step(s, nw > 0, false, res, st);
            if (res != residuals)
                for (int l = 0; l < s->d.n_layers; ++l)
                    (void)hipMemcpyAsync(residuals + ((size_t)l * n + off) * width, res + (size_t)l * width, (size_t)width * 4, hipMemcpyDeviceToDevice, st);
            if (rc == CFPP_OK && nw > 0) {
                const hipError_t e = hipMemcpyAsync(logits + (size_t)w * V, s->logits, (size_t)V * 4, hipMemcpyDeviceToDevice, st);
                if (e != hipSuccess) rc = (int)e;
            }
        } else {
            std::vector<int> places(nw);
            for (int i = 0; i < nw; ++i) places[i] = want[w + i] - off;
            hipError_t e = hipMemcpyAsync(s->tokens, tokens + off, (size_t)T * 4, hipMemcpyHostToDevice, st);
            if (e == hipSuccess && nw > 0) e = hipMemcpyAsync(s->want, places.data(), (size_t)nw * 4, hipMemcpyHostToDevice, st);
            if (e == hipSuccess) e = hipStreamSynchronize(st);           // the host arrays are the caller's and this frame's
            if (e != hipSuccess) return (int)e;
            float* res = residuals != nullptr ? residuals + (size_t)off * width : nullptr;
            float* lg = nw > 0 ? logits + (size_t)w * V : nullptr;
            const size_t rs = (size_t)n * width;
            rc = s->d.dtype == CFPP_SEQ_BF16 ? run_portion<bf16_t>(s, slot, T, pos + off, nw, lg, res, rs, st)
                                             : run_portion<float>(s, slot, T, pos + off, nw, lg, res, rs, st);
        }
        if (rc != CFPP_OK) return rc;
        off += T;
        w = w1;
    }
    return CFPP_OK;
}

int cfpp_seq_set_state(cfpp_seq* s, int32_t slot, int32_t token, int32_t pos, void* stream) {
    if (s == nullptr) return CFPP_ERR_NULL;
    if (slot < 0 || slot >= s->d.slots) return CFPP_ERR_CONTEXT;
    if (token < 0 || token >= s->d.vocab) return CFPP_ERR_DIMS;
    if (pos < 0 || pos >= s->d.capacity) return CFPP_ERR_SEQ;
    hipLaunchKernelGGL(k_seq_set_state, dim3(1), dim3(64), 0, (hipStream_t)stream, s->state, slot, token, pos, 0);
    s->pos = pos;
    return last_error();
}

int cfpp_seq_steps(cfpp_seq* s, int32_t n, void* stream) {
    if (s == nullptr) return CFPP_ERR_NULL;
    if (n < 0 || n > s->d.capacity - s->pos) return CFPP_ERR_SEQ;
    for (int i = 0; i < n; ++i) {
        const int rc = step(s, true, true, nullptr, (hipStream_t)stream);
        if (rc != CFPP_OK) return rc;
        ++s->pos;
    }
    return CFPP_OK;
}

int cfpp_seq_graph_steps(cfpp_seq* s, int32_t n, void* stream) {
    if (s == nullptr) return CFPP_ERR_NULL;
    if (n < 0 || n > s->d.capacity - s->pos) return CFPP_ERR_SEQ;
    if (s->graph == nullptr) {
        hipGraph_t g = nullptr;
        hipError_t e = s->capture != nullptr ? hipSuccess : hipStreamCreateWithFlags(&s->capture, hipStreamNonBlocking);
        if (e == hipSuccess) e = hipStreamBeginCapture(s->capture, hipStreamCaptureModeThreadLocal);
        if (e != hipSuccess) return (int)e;
        const int rc = step(s, true, true, nullptr, s->capture);
        e = hipStreamEndCapture(s->capture, &g);
        if (rc != CFPP_OK || e != hipSuccess) {
            if (g != nullptr) (void)hipGraphDestroy(g);
            return rc != CFPP_OK ? rc : (int)e;
        }
        e = hipGraphInstantiate(&s->graph, g, nullptr, nullptr, 0);
        (void)hipGraphDestroy(g);
        if (e != hipSuccess) {
            s->graph = nullptr;
            return (int)e;
        }
    }
    for (int i = 0; i < n; ++i) {
        const hipError_t e = hipGraphLaunch(s->graph, (hipStream_t)stream);
        if (e != hipSuccess) return (int)e;
        ++s->pos;
    }
    return CFPP_OK;
}

int cfpp_seq_launches_per_step(const cfpp_seq* s) { return s != nullptr ? s->launches : 0; }

int cfpp_seq_buffers(cfpp_seq* s, float** logits, int32_t** state, int32_t** history, int32_t* history_capacity) {
    if (s == nullptr) return CFPP_ERR_NULL;
    if (logits) *logits = s->logits;
    if (state) *state = s->state;
    if (history) *history = s->history;
    if (history_capacity) *history_capacity = s->history_cap;
    return CFPP_OK;
}

}  // extern "C"
