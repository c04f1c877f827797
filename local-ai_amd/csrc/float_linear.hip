// Products of activations with bf16 weights [N, K]:
//   linear_mfma_kernel   bf16 activations, K a multiple of 8: LDS-tiled bf16 MFMA 16x16x32, tiles loaded straight into LDS
//   linear_plain_kernel  everything else: f32 FMA on 64 x 64 tiles (the 32-bit runs, ragged K)
//   matvec_bf16_kernel   one row, HBM-bound weight streaming, with the norm before the product done while x is staged
// All three end in the same column segments (bias, activation, layout, residual add), and the first two also run the
// experts of a mixture on the tiles of a routing plan.
#include "float_linear.hpp"
#include <algorithm>
#include <cstring>

namespace {

typedef __attribute__((address_space(1))) const void gvoid;
typedef __attribute__((address_space(3))) void lvoid;

// 16 bytes per lane from global memory into LDS: lane i of the wave lands at lds + 16 i (`lds` wave-uniform).
__device__ __forceinline__ void load_lds16(const void* g, void* lds) {
    __builtin_amdgcn_global_load_lds((gvoid*)g, (lvoid*)lds, 16, 0, 0);
}

__device__ uint4 g_zero16 = {0u, 0u, 0u, 0u};   // what activation chunks past K read

// The rows this workgroup multiplies: tile `mt` of an ordinary product or of an expert plan.
struct RowTile { uint32_t begin, end, expert; };
__device__ __forceinline__ RowTile row_tile(const LhLinear& a, uint32_t mt, uint32_t bm) {
    if (a.ex.tiles == nullptr) return RowTile{mt * bm, min(mt * bm + bm, a.M), 0u};
    const uint32_t* t = a.ex.tiles + 3 * mt;
    RowTile r{t[1], min(t[2], a.ex.slots), t[0]};
    if (r.expert >= a.ex.experts || r.begin >= r.end) r.begin = r.end = r.expert = 0;
    return r;
}
__device__ __forceinline__ uint32_t a_row(const LhLinear& a, uint32_t slot) {
    if (!a.ex.gather) return slot;
    const uint32_t r = a.ex.slot_row[slot];
    return r < a.ex.rows ? r : 0u;
}
struct OutRow { uint32_t row; float weight; };
__device__ __forceinline__ OutRow out_row(const LhLinear& a, uint32_t slot) {
    OutRow o{slot, 1.0f};
    if (a.ex.tiles != nullptr) {
        if (a.ex.scatter) o.row = a.ex.slot_row[slot];
        if (a.ex.slot_weight) o.weight = a.ex.slot_weight[slot];
    }
    return o;
}

// Column and row tile of a workgroup: workgroups are dealt to the eight XCDs round robin, so each XCD gets a contiguous
// range of tiles (its L2 then sees the same weight panels again), walked in groups of four row tiles.
__device__ __forceinline__ void tile_of_block(uint32_t mt_n, uint32_t nt_n, uint32_t& mt, uint32_t& nt) {
    const uint32_t total = mt_n * nt_n, id = blockIdx.x;
    const uint32_t q = total >> 3, rem = total & 7, x = id & 7, i = id >> 3;
    const uint32_t t = (x < rem ? x * (q + 1) : rem * (q + 1) + (x - rem) * q) + i;
    const uint32_t gsz = 4 * nt_n, g = t / gsz, m_in = min(4u, mt_n - g * 4), r = t - g * gsz;
    mt = g * 4 + r % m_in;
    nt = r / m_in;
}

// Bias, activation and destination of columns n .. n + 3 (those below N) of one row of a product.
__device__ __forceinline__ void store4(const LhLinear& a, uint32_t slot, uint32_t n, const float4 acc, uint32_t pos0) {
    const OutRow o = out_row(a, slot);
    float v[4] = {acc.x, acc.y, acc.z, acc.w};
#pragma unroll
    for (int r = 0; r < 4; r++) v[r] = v[r] * o.weight + (a.bias && n + r < a.N ? a.bias[n + r] : 0.0f);
    const uint32_t s = lh_segment_of(a.seg, n);              // (of all four columns where the boundaries are aligned)
    if (a.seg.pairs) {
        if (a.seg.aligned4 && a.seg.act[s] == LH_ACT_SILU_PAIRS && !a.seg.f32[s]) {
            *reinterpret_cast<uint32_t*>(static_cast<uint16_t*>(a.seg.out[s]) + (size_t)o.row * a.seg.ld[s] + (n - a.seg.n0[s]) / 2) =
                lh_pack_bf(v[0] * lh_sigmoid(v[0]) * v[1], v[2] * lh_sigmoid(v[2]) * v[3]);
            return;
        }
        lh_segment_store_pair(a.seg, o.row, n, v[0], v[1], pos0);   // every count of columns is even here
        if (n + 2 < a.N) lh_segment_store_pair(a.seg, o.row, n + 2, v[2], v[3], pos0);
        return;
    }
    if (!a.seg.aligned4 || !a.seg.vec4[s]) {
#pragma unroll 1
        for (uint32_t r = 0; r < 4 && n + r < a.N; r++) lh_segment_store(a.seg, o.row, n + r, r == 0 ? v[0] : r == 1 ? v[1] : r == 2 ? v[2] : v[3], pos0);
        return;
    }
    const uint32_t p = lh_segment_at_position(a.seg, s) ? pos0 + o.row : o.row;
    if (p >= a.seg.rows[s]) return;
    uint32_t c = n - a.seg.n0[s];
    if (a.seg.head[s] != a.seg.padded[s]) { const uint32_t h = c / a.seg.head[s]; c = h * a.seg.padded[s] + (c - h * a.seg.head[s]); }
    const size_t idx = (size_t)p * a.seg.ld[s] + c;
    const uint32_t act = a.seg.act[s];
    if (act != LH_ACT_NONE) {
#pragma unroll
        for (int r = 0; r < 4; r++) v[r] = lh_activate(v[r], act);
    }
    if (a.seg.f32[s]) {
        float4* d = reinterpret_cast<float4*>(static_cast<float*>(a.seg.out[s]) + idx);
        float4 t = make_float4(v[0], v[1], v[2], v[3]);
        if (a.seg.accumulate) { const float4 x = *d; t.x += x.x; t.y += x.y; t.z += x.z; t.w += x.w; }
        *d = t;
    } else {
        *reinterpret_cast<uint2*>(static_cast<uint16_t*>(a.seg.out[s]) + idx) = make_uint2(lh_pack_bf(v[0], v[1]), lh_pack_bf(v[2], v[3]));
    }
}

// A finished tile into a value cache: a thread stores a quarter of a block of 32 positions of one column, which is 16 bytes where
// the tile has all of them.  `tile` as linear_mfma_kernel leaves it.
template <int BM, int BN>
__device__ __forceinline__ void store_blocks(const LhLinear& a, uint32_t s, const float* tile, const RowTile& rt, uint32_t n0, uint32_t pos0) {
    const uint32_t first = pos0 + rt.begin, last = min(pos0 + rt.end, a.seg.rows[s]), b0 = first >> 5;      // positions [first, last)
    if (first >= last) return;
    const uint32_t blocks = ((last - 1) >> 5) - b0 + 1, cols = min((uint32_t)BN, a.N - n0);
    uint16_t* out = static_cast<uint16_t*>(a.seg.out[s]);
#pragma unroll 1
    for (uint32_t e = threadIdx.x; e < blocks * cols * 4; e += 256) {
        const uint32_t g = e & 3, j = (e >> 2) % cols, b = b0 + (e >> 2) / cols, n = n0 + j;
        uint32_t c = n - a.seg.n0[s];
        if (a.seg.head[s] != a.seg.padded[s]) { const uint32_t h = c / a.seg.head[s]; c = h * a.seg.padded[s] + (c - h * a.seg.head[s]); }
        uint16_t* d = out + ((size_t)b * a.seg.ld[s] + c) * 32 + g * 8;
        const float bias = a.bias ? a.bias[n] : 0.0f;
        uint16_t v[8];
        bool all = true, in[8];
#pragma unroll
        for (uint32_t i = 0; i < 8; i++) {                    // entries 8 g + i: positions 4 g + i and 16 + 4 g + i - 4
            const uint32_t p = b * 32 + (i >> 2) * 16 + g * 4 + (i & 3);
            in[i] = p >= first && p < last;
            all = all && in[i];
            const uint32_t m = in[i] ? p - first : 0u;
            v[i] = lh_f2bf(lh_activate(tile[(m * (BN / 4) + ((j >> 2) ^ (m & 7))) * 4 + (j & 3)] + bias, a.seg.act[s]));
        }
        if (all) *reinterpret_cast<uint4*>(d) = make_uint4(v[0] | (uint32_t)v[1] << 16, v[2] | (uint32_t)v[3] << 16, v[4] | (uint32_t)v[5] << 16, v[6] | (uint32_t)v[7] << 16);
        else {
#pragma unroll
            for (uint32_t i = 0; i < 8; i++) if (in[i]) d[i] = v[i];
        }
    }
}

// ---- matrix cores ------------------------------------------------------------------------------------------------------
// 256 threads, 2 x 2 waves of BM/2 x BN/2 outputs.  A k step is 64 wide: a tile row is eight 16-byte chunks, chunk c of row r
// kept at place c ^ (r & 7) of its row so that the fragment reads of sixteen rows fall on different banks (the loads
// write LDS in order, so the permutation is applied to their global addresses).  NS buffers, one barrier per step: step kt is
// multiplied while the loads of the NS - 1 steps after it are on their way.
// The weights are the MFMA's row operand: lane = output row (lane & 15), four consecutive output columns per tile.
template <int N> __device__ __forceinline__ void wait_loads() { asm volatile("s_waitcnt vmcnt(%0)" :: "n"(N) : "memory"); }

template <int BM, int BN, int NS>
__global__ __launch_bounds__(256) void linear_mfma_kernel(const LhLinear a) {
    constexpr int TI = BM / 32, TJ = BN / 32, CA = BM / 32, CB = BN / 32;
    static_assert(NS * (BM + BN) * 128 >= BM * BN * 4, "the output tile must fit the staging buffers");
    __shared__ uint4 sm[NS][(BM + BN) * 8];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, wm = wave >> 1, wn = wave & 1;
    const uint32_t mt_n = a.ex.tiles ? a.ex.n_tiles : (a.M + BM - 1) / BM, nt_n = (a.N + BN - 1) / BN;
    uint32_t mt, nt;
    tile_of_block(mt_n, nt_n, mt, nt);
    const RowTile rt = row_tile(a, mt, BM);
    if (rt.begin >= rt.end) return;
    const uint32_t n0 = nt * BN, K = a.K, nk = (K + 63) / 64;
    const uint16_t* A = static_cast<const uint16_t*>(a.A);
    const uint16_t* W = a.W + (size_t)rt.expert * a.N * K;

    const uint16_t* pa[CA];
    const uint16_t* pb[CB];
    const uint32_t src = (tid & 7) ^ ((tid >> 3) & 7);        // the chunk this thread brings in, of every row it serves
#pragma unroll
    for (int i = 0; i < CA; i++) {
        const uint32_t r = min(rt.begin + i * 32 + (tid >> 3), rt.end - 1);
        pa[i] = A + (size_t)a_row(a, r) * a.lda + src * 8;
    }
#pragma unroll
    for (int i = 0; i < CB; i++) pb[i] = W + (size_t)min(n0 + i * 32 + (tid >> 3), a.N - 1) * K + src * 8;

    auto load_step = [&](int buf, uint32_t kt) {
        uint4* base = &sm[buf][wave * 64];
        if (kt * 64 + 64 <= K) {
#pragma unroll
            for (int i = 0; i < CA; i++) load_lds16(pa[i] + kt * 64, base + i * 256);
#pragma unroll
            for (int i = 0; i < CB; i++) load_lds16(pb[i] + kt * 64, base + (CA + i) * 256);
        } else {                                             // the last step of a ragged K: chunks past it read zeros
            const bool past = kt * 64 + src * 8 >= K;
#pragma unroll
            for (int i = 0; i < CA; i++) load_lds16(past ? (const void*)&g_zero16 : (const void*)(pa[i] + kt * 64), base + i * 256);
#pragma unroll
            for (int i = 0; i < CB; i++) load_lds16(past ? (const void*)&g_zero16 : (const void*)(pb[i] + kt * 64), base + (CA + i) * 256);
        }
    };

    lh_f32x4 acc[TI][TJ];
#pragma unroll
    for (int i = 0; i < TI; i++)
#pragma unroll
        for (int j = 0; j < TJ; j++) acc[i][j] = (lh_f32x4){0.f, 0.f, 0.f, 0.f};

#pragma unroll
    for (int i = 0; i < NS - 1; i++) if (i < (int)nk) load_step(i, i);
    uint32_t buf = 0;
    for (uint32_t kt = 0; kt < nk; kt++) {
        if (kt + NS - 1 <= nk) wait_loads<(NS - 2) * (CA + CB)>();   // step kt has arrived; the later steps may still be coming
        else wait_loads<0>();
        lh_lds_barrier();
        if (kt + NS - 1 < nk) load_step(buf == 0 ? NS - 1 : buf - 1, kt + NS - 1);
        const uint4* as = sm[buf];
        buf = buf + 1 == NS ? 0 : buf + 1;
        const uint4* bs = as + BM * 8;
#pragma unroll
        for (int ks = 0; ks < 2; ks++) {
            lh_bf16x8 fa[TI], fb[TJ];
            const uint32_t c = ks * 4 + (lane >> 4);
#pragma unroll
            for (int i = 0; i < TI; i++) {
                const uint32_t r = wm * (BM / 2) + i * 16 + (lane & 15);
                fa[i] = __builtin_bit_cast(lh_bf16x8, as[r * 8 + (c ^ (r & 7))]);
            }
#pragma unroll
            for (int j = 0; j < TJ; j++) {
                const uint32_t r = wn * (BN / 2) + j * 16 + (lane & 15);
                fb[j] = __builtin_bit_cast(lh_bf16x8, bs[r * 8 + (c ^ (r & 7))]);
            }
#pragma unroll
            for (int i = 0; i < TI; i++)
#pragma unroll
                for (int j = 0; j < TJ; j++) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fb[j], fa[i], acc[i][j], 0, 0, 0);
        }
    }

    // The tile goes through LDS, so that a wave stores whole stretches of a row (and the store code exists once): four columns
    // of row m are the 16-byte piece n / 4, kept at place (n / 4) ^ (m & 7).
    __syncthreads();
    float4* tile = reinterpret_cast<float4*>(&sm[0][0]);
#pragma unroll
    for (int i = 0; i < TI; i++)
#pragma unroll
        for (int j = 0; j < TJ; j++) {
            const uint32_t m = wm * (BM / 2) + i * 16 + (lane & 15), c = (wn * (BN / 2) + j * 16) / 4 + (lane >> 4);
            tile[m * (BN / 4) + (c ^ (m & 7))] = make_float4(acc[i][j][0], acc[i][j][1], acc[i][j][2], acc[i][j][3]);
        }
    __syncthreads();
    const uint32_t pos0 = a.seg.position ? *a.seg.position : 0u;
    const uint32_t s = lh_segment_of(a.seg, n0);
    if (a.seg.layout[s] == LH_BLOCKS_AT_POSITION && !a.seg.f32[s] && s == lh_segment_of(a.seg, min(n0 + BN, a.N) - 1) && a.ex.tiles == nullptr) {
        store_blocks<BM, BN>(a, s, reinterpret_cast<const float*>(tile), rt, n0, pos0);
        return;
    }
#pragma unroll 1
    for (uint32_t e = tid; e < BM * BN / 4; e += 256) {
        const uint32_t m = e / (BN / 4), c = e % (BN / 4), n = n0 + c * 4, slot = rt.begin + m;
        if (slot >= rt.end || n >= a.N) continue;
        store4(a, slot, n, tile[m * (BN / 4) + (c ^ (m & 7))], pos0);
    }
}

// ---- f32 FMA -----------------------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void linear_plain_kernel(const LhLinear a) {
    constexpr int BK = 16;
    __shared__ float as[BK][64 + 4], bs[BK][64 + 4];
    const uint32_t tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
    const uint32_t bm = a.ex.tiles ? a.ex.tile_rows : 64u, nt_n = (a.N + 63) / 64, mt = blockIdx.x / nt_n, nt = blockIdx.x % nt_n;
    const RowTile rt = row_tile(a, mt, bm);
    const T* A = static_cast<const T*>(a.A);
    const uint16_t* W = a.W + (size_t)rt.expert * a.N * a.K;
    const uint32_t n0 = nt * 64, K = a.K, pos0 = a.seg.position ? *a.seg.position : 0u;
    for (uint32_t begin = rt.begin; begin < rt.end; begin += 64) {
        float acc[4][4] = {};
        for (uint32_t k0 = 0; k0 < K; k0 += BK) {
            for (uint32_t e = tid; e < 64 * BK; e += 256) {
                const uint32_t r = e >> 4, k = k0 + (e & 15);
                const bool ka = k < K;
                as[e & 15][r] = ka && begin + r < rt.end ? lh_ld(A, (size_t)a_row(a, begin + r) * a.lda + k) : 0.0f;
                bs[e & 15][r] = ka && n0 + r < a.N ? lh_bf2f(W[(size_t)(n0 + r) * K + k]) : 0.0f;
            }
            __syncthreads();
#pragma unroll
            for (int k = 0; k < BK; k++) {
                float x[4], w[4];
#pragma unroll
                for (int i = 0; i < 4; i++) { x[i] = as[k][ty * 4 + i]; w[i] = bs[k][tx * 4 + i]; }
#pragma unroll
                for (int i = 0; i < 4; i++)
#pragma unroll
                    for (int j = 0; j < 4; j++) acc[i][j] = __builtin_fmaf(x[i], w[j], acc[i][j]);
            }
            __syncthreads();
        }
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const uint32_t slot = begin + ty * 4 + i;
            if (slot >= rt.end) continue;
            const OutRow o = out_row(a, slot);
            if (a.seg.pairs) {                                // (an expert's weight and a bias do not occur with pairs of a plain product)
#pragma unroll
                for (int j = 0; j < 4; j += 2) {
                    const uint32_t n = n0 + tx * 4 + j;
                    if (n < a.N) lh_segment_store_pair(a.seg, o.row, n, acc[i][j] + (a.bias ? a.bias[n] : 0.0f), acc[i][j + 1] + (a.bias ? a.bias[n + 1] : 0.0f), pos0);
                }
                continue;
            }
#pragma unroll
            for (int j = 0; j < 4; j++) {
                const uint32_t n = n0 + tx * 4 + j;
                if (n < a.N) lh_segment_store(a.seg, o.row, n, acc[i][j] * o.weight + (a.bias ? a.bias[n] : 0.0f), pos0);
            }
        }
    }
}

// ---- one row -----------------------------------------------------------------------------------------------------------
// Place of element k in the staged vector: the two halves of an 8-element chunk lie in planes of 64 x 16 bytes, so that the
// 16-byte reads of a wave (lane = chunk) are in order.
__device__ __forceinline__ uint32_t x_place(uint32_t k) {
    const uint32_t chunk = k >> 3, j = k & 7;
    return (((chunk >> 6) * 2 + (j >> 2)) << 8) + ((chunk & 63) << 2) + (j & 3);
}

template <int STAGE>
__device__ void stage_vector(const VectorStage& st, float* xs, float* scratch, uint32_t K) {
    auto gate = [&](uint32_t k) { return lh_gate(st.gate_f32 ? static_cast<const float*>(st.gate)[k] : lh_bf2f(static_cast<const uint16_t*>(st.gate)[k]), st.gate_act); };
    auto value = [&](uint32_t k) {
        if constexpr (STAGE == kPlain) return st.x_f32 ? static_cast<const float*>(st.x)[k] : lh_bf2f(static_cast<const uint16_t*>(st.x)[k]);
        float v = static_cast<const float*>(st.x)[k];
        if (STAGE == kNorm && st.add) v += st.add[k];
        if constexpr (STAGE == kGated) if (st.gate_first) v *= gate(k);
        return v;
    };
    auto weight = [&](uint32_t k) {
        const float w = STAGE != kGated || st.norm_weight ? st.norm_weight[k] : 1.0f;
        if constexpr (STAGE == kGated) return st.gate_first ? w : w * gate(k);
        return w;
    };
    const uint32_t padded = (K + 511) / 512 * 512;
    if constexpr (STAGE == kResidual) {
        float s = 0.0f;
        for (uint32_t k = threadIdx.x; k < K; k += blockDim.x) { const float y = st.add[k]; s += y * y; }
        const float r = rsqrtf(lh_block_sum(s, scratch) / (float)K + st.eps);
        for (uint32_t k = threadIdx.x; k < padded; k += blockDim.x) {
            const float v = k < K ? __builtin_fmaf(st.add[k] * st.norm_weight[k], r, value(k)) : 0.0f;
            xs[x_place(k)] = v;
            if (st.store && blockIdx.x == 0 && k < K) st.store[k] = v;
        }
    } else if constexpr (STAGE == kPlain) {
        for (uint32_t k = threadIdx.x; k < padded; k += blockDim.x) xs[x_place(k)] = k < K ? value(k) : 0.0f;
    } else {
        constexpr int R = 8;                                  // elements a thread keeps between the passes; the rest are read again
        float keep[R], wk[R];
        float s = 0.0f;
#pragma unroll
        for (int i = 0; i < R; i++) {
            const uint32_t k = threadIdx.x + i * blockDim.x;
            keep[i] = k < K ? value(k) : 0.0f;
            wk[i] = k < K ? weight(k) : 0.0f;
            s += keep[i] * keep[i];
        }
        for (uint32_t k = threadIdx.x + R * blockDim.x; k < K; k += blockDim.x) { const float v = value(k); s += v * v; }
        const float r = rsqrtf(lh_block_sum(s, scratch) / (float)K + st.eps);
        const bool store = STAGE == kNorm && st.store != nullptr && blockIdx.x == 0;
#pragma unroll
        for (int i = 0; i < R; i++) {
            const uint32_t k = threadIdx.x + i * blockDim.x;
            if (k < padded) xs[x_place(k)] = keep[i] * r * wk[i];
            if (store && k < K) st.store[k] = keep[i];
        }
        for (uint32_t k = threadIdx.x + R * blockDim.x; k < padded; k += blockDim.x) {
            float v = 0.0f, w = 0.0f;
            if (k < K) {
                v = value(k);
                w = weight(k);
                if (store) st.store[k] = v;
            }
            xs[x_place(k)] = v * r * w;
        }
    }
    __syncthreads();
}

// Which rows a wave (or workgroup) takes: every `count`-th from `first` on; of (gate, up) pairs both.
struct RowWalk {
    const uint32_t first, count, pairs;
    __device__ __forceinline__ uint32_t row(uint32_t i) const { return pairs ? 2 * (first + (i >> 1) * count) + (i & 1) : first + i * count; }
};

// Stores the finished sums of rows i0 .. i0 + n - 1 of a walk, one per lane.
__device__ __forceinline__ void store_sums(const LhSegments& seg, const float* bias, const RowWalk& walk, uint32_t i0, uint32_t n, uint32_t lane, float v) {
    const uint32_t row = walk.row(i0 + lane);
    if (bias && lane < n) v += bias[row];
    if (walk.pairs) {                                         // n is even, and a pair's factors are in neighbouring lanes
        const float up = lh_dpp_f<LH_DPP_QUAD_XOR1>(v);
        if (lane < n && !(lane & 1)) lh_segment_put(seg, 0, row >> 1, v * lh_sigmoid(v) * up);
    } else if (lane < n) lh_segment_store(seg, 0, row, v, seg.position ? *seg.position : 0u);
}

// The finished sums of a wave's rows, one per lane, stored 64 at a time: bias, activation and destination then cost one pass
// for all of them, and no load of that pass has to wait for weights that were requested in between.
struct RowSums {
    const LhSegments& seg;
    const float* bias;
    const RowWalk& walk;
    const uint32_t lane;
    uint32_t i0 = 0, n = 0;
    float mine = 0.0f;
    __device__ __forceinline__ void add(float total) {
        mine = n == lane ? total : mine;
        if (++n == 64) flush();
    }
    __device__ __forceinline__ void flush() {
        store_sums(seg, bias, walk, i0, n, lane, mine);
        i0 += n;
        n = 0;
    }
};

// A wave takes rows round robin over the grid, 8 weights (16 bytes) per lane and load, NL loads per pass of a row; the loads
// of the next pass are issued before the arithmetic of the current one.  Past the row's end the address is clamped and the
// staged vector is zero.  VEC false (K not a multiple of 8): single weights.
template <int STAGE, int NL, bool VEC>
__global__ __launch_bounds__(256) void matvec_bf16_kernel(const VectorStage st, const uint16_t* __restrict__ W, const float* __restrict__ bias, const LhSegments seg,
                                                         uint32_t N, uint32_t K) {
    extern __shared__ __align__(16) float xs[];
    __shared__ float scratch[4];
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    stage_vector<STAGE>(st, xs, scratch, K);
    const RowWalk walk{blockIdx.x * 4 + wave, gridDim.x * 4, seg.pairs};
    RowSums sums{seg, bias, walk, lane};
    if constexpr (VEC) {
        constexpr uint32_t kPass = 512u * NL;
        const uint32_t ppr = (K + kPass - 1) / kPass, last = (K >> 3) - 1;
        uint32_t at = 0, row = walk.row(0), pass = 0;
        auto issue = [&](uint4 (&v)[NL], uint32_t r, uint32_t ps) {
            const uint16_t* wr = W + (size_t)r * K;
#pragma unroll
            for (int c = 0; c < NL; c++) v[c] = lh_ld16_stream(wr + 8 * min(ps * (kPass >> 3) + 64u * c + lane, last));
        };
        float acc = 0.0f;
        auto consume = [&](const uint4 (&v)[NL], uint32_t r, uint32_t ps) {
#pragma unroll
            for (int c = 0; c < NL; c++) {
                const uint32_t q = ps * NL + c;
                if (q * 512 >= K) break;
                const float4 x0 = *reinterpret_cast<const float4*>(&xs[(q * 2) * 256 + lane * 4]), x1 = *reinterpret_cast<const float4*>(&xs[(q * 2 + 1) * 256 + lane * 4]);
                const float xv[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
                const uint32_t wv[4] = {v[c].x, v[c].y, v[c].z, v[c].w};
#pragma unroll
                for (int j = 0; j < 4; j++) {
                    acc = __builtin_fmaf(__builtin_bit_cast(float, wv[j] << 16), xv[2 * j], acc);
                    acc = __builtin_fmaf(__builtin_bit_cast(float, wv[j] & 0xFFFF0000u), xv[2 * j + 1], acc);
                }
            }
            if (ps + 1 == ppr) { sums.add(lh_group_sum(acc, 64)); acc = 0.0f; }
        };
        auto step = [&](const uint4 (&cur)[NL], uint4 (&nxt)[NL]) {   // false: that was the wave's last pass
            uint32_t nrow = row, npass = pass + 1;
            if (npass == ppr) { npass = 0; nrow = walk.row(++at); }
            const bool more = nrow < N;
            if (more) issue(nxt, nrow, npass);
            consume(cur, row, pass);
            row = nrow; pass = npass;
            return more;
        };
        uint4 p[NL], q[NL];
        if (row < N) {
            issue(p, row, 0);
            while (step(p, q) && step(q, p)) {}
        }
    } else {
        for (uint32_t i = 0, row; (row = walk.row(i)) < N; i++) {
            float acc = 0.0f;
            for (uint32_t k = lane; k < K; k += 64) acc = __builtin_fmaf(lh_bf2f(W[(size_t)row * K + k]), xs[x_place(k)], acc);
            sums.add(lh_group_sum(acc, 64));
        }
    }
    sums.flush();
}

// The same with the vector in registers (K up to 512 * NL): the first row's weights are requested before the vector.
template <int STAGE, int NL>
__global__ __launch_bounds__(256) void matvec_bf16_reg_kernel(const VectorStage st, const uint16_t* __restrict__ W, const float* __restrict__ bias, const LhSegments seg,
                                                             uint32_t N, uint32_t K) {
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6, last = (K >> 3) - 1;
    const RowWalk walk{blockIdx.x * 4 + wave, gridDim.x * 4, seg.pairs};
    auto issue = [&](uint4 (&v)[NL], uint32_t r) {
        const uint16_t* wr = W + (size_t)r * K;
#pragma unroll
        for (int c = 0; c < NL; c++) v[c] = lh_ld16_stream(wr + 8 * min(64u * c + lane, last));
    };
    uint32_t at = 0;
    if (walk.row(0) >= N) return;
    uint4 p[NL], q[NL];
    issue(p, walk.row(0));
    RowSums sums{seg, bias, walk, lane};
    float xr[NL][8];
    lh_vector_registers<STAGE, NL>(st, K, lane, blockIdx.x == 0 && wave == 0 && st.store != nullptr, xr);
    auto step = [&](const uint4 (&cur)[NL], uint4 (&nxt)[NL]) {   // false: that was the wave's last row
        const uint32_t next = walk.row(++at);
        const bool more = next < N;
        if (more) issue(nxt, next);
        float acc = 0.0f;
#pragma unroll
        for (int c = 0; c < NL; c++) acc = lh_dot8(cur[c], xr[c], acc);
        sums.add(lh_group_sum(acc, 64));
        return more;
    };
    while (step(p, q) && step(q, p)) {}
    sums.flush();
}

// Rows longer than a wave's registers: the four waves of a workgroup take a quarter of the columns each, and the quarters of up to 64 rows meet in LDS.  Plain vectors only: a norm would need all quarters.
template <int NL>
__global__ __launch_bounds__(256) void matvec_bf16_quarter_kernel(const VectorStage st, const uint16_t* __restrict__ W, const float* __restrict__ bias, const LhSegments seg,
                                                                 uint32_t N, uint32_t K, uint32_t quarter) {
    __shared__ float sums[4][64];
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6, k0 = wave * quarter, len = k0 < K ? min(quarter, K - k0) : 0u;   // quarter: a multiple of 8
    const uint32_t last = len ? (len >> 3) - 1 : 0u, kb = len ? k0 : 0u;
    auto issue = [&](uint4 (&v)[NL], uint32_t r) {
        const uint16_t* wr = W + (size_t)r * K + kb;
#pragma unroll
        for (int c = 0; c < NL; c++) v[c] = lh_ld16_stream(wr + 8 * min(64u * c + lane, last));
    };
    const RowWalk walk{blockIdx.x, gridDim.x, seg.pairs};
    uint32_t at = 0, i0 = 0, n = 0;
    if (walk.row(0) >= N) return;
    uint4 p[NL], q[NL];
    issue(p, walk.row(0));
    VectorStage part = st;
    part.x = st.x_f32 ? (const void*)(static_cast<const float*>(st.x) + kb) : (const void*)(static_cast<const uint16_t*>(st.x) + kb);
    float xr[NL][8], mine = 0.0f;
    lh_vector_registers<kPlain, NL>(part, len, lane, false, xr);
    auto flush = [&]() {
        sums[wave][lane] = mine;
        __syncthreads();
        if (wave == 0) store_sums(seg, bias, walk, i0, n, lane, (sums[0][lane] + sums[1][lane]) + (sums[2][lane] + sums[3][lane]));
        __syncthreads();
        i0 += n;
        n = 0;
    };
    auto step = [&](const uint4 (&cur)[NL], uint4 (&nxt)[NL]) {
        const uint32_t next = walk.row(++at);
        const bool more = next < N;
        if (more) issue(nxt, next);
        float acc = 0.0f;
#pragma unroll
        for (int c = 0; c < NL; c++) acc = lh_dot8(cur[c], xr[c], acc);
        acc = lh_group_sum(acc, 64);
        mine = n == lane ? acc : mine;
        if (++n == 64) flush();
        return more;
    };
    while (step(p, q) && step(q, p)) {}
    if (n) flush();
}

constexpr uint32_t kMaxVectorK = 36864;   // 144 KB of staged f32 activations

template <int STAGE>
int launch_vector(lh_context* ctx, const VectorStage& st, const uint16_t* W, const float* bias, const LhSegments& seg, uint32_t N, uint32_t K, const char* op) {
    LH_REQUIRE(K > 0 && K <= kMaxVectorK, "%s: k %u outside 1..=%u", op, K, kMaxVectorK);
    const size_t lds = (size_t)(K + 511) / 512 * 512 * 4;
    const uint32_t takes = seg.pairs ? N / 2 : N;             // rows, or pairs of rows
    const bool vec = K % 8 == 0 && ((uintptr_t)W & 15) == 0;
    if (vec && K <= 4096 && lh_stage_aligned(st)) {
        const uint32_t grid = (uint32_t)std::min<uint64_t>(((uint64_t)takes + 3) / 4, (uint64_t)ctx->cu_count * (K <= 2048 ? 4 : 2));
#define LH_MVR(NLOADS) hipLaunchKernelGGL((matvec_bf16_reg_kernel<STAGE, NLOADS>), dim3(grid), dim3(256), 0, ctx->stream, st, W, bias, seg, N, K)
        if (K <= 512) LH_MVR(1);
        else if (K <= 1024) LH_MVR(2);
        else if (K <= 2048) LH_MVR(4);
        else LH_MVR(8);
#undef LH_MVR
        return lh_check_launch(op);
    }
    if constexpr (STAGE == kPlain) if (vec && K <= 16384 && lh_stage_aligned(st)) {
        const uint32_t quarter = ((K + 3) / 4 + 7) / 8 * 8, grid = (uint32_t)std::min<uint64_t>(takes, (uint64_t)ctx->cu_count * 4);
        if (quarter <= 1024) hipLaunchKernelGGL((matvec_bf16_quarter_kernel<2>), dim3(grid), dim3(256), 0, ctx->stream, st, W, bias, seg, N, K, quarter);
        else if (quarter <= 2048) hipLaunchKernelGGL((matvec_bf16_quarter_kernel<4>), dim3(grid), dim3(256), 0, ctx->stream, st, W, bias, seg, N, K, quarter);
        else hipLaunchKernelGGL((matvec_bf16_quarter_kernel<8>), dim3(grid), dim3(256), 0, ctx->stream, st, W, bias, seg, N, K, quarter);
        return lh_check_launch(op);
    }
    const uint32_t grid = (uint32_t)std::min<uint64_t>(((uint64_t)takes + 3) / 4, (uint64_t)ctx->cu_count * 4);
#define LH_MV(NLOADS, V)                                                                                                               \
    do {                                                                                                                               \
        if (lds > 64 * 1024 - 64) {                                                                                                    \
            const int rr = lh_raise_dynamic_lds(ctx, (const void*)matvec_bf16_kernel<STAGE, NLOADS, V>, lds, op);                      \
            if (rr != LH_OK) return rr;                                                                                                \
        }                                                                                                                              \
        hipLaunchKernelGGL((matvec_bf16_kernel<STAGE, NLOADS, V>), dim3(grid), dim3(256), lds, ctx->stream, st, W, bias, seg, N, K);    \
    } while (0)
    if (!vec) LH_MV(1, false);
    else if (K <= 512) LH_MV(1, true);
    else if (K <= 1024) LH_MV(2, true);
    else LH_MV(4, true);
#undef LH_MV
    return lh_check_launch(op);
}

int check_common(lh_batch* batch, const lh_buffer* weight, const lh_buffer* bias, uint32_t k, uint64_t n, const char* op) {
    LH_REQUIRE(k > 0, "%s: k is 0", op);
    LH_NEED(weight, (size_t)n * k * 2, op, "weight");
    if (bias) LH_NEED(bias, (size_t)n * 4, op, "bias");
    return LH_OK;
}
#define LH_TRY(expr)                  \
    do {                              \
        const int rt__ = (expr);      \
        if (rt__ != LH_OK) return rt__; \
    } while (0)

int vector_entry(lh_batch* batch, const char* op, int stage, const VectorStage& st, const lh_buffer* weight, const lh_buffer* bias, uint32_t k,
                 uint32_t count, const uint32_t* ns, const uint32_t* acts, const uint32_t* heads, const uint32_t* padded, const uint32_t* layouts,
                 lh_buffer* const* outputs, int output_dtype, int accumulate, const lh_buffer* position) {
    LhSegments seg;
    LH_TRY(lh_make_segments(seg, op, 1, 0, count, ns, acts, heads, padded, layouts, outputs, output_dtype, accumulate, position));
    LH_REQUIRE(!seg.pairs || seg.count == 1, "%s: pairs beside other segments", op);
    const uint32_t n = seg.n0[seg.count];
    LH_TRY(check_common(batch, weight, bias, k, n, op));
    const uint16_t* W = (const uint16_t*)weight->ptr;
    const float* b = bias ? (const float*)bias->ptr : nullptr;
    int r;
    if (stage == kResidual) r = launch_vector<kResidual>(batch->ctx, st, W, b, seg, n, k, op);
    else if (stage == kPlain) r = launch_vector<kPlain>(batch->ctx, st, W, b, seg, n, k, op);
    else if (stage == kNorm) r = launch_vector<kNorm>(batch->ctx, st, W, b, seg, n, k, op);
    else r = launch_vector<kGated>(batch->ctx, st, W, b, seg, n, k, op);
    if (r == LH_OK) batch->dispatch_count++;
    return r;
}

}  // namespace

uint32_t lh_expert_tile_rows(uint32_t slots, uint32_t experts) { return slots / (experts ? experts : 1) >= 128 ? 128u : 64u; }

int lh_launch_linear(lh_context* ctx, const LhLinear& given, const char* op) {
    LhLinear a = given;
    if (a.lda == 0) a.lda = a.K;
    const bool mfma = !a.a_f32 && a.K % 8 == 0 && a.lda % 8 == 0 && (((uintptr_t)a.A | (uintptr_t)a.W) & 15) == 0;
    if (!mfma) {
        const uint64_t mt = a.ex.tiles ? a.ex.n_tiles : ((uint64_t)a.M + 63) / 64, grid = mt * ((a.N + 63) / 64);
        LH_REQUIRE(grid < 0x7FFFFFFFull, "%s: %u x %u outputs", op, a.M, a.N);
        if (grid == 0) return LH_OK;
        if (a.a_f32) hipLaunchKernelGGL((linear_plain_kernel<float>), dim3((uint32_t)grid), dim3(256), 0, ctx->stream, a);
        else hipLaunchKernelGGL((linear_plain_kernel<uint16_t>), dim3((uint32_t)grid), dim3(256), 0, ctx->stream, a);
        return lh_check_launch(op);
    }
    auto tiles = [&](uint32_t bm, uint32_t bn) { return (uint64_t)(a.ex.tiles ? a.ex.n_tiles : (a.M + bm - 1) / bm) * ((a.N + bn - 1) / bn); };
#define LH_GEMM(BM_, BN_, NS_)                                                                                             \
    do {                                                                                                                \
        const uint64_t grid = tiles(BM_, BN_);                                                                          \
        LH_REQUIRE(grid < 0x7FFFFFFFull, "%s: %u x %u outputs", op, a.M, a.N);                                          \
        if (grid) hipLaunchKernelGGL((linear_mfma_kernel<BM_, BN_, NS_>), dim3((uint32_t)grid), dim3(256), 0, ctx->stream, a); \
    } while (0)
    const uint64_t want = (uint64_t)ctx->cu_count;
    if (a.ex.tiles) {
        if (a.ex.tile_rows == 128) { if (tiles(128, 128) >= want) LH_GEMM(128, 128, 2); else LH_GEMM(128, 64, 3); }
        else LH_GEMM(64, 64, 4);
    } else if (tiles(128, 128) >= 2 * want) LH_GEMM(128, 128, 2);
    else if (tiles(128, 64) >= want) LH_GEMM(128, 64, 3);
    else if (tiles(64, 64) >= want || a.M > 32) LH_GEMM(64, 64, 4);
    else LH_GEMM(32, 32, 4);
#undef LH_GEMM
    return lh_check_launch(op);
}

extern "C" {

int lh_linear_rows_into(lh_batch* batch, const lh_buffer* input, int input_dtype, const lh_buffer* weight, const lh_buffer* bias, uint32_t m, uint32_t k,
                        uint32_t count, const uint32_t* ns, const uint32_t* acts, const uint32_t* heads, const uint32_t* padded, const uint32_t* layouts,
                        lh_buffer* const* outputs, int output_dtype, int accumulate, const lh_buffer* position) {
    const char* op = "linear_rows";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(input_dtype == LH_F32 || input_dtype == LH_BF16, "%s: input dtype %d", op, input_dtype);
    if (m == 0) return LH_OK;
    LhLinear a;
    memset(&a, 0, sizeof a);
    LH_TRY(lh_make_segments(a.seg, op, m, 0, count, ns, acts, heads, padded, layouts, outputs, output_dtype, accumulate, position));
    a.N = a.seg.n0[a.seg.count];
    LH_TRY(check_common(batch, weight, bias, k, a.N, op));
    LH_NEED(input, (size_t)m * k * (input_dtype == LH_F32 ? 4 : 2), op, "input");
    a.A = input->ptr; a.a_f32 = input_dtype == LH_F32;
    a.W = (const uint16_t*)weight->ptr; a.bias = bias ? (const float*)bias->ptr : nullptr;
    a.M = m; a.K = k;
    const int r = lh_launch_linear(batch->ctx, a, op);
    if (r == LH_OK) batch->dispatch_count++;
    return r;
}

int lh_linear_vector_into(lh_batch* batch, const lh_buffer* input, int input_dtype, const lh_buffer* weight, const lh_buffer* bias, uint32_t k,
                          uint32_t count, const uint32_t* ns, const uint32_t* acts, const uint32_t* heads, const uint32_t* padded,
                          const uint32_t* layouts, lh_buffer* const* outputs, int output_dtype, int accumulate, const lh_buffer* position) {
    const char* op = "linear_vector";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(input_dtype == LH_F32 || input_dtype == LH_BF16, "%s: input dtype %d", op, input_dtype);
    LH_NEED(input, (size_t)k * (input_dtype == LH_F32 ? 4 : 2), op, "input");
    VectorStage st{};
    st.x = input->ptr; st.x_f32 = input_dtype == LH_F32;
    return vector_entry(batch, op, kPlain, st, weight, bias, k, count, ns, acts, heads, padded, layouts, outputs, output_dtype, accumulate, position);
}

int lh_linear_norm_vector_into(lh_batch* batch, const lh_buffer* input, const lh_buffer* add, lh_buffer* store, const lh_buffer* norm_weight, float eps,
                               const lh_buffer* weight, const lh_buffer* bias, uint32_t k, uint32_t count, const uint32_t* ns, const uint32_t* acts,
                               const uint32_t* heads, const uint32_t* padded, const uint32_t* layouts, lh_buffer* const* outputs, int output_dtype,
                               int accumulate, const lh_buffer* position) {
    const char* op = "linear_norm_vector";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_NEED(input, (size_t)k * 4, op, "input");
    LH_NEED(norm_weight, (size_t)k * 4, op, "norm_weight");
    if (add) LH_NEED(add, (size_t)k * 4, op, "add");
    if (store) {
        LH_NEED(store, (size_t)k * 4, op, "store");
        LH_REQUIRE(store->ptr != input->ptr && (!add || store->ptr != add->ptr), "%s: store must not be read by the other workgroups", op);
    }
    VectorStage st{};
    st.x = input->ptr; st.x_f32 = 1; st.add = add ? (const float*)add->ptr : nullptr; st.store = store ? (float*)store->ptr : nullptr;
    st.norm_weight = (const float*)norm_weight->ptr; st.eps = eps;
    return vector_entry(batch, op, kNorm, st, weight, bias, k, count, ns, acts, heads, padded, layouts, outputs, output_dtype, accumulate, position);
}

int lh_linear_residual_vector_into(lh_batch* batch, const lh_buffer* input, const lh_buffer* branch, lh_buffer* store, const lh_buffer* norm_weight,
                                   float eps, const lh_buffer* weight, const lh_buffer* bias, uint32_t k, uint32_t count, const uint32_t* ns,
                                   const uint32_t* acts, const uint32_t* heads, const uint32_t* padded, const uint32_t* layouts, lh_buffer* const* outputs,
                                   int output_dtype, int accumulate, const lh_buffer* position) {
    const char* op = "linear_residual_vector";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_NEED(input, (size_t)k * 4, op, "input");
    LH_NEED(branch, (size_t)k * 4, op, "branch");
    LH_NEED(norm_weight, (size_t)k * 4, op, "norm_weight");
    if (store) {
        LH_NEED(store, (size_t)k * 4, op, "store");
        LH_REQUIRE(store->ptr != input->ptr && store->ptr != branch->ptr, "%s: store must not be read by the other workgroups", op);
    }
    VectorStage st{};
    st.x = input->ptr; st.x_f32 = 1; st.add = (const float*)branch->ptr; st.store = store ? (float*)store->ptr : nullptr;
    st.norm_weight = (const float*)norm_weight->ptr; st.eps = eps;
    return vector_entry(batch, op, kResidual, st, weight, bias, k, count, ns, acts, heads, padded, layouts, outputs, output_dtype, accumulate, position);
}

uint32_t lh_gated_vector_fits(uint32_t k, uint32_t group) {
    if (group == k) return 1;
    if (group == 0 || k % group || group % 8 || k > 4096) return 0;
    const uint32_t c = group / 8;
    return c % 64 == 0 || (c < 64 && (c & (c - 1)) == 0);
}

int lh_linear_gated_vector_into(lh_batch* batch, const lh_buffer* input, const lh_buffer* gate, int gate_dtype, uint32_t gate_act, int gate_first,
                                const lh_buffer* norm_weight, uint32_t group, float eps, const lh_buffer* weight, const lh_buffer* bias, uint32_t k, uint32_t count, const uint32_t* ns, const uint32_t* acts,
                                const uint32_t* heads, const uint32_t* padded, const uint32_t* layouts, lh_buffer* const* outputs, int output_dtype,
                                int accumulate, const lh_buffer* position) {
    const char* op = "linear_gated_vector";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(gate_dtype == LH_F32 || gate_dtype == LH_BF16, "%s: gate dtype %d", op, gate_dtype);
    LH_NEED(input, (size_t)k * 4, op, "input");
    LH_NEED(gate, (size_t)k * (gate_dtype == LH_F32 ? 4 : 2), op, "gate");
    if (norm_weight) LH_NEED(norm_weight, (size_t)k * 4, op, "norm_weight");
    LH_REQUIRE(gate_act == LH_ACT_SIGMOID || gate_act == LH_ACT_SILU, "%s: gate activation %u", op, gate_act);
    LH_REQUIRE(lh_gated_vector_fits(k, group), "%s: %u values in parts of %u", op, k, group);
    VectorStage st{};
    st.x = input->ptr; st.x_f32 = 1; st.norm_weight = norm_weight ? (const float*)norm_weight->ptr : nullptr; st.gate = gate->ptr;
    st.gate_f32 = gate_dtype == LH_F32; st.gate_act = gate_act; st.gate_first = gate_first != 0; st.group = group; st.eps = eps;
    LH_REQUIRE(group == k || lh_stage_aligned(st), "%s: buffers must be 16-byte aligned", op);
    LH_REQUIRE(group == k || ((uintptr_t)weight->ptr & 15) == 0, "%s: the weight must be 16-byte aligned", op);
    return vector_entry(batch, op, kGated, st, weight, bias, k, count, ns, acts, heads, padded, layouts, outputs, output_dtype, accumulate, position);
}

}  // extern "C"
