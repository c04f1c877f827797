// Causal softmax attention over bf16 (or f32) caches, with one or two score maps per head.  With two maps (differential
// attention) both share the head's values and are combined in the same kernel: the difference of the two averages, the
// second times lambda, an RMS norm over the head, a constant factor.
//
// Caches: keys [position][kv head][map][DQ], values in blocks of 32 positions [block][kv head][DV][32] whose 32 entries
// are in lh_block_slot order.  The queries of one kv head's group are packed: packed row r = query row r / R, head r % R of
// the group (R heads per kv head), so a tile of 16 packed rows uses the matrix cores fully also for one query row.
//
// Matrix-core form (bf16): a step of 32 keys computes S^T = K Q^T (two 16 x 16 tiles; lane = packed row (lane & 15), keys
// 4g .. 4g + 3 of each tile, g = lane >> 4), so a row's maximum and sum are eight registers and two lane exchanges, and
// the weights are already where O^T = V^T P^T wants them: its k index 8g + j is key 4g + j of tile 0 (j < 4) or key
// 4g + j - 4 of tile 1, which is the order of the value blocks.  Scores, weights and sums are f32; a weight enters the
// product as the sum of three bf16 terms, which is all of its 24 bits.
//   attention_tile_kernel   many rows: four waves share key and value blocks through LDS
//   attention_split_kernel  few rows: every wave walks its own share of the blocks straight from global memory; the
//                           workgroup's four partial results are merged in LDS, the workgroups' by attention_merge_kernel
// Plain form (any dtype, any dim): attention_plain_kernel, one workgroup per query row and head.
#include "float_ops.hpp"
#include <algorithm>
#include <cmath>

namespace {

struct AttentionArgs {
    const void* q;
    const void* keys;
    const void* values;
    void* out;
    const uint32_t* position;
    uint32_t rows, heads, kv_heads, maps, dim, dq, vdim, dv, capacity;
    float scale, lambda, out_scale, eps;
    float* partial;            // records [16-row tile][kv head][split][map][16] of dv unnormalised sums, maximum, sum of weights
    uint32_t splits;
};

constexpr float kLog2e = 1.4426950408889634f;

typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));

// The B operand of S^T: query values of packed row `row` (zero past the rows and past dim).
template <int DQ, int MAPS>
__device__ __forceinline__ void load_queries(lh_bf16x8 (&qf)[MAPS][DQ / 32], const AttentionArgs& a, uint32_t g, uint32_t row, uint32_t lane) {
    const uint32_t R = a.heads / a.kv_heads, t = row / R, h = g * R + (row - t * R);
    const bool on = t < a.rows;
#pragma unroll
    for (int mp = 0; mp < MAPS; mp++)
#pragma unroll
        for (int c = 0; c < DQ / 32; c++) {
            const uint32_t k = c * 32 + (lane >> 4) * 8;
            u32x4 v = {0u, 0u, 0u, 0u};
            if (on && k < a.dim) {
                v = *reinterpret_cast<const u32x4*>(static_cast<const uint16_t*>(a.q) + (((size_t)t * a.heads + h) * MAPS + mp) * DQ + k);
#pragma unroll
                for (int j = 0; j < 4; j++) {
                    if (k + 2 * j >= a.dim) v[j] = 0u;
                    else if (k + 2 * j + 1 >= a.dim) v[j] &= 0xFFFFu;
                }
            }
            qf[mp][c] = __builtin_bit_cast(lh_bf16x8, v);
        }
}

// A row tile's running softmax state for one map; every lane holds the values of packed row (lane & 15).
struct RowState { float m, l; };

// Scores of NB steps of 32 keys -> weights in P V operand order, as three bf16 terms; returns the factor for what was summed
// before.  `first` is the first key, `limit` the row's last visible key, `bound` whether any lane may have to mask.
template <int NB>
__device__ __forceinline__ float softmax_step(lh_f32x4 (&s)[2 * NB], RowState& st, float scale2, uint32_t first, uint32_t limit, bool bound, uint32_t lane,
                                              lh_bf16x8 (&w)[NB][3]) {
    float v[8 * NB], mx = -INFINITY;
    const uint32_t g = lane >> 4;
#pragma unroll
    for (int i = 0; i < 8 * NB; i++) {
        v[i] = s[i >> 2][i & 3] * scale2;
        if (bound && first + (i >> 2) * 16 + g * 4 + (i & 3) > limit) v[i] = -INFINITY;
        mx = fmaxf(mx, v[i]);
    }
    const float nm = fmaxf(st.m, lh_column_max(mx)), base = nm == -INFINITY ? 0.0f : nm;
    const float alpha = __builtin_amdgcn_exp2f(st.m - base);
    float sum = 0.0f;
#pragma unroll
    for (int b = 0; b < NB; b++) {
        uint32_t h[4], m[4], l[4];
#pragma unroll
        for (int i = 0; i < 4; i++) {
            float p0 = __builtin_amdgcn_exp2f(v[8 * b + 2 * i] - base), p1 = __builtin_amdgcn_exp2f(v[8 * b + 2 * i + 1] - base);
            sum += p0 + p1;
            h[i] = lh_pack_bf(p0, p1);
            p0 -= __builtin_bit_cast(float, h[i] << 16); p1 -= __builtin_bit_cast(float, h[i] & 0xFFFF0000u);
            m[i] = lh_pack_bf(p0, p1);
            l[i] = lh_pack_bf(p0 - __builtin_bit_cast(float, m[i] << 16), p1 - __builtin_bit_cast(float, m[i] & 0xFFFF0000u));
        }
        w[b][0] = __builtin_bit_cast(lh_bf16x8, (u32x4){h[0], h[1], h[2], h[3]});
        w[b][1] = __builtin_bit_cast(lh_bf16x8, (u32x4){m[0], m[1], m[2], m[3]});
        w[b][2] = __builtin_bit_cast(lh_bf16x8, (u32x4){l[0], l[1], l[2], l[3]});
    }
    st.l = st.l * alpha + sum;      // this lane's keys only; the four lanes of a row are added at the end
    st.m = nm;
    return alpha;
}

// A finished row: o[i][r] holds value 16 i + 4g + r of packed row (lane & 15), for every map unnormalised with sum l.
template <int DV, int MAPS>
__device__ __forceinline__ void finish_row(const AttentionArgs& a, lh_f32x4 (&o)[MAPS][DV / 16], const float (&l)[MAPS], uint32_t g, uint32_t row, uint32_t lane) {
    const uint32_t R = a.heads / a.kv_heads, t = row / R, h = g * R + (row - t * R);
    float inv[MAPS];
#pragma unroll
    for (int mp = 0; mp < MAPS; mp++) inv[mp] = 1.0f / l[mp];
    float ss = 0.0f;
#pragma unroll
    for (int i = 0; i < DV / 16; i++)
#pragma unroll
        for (int r = 0; r < 4; r++) {
            float v = o[0][i][r] * inv[0];
            if constexpr (MAPS == 2) v -= a.lambda * (o[MAPS - 1][i][r] * inv[MAPS - 1]);
            o[0][i][r] = v;
            if ((uint32_t)(i * 16 + (lane >> 4) * 4 + r) < a.vdim) ss += v * v;
        }
    float f = 1.0f;
    if constexpr (MAPS == 2) {
        ss = lh_column_sum(ss);
        f = rsqrtf(ss / (float)a.vdim + a.eps) * a.out_scale;
    }
    if (t >= a.rows) return;
    uint16_t* out = static_cast<uint16_t*>(a.out) + ((size_t)t * a.heads + h) * a.vdim;
#pragma unroll
    for (int i = 0; i < DV / 16; i++) {
        const uint32_t c = i * 16 + (lane >> 4) * 4;
        if ((a.vdim & 3) == 0) {
            if (c < a.vdim) *reinterpret_cast<uint2*>(out + c) = make_uint2(lh_pack_bf(o[0][i][0] * f, o[0][i][1] * f), lh_pack_bf(o[0][i][2] * f, o[0][i][3] * f));
        } else {
#pragma unroll
            for (int r = 0; r < 4; r++) if (c + r < a.vdim) out[c + r] = lh_f2bf(o[0][i][r] * f);
        }
    }
}

typedef __attribute__((address_space(1))) const void gvoid;
typedef __attribute__((address_space(3))) void lvoid;

// 64 packed rows, 16 per wave; steps of 32 * NB keys through two LDS buffers.  A key row of the buffer is MAPS * DQ / 8 chunks
// of 16 bytes, chunk c at place c ^ (key & 7) (see linear_mfma_kernel for why and how).  With more than one split a
// workgroup takes its share of the key steps and leaves partial records.
template <int DQ, int DV, int MAPS, int NB>
__global__ __launch_bounds__(256, MAPS * DV <= 256 ? 2 : 1) void attention_tile_kernel(const AttentionArgs a) {
    constexpr int KC = MAPS * DQ / 8, KCH = 32 * NB * KC, VB = DV * 4, VCH = NB * VB;    // chunks per key row; per step: keys, values
    constexpr uint32_t kSwizzle = KC >= 8 ? 7 : KC - 1;
    __shared__ uint4 sm[2][KCH + VCH];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const uint32_t R = a.heads / a.kv_heads, packed = a.rows * R, tiles = (packed + 63) / 64;
    const uint32_t split = blockIdx.x % a.splits, gt = blockIdx.x / a.splits;
    const uint32_t g = gt % a.kv_heads, tile = tiles - 1 - gt / a.kv_heads;              // the long tiles first
    const uint32_t start = *a.position;
    const uint32_t row0 = tile * 64, row_last = min(row0 + 64, packed) - 1;
    const uint32_t last_key = min(start + row_last / R, a.capacity - 1), last_block = last_key / 32, nstep = last_block / NB + 1;
    const uint32_t per = (nstep + a.splits - 1) / a.splits, s0 = min(split * per, nstep), s1 = min(s0 + per, nstep);
    const uint32_t wrow = row0 + wave * 16, row = wrow + (lane & 15);

    lh_bf16x8 qf[MAPS][DQ / 32];
    load_queries<DQ, MAPS>(qf, a, g, row, lane);
    const uint32_t limit = min(start + row / R, last_key), first_limit = start + wrow / R, wave_last = min(start + (wrow + 15) / R, last_key);
    lh_f32x4 o[MAPS][DV / 16];
    RowState st[MAPS];
#pragma unroll
    for (int mp = 0; mp < MAPS; mp++) {
        st[mp] = RowState{-INFINITY, 0.0f};
#pragma unroll
        for (int d = 0; d < DV / 16; d++) o[mp][d] = (lh_f32x4){0.f, 0.f, 0.f, 0.f};
    }

    const uint16_t* K = static_cast<const uint16_t*>(a.keys) + (size_t)g * MAPS * DQ;
    const uint16_t* V = static_cast<const uint16_t*>(a.values) + (size_t)g * DV * 32;
    const size_t krow = (size_t)a.kv_heads * MAPS * DQ, vblock = (size_t)a.kv_heads * DV * 32;
    auto load_step = [&](int buf, uint32_t s) {
#pragma unroll
        for (int i = 0; i < (KCH + 255) / 256; i++) {
            if (KCH % 256 != 0 && i * 256 + wave * 64 >= KCH) break;                     // whole waves (KCH is a multiple of 64)
            const uint32_t c = i * 256 + tid, key = c / KC, ch = (c % KC) ^ (key & kSwizzle);
            const uint32_t p = min(s * (32 * NB) + key, last_key);                        // keys past the last are masked
            __builtin_amdgcn_global_load_lds((gvoid*)(K + p * krow + ch * 8), (lvoid*)&sm[buf][i * 256 + wave * 64], 16, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < (VCH + 255) / 256; i++) {
            if (VCH % 256 != 0 && i * 256 + wave * 64 >= VCH) break;
            const uint32_t c = i * 256 + tid;
            __builtin_amdgcn_global_load_lds((gvoid*)(V + min(s * NB + c / VB, last_block) * vblock + (c % VB) * 8), (lvoid*)&sm[buf][KCH + i * 256 + wave * 64], 16, 0, 0);
        }
    };
    const float scale2 = a.scale * kLog2e;
    if (s0 < s1) load_step(s0 & 1, s0);
    for (uint32_t s = s0; s < s1; s++) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
        if (s + 1 < s1) load_step((s + 1) & 1, s + 1);
        const uint32_t first = s * (32 * NB);
        if (first > wave_last) continue;                                                  // nothing here is visible to this wave
        const uint4* ks = sm[s & 1];
        const uint4* vs = ks + KCH;
        const bool bound = first + 32 * NB - 1 > first_limit;
#pragma unroll
        for (int mp = 0; mp < MAPS; mp++) {                                               // (a map at a time: the registers of two halve the waves)
            lh_bf16x8 w[NB][3];
            lh_f32x4 sc[2 * NB];
#pragma unroll
            for (int t = 0; t < 2 * NB; t++) {
                sc[t] = (lh_f32x4){0.f, 0.f, 0.f, 0.f};
                const uint32_t key = t * 16 + (lane & 15);
#pragma unroll
                for (int c = 0; c < DQ / 32; c++) {
                    const uint32_t ch = mp * (DQ / 8) + c * 4 + (lane >> 4);
                    sc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(lh_bf16x8, ks[key * KC + (ch ^ (key & kSwizzle))]), qf[mp][c], sc[t], 0, 0, 0);
                }
            }
            const float alpha = softmax_step<NB>(sc, st[mp], scale2, first, limit, bound, lane, w);
            if (__ballot(alpha != 1.0f)) {
#pragma unroll
                for (int d = 0; d < DV / 16; d++)
#pragma unroll
                    for (int r = 0; r < 4; r++) o[mp][d][r] *= alpha;
            }
#pragma unroll
            for (int b = 0; b < NB; b++)
#pragma unroll
                for (int d = 0; d < DV / 16; d++) {
                    const lh_bf16x8 vf = __builtin_bit_cast(lh_bf16x8, vs[b * VB + (d * 16 + (lane & 15)) * 4 + (lane >> 4)]);
#pragma unroll
                    for (int z = 2; z >= 0; z--) o[mp][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, w[b][z], o[mp][d], 0, 0, 0);
                }
        }
    }
    float l[MAPS];
#pragma unroll
    for (int mp = 0; mp < MAPS; mp++) l[mp] = lh_column_sum(st[mp].l);
    if (a.splits == 1) { finish_row<DV, MAPS>(a, o, l, g, row, lane); return; }
    if (row >= packed) return;
    constexpr uint32_t kRow = DV + 4;
#pragma unroll
    for (int mp = 0; mp < MAPS; mp++) {
        float* r = a.partial + ((((size_t)(wrow >> 4) * a.kv_heads + g) * a.splits + split) * MAPS + mp) * 16 * kRow + (lane & 15) * kRow;
#pragma unroll
        for (int d = 0; d < DV / 16; d++) *reinterpret_cast<float4*>(r + d * 16 + (lane >> 4) * 4) = make_float4(o[mp][d][0], o[mp][d][1], o[mp][d][2], o[mp][d][3]);
        if (lane < 16) { r[DV] = st[mp].m; r[DV + 1] = l[mp]; }
    }
}

// grid: row tiles x kv heads x splits.  The blocks of the visible range are dealt out in contiguous runs to the 4 * splits
// waves of a (tile, kv head); where two blocks' operands fit the registers a wave loads one block ahead.
template <int DQ, int DV, int MAPS>
__global__ __launch_bounds__(256) void attention_split_kernel(const AttentionArgs a) {
    extern __shared__ __align__(16) float merge[];                          // [4 waves][MAPS][16 rows][DV + 4]: values, maximum, sum
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const uint32_t split = blockIdx.x % a.splits, g = (blockIdx.x / a.splits) % a.kv_heads, tile = blockIdx.x / (a.splits * a.kv_heads);
    const uint32_t R = a.heads / a.kv_heads, packed = a.rows * R, start = *a.position;
    const uint32_t row0 = tile * 16, row_last = min(row0 + 16, packed) - 1, row = row0 + (lane & 15);
    const uint32_t last_key = min(start + row_last / R, a.capacity - 1), nb = last_key / 32 + 1;
    const uint32_t limit = min(start + row / R, last_key), first_limit = start + row0 / R;
    const uint32_t per = (nb + 4 * a.splits - 1) / (4 * a.splits), w = split * 4 + wave;
    const uint32_t b0 = min(w * per, nb), b1 = min(b0 + per, nb);

    lh_bf16x8 qf[MAPS][DQ / 32];
    load_queries<DQ, MAPS>(qf, a, g, row, lane);
    lh_f32x4 o[MAPS][DV / 16];
    RowState st[MAPS];
#pragma unroll
    for (int mp = 0; mp < MAPS; mp++) {
        st[mp] = RowState{-INFINITY, 0.0f};
#pragma unroll
        for (int d = 0; d < DV / 16; d++) o[mp][d] = (lh_f32x4){0.f, 0.f, 0.f, 0.f};
    }
    const uint16_t* K = static_cast<const uint16_t*>(a.keys) + (size_t)g * MAPS * DQ + (lane >> 4) * 8;
    const uint16_t* V = static_cast<const uint16_t*>(a.values) + (size_t)g * DV * 32;
    const size_t krow = (size_t)a.kv_heads * MAPS * DQ, vblock = (size_t)a.kv_heads * DV * 32;
    struct Block { u32x4 k[2][MAPS][DQ / 32], v[DV / 16]; };
    auto issue = [&](Block& f, uint32_t b) {
#pragma unroll
        for (int t = 0; t < 2; t++) {
            const uint32_t p = min(b * 32 + t * 16 + (lane & 15), last_key);
#pragma unroll
            for (int mp = 0; mp < MAPS; mp++)
#pragma unroll
                for (int c = 0; c < DQ / 32; c++) f.k[t][mp][c] = *reinterpret_cast<const u32x4*>(K + p * krow + mp * DQ + c * 32);
        }
#pragma unroll
        for (int d = 0; d < DV / 16; d++) f.v[d] = *reinterpret_cast<const u32x4*>(V + b * vblock + ((d * 16 + (lane & 15)) * 4 + (lane >> 4)) * 8);
    };
    const float scale2 = a.scale * kLog2e;
    auto consume = [&](const Block& f, uint32_t b) {
        const bool bound = b * 32 + 31 > first_limit;
        lh_bf16x8 w[MAPS][1][3];
#pragma unroll
        for (int mp = 0; mp < MAPS; mp++) {
            lh_f32x4 s[2];
#pragma unroll
            for (int t = 0; t < 2; t++) {
                s[t] = (lh_f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int c = 0; c < DQ / 32; c++) s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(lh_bf16x8, f.k[t][mp][c]), qf[mp][c], s[t], 0, 0, 0);
            }
            const float alpha = softmax_step<1>(s, st[mp], scale2, b * 32, limit, bound, lane, w[mp]);
            if (__ballot(alpha != 1.0f)) {
#pragma unroll
                for (int d = 0; d < DV / 16; d++)
#pragma unroll
                    for (int r = 0; r < 4; r++) o[mp][d][r] *= alpha;
            }
        }
#pragma unroll
        for (int d = 0; d < DV / 16; d++)
#pragma unroll
            for (int mp = 0; mp < MAPS; mp++) {
#pragma unroll
                for (int z = 2; z >= 0; z--)
                    o[mp][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(lh_bf16x8, f.v[d]), w[mp][0][z], o[mp][d], 0, 0, 0);
            }
    };
    if constexpr (sizeof(Block) > 256) {                      // two blocks would not fit the registers
        for (uint32_t b = b0; b < b1; b++) {
            Block x;
            issue(x, b);
            consume(x, b);
        }
    } else if (b0 < b1) {
        Block x, y;
        issue(x, b0);
        for (uint32_t b = b0; b < b1; b += 2) {
            issue(y, min(b + 1, b1 - 1));
            consume(x, b);
            if (b + 1 < b1) {
                issue(x, min(b + 2, b1 - 1));
                consume(y, b + 1);
            }
        }
    }
    constexpr uint32_t kRow = DV + 4;
#pragma unroll
    for (int mp = 0; mp < MAPS; mp++) {
        const float l = lh_column_sum(st[mp].l);
        float* d0 = merge + ((wave * MAPS + mp) * 16 + (lane & 15)) * kRow;
        if (lane < 16) { d0[DV] = st[mp].m; d0[DV + 1] = l; }
#pragma unroll
        for (int d = 0; d < DV / 16; d++) *reinterpret_cast<float4*>(d0 + d * 16 + (lane >> 4) * 4) = make_float4(o[mp][d][0], o[mp][d][1], o[mp][d][2], o[mp][d][3]);
    }
    __syncthreads();
    float* rec = a.partial + (size_t)((tile * a.kv_heads + g) * a.splits + split) * MAPS * 16 * kRow;
    const uint32_t used = row_last - row0 + 1;
    for (uint32_t i = tid; i < (uint32_t)MAPS * used * DV; i += 256) {
        const uint32_t mp = i / (used * DV), rr = (i / DV) % used, d = i % DV;
        float m = -INFINITY, acc = 0.0f, l = 0.0f;
#pragma unroll
        for (int wv = 0; wv < 4; wv++) m = fmaxf(m, merge[((wv * MAPS + mp) * 16 + rr) * kRow + DV]);
        const float base = m == -INFINITY ? 0.0f : m;
#pragma unroll
        for (int wv = 0; wv < 4; wv++) {
            const float* s = merge + ((wv * MAPS + mp) * 16 + rr) * kRow;
            const float f = __builtin_amdgcn_exp2f(s[DV] - base);
            l += f * s[DV + 1];
            acc += f * s[d];
        }
        float* r = rec + (mp * 16 + rr) * kRow;
        r[d] = acc;
        if (d == 0) { r[DV] = m; r[DV + 1] = l; }
    }
}

// One workgroup per (query row, head): merges the splits of every map, combines the maps, norms and stores.  Groups of dv / 4
// threads take the splits in turn, four values a thread, several loads on their way; the groups are added through LDS.
constexpr uint32_t kMergeThreads = 512;
template <int MAPS>
__global__ __launch_bounds__(kMergeThreads) void attention_merge_kernel(const AttentionArgs a) {
    __shared__ float factor[MAPS][512], total[MAPS], scratch[kMergeThreads / 64];
    __shared__ float4 sums[MAPS][kMergeThreads];
    const uint32_t t = blockIdx.x / a.heads, h = blockIdx.x % a.heads, R = a.heads / a.kv_heads, g = h / R, row = t * R + h % R;
    const uint32_t kRow = a.dv + 4, rr = row & 15;
    const size_t stride = (size_t)MAPS * 16 * kRow;
    const float* rec = a.partial + (size_t)(((row >> 4) * a.kv_heads + g) * a.splits) * stride + rr * kRow;
    const uint32_t wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    if (wave < MAPS) {                                        // splits <= 512
        const float* r = rec + wave * 16 * kRow + a.dv;
        float m = -INFINITY, l = 0.0f, mine[8], ml[8];
#pragma unroll
        for (uint32_t i = 0; i < 8; i++) {
            const uint32_t s = i * 64 + lane;
            mine[i] = -INFINITY; ml[i] = 0.0f;
            if (i * 64 >= a.splits) break;
            if (s < a.splits) { const float2 x = *reinterpret_cast<const float2*>(r + s * stride); mine[i] = x.x; ml[i] = x.y; }
            m = fmaxf(m, mine[i]);
        }
        m = lh_group_max(m, 64);
#pragma unroll
        for (uint32_t i = 0; i < 8; i++) {
            if (i * 64 >= a.splits) break;
            const float f = __builtin_amdgcn_exp2f(mine[i] - m);
            if (i * 64 + lane < a.splits) factor[wave][i * 64 + lane] = f;
            l += f * ml[i];
        }
        l = lh_group_sum(l, 64);
        if (lane == 0) total[wave] = 1.0f / l;
    }
    __syncthreads();
    const uint32_t quads = a.dv / 4, groups = kMergeThreads / quads, grp = threadIdx.x / quads, q = threadIdx.x % quads;   // quads <= 64
    float4 acc[MAPS];
#pragma unroll
    for (int mp = 0; mp < MAPS; mp++) acc[mp] = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 4
    for (uint32_t s = grp; s < a.splits; s += groups)
#pragma unroll
        for (int mp = 0; mp < MAPS; mp++) {
            const float4 x = *reinterpret_cast<const float4*>(rec + s * stride + mp * 16 * kRow + q * 4);
            const float f = factor[mp][s];
            acc[mp].x += f * x.x; acc[mp].y += f * x.y; acc[mp].z += f * x.z; acc[mp].w += f * x.w;
        }
#pragma unroll
    for (int mp = 0; mp < MAPS; mp++) sums[mp][threadIdx.x] = acc[mp];
    __syncthreads();
    float v = 0.0f;
    const uint32_t d = threadIdx.x;                           // dv <= 256
    if (d < a.vdim) {
        float s[MAPS] = {};
        for (uint32_t i = 0; i < groups; i++)
#pragma unroll
            for (int mp = 0; mp < MAPS; mp++) s[mp] += reinterpret_cast<const float*>(&sums[mp][i * quads])[d];
        v = s[0] * total[0];
        if constexpr (MAPS == 2) v -= a.lambda * (s[MAPS - 1] * total[MAPS - 1]);
    }
    float f = 1.0f;
    if constexpr (MAPS == 2) f = rsqrtf(lh_block_sum(v * v, scratch) / (float)a.vdim + a.eps) * a.out_scale;
    if (d < a.vdim) static_cast<uint16_t*>(a.out)[((size_t)t * a.heads + h) * a.vdim + d] = lh_f2bf(v * f);
}

// One workgroup per (query row, head), 256 keys at a time; f32 arithmetic throughout.
template <typename T>
__global__ __launch_bounds__(256) void attention_plain_kernel(const AttentionArgs a) {
    extern __shared__ float dyn[];                            // the query's maps * dim values
    __shared__ float p[2][256], scratch[4];
    const uint32_t t = blockIdx.x / a.heads, h = blockIdx.x % a.heads, g = h / (a.heads / a.kv_heads), tid = threadIdx.x;
    const uint32_t start = *a.position, last = min(start + t, a.capacity - 1);
    const T* q = static_cast<const T*>(a.q) + ((size_t)t * a.heads + h) * a.maps * a.dq;
    for (uint32_t i = tid; i < a.maps * a.dim; i += 256) dyn[i] = lh_ld(q, (size_t)(i / a.dim) * a.dq + i % a.dim);
    __syncthreads();
    float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.0f, 0.0f}, acc[2][4] = {};
    for (uint32_t k0 = 0; k0 <= last; k0 += 256) {
        const uint32_t n = min(256u, last + 1 - k0);
        for (uint32_t mp = 0; mp < a.maps; mp++) {
            float s = -INFINITY;
            if (tid < n) {
                const T* k = static_cast<const T*>(a.keys) + (((size_t)(k0 + tid) * a.kv_heads + g) * a.maps + mp) * a.dq;
                float dot = 0.0f;
                for (uint32_t i = 0; i < a.dim; i++) dot = __builtin_fmaf(dyn[mp * a.dim + i], lh_ld(k, i), dot);
                s = dot * a.scale;
            }
            float mx = lh_group_max(s, 64);
            if ((tid & 63) == 0) scratch[tid >> 6] = mx;
            __syncthreads();
            mx = fmaxf(fmaxf(scratch[0], scratch[1]), fmaxf(scratch[2], scratch[3]));
            __syncthreads();
            const float nm = fmaxf(m[mp], mx), alpha = expf(m[mp] - nm), w = tid < n ? expf(s - nm) : 0.0f;
            p[mp][tid] = w;
            const float sum = lh_block_sum(w, scratch);
            l[mp] = l[mp] * alpha + sum;
            m[mp] = nm;
#pragma unroll
            for (int i = 0; i < 4; i++) acc[mp][i] *= alpha;
        }
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const uint32_t d = tid + i * 256;
            if (d >= a.vdim) break;
            for (uint32_t j0 = 0; j0 < n; j0 += 32) {          // k0 is a multiple of 32
                const T* v = static_cast<const T*>(a.values) + ((size_t)((k0 + j0) >> 5) * a.kv_heads * a.dv + (size_t)g * a.dv + d) * 32;
                for (uint32_t j = 0; j < min(32u, n - j0); j++) {
                    const float x = lh_ld(v, lh_block_slot(j));
                    acc[0][i] = __builtin_fmaf(p[0][j0 + j], x, acc[0][i]);
                    if (a.maps == 2) acc[1][i] = __builtin_fmaf(p[1][j0 + j], x, acc[1][i]);
                }
            }
        }
        __syncthreads();
    }
    float v[4], ss = 0.0f;
#pragma unroll
    for (int i = 0; i < 4; i++) {
        v[i] = acc[0][i] / l[0];
        if (a.maps == 2) v[i] -= a.lambda * (acc[1][i] / l[1]);
        if (tid + i * 256 < a.vdim) ss += v[i] * v[i];
    }
    float f = 1.0f;
    if (a.maps == 2) f = rsqrtf(lh_block_sum(ss, scratch) / (float)a.vdim + a.eps) * a.out_scale;
#pragma unroll
    for (int i = 0; i < 4; i++)
        if (tid + i * 256 < a.vdim) lh_st(static_cast<T*>(a.out), ((size_t)t * a.heads + h) * a.vdim + tid + i * 256, v[i] * f);
}

constexpr uint32_t kMaxSplits = 512;

template <int DQ, int DV, int MAPS>
int launch_mfma(lh_context* ctx, AttentionArgs& a, uint32_t max_position, const char* op, uint32_t& launches) {
    const uint32_t R = a.heads / a.kv_heads;
    const uint64_t packed = (uint64_t)a.rows * R, tiles16 = (packed + 15) / 16, cus = ctx->cu_count;
    const uint32_t max_blocks = (uint32_t)std::min<uint64_t>((uint64_t)max_position + a.rows, a.capacity) / 32 + 1;
    const size_t rec = (size_t)tiles16 * a.kv_heads * MAPS * 16 * (DV + 4) * 4;
    const uint32_t room = (uint32_t)std::min<size_t>(ctx->workspace_bytes / rec, kMaxSplits);
    auto merge = [&]() {
        hipLaunchKernelGGL((attention_merge_kernel<MAPS>), dim3(a.rows * a.heads), dim3(kMergeThreads), 0, ctx->stream, a);
        launches++;
        return lh_check_launch(op);
    };
    a.partial = (float*)ctx->workspace;
    launches = 1;
    if (packed > 64) {
        constexpr int NB = MAPS * DQ + DV <= 256 ? 2 : 1;
        const uint64_t groups = (packed + 63) / 64 * a.kv_heads;
        // a share of eight key steps at least, and no more workgroups than two per CU
        a.splits = (uint32_t)std::max<uint64_t>(1, std::min<uint64_t>({2 * cus / groups, max_blocks / (8 * NB), room}));
        LH_REQUIRE(groups * a.splits < 0x7FFFFFFFull, "%s: %u rows", op, a.rows);
        hipLaunchKernelGGL((attention_tile_kernel<DQ, DV, MAPS, NB>), dim3((uint32_t)(groups * a.splits)), dim3(256), 0, ctx->stream, a);
        const int r = lh_check_launch(op);
        return r != LH_OK || a.splits == 1 ? r : merge();
    }
    // one block per wave at least, no more workgroups than one per CU
    const uint64_t groups = tiles16 * a.kv_heads;
    LH_REQUIRE(room >= 1, "%s: %u heads of %u values exceed the workspace", op, a.heads, a.vdim);
    a.splits = (uint32_t)std::max<uint64_t>(1, std::min<uint64_t>({max_blocks / 4, (cus + groups - 1) / groups, room}));
    constexpr size_t lds = (size_t)4 * MAPS * 16 * (DV + 4) * 4;
    if (lds > 64 * 1024) {
        const int r = lh_raise_dynamic_lds(ctx, (const void*)attention_split_kernel<DQ, DV, MAPS>, lds, op);
        if (r != LH_OK) return r;
    }
    hipLaunchKernelGGL((attention_split_kernel<DQ, DV, MAPS>), dim3((uint32_t)(groups * a.splits)), dim3(256), lds, ctx->stream, a);
    const int r = lh_check_launch(op);
    return r != LH_OK ? r : merge();
}

template <int DQ, int DV>
int launch_maps(lh_context* ctx, AttentionArgs& a, uint32_t mp, const char* op, uint32_t& n) {
    return a.maps == 2 ? launch_mfma<DQ, DV, 2>(ctx, a, mp, op, n) : launch_mfma<DQ, DV, 1>(ctx, a, mp, op, n);
}
template <int DQ>
int launch_dv(lh_context* ctx, AttentionArgs& a, uint32_t mp, const char* op, uint32_t& n) {
    switch (a.dv) {
        case 32: return launch_maps<DQ, 32>(ctx, a, mp, op, n);
        case 64: return launch_maps<DQ, 64>(ctx, a, mp, op, n);
        case 128: return launch_maps<DQ, 128>(ctx, a, mp, op, n);
        default: return launch_maps<DQ, 256>(ctx, a, mp, op, n);
    }
}

}  // namespace

extern "C" {

uint32_t lh_attention_padded_dim(uint32_t dim) { return dim <= 32 ? 32u : dim <= 64 ? 64u : (dim + 127) / 128 * 128; }
uint32_t lh_attention_padded_vdim(uint32_t vdim) { return vdim <= 32 ? 32u : vdim <= 64 ? 64u : vdim <= 128 ? 128u : (vdim + 255) / 256 * 256; }

int lh_attention_rows_into(lh_batch* batch, const lh_buffer* q, const lh_buffer* keys, const lh_buffer* values, lh_buffer* output, int dtype,
                           const lh_buffer* position, uint32_t max_position, uint32_t rows, uint32_t heads, uint32_t kv_heads, uint32_t maps, uint32_t dim,
                           uint32_t vdim, uint32_t capacity, float scale, float lambda, float out_scale, float eps) {
    const char* op = "attention_rows";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(dtype == LH_F32 || dtype == LH_BF16, "%s: dtype %d", op, dtype);
    LH_REQUIRE(maps == 1 || maps == 2, "%s: %u maps", op, maps);
    LH_REQUIRE(kv_heads > 0 && heads > 0 && heads % kv_heads == 0, "%s: heads %u is not a multiple of kv_heads %u", op, heads, kv_heads);
    LH_REQUIRE(dim > 0 && dim <= 4096 && vdim > 0 && vdim <= 1024, "%s: dim %u, vdim %u", op, dim, vdim);
    if (rows == 0) return LH_OK;
    LH_REQUIRE(capacity > 0 && capacity % 32 == 0 && (uint64_t)max_position + rows <= capacity, "%s: positions up to %llu in caches of %u", op,
               (unsigned long long)max_position + rows, capacity);
    AttentionArgs a{};
    a.dq = lh_attention_padded_dim(dim);
    a.dv = lh_attention_padded_vdim(vdim);
    const size_t es = dtype == LH_F32 ? 4 : 2;
    LH_NEED(q, (size_t)rows * heads * maps * a.dq * es, op, "q");
    LH_NEED(keys, (size_t)capacity * kv_heads * maps * a.dq * es, op, "keys");
    LH_NEED(values, (size_t)capacity * kv_heads * a.dv * es, op, "values");
    LH_NEED(output, (size_t)rows * heads * vdim * es, op, "output");
    LH_NEED(position, 4, op, "position");
    a.q = q->ptr; a.keys = keys->ptr; a.values = values->ptr; a.out = output->ptr; a.position = (const uint32_t*)position->ptr;
    a.rows = rows; a.heads = heads; a.kv_heads = kv_heads; a.maps = maps; a.dim = dim; a.vdim = vdim; a.capacity = capacity;
    a.scale = scale; a.lambda = lambda; a.out_scale = out_scale; a.eps = eps;
    const bool aligned = (((uintptr_t)a.q | (uintptr_t)a.keys | (uintptr_t)a.values | (uintptr_t)a.out) & 15) == 0;
    uint32_t launches = 0;
    int r;
    if (dtype == LH_BF16 && aligned && a.dq <= 128 && a.dv <= 256) {
        if (a.dq == 32) r = launch_dv<32>(batch->ctx, a, max_position, op, launches);
        else if (a.dq == 64) r = launch_dv<64>(batch->ctx, a, max_position, op, launches);
        else r = launch_dv<128>(batch->ctx, a, max_position, op, launches);
    } else {
        LH_REQUIRE((uint64_t)rows * heads < 0x7FFFFFFFull, "%s: %u rows", op, rows);
        const size_t lds = (size_t)maps * dim * 4;
        if (dtype == LH_F32) hipLaunchKernelGGL((attention_plain_kernel<float>), dim3(rows * heads), dim3(256), lds, batch->ctx->stream, a);
        else hipLaunchKernelGGL((attention_plain_kernel<uint16_t>), dim3(rows * heads), dim3(256), lds, batch->ctx->stream, a);
        launches = 1;
        r = lh_check_launch(op);
    }
    batch->dispatch_count += launches;
    return r;
}

}  // extern "C"
