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
#include "softmax_attention.hpp"

namespace {

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

// A finished row: o[i][r] holds value 16 i + 4g + r of packed row (lane & 15), for every map unnormalised with sum l.
template <int DV, int MAPS>
__device__ __forceinline__ void finish_row(const AttentionArgs& a, lh_f32x4 (&o)[MAPS][DV / 16], const float (&l)[MAPS], float m0, uint32_t g, uint32_t row, uint32_t lane) {   // m0: the first map's maximum
    const uint32_t R = a.heads / a.kv_heads, t = row / R, h = g * R + (row - t * R);
    float inv[MAPS];
#pragma unroll
    for (int mp = 0; mp < MAPS; mp++) inv[mp] = 1.0f / l[mp];
    if (MAPS == 1 && a.sink) inv[0] = 1.0f / (l[0] + __builtin_amdgcn_exp2f(a.sink[h] * kLog2e - m0));
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
    if (MAPS == 1 && a.gate) f = lh_sigmoid(a.gate[(size_t)t * a.heads + h]);
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
    if (a.splits == 1) { finish_row<DV, MAPS>(a, o, l, st[0].m, g, row, lane); return; }
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

template <int DQ, int DV, int MAPS>
int launch_mfma(lh_context* ctx, AttentionArgs& a, uint32_t max_position, const char* op, uint32_t& launches) {
    const uint32_t R = a.heads / a.kv_heads;
    const uint64_t packed = (uint64_t)a.rows * R, tiles16 = (packed + 15) / 16, cus = ctx->cu_count;
    const uint32_t max_blocks = (uint32_t)std::min<uint64_t>((uint64_t)max_position + a.rows, a.capacity) / 32 + 1;
    const size_t rec = (size_t)tiles16 * a.kv_heads * MAPS * 16 * (DV + 4) * 4;
    const uint32_t room = (uint32_t)std::min<size_t>(ctx->workspace_bytes / rec, kMaxSplits);
    auto merge = [&]() {
        launches++;
        return launch_merge<MAPS>(ctx, a, op);
    };
    a.partial = (float*)ctx->workspace;
    launches = 1;
    if (packed > 64) {
        constexpr int NB = MAPS * DQ + DV <= (MAPS == 1 ? 320 : 256) ? 2 : 1;
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
    if constexpr (DQ <= 128) if (a.maps == 2) return launch_mfma<DQ, DV, 2>(ctx, a, mp, op, n);
    return launch_mfma<DQ, DV, 1>(ctx, a, mp, op, n);
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

uint32_t lh_attention_padded_dim(uint32_t dim) { return dim <= 32 ? 32u : dim <= 64 ? 64u : dim > 128 && dim <= 192 ? 192u : (dim + 127) / 128 * 128; }
uint32_t lh_attention_padded_vdim(uint32_t vdim) { return vdim <= 32 ? 32u : vdim <= 64 ? 64u : vdim <= 128 ? 128u : (vdim + 255) / 256 * 256; }

int lh_attention_rows_into(lh_batch* batch, const lh_buffer* q, const lh_buffer* keys, const lh_buffer* values, lh_buffer* output, int dtype,
                           const lh_buffer* position, uint32_t max_position, uint32_t rows, uint32_t heads, uint32_t kv_heads, uint32_t maps, uint32_t dim,
                           uint32_t vdim, uint32_t capacity, float scale, float lambda, float out_scale, float eps,
                           const lh_buffer* sink, const lh_buffer* gate) {
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
    LH_REQUIRE(maps == 1 || (!sink && !gate), "%s: a sink or a gate with two maps", op);
    if (sink) { LH_NEED(sink, (size_t)heads * 4, op, "sink"); a.sink = (const float*)sink->ptr; }
    if (gate) { LH_NEED(gate, (size_t)rows * heads * 4, op, "gate"); a.gate = (const float*)gate->ptr; }
    const bool aligned = (((uintptr_t)a.q | (uintptr_t)a.keys | (uintptr_t)a.values | (uintptr_t)a.out) & 15) == 0;
    uint32_t launches = 0;
    int r;
    if (dtype == LH_BF16 && aligned && a.dq <= (maps == 2 ? 128u : 256u) && a.dv <= 256) {
        if (a.dq == 32) r = launch_dv<32>(batch->ctx, a, max_position, op, launches);
        else if (a.dq == 64) r = launch_dv<64>(batch->ctx, a, max_position, op, launches);
        else if (a.dq == 128) r = launch_dv<128>(batch->ctx, a, max_position, op, launches);
        else if (a.dq == 192) r = launch_dv<192>(batch->ctx, a, max_position, op, launches);
        else r = launch_dv<256>(batch->ctx, a, max_position, op, launches);
    } else {
        LH_REQUIRE((uint64_t)rows * heads < 0x7FFFFFFFull, "%s: %u rows", op, rows);
        const size_t lds = (size_t)maps * dim * 4;
        if (dtype == LH_F32) hipLaunchKernelGGL((attention_plain_kernel<float, float>), dim3(rows * heads), dim3(256), lds, batch->ctx->stream, a);
        else hipLaunchKernelGGL((attention_plain_kernel<uint16_t, uint16_t>), dim3(rows * heads), dim3(256), lds, batch->ctx->stream, a);
        launches = 1;
        r = lh_check_launch(op);
    }
    batch->dispatch_count += launches;
    return r;
}

}  // extern "C"
