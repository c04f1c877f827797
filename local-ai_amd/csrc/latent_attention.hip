// Latent attention: one cached row per position serves all heads, [latent (DV) | rotated key part (64)], as key in full and as
// value with its latent columns.  Two forms of the same attention:
//   few rows    the key projection is applied to the queries and the value projection to the output, so that the cache is read
//               as it is (latent_split_kernel, whose 16 packed rows are heads of query rows)
//   many rows   keys and values of every head are made from the cache first (lh_latent_expand_into), and the kernels of
//               softmax_attention.hip run over them
#include "float_linear.hpp"
#include "softmax_attention.hpp"
#include <cstring>

namespace {

constexpr uint32_t kRotPad = 64;
uint32_t padded_rank(uint32_t rank) { return rank <= 64 ? 64u : rank <= 128 ? 128u : (rank + 255) / 256 * 256; }
uint32_t padded_rot(uint32_t rot) { return rot <= kRotPad ? kRotPad : (rot + 63) / 64 * 64; }

// ---- cache rows and rotated queries ----------------------------------------------------------------------------------------
struct PrepareArgs {
    const float *q_rot, *down, *norm_weight, *frequencies;
    const uint32_t* position;
    void *q, *cache;
    uint32_t heads, rank, dv, rot, row, q_ld, rot_column, clear_column, capacity;
    float eps;
};

// Value i of a rotated vector whose pairs (2i, 2i + 1) turn by position * frequency.
__device__ __forceinline__ float rotated(const float* v, uint32_t i, float position, const float* frequencies) {
    float s, c;
    sincosf(position * frequencies[i >> 1], &s, &c);
    const float u = v[i & ~1u], w = v[i | 1u];
    return i & 1 ? w * c + u * s : u * c - w * s;
}

// Row t; piece 0 writes the cache row, the others 1024 columns of the queries each.
template <typename TQ, typename T>
__device__ __forceinline__ void prepare_piece(const PrepareArgs& a, uint32_t t, uint32_t piece, float* scratch) {
    const uint32_t pos = *a.position + t;
    if (piece == 0) {
        if (!a.down || pos >= a.capacity) return;
        const float* d = a.down + (size_t)t * (a.rank + a.rot);
        T* row = static_cast<T*>(a.cache) + (size_t)pos * a.row;
        float s = 0.0f;
        for (uint32_t i = threadIdx.x; i < a.rank; i += 256) s += d[i] * d[i];
        const float r = rsqrtf(lh_block_sum(s, scratch) / (float)a.rank + a.eps);
        for (uint32_t i = threadIdx.x; i < a.row; i += 256) {
            float v = 0.0f;
            if (i < a.rank) v = d[i] * r * a.norm_weight[i];
            else if (i >= a.dv && i < a.dv + a.rot) v = rotated(d + a.rank, i - a.dv, (float)pos, a.frequencies);
            lh_st(row, i, v);
        }
        return;
    }
    const uint32_t width = a.q_ld - a.clear_column, total = a.heads * width;
#pragma unroll
    for (uint32_t j = 0; j < 4; j++) {
        const uint32_t e = (piece - 1) * 1024 + j * 256 + threadIdx.x;
        if (e >= total) return;
        const uint32_t h = e / width, c = a.clear_column + e % width;
        const float v = c >= a.rot_column && c < a.rot_column + a.rot
                            ? rotated(a.q_rot + ((size_t)t * a.heads + h) * a.rot, c - a.rot_column, (float)pos, a.frequencies) : 0.0f;
        lh_st(static_cast<TQ*>(a.q), ((size_t)t * a.heads + h) * a.q_ld + c, v);
    }
}

template <typename TQ, typename T>
__global__ __launch_bounds__(256) void latent_prepare_kernel(const PrepareArgs a) {
    __shared__ float scratch[4];
    prepare_piece<TQ, T>(a, blockIdx.x, blockIdx.y, scratch);
}

// ---- one small product per head --------------------------------------------------------------------------------------------
struct HeadArgs {
    const void* x;             // [rows, heads, K]
    const uint16_t* W;         // [heads, N, K]
    void* out;                 // [rows, heads, ld]
    uint32_t rows, heads, N, K, ld, vec;
};

// Eight values of a row of K at k, zeros past its end.
__device__ __forceinline__ lh_bf16x8 operand8(const uint16_t* row, uint32_t k, uint32_t K, bool vec) {
    u32x4 v = {0u, 0u, 0u, 0u};
    if (vec) { if (k < K) v = *reinterpret_cast<const u32x4*>(row + k); }
    else {
#pragma unroll
        for (uint32_t j = 0; j < 8; j++) if (k + j < K) v[j >> 1] |= (uint32_t)row[k + j] << (16 * (j & 1));
    }
    return __builtin_bit_cast(lh_bf16x8, v);
}

// 16 columns x 16 rows of one head, the four waves take quarters of K.
template <typename TO>
__device__ __forceinline__ void head_tile(const HeadArgs& a, uint32_t h, uint32_t n0, uint32_t m0, lh_f32x4 (&part)[4][64]) {
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const uint32_t steps = (a.K + 31) / 32, per = (steps + 3) / 4, s0 = min(wave * per, steps), s1 = min(s0 + per, steps);
    const uint16_t* w = a.W + ((size_t)h * a.N + min(n0 + (lane & 15), a.N - 1)) * a.K;
    const uint16_t* x = static_cast<const uint16_t*>(a.x) + ((size_t)min(m0 + (lane & 15), a.rows - 1) * a.heads + h) * a.K;
    lh_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (uint32_t s = s0; s < s1; s++) {
        const uint32_t k = s * 32 + (lane >> 4) * 8;
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(operand8(w, k, a.K, a.vec), operand8(x, k, a.K, a.vec), acc, 0, 0, 0);
    }
    part[wave][lane] = acc;
    __syncthreads();
    const uint32_t l = threadIdx.x >> 2, r = threadIdx.x & 3, m = m0 + (l & 15), n = n0 + (l >> 4) * 4 + r;   // thread: one output
    if (m >= a.rows || n >= a.N) return;
    lh_st(static_cast<TO*>(a.out), ((size_t)m * a.heads + h) * a.ld + n, (part[0][l][r] + part[1][l][r]) + (part[2][l][r] + part[3][l][r]));
}

// grid (column tiles, heads, row tiles)
template <typename TO>
__global__ __launch_bounds__(256) void head_linear_mfma_kernel(const HeadArgs a) {
    __shared__ lh_f32x4 part[4][64];
    head_tile<TO>(a, blockIdx.y, blockIdx.x * 16, blockIdx.z * 16, part);
}

// Both steps in front of the attention of few rows: the tiles of the key projection, then the pieces of the preparation.
__global__ __launch_bounds__(256) void latent_queries_kernel(const HeadArgs a, const PrepareArgs p, uint32_t tiles, uint32_t pieces) {
    __shared__ lh_f32x4 part[4][64];
    const uint32_t nt = (a.N + 15) / 16, i = blockIdx.x;
    if (i < tiles) head_tile<float>(a, i / nt % a.heads, i % nt * 16, i / (nt * a.heads) * 16, part);
    else prepare_piece<float, uint16_t>(p, (i - tiles) / pieces, (i - tiles) % pieces, reinterpret_cast<float*>(&part[0][0]));
}

// f32: a wave per output.
__global__ __launch_bounds__(256) void head_linear_plain_kernel(const HeadArgs a) {
    const uint32_t n = blockIdx.x * 4 + (threadIdx.x >> 6), h = blockIdx.y, m = blockIdx.z, lane = threadIdx.x & 63;
    if (n >= a.N) return;
    const uint16_t* w = a.W + ((size_t)h * a.N + n) * a.K;
    const float* x = static_cast<const float*>(a.x) + ((size_t)m * a.heads + h) * a.K;
    float s = 0.0f;
    for (uint32_t k = lane; k < a.K; k += 64) s = __builtin_fmaf(lh_bf2f(w[k]), x[k], s);
    s = lh_group_sum(s, 64);
    if (lane == 0) static_cast<float*>(a.out)[((size_t)m * a.heads + h) * a.ld + n] = s;
}

// ---- keys of every head: the shared rotated part ---------------------------------------------------------------------------
// T: as many values as move together.
template <typename T>
__global__ __launch_bounds__(256) void expand_rotated_kernel(const T* __restrict__ cache, T* __restrict__ keys, uint32_t heads, uint32_t row, uint32_t dv,
                                                            uint32_t dim, uint32_t rot, uint32_t dq) {
    const uint32_t p = blockIdx.x;
    for (uint32_t e = threadIdx.x; e < heads * rot; e += 256) keys[((size_t)p * heads + e / rot) * dq + dim + e % rot] = cache[(size_t)p * row + dv + e % rot];
}

// ---- attention over the cache rows -----------------------------------------------------------------------------------------
typedef __attribute__((address_space(1))) const void gvoid;
typedef __attribute__((address_space(3))) void lvoid;
typedef short s16x4 __attribute__((ext_vector_type(4)));

// Four rows of 16 columns out of LDS, transposed: over a group of 16 lanes, lane l names columns 4 (l & 3) .. + 3 of row l / 4 and
// receives column l of the four rows.
__device__ __forceinline__ s16x4 transposed4(const void* lds) {
    typedef __attribute__((address_space(3))) s16x4 lds_s16x4;
    return __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)lds);
}

// grid: row tiles x splits; packed row r = head r % heads of query row r / heads.  The blocks of 32 positions of the visible range
// are dealt out in contiguous runs to the splits of a row tile.  The four waves share a block in LDS, in tiles of 8 key rows x 8
// chunks of 16 bytes, chunk c of row k at place c ^ k of its row (a load fills one tile, and every address is one of a few per
// lane plus a constant), while the next block is on its way into a second buffer.  A wave takes every fourth 32 columns of the
// scores' sums, which meet in LDS, and a quarter of the value columns, which it reads through the transposing LDS read.  A query
// value enters as the sum of two bf16 terms.
template <int DV>
__global__ __launch_bounds__(256) void latent_split_kernel(const AttentionArgs a) {
    constexpr int DQ = DV + kRotPad, KT = DQ / 64, NC = (DQ / 32 + 3) / 4, ND = DV / 64, kBlock = 4 * KT * 64;
    extern __shared__ __align__(16) uint4 sm[];             // two blocks, then the partial scores [4 waves][2 tiles][64 lanes]
    lh_f32x4* sums = reinterpret_cast<lh_f32x4*>(sm + 2 * kBlock);
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, lc = lane & 15;
    const uint32_t split = blockIdx.x % a.splits, tile = blockIdx.x / a.splits, packed = a.rows * a.heads, start = *a.position;
    const uint32_t row0 = tile * 16, row_last = min(row0 + 16, packed) - 1, row = row0 + lc;
    const uint32_t last_key = min(start + row_last / a.heads, a.capacity - 1), nb = last_key / 32 + 1;
    const uint32_t limit = min(start + row / a.heads, last_key), first_limit = start + row0 / a.heads;
    const uint32_t per = (nb + a.splits - 1) / a.splits, b0 = min(split * per, nb), b1 = min(b0 + per, nb);
    const uint16_t* cache = static_cast<const uint16_t*>(a.keys) + ((lane & 7) ^ (lane >> 3)) * 8;
    auto load_block = [&](uint32_t b) {                       // a wave brings in eight key rows
        const uint16_t* key = cache + (size_t)min(b * 32 + wave * 8 + (lane >> 3), last_key) * DQ;               // keys past the last are masked
        uint4* to = sm + (b & 1) * kBlock + wave * KT * 64;
#pragma unroll
        for (int i = 0; i < KT; i++) __builtin_amdgcn_global_load_lds((gvoid*)(key + i * 64), (lvoid*)(to + i * 64), 16, 0, 0);
    };
    lh_bf16x8 qh[NC], ql[NC];
#pragma unroll
    for (int i = 0; i < NC; i++) {
        const uint32_t c = i * 4 + wave;
        float f[8];
        if (row < packed && c < DQ / 32) lh_ld8(static_cast<const float*>(a.q) + (size_t)row * DQ + c * 32 + g * 8, f);
        else
#pragma unroll
            for (int j = 0; j < 8; j++) f[j] = 0.0f;
        uint32_t h[4], l[4];
#pragma unroll
        for (int j = 0; j < 4; j++) {
            h[j] = lh_pack_bf(f[2 * j], f[2 * j + 1]);
            l[j] = lh_pack_bf(f[2 * j] - __builtin_bit_cast(float, h[j] << 16), f[2 * j + 1] - __builtin_bit_cast(float, h[j] & 0xFFFF0000u));
        }
        qh[i] = __builtin_bit_cast(lh_bf16x8, (u32x4){h[0], h[1], h[2], h[3]});
        ql[i] = __builtin_bit_cast(lh_bf16x8, (u32x4){l[0], l[1], l[2], l[3]});
    }
    if (b0 < b1) load_block(b0);
    lh_f32x4 o[ND];
#pragma unroll
    for (int d = 0; d < ND; d++) o[d] = (lh_f32x4){0.f, 0.f, 0.f, 0.f};
    RowState st{-INFINITY, 0.0f};
    const float scale2 = a.scale * kLog2e;
    // score operand: key lc (+ 16), chunk 4 c + g; value operand: key 4 g + lc / 4 (+ 16), columns 16 d + 4 (lane & 3) ..
    const uint4* kp = sm + (lc >> 3) * (KT * 64) + (lc & 7) * 8;
    const uint32_t vk = g * 4 + (lc >> 2);
    const char* vp = reinterpret_cast<const char*>(sm + (vk >> 3) * (KT * 64) + (vk & 7) * 8) + (lane & 1) * 8;

    for (uint32_t b = b0; b < b1; b++) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        lh_lds_barrier();                                     // the block has arrived, and the one before has been read by all
        if (b + 1 < b1) load_block(b + 1);
        const uint32_t buf = (b & 1) * kBlock;
        lh_f32x4 s[2], low[2];                                // four sums that do not wait for each other
#pragma unroll
        for (int t = 0; t < 2; t++) s[t] = low[t] = (lh_f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < NC; i++) {
            const uint32_t c = i * 4 + wave;
            if (i * 4 + 3 >= DQ / 32 && c >= DQ / 32) break;
#pragma unroll
            for (int t = 0; t < 2; t++) {
                const lh_bf16x8 k = __builtin_bit_cast(lh_bf16x8, kp[buf + t * 2 * KT * 64 + (c >> 1) * 64 + (((c & 1) * 4 + g) ^ (lc & 7))]);
                low[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k, ql[i], low[t], 0, 0, 0);
                s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k, qh[i], s[t], 0, 0, 0);
            }
        }
#pragma unroll
        for (int t = 0; t < 2; t++) sums[(wave * 2 + t) * 64 + lane] = s[t] + low[t];
        lh_lds_barrier();
#pragma unroll
        for (int t = 0; t < 2; t++) s[t] = (sums[t * 64 + lane] + sums[(2 + t) * 64 + lane]) + (sums[(4 + t) * 64 + lane] + sums[(6 + t) * 64 + lane]);
        lh_bf16x8 p[1][3];
        const float alpha = softmax_step<1>(s, st, scale2, b * 32, limit, b * 32 + 31 > first_limit, lane, p);
        if (__ballot(alpha != 1.0f)) {
#pragma unroll
            for (int d = 0; d < ND; d++)
#pragma unroll
                for (int r = 0; r < 4; r++) o[d][r] *= alpha;
        }
        lh_bf16x8 vf[ND];
#pragma unroll
        for (int d = 0; d < ND; d++) {
            const uint32_t ch = 2 * (wave * ND + d) + ((lane & 3) >> 1);
            const char* v0 = vp + (buf + ((ch & 7) ^ (vk & 7)) + (ch >> 3) * 64) * 16;
            struct { s16x4 x, y; } v = {transposed4(v0), transposed4(v0 + 2 * KT * 64 * 16)};
            vf[d] = __builtin_bit_cast(lh_bf16x8, v);
        }
#pragma unroll
        for (int z = 2; z >= 0; z--)
#pragma unroll
            for (int d = 0; d < ND; d++) o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[d], p[0][z], o[d], 0, 0, 0);
    }
    const float l = lh_column_sum(st.l);
    if (row > row_last) return;
    constexpr uint32_t kRow = DV + 4;
    float* rec = a.partial + (size_t)(tile * a.splits + split) * 16 * kRow + lc * kRow;
#pragma unroll
    for (int d = 0; d < ND; d++) *reinterpret_cast<float4*>(rec + (wave * ND + d) * 16 + g * 4) = make_float4(o[d][0], o[d][1], o[d][2], o[d][3]);
    if (tid < 16) { rec[DV] = st.m; rec[DV + 1] = l; }
}

template <int DV>
int launch_split(lh_context* ctx, AttentionArgs& a, uint32_t max_position, const char* op, uint32_t& launches) {
    constexpr size_t lds = 2 * 32 * (DV + kRotPad) * 2 + 4 * 2 * 64 * 16;
    const uint64_t tiles = ((uint64_t)a.rows * a.heads + 15) / 16, want = (uint64_t)ctx->cu_count * (tiles > 2 ? 2 : 1);
    const uint32_t max_blocks = (uint32_t)std::min<uint64_t>((uint64_t)max_position + a.rows, a.capacity) / 32 + 1;
    const size_t rec = (size_t)tiles * 16 * (DV + 4) * 4;
    const uint32_t room = (uint32_t)std::min<size_t>(ctx->workspace_bytes / rec, kMaxSplits);
    LH_REQUIRE(room >= 1, "%s: %u rows of %u heads exceed the workspace", op, a.rows, a.heads);
    a.splits = (uint32_t)std::max<uint64_t>(1, std::min<uint64_t>({max_blocks / 2, (want + tiles - 1) / tiles, room}));
    LH_REQUIRE(tiles * a.splits < 0x7FFFFFFFull && (uint64_t)a.rows * a.heads < 0x7FFFFFFFull, "%s: %u rows", op, a.rows);
    a.partial = (float*)ctx->workspace;
    if (lds > 64 * 1024) {
        const int r = lh_raise_dynamic_lds(ctx, (const void*)latent_split_kernel<DV>, lds, op);
        if (r != LH_OK) return r;
    }
    hipLaunchKernelGGL((latent_split_kernel<DV>), dim3((uint32_t)(tiles * a.splits)), dim3(256), lds, ctx->stream, a);
    int r = lh_check_launch(op);
    if (r != LH_OK) return r;
    launches = 2;
    return launch_merge<1>(ctx, a, op);
}

// Checks and arguments of an attention over cache rows; the output is the caller's.
int latent_args(AttentionArgs& a, const char* op, const lh_buffer* q, const lh_buffer* cache, int dtype, const lh_buffer* position, uint32_t max_position,
                uint32_t rows, uint32_t heads, uint32_t rank, uint32_t rot, uint32_t capacity, float scale, const lh_buffer* sink, const lh_buffer* gate) {
    LH_REQUIRE(dtype == LH_F32 || dtype == LH_BF16, "%s: dtype %d", op, dtype);
    LH_REQUIRE(heads > 0 && rank > 0 && rank <= 1024 && rot > 0 && rot <= 2048, "%s: heads %u, rank %u, rot %u", op, heads, rank, rot);
    LH_REQUIRE(capacity > 0 && capacity % 32 == 0 && (uint64_t)max_position + rows <= capacity, "%s: positions up to %llu in caches of %u", op,
               (unsigned long long)max_position + rows, capacity);
    a = AttentionArgs{};
    a.dv = padded_rank(rank);
    a.dq = lh_latent_row(rank, rot);
    LH_NEED(q, (size_t)rows * heads * a.dq * 4, op, "q");
    LH_NEED(cache, (size_t)capacity * a.dq * (dtype == LH_F32 ? 4 : 2), op, "cache");
    LH_NEED(position, 4, op, "position");
    if (sink) { LH_NEED(sink, (size_t)heads * 4, op, "sink"); a.sink = (const float*)sink->ptr; }
    if (gate) { LH_NEED(gate, (size_t)rows * heads * 4, op, "gate"); a.gate = (const float*)gate->ptr; }
    a.q = q->ptr; a.keys = cache->ptr; a.values = cache->ptr; a.position = (const uint32_t*)position->ptr;
    a.rows = rows; a.heads = heads; a.kv_heads = 1; a.maps = 1; a.dim = a.dq; a.vdim = rank; a.capacity = capacity; a.scale = scale; a.out_scale = 1.0f;
    a.values_in_keys = 1;
    return LH_OK;
}
bool tiled(const AttentionArgs& a, int dtype, uint32_t rot) {
    return dtype == LH_BF16 && (((uintptr_t)a.q | (uintptr_t)a.keys) & 15) == 0 && rot <= kRotPad && a.dv <= 512;
}
int launch_tiled(lh_context* ctx, AttentionArgs& a, uint32_t max_position, const char* op, uint32_t& launches) {
    if (a.dv == 64) return launch_split<64>(ctx, a, max_position, op, launches);
    if (a.dv == 128) return launch_split<128>(ctx, a, max_position, op, launches);
    if (a.dv == 256) return launch_split<256>(ctx, a, max_position, op, launches);
    return launch_split<512>(ctx, a, max_position, op, launches);
}

int prepare_args(PrepareArgs& a, uint32_t& pieces, const char* op, const lh_buffer* q_rot, const lh_buffer* down, const lh_buffer* norm_weight,
                 const lh_buffer* frequencies, const lh_buffer* position, lh_buffer* q, int q_dtype, lh_buffer* cache, int dtype, uint32_t rows, uint32_t heads,
                 uint32_t rank, uint32_t rot, uint32_t q_ld, uint32_t rot_column, uint32_t clear_column, uint32_t capacity, float eps) {
    LH_REQUIRE((dtype == LH_F32 || dtype == LH_BF16) && (q_dtype == LH_F32 || q_dtype == LH_BF16), "%s: dtypes %d, %d", op, q_dtype, dtype);
    LH_REQUIRE(q_dtype == LH_F32 || dtype == LH_BF16, "%s: bf16 queries of an f32 cache", op);
    LH_REQUIRE(heads > 0 && rank > 0 && rot > 0 && rot % 2 == 0, "%s: heads %u, rank %u, rot %u", op, heads, rank, rot);
    LH_REQUIRE(clear_column <= rot_column && (uint64_t)rot_column + rot <= q_ld && (uint64_t)heads * q_ld < 0x7FFFFFFFull, "%s: columns %u and %u of %u", op,
               clear_column, rot_column, q_ld);
    const uint32_t row = lh_latent_row(rank, rot);
    LH_NEED(q_rot, (size_t)rows * heads * rot * 4, op, "q_rot");
    LH_NEED(frequencies, (size_t)(rot / 2) * 4, op, "frequencies");
    LH_NEED(position, 4, op, "position");
    LH_NEED(q, (size_t)rows * heads * q_ld * (q_dtype == LH_F32 ? 4 : 2), op, "q");
    LH_NEED(cache, (size_t)capacity * row * (dtype == LH_F32 ? 4 : 2), op, "cache");
    if (down) {
        LH_NEED(down, (size_t)rows * (rank + rot) * 4, op, "down");
        LH_NEED(norm_weight, (size_t)rank * 4, op, "norm_weight");
    }
    a = PrepareArgs{};
    a.q_rot = (const float*)q_rot->ptr; a.down = down ? (const float*)down->ptr : nullptr; a.norm_weight = down ? (const float*)norm_weight->ptr : nullptr;
    a.frequencies = (const float*)frequencies->ptr; a.position = (const uint32_t*)position->ptr; a.q = q->ptr; a.cache = cache->ptr;
    a.heads = heads; a.rank = rank; a.dv = padded_rank(rank); a.rot = rot; a.row = row; a.q_ld = q_ld; a.rot_column = rot_column; a.clear_column = clear_column;
    a.capacity = capacity; a.eps = eps;
    const uint64_t parts = ((uint64_t)heads * (q_ld - clear_column) + 1023) / 1024;
    LH_REQUIRE(parts < 65535, "%s: %u heads of %u columns", op, heads, q_ld);
    pieces = (uint32_t)parts + 1;
    return LH_OK;
}
int head_args(HeadArgs& a, const char* op, const lh_buffer* input, int dtype, const lh_buffer* weight, lh_buffer* output, int output_dtype, uint32_t rows,
              uint32_t heads, uint32_t n, uint32_t k, uint32_t output_ld) {
    LH_REQUIRE((dtype == LH_F32 && output_dtype == LH_F32) || (dtype == LH_BF16 && (output_dtype == LH_F32 || output_dtype == LH_BF16)), "%s: dtypes %d, %d", op, dtype,
               output_dtype);
    LH_REQUIRE(heads > 0 && heads < 65536 && n > 0 && k > 0 && output_ld >= n, "%s: %u heads of %u x %u into %u columns", op, heads, n, k, output_ld);
    LH_REQUIRE(rows < 65536, "%s: %u rows", op, rows);
    LH_NEED(input, (size_t)rows * heads * k * (dtype == LH_F32 ? 4 : 2), op, "input");
    LH_NEED(weight, (size_t)heads * n * k * 2, op, "weight");
    LH_NEED(output, (size_t)rows * heads * output_ld * (output_dtype == LH_F32 ? 4 : 2), op, "output");
    a = HeadArgs{input->ptr, (const uint16_t*)weight->ptr, output->ptr, rows, heads, n, k, output_ld,
                 k % 8 == 0 && (((uintptr_t)input->ptr | (uintptr_t)weight->ptr) & 15) == 0};
    return LH_OK;
}

}  // namespace

extern "C" {

uint32_t lh_latent_padded_rank(uint32_t rank) { return padded_rank(rank); }
uint32_t lh_latent_row(uint32_t rank, uint32_t rot) { return padded_rank(rank) + padded_rot(rot); }

int lh_latent_prepare_into(lh_batch* batch, const lh_buffer* q_rot, const lh_buffer* down, const lh_buffer* norm_weight, const lh_buffer* frequencies,
                           const lh_buffer* position, lh_buffer* q, int q_dtype, lh_buffer* cache, int dtype, uint32_t rows, uint32_t heads, uint32_t rank,
                           uint32_t rot, uint32_t q_ld, uint32_t rot_column, uint32_t clear_column, uint32_t capacity, float eps) {
    const char* op = "latent_prepare";
    LH_REQUIRE(batch, "%s: batch is null", op);
    if (rows == 0) return LH_OK;
    PrepareArgs a;
    uint32_t pieces = 0;
    int r = prepare_args(a, pieces, op, q_rot, down, norm_weight, frequencies, position, q, q_dtype, cache, dtype, rows, heads, rank, rot, q_ld, rot_column, clear_column,
                         capacity, eps);
    if (r != LH_OK) return r;
    const dim3 grid(rows, pieces);
    if (dtype == LH_F32) hipLaunchKernelGGL((latent_prepare_kernel<float, float>), grid, dim3(256), 0, batch->ctx->stream, a);
    else if (q_dtype == LH_F32) hipLaunchKernelGGL((latent_prepare_kernel<float, uint16_t>), grid, dim3(256), 0, batch->ctx->stream, a);
    else hipLaunchKernelGGL((latent_prepare_kernel<uint16_t, uint16_t>), grid, dim3(256), 0, batch->ctx->stream, a);
    r = lh_check_launch(op);
    if (r == LH_OK) batch->dispatch_count++;
    return r;
}

int lh_head_linear_into(lh_batch* batch, const lh_buffer* input, int dtype, const lh_buffer* weight, lh_buffer* output, int output_dtype, uint32_t rows,
                        uint32_t heads, uint32_t n, uint32_t k, uint32_t output_ld) {
    const char* op = "head_linear";
    LH_REQUIRE(batch, "%s: batch is null", op);
    if (rows == 0) return LH_OK;
    HeadArgs a;
    int r = head_args(a, op, input, dtype, weight, output, output_dtype, rows, heads, n, k, output_ld);
    if (r != LH_OK) return r;
    if (dtype == LH_F32) hipLaunchKernelGGL(head_linear_plain_kernel, dim3((n + 3) / 4, heads, rows), dim3(256), 0, batch->ctx->stream, a);
    else {
        const dim3 grid((n + 15) / 16, heads, (rows + 15) / 16);
        if (output_dtype == LH_F32) hipLaunchKernelGGL((head_linear_mfma_kernel<float>), grid, dim3(256), 0, batch->ctx->stream, a);
        else hipLaunchKernelGGL((head_linear_mfma_kernel<uint16_t>), grid, dim3(256), 0, batch->ctx->stream, a);
    }
    r = lh_check_launch(op);
    if (r == LH_OK) batch->dispatch_count++;
    return r;
}

int lh_latent_expand_into(lh_batch* batch, const lh_buffer* cache, int dtype, const lh_buffer* weight, lh_buffer* keys, lh_buffer* values, uint32_t positions,
                          uint32_t heads, uint32_t dim, uint32_t rot, uint32_t vdim, uint32_t rank) {
    const char* op = "latent_expand";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(dtype == LH_F32 || dtype == LH_BF16, "%s: dtype %d", op, dtype);
    LH_REQUIRE(heads > 0 && dim > 0 && rot > 0 && vdim > 0 && rank > 0, "%s: heads %u, dim %u + %u, vdim %u, rank %u", op, heads, dim, rot, vdim, rank);
    if (positions == 0) return LH_OK;
    const size_t es = dtype == LH_F32 ? 4 : 2;
    const uint32_t row = lh_latent_row(rank, rot), dq = lh_attention_padded_dim(dim + rot), dv = lh_attention_padded_vdim(vdim);
    LH_REQUIRE(positions % 32 == 0, "%s: %u positions are not whole blocks", op, positions);
    LH_NEED(cache, (size_t)positions * row * es, op, "cache");
    LH_NEED(weight, (size_t)heads * (dim + vdim) * rank * 2, op, "weight");
    LH_NEED(keys, (size_t)positions * heads * dq * es, op, "keys");
    LH_NEED(values, (size_t)positions * heads * dv * es, op, "values");
    LhLinear a;
    memset(&a, 0, sizeof a);
    const uint32_t ns[2] = {heads * dim, heads * vdim}, acts[2] = {LH_ACT_NONE, LH_ACT_NONE}, head[2] = {dim, vdim}, padded[2] = {dq, dv},
                   layouts[2] = {LH_ROWS, LH_ROWS};
    lh_buffer* const outs[2] = {keys, values};
    const int rs = lh_make_segments(a.seg, op, positions, 0, 2, ns, acts, head, padded, layouts, outs, dtype, 0, nullptr);
    if (rs != LH_OK) return rs;
    a.seg.layout[1] = LH_BLOCKS_AT_POSITION;                  // the portion is the whole cache: position 0
    a.seg.vec4[1] = 0;
    a.A = cache->ptr; a.a_f32 = dtype == LH_F32; a.W = (const uint16_t*)weight->ptr;
    a.M = positions; a.N = heads * (dim + vdim); a.K = rank; a.lda = row;
    int r = lh_launch_linear(batch->ctx, a, op);
    if (r != LH_OK) return r;
    const uint32_t dl = padded_rank(rank);
    const bool aligned = (((uintptr_t)cache->ptr | (uintptr_t)keys->ptr) & 15) == 0;
#define LH_EXPAND(T, N) hipLaunchKernelGGL((expand_rotated_kernel<T>), dim3(positions), dim3(256), 0, batch->ctx->stream, (const T*)cache->ptr, (T*)keys->ptr, heads, row / N, dl / N, dim / N, rot / N, dq / N)
    if (dtype == LH_F32) LH_EXPAND(float, 1);
    else if (aligned && dim % 8 == 0 && rot % 8 == 0) LH_EXPAND(uint4, 8);
    else LH_EXPAND(uint16_t, 1);
#undef LH_EXPAND
    r = lh_check_launch(op);
    if (r == LH_OK) batch->dispatch_count += 2;
    return r;
}

int lh_latent_attention_rows_into(lh_batch* batch, const lh_buffer* q, const lh_buffer* cache, lh_buffer* output, int dtype, const lh_buffer* position,
                                  uint32_t max_position, uint32_t rows, uint32_t heads, uint32_t rank, uint32_t rot, uint32_t capacity, float scale,
                                  const lh_buffer* sink, const lh_buffer* gate) {
    const char* op = "latent_attention_rows";
    LH_REQUIRE(batch, "%s: batch is null", op);
    if (rows == 0) return LH_OK;
    AttentionArgs a;
    int r = latent_args(a, op, q, cache, dtype, position, max_position, rows, heads, rank, rot, capacity, scale, sink, gate);
    if (r != LH_OK) return r;
    LH_NEED(output, (size_t)rows * heads * rank * (dtype == LH_F32 ? 4 : 2), op, "output");
    a.out = output->ptr;
    uint32_t launches = 1;
    if (tiled(a, dtype, rot)) r = launch_tiled(batch->ctx, a, max_position, op, launches);
    else {
        LH_REQUIRE((uint64_t)rows * heads < 0x7FFFFFFFull, "%s: %u rows", op, rows);
        if (dtype == LH_F32) hipLaunchKernelGGL((attention_plain_kernel<float, float>), dim3(rows * heads), dim3(256), (size_t)a.dim * 4, batch->ctx->stream, a);
        else hipLaunchKernelGGL((attention_plain_kernel<float, uint16_t>), dim3(rows * heads), dim3(256), (size_t)a.dim * 4, batch->ctx->stream, a);
        r = lh_check_launch(op);
    }
    batch->dispatch_count += launches;
    return r;
}

int lh_latent_queries_into(lh_batch* batch, const lh_buffer* q, const lh_buffer* key_weight, const lh_buffer* q_rot, const lh_buffer* down,
                           const lh_buffer* norm_weight, const lh_buffer* frequencies, const lh_buffer* position, lh_buffer* output, lh_buffer* cache, int dtype,
                           uint32_t rows, uint32_t heads, uint32_t dim, uint32_t rank, uint32_t rot, uint32_t capacity, float eps) {
    const char* op = "latent_queries";
    LH_REQUIRE(batch, "%s: batch is null", op);
    if (rows == 0) return LH_OK;
    PrepareArgs p;
    uint32_t pieces = 0;
    const uint32_t row = lh_latent_row(rank, rot);
    int r = prepare_args(p, pieces, op, q_rot, down, norm_weight, frequencies, position, output, LH_F32, cache, dtype, rows, heads, rank, rot, row, padded_rank(rank), rank,
                         capacity, eps);
    if (r != LH_OK) return r;
    HeadArgs a;
    r = head_args(a, op, q, dtype, key_weight, output, LH_F32, rows, heads, rank, dim, row);
    if (r != LH_OK) return r;
    const uint64_t tiles = (uint64_t)((rank + 15) / 16) * heads * ((rows + 15) / 16);
    if (dtype == LH_F32 || tiles + (uint64_t)rows * pieces >= 0x7FFFFFFFull) {
        r = lh_head_linear_into(batch, q, dtype, key_weight, output, LH_F32, rows, heads, rank, dim, row);
        return r != LH_OK ? r : lh_latent_prepare_into(batch, q_rot, down, norm_weight, frequencies, position, output, LH_F32, cache, dtype, rows, heads, rank, rot, row,
                                                       padded_rank(rank), rank, capacity, eps);
    }
    hipLaunchKernelGGL(latent_queries_kernel, dim3((uint32_t)tiles + rows * pieces), dim3(256), 0, batch->ctx->stream, a, p, (uint32_t)tiles, pieces);
    r = lh_check_launch(op);
    if (r == LH_OK) batch->dispatch_count++;
    return r;
}

}  // extern "C"
