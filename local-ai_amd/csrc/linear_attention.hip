// Linear attention with a decay a per head: for every token M <- a M + k (x) v, y = q M.  The decay is fixed, or computed from
// the token together with a step size that scales k (x) v (selective state space; heads may then share q and k in groups, and
// a multiple of v is added to y).  The state M is f32,
// kept as [head][value column][DQ key columns] (the key columns that exist, then zeros).
//
// Recurrent form: one workgroup per head and 16 value columns; a row of 16 lanes holds one value column's state in
// registers (DQ / 16 values each) and walks the rows.
//
// Chunked form (64 rows a chunk, bf16 inputs on the matrix cores, everything else f32):
//   1. every chunk's own contribution to the state, U = sum over rows s of a^(L-1-s) k_s (x) v_s (all chunks at once)
//   2. a scan over the chunks, M <- a^L M + U, that leaves each chunk's incoming state in place of its U
//   3. all outputs: y_t = a^(t+1) q_t M_in + sum over s <= t of a^(t-s) (q_t . k_s) v_s
// With decays per token, a power becomes the exponential of a difference of running sums of the decays' logarithms.
// Where an f32 quantity enters a product (decayed keys, decayed scores, the state) it does so as the sum of three bf16
// terms, which is all of its 24 bits; the products of bf16 values are exact and summed in f32.
#include "float_ops.hpp"
#include <algorithm>

namespace {

constexpr uint32_t kChunk = 64;

// What the step of a token is: fixed per head, or computed from the token (selective state space).
__device__ __forceinline__ float softplus(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }

struct RecurrentArgs {
    const void *q, *k, *v;
    float* state;
    const float* decay;                                     // [heads]
    const float *dt_raw, *dt_bias, *a_log, *skip;           // selective: [rows, heads], then [heads] each
    float* out;
    uint32_t rows, heads, key_heads, dim, dq, vdim;
    float scale;
};

template <typename T, int NR, bool SELECTIVE>
__global__ __launch_bounds__(256) void recurrent_kernel(const RecurrentArgs a) {
    const T *q = static_cast<const T*>(a.q), *k = static_cast<const T*>(a.k), *v = static_cast<const T*>(a.v);
    const uint32_t dim = a.dim, dq = a.dq, vdim = a.vdim, heads = a.heads, rows = a.rows;
    const uint32_t vt = (vdim + 15) / 16, h = blockIdx.x / vt, col = (blockIdx.x % vt) * 16 + (threadIdx.x >> 4), part = threadIdx.x & 15;
    const uint32_t kh = h / (heads / a.key_heads);
    const bool on = col < vdim;
    const uint32_t c = on ? col : vdim - 1, k0 = part * NR;
    float* st = a.state + ((size_t)h * vdim + c) * dq + k0;
    float s[NR];
#pragma unroll
    for (int i = 0; i < NR; i++) s[i] = k0 + i < dq ? st[i] : 0.0f;
    const float fixed = SELECTIVE ? 0.0f : a.decay[h], rate = SELECTIVE ? -expf(a.a_log[h]) : 0.0f, bias = SELECTIVE ? a.dt_bias[h] : 0.0f,
                skip = SELECTIVE ? a.skip[h] : 0.0f;
    float kn[NR], qn[NR], vn, zn = 0.0f;
    auto fetch = [&](uint32_t t) {
        const size_t row = ((size_t)t * a.key_heads + kh) * dq + k0;
#pragma unroll
        for (int i = 0; i < NR; i++) {
            const bool in = k0 + i < dim;
            kn[i] = in ? lh_ld(k, row + i) : 0.0f;
            qn[i] = in ? lh_ld(q, row + i) : 0.0f;
        }
        vn = lh_ld(v, ((size_t)t * heads + h) * vdim + c);
        if (SELECTIVE) zn = a.dt_raw[(size_t)t * heads + h];
    };
    fetch(0);
    for (uint32_t t = 0; t < rows; t++) {
        float kc[NR], qc[NR];
        const float x = vn, dt = SELECTIVE ? softplus(zn + bias) : 1.0f, d = SELECTIVE ? expf(rate * dt) : fixed, vc = SELECTIVE ? dt * x : x;
#pragma unroll
        for (int i = 0; i < NR; i++) { kc[i] = kn[i]; qc[i] = qn[i]; }
        if (t + 1 < rows) fetch(t + 1);
        float o = 0.0f;
#pragma unroll
        for (int i = 0; i < NR; i++) {
            s[i] = __builtin_fmaf(kc[i], vc, d * s[i]);
            o = __builtin_fmaf(s[i], qc[i], o);
        }
        o = lh_group_sum(o, 16);
        if (part == 0 && on) a.out[((size_t)t * heads + h) * vdim + col] = SELECTIVE ? __builtin_fmaf(skip, x, o) : o * a.scale;
    }
    if (on) {
#pragma unroll
        for (int i = 0; i < NR; i++) if (k0 + i < dq) st[i] = s[i];
    }
}

// The steps of a selective state space, one wave per head and chunk: step sizes, and the running sum of the logarithms of the
// decays within the chunk.  Rows past the last have step 0 and decay 1.
__global__ __launch_bounds__(64) void chunk_steps_kernel(const float* __restrict__ dt_raw, const float* __restrict__ dt_bias, const float* __restrict__ a_log,
                                                        float* __restrict__ sums, float* __restrict__ sizes, uint32_t rows, uint32_t heads, uint32_t chunks) {
    const uint32_t h = blockIdx.x % heads, c = blockIdx.x / heads, lane = threadIdx.x, t = c * kChunk + lane;
    const float dt = t < rows ? softplus(dt_raw[(size_t)t * heads + h] + dt_bias[h]) : 0.0f;
    float sum = -expf(a_log[h]) * dt;
#pragma unroll
    for (uint32_t d = 1; d < 64; d <<= 1) {
        const float o = __shfl_up(sum, d, 64);
        if (lane >= d) sum += o;
    }
    const size_t i = ((size_t)h * chunks + c) * kChunk + lane;
    sums[i] = sum;
    sizes[i] = dt;
}

struct ChunkArgs {
    const uint16_t *q, *k, *v;
    float* state;
    const float* powers;       // fixed decays: [heads][65]
    const float *sums, *sizes; // selective: [heads][chunks][64]
    const float* skip;         // selective: [heads]
    float* chunk_state;        // [chunk][heads][vdim][dq]
    float* out;
    uint32_t rows, heads, key_heads, dim, vdim, chunks;
    float scale;
};

__device__ __forceinline__ lh_bf16x8 bf8(const uint32_t (&w)[4]) {
    struct { uint32_t v[4]; } t = {{w[0], w[1], w[2], w[3]}};
    return __builtin_bit_cast(lh_bf16x8, t);
}

constexpr uint32_t kLdT = kChunk + 8;     // row length of a transposed tile: 16-byte aligned, rows on different banks

// 64 rows of 64 value columns, transposed into LDS: thread t brings in rows t / 8 and t / 8 + 32, eight columns each.
struct ValueTile { uint4 x[2]; };
__device__ __forceinline__ void load_values(ValueTile& f, const ChunkArgs& a, uint32_t t0, uint32_t L, uint32_t h, uint32_t v0, uint32_t tid) {
    const uint32_t d = v0 + (tid & 7) * 8;
#pragma unroll
    for (int i = 0; i < 2; i++) {
        const uint32_t s = (tid >> 3) + 32 * i;
        f.x[i] = make_uint4(0u, 0u, 0u, 0u);
        if (s >= L || d >= a.vdim) continue;
        const uint16_t* p = a.v + ((size_t)(t0 + s) * a.heads + h) * a.vdim + d;
        if ((a.vdim & 7) == 0) f.x[i] = *reinterpret_cast<const uint4*>(p);
        else {
            uint32_t w[4] = {0u, 0u, 0u, 0u};
#pragma unroll
            for (uint32_t j = 0; j < 8; j++) if (d + j < a.vdim) w[j >> 1] |= (uint32_t)p[j] << (16 * (j & 1));
            f.x[i] = make_uint4(w[0], w[1], w[2], w[3]);
        }
    }
}
template <bool SLOTS>
__device__ __forceinline__ void park_values(const ValueTile& f, uint16_t (&vt)[64][kLdT], uint32_t tid) {
#pragma unroll
    for (int i = 0; i < 2; i++) {
        const uint32_t s = (tid >> 3) + 32 * i, place = SLOTS ? (s & 32) + lh_block_slot(s & 31) : s;
        const uint32_t w[4] = {f.x[i].x, f.x[i].y, f.x[i].z, f.x[i].w};
#pragma unroll
        for (uint32_t j = 0; j < 8; j++) vt[(tid & 7) * 8 + j][place] = (uint16_t)(w[j >> 1] >> (16 * (j & 1)));
    }
}

// Step 1.  A workgroup takes one chunk of one head, 32 key columns and 64 value columns; wave w the value columns 16 w ..
// 16 w + 15.  Row operand = decayed keys (16 key columns x rows), column operand = values (16 value columns x rows).
template <int DQ, bool SELECTIVE>
__global__ __launch_bounds__(256) void chunk_state_kernel(const ChunkArgs a) {
    __shared__ __align__(16) uint16_t kt[3][32][kLdT], vt[64][kLdT];
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const uint32_t vtiles = (a.vdim + 63) / 64, k0 = blockIdx.x % (DQ / 32) * 32, r = blockIdx.x / (DQ / 32);
    const uint32_t vb = r % vtiles, h = (r / vtiles) % a.heads, c = r / (vtiles * a.heads);
    const uint32_t t0 = c * kChunk, L = min(kChunk, a.rows - t0), v0 = vb * 64;
    ValueTile f;
    load_values(f, a, t0, L, h, v0, tid);
    {   // eight key columns of one row per thread
        const uint32_t s = tid >> 2, d = (tid & 3) * 8;
        uint4 x = make_uint4(0u, 0u, 0u, 0u);
        float p = 0.0f;
        if (s < L) {
            x = *reinterpret_cast<const uint4*>(a.k + ((size_t)(t0 + s) * a.key_heads + h / (a.heads / a.key_heads)) * DQ + k0 + d);
            if constexpr (SELECTIVE) {
                const size_t i = ((size_t)h * a.chunks + c) * kChunk;
                p = expf(a.sums[i + L - 1] - a.sums[i + s]) * a.sizes[i + s];
            } else p = a.powers[h * (kChunk + 1) + L - 1 - s];
        }
        const uint32_t w[4] = {x.x, x.y, x.z, x.w};
#pragma unroll
        for (uint32_t j = 0; j < 8; j++) {
            const LhSplit3 e = lh_split3(s < L && k0 + d + j < a.dim ? lh_bf2f((uint16_t)(w[j >> 1] >> (16 * (j & 1)))) * p : 0.0f);
            kt[0][d + j][s] = e.hi; kt[1][d + j][s] = e.mid; kt[2][d + j][s] = e.lo;
        }
    }
    park_values<false>(f, vt, tid);
    __syncthreads();
    lh_f32x4 acc[2] = {(lh_f32x4){0.f, 0.f, 0.f, 0.f}, (lh_f32x4){0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int ks = 0; ks < 2; ks++) {
        const uint32_t s = ks * 32 + (lane >> 4) * 8;
        const lh_bf16x8 vf = *reinterpret_cast<const lh_bf16x8*>(&vt[wave * 16 + (lane & 15)][s]);
#pragma unroll
        for (int i = 0; i < 2; i++)
#pragma unroll
            for (int p = 0; p < 3; p++)
                acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const lh_bf16x8*>(&kt[p][i * 16 + (lane & 15)][s]), vf, acc[i], 0, 0, 0);
    }
    const uint32_t col = v0 + wave * 16 + (lane & 15);
    if (col >= a.vdim) return;
    float* U = a.chunk_state + ((size_t)c * a.heads + h) * a.vdim * DQ + (size_t)col * DQ + k0 + (lane >> 4) * 4;
#pragma unroll
    for (int i = 0; i < 2; i++) *reinterpret_cast<float4*>(U + i * 16) = make_float4(acc[i][0], acc[i][1], acc[i][2], acc[i][3]);
}

// Step 2.  A thread owns four neighbouring state values and walks the chunks, eight loads ahead.
template <bool SELECTIVE>
__global__ __launch_bounds__(256) void chunk_scan_kernel(const ChunkArgs a, uint32_t dq) {
    const size_t per_head4 = (size_t)a.vdim * dq / 4, total4 = per_head4 * a.heads, i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= total4) return;
    const uint32_t h = (uint32_t)(i / per_head4);
    const float* pw = SELECTIVE ? nullptr : a.powers + h * (kChunk + 1);
    const float full = SELECTIVE ? 0.0f : pw[kChunk];
    float4* st = reinterpret_cast<float4*>(a.state) + i;
    float4* u = reinterpret_cast<float4*>(a.chunk_state) + i;
    float4 s = *st;
    constexpr uint32_t P = 8;
    for (uint32_t c0 = 0; c0 < a.chunks; c0 += P) {
        float4 x[P];
#pragma unroll
        for (uint32_t j = 0; j < P; j++) x[j] = u[(size_t)min(c0 + j, a.chunks - 1) * total4];
#pragma unroll
        for (uint32_t j = 0; j < P; j++) {
            if (c0 + j >= a.chunks) break;
            u[(size_t)(c0 + j) * total4] = s;
            const float d = SELECTIVE ? expf(a.sums[((size_t)h * a.chunks + c0 + j) * kChunk + kChunk - 1]) : c0 + j + 1 < a.chunks ? full : pw[a.rows - (a.chunks - 1) * kChunk];
            s.x = __builtin_fmaf(d, s.x, x[j].x); s.y = __builtin_fmaf(d, s.y, x[j].y);
            s.z = __builtin_fmaf(d, s.z, x[j].z); s.w = __builtin_fmaf(d, s.w, x[j].w);
        }
    }
    *st = s;
}

// Step 3.  A workgroup takes one chunk of one head and 64 value columns; wave w the rows 16 w .. 16 w + 15.
// Scores transposed (row operand keys, column operand queries), so that the decayed scores are in operand order for
// O^T = V^T P^T, whose k index 8g + j is row 4g + j of the first 16-row tile (j < 4) or 4g + j - 4 of the second.
template <int DQ, bool SELECTIVE>
__global__ __launch_bounds__(256) void chunk_output_kernel(const ChunkArgs a) {
    __shared__ __align__(16) uint16_t vt[64][kLdT];            // [value column][32-row half][slot]
    __shared__ float pws[kChunk + 1], sizes[SELECTIVE ? kChunk : 1];   // powers of the decay, or running sums of its logarithm
    const uint32_t tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4;
    const uint32_t vtiles = (a.vdim + 63) / 64, vb = blockIdx.x % vtiles, h = (blockIdx.x / vtiles) % a.heads, c = blockIdx.x / (vtiles * a.heads);
    const uint32_t t0 = c * kChunk, L = min(kChunk, a.rows - t0), v0 = vb * 64;
    ValueTile f;
    load_values(f, a, t0, L, h, v0, tid);
    const uint32_t kh = h / (a.heads / a.key_heads);
    if constexpr (SELECTIVE) {
        if (tid < kChunk) { pws[tid] = a.sums[((size_t)h * a.chunks + c) * kChunk + tid]; sizes[tid] = a.sizes[((size_t)h * a.chunks + c) * kChunk + tid]; }
    } else if (tid <= kChunk) pws[tid] = a.powers[h * (kChunk + 1) + tid];
    const uint32_t t = wave * 16 + (lane & 15), tr = min(t, L - 1);
    lh_bf16x8 qf[DQ / 32];
#pragma unroll
    for (int i = 0; i < DQ / 32; i++) {
        const uint32_t k = i * 32 + g * 8;
        uint32_t w[4] = {0u, 0u, 0u, 0u};
        if (k < a.dim) {
            const uint4 x = *reinterpret_cast<const uint4*>(a.q + ((size_t)(t0 + tr) * a.key_heads + kh) * DQ + k);
            w[0] = x.x; w[1] = x.y; w[2] = x.z; w[3] = x.w;
#pragma unroll
            for (int j = 0; j < 4; j++) {
                if (k + 2 * j >= a.dim) w[j] = 0u;
                else if (k + 2 * j + 1 >= a.dim) w[j] &= 0xFFFFu;
            }
        }
        qf[i] = bf8(w);
    }
    park_values<true>(f, vt, tid);
    __syncthreads();
    if (wave * 16 >= L) return;
    lh_f32x4 o[4];
    // the state's part, scaled by decay^(t + 1) afterwards
    const float* S = a.chunk_state + ((size_t)c * a.heads + h) * a.vdim * DQ;
#pragma unroll
    for (int d = 0; d < 4; d++) {
        o[d] = (lh_f32x4){0.f, 0.f, 0.f, 0.f};
        if (v0 + d * 16 >= a.vdim) continue;
        const float* srow = S + (size_t)min(v0 + d * 16 + (lane & 15), a.vdim - 1) * DQ + g * 8;
#pragma unroll
        for (int i = 0; i < DQ / 32; i++) {
            const float4 x = *reinterpret_cast<const float4*>(srow + i * 32), y = *reinterpret_cast<const float4*>(srow + i * 32 + 4);
            const float f[8] = {x.x, x.y, x.z, x.w, y.x, y.y, y.z, y.w};
            uint32_t p[3][4];
#pragma unroll
            for (int j = 0; j < 4; j++) {
                const LhSplit3 e = lh_split3(f[2 * j]), m = lh_split3(f[2 * j + 1]);
                p[0][j] = (uint32_t)e.hi | ((uint32_t)m.hi << 16);
                p[1][j] = (uint32_t)e.mid | ((uint32_t)m.mid << 16);
                p[2][j] = (uint32_t)e.lo | ((uint32_t)m.lo << 16);
            }
#pragma unroll
            for (int z = 2; z >= 0; z--) o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf8(p[z]), qf[i], o[d], 0, 0, 0);
        }
    }
    const float carry = SELECTIVE ? expf(pws[tr]) : pws[tr + 1];
#pragma unroll
    for (int d = 0; d < 4; d++)
#pragma unroll
        for (int r = 0; r < 4; r++) o[d][r] *= carry;
    // the chunk's own rows, 32 at a time
    for (uint32_t s0 = 0; s0 <= wave * 16 + 15 && s0 < L; s0 += 32) {
        lh_f32x4 sc[2];
#pragma unroll
        for (int u = 0; u < 2; u++) {
            sc[u] = (lh_f32x4){0.f, 0.f, 0.f, 0.f};
            const uint32_t s = min(s0 + u * 16 + (lane & 15), L - 1);
            const uint16_t* kr = a.k + ((size_t)(t0 + s) * a.key_heads + kh) * DQ + g * 8;
#pragma unroll
            for (int i = 0; i < DQ / 32; i++) sc[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const lh_bf16x8*>(kr + i * 32), qf[i], sc[u], 0, 0, 0);
        }
        uint32_t p[3][4];
#pragma unroll
        for (int j = 0; j < 4; j++) {
            LhSplit3 e[2];
#pragma unroll
            for (int b = 0; b < 2; b++) {
                const int n = 2 * j + b;
                const uint32_t s = s0 + (n >> 2) * 16 + g * 4 + (n & 3);
                const float f = SELECTIVE ? expf(fminf(pws[tr] - pws[min(s, kChunk - 1)], 0.0f)) * sizes[min(s, kChunk - 1)] : pws[min(t - s, kChunk)];
                e[b] = lh_split3(s <= t && s < L ? sc[n >> 2][n & 3] * f : 0.0f);
            }
            p[0][j] = (uint32_t)e[0].hi | ((uint32_t)e[1].hi << 16);
            p[1][j] = (uint32_t)e[0].mid | ((uint32_t)e[1].mid << 16);
            p[2][j] = (uint32_t)e[0].lo | ((uint32_t)e[1].lo << 16);
        }
#pragma unroll
        for (int d = 0; d < 4; d++) {
            const lh_bf16x8 vf = *reinterpret_cast<const lh_bf16x8*>(&vt[d * 16 + (lane & 15)][s0 + g * 8]);
#pragma unroll
            for (int z = 2; z >= 0; z--) o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, bf8(p[z]), o[d], 0, 0, 0);
        }
    }
    if (t >= L) return;
    float* out = a.out + ((size_t)(t0 + t) * a.heads + h) * a.vdim + v0;
    const uint16_t* x = a.v + ((size_t)(t0 + t) * a.heads + h) * a.vdim + v0;
    const float skip = SELECTIVE ? a.skip[h] : 0.0f;
#pragma unroll
    for (int d = 0; d < 4; d++) {
        const uint32_t col = d * 16 + g * 4;
        if (v0 + col >= a.vdim) continue;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            if constexpr (SELECTIVE) o[d][r] = __builtin_fmaf(skip, lh_bf2f(x[min(col + r, a.vdim - 1 - v0)]), o[d][r]);
            else o[d][r] *= a.scale;
        }
        if ((a.vdim & 3) == 0) { if (v0 + col < a.vdim) *reinterpret_cast<float4*>(out + col) = make_float4(o[d][0], o[d][1], o[d][2], o[d][3]); }
        else {
#pragma unroll
            for (int r = 0; r < 4; r++) if (v0 + col + r < a.vdim) out[col + r] = o[d][r];
        }
    }
}

template <int DQ, bool SELECTIVE>
int launch_chunked(lh_context* ctx, const ChunkArgs& a, const char* op) {
    const uint32_t grid = a.chunks * a.heads * ((a.vdim + 63) / 64);
    hipLaunchKernelGGL((chunk_state_kernel<DQ, SELECTIVE>), dim3(grid * (DQ / 32)), dim3(256), 0, ctx->stream, a);
    int r = lh_check_launch(op);
    if (r != LH_OK) return r;
    const size_t total4 = (size_t)a.heads * a.vdim * DQ / 4;
    hipLaunchKernelGGL((chunk_scan_kernel<SELECTIVE>), dim3((uint32_t)((total4 + 255) / 256)), dim3(256), 0, ctx->stream, a, (uint32_t)DQ);
    r = lh_check_launch(op);
    if (r != LH_OK) return r;
    hipLaunchKernelGGL((chunk_output_kernel<DQ, SELECTIVE>), dim3(grid), dim3(256), 0, ctx->stream, a);
    return lh_check_launch(op);
}
template <bool SELECTIVE>
int launch_chunked_dim(lh_context* ctx, const ChunkArgs& a, const char* op) {
    switch (lh_linear_attention_padded_dim(a.dim)) {
        case 32: return launch_chunked<32, SELECTIVE>(ctx, a, op);
        case 64: return launch_chunked<64, SELECTIVE>(ctx, a, op);
        case 128: return launch_chunked<128, SELECTIVE>(ctx, a, op);
        default: return launch_chunked<256, SELECTIVE>(ctx, a, op);
    }
}

template <typename T, bool SELECTIVE>
int launch_recurrent(lh_context* ctx, const RecurrentArgs& a, const char* op) {
    const uint64_t grid = (uint64_t)a.heads * ((a.vdim + 15) / 16);
    LH_REQUIRE(grid < 0x7FFFFFFFull, "%s: heads %u, vdim %u", op, a.heads, a.vdim);
#define LH_REC(NR_) hipLaunchKernelGGL((recurrent_kernel<T, NR_, SELECTIVE>), dim3((uint32_t)grid), dim3(256), 0, ctx->stream, a)
    if (a.dq <= 32) LH_REC(2);
    else if (a.dq <= 64) LH_REC(4);
    else if (a.dq <= 128) LH_REC(8);
    else if (a.dq <= 256) LH_REC(16);
    else if (a.dq <= 512) LH_REC(32);
    else LH_REC(64);
#undef LH_REC
    return lh_check_launch(op);
}

}  // namespace

extern "C" {

uint32_t lh_linear_attention_padded_dim(uint32_t dim) { return dim <= 32 ? 32u : dim <= 64 ? 64u : (dim + 127) / 128 * 128; }

size_t lh_linear_attention_workspace_bytes(uint32_t rows, uint32_t heads, uint32_t dim, uint32_t vdim) {
    return (size_t)((rows + kChunk - 1) / kChunk) * heads * vdim * lh_linear_attention_padded_dim(dim) * 4;
}

int lh_linear_attention_recurrent_into(lh_batch* batch, const lh_buffer* q, const lh_buffer* k, const lh_buffer* v, int dtype, lh_buffer* state,
                                       const lh_buffer* decay, lh_buffer* output, uint32_t rows, uint32_t heads, uint32_t dim, uint32_t vdim, float scale) {
    const char* op = "linear_attention_recurrent";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(dtype == LH_F32 || dtype == LH_BF16, "%s: dtype %d", op, dtype);
    LH_REQUIRE(heads > 0 && dim > 0 && dim <= 1024 && vdim > 0, "%s: heads %u, dim %u, vdim %u", op, heads, dim, vdim);
    if (rows == 0) return LH_OK;
    const uint32_t dq = lh_linear_attention_padded_dim(dim);
    const size_t es = dtype == LH_F32 ? 4 : 2;
    LH_NEED(q, (size_t)rows * heads * dq * es, op, "q");
    LH_NEED(k, (size_t)rows * heads * dq * es, op, "k");
    LH_NEED(v, (size_t)rows * heads * vdim * es, op, "v");
    LH_NEED(state, (size_t)heads * vdim * dq * 4, op, "state");
    LH_NEED(decay, (size_t)heads * 4, op, "decay");
    LH_NEED(output, (size_t)rows * heads * vdim * 4, op, "output");
    RecurrentArgs a{};
    a.q = q->ptr; a.k = k->ptr; a.v = v->ptr; a.state = (float*)state->ptr; a.decay = (const float*)decay->ptr; a.out = (float*)output->ptr;
    a.rows = rows; a.heads = a.key_heads = heads; a.dim = dim; a.dq = dq; a.vdim = vdim; a.scale = scale;
    const int r = dtype == LH_F32 ? launch_recurrent<float, false>(batch->ctx, a, op) : launch_recurrent<uint16_t, false>(batch->ctx, a, op);
    if (r == LH_OK) batch->dispatch_count++;
    return r;
}

int lh_linear_attention_chunked_into(lh_batch* batch, const lh_buffer* q, const lh_buffer* k, const lh_buffer* v, lh_buffer* state,
                                     const lh_buffer* decay_powers, lh_buffer* workspace, lh_buffer* output, uint32_t rows, uint32_t heads, uint32_t dim,
                                     uint32_t vdim, float scale) {
    const char* op = "linear_attention_chunked";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(heads > 0 && dim > 0 && dim <= 256 && vdim > 0, "%s: heads %u, dim %u, vdim %u", op, heads, dim, vdim);
    if (rows == 0) return LH_OK;
    const uint32_t dq = lh_linear_attention_padded_dim(dim);
    LH_NEED(q, (size_t)rows * heads * dq * 2, op, "q");
    LH_NEED(k, (size_t)rows * heads * dq * 2, op, "k");
    LH_NEED(v, (size_t)rows * heads * vdim * 2, op, "v");
    LH_NEED(state, (size_t)heads * vdim * dq * 4, op, "state");
    LH_NEED(decay_powers, (size_t)heads * (kChunk + 1) * 4, op, "decay_powers");
    LH_NEED(workspace, lh_linear_attention_workspace_bytes(rows, heads, dim, vdim), op, "workspace");
    LH_NEED(output, (size_t)rows * heads * vdim * 4, op, "output");
    LH_REQUIRE((((uintptr_t)q->ptr | (uintptr_t)k->ptr | (uintptr_t)v->ptr | (uintptr_t)state->ptr | (uintptr_t)workspace->ptr | (uintptr_t)output->ptr) & 15) == 0,
               "%s: buffers must be 16-byte aligned", op);
    ChunkArgs a{};
    a.q = (const uint16_t*)q->ptr; a.k = (const uint16_t*)k->ptr; a.v = (const uint16_t*)v->ptr; a.state = (float*)state->ptr;
    a.powers = (const float*)decay_powers->ptr; a.chunk_state = (float*)workspace->ptr; a.out = (float*)output->ptr;
    a.rows = rows; a.heads = a.key_heads = heads; a.dim = dim; a.vdim = vdim; a.chunks = (rows + kChunk - 1) / kChunk; a.scale = scale;
    LH_REQUIRE((uint64_t)a.chunks * heads * ((vdim + 63) / 64) * 8 < 0x7FFFFFFFull, "%s: %u rows", op, rows);
    const int r = launch_chunked_dim<false>(batch->ctx, a, op);
    if (r == LH_OK) batch->dispatch_count += 3;
    return r;
}

// [heads][chunks][64] running sums, then as many step sizes
size_t lh_selective_steps_bytes(uint32_t rows, uint32_t heads) { return (size_t)((rows + kChunk - 1) / kChunk) * kChunk * heads * 2 * 4; }

int lh_selective_recurrent_into(lh_batch* batch, const lh_buffer* x, const lh_buffer* b, const lh_buffer* c, int dtype, const lh_buffer* dt_raw,
                                const lh_buffer* dt_bias, const lh_buffer* a_log, const lh_buffer* skip, lh_buffer* memory, lh_buffer* output, uint32_t rows,
                                uint32_t heads, uint32_t vdim, uint32_t groups, uint32_t state) {
    const char* op = "selective_recurrent";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(dtype == LH_F32 || dtype == LH_BF16, "%s: dtype %d", op, dtype);
    LH_REQUIRE(heads > 0 && groups > 0 && heads % groups == 0 && state > 0 && state <= 1024 && vdim > 0, "%s: heads %u over %u groups, state %u, vdim %u", op, heads,
               groups, state, vdim);
    if (rows == 0) return LH_OK;
    const uint32_t dq = lh_linear_attention_padded_dim(state);
    const size_t es = dtype == LH_F32 ? 4 : 2;
    LH_NEED(x, (size_t)rows * heads * vdim * es, op, "x");
    LH_NEED(b, (size_t)rows * groups * dq * es, op, "b");
    LH_NEED(c, (size_t)rows * groups * dq * es, op, "c");
    LH_NEED(dt_raw, (size_t)rows * heads * 4, op, "dt_raw");
    LH_NEED(dt_bias, (size_t)heads * 4, op, "dt_bias");
    LH_NEED(a_log, (size_t)heads * 4, op, "a_log");
    LH_NEED(skip, (size_t)heads * 4, op, "skip");
    LH_NEED(memory, (size_t)heads * vdim * dq * 4, op, "memory");
    LH_NEED(output, (size_t)rows * heads * vdim * 4, op, "output");
    RecurrentArgs a{};
    a.q = c->ptr; a.k = b->ptr; a.v = x->ptr; a.state = (float*)memory->ptr; a.out = (float*)output->ptr;
    a.dt_raw = (const float*)dt_raw->ptr; a.dt_bias = (const float*)dt_bias->ptr; a.a_log = (const float*)a_log->ptr; a.skip = (const float*)skip->ptr;
    a.rows = rows; a.heads = heads; a.key_heads = groups; a.dim = state; a.dq = dq; a.vdim = vdim; a.scale = 1.0f;
    const int r = dtype == LH_F32 ? launch_recurrent<float, true>(batch->ctx, a, op) : launch_recurrent<uint16_t, true>(batch->ctx, a, op);
    if (r == LH_OK) batch->dispatch_count++;
    return r;
}

int lh_selective_chunked_into(lh_batch* batch, const lh_buffer* x, const lh_buffer* b, const lh_buffer* c, const lh_buffer* dt_raw, const lh_buffer* dt_bias,
                              const lh_buffer* a_log, const lh_buffer* skip, lh_buffer* memory, lh_buffer* steps, lh_buffer* workspace, lh_buffer* output,
                              uint32_t rows, uint32_t heads, uint32_t vdim, uint32_t groups, uint32_t state) {
    const char* op = "selective_chunked";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(heads > 0 && groups > 0 && heads % groups == 0 && state > 0 && state <= 256 && vdim > 0, "%s: heads %u over %u groups, state %u, vdim %u", op, heads,
               groups, state, vdim);
    if (rows == 0) return LH_OK;
    const uint32_t dq = lh_linear_attention_padded_dim(state);
    LH_NEED(x, (size_t)rows * heads * vdim * 2, op, "x");
    LH_NEED(b, (size_t)rows * groups * dq * 2, op, "b");
    LH_NEED(c, (size_t)rows * groups * dq * 2, op, "c");
    LH_NEED(dt_raw, (size_t)rows * heads * 4, op, "dt_raw");
    LH_NEED(dt_bias, (size_t)heads * 4, op, "dt_bias");
    LH_NEED(a_log, (size_t)heads * 4, op, "a_log");
    LH_NEED(skip, (size_t)heads * 4, op, "skip");
    LH_NEED(memory, (size_t)heads * vdim * dq * 4, op, "memory");
    LH_NEED(steps, lh_selective_steps_bytes(rows, heads), op, "steps");
    LH_NEED(workspace, lh_linear_attention_workspace_bytes(rows, heads, state, vdim), op, "workspace");
    LH_NEED(output, (size_t)rows * heads * vdim * 4, op, "output");
    LH_REQUIRE((((uintptr_t)x->ptr | (uintptr_t)b->ptr | (uintptr_t)c->ptr | (uintptr_t)memory->ptr | (uintptr_t)workspace->ptr | (uintptr_t)output->ptr) & 15) == 0,
               "%s: buffers must be 16-byte aligned", op);
    ChunkArgs a{};
    a.q = (const uint16_t*)c->ptr; a.k = (const uint16_t*)b->ptr; a.v = (const uint16_t*)x->ptr; a.state = (float*)memory->ptr;
    a.chunk_state = (float*)workspace->ptr; a.out = (float*)output->ptr; a.skip = (const float*)skip->ptr;
    a.rows = rows; a.heads = heads; a.key_heads = groups; a.dim = state; a.vdim = vdim; a.chunks = (rows + kChunk - 1) / kChunk; a.scale = 1.0f;
    LH_REQUIRE((uint64_t)a.chunks * heads * ((vdim + 63) / 64) * 8 < 0x7FFFFFFFull, "%s: %u rows", op, rows);
    float* sums = (float*)steps->ptr;
    float* sizes = sums + (size_t)a.chunks * kChunk * heads;
    a.sums = sums; a.sizes = sizes;
    hipLaunchKernelGGL(chunk_steps_kernel, dim3(a.chunks * heads), dim3(64), 0, batch->ctx->stream, (const float*)dt_raw->ptr, (const float*)dt_bias->ptr,
                       (const float*)a_log->ptr, sums, sizes, rows, heads, a.chunks);
    int r = lh_check_launch(op);
    if (r == LH_OK) r = launch_chunked_dim<true>(batch->ctx, a, op);
    if (r == LH_OK) batch->dispatch_count += 4;
    return r;
}

}  // extern "C"
