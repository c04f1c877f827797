// What the softmax-attention kernels share (softmax_attention.hip: caches of keys and values per head; latent_attention.hip:
// caches of one latent for all heads): the running softmax, the merge of partial results, the plain form.
#pragma once
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
    const float* sink;         // [heads]: exp(sink) joins every denominator (may be null; one map)
    const float* gate;         // [rows, heads]: the output is multiplied by sigmoid(gate) (may be null; one map)
    uint32_t values_in_keys;   // plain form: a position's values are the first columns of its key row
    float* partial;            // records [16-row tile][kv head][split][map][16] of dv unnormalised sums, maximum, sum of weights
    uint32_t splits;
    uint32_t parts;            // workgroups that share a row's columns in the merge (one map)
};

constexpr float kLog2e = 1.4426950408889634f;

typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));

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

// Merges the splits of every map of one (query row, head) in columns col0 .. col0 + cols - 1 (cols a multiple of 4, at most 512):
// thread i returns column col0 + i, the maps combined (no norm, no gate).  Groups of cols / 4 threads take the splits in turn,
// four values a thread, several loads on their way; the groups are added through LDS.
constexpr uint32_t kMergeThreads = 512;
template <int MAPS>
struct MergeSpace { float factor[MAPS][512], total[MAPS]; float4 sums[MAPS][kMergeThreads]; };
template <int MAPS>
__device__ __forceinline__ float merge_columns(const AttentionArgs& a, uint32_t t, uint32_t h, uint32_t col0, uint32_t cols, MergeSpace<MAPS>& sp) {
    const uint32_t R = a.heads / a.kv_heads, g = h / R, row = t * R + h % R;
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
        const float sink = a.sink ? a.sink[h] * kLog2e : -INFINITY;
        m = fmaxf(m, sink);
#pragma unroll
        for (uint32_t i = 0; i < 8; i++) {
            if (i * 64 >= a.splits) break;
            const float f = __builtin_amdgcn_exp2f(mine[i] - m);
            if (i * 64 + lane < a.splits) sp.factor[wave][i * 64 + lane] = f;
            l += f * ml[i];
        }
        l = lh_group_sum(l, 64) + __builtin_amdgcn_exp2f(sink - m);
        if (lane == 0) sp.total[wave] = 1.0f / l;
    }
    __syncthreads();
    const uint32_t quads = cols / 4, groups = kMergeThreads / quads, grp = threadIdx.x / quads, q = threadIdx.x % quads;   // quads <= 128
    float4 acc[MAPS];
#pragma unroll
    for (int mp = 0; mp < MAPS; mp++) acc[mp] = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 4
    for (uint32_t s = grp; s < a.splits; s += groups)
#pragma unroll
        for (int mp = 0; mp < MAPS; mp++) {
            const float4 x = *reinterpret_cast<const float4*>(rec + s * stride + mp * 16 * kRow + col0 + q * 4);
            const float f = sp.factor[mp][s];
            acc[mp].x += f * x.x; acc[mp].y += f * x.y; acc[mp].z += f * x.z; acc[mp].w += f * x.w;
        }
#pragma unroll
    for (int mp = 0; mp < MAPS; mp++) sp.sums[mp][threadIdx.x] = acc[mp];
    __syncthreads();
    float v = 0.0f;
    if (threadIdx.x < cols && col0 + threadIdx.x < a.vdim) {
        float s[MAPS] = {};
        for (uint32_t i = 0; i < groups; i++)
#pragma unroll
            for (int mp = 0; mp < MAPS; mp++) s[mp] += reinterpret_cast<const float*>(&sp.sums[mp][i * quads])[threadIdx.x];
        v = s[0] * sp.total[0];
        if constexpr (MAPS == 2) v -= a.lambda * (s[MAPS - 1] * sp.total[MAPS - 1]);
    }
    return v;
}

// One workgroup per (query row, head) and part of the columns: merges, norms or gates, and stores.
template <int MAPS>
__global__ __launch_bounds__(kMergeThreads) void attention_merge_kernel(const AttentionArgs a) {
    __shared__ MergeSpace<MAPS> space;
    __shared__ float scratch[kMergeThreads / 64];
    const uint32_t part = blockIdx.x % a.parts, th = blockIdx.x / a.parts, t = th / a.heads, h = th % a.heads;
    const uint32_t cols = a.dv / a.parts, d = part * cols + threadIdx.x;
    const float v = merge_columns<MAPS>(a, t, h, part * cols, cols, space);
    float f = 1.0f;
    if constexpr (MAPS == 2) f = rsqrtf(lh_block_sum(v * v, scratch) / (float)a.vdim + a.eps) * a.out_scale;
    if (MAPS == 1 && a.gate) f = lh_sigmoid(a.gate[(size_t)t * a.heads + h]);
    if (threadIdx.x < cols && d < a.vdim) static_cast<uint16_t*>(a.out)[((size_t)t * a.heads + h) * a.vdim + d] = lh_f2bf(v * f);
}

template <int MAPS>
int launch_merge(lh_context* ctx, AttentionArgs& a, const char* op) {
    a.parts = 1;                                              // two maps: the norm needs all columns
    if (MAPS == 1) while (a.dv / a.parts > 64 && (uint64_t)a.rows * a.heads * a.parts * 2 <= (uint64_t)ctx->cu_count) a.parts *= 2;
    hipLaunchKernelGGL((attention_merge_kernel<MAPS>), dim3(a.rows * a.heads * a.parts), dim3(kMergeThreads), 0, ctx->stream, a);
    return lh_check_launch(op);
}

// One workgroup per (query row, head), 256 keys at a time; f32 arithmetic throughout.
// TQ: type of the queries.
template <typename TQ, typename T>
__global__ __launch_bounds__(256) void attention_plain_kernel(const AttentionArgs a) {
    extern __shared__ float dyn[];                            // the query's maps * dim values
    __shared__ float p[2][256], scratch[4];
    const uint32_t t = blockIdx.x / a.heads, h = blockIdx.x % a.heads, g = h / (a.heads / a.kv_heads), tid = threadIdx.x;
    const uint32_t start = *a.position, last = min(start + t, a.capacity - 1);
    const TQ* q = static_cast<const TQ*>(a.q) + ((size_t)t * a.heads + h) * a.maps * a.dq;
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
            if (a.values_in_keys) {
                const T* v = static_cast<const T*>(a.keys) + (size_t)k0 * a.dq + d;
                for (uint32_t j = 0; j < n; j++) acc[0][i] = __builtin_fmaf(p[0][j], lh_ld(v, (size_t)j * a.dq), acc[0][i]);
                continue;
            }
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
    if (a.sink) {
        const float nm = fmaxf(m[0], a.sink[h]), alpha = expf(m[0] - nm);
        l[0] = l[0] * alpha + expf(a.sink[h] - nm);
#pragma unroll
        for (int i = 0; i < 4; i++) acc[0][i] *= alpha;
    }
    float v[4], ss = 0.0f;
#pragma unroll
    for (int i = 0; i < 4; i++) {
        v[i] = acc[0][i] / l[0];
        if (a.maps == 2) v[i] -= a.lambda * (acc[1][i] / l[1]);
        if (tid + i * 256 < a.vdim) ss += v[i] * v[i];
    }
    float f = 1.0f;
    if (a.gate) f = lh_sigmoid(a.gate[(size_t)t * a.heads + h]);
    if (a.maps == 2) f = rsqrtf(lh_block_sum(ss, scratch) / (float)a.vdim + a.eps) * a.out_scale;
#pragma unroll
    for (int i = 0; i < 4; i++)
        if (tid + i * 256 < a.vdim) lh_st(static_cast<T*>(a.out), ((size_t)t * a.heads + h) * a.vdim + tid + i * 256, v[i] * f);
}

constexpr uint32_t kMaxSplits = 512;

}  // namespace
