// Shared pieces of the kernels that serve models with bf16 weights: element types, activations, and the description of
// where the columns of a product go.
#pragma once
#include "common.hpp"

typedef float lh_f32x4 __attribute__((ext_vector_type(4)));
typedef __bf16 lh_bf16x8 __attribute__((ext_vector_type(8)));

// Storage types of activations and caches: bf16 (raw bits) and f32.
__device__ __forceinline__ uint16_t lh_f2bf(float f) { return __builtin_bit_cast(uint16_t, (__bf16)f); }   // round to nearest even
__device__ __forceinline__ float lh_ld(const uint16_t* p, size_t i) { return lh_bf2f(p[i]); }
__device__ __forceinline__ float lh_ld(const float* p, size_t i) { return p[i]; }
__device__ __forceinline__ void lh_st(uint16_t* p, size_t i, float v) { p[i] = lh_f2bf(v); }
__device__ __forceinline__ void lh_st(float* p, size_t i, float v) { p[i] = v; }

__device__ __forceinline__ uint32_t lh_pack_bf(float a, float b) { return (uint32_t)lh_f2bf(a) | ((uint32_t)lh_f2bf(b) << 16); }

// x as the sum of bf16 terms, each the rounding of what the terms before it leave: two carry 16 bits of x, three all 24.
struct LhSplit3 { uint16_t hi, mid, lo; };
__device__ __forceinline__ LhSplit3 lh_split3(float x) {
    const uint16_t h = lh_f2bf(x);
    const float r = x - lh_bf2f(h);
    const uint16_t m = lh_f2bf(r);
    return LhSplit3{h, m, lh_f2bf(r - lh_bf2f(m))};
}

__device__ __forceinline__ float lh_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
// the tanh form of gelu as z times a sigmoid of twice the tanh's argument
__device__ __forceinline__ float lh_gelu_tanh(float z) {
    const float u = 0.7978845608028654f * (z + 0.044715f * z * z * z);
    return z / (1.0f + expf(-2.0f * u));
}
__device__ __forceinline__ float lh_activate(float v, uint32_t act) {
    switch (act) {
        case LH_ACT_SILU: return v * lh_sigmoid(v);
        case LH_ACT_GELU_TANH: return lh_gelu_tanh(v);
        case LH_ACT_RELU_SQUARED: { const float r = fmaxf(v, 0.0f); return r * r; }
        case LH_ACT_SIGMOID: return lh_sigmoid(v);
        default: return v;
    }
}
__device__ __forceinline__ float lh_gate(float g, uint32_t act) { const float s = lh_sigmoid(g); return act == LH_ACT_SILU ? g * s : s; }

// Inside a 32-position block of a value cache the positions are kept in the order in which a lane of the matrix product
// P V needs them: the scores of a 32-key step leave lane group g with keys 4g .. 4g + 3 of both 16-key tiles, so those
// eight are neighbours.
__host__ __device__ __forceinline__ uint32_t lh_block_slot(uint32_t p) { return ((p >> 2) & 3u) * 8u + ((p >> 4) & 1u) * 4u + (p & 3u); }

// Column ranges ("segments") of one stacked product, each with its own activation, destination and layout.
struct LhSegments {
    uint32_t count;
    uint32_t n0[5];                 // first column of each segment; n0[count] = all columns
    void* out[4];
    uint32_t ld[4];                 // columns of a destination row, padding included
    uint32_t head[4], padded[4];    // column n of the segment lands at (n / head) * padded + n % head
    uint32_t act[4];
    uint32_t layout[4];             // LH_ROWS, LH_ROWS_AT_POSITION, LH_BLOCKS_AT_POSITION, LH_ROWS_F32
    uint32_t rows[4];               // rows (positions) the destination holds: writes past it are dropped
    uint32_t f32[4];                // the destination is f32 (else bf16)
    uint32_t accumulate;            // add to the destination (f32 only)
    uint32_t aligned4;              // every boundary is a multiple of 4: four neighbouring columns are of one segment
    uint32_t vec4[4];               // and stay together in the destination
    uint32_t pairs;                 // some segment has LH_ACT_SILU_PAIRS
    const uint32_t* position;       // device word: position of row 0 (layouts AT_POSITION)
};
__device__ __forceinline__ bool lh_segment_at_position(const LhSegments& s, uint32_t i) {
    return s.layout[i] == LH_ROWS_AT_POSITION || s.layout[i] == LH_BLOCKS_AT_POSITION;
}
__device__ __forceinline__ uint32_t lh_segment_of(const LhSegments& s, uint32_t n) {
    uint32_t i = 0;
#pragma unroll
    for (uint32_t j = 1; j < 4; j++) if (j < s.count && n >= s.n0[j]) i = j;
    return i;
}
__device__ __forceinline__ void lh_segment_put(const LhSegments& s, uint32_t i, size_t idx, float v) {
    if (s.f32[i]) { float* o = static_cast<float*>(s.out[i]); o[idx] = s.accumulate ? o[idx] + v : v; }
    else static_cast<uint16_t*>(s.out[i])[idx] = lh_f2bf(v);
}
// Stores column n of row m (activation applied here); `pos0` is *s.position, or 0.
__device__ __forceinline__ void lh_segment_store(const LhSegments& s, uint32_t m, uint32_t n, float v, uint32_t pos0) {
    const uint32_t i = lh_segment_of(s, n);
    uint32_t c = n - s.n0[i];
    if (s.head[i] != s.padded[i]) { const uint32_t h = c / s.head[i]; c = h * s.padded[i] + (c - h * s.head[i]); }
    v = lh_activate(v, s.act[i]);
    const uint32_t p = lh_segment_at_position(s, i) ? pos0 + m : m;
    if (p >= s.rows[i]) return;
    const size_t idx = s.layout[i] == LH_BLOCKS_AT_POSITION ? ((size_t)(p >> 5) * s.ld[i] + c) * 32 + lh_block_slot(p & 31u) : (size_t)p * s.ld[i] + c;
    lh_segment_put(s, i, idx, v);
}
// Columns n and n + 1 (n even) of row m: a (gate, up) pair of an LH_ACT_SILU_PAIRS segment becomes one value.
__device__ __forceinline__ void lh_segment_store_pair(const LhSegments& s, uint32_t m, uint32_t n, float a, float b, uint32_t pos0) {
    const uint32_t i = lh_segment_of(s, n);
    if (s.act[i] == LH_ACT_SILU_PAIRS) { lh_segment_put(s, i, (size_t)m * s.ld[i] + (n - s.n0[i]) / 2, a * lh_sigmoid(a) * b); return; }
    lh_segment_store(s, m, n, a, pos0);
    lh_segment_store(s, m, n + 1, b, pos0);
}

// Host side of the above, from the arrays of the C ABI; validates every destination against its shape.
int lh_make_segments(LhSegments& s, const char* op, uint32_t m, uint32_t n_total, uint32_t count, const uint32_t* ns, const uint32_t* acts,
                     const uint32_t* heads, const uint32_t* padded, const uint32_t* layouts, lh_buffer* const* outputs, int output_dtype,
                     int accumulate, const lh_buffer* position);

// Sum over a workgroup of up to 16 waves.
__device__ __forceinline__ float lh_block_sum(float v, float* scratch) {
    v = lh_group_sum(v, 64);
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nwaves = (blockDim.x + 63) >> 6;
    if (lane == 0) scratch[wave] = v;
    __syncthreads();
    float t = 0.0f;
    for (int w = 0; w < nwaves; w++) t += scratch[w];
    __syncthreads();
    return t;
}

// Barrier over LDS accesses only: global loads that are on their way stay on their way.
__device__ __forceinline__ void lh_lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// Maximum and sum over the four lanes that differ in their 16s and 32s (the column of a 16 x 16 matrix-product tile).
// v_permlane16_swap / v_permlane32_swap on two copies leave the even and the odd rows (the lower and the upper half) of a
// value in all rows (both halves).
__device__ __forceinline__ void lh_pair16(float v, float& a, float& b) {
    const auto r = __builtin_amdgcn_permlane16_swap(__builtin_bit_cast(uint32_t, v), __builtin_bit_cast(uint32_t, v), false, false);
    const uint32_t x = r[0], y = r[1];      // (__builtin_bit_cast of a vector's element reads element 0, whichever is named)
    a = __builtin_bit_cast(float, x); b = __builtin_bit_cast(float, y);
}
__device__ __forceinline__ void lh_pair32(float v, float& a, float& b) {
    const auto r = __builtin_amdgcn_permlane32_swap(__builtin_bit_cast(uint32_t, v), __builtin_bit_cast(uint32_t, v), false, false);
    const uint32_t x = r[0], y = r[1];      // (__builtin_bit_cast of a vector's element reads element 0, whichever is named)
    a = __builtin_bit_cast(float, x); b = __builtin_bit_cast(float, y);
}
__device__ __forceinline__ float lh_column_max(float v) {
    float a, b;
    lh_pair16(v, a, b);
    lh_pair32(fmaxf(a, b), a, b);
    return fmaxf(a, b);
}
__device__ __forceinline__ float lh_column_sum(float v) {
    float a, b;
    lh_pair16(v, a, b);
    lh_pair32(a + b, a, b);
    return a + b;
}
