// Internal interface of the bf16-weight products (float_linear.hip) for the mixture-of-experts entries (float_moe.hip).
#pragma once
#include "float_ops.hpp"

// Rows of an expert product: the plan's tiles (see float_moe.hip), each `tile_rows` plan slots of one expert.
struct LhExpertRows {
    const uint32_t* tiles;          // null: an ordinary product.  [n_tiles][3]: expert, first slot, one past the last slot
    uint32_t n_tiles, tile_rows;    // 64 or 128
    const uint32_t* slot_row;       // slot -> row of the activations
    const float* slot_weight;       // slot -> weight of the expert's input (null: 1)
    uint32_t gather;                // activations are indexed by slot_row (else by the slot itself)
    uint32_t scatter;               // outputs go to slot_row (else to the slot itself)
    uint32_t experts, slots, rows;  // bounds of the above
};

struct LhLinear {
    const void* A;                  // [M, K], bf16 or f32, rows `lda` elements apart (0: K)
    uint32_t a_f32;
    const uint16_t* W;              // [N, K] (of every expert, one after the other)
    const float* bias;
    uint32_t M, N, K, lda;
    LhSegments seg;
    LhExpertRows ex;
};
int lh_launch_linear(lh_context* ctx, const LhLinear& a, const char* op);
uint32_t lh_expert_tile_rows(uint32_t slots, uint32_t experts);

// ---- one row: the activation vector in registers -------------------------------------------------------------------------
// Up to 4096 columns a wave keeps the vector itself: lane l holds the NL chunks of eight elements 8 (64 c + l), which is what
// it multiplies in every row.  The norm before the product is then a sum over the wave, with no barrier and no LDS.
enum { kPlain = 0, kNorm = 1, kGated = 2, kResidual = 3 };
struct VectorStage {
    const void* x;             // plain: x_f32 ? f32 : bf16; the others: f32
    uint32_t x_f32;
    const float* add;          // norm: may be null; residual: what is normed and added
    float* store;              // norm, residual: receives the sum (workgroup 0), may be null
    const float* norm_weight;  // gated: may be null
    const void* gate;          // gated
    uint32_t gate_f32, gate_act, gate_first, group;   // gated: the gate multiplies before the norm; elements per normed part
    float eps;
};

__device__ __forceinline__ void lh_ld8(const float* p, float (&v)[8]) {
    const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
    v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}
__device__ __forceinline__ void lh_ld8(const uint16_t* p, float (&v)[8]) {
    const uint4 a = *reinterpret_cast<const uint4*>(p);
    const uint32_t w[4] = {a.x, a.y, a.z, a.w};
#pragma unroll
    for (int j = 0; j < 4; j++) { v[2 * j] = __builtin_bit_cast(float, w[j] << 16); v[2 * j + 1] = __builtin_bit_cast(float, w[j] & 0xFFFF0000u); }
}

// K a multiple of 8, all pointers 16-byte aligned; chunks past K are zero.  `store` whether this wave stores x + add.
template <int STAGE, int NL>
__device__ __forceinline__ void lh_vector_registers(const VectorStage& st, uint32_t K, uint32_t lane, bool store, float (&xr)[NL][8]) {
    constexpr bool kNormed = STAGE == kNorm || STAGE == kGated || STAGE == kResidual;
    float w[kNormed ? NL : 1][8], s[kNormed ? NL : 1], total = 0.0f;
#pragma unroll
    for (int c = 0; c < NL; c++) {
        const uint32_t k = (64 * c + lane) * 8;
#pragma unroll
        for (int j = 0; j < 8; j++) xr[c][j] = 0.0f;
        if constexpr (kNormed) s[c] = 0.0f;
        if (k >= K) continue;
        if (STAGE == kPlain && !st.x_f32) lh_ld8(static_cast<const uint16_t*>(st.x) + k, xr[c]);
        else lh_ld8(static_cast<const float*>(st.x) + k, xr[c]);
        if constexpr (STAGE == kNorm) if (st.add) {
            float b[8];
            lh_ld8(st.add + k, b);
#pragma unroll
            for (int j = 0; j < 8; j++) xr[c][j] += b[j];
        }
        if constexpr (kNormed) {
            if (STAGE != kGated || st.norm_weight) lh_ld8(st.norm_weight + k, w[c]);
            else
#pragma unroll
                for (int j = 0; j < 8; j++) w[c][j] = 1.0f;
            if constexpr (STAGE == kGated) {
                float g[8];
                if (st.gate_f32) lh_ld8(static_cast<const float*>(st.gate) + k, g);
                else lh_ld8(static_cast<const uint16_t*>(st.gate) + k, g);
#pragma unroll
                for (int j = 0; j < 8; j++) {
                    const float f = lh_gate(g[j], st.gate_act);
                    if (st.gate_first) xr[c][j] *= f; else w[c][j] *= f;
                }
            }
            if constexpr (STAGE == kResidual) {               // w becomes the weighted branch
                float y[8];
                lh_ld8(st.add + k, y);
#pragma unroll
                for (int j = 0; j < 8; j++) { s[c] += y[j] * y[j]; w[c][j] *= y[j]; }
            } else
#pragma unroll
                for (int j = 0; j < 8; j++) s[c] += xr[c][j] * xr[c][j];
            total += s[c];
        }
    }
    if constexpr (kNormed) {
        float r[NL];
        if (STAGE == kGated && st.group != K) {               // group / 8 chunks: a power of two of lanes, or whole sets of 64
            const uint32_t cg = st.group >> 3;
#pragma unroll
            for (int c = 0; c < NL; c++) s[c] = lh_group_sum(s[c], (int)min(cg, 64u));
            const uint32_t per = cg > 64 ? cg >> 6 : 1u;
#pragma unroll
            for (int c = 0; c < NL; c++) {
                float t = 0.0f;
#pragma unroll
                for (int e = 0; e < NL; e++) t += (uint32_t)e / per == (uint32_t)c / per ? s[e] : 0.0f;
                r[c] = rsqrtf(t / (float)st.group + st.eps);
            }
        } else {
            const float all = rsqrtf(lh_group_sum(total, 64) / (float)K + st.eps);
#pragma unroll
            for (int c = 0; c < NL; c++) r[c] = all;
        }
#pragma unroll
        for (int c = 0; c < NL; c++) {
            const uint32_t k = (64 * c + lane) * 8;
            if (k >= K) continue;
            if constexpr (STAGE == kResidual)
#pragma unroll
                for (int j = 0; j < 8; j++) xr[c][j] = __builtin_fmaf(w[c][j], r[c], xr[c][j]);
            if (STAGE != kGated && store) {
                *reinterpret_cast<float4*>(st.store + k) = make_float4(xr[c][0], xr[c][1], xr[c][2], xr[c][3]);
                *reinterpret_cast<float4*>(st.store + k + 4) = make_float4(xr[c][4], xr[c][5], xr[c][6], xr[c][7]);
            }
            if constexpr (STAGE != kResidual)
#pragma unroll
                for (int j = 0; j < 8; j++) xr[c][j] = xr[c][j] * r[c] * w[c][j];
        }
    }
}
static inline bool lh_stage_aligned(const VectorStage& st) {
    return (((uintptr_t)st.x | (uintptr_t)st.add | (uintptr_t)st.store | (uintptr_t)st.norm_weight | (uintptr_t)st.gate) & 15) == 0;
}

// Weights are read once per launch: streaming loads.
__device__ __forceinline__ uint4 lh_ld16_stream(const uint16_t* p) {
    typedef uint32_t u32x4_t __attribute__((ext_vector_type(4)));
    const u32x4_t v = __builtin_nontemporal_load(reinterpret_cast<const u32x4_t*>(p));
    return make_uint4(v.x, v.y, v.z, v.w);
}
__device__ __forceinline__ float lh_dot8(const uint4& v, const float* x, float acc) {
    const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
    for (int j = 0; j < 4; j++) {
        acc = __builtin_fmaf(__builtin_bit_cast(float, w[j] << 16), x[2 * j], acc);
        acc = __builtin_fmaf(__builtin_bit_cast(float, w[j] & 0xFFFF0000u), x[2 * j + 1], acc);
    }
    return acc;
}
