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
    const void* A;                  // [M, K], bf16 or f32
    uint32_t a_f32;
    const uint16_t* W;              // [N, K] (of every expert, one after the other)
    const float* bias;
    uint32_t M, N, K;
    LhSegments seg;
    LhExpertRows ex;
};
int lh_launch_linear(lh_context* ctx, const LhLinear& a, const char* op);
uint32_t lh_expert_tile_rows(uint32_t slots, uint32_t experts);
