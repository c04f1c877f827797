// Mixture of experts with sigmoid scores: every row goes to its `top` best experts, and what enters an expert is scaled by
// the score itself.  The first product of an expert is linear, so the weight
// is applied to that product's result, before the activation.
//
// Many rows: route_kernel picks the experts of every row (one wave per row), place_kernel groups the (row, choice) slots by
// expert in row order (one workgroup per expert, no atomics: the order is fixed) and lays out the row tiles, and the two
// products run on those tiles (float_linear.hip).  One row: both products select the experts themselves from the logits.
//
// Plan layout (u32 words), S = rows * top slots, T = S / tile + experts tiles:
//   [0, S)       expert of slot (row, choice)          [S, 2S)      its weight (f32 bits)
//   [2S, 3S)     plan position of (row, choice)        [3S, 4S)     row of a plan position
//   [4S, 5S)     weight of a plan position             [5S, 5S + 3T) tiles: expert, first position, one past the last
#include "float_linear.hpp"
#include <algorithm>
#include <cstring>

namespace {

constexpr uint32_t kMaxExperts = 1024, kMaxTop = 64;

// The `top` largest of `experts` logits, best first, by one wave; ids and weights go to LDS or global memory.  (Sigmoid is
// monotone, so the logits decide; ties go to the lower index.)
template <uint32_t PER>
__device__ __forceinline__ void select_experts_of(const float* logits, uint32_t experts, uint32_t top, uint32_t lane, uint32_t* ids, float* weights) {
    float v[PER];
#pragma unroll
    for (uint32_t i = 0; i < PER; i++) v[i] = i * 64 + lane < experts ? logits[i * 64 + lane] : -INFINITY;
    for (uint32_t c = 0; c < top; c++) {
        float best = -INFINITY;
        uint32_t at = 0xFFFFFFFFu;
#pragma unroll
        for (uint32_t i = 0; i < PER; i++) if (v[i] > best) { best = v[i]; at = i * 64 + lane; }
        const float m = lh_group_max(best, 64);
        // the lowest index among the lanes that hold the maximum: a minimum as the maximum of the complements
        uint32_t win = ~lh_group_max_u(best == m && at != 0xFFFFFFFFu ? ~at : 0u, 64);
        if (win >= experts) win = min(c, experts - 1);        // no finite logit left
#pragma unroll
        for (uint32_t i = 0; i < PER; i++) if (i * 64 + lane == win) v[i] = -INFINITY;
        if (lane == 0) { ids[c] = win; weights[c] = lh_sigmoid(m); }
    }
}
__device__ void select_experts(const float* logits, uint32_t experts, uint32_t top, uint32_t lane, uint32_t* ids, float* weights) {
    if (experts <= 64) select_experts_of<1>(logits, experts, top, lane, ids, weights);
    else if (experts <= 256) select_experts_of<4>(logits, experts, top, lane, ids, weights);
    else select_experts_of<kMaxExperts / 64>(logits, experts, top, lane, ids, weights);
}

__global__ __launch_bounds__(256) void route_kernel(const float* __restrict__ logits, uint32_t* __restrict__ plan, uint32_t rows, uint32_t experts, uint32_t top) {
    __shared__ uint32_t ids[4][kMaxTop];
    __shared__ float weights[4][kMaxTop];
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6, row = blockIdx.x * 4 + wave, S = rows * top;
    if (row < rows) select_experts(logits + (size_t)row * experts, experts, top, lane, ids[wave], weights[wave]);
    __syncthreads();
    if (row < rows && lane < top) {
        plan[row * top + lane] = ids[wave][lane];
        plan[S + row * top + lane] = __builtin_bit_cast(uint32_t, weights[wave][lane]);
    }
}

__global__ __launch_bounds__(256) void place_kernel(uint32_t* __restrict__ plan, uint32_t rows, uint32_t experts, uint32_t top, uint32_t tile) {
    __shared__ uint32_t less[4], same[4];
    const uint32_t e = blockIdx.x, S = rows * top, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    uint32_t nl = 0, ns = 0;
    for (uint32_t i = threadIdx.x; i < S; i += 256) { const uint32_t x = plan[i]; nl += x < e; ns += x == e; }
    nl = (uint32_t)lh_group_sum_i((int)nl, 64);
    ns = (uint32_t)lh_group_sum_i((int)ns, 64);
    if (lane == 0) { less[wave] = nl; same[wave] = ns; }
    __syncthreads();
    const uint32_t base = less[0] + less[1] + less[2] + less[3], count = same[0] + same[1] + same[2] + same[3];
    uint32_t at = base;
    for (uint32_t i0 = 0; i0 < S; i0 += 256) {                // in slot order
        const uint32_t i = i0 + threadIdx.x;
        const bool mine = i < S && plan[i] == e;
        const uint64_t mask = __ballot(mine);
        __syncthreads();
        if (lane == 0) same[wave] = (uint32_t)__popcll(mask);
        __syncthreads();
        uint32_t before = at;
        for (uint32_t w = 0; w < wave; w++) before += same[w];
        if (mine) {
            const uint32_t p = before + (uint32_t)__popcll(mask & ((1ull << lane) - 1));
            plan[2 * S + i] = p;
            plan[3 * S + p] = i / top;
            plan[4 * S + p] = plan[S + i];
        }
        at += same[0] + same[1] + same[2] + same[3];
    }
    // expert e's tiles start at base / tile + e: there is always room for its ceil(count / tile) before the next expert's
    const uint32_t t0 = base / tile + e, t1 = (base + count) / tile + e + 1;
    for (uint32_t t = t0 + threadIdx.x; t < t1; t += 256) {
        const uint32_t b = min(base + (t - t0) * tile, base + count);
        uint32_t* w = plan + 5 * S + 3 * t;
        w[0] = e; w[1] = b; w[2] = min(b + tile, base + count);
    }
}

// residual[row] += the row's slots in choice order
__global__ __launch_bounds__(256) void combine_kernel(const float* __restrict__ slots, const uint32_t* __restrict__ plan, float* __restrict__ residual, uint32_t rows,
                                                     uint32_t top, uint32_t width) {
    const uint32_t row = blockIdx.x, S = rows * top;
    for (uint32_t i = threadIdx.x; i < width; i += 256) {
        float s = 0.0f;
        for (uint32_t c = 0; c < top; c++) s += slots[(size_t)plan[2 * S + row * top + c] * width + i];
        residual[(size_t)row * width + i] += s;
    }
}

// Dot product of one weight row with a vector in LDS, by a wave.
__device__ __forceinline__ float wave_dot(const uint16_t* __restrict__ w, const float* x, uint32_t K, uint32_t lane, bool vec) {
    float acc = 0.0f;
    if (vec) {
#pragma unroll 4
        for (uint32_t k = lane * 8; k < K; k += 512) {
            const uint4 v = *reinterpret_cast<const uint4*>(w + k);
            const float4 a = *reinterpret_cast<const float4*>(x + k), b = *reinterpret_cast<const float4*>(x + k + 4);
            acc = __builtin_fmaf(__builtin_bit_cast(float, v.x << 16), a.x, acc);
            acc = __builtin_fmaf(__builtin_bit_cast(float, v.x & 0xFFFF0000u), a.y, acc);
            acc = __builtin_fmaf(__builtin_bit_cast(float, v.y << 16), a.z, acc);
            acc = __builtin_fmaf(__builtin_bit_cast(float, v.y & 0xFFFF0000u), a.w, acc);
            acc = __builtin_fmaf(__builtin_bit_cast(float, v.z << 16), b.x, acc);
            acc = __builtin_fmaf(__builtin_bit_cast(float, v.z & 0xFFFF0000u), b.y, acc);
            acc = __builtin_fmaf(__builtin_bit_cast(float, v.w << 16), b.z, acc);
            acc = __builtin_fmaf(__builtin_bit_cast(float, v.w & 0xFFFF0000u), b.w, acc);
        }
    } else {
        for (uint32_t k = lane; k < K; k += 64) acc = __builtin_fmaf(lh_bf2f(w[k]), x[k], acc);
    }
    return lh_group_sum(acc, 64);
}

// hidden[c * ff + r] = act(weight_c * (up[e_c][r] . rms_norm(input)))
__global__ __launch_bounds__(256) void vector_up_kernel(const float* __restrict__ input, const float* __restrict__ norm_weight, float eps, const float* __restrict__ logits,
                                                       const uint16_t* __restrict__ up, float* __restrict__ hidden, uint32_t experts, uint32_t top, uint32_t width,
                                                       uint32_t ff, uint32_t act, uint32_t vec) {
    extern __shared__ __align__(16) float xs[];
    __shared__ uint32_t ids[kMaxTop];
    __shared__ float weights[kMaxTop], scratch[4];
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    float s = 0.0f;
    for (uint32_t k = threadIdx.x; k < width; k += 256) { const float v = input[k]; xs[k] = v; s += v * v; }
    const float r = rsqrtf(lh_block_sum(s, scratch) / (float)width + eps);
    for (uint32_t k = threadIdx.x; k < width; k += 256) xs[k] *= r * norm_weight[k];
    if (wave == 0) select_experts(logits, experts, top, lane, ids, weights);
    __syncthreads();
    const uint32_t total = top * ff;
    for (uint32_t i = blockIdx.x * 4 + wave; i < total; i += gridDim.x * 4) {
        const uint32_t c = i / ff, e = ids[c];
        const float v = wave_dot(up + ((size_t)e * ff + (i - c * ff)) * width, xs, width, lane, vec);
        if (lane == 0) hidden[i] = lh_activate(weights[c] * v, act);
    }
}

// The same with the normed vector in registers (width a multiple of 8, up to 512 * NL): a workgroup keeps to one expert's rows
// (blockIdx.y: the choice), and the first row's weights are requested as soon as the selection is known.
template <int NL>
__global__ __launch_bounds__(256) void vector_up_reg_kernel(const VectorStage st, const float* __restrict__ logits, const uint16_t* __restrict__ up,
                                                           float* __restrict__ hidden, uint32_t experts, uint32_t top, uint32_t width, uint32_t ff, uint32_t act) {
    __shared__ uint32_t ids[4][kMaxTop];
    __shared__ float weights[4][kMaxTop];
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c = blockIdx.y, last = (width >> 3) - 1;
    select_experts(logits, experts, c + 1, lane, ids[wave], weights[wave]);    // every wave for itself: no barrier
    const uint32_t e = ids[wave][c];
    const float weight = weights[wave][c];
    const uint16_t* base = up + (size_t)e * ff * width;
    uint32_t row = blockIdx.x * 4 + wave;
    uint4 w[NL];
    auto issue = [&](uint32_t r) {
#pragma unroll
        for (int i = 0; i < NL; i++) w[i] = lh_ld16_stream(base + (size_t)min(r, ff - 1) * width + 8 * min(64u * i + lane, last));
    };
    issue(row);
    float xr[NL][8];
    lh_vector_registers<kNorm, NL>(st, width, lane, false, xr);
    for (; row < ff; row += gridDim.x * 4) {
        float acc = 0.0f;
#pragma unroll
        for (int i = 0; i < NL; i++) acc = lh_dot8(w[i], xr[i], acc);
        if (row + gridDim.x * 4 < ff) issue(row + gridDim.x * 4);
        acc = lh_group_sum(acc, 64);
        if (lane == 0) hidden[c * ff + row] = lh_activate(weight * acc, act);
    }
}

// residual[r] += sum_c down[e_c][r] . hidden[c]
__global__ __launch_bounds__(256) void vector_down_kernel(const float* __restrict__ hidden, const float* __restrict__ logits, const uint16_t* __restrict__ down,
                                                         float* __restrict__ residual, uint32_t experts, uint32_t top, uint32_t width, uint32_t ff, uint32_t vec) {
    extern __shared__ __align__(16) float xs[];
    __shared__ uint32_t ids[kMaxTop];
    __shared__ float weights[kMaxTop];
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6, ffp = (ff + 3) / 4 * 4;   // a choice's values start 16-byte aligned
    for (uint32_t i = threadIdx.x; i < top * ff; i += 256) { const uint32_t c = i / ff; xs[c * ffp + (i - c * ff)] = hidden[i]; }
    if (wave == 0) select_experts(logits, experts, top, lane, ids, weights);
    __syncthreads();
    for (uint32_t n = blockIdx.x * 4 + wave; n < width; n += gridDim.x * 4) {
        float v = 0.0f;
        for (uint32_t c = 0; c < top; c++) v += wave_dot(down + ((size_t)ids[c] * width + n) * ff, xs + c * ffp, ff, lane, vec);
        if (lane == 0) residual[n] += v;
    }
}

// The same with the hidden values of all choices in registers as one vector of top * ff (ff a multiple of 8): a lane's chunk
// belongs to one choice, so it has its own place in the weights.
template <int NL>
__global__ __launch_bounds__(256) void vector_down_reg_kernel(const float* __restrict__ hidden, const float* __restrict__ logits, const uint16_t* __restrict__ down,
                                                             float* __restrict__ residual, uint32_t experts, uint32_t top, uint32_t width, uint32_t ff) {
    __shared__ uint32_t ids[4][kMaxTop];
    __shared__ float weights[4][kMaxTop];
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6, chunks = top * (ff >> 3), row_step = gridDim.x * 4;
    VectorStage st{};
    st.x = hidden; st.x_f32 = 1;
    float xr[NL][8];
    lh_vector_registers<kPlain, NL>(st, top * ff, lane, false, xr);
    select_experts(logits, experts, top, lane, ids[wave], weights[wave]);
    const uint16_t* base[NL];
#pragma unroll
    for (int i = 0; i < NL; i++) {
        const uint32_t q = min(64u * i + lane, chunks - 1), c = q / (ff >> 3);
        base[i] = down + (size_t)ids[wave][c] * width * ff + 8 * (q - c * (ff >> 3));
    }
    uint32_t n = blockIdx.x * 4 + wave;
    if (n >= width) return;
    uint4 w[NL];
    auto issue = [&](uint32_t r) {
#pragma unroll
        for (int i = 0; i < NL; i++) w[i] = lh_ld16_stream(base[i] + (size_t)r * ff);
    };
    issue(n);
    for (; n < width; n += row_step) {
        const float before = lane == 0 ? residual[n] : 0.0f;
        float acc = 0.0f;
#pragma unroll
        for (int i = 0; i < NL; i++) acc = lh_dot8(w[i], xr[i], acc);
        if (n + row_step < width) issue(n + row_step);
        acc = lh_group_sum(acc, 64);
        if (lane == 0) residual[n] = before + acc;
    }
}

int check_shape(const char* op, uint32_t rows, uint32_t experts, uint32_t top) {
    LH_REQUIRE(experts > 0 && experts <= kMaxExperts, "%s: %u experts outside 1..=%u", op, experts, kMaxExperts);
    LH_REQUIRE(top > 0 && top <= experts && top <= kMaxTop, "%s: top %u of %u experts", op, top, experts);
    LH_REQUIRE((uint64_t)rows * top < 0x10000000ull, "%s: %u rows", op, rows);
    return LH_OK;
}
uint32_t plan_tiles(uint32_t slots, uint32_t experts) { return slots / lh_expert_tile_rows(slots, experts) + experts; }

void expert_rows(LhExpertRows& x, const lh_buffer* plan, uint32_t rows, uint32_t experts, uint32_t top) {
    const uint32_t S = rows * top;
    const uint32_t* p = (const uint32_t*)plan->ptr;
    x.tiles = p + 5 * (size_t)S;
    x.n_tiles = plan_tiles(S, experts);
    x.tile_rows = lh_expert_tile_rows(S, experts);
    x.slot_row = p + 3 * (size_t)S;
    x.slot_weight = nullptr;
    x.experts = experts; x.slots = S; x.rows = rows;
}
#define LH_TRY(expr)                  \
    do {                              \
        const int rt__ = (expr);      \
        if (rt__ != LH_OK) return rt__; \
    } while (0)

int vector_lds(lh_context* ctx, const void* kernel, size_t bytes, const char* op) {
    LH_REQUIRE(bytes <= 144 * 1024, "%s: %zu values do not fit the staging memory", op, bytes / 4);
    return bytes > 60 * 1024 ? lh_raise_dynamic_lds(ctx, kernel, bytes, op) : LH_OK;
}

}  // namespace

extern "C" {

uint32_t lh_moe_plan_words(uint32_t rows, uint32_t experts, uint32_t top) {
    const uint32_t S = rows * top;
    return 5 * S + 3 * plan_tiles(S, experts);
}

int lh_moe_route_into(lh_batch* batch, const lh_buffer* logits, lh_buffer* plan, uint32_t rows, uint32_t experts, uint32_t top) {
    const char* op = "moe_route";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_TRY(check_shape(op, rows, experts, top));
    if (rows == 0) return LH_OK;
    LH_NEED(logits, (size_t)rows * experts * 4, op, "logits");
    LH_NEED(plan, (size_t)lh_moe_plan_words(rows, experts, top) * 4, op, "plan");
    hipLaunchKernelGGL(route_kernel, dim3((rows + 3) / 4), dim3(256), 0, batch->ctx->stream, (const float*)logits->ptr, (uint32_t*)plan->ptr, rows, experts, top);
    LH_TRY(lh_check_launch(op));
    hipLaunchKernelGGL(place_kernel, dim3(experts), dim3(256), 0, batch->ctx->stream, (uint32_t*)plan->ptr, rows, experts, top,
                       lh_expert_tile_rows(rows * top, experts));
    LH_TRY(lh_check_launch(op));
    batch->dispatch_count += 2;
    return LH_OK;
}

int lh_moe_up_into(lh_batch* batch, const lh_buffer* input, int dtype, const lh_buffer* plan, const lh_buffer* up, lh_buffer* hidden, uint32_t rows,
                   uint32_t experts, uint32_t top, uint32_t width, uint32_t ff, uint32_t act) {
    const char* op = "moe_up";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(dtype == LH_F32 || dtype == LH_BF16, "%s: dtype %d", op, dtype);
    LH_TRY(check_shape(op, rows, experts, top));
    LH_REQUIRE(width > 0 && ff > 0, "%s: width %u, ff %u", op, width, ff);
    if (rows == 0) return LH_OK;
    const size_t es = dtype == LH_F32 ? 4 : 2;
    LH_NEED(input, (size_t)rows * width * es, op, "input");
    LH_NEED(plan, (size_t)lh_moe_plan_words(rows, experts, top) * 4, op, "plan");
    LH_NEED(up, (size_t)experts * ff * width * 2, op, "up");
    LH_NEED(hidden, (size_t)rows * top * ff * es, op, "hidden");
    LhLinear a;
    memset(&a, 0, sizeof a);
    const uint32_t layout = LH_ROWS;
    lh_buffer* outs[1] = {hidden};
    LH_TRY(lh_make_segments(a.seg, op, rows * top, ff, 1, &ff, &act, &ff, &ff, &layout, outs, dtype, 0, nullptr));
    a.A = input->ptr; a.a_f32 = dtype == LH_F32; a.W = (const uint16_t*)up->ptr;
    a.M = rows * top; a.N = ff; a.K = width;
    expert_rows(a.ex, plan, rows, experts, top);
    a.ex.slot_weight = (const float*)plan->ptr + 4 * (size_t)(rows * top);
    a.ex.gather = 1;
    LH_TRY(lh_launch_linear(batch->ctx, a, op));
    batch->dispatch_count++;
    return LH_OK;
}

int lh_moe_down_into(lh_batch* batch, const lh_buffer* hidden, int dtype, const lh_buffer* plan, const lh_buffer* down, lh_buffer* slots, lh_buffer* residual,
                     uint32_t rows, uint32_t experts, uint32_t top, uint32_t width, uint32_t ff) {
    const char* op = "moe_down";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(dtype == LH_F32 || dtype == LH_BF16, "%s: dtype %d", op, dtype);
    LH_TRY(check_shape(op, rows, experts, top));
    LH_REQUIRE(width > 0 && ff > 0, "%s: width %u, ff %u", op, width, ff);
    if (rows == 0) return LH_OK;
    const size_t es = dtype == LH_F32 ? 4 : 2;
    LH_NEED(hidden, (size_t)rows * top * ff * es, op, "hidden");
    LH_NEED(plan, (size_t)lh_moe_plan_words(rows, experts, top) * 4, op, "plan");
    LH_NEED(down, (size_t)experts * ff * width * 2, op, "down");
    LH_NEED(residual, (size_t)rows * width * 4, op, "residual");
    const bool direct = top == 1;                            // one slot per row: add it where it belongs
    if (!direct) LH_NEED(slots, (size_t)rows * top * width * 4, op, "slots");
    LhLinear a;
    memset(&a, 0, sizeof a);
    const uint32_t layout = LH_ROWS, act = LH_ACT_NONE;
    lh_buffer* outs[1] = {direct ? residual : slots};
    LH_TRY(lh_make_segments(a.seg, op, rows * top, width, 1, &width, &act, &width, &width, &layout, outs, LH_F32, direct, nullptr));
    a.A = hidden->ptr; a.a_f32 = dtype == LH_F32; a.W = (const uint16_t*)down->ptr;
    a.M = rows * top; a.N = width; a.K = ff;
    expert_rows(a.ex, plan, rows, experts, top);
    a.ex.scatter = direct;
    LH_TRY(lh_launch_linear(batch->ctx, a, op));
    batch->dispatch_count++;
    if (direct) return LH_OK;
    hipLaunchKernelGGL(combine_kernel, dim3(rows), dim3(256), 0, batch->ctx->stream, (const float*)slots->ptr, (const uint32_t*)plan->ptr, (float*)residual->ptr, rows,
                       top, width);
    LH_TRY(lh_check_launch(op));
    batch->dispatch_count++;
    return LH_OK;
}

int lh_moe_vector_up_into(lh_batch* batch, const lh_buffer* input, const lh_buffer* norm_weight, float eps, const lh_buffer* logits, const lh_buffer* up,
                          lh_buffer* hidden, uint32_t experts, uint32_t top, uint32_t width, uint32_t ff, uint32_t act) {
    const char* op = "moe_vector_up";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_TRY(check_shape(op, 1, experts, top));
    LH_REQUIRE(width > 0 && ff > 0 && act <= LH_ACT_SIGMOID, "%s: width %u, ff %u, activation %u", op, width, ff, act);
    LH_NEED(input, (size_t)width * 4, op, "input");
    LH_NEED(norm_weight, (size_t)width * 4, op, "norm_weight");
    LH_NEED(logits, (size_t)experts * 4, op, "logits");
    LH_NEED(up, (size_t)experts * ff * width * 2, op, "up");
    LH_NEED(hidden, (size_t)top * ff * 4, op, "hidden");
    VectorStage st{};
    st.x = input->ptr; st.x_f32 = 1; st.norm_weight = (const float*)norm_weight->ptr; st.eps = eps;
    if (width % 8 == 0 && width <= 4096 && ((uintptr_t)up->ptr & 15) == 0 && lh_stage_aligned(st)) {
        const dim3 grid(std::min<uint32_t>((ff + 3) / 4, std::max<uint32_t>(1, (uint32_t)batch->ctx->cu_count * 4 / top)), top);
#define LH_UP(NL) hipLaunchKernelGGL((vector_up_reg_kernel<NL>), grid, dim3(256), 0, batch->ctx->stream, st, (const float*)logits->ptr, (const uint16_t*)up->ptr, \
                                     (float*)hidden->ptr, experts, top, width, ff, act)
        if (width <= 512) LH_UP(1);
        else if (width <= 1024) LH_UP(2);
        else if (width <= 2048) LH_UP(4);
        else LH_UP(8);
#undef LH_UP
        LH_TRY(lh_check_launch(op));
        batch->dispatch_count++;
        return LH_OK;
    }
    const size_t lds = (size_t)width * 4;
    LH_TRY(vector_lds(batch->ctx, (const void*)vector_up_kernel, lds, op));
    const uint32_t grid = (uint32_t)std::min<uint64_t>(((uint64_t)top * ff + 3) / 4, (uint64_t)batch->ctx->cu_count * 4);
    hipLaunchKernelGGL(vector_up_kernel, dim3(grid), dim3(256), lds, batch->ctx->stream, (const float*)input->ptr, (const float*)norm_weight->ptr, eps,
                       (const float*)logits->ptr, (const uint16_t*)up->ptr, (float*)hidden->ptr, experts, top, width, ff, act,
                       (uint32_t)(width % 8 == 0 && ((uintptr_t)up->ptr & 15) == 0));
    LH_TRY(lh_check_launch(op));
    batch->dispatch_count++;
    return LH_OK;
}

int lh_moe_vector_down_into(lh_batch* batch, const lh_buffer* hidden, const lh_buffer* logits, const lh_buffer* down, lh_buffer* residual, uint32_t experts,
                            uint32_t top, uint32_t width, uint32_t ff) {
    const char* op = "moe_vector_down";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_TRY(check_shape(op, 1, experts, top));
    LH_REQUIRE(width > 0 && ff > 0, "%s: width %u, ff %u", op, width, ff);
    LH_NEED(hidden, (size_t)top * ff * 4, op, "hidden");
    LH_NEED(logits, (size_t)experts * 4, op, "logits");
    LH_NEED(down, (size_t)experts * ff * width * 2, op, "down");
    LH_NEED(residual, (size_t)width * 4, op, "residual");
    if (ff % 8 == 0 && (uint64_t)top * ff <= 4096 && (((uintptr_t)down->ptr | (uintptr_t)hidden->ptr) & 15) == 0) {
        const uint32_t blocks = (uint32_t)std::min<uint64_t>(((uint64_t)width + 3) / 4, (uint64_t)batch->ctx->cu_count * 4);
#define LH_DOWN(NL) hipLaunchKernelGGL((vector_down_reg_kernel<NL>), dim3(blocks), dim3(256), 0, batch->ctx->stream, (const float*)hidden->ptr, (const float*)logits->ptr, \
                                       (const uint16_t*)down->ptr, (float*)residual->ptr, experts, top, width, ff)
        if (top * ff <= 512) LH_DOWN(1);
        else if (top * ff <= 1024) LH_DOWN(2);
        else if (top * ff <= 2048) LH_DOWN(4);
        else LH_DOWN(8);
#undef LH_DOWN
        LH_TRY(lh_check_launch(op));
        batch->dispatch_count++;
        return LH_OK;
    }
    const size_t lds = (size_t)top * ((ff + 3) / 4 * 4) * 4;
    LH_TRY(vector_lds(batch->ctx, (const void*)vector_down_kernel, lds, op));
    const uint32_t grid = (uint32_t)std::min<uint64_t>(((uint64_t)width + 3) / 4, (uint64_t)batch->ctx->cu_count * 4);
    hipLaunchKernelGGL(vector_down_kernel, dim3(grid), dim3(256), lds, batch->ctx->stream, (const float*)hidden->ptr, (const float*)logits->ptr,
                       (const uint16_t*)down->ptr, (float*)residual->ptr, experts, top, width, ff, (uint32_t)(ff % 8 == 0 && ((uintptr_t)down->ptr & 15) == 0));
    LH_TRY(lh_check_launch(op));
    batch->dispatch_count++;
    return LH_OK;
}

}  // extern "C"
