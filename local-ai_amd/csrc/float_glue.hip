// Row kernels around the products of models with bf16 weights: embedding gather, RMS norms of the f32 residual stream,
// the gated norm of a linear-attention layer, position counter and argmax.  One workgroup per row, f32 arithmetic.
#include "float_ops.hpp"
#include <cstring>

namespace {

__global__ __launch_bounds__(256) void embed_rows_kernel(const uint16_t* __restrict__ table, uint32_t table_rows, uint32_t cols,
                                                        const uint32_t* __restrict__ rows, float* __restrict__ out) {
    const uint32_t r = rows[blockIdx.x], src = r < table_rows ? r : table_rows - 1;
    for (uint32_t i = threadIdx.x; i < cols; i += blockDim.x) out[(size_t)blockIdx.x * cols + i] = lh_bf2f(table[(size_t)src * cols + i]);
}

// VEC: dim a multiple of 4 and at most 4 * 4 * blockDim (a thread keeps its elements between the two passes).
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void norm_rows_kernel(const float* in, const float* __restrict__ add, const float* __restrict__ w, float* store,   // store may be in
                                                       const uint32_t* __restrict__ index, uint32_t index_limit, T* __restrict__ out, uint32_t dim, float eps) {
    __shared__ float scratch[4];
    uint32_t src = blockIdx.x;
    if (index) { src = index[blockIdx.x]; src = src < index_limit ? src : index_limit - 1; }
    const size_t base = (size_t)src * dim, obase = (size_t)blockIdx.x * dim;
    float s = 0.0f;
    if constexpr (VEC) {
        float4 v[4], g[4];
#pragma unroll
        for (int it = 0; it < 4; it++) {
            const uint32_t i = (threadIdx.x + it * blockDim.x) * 4;
            v[it] = g[it] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (i >= dim) break;
            v[it] = *reinterpret_cast<const float4*>(in + base + i);
            g[it] = *reinterpret_cast<const float4*>(w + i);
            if (add) { const float4 b = *reinterpret_cast<const float4*>(add + base + i); v[it].x += b.x; v[it].y += b.y; v[it].z += b.z; v[it].w += b.w; }
            if (store) *reinterpret_cast<float4*>(store + base + i) = v[it];
            s += v[it].x * v[it].x + v[it].y * v[it].y + v[it].z * v[it].z + v[it].w * v[it].w;
        }
        const float r = rsqrtf(lh_block_sum(s, scratch) / (float)dim + eps);
#pragma unroll
        for (int it = 0; it < 4; it++) {
            const uint32_t i = (threadIdx.x + it * blockDim.x) * 4;
            if (i >= dim) break;
            const float a = v[it].x * r * g[it].x, b = v[it].y * r * g[it].y, c = v[it].z * r * g[it].z, d = v[it].w * r * g[it].w;
            if constexpr (sizeof(T) == 4) *reinterpret_cast<float4*>(out + obase + i) = make_float4(a, b, c, d);
            else *reinterpret_cast<uint2*>(out + obase + i) = make_uint2(lh_pack_bf(a, b), lh_pack_bf(c, d));
        }
    } else {
        for (uint32_t i = threadIdx.x; i < dim; i += blockDim.x) {
            float v = in[base + i];
            if (add) v += add[base + i];
            if (store) store[base + i] = v;
            s += v * v;
        }
        const float r = rsqrtf(lh_block_sum(s, scratch) / (float)dim + eps);
        for (uint32_t i = threadIdx.x; i < dim; i += blockDim.x) {   // a thread reads back what it stored itself
            float v = store ? store[base + i] : in[base + i];
            if (add && !store) v += add[base + i];
            lh_st(out, obase + i, v * r * w[i]);
        }
    }
}

// A residual branch whose norm comes behind it: store = x + rms_norm(branch) * w, and a copy of the sum in the dtype the next
// product reads.  Without a branch only the copy is made.  VEC as above.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void residual_rows_kernel(const float* x, const float* __restrict__ branch, const float* __restrict__ w, float* store,   // store may be x
                                                           T* __restrict__ out, uint32_t dim, float eps) {
    __shared__ float scratch[4];
    const size_t base = (size_t)blockIdx.x * dim;
    float s = 0.0f;
    if constexpr (VEC) {
        float4 v[4], y[4];
#pragma unroll
        for (int it = 0; it < 4; it++) {
            const uint32_t i = (threadIdx.x + it * blockDim.x) * 4;
            v[it] = y[it] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (i >= dim) break;
            v[it] = *reinterpret_cast<const float4*>(x + base + i);
            if (!branch) continue;
            const float4 b = *reinterpret_cast<const float4*>(branch + base + i), g = *reinterpret_cast<const float4*>(w + i);
            s += b.x * b.x + b.y * b.y + b.z * b.z + b.w * b.w;
            y[it] = make_float4(b.x * g.x, b.y * g.y, b.z * g.z, b.w * g.w);
        }
        const float r = branch ? rsqrtf(lh_block_sum(s, scratch) / (float)dim + eps) : 0.0f;
#pragma unroll
        for (int it = 0; it < 4; it++) {
            const uint32_t i = (threadIdx.x + it * blockDim.x) * 4;
            if (i >= dim) break;
            const float4 t = make_float4(__builtin_fmaf(y[it].x, r, v[it].x), __builtin_fmaf(y[it].y, r, v[it].y), __builtin_fmaf(y[it].z, r, v[it].z), __builtin_fmaf(y[it].w, r, v[it].w));
            if (store) *reinterpret_cast<float4*>(store + base + i) = t;
            if (!out) continue;
            if constexpr (sizeof(T) == 4) *reinterpret_cast<float4*>(out + base + i) = t;
            else *reinterpret_cast<uint2*>(out + base + i) = make_uint2(lh_pack_bf(t.x, t.y), lh_pack_bf(t.z, t.w));
        }
    } else {
        if (branch) for (uint32_t i = threadIdx.x; i < dim; i += blockDim.x) { const float b = branch[base + i]; s += b * b; }
        const float r = branch ? rsqrtf(lh_block_sum(s, scratch) / (float)dim + eps) : 0.0f;
        for (uint32_t i = threadIdx.x; i < dim; i += blockDim.x) {
            const float t = branch ? __builtin_fmaf(branch[base + i] * w[i], r, x[base + i]) : x[base + i];
            if (store) store[base + i] = t;
            if (out) lh_st(out, base + i, t);
        }
    }
}

// RMS norm in parts of `group` columns with a gate, which multiplies before the norm (gate_first) or after it.
// WAVE: a wave per part, no barrier; else the workgroup takes one part after the other.
template <typename T, bool WAVE>
__global__ __launch_bounds__(256) void gated_norm_rows_kernel(const float* __restrict__ in, const T* __restrict__ gate, const float* __restrict__ w, T* __restrict__ out,
                                                             uint32_t dim, uint32_t group, uint32_t gate_act, uint32_t gate_first, float eps) {
    __shared__ float scratch[4];
    const size_t base = (size_t)blockIdx.x * dim;
    const uint32_t first = WAVE ? threadIdx.x & 63 : threadIdx.x, step = WAVE ? 64 : blockDim.x;
    for (uint32_t g0 = WAVE ? (threadIdx.x >> 6) * group : 0; g0 < dim; g0 += WAVE ? 4 * group : group) {
        constexpr int R = 16;                                 // elements a thread keeps between the passes; the rest are read again
        float keep[R], gt[R], s = 0.0f;
        auto value = [&](uint32_t i, float& f) {
            f = lh_gate(lh_ld(gate, base + i), gate_act);
            const float v = in[base + i];
            return gate_first ? v * f : v;
        };
#pragma unroll
        for (int j = 0; j < R; j++) {
            const uint32_t i = first + j * step;
            keep[j] = 0.0f; gt[j] = 1.0f;
            if (i < group) keep[j] = value(g0 + i, gt[j]);
            s += keep[j] * keep[j];
        }
        for (uint32_t i = first + R * step; i < group; i += step) { float f; const float v = value(g0 + i, f); s += v * v; }
        s = WAVE ? lh_group_sum(s, 64) : lh_block_sum(s, scratch);
        const float r = rsqrtf(s / (float)group + eps);
        auto put = [&](uint32_t i, float v, float f) { lh_st(out, base + i, v * r * (w ? w[i] : 1.0f) * (gate_first ? 1.0f : f)); };
#pragma unroll
        for (int j = 0; j < R; j++) if (first + j * step < group) put(g0 + first + j * step, keep[j], gt[j]);
        for (uint32_t i = first + R * step; i < group; i += step) { float f; const float v = value(g0 + i, f); put(g0 + i, v, f); }
    }
}

__global__ __launch_bounds__(256) void softcap_kernel(float* x, size_t n, float cap) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i < n) x[i] = cap * tanhf(x[i] / cap);
}

__global__ void advance_position_kernel(uint32_t* position, uint32_t by) { *position += by; }

__global__ __launch_bounds__(1024) void argmax_rows_kernel(const float* __restrict__ x, uint32_t* __restrict__ index, uint32_t n) {
    __shared__ float sv[1024];
    __shared__ uint32_t si[1024];
    const float* row = x + (size_t)blockIdx.x * n;
    float best = -INFINITY;
    uint32_t at = 0xFFFFFFFFu;
    for (uint32_t i0 = threadIdx.x; i0 < n; i0 += 16 * 1024) {   // sixteen loads on their way at a time
        float v[16];
#pragma unroll
        for (uint32_t j = 0; j < 16; j++) v[j] = row[min(i0 + j * 1024, n - 1)];
#pragma unroll
        for (uint32_t j = 0; j < 16; j++) if (i0 + j * 1024 < n && (v[j] > best || at == 0xFFFFFFFFu)) { best = v[j]; at = i0 + j * 1024; }
    }
    sv[threadIdx.x] = best; si[threadIdx.x] = at;
    __syncthreads();
    for (uint32_t h = 512; h > 0; h >>= 1) {
        if (threadIdx.x < h) {
            const float v = sv[threadIdx.x + h];
            const uint32_t i = si[threadIdx.x + h];
            if (i != 0xFFFFFFFFu && (si[threadIdx.x] == 0xFFFFFFFFu || v > sv[threadIdx.x] || (v == sv[threadIdx.x] && i < si[threadIdx.x]))) { sv[threadIdx.x] = v; si[threadIdx.x] = i; }
        }
        __syncthreads();
    }
    if (threadIdx.x == 0) index[blockIdx.x] = si[0];
}

int done(lh_batch* batch, const char* op) {
    const int r = lh_check_launch(op);
    if (r == LH_OK) batch->dispatch_count++;
    return r;
}

}  // namespace

static inline bool lh_segment_at(uint32_t layout) { return layout == LH_ROWS_AT_POSITION || layout == LH_BLOCKS_AT_POSITION; }

int lh_make_segments(LhSegments& s, const char* op, uint32_t m, uint32_t n_total, uint32_t count, const uint32_t* ns, const uint32_t* acts,
                     const uint32_t* heads, const uint32_t* padded, const uint32_t* layouts, lh_buffer* const* outputs, int output_dtype,
                     int accumulate, const lh_buffer* position) {
    LH_REQUIRE(count >= 1 && count <= 4, "%s: %u segments", op, count);
    LH_REQUIRE(ns && acts && heads && padded && layouts && outputs, "%s: null argument", op);
    LH_REQUIRE(output_dtype == LH_F32 || output_dtype == LH_BF16, "%s: output dtype %d must be f32 or bf16", op, output_dtype);
    LH_REQUIRE(!accumulate || output_dtype == LH_F32, "%s: only f32 outputs accumulate", op);
    memset(&s, 0, sizeof s);
    s.count = count;
    s.accumulate = accumulate != 0;
    uint64_t n = 0;
    bool at_position = false;
    s.aligned4 = 1;
    for (uint32_t i = 0; i < count; i++) {
        LH_REQUIRE(ns[i] > 0 && heads[i] > 0 && ns[i] % heads[i] == 0 && padded[i] >= heads[i], "%s: segment %u: %u columns in heads of %u padded to %u",
                   op, i, ns[i], heads[i], padded[i]);
        LH_REQUIRE(acts[i] <= LH_ACT_SILU_PAIRS && layouts[i] <= LH_ROWS_F32, "%s: segment %u: activation %u, layout %u", op, i, acts[i], layouts[i]);
        const bool pairs = acts[i] == LH_ACT_SILU_PAIRS;
        LH_REQUIRE(!pairs || (ns[i] % 2 == 0 && n % 2 == 0 && heads[i] == padded[i] && (layouts[i] == LH_ROWS || layouts[i] == LH_ROWS_F32)),
                   "%s: segment %u: pairs need an even number of columns and plain rows", op, i);
        LH_REQUIRE(outputs[i] != nullptr, "%s: output %u is null", op, i);
        s.n0[i] = (uint32_t)n;
        n += ns[i];
        s.head[i] = heads[i]; s.padded[i] = padded[i]; s.act[i] = acts[i]; s.layout[i] = layouts[i];
        s.ld[i] = pairs ? ns[i] / 2 : ns[i] / heads[i] * padded[i];
        s.f32[i] = output_dtype == LH_F32 || layouts[i] == LH_ROWS_F32;
        s.pairs |= pairs;
        s.out[i] = outputs[i]->ptr;
        uint64_t rows = outputs[i]->len / ((s.f32[i] ? 4ull : 2ull) * s.ld[i]);
        if (layouts[i] == LH_BLOCKS_AT_POSITION) rows = rows / 32 * 32;
        if (!lh_segment_at(layouts[i])) LH_REQUIRE(rows >= m, "%s: output %u holds %llu rows of %u, needs %u", op, i, (unsigned long long)rows, s.ld[i], m);
        else at_position = true;
        s.rows[i] = rows > 0xFFFFFFFFull ? 0xFFFFFFFFu : (uint32_t)rows;
        s.aligned4 &= ns[i] % 4 == 0;
        s.vec4[i] = !pairs && heads[i] % 4 == 0 && padded[i] % 4 == 0 && layouts[i] != LH_BLOCKS_AT_POSITION && ((uintptr_t)s.out[i] & 15) == 0;
    }
    LH_REQUIRE(n == n_total || n_total == 0, "%s: segments cover %llu of %u columns", op, (unsigned long long)n, n_total);
    LH_REQUIRE(n < 0x7FFFFFFFull, "%s: %llu columns", op, (unsigned long long)n);
    for (uint32_t i = count; i < 5; i++) s.n0[i] = (uint32_t)n;
    if (at_position) { LH_NEED(position, 4, op, "position"); s.position = (const uint32_t*)position->ptr; }
    return LH_OK;
}

extern "C" {

int lh_embed_rows_bf16_into(lh_batch* batch, const lh_buffer* table, uint32_t table_rows, uint32_t cols, const lh_buffer* rows, uint32_t n_rows,
                            lh_buffer* output) {
    const char* op = "embed_rows_bf16";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(table_rows > 0 && cols > 0, "%s: empty table", op);
    if (n_rows == 0) return LH_OK;
    LH_NEED(table, (size_t)table_rows * cols * 2, op, "table");
    LH_NEED(rows, (size_t)n_rows * 4, op, "rows");
    LH_NEED(output, (size_t)n_rows * cols * 4, op, "output");
    hipLaunchKernelGGL(embed_rows_kernel, dim3(n_rows), dim3(256), 0, batch->ctx->stream, (const uint16_t*)table->ptr, table_rows, cols,
                       (const uint32_t*)rows->ptr, (float*)output->ptr);
    return done(batch, op);
}

int lh_norm_rows_f32_into(lh_batch* batch, const lh_buffer* input, const lh_buffer* add, const lh_buffer* weight, lh_buffer* store,
                          const lh_buffer* row_index, lh_buffer* output, int output_dtype, uint32_t dim, uint32_t rows, float eps) {
    const char* op = "norm_rows_f32";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(output_dtype == LH_F32 || output_dtype == LH_BF16, "%s: output dtype %d", op, output_dtype);
    LH_REQUIRE(dim > 0, "%s: dim is 0", op);
    LH_REQUIRE(!row_index || (!add && !store), "%s: picked rows are only normed", op);
    if (rows == 0) return LH_OK;
    LH_NEED(input, row_index ? (size_t)dim * 4 : (size_t)rows * dim * 4, op, "input");
    LH_NEED(weight, (size_t)dim * 4, op, "weight");
    LH_NEED(output, (size_t)rows * dim * (output_dtype == LH_F32 ? 4 : 2), op, "output");
    if (add) LH_NEED(add, (size_t)rows * dim * 4, op, "add");
    if (store) LH_NEED(store, (size_t)rows * dim * 4, op, "store");
    if (row_index) LH_NEED(row_index, (size_t)rows * 4, op, "row_index");
    const uint32_t limit = (uint32_t)(input->len / ((size_t)dim * 4));
    auto al = [](const lh_buffer* b) { return b == nullptr || ((uintptr_t)b->ptr & 15) == 0; };
    const bool vec = dim % 4 == 0 && dim <= 4096 && al(input) && al(add) && al(weight) && al(store) && al(output);
    const uint32_t threads = dim <= 256 ? 64 : dim <= 1024 ? 128 : 256;
#define LH_NORM(T, V)                                                                                                                             \
    hipLaunchKernelGGL((norm_rows_kernel<T, V>), dim3(rows), dim3(threads), 0, batch->ctx->stream, (const float*)input->ptr,                      \
                       add ? (const float*)add->ptr : nullptr, (const float*)weight->ptr, store ? (float*)store->ptr : nullptr,                   \
                       row_index ? (const uint32_t*)row_index->ptr : nullptr, limit, (T*)output->ptr, dim, eps)
    if (output_dtype == LH_F32) { if (vec) LH_NORM(float, true); else LH_NORM(float, false); }
    else { if (vec) LH_NORM(uint16_t, true); else LH_NORM(uint16_t, false); }
#undef LH_NORM
    return done(batch, op);
}

int lh_residual_rows_into(lh_batch* batch, const lh_buffer* input, const lh_buffer* branch, const lh_buffer* weight, lh_buffer* store, lh_buffer* output,
                          int output_dtype, uint32_t dim, uint32_t rows, float eps) {
    const char* op = "residual_rows";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(output_dtype == LH_F32 || output_dtype == LH_BF16, "%s: output dtype %d", op, output_dtype);
    LH_REQUIRE(dim > 0, "%s: dim is 0", op);
    if (rows == 0) return LH_OK;
    LH_NEED(input, (size_t)rows * dim * 4, op, "input");
    if (branch) { LH_NEED(branch, (size_t)rows * dim * 4, op, "branch"); LH_NEED(weight, (size_t)dim * 4, op, "weight"); }
    if (store) LH_NEED(store, (size_t)rows * dim * 4, op, "store");
    if (output) LH_NEED(output, (size_t)rows * dim * (output_dtype == LH_F32 ? 4 : 2), op, "output");
    auto al = [](const lh_buffer* b) { return b == nullptr || ((uintptr_t)b->ptr & 15) == 0; };
    const bool vec = dim % 4 == 0 && dim <= 4096 && al(input) && al(branch) && al(weight) && al(store) && al(output);
    const uint32_t threads = dim <= 256 ? 64 : dim <= 1024 ? 128 : 256;
#define LH_RESIDUAL(T, V)                                                                                                                   \
    hipLaunchKernelGGL((residual_rows_kernel<T, V>), dim3(rows), dim3(threads), 0, batch->ctx->stream, (const float*)input->ptr,            \
                       branch ? (const float*)branch->ptr : nullptr, branch ? (const float*)weight->ptr : nullptr,                          \
                       store ? (float*)store->ptr : nullptr, output ? (T*)output->ptr : nullptr, dim, eps)
    if (output_dtype == LH_F32) { if (vec) LH_RESIDUAL(float, true); else LH_RESIDUAL(float, false); }
    else { if (vec) LH_RESIDUAL(uint16_t, true); else LH_RESIDUAL(uint16_t, false); }
#undef LH_RESIDUAL
    return done(batch, op);
}

int lh_gated_norm_rows_into(lh_batch* batch, const lh_buffer* input, const lh_buffer* gate, uint32_t gate_act, int gate_first, const lh_buffer* weight,
                            lh_buffer* output, int dtype, uint32_t dim, uint32_t group, uint32_t rows, float eps) {
    const char* op = "gated_norm_rows";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(dtype == LH_F32 || dtype == LH_BF16, "%s: dtype %d", op, dtype);
    LH_REQUIRE(gate_act == LH_ACT_SIGMOID || gate_act == LH_ACT_SILU, "%s: gate activation %u", op, gate_act);
    LH_REQUIRE(dim > 0 && group > 0 && dim % group == 0, "%s: %u columns in parts of %u", op, dim, group);
    if (rows == 0) return LH_OK;
    const size_t es = dtype == LH_F32 ? 4 : 2;
    LH_NEED(input, (size_t)rows * dim * 4, op, "input");
    LH_NEED(gate, (size_t)rows * dim * es, op, "gate");
    if (weight) LH_NEED(weight, (size_t)dim * 4, op, "weight");
    LH_NEED(output, (size_t)rows * dim * es, op, "output");
    const bool wave = dim / group >= 4;
#define LH_GATED(T, W)                                                                                                                      \
    hipLaunchKernelGGL((gated_norm_rows_kernel<T, W>), dim3(rows), dim3(256), 0, batch->ctx->stream, (const float*)input->ptr,              \
                       (const T*)gate->ptr, weight ? (const float*)weight->ptr : nullptr, (T*)output->ptr, dim, group, gate_act,            \
                       (uint32_t)(gate_first != 0), eps)
    if (dtype == LH_F32) { if (wave) LH_GATED(float, true); else LH_GATED(float, false); }
    else { if (wave) LH_GATED(uint16_t, true); else LH_GATED(uint16_t, false); }
#undef LH_GATED
    return done(batch, op);
}

int lh_softcap_f32_into(lh_batch* batch, lh_buffer* logits, size_t n, float cap) {
    const char* op = "softcap_f32";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(cap > 0.0f, "%s: cap %g", op, (double)cap);
    if (n == 0) return LH_OK;
    LH_NEED(logits, n * 4, op, "logits");
    LH_REQUIRE((n + 255) / 256 < 0x7FFFFFFFull, "%s: %zu values", op, n);
    hipLaunchKernelGGL(softcap_kernel, dim3((uint32_t)((n + 255) / 256)), dim3(256), 0, batch->ctx->stream, (float*)logits->ptr, n, cap);
    return done(batch, op);
}

int lh_advance_position_into(lh_batch* batch, lh_buffer* position, uint32_t by) {
    LH_REQUIRE(batch, "advance_position: batch is null");
    LH_NEED(position, 4, "advance_position", "position");
    hipLaunchKernelGGL(advance_position_kernel, dim3(1), dim3(1), 0, batch->ctx->stream, (uint32_t*)position->ptr, by);
    return done(batch, "advance_position");
}

int lh_argmax_rows_f32_into(lh_batch* batch, const lh_buffer* logits, lh_buffer* index, uint32_t rows, uint32_t n) {
    const char* op = "argmax_rows_f32";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(n > 0, "%s: no columns", op);
    if (rows == 0) return LH_OK;
    LH_NEED(logits, (size_t)rows * n * 4, op, "logits");
    LH_NEED(index, (size_t)rows * 4, op, "index");
    hipLaunchKernelGGL(argmax_rows_kernel, dim3(rows), dim3(1024), 0, batch->ctx->stream, (const float*)logits->ptr, (uint32_t*)index->ptr, n);
    return done(batch, op);
}

}  // extern "C"
