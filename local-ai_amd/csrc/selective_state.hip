// Selective state space: the causal convolution in front of it, and the whole step for one row (the recurrence over many rows
// is in linear_attention.hip).  Per channel of [x | B | C] the last `taps` inputs are kept in a ring, row (position mod taps).
#include "float_ops.hpp"

namespace {

struct ConvArgs {
    const void* input;          // [rows, channels]
    float* ring;                // [taps, channels]
    const float *weight, *bias; // [taps, channels], [channels]
    const uint32_t* position;
    void *x, *b, *c;            // [rows, inner], [rows, groups, dq] twice
    uint32_t rows, channels, inner, groups, state, dq, taps;
    uint32_t tile;              // rows of a workgroup, taps - 1 at least
};
constexpr uint32_t kMaxTaps = 32;

// Where channel ch of row t goes.
template <typename T>
__device__ __forceinline__ T* conv_place(const ConvArgs& a, uint32_t ch, size_t t) {
    if (ch < a.inner) return static_cast<T*>(a.x) + t * a.inner + ch;
    const uint32_t n = a.groups * a.state, r = ch - a.inner, i = r < n ? r : r - n;
    return static_cast<T*>(r < n ? a.b : a.c) + (t * a.groups + i / a.state) * a.dq + i % a.state;
}

// Thread = channel, workgroup = a.tile rows.  Only the first rows' workgroup reads the ring, and it writes the ring
// afterwards (the inputs it keeps are those of the last rows, which nobody changes).  TAPS 0: any number.
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void conv_rows_kernel(const ConvArgs a) {
    const uint32_t ch = blockIdx.x * 256 + threadIdx.x, t0 = blockIdx.y * a.tile, t1 = min(t0 + a.tile, a.rows);
    if (ch >= a.channels) {                                   // the threads behind the channels clear the padding of B and C
        const uint32_t i = ch - a.channels, padding = a.dq - a.state;
        if (i < 2 * a.groups * padding) {
            T* d = static_cast<T*>(i < a.groups * padding ? a.b : a.c);
            const uint32_t j = i % (a.groups * padding);
            for (uint32_t t = t0; t < t1; t++) lh_st(d, ((size_t)t * a.groups + j / padding) * a.dq + a.state + j % padding, 0.0f);
        }
        return;
    }
    const uint32_t taps = TAPS ? TAPS : a.taps, pos0 = *a.position;
    const T* in = static_cast<const T*>(a.input) + ch;
    auto value = [&](int64_t t) {                             // the input of row t, rows before this portion from the ring
        if (t >= 0) return lh_ld(in, (size_t)t * a.channels);
        const int64_t p = (int64_t)pos0 + t;
        return p >= 0 ? a.ring[(size_t)(p % taps) * a.channels + ch] : 0.0f;
    };
    const float bias = a.bias[ch];
    T* out = conv_place<T>(a, ch, t0);
    const size_t step = ch < a.inner ? a.inner : (size_t)a.groups * a.dq;
    if constexpr (TAPS != 0) {
        float w[TAPS], v[TAPS];                               // v: the inputs of rows t - TAPS + 1 .. t
#pragma unroll
        for (int j = 0; j < TAPS; j++) { w[j] = a.weight[(size_t)j * a.channels + ch]; v[j] = j + 1 < TAPS ? value((int64_t)t0 + j + 1 - TAPS) : 0.0f; }
        // v[0 .. TAPS - 2] hold rows t0 - TAPS + 1 .. t0 - 1
        for (uint32_t t = t0; t < t1; t += 8) {
            float x[8];
#pragma unroll
            for (int i = 0; i < 8; i++) x[i] = t + i < t1 ? lh_ld(in, (size_t)(t + i) * a.channels) : 0.0f;
#pragma unroll
            for (int i = 0; i < 8; i++) {
                v[TAPS - 1] = x[i];
                float s = bias;
#pragma unroll
                for (int j = 0; j < TAPS; j++) s = __builtin_fmaf(w[j], v[j], s);
                if (t + i < t1) lh_st(out, (size_t)(t + i - t0) * step, s * lh_sigmoid(s));
#pragma unroll
                for (int j = 0; j + 1 < TAPS; j++) v[j] = v[j + 1];
            }
        }
    } else {
        for (uint32_t t = t0; t < t1; t++) {
            float s = bias;
            for (uint32_t j = 0; j < taps; j++) s = __builtin_fmaf(a.weight[(size_t)j * a.channels + ch], value((int64_t)t + j + 1 - taps), s);
            lh_st(out, (size_t)(t - t0) * step, s * lh_sigmoid(s));
        }
    }
    if (t0 == 0)
        for (uint32_t t = a.rows > taps ? a.rows - taps : 0; t < a.rows; t++) a.ring[(size_t)((pos0 + t) % taps) * a.channels + ch] = lh_ld(in, (size_t)t * a.channels);
}

struct StepArgs {
    ConvArgs conv;
    const float *dt_raw, *dt_bias, *a_log, *skip;
    float* memory;              // [heads, vdim, dq]
    float* out;                 // [heads * vdim]
    uint32_t heads, vdim;
};

__device__ __forceinline__ float softplus(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }

// A workgroup takes 16 value columns of a head, as recurrent_kernel does; the convolution of what it needs (its columns of x,
// the group's B and C) goes through LDS.  The ring row of the current position is not read, so it can be written in passing.
template <int NR>
__global__ __launch_bounds__(256) void selective_step_kernel(const StepArgs a) {
    extern __shared__ float bc[];                             // B [dq], C [dq], x [16]
    const ConvArgs& cv = a.conv;
    const uint32_t vt = (a.vdim + 15) / 16, h = blockIdx.x / vt, v0 = (blockIdx.x % vt) * 16, per = a.heads / cv.groups, g = h / per;
    const uint32_t slot = threadIdx.x >> 4, part = threadIdx.x & 15, k0 = part * NR, col = v0 + slot, dq = cv.dq;
    const bool on = col < a.vdim;
    float* st = a.memory + ((size_t)h * a.vdim + (on ? col : a.vdim - 1)) * dq + k0;
    float s[NR];
#pragma unroll
    for (int i = 0; i < NR; i++) s[i] = k0 + i < dq ? st[i] : 0.0f;
    const float dt = softplus(a.dt_raw[h] + a.dt_bias[h]), d = expf(-expf(a.a_log[h]) * dt), skip = a.skip[h];
    const uint32_t pos = *cv.position;
    for (uint32_t i = threadIdx.x; i < 2 * dq + 16; i += 256) {
        const uint32_t which = i < dq ? 0u : i < 2 * dq ? 1u : 2u, j = i - which * dq;
        const bool real = which < 2 ? j < cv.state : v0 + j < a.vdim;
        float y = 0.0f;
        if (real) {
            const uint32_t ch = which < 2 ? cv.inner + (which * cv.groups + g) * cv.state + j : h * a.vdim + v0 + j;
            const float now = static_cast<const float*>(cv.input)[ch];
            y = __builtin_fmaf(cv.weight[(size_t)(cv.taps - 1) * cv.channels + ch], now, cv.bias[ch]);
            for (uint32_t b = 1; b < cv.taps; b++)
                if (b <= pos) y = __builtin_fmaf(cv.weight[(size_t)(cv.taps - 1 - b) * cv.channels + ch], cv.ring[(size_t)((pos - b) % cv.taps) * cv.channels + ch], y);
            y *= lh_sigmoid(y);
            if (which == 2 || (h == g * per && v0 == 0)) cv.ring[(size_t)(pos % cv.taps) * cv.channels + ch] = now;
        }
        bc[i] = y;
    }
    __syncthreads();
    const float x = bc[2 * dq + slot], xd = dt * x;
    float o = 0.0f;
#pragma unroll
    for (int i = 0; i < NR; i++) {
        if (k0 + i >= dq) break;
        s[i] = __builtin_fmaf(bc[k0 + i], xd, d * s[i]);
        o = __builtin_fmaf(s[i], bc[dq + k0 + i], o);
        if (on) st[i] = s[i];
    }
    o = lh_group_sum(o, 16);
    if (part == 0 && on) a.out[(size_t)h * a.vdim + col] = __builtin_fmaf(skip, x, o);
}

int conv_args(ConvArgs& a, const char* op, const lh_buffer* input, size_t es, lh_buffer* ring, const lh_buffer* taps_weight, const lh_buffer* bias,
              const lh_buffer* position, uint32_t rows, uint32_t heads, uint32_t vdim, uint32_t groups, uint32_t state, uint32_t taps) {
    LH_REQUIRE(heads > 0 && groups > 0 && heads % groups == 0 && state > 0 && state <= 1024 && vdim > 0, "%s: heads %u over %u groups, state %u, vdim %u", op, heads,
               groups, state, vdim);
    LH_REQUIRE(taps >= 1 && taps <= kMaxTaps, "%s: %u taps", op, taps);
    const uint64_t channels = (uint64_t)heads * vdim + 2ull * groups * state;
    LH_REQUIRE(channels < 0x7FFFFFFull, "%s: %llu channels", op, (unsigned long long)channels);
    LH_NEED(input, (size_t)rows * channels * es, op, "input");
    LH_NEED(ring, (size_t)taps * channels * 4, op, "ring");
    LH_NEED(taps_weight, (size_t)taps * channels * 4, op, "taps_weight");
    LH_NEED(bias, (size_t)channels * 4, op, "bias");
    LH_NEED(position, 4, op, "position");
    a = ConvArgs{};
    a.input = input->ptr; a.ring = (float*)ring->ptr; a.weight = (const float*)taps_weight->ptr; a.bias = (const float*)bias->ptr;
    a.position = (const uint32_t*)position->ptr;
    a.rows = rows; a.channels = (uint32_t)channels; a.inner = heads * vdim; a.groups = groups; a.state = state;
    a.dq = lh_linear_attention_padded_dim(state); a.taps = taps;
    return LH_OK;
}

}  // namespace

extern "C" {

int lh_selective_conv_into(lh_batch* batch, const lh_buffer* input, int dtype, lh_buffer* ring, const lh_buffer* taps_weight, const lh_buffer* bias,
                           const lh_buffer* position, lh_buffer* x, lh_buffer* b, lh_buffer* c, uint32_t rows, uint32_t heads, uint32_t vdim, uint32_t groups,
                           uint32_t state, uint32_t taps) {
    const char* op = "selective_conv";
    LH_REQUIRE(batch, "%s: batch is null", op);
    LH_REQUIRE(dtype == LH_F32 || dtype == LH_BF16, "%s: dtype %d", op, dtype);
    if (rows == 0) return LH_OK;
    const size_t es = dtype == LH_F32 ? 4 : 2;
    ConvArgs a;
    const int r = conv_args(a, op, input, es, ring, taps_weight, bias, position, rows, heads, vdim, groups, state, taps);
    if (r != LH_OK) return r;
    LH_NEED(x, (size_t)rows * a.inner * es, op, "x");
    LH_NEED(b, (size_t)rows * groups * a.dq * es, op, "b");
    LH_NEED(c, (size_t)rows * groups * a.dq * es, op, "c");
    a.x = x->ptr; a.b = b->ptr; a.c = c->ptr;
    a.tile = taps > 17 ? 32 : 16;
    const uint32_t threads = a.channels + 2 * groups * (a.dq - state), tiles = (rows + a.tile - 1) / a.tile;
    LH_REQUIRE(tiles < 65536, "%s: %u rows", op, rows);
    const dim3 grid((threads + 255) / 256, tiles);
#define LH_CONV(T, N) hipLaunchKernelGGL((conv_rows_kernel<T, N>), grid, dim3(256), 0, batch->ctx->stream, a)
#define LH_CONV_T(T)                                                                                                  \
    do {                                                                                                              \
        if (taps == 2) LH_CONV(T, 2); else if (taps == 3) LH_CONV(T, 3); else if (taps == 4) LH_CONV(T, 4); else LH_CONV(T, 0); \
    } while (0)
    if (dtype == LH_F32) LH_CONV_T(float);
    else LH_CONV_T(uint16_t);
#undef LH_CONV_T
#undef LH_CONV
    const int rc = lh_check_launch(op);
    if (rc == LH_OK) batch->dispatch_count++;
    return rc;
}

int lh_selective_step_into(lh_batch* batch, const lh_buffer* input, lh_buffer* ring, const lh_buffer* taps_weight, const lh_buffer* bias,
                           const lh_buffer* position, const lh_buffer* dt_raw, const lh_buffer* dt_bias, const lh_buffer* a_log, const lh_buffer* skip,
                           lh_buffer* memory, lh_buffer* output, uint32_t heads, uint32_t vdim, uint32_t groups, uint32_t state, uint32_t taps) {
    const char* op = "selective_step";
    LH_REQUIRE(batch, "%s: batch is null", op);
    StepArgs a{};
    const int r = conv_args(a.conv, op, input, 4, ring, taps_weight, bias, position, 1, heads, vdim, groups, state, taps);
    if (r != LH_OK) return r;
    const uint32_t dq = a.conv.dq;
    LH_NEED(dt_raw, (size_t)heads * 4, op, "dt_raw");
    LH_NEED(dt_bias, (size_t)heads * 4, op, "dt_bias");
    LH_NEED(a_log, (size_t)heads * 4, op, "a_log");
    LH_NEED(skip, (size_t)heads * 4, op, "skip");
    LH_NEED(memory, (size_t)heads * vdim * dq * 4, op, "memory");
    LH_NEED(output, (size_t)heads * vdim * 4, op, "output");
    a.dt_raw = (const float*)dt_raw->ptr; a.dt_bias = (const float*)dt_bias->ptr; a.a_log = (const float*)a_log->ptr; a.skip = (const float*)skip->ptr;
    a.memory = (float*)memory->ptr; a.out = (float*)output->ptr; a.heads = heads; a.vdim = vdim;
    const uint64_t grid = (uint64_t)heads * ((vdim + 15) / 16);
    LH_REQUIRE(grid < 0x7FFFFFFFull, "%s: heads %u, vdim %u", op, heads, vdim);
    const size_t lds = (size_t)(2 * dq + 16) * 4;
#define LH_STEP(NR_) hipLaunchKernelGGL((selective_step_kernel<NR_>), dim3((uint32_t)grid), dim3(256), lds, batch->ctx->stream, a)
    if (dq <= 32) LH_STEP(2);
    else if (dq <= 64) LH_STEP(4);
    else if (dq <= 128) LH_STEP(8);
    else if (dq <= 256) LH_STEP(16);
    else if (dq <= 512) LH_STEP(32);
    else LH_STEP(64);
#undef LH_STEP
    const int rc = lh_check_launch(op);
    if (rc == LH_OK) batch->dispatch_count++;
    return rc;
}

}  // extern "C"
