// What stands around a sublayer whose OUTPUT is normed before it joins the residual stream:
//     x <- x + mult * rmsnorm(scale_a * a + scale_b * b) * w
// (b optional: two branches that read the same input and are mixed with fixed weights), the rounded
// copy of the new x that the next sublayer's products read, and a gated linear unit with clamped
// halves. Sums and the residual stream are float32.
#include "fw_common.h"
#include "fw_kernels.h"

__device__ __forceinline__ float sublayer_sigmoid(float g) {
    if (g >= 0.0f) return 1.0f / (1.0f + expf(-g));
    const float e = expf(g);
    return e / (1.0f + e);
}

// One workgroup per row. y = scale_a a (+ scale_b b) is formed once and kept in registers (rows of up
// to 256 * NORM_ADD_HELD channels) or formed again in the second pass (wider rows).
#define NORM_ADD_HELD 16
template <typename T>
__global__ __launch_bounds__(256) void norm_scale_add_kernel(
    float* __restrict__ x, const float* __restrict__ a, const float* __restrict__ b, float scale_a, float scale_b,
    const float* __restrict__ weight, int one_centered, float eps, float mult, T* __restrict__ rounded, int hidden) {
    __shared__ float scratch[16];
    const size_t row0 = (size_t)blockIdx.x * hidden;
    const bool held_all = hidden <= 256 * NORM_ADD_HELD;
    float held[NORM_ADD_HELD], was[NORM_ADD_HELD], scale[NORM_ADD_HELD];
    float sum = 0.0f;
    if (held_all) {
        // everything the row needs is asked for at once: the old x and the weight travel with a and b
#pragma unroll
        for (int u = 0; u < NORM_ADD_HELD; ++u) {
            const int i = threadIdx.x + 256 * u;
            float y = 0.0f;
            was[u] = scale[u] = 0.0f;
            if (i < hidden) {
                y = scale_a * a[row0 + i];
                if (b) y = fmaf(scale_b, b[row0 + i], y);
                was[u] = x[row0 + i];
                scale[u] = weight[i];
            }
            held[u] = y;
            sum = fmaf(y, y, sum);
        }
    } else {
        for (int i = threadIdx.x; i < hidden; i += 256) {
            float y = scale_a * a[row0 + i];
            if (b) y = fmaf(scale_b, b[row0 + i], y);
            sum = fmaf(y, y, sum);
        }
    }
    sum = block_sum(sum, scratch);
    const float inv = 1.0f / sqrtf(sum / (float)hidden + eps);
    const float one = one_centered ? 1.0f : 0.0f;
    if (held_all) {
#pragma unroll
        for (int u = 0; u < NORM_ADD_HELD; ++u) {
            const int i = threadIdx.x + 256 * u;
            if (i < hidden) {
                const float updated = was[u] + mult * (held[u] * inv * (scale[u] + one));
                x[row0 + i] = updated;
                if (rounded) store_from_float(rounded, row0 + i, updated);
            }
        }
    } else {
        for (int i = threadIdx.x; i < hidden; i += 256) {
            float y = scale_a * a[row0 + i];
            if (b) y = fmaf(scale_b, b[row0 + i], y);
            const float updated = x[row0 + i] + mult * (y * inv * (weight[i] + one));
            x[row0 + i] = updated;
            if (rounded) store_from_float(rounded, row0 + i, updated);
        }
    }
}

extern "C" int fw_norm_scale_add(float* x, const float* a, const float* b, float scale_a, float scale_b, const float* weight,
                                 int one_centered, float eps, float mult, void* rounded, int rounded_dtype, int rows,
                                 int hidden, void* stream) {
    FW_REQUIRE(rows >= 0 && hidden > 0, "norm_scale_add: bad sizes rows=%d hidden=%d", rows, hidden);
    FW_REQUIRE(eps > 0.0f, "norm_scale_add: eps must be positive");
    FW_REQUIRE(x && a && weight, "norm_scale_add: x, a and the weight are needed");
    if (rows == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    if (!rounded || rounded_dtype == FW_F32)
        norm_scale_add_kernel<float><<<rows, 256, 0, s>>>(x, a, b, scale_a, scale_b, weight, one_centered, eps, mult, (float*)rounded, hidden);
    else if (rounded_dtype == FW_BF16)
        norm_scale_add_kernel<bf16_t><<<rows, 256, 0, s>>>(x, a, b, scale_a, scale_b, weight, one_centered, eps, mult, (bf16_t*)rounded, hidden);
    else
        FW_REQUIRE(false, "norm_scale_add: unknown dtype %d", rounded_dtype);
    FW_LAUNCH_CHECK("norm_scale_add");
    return 0;
}

// float32 rows rounded to the activation type
__global__ void round_rows_kernel(const float* __restrict__ x, bf16_t* __restrict__ out, long long count) {
    for (long long i = blockIdx.x * (long long)blockDim.x + threadIdx.x; i < count; i += (long long)gridDim.x * blockDim.x)
        out[i] = float_to_bf16(x[i]);
}

extern "C" int fw_round_rows(const float* x, void* out, long long count, void* stream) {
    FW_REQUIRE(count >= 0, "round_rows: negative count");
    if (count == 0) return 0;
    const int blocks = (int)((count + 255) / 256 < 4096 ? (count + 255) / 256 : 4096);
    round_rows_kernel<<<blocks, 256, 0, (hipStream_t)stream>>>(x, (bf16_t*)out, count);
    FW_LAUNCH_CHECK("round_rows");
    return 0;
}

// The same into some columns of wider rows: out[r][col0 .. col0 + hidden - 1] = x[r], and with `twice` once more `hidden`
// columns on (rows joined with themselves).
template <typename T>
__global__ __launch_bounds__(256) void place_rows_kernel(const float* __restrict__ x, int x_stride, T* __restrict__ out, int hidden, int out_stride,
                                                        int col0, int twice) {
    const int row = blockIdx.x;
    T* to = out + (size_t)row * out_stride + col0;
    for (int i = threadIdx.x; i < hidden; i += 256) {
        const float v = x[(size_t)row * x_stride + i];
        store_from_float(to, i, v);
        if (twice) store_from_float(to, hidden + i, v);
    }
}

extern "C" int fw_place_rows(const float* x, int x_stride, void* out, int out_dtype, int rows, int hidden, int out_stride, int col0, int twice,
                             void* stream) {
    FW_REQUIRE(x_stride >= hidden, "place_rows: rows of %d do not lie %d apart", hidden, x_stride);
    FW_REQUIRE(rows >= 0 && hidden > 0 && col0 >= 0 && col0 + (twice ? 2 : 1) * hidden <= out_stride,
               "place_rows: %d columns from %d on do not fit rows of %d", (twice ? 2 : 1) * hidden, col0, out_stride);
    if (rows == 0) return 0;
    if (out_dtype == FW_F32) place_rows_kernel<float><<<rows, 256, 0, (hipStream_t)stream>>>(x, x_stride, (float*)out, hidden, out_stride, col0, twice);
    else if (out_dtype == FW_BF16) place_rows_kernel<bf16_t><<<rows, 256, 0, (hipStream_t)stream>>>(x, x_stride, (bf16_t*)out, hidden, out_stride, col0, twice);
    else FW_REQUIRE(false, "place_rows: unknown dtype %d", out_dtype);
    FW_LAUNCH_CHECK("place_rows");
    return 0;
}

// the error-function gelu of float32 sums, rounded once
template <typename T>
__global__ void gelu_rows_kernel(const float* __restrict__ z, T* __restrict__ out, long long count) {
    for (long long i = blockIdx.x * (long long)blockDim.x + threadIdx.x; i < count; i += (long long)gridDim.x * blockDim.x)
        store_from_float(out, (size_t)i, fw_gelu(z[i]));
}

extern "C" int fw_gelu_rows(const float* z, void* out, int out_dtype, long long count, void* stream) {
    FW_REQUIRE(count >= 0, "gelu_rows: negative count");
    if (count == 0) return 0;
    const int blocks = (int)((count + 255) / 256 < 8192 ? (count + 255) / 256 : 8192);
    if (out_dtype == FW_F32) gelu_rows_kernel<float><<<blocks, 256, 0, (hipStream_t)stream>>>(z, (float*)out, count);
    else if (out_dtype == FW_BF16) gelu_rows_kernel<bf16_t><<<blocks, 256, 0, (hipStream_t)stream>>>(z, (bf16_t*)out, count);
    else FW_REQUIRE(false, "gelu_rows: unknown dtype %d", out_dtype);
    FW_LAUNCH_CHECK("gelu_rows");
    return 0;
}

// Gated linear unit with clamped halves: g = min(gate, limit), u = clamp(up, -limit, limit),
// out = g * sigmoid(alpha * g) * (u + shift). gate_up [rows][2 I]: gate columns, then up columns.
template <typename TI, typename TO>
__global__ void clamped_glu_kernel(const TI* __restrict__ gate_up, TO* __restrict__ out, int intermediate, float limit,
                                   float alpha, float shift) {
    const int row = blockIdx.y;
    const TI* source = gate_up + (size_t)row * 2 * intermediate;
    for (int i = blockIdx.x * blockDim.x + threadIdx.x; i < intermediate; i += gridDim.x * blockDim.x) {
        const float g = fminf(load_as_float(source, i), limit);
        const float u = fminf(fmaxf(load_as_float(source, (size_t)intermediate + i), -limit), limit);
        store_from_float(out, (size_t)row * intermediate + i, g * sublayer_sigmoid(alpha * g) * (u + shift));
    }
}

extern "C" int fw_clamped_glu(const void* gate_up, int in_dtype, void* out, int out_dtype, int rows, int intermediate,
                              float limit, float alpha, float shift, void* stream) {
    FW_REQUIRE(rows >= 0 && rows <= 65535 * 16 && intermediate > 0, "clamped_glu: bad sizes rows=%d intermediate=%d", rows, intermediate);
    FW_REQUIRE(limit > 0.0f, "clamped_glu: the limit must be positive");
    if (rows == 0) return 0;
    int across = (intermediate + 255) / 256;
    if (across > 64) across = 64;
    hipStream_t s = (hipStream_t)stream;
    for (int row0 = 0; row0 < rows; row0 += 65535) {
        const int now = rows - row0 < 65535 ? rows - row0 : 65535;
        dim3 grid(across, now);
        const size_t in_at = (size_t)row0 * 2 * intermediate, out_at = (size_t)row0 * intermediate;
#define FW_GLU_LAUNCH(TI, TO) \
    clamped_glu_kernel<TI, TO><<<grid, 256, 0, s>>>((const TI*)gate_up + in_at, (TO*)out + out_at, intermediate, limit, alpha, shift)
        if (in_dtype == FW_F32 && out_dtype == FW_F32) FW_GLU_LAUNCH(float, float);
        else if (in_dtype == FW_F32 && out_dtype == FW_BF16) FW_GLU_LAUNCH(float, bf16_t);
        else if (in_dtype == FW_BF16 && out_dtype == FW_BF16) FW_GLU_LAUNCH(bf16_t, bf16_t);
        else FW_REQUIRE(false, "clamped_glu: unsupported dtypes in=%d out=%d", in_dtype, out_dtype);
#undef FW_GLU_LAUNCH
    }
    FW_LAUNCH_CHECK("clamped_glu");
    return 0;
}

// ---- a sublayer between two norms ---------------------------------------------------------------------
// What joins a sublayer whose output passes a norm of its own to the residual stream, and hands the
// stream to the next reader, in one pass over the row:
//     x <- x + mult * (norm_a(a) * w + bias)   (norm_a: RMS, or with `centered` the mean taken off first; bias null: none)
//     next_out = next(x)                (next_kind 0: nothing; 1: x rounded to next_dtype; 2: RMS norm
//                                        of x times next_weight (+ next_bias); 3: the same with the mean taken off)
// The rows of next_out may lie next_stride apart (they are then some columns of wider rows).
// A norm here is v / sqrt(mean(v^2) + eps), v the values or their deviations from the row's mean. One
// workgroup per row; a row of up to 256 * JOIN_HELD values stays in registers between the passes, a
// wider one is read again. Every sum is a function of the row alone.
// A row that stays in registers asks for everything it will need at once (with few rows nothing else hides a
// second trip to memory), meets over LDS alone, and writes x last (a barrier behind a store would wait for it).
#define JOIN_HELD 16
template <typename T, int N>
__global__ __launch_bounds__(256) void norm_add_norm_held_kernel(
    float* __restrict__ x, const float* __restrict__ a, const float* __restrict__ weight, const float* __restrict__ bias, float mult,
    int centered, float eps, int next_kind, const float* __restrict__ next_weight, const float* __restrict__ next_bias, float next_eps,
    T* __restrict__ next_out, int next_stride, int hidden) {
    __shared__ float scratch[4][4];
    const size_t row0 = (size_t)blockIdx.x * hidden;
    const float count = (float)hidden;
    float held[N], was[N], scale[N], shift[N], next_scale[N], next_shift[N];
    float sum = 0.0f;
#pragma unroll
    for (int u = 0; u < N; ++u) {
        const int i = threadIdx.x + 256 * u < hidden ? threadIdx.x + 256 * u : hidden - 1;      // past the end: read again, not used
        held[u] = a[row0 + i];
        was[u] = x[row0 + i];
        scale[u] = weight[i];
        shift[u] = bias ? bias[i] : 0.0f;
        next_scale[u] = next_kind >= 2 ? next_weight[i] : 0.0f;
        next_shift[u] = (next_kind >= 2 && next_bias) ? next_bias[i] : 0.0f;
    }
#pragma unroll
    for (int u = 0; u < N; ++u) sum += threadIdx.x + 256 * u < hidden ? held[u] : 0.0f;
    const float mean = centered ? block_sum_by_lds(sum, scratch[0]) / count : 0.0f;
    float squares = 0.0f;
#pragma unroll
    for (int u = 0; u < N; ++u) {
        const float d = threadIdx.x + 256 * u < hidden ? held[u] - mean : 0.0f;
        squares = fmaf(d, d, squares);
    }
    const float inv = 1.0f / sqrtf(block_sum_by_lds(squares, scratch[1]) / count + eps);
    float new_sum = 0.0f;
#pragma unroll
    for (int u = 0; u < N; ++u) {
        const float normed = (held[u] - mean) * inv * scale[u];
        was[u] = fmaf(mult, bias ? normed + shift[u] : normed, was[u]);
        new_sum += threadIdx.x + 256 * u < hidden ? was[u] : 0.0f;
    }
    float next_mean = 0.0f, next_inv = 1.0f;
    if (next_kind >= 2) {
        next_mean = next_kind == 3 ? block_sum_by_lds(new_sum, scratch[2]) / count : 0.0f;
        float next_squares = 0.0f;
#pragma unroll
        for (int u = 0; u < N; ++u) {
            const float d = threadIdx.x + 256 * u < hidden ? was[u] - next_mean : 0.0f;
            next_squares = fmaf(d, d, next_squares);
        }
        next_inv = 1.0f / sqrtf(block_sum_by_lds(next_squares, scratch[3]) / count + next_eps);
    }
    next_out += (size_t)blockIdx.x * next_stride;
#pragma unroll
    for (int u = 0; u < N; ++u) {
        const int i = threadIdx.x + 256 * u;
        if (i >= hidden) break;
        x[row0 + i] = was[u];
        if (next_kind == 1) store_from_float(next_out, i, was[u]);
        if (next_kind >= 2) {
            const float normed = (was[u] - next_mean) * next_inv * next_scale[u];
            store_from_float(next_out, i, next_bias ? normed + next_shift[u] : normed);
        }
    }
}

template <typename T>
__global__ __launch_bounds__(256) void norm_add_norm_wide_kernel(
    float* __restrict__ x, const float* __restrict__ a, const float* __restrict__ weight, const float* __restrict__ bias, float mult,
    int centered, float eps, int next_kind, const float* __restrict__ next_weight, const float* __restrict__ next_bias, float next_eps,
    T* __restrict__ next_out, int next_stride, int hidden) {
    __shared__ float scratch[16];
    const size_t row0 = (size_t)blockIdx.x * hidden;
    next_out += (size_t)blockIdx.x * next_stride;
    const float count = (float)hidden;
    float sum = 0.0f;
    for (int i = threadIdx.x; i < hidden; i += 256) sum += a[row0 + i];
    const float mean = centered ? block_sum(sum, scratch) / count : 0.0f;
    float squares = 0.0f;
    for (int i = threadIdx.x; i < hidden; i += 256) {
        const float d = a[row0 + i] - mean;
        squares = fmaf(d, d, squares);
    }
    const float inv = 1.0f / sqrtf(block_sum(squares, scratch) / count + eps);
    float new_sum = 0.0f;
    for (int i = threadIdx.x; i < hidden; i += 256) {
        const float normed = (a[row0 + i] - mean) * inv * weight[i];
        const float updated = fmaf(mult, bias ? normed + bias[i] : normed, x[row0 + i]);
        x[row0 + i] = updated;          // read again below by the thread that wrote it
        new_sum += updated;
    }
    if (next_kind == 0) return;
    if (next_kind == 1) {
        for (int i = threadIdx.x; i < hidden; i += 256) store_from_float(next_out, i, x[row0 + i]);
        return;
    }
    const float next_mean = next_kind == 3 ? block_sum(new_sum, scratch) / count : 0.0f;
    float next_squares = 0.0f;
    for (int i = threadIdx.x; i < hidden; i += 256) {
        const float d = x[row0 + i] - next_mean;
        next_squares = fmaf(d, d, next_squares);
    }
    const float next_inv = 1.0f / sqrtf(block_sum(next_squares, scratch) / count + next_eps);
    for (int i = threadIdx.x; i < hidden; i += 256) {
        const float normed = (x[row0 + i] - next_mean) * next_inv * next_weight[i];
        store_from_float(next_out, i, next_bias ? normed + next_bias[i] : normed);
    }
}

extern "C" int fw_norm_add_norm(float* x, const float* a, const float* weight, const float* bias, float mult, int centered, float eps,
                                int next_kind, const float* next_weight, const float* next_bias, float next_eps, void* next_out,
                                int next_dtype, int next_stride, int rows, int hidden, void* stream) {
    if (next_stride <= 0) next_stride = hidden;
    FW_REQUIRE(next_stride >= hidden, "norm_add_norm: rows of %d do not fit %d apart", hidden, next_stride);
    FW_REQUIRE(rows >= 0 && hidden > 0, "norm_add_norm: bad sizes rows=%d hidden=%d", rows, hidden);
    FW_REQUIRE(eps > 0.0f, "norm_add_norm: eps must be positive");
    FW_REQUIRE(x && a && weight, "norm_add_norm: x, a and the weight are needed");
    FW_REQUIRE(next_kind >= 0 && next_kind <= 3, "norm_add_norm: unknown kind %d of what follows", next_kind);
    FW_REQUIRE(next_kind == 0 || next_out, "norm_add_norm: what follows has nowhere to go");
    FW_REQUIRE(next_kind < 2 || (next_weight && next_eps > 0.0f), "norm_add_norm: the norm that follows needs a weight and a positive eps");
    FW_REQUIRE(next_kind == 0 || next_dtype == FW_F32 || next_dtype == FW_BF16, "norm_add_norm: unknown dtype %d", next_dtype);
    if (rows == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
#define FW_JOIN_LAUNCH(KERNEL, T)                                                                                                    \
    KERNEL<<<rows, 256, 0, s>>>(x, a, weight, bias, mult, centered, eps, next_kind, next_weight, next_bias, next_eps, (T*)next_out, \
                                next_stride, hidden)
#define FW_JOIN_BY_WIDTH(T)                                                                            \
    if (hidden <= 256 * 4) FW_JOIN_LAUNCH((norm_add_norm_held_kernel<T, 4>), T);                       \
    else if (hidden <= 256 * 8) FW_JOIN_LAUNCH((norm_add_norm_held_kernel<T, 8>), T);                  \
    else if (hidden <= 256 * JOIN_HELD) FW_JOIN_LAUNCH((norm_add_norm_held_kernel<T, JOIN_HELD>), T); \
    else FW_JOIN_LAUNCH((norm_add_norm_wide_kernel<T>), T)
    if (next_kind == 0 || next_dtype == FW_F32) {
        FW_JOIN_BY_WIDTH(float);
    } else {
        FW_JOIN_BY_WIDTH(bf16_t);
    }
#undef FW_JOIN_BY_WIDTH
#undef FW_JOIN_LAUNCH
    FW_LAUNCH_CHECK("norm_add_norm");
    return 0;
}
