// A residual stream of several rows side by side ("hyper-connections"): what stands between two sublayers.
//
//   read   u = sum_s in[s] x_s;  out = norm(u)
//   join   x_t <- sum_s mix[s][t] x_s + out[t] * (ls * y), all t from the old rows; then the next reader's read
//
// x [rows][streams][hidden] float32. The norm is tanh(alpha u) w + b, no statistics of the row, so that a channel
// of all streams can be worked on by one thread alone. y is given as what the sublayer left:
//   ROWS      rows of its own
//   BRANCHES  scale_a rms(a) w_a + scale_b rms(b) w_b (two branches, each brought to unit root mean square first)
//   CHOSEN    sum_j weight[r][j] a[place[r][j]] (+ sigmoid(gate[r]) b[r]): the outputs of the experts a row chose,
//             in the order of the choices, and of a unit that every row runs
// Everything is float32 and every sum is in an order fixed by the row alone.
#include "fw_common.h"
#include "fw_kernels.h"

#define STREAM_ROWS 0
#define STREAM_BRANCHES 1
#define STREAM_CHOSEN 2
// what reads the streams next
#define STREAM_NEXT_NOTHING 0
#define STREAM_NEXT_SUM 1       // u as it is
#define STREAM_NEXT_TANH 2      // tanh(alpha u) w + b
#define STREAM_MAX 32
#define STREAM_BRANCH_HELD 4    // pieces of four channels a thread keeps of either branch

typedef __attribute__((ext_vector_type(4))) float st_f32x4;
typedef __attribute__((ext_vector_type(2))) uint32_t st_u32x2;

struct StreamSource {
    const float* a;
    const float* b;
    const float* weight_a;
    const float* weight_b;
    float scale_a, scale_b, eps;
    const float* choice_weight;
    const int32_t* pair_place;
    int top;
    const float* gate;
    int gate_stride;
};

struct StreamReader {
    int kind;
    const float* in;        // [streams], null: all ones
    const float* weight;
    const float* bias;
    const float* alpha;
};

// V consecutive channels
template <int V> struct Channels {
    float v[V];
};
template <int V> __device__ __forceinline__ Channels<V> st_load(const float* p) {
    Channels<V> c;
    if constexpr (V == 4) {
        const st_f32x4 f = *reinterpret_cast<const st_f32x4*>(p);
#pragma unroll
        for (int e = 0; e < 4; ++e) c.v[e] = f[e];
    } else {
        c.v[0] = p[0];
    }
    return c;
}
template <int V> __device__ __forceinline__ void st_store(float* p, const Channels<V>& c) {
    if constexpr (V == 4) *reinterpret_cast<st_f32x4*>(p) = st_f32x4{c.v[0], c.v[1], c.v[2], c.v[3]};
    else p[0] = c.v[0];
}
template <int V> __device__ __forceinline__ void st_store(bf16_t* p, const Channels<V>& c) {
    if constexpr (V == 4) {
        *reinterpret_cast<st_u32x2*>(p) = st_u32x2{(uint32_t)float_to_bf16_bits(c.v[0]) | ((uint32_t)float_to_bf16_bits(c.v[1]) << 16),
                                                   (uint32_t)float_to_bf16_bits(c.v[2]) | ((uint32_t)float_to_bf16_bits(c.v[3]) << 16)};
    } else {
        p[0] = float_to_bf16(c.v[0]);
    }
}

__device__ __forceinline__ float st_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// tanh with the sign apart: 1 - 2 / (e^(2 |z|) + 1), and a short odd series where that difference would lose its digits
// (|z| < 0.25: the next term is below 2e-8 of the result)
__device__ __forceinline__ float st_tanh(float z) {
    const float x = fabsf(z);
    const float e = __expf(2.0f * x);
    const float far = 1.0f - 2.0f / (e + 1.0f);
    const float s = x * x;
    const float near = x * fmaf(s, fmaf(s, fmaf(s, fmaf(s, fmaf(s, -1382.0f / 155925.0f, 62.0f / 2835.0f), -17.0f / 315.0f), 2.0f / 15.0f), -1.0f / 3.0f), 1.0f);
    return copysignf(x < 0.25f ? near : far, z);
}

template <int V, typename T>
__device__ __forceinline__ void st_next(const StreamReader& reader, float alpha, Channels<V> u, int i, T* to) {
    if (reader.kind == STREAM_NEXT_TANH) {
        const Channels<V> w = st_load<V>(reader.weight + i), b = st_load<V>(reader.bias + i);
#pragma unroll
        for (int e = 0; e < V; ++e) u.v[e] = fmaf(st_tanh(alpha * u.v[e]), w.v[e], b.v[e]);
    }
    st_store<V>(to, u);
}

// ---- read ---------------------------------------------------------------------------------------------------
template <int V, typename T>
__global__ __launch_bounds__(256) void stream_read_kernel(const float* __restrict__ x, int streams, const StreamReader reader,
                                                          const int32_t* __restrict__ row_index, T* __restrict__ out, int hidden) {
    const int row = blockIdx.x;
    const float* source = x + (size_t)(row_index ? row_index[row] : row) * streams * hidden;
    const float alpha = reader.kind == STREAM_NEXT_TANH ? reader.alpha[0] : 0.0f;
    for (int i = (blockIdx.y * 256 + threadIdx.x) * V; i < hidden; i += gridDim.y * 256 * V) {
        Channels<V> u;
#pragma unroll
        for (int e = 0; e < V; ++e) u.v[e] = 0.0f;
        for (int s = 0; s < streams; ++s) {
            const Channels<V> c = st_load<V>(source + (size_t)s * hidden + i);
            const float w = reader.in ? reader.in[s] : 1.0f;
#pragma unroll
            for (int e = 0; e < V; ++e) u.v[e] = fmaf(w, c.v[e], u.v[e]);
        }
        st_next<V, T>(reader, alpha, u, i, out + (size_t)row * hidden + i);
    }
}

// ---- join ---------------------------------------------------------------------------------------------------
// The streams of V channels from the old ones and y (already times ls), stored, and the next reader's sum of the new ones.
// S > 0: that many streams, held in registers; S = 0: any number up to STREAM_MAX.
template <int S, int V>
__device__ __forceinline__ Channels<V> st_mix(float* x, const Channels<V> (&old)[S > 0 ? S : STREAM_MAX], const Channels<V>& y, int streams,
                                              const float* __restrict__ mix, const float* __restrict__ out_weight,
                                              const float* __restrict__ next_in, int hidden) {
    const int n = S > 0 ? S : streams;
    Channels<V> u;
#pragma unroll
    for (int e = 0; e < V; ++e) u.v[e] = 0.0f;
#pragma unroll
    for (int t = 0; t < (S > 0 ? S : STREAM_MAX); ++t) {
        if (t >= n) break;
        Channels<V> now;
        const float o = out_weight[t];
#pragma unroll
        for (int e = 0; e < V; ++e) now.v[e] = o * y.v[e];
#pragma unroll
        for (int s = 0; s < (S > 0 ? S : STREAM_MAX); ++s) {
            if (s >= n) break;
            const float m = mix[s * n + t];
#pragma unroll
            for (int e = 0; e < V; ++e) now.v[e] = fmaf(m, old[s].v[e], now.v[e]);
        }
        st_store<V>(x + (size_t)t * hidden, now);
        const float w = next_in ? next_in[t] : 1.0f;
#pragma unroll
        for (int e = 0; e < V; ++e) u.v[e] = fmaf(w, now.v[e], u.v[e]);
    }
    return u;
}

template <int S, int V, int SOURCE, typename T>
__global__ __launch_bounds__(256) void stream_join_kernel(float* __restrict__ x, int streams, const float* __restrict__ ls,
                                                          const float* __restrict__ mix, const float* __restrict__ out_weight,
                                                          const StreamSource source, const StreamReader reader, T* __restrict__ next_out,
                                                          int hidden) {
    const int row = blockIdx.x;
    const int n = S > 0 ? S : streams;
    float* rows = x + (size_t)row * n * hidden;
    const float alpha = reader.kind == STREAM_NEXT_TANH ? reader.alpha[0] : 0.0f;
    const float shared = (SOURCE == STREAM_CHOSEN && source.b) ? (source.gate ? st_sigmoid(source.gate[(size_t)row * source.gate_stride]) : 1.0f) : 0.0f;
    for (int i = (blockIdx.y * 256 + threadIdx.x) * V; i < hidden; i += gridDim.y * 256 * V) {
        Channels<V> old[S > 0 ? S : STREAM_MAX];
#pragma unroll
        for (int s = 0; s < (S > 0 ? S : STREAM_MAX); ++s)
            if (s < n) old[s] = st_load<V>(rows + (size_t)s * hidden + i);
        const Channels<V> scale = st_load<V>(ls + i);
        Channels<V> y;
        if constexpr (SOURCE == STREAM_ROWS) {
            y = st_load<V>(source.a + (size_t)row * hidden + i);
        } else {
            Channels<V> b;
#pragma unroll
            for (int e = 0; e < V; ++e) y.v[e] = b.v[e] = 0.0f;
            if (source.b) b = st_load<V>(source.b + (size_t)row * hidden + i);
#pragma unroll 4
            for (int j = 0; j < source.top; ++j) {
                const float w = source.choice_weight[(size_t)row * source.top + j];
                const Channels<V> c = st_load<V>(source.a + (size_t)source.pair_place[(size_t)row * source.top + j] * hidden + i);
#pragma unroll
                for (int e = 0; e < V; ++e) y.v[e] = fmaf(w, c.v[e], y.v[e]);
            }
            if (source.b)
#pragma unroll
                for (int e = 0; e < V; ++e) y.v[e] = fmaf(shared, b.v[e], y.v[e]);
        }
#pragma unroll
        for (int e = 0; e < V; ++e) y.v[e] *= scale.v[e];
        const Channels<V> u = st_mix<S, V>(rows + i, old, y, n, mix, out_weight, reader.in, hidden);
        if (reader.kind != STREAM_NEXT_NOTHING) st_next<V, T>(reader, alpha, u, i, next_out + (size_t)row * hidden + i);
    }
}

// Two branches: the row's two sums of squares first, a workgroup per row. Rows of up to 256 * V * STREAM_BRANCH_HELD
// channels keep both branches in registers between the passes, wider ones are read again.
template <int S, int V, typename T>
__global__ __launch_bounds__(256) void stream_join_branches_kernel(float* __restrict__ x, int streams, const float* __restrict__ ls,
                                                                   const float* __restrict__ mix, const float* __restrict__ out_weight,
                                                                   const StreamSource source, const StreamReader reader,
                                                                   T* __restrict__ next_out, int hidden) {
    __shared__ float scratch[2][4];
    const int row = blockIdx.x;
    const int n = S > 0 ? S : streams;
    float* rows = x + (size_t)row * n * hidden;
    const float* a = source.a + (size_t)row * hidden;
    const float* b = source.b + (size_t)row * hidden;
    const float alpha = reader.kind == STREAM_NEXT_TANH ? reader.alpha[0] : 0.0f;
    const bool held_all = hidden <= 256 * V * STREAM_BRANCH_HELD;
    Channels<V> held_a[STREAM_BRANCH_HELD], held_b[STREAM_BRANCH_HELD];
    float squares_a = 0.0f, squares_b = 0.0f;
    auto count = [&](const Channels<V>& ca, const Channels<V>& cb) {
#pragma unroll
        for (int e = 0; e < V; ++e) {
            squares_a = fmaf(ca.v[e], ca.v[e], squares_a);
            squares_b = fmaf(cb.v[e], cb.v[e], squares_b);
        }
    };
    if (held_all) {
#pragma unroll
        for (int p = 0; p < STREAM_BRANCH_HELD; ++p) {
            const int i = (p * 256 + threadIdx.x) * V;
            const int from = i < hidden ? i : 0;
            held_a[p] = st_load<V>(a + from);
            held_b[p] = st_load<V>(b + from);
        }
#pragma unroll
        for (int p = 0; p < STREAM_BRANCH_HELD; ++p)
            if ((p * 256 + threadIdx.x) * V < hidden) count(held_a[p], held_b[p]);
    } else {
        for (int i = threadIdx.x * V; i < hidden; i += 256 * V) count(st_load<V>(a + i), st_load<V>(b + i));
    }
    squares_a = wave_sum(squares_a);
    squares_b = wave_sum(squares_b);
    if ((threadIdx.x & 63) == 0) {
        scratch[0][threadIdx.x >> 6] = squares_a;
        scratch[1][threadIdx.x >> 6] = squares_b;
    }
    fw_lds_barrier();
    const float sum_a = ((scratch[0][0] + scratch[0][1]) + scratch[0][2]) + scratch[0][3];
    const float sum_b = ((scratch[1][0] + scratch[1][1]) + scratch[1][2]) + scratch[1][3];
    const float inv_a = source.scale_a / sqrtf(sum_a / (float)hidden + source.eps);
    const float inv_b = source.scale_b / sqrtf(sum_b / (float)hidden + source.eps);
    auto finish = [&](const Channels<V>& ca, const Channels<V>& cb, int i) {
        Channels<V> old[S > 0 ? S : STREAM_MAX];
#pragma unroll
        for (int s = 0; s < (S > 0 ? S : STREAM_MAX); ++s)
            if (s < n) old[s] = st_load<V>(rows + (size_t)s * hidden + i);
        const Channels<V> scale = st_load<V>(ls + i), wa = st_load<V>(source.weight_a + i), wb = st_load<V>(source.weight_b + i);
        Channels<V> y;
#pragma unroll
        for (int e = 0; e < V; ++e) y.v[e] = (ca.v[e] * inv_a * wa.v[e] + cb.v[e] * inv_b * wb.v[e]) * scale.v[e];
        const Channels<V> u = st_mix<S, V>(rows + i, old, y, n, mix, out_weight, reader.in, hidden);
        if (reader.kind != STREAM_NEXT_NOTHING) st_next<V, T>(reader, alpha, u, i, next_out + (size_t)row * hidden + i);
    };
    if (held_all) {
#pragma unroll
        for (int p = 0; p < STREAM_BRANCH_HELD; ++p) {
            const int i = (p * 256 + threadIdx.x) * V;
            if (i < hidden) finish(held_a[p], held_b[p], i);
        }
    } else {
        for (int i = threadIdx.x * V; i < hidden; i += 256 * V) finish(st_load<V>(a + i), st_load<V>(b + i), i);
    }
}

static bool st_aligned(const void* p, int bytes) { return (uintptr_t)p % bytes == 0; }

extern "C" int fw_stream_read(const float* x, int streams, int next_kind, const float* next_in, const float* next_weight,
                              const float* next_bias, const float* next_alpha, const int32_t* row_index, void* out, int out_dtype, int rows,
                              int hidden, void* stream) {
    FW_REQUIRE(rows >= 0 && hidden > 0 && streams >= 1, "stream_read: bad sizes rows=%d streams=%d hidden=%d", rows, streams, hidden);
    FW_REQUIRE(next_kind == STREAM_NEXT_SUM || (next_kind == STREAM_NEXT_TANH && next_weight && next_bias && next_alpha),
               "stream_read: unknown kind %d of norm, or one without its weight, bias and alpha", next_kind);
    FW_REQUIRE(out_dtype == FW_F32 || out_dtype == FW_BF16, "stream_read: unknown dtype %d", out_dtype);
    if (rows == 0) return 0;
    const StreamReader reader = {next_kind, next_in, next_weight, next_bias, next_alpha};
    hipStream_t s = (hipStream_t)stream;
    const bool four = hidden % 4 == 0 && st_aligned(x, 16) && st_aligned(out, 16) &&
                      (next_kind != STREAM_NEXT_TANH || (st_aligned(next_weight, 16) && st_aligned(next_bias, 16)));
    const dim3 grid(rows, fw_ceil_div(hidden, four ? 1024 : 256) < 64 ? fw_ceil_div(hidden, four ? 1024 : 256) : 64);
#define FW_READ_LAUNCH(V, T) stream_read_kernel<V, T><<<grid, 256, 0, s>>>(x, streams, reader, row_index, (T*)out, hidden)
    if (four) {
        if (out_dtype == FW_F32) FW_READ_LAUNCH(4, float);
        else FW_READ_LAUNCH(4, bf16_t);
    } else {
        if (out_dtype == FW_F32) FW_READ_LAUNCH(1, float);
        else FW_READ_LAUNCH(1, bf16_t);
    }
#undef FW_READ_LAUNCH
    FW_LAUNCH_CHECK("stream_read");
    return 0;
}

template <int S, int V, typename T>
static void stream_join_launch(float* x, int streams, const float* ls, const float* mix, const float* out_weight, int kind,
                               const StreamSource& source, const StreamReader& reader, void* next_out, int rows, int hidden, hipStream_t s) {
    if (kind == STREAM_BRANCHES) {
        stream_join_branches_kernel<S, V, T><<<rows, 256, 0, s>>>(x, streams, ls, mix, out_weight, source, reader, (T*)next_out, hidden);
        return;
    }
    const int across = fw_ceil_div(hidden, 256 * V);
    const dim3 grid(rows, across < 64 ? across : 64);
    if (kind == STREAM_ROWS)
        stream_join_kernel<S, V, STREAM_ROWS, T><<<grid, 256, 0, s>>>(x, streams, ls, mix, out_weight, source, reader, (T*)next_out, hidden);
    else
        stream_join_kernel<S, V, STREAM_CHOSEN, T><<<grid, 256, 0, s>>>(x, streams, ls, mix, out_weight, source, reader, (T*)next_out, hidden);
}

extern "C" int fw_stream_join(float* x, int streams, const float* ls, const float* mix, const float* out_weight, int source_kind,
                              const float* a, const float* b, const float* weight_a, const float* weight_b, float scale_a, float scale_b,
                              float eps, const float* choice_weight, const int32_t* pair_place, int top, const float* gate, int gate_stride,
                              int next_kind, const float* next_in, const float* next_weight, const float* next_bias,
                              const float* next_alpha, void* next_out, int next_dtype, int rows, int hidden, void* stream) {
    FW_REQUIRE(rows >= 0 && hidden > 0 && streams >= 1 && streams <= STREAM_MAX, "stream_join: bad sizes rows=%d streams=%d (1..%d) hidden=%d",
               rows, streams, STREAM_MAX, hidden);
    FW_REQUIRE(x && ls && mix && out_weight && a, "stream_join: x, the scales, the mix and the sublayer's output are needed");
    FW_REQUIRE(source_kind >= STREAM_ROWS && source_kind <= STREAM_CHOSEN, "stream_join: unknown kind %d of output", source_kind);
    FW_REQUIRE(source_kind != STREAM_BRANCHES || (b && weight_a && weight_b && eps > 0.0f), "stream_join: two branches need their weights and a positive eps");
    FW_REQUIRE(source_kind != STREAM_CHOSEN || (choice_weight && pair_place && top >= 1), "stream_join: chosen rows need their places and weights");
    FW_REQUIRE(next_kind >= STREAM_NEXT_NOTHING && next_kind <= STREAM_NEXT_TANH, "stream_join: unknown kind %d of what follows", next_kind);
    FW_REQUIRE(next_kind == STREAM_NEXT_NOTHING || next_out, "stream_join: what follows has nowhere to go");
    FW_REQUIRE(next_kind != STREAM_NEXT_TANH || (next_weight && next_bias && next_alpha), "stream_join: the norm that follows needs its weight, bias and alpha");
    FW_REQUIRE(next_kind == STREAM_NEXT_NOTHING || next_dtype == FW_F32 || next_dtype == FW_BF16, "stream_join: unknown dtype %d", next_dtype);
    if (rows == 0) return 0;
    const StreamSource source = {a, b, weight_a, weight_b, scale_a, scale_b, eps, choice_weight, pair_place, top, gate, gate_stride};
    const StreamReader reader = {next_kind, next_in, next_weight, next_bias, next_alpha};
    hipStream_t s = (hipStream_t)stream;
    const bool to_float = next_kind == STREAM_NEXT_NOTHING || next_dtype == FW_F32;
    bool four = hidden % 4 == 0;
    const void* wide[] = {x, ls, a, b, weight_a, weight_b, next_weight, next_bias, next_out};
    for (const void* p : wide) four = four && st_aligned(p, 16);
#define FW_STREAM_LAUNCH(S, V)                                                                                                               \
    {                                                                                                                                        \
        if (to_float) stream_join_launch<S, V, float>(x, streams, ls, mix, out_weight, source_kind, source, reader, next_out, rows, hidden, s); \
        else stream_join_launch<S, V, bf16_t>(x, streams, ls, mix, out_weight, source_kind, source, reader, next_out, rows, hidden, s);         \
    }
    if (four && streams == 1) FW_STREAM_LAUNCH(1, 4)
    else if (four && streams == 2) FW_STREAM_LAUNCH(2, 4)
    else if (four && streams == 3) FW_STREAM_LAUNCH(3, 4)
    else if (four && streams == 4) FW_STREAM_LAUNCH(4, 4)
    else if (four && streams == 6) FW_STREAM_LAUNCH(6, 4)
    else if (four && streams == 8) FW_STREAM_LAUNCH(8, 4)
    else FW_STREAM_LAUNCH(0, 1)
#undef FW_STREAM_LAUNCH
    FW_LAUNCH_CHECK("stream_join");
    return 0;
}
