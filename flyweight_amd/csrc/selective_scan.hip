// The selective scan: a linear recurrence per channel and state whose decay, input and read-out the token itself forms
// (Mamba: Gu and Dao, "Mamba: Linear-Time Sequence Modeling with Selective State Spaces"). Per channel c and state n,
// with the step size dt = softplus(z_c):
//     S[n] <- exp(dt A[n]) S[n] + dt x B[n];   y = sum_n S[n] C[n] + D x;   out = y * silu(gate)
// All float32; only `out` is rounded. State [slot][n][channel], zero at a request's start. A's rows come times log2(e):
// exp(dt A) = 2^(dt A').
#include "fw_common.h"
#include "fw_kernels.h"

#define SS_TOKENS 16            // tokens whose B and C are staged together
#define SS_CHUNK 64
#define SS_MAX_STATE 128

// softplus(x) = ln(1 + e^x). The logarithm of the rounded u = 1 + e is corrected by e / (u - 1), which is exact to the last
// digits however small e is; beyond 20 e^-x no longer shows.
// QUICK (the bfloat16 runs): the hardware's exponential and reciprocal, a few units in the last place of float32.
template <bool QUICK>
__device__ __forceinline__ float ss_softplus(float x) {
    const float e = QUICK ? __expf(x) : expf(x);
    const float u = 1.0f + e, d = u - 1.0f;
    const float ln = __builtin_amdgcn_logf(u) * 0.69314718055994531f;
    const float corrected = d == 0.0f ? e : ln * (QUICK ? e * __builtin_amdgcn_rcpf(d) : e / d);
    return x > 20.0f ? x : corrected;
}
template <bool QUICK>
__device__ __forceinline__ float ss_silu(float z) {
    return QUICK ? z * __builtin_amdgcn_rcpf(1.0f + __expf(-z)) : z / (1.0f + expf(-z));
}

// A run of rows row0 .. row0 + count - 1 for one channel a lane: S moves on; with OUT the outputs are formed, else the steps' sum
// is. All lanes of the workgroup (one wave) call it together: they share the staged B and C.
// EXACT: the model has N states, and B and C are read where they lie: the row is the same for all lanes, so they travel as
// scalars and enter the arithmetic as such, with no trip through LDS.
template <int N, bool EXACT, bool OUT, bool QUICK, typename TO>
__device__ __forceinline__ float ss_run(float (&S)[N], const float (&a)[N], float d, const float* __restrict__ x, int x_stride,
                                        const float* __restrict__ z, int z_stride, const float* __restrict__ bc, int bc_stride,
                                        const float* __restrict__ gate, int gate_stride, TO* __restrict__ out, int row0, int count, int at,
                                        bool live, int channels, int states, float* staged) {
    constexpr int SS_AHEAD = N <= 32 ? 8 : 2;           // tokens whose inputs are asked for together
    float total = 0.0f;
    for (int base = 0; base < count; base += SS_TOKENS) {
        const int tokens = count - base < SS_TOKENS ? count - base : SS_TOKENS;
        if (!EXACT) {
            __syncthreads();
            for (int i = threadIdx.x; i < tokens * 2 * N; i += 64) {
                const int token = i / (2 * N), j = i % (2 * N), n = j % N;
                staged[i] = n < states ? bc[(size_t)(row0 + base + token) * bc_stride + (j < N ? n : states + n)] : 0.0f;
            }
            __syncthreads();
        }
        for (int t0 = 0; t0 < tokens; t0 += SS_AHEAD) {
            float xs[SS_AHEAD], zs[SS_AHEAD], gs[SS_AHEAD];
#pragma unroll
            for (int u = 0; u < SS_AHEAD; ++u) {        // (past the end: the last row again, not used)
                const size_t row = (size_t)(row0 + base + (t0 + u < tokens ? t0 + u : tokens - 1));
                xs[u] = x[row * x_stride + at];
                zs[u] = z[row * z_stride + at];
                gs[u] = OUT ? gate[row * gate_stride + at] : 0.0f;
            }
            auto token = [&](int u) {
                const float dt = ss_softplus<QUICK>(zs[u]);
                const float dx = dt * xs[u];
                const float* B = EXACT ? bc + (size_t)(row0 + base + t0 + u) * bc_stride : staged + (t0 + u) * 2 * N;
                float y = 0.0f;
#pragma unroll
                for (int n = 0; n < N; ++n) {
                    S[n] = fmaf(__builtin_amdgcn_exp2f(dt * a[n]), S[n], dx * B[n]);
                    if (OUT) y = fmaf(S[n], B[N + n], y);
                }
                if (OUT) {
                    y = fmaf(d, xs[u], y);
                    if (live) store_from_float(out, (size_t)(row0 + base + t0 + u) * channels + at, y * ss_silu<QUICK>(gs[u]));
                } else {
                    total += dt;
                }
            };
            if (t0 + SS_AHEAD <= tokens) {              // no branch between the tokens: what the next one needs is asked for ahead
#pragma unroll
                for (int u = 0; u < SS_AHEAD; ++u) token(u);
            } else {
#pragma unroll
                for (int u = 0; u < SS_AHEAD; ++u) {
                    if (t0 + u >= tokens) break;
                    token(u);
                }
            }
        }
    }
    return total;
}

// ---- in order ---------------------------------------------------------------------------------------------------
// A thread per (segment, channel), its N states in registers (N: the template's size, the model's states of it used; the
// others have A = B = C = 0 and stay zero). Segments of more than long_rows rows (> 0) are left to the chunked kernels.
template <int N, bool EXACT, typename TO>
__global__ __launch_bounds__(64) void selective_scan_step_kernel(
    const float* __restrict__ x, int x_stride, const float* __restrict__ z, int z_stride, const float* __restrict__ bc, int bc_stride,
    const float* __restrict__ gate, int gate_stride, const float* __restrict__ A2, const float* __restrict__ D, float* __restrict__ state,
    TO* __restrict__ out, const int32_t* __restrict__ seg_row0, const int32_t* __restrict__ seg_slot, int channels, int states, int long_rows) {
    __shared__ __attribute__((aligned(16))) float staged[EXACT ? 4 : SS_TOKENS * 2 * N];
    const int seg = blockIdx.x;
    const int first = seg_row0[seg], count = seg_row0[seg + 1] - first;
    if (long_rows > 0 && count > long_rows) return;
    const int c = blockIdx.y * 64 + threadIdx.x;
    const bool live = c < channels;
    const int at = live ? c : channels - 1;
    float* mine = state + (size_t)seg_slot[seg] * states * channels + at;
    float S[N], a[N];
#pragma unroll
    for (int n = 0; n < N; ++n) {
        S[n] = n < states ? mine[(size_t)n * channels] : 0.0f;
        a[n] = n < states ? A2[(size_t)n * channels + at] : 0.0f;
    }
    ss_run<N, EXACT, true, sizeof(TO) == 2, TO>(S, a, D[at], x, x_stride, z, z_stride, bc, bc_stride, gate, gate_stride, out, first, count, at, live, channels, states, staged);
    if (live)
#pragma unroll
        for (int n = 0; n < N; ++n)
            if (n < states) mine[(size_t)n * channels] = S[n];
}

// ---- in chunks --------------------------------------------------------------------------------------------------
// Long segments are cut into chunks of SS_CHUNK rows that are walked side by side, in three launches: every chunk from a zero
// state (leaving its last state and the sum of its steps), the states ahead of the chunks (S_out = 2^(sum dt A') S_in + the
// chunk's own, a thread per channel and state), and every chunk once more from its S_in, with the outputs.
// local [chunk][n][channel], steps [chunk][channel].
template <int N, bool EXACT, bool QUICK>
__global__ __launch_bounds__(64) void selective_scan_chunk_kernel(
    const float* __restrict__ x, int x_stride, const float* __restrict__ z, int z_stride, const float* __restrict__ bc, int bc_stride,
    const float* __restrict__ A2, float* __restrict__ local, float* __restrict__ steps, const int32_t* __restrict__ chunk_seg,
    const int32_t* __restrict__ chunk_row0, const int32_t* __restrict__ seg_row0, int channels, int states) {
    __shared__ __attribute__((aligned(16))) float staged[EXACT ? 4 : SS_TOKENS * 2 * N];
    const int chunk = blockIdx.x;
    const int row0 = chunk_row0[chunk], end = seg_row0[chunk_seg[chunk] + 1];
    const int count = end - row0 < SS_CHUNK ? end - row0 : SS_CHUNK;
    const int c = blockIdx.y * 64 + threadIdx.x;
    const bool live = c < channels;
    const int at = live ? c : channels - 1;
    float S[N], a[N];
#pragma unroll
    for (int n = 0; n < N; ++n) {
        S[n] = 0.0f;
        a[n] = n < states ? A2[(size_t)n * channels + at] : 0.0f;
    }
    const float total = ss_run<N, EXACT, false, QUICK, float>(S, a, 0.0f, x, x_stride, z, z_stride, bc, bc_stride, nullptr, 0, nullptr, row0, count, at, live,
                                                channels, states, staged);
    if (!live) return;
    float* to = local + (size_t)chunk * states * channels + c;
#pragma unroll
    for (int n = 0; n < N; ++n)
        if (n < states) to[(size_t)n * channels] = S[n];
    steps[(size_t)chunk * channels + c] = total;
}

__global__ __launch_bounds__(256) void selective_scan_state_kernel(const float* __restrict__ A2, float* __restrict__ local,
                                                                   const float* __restrict__ steps, float* __restrict__ state,
                                                                   const int32_t* __restrict__ seg_chunk0, const int32_t* __restrict__ seg_slot,
                                                                   int channels, int states) {
    const int seg = blockIdx.x;
    const int begin = seg_chunk0[seg], chunks = seg_chunk0[seg + 1] - begin;
    const int i = blockIdx.y * 256 + threadIdx.x;       // n * channels + c
    const int size = channels * states;
    if (chunks <= 0 || i >= size) return;
    const int c = i % channels;
    const float a = A2[i];
    float* slot = state + (size_t)seg_slot[seg] * size + i;
    float* at = local + (size_t)begin * size + i;
    const float* step = steps + (size_t)begin * channels + c;
    float S = *slot;
    for (int k = 0; k < chunks; k += 8) {
        float own[8], dt[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            const int from = k + u < chunks ? k + u : chunks - 1;
            own[u] = at[(size_t)from * size];
            dt[u] = step[(size_t)from * channels];
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            if (k + u >= chunks) break;
            at[(size_t)(k + u) * size] = S;
            S = fmaf(__builtin_amdgcn_exp2f(dt[u] * a), S, own[u]);
        }
    }
    *slot = S;
}

template <int N, bool EXACT, typename TO>
__global__ __launch_bounds__(64) void selective_scan_finish_kernel(
    const float* __restrict__ x, int x_stride, const float* __restrict__ z, int z_stride, const float* __restrict__ bc, int bc_stride,
    const float* __restrict__ gate, int gate_stride, const float* __restrict__ A2, const float* __restrict__ D,
    const float* __restrict__ local, TO* __restrict__ out, const int32_t* __restrict__ chunk_seg, const int32_t* __restrict__ chunk_row0,
    const int32_t* __restrict__ seg_row0, int channels, int states) {
    __shared__ __attribute__((aligned(16))) float staged[EXACT ? 4 : SS_TOKENS * 2 * N];
    const int chunk = blockIdx.x;
    const int row0 = chunk_row0[chunk], end = seg_row0[chunk_seg[chunk] + 1];
    const int count = end - row0 < SS_CHUNK ? end - row0 : SS_CHUNK;
    const int c = blockIdx.y * 64 + threadIdx.x;
    const bool live = c < channels;
    const int at = live ? c : channels - 1;
    const float* from = local + (size_t)chunk * states * channels + at;
    float S[N], a[N];
#pragma unroll
    for (int n = 0; n < N; ++n) {
        S[n] = n < states ? from[(size_t)n * channels] : 0.0f;
        a[n] = n < states ? A2[(size_t)n * channels + at] : 0.0f;
    }
    ss_run<N, EXACT, true, sizeof(TO) == 2, TO>(S, a, D[at], x, x_stride, z, z_stride, bc, bc_stride, gate, gate_stride, out, row0, count, at, live, channels, states, staged);
}

extern "C" int fw_scan_chunk_rows(void) { return SS_CHUNK; }

extern "C" int fw_selective_scan(const float* x, int x_stride, const float* z, int z_stride, const float* bc, int bc_stride, const float* gate,
                                 int gate_stride, const float* A2, const float* D, float* state, int slots, void* out, int out_dtype,
                                 const int32_t* seg_row0, const int32_t* seg_slot, int rows, int segments, int channels, int states,
                                 const int32_t* chunk_seg, const int32_t* chunk_row0, const int32_t* seg_chunk0, int chunks, int long_rows,
                                 int all_long, float* workspace, void* stream) {
    FW_REQUIRE(rows >= 0 && segments >= 0 && channels > 0 && slots > 0, "selective_scan: bad sizes rows=%d segments=%d channels=%d", rows, segments, channels);
    FW_REQUIRE(states >= 1 && states <= SS_MAX_STATE, "selective_scan: %d states a channel (1..%d)", states, SS_MAX_STATE);
    FW_REQUIRE((long long)channels * states < (1ll << 24), "selective_scan: too many channels (%d)", channels);
    FW_REQUIRE(x_stride >= channels && z_stride >= channels && gate_stride >= channels && bc_stride >= 2 * states,
               "selective_scan: rows of %d / %d / %d / %d values do not hold %d channels and %d states", x_stride, z_stride, gate_stride, bc_stride, channels, states);
    FW_REQUIRE(out_dtype == FW_F32 || out_dtype == FW_BF16, "selective_scan: unknown dtype %d", out_dtype);
    FW_REQUIRE(chunks >= 0 && (chunks == 0 || (chunk_seg && chunk_row0 && seg_chunk0 && workspace && long_rows > 0)),
               "selective_scan: chunks come with their places, a workspace and the length from which they are used");
    if (rows == 0 || segments == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const int across = fw_ceil_div(channels, 64);
    const dim3 grid(segments, across), by_chunk(chunks > 0 ? chunks : 1, across);
    const dim3 by_state(segments, fw_ceil_div((long long)channels * states, 256));
    float* local = workspace;
    float* steps = workspace ? workspace + (size_t)chunks * states * channels : nullptr;
#define FW_SCAN_OUT(N, EXACT, TO)                                                                                                            \
    if (chunks == 0 || !all_long)                                                                                                            \
        selective_scan_step_kernel<N, EXACT, TO><<<grid, 64, 0, s>>>(x, x_stride, z, z_stride, bc, bc_stride, gate, gate_stride, A2, D,      \
                                                                     state, (TO*)out, seg_row0, seg_slot, channels, states,                  \
                                                                     chunks > 0 ? long_rows : 0);                                            \
    if (chunks > 0) {                                                                                                                        \
        selective_scan_chunk_kernel<N, EXACT, sizeof(TO) == 2><<<by_chunk, 64, 0, s>>>(x, x_stride, z, z_stride, bc, bc_stride, A2, local, steps, chunk_seg,  \
                                                                      chunk_row0, seg_row0, channels, states);                               \
        selective_scan_state_kernel<<<by_state, 256, 0, s>>>(A2, local, steps, state, seg_chunk0, seg_slot, channels, states);               \
        selective_scan_finish_kernel<N, EXACT, TO><<<by_chunk, 64, 0, s>>>(x, x_stride, z, z_stride, bc, bc_stride, gate, gate_stride, A2,   \
                                                                           D, local, (TO*)out, chunk_seg, chunk_row0, seg_row0, channels,    \
                                                                           states);                                                          \
    }
#define FW_SCAN_LAUNCH(N, EXACT)                                 \
    {                                                            \
        if (out_dtype == FW_F32) { FW_SCAN_OUT(N, EXACT, float) } \
        else { FW_SCAN_OUT(N, EXACT, bf16_t) }                   \
    }
    if (states == 8) FW_SCAN_LAUNCH(8, true)
    else if (states == 16) FW_SCAN_LAUNCH(16, true)
    else if (states == 32) FW_SCAN_LAUNCH(32, true)
    else if (states == 64) FW_SCAN_LAUNCH(64, true)
    else if (states <= 8) FW_SCAN_LAUNCH(8, false)
    else if (states <= 16) FW_SCAN_LAUNCH(16, false)
    else if (states <= 24) FW_SCAN_LAUNCH(24, false)
    else if (states <= 32) FW_SCAN_LAUNCH(32, false)
    else if (states <= 64) FW_SCAN_LAUNCH(64, false)
    else FW_SCAN_LAUNCH(128, false)
#undef FW_SCAN_LAUNCH
#undef FW_SCAN_OUT
    FW_LAUNCH_CHECK("selective_scan");
    return 0;
}

// ---- the steps of single rows, with the low-rank map in front ----------------------------------------------------
// Every segment is one row (row r is segment r). z[c] = sum_j low[j] W[j][c] + bias[c], W [rank][channels] in two
// neighbouring ranks a word where it is bfloat16: the map is a few loads of whole rows beside the state's, and spares
// two launches. low: the first `rank` columns of bc's rows; B and C behind them.
template <int N, typename TW, typename TO>
__global__ __launch_bounds__(256) void selective_scan_low_rank_kernel(
    const float* __restrict__ x, int x_stride, const float* __restrict__ low, int low_stride, int rank, const TW* __restrict__ w,
    const float* __restrict__ bias, const float* __restrict__ gate, int gate_stride, const float* __restrict__ A2, const float* __restrict__ D,
    float* __restrict__ state, TO* __restrict__ out, const int32_t* __restrict__ seg_slot, int channels, int states) {
    extern __shared__ __attribute__((aligned(16))) float shared[];      // the row's low part, B, C; then four partial sums a channel
    const int row = blockIdx.x;
    const int lane = threadIdx.x & 63, part = threadIdx.x >> 6;         // four waves share the ranks of 64 channels
    const int c = blockIdx.y * 64 + lane;
    const bool live = c < channels;
    const int at = live ? c : channels - 1;
    const int width = rank + 2 * states;
    float* B = shared + ((rank + 3) & ~3);                              // B, C: N places each, zeros behind the states
    float* parts = B + 2 * N;
    for (int i = threadIdx.x; i < width; i += 256) {
        const float value = low[(size_t)row * low_stride + i];
        if (i < rank) shared[i] = value;
        else B[i - rank < states ? i - rank : N + (i - rank - states)] = value;
    }
    for (int i = states + threadIdx.x; i < N; i += 256) B[i] = B[N + i] = 0.0f;
    float* mine = state + (size_t)seg_slot[row] * states * channels + at;
    float S[N], a[N];
    float xx = 0.0f, g = 0.0f;
    if (part == 0) {            // the wave that walks the states asks for them ahead of the map
#pragma unroll
        for (int n = 0; n < N; ++n) {
            S[n] = mine[(size_t)(n < states ? n : 0) * channels];
            a[n] = A2[(size_t)(n < states ? n : 0) * channels + at];
        }
        xx = x[(size_t)row * x_stride + at];
        g = gate[(size_t)row * gate_stride + at];
    }
    __syncthreads();
    float sum = 0.0f;
    if constexpr (sizeof(TW) == 2) {
        const uint32_t* pairs = reinterpret_cast<const uint32_t*>(w);   // [rank / 2][channels]
#pragma unroll 16
        for (int j = part; j < rank / 2; j += 4) {
            const uint32_t two = pairs[(size_t)j * channels + at];
            sum = fmaf(bf16_bits_to_float(two & 0xffffu), shared[2 * j], sum);
            sum = fmaf(bf16_bits_to_float(two >> 16), shared[2 * j + 1], sum);
        }
    } else {
#pragma unroll 16
        for (int j = part; j < rank; j += 4) sum = fmaf(load_as_float(w, (size_t)j * channels + at), shared[j], sum);
    }
    parts[threadIdx.x] = sum;
    __syncthreads();
    if (part != 0) return;
    const float z = (((parts[lane] + parts[64 + lane]) + parts[128 + lane]) + parts[192 + lane]) + bias[at];
    const float dt = ss_softplus<sizeof(TO) == 2>(z), dx = dt * xx;
    float y = 0.0f;
#pragma unroll
    for (int n = 0; n < N; ++n) {
        S[n] = fmaf(__builtin_amdgcn_exp2f(dt * a[n]), S[n], dx * B[n]);
        y = fmaf(S[n], B[N + n], y);
    }
    if (!live) return;
    store_from_float(out, (size_t)row * channels + c, fmaf(D[c], xx, y) * ss_silu<sizeof(TO) == 2>(g));
#pragma unroll
    for (int n = 0; n < N; ++n)
        if (n < states) mine[(size_t)n * channels] = S[n];
}

extern "C" int fw_selective_scan_low_rank(const float* x, int x_stride, const float* low, int low_stride, int rank, const void* w, int w_dtype,
                                          const float* bias, const float* gate, int gate_stride, const float* A2, const float* D, float* state,
                                          int slots, void* out, int out_dtype, const int32_t* seg_slot, int rows, int channels, int states,
                                          void* stream) {
    FW_REQUIRE(rows >= 0 && channels > 0 && slots > 0 && rank >= 1, "selective_scan_low_rank: bad sizes rows=%d channels=%d rank=%d", rows, channels, rank);
    FW_REQUIRE(states >= 1 && states <= SS_MAX_STATE, "selective_scan_low_rank: %d states a channel (1..%d)", states, SS_MAX_STATE);
    FW_REQUIRE(x_stride >= channels && gate_stride >= channels && low_stride >= rank + 2 * states,
               "selective_scan_low_rank: rows of %d / %d / %d values do not hold %d channels and %d + 2 * %d numbers", x_stride, gate_stride, low_stride,
               channels, rank, states);
    FW_REQUIRE(w_dtype == FW_F32 || (w_dtype == FW_BF16 && rank % 2 == 0 && (uintptr_t)w % 4 == 0), "selective_scan_low_rank: an odd rank of bfloat16");
    FW_REQUIRE(rank + 2 * states <= 8192, "selective_scan_low_rank: a rank of %d", rank);
    if (rows == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid(rows, fw_ceil_div(channels, 64));
    const int rank_bytes = ((rank + 3) & ~3) * 4;
#define FW_LOW_LAUNCH(N, TW, TO)                                                                                                         \
    selective_scan_low_rank_kernel<N, TW, TO><<<grid, 256, rank_bytes + (2 * N + 256) * 4, s>>>(x, x_stride, low, low_stride, rank, (const TW*)w, bias, gate, \
                                                                           gate_stride, A2, D, state, (TO*)out, seg_slot, channels, states)
#define FW_LOW_BY_DTYPE(N)                                                                 \
    {                                                                                      \
        if (w_dtype == FW_BF16 && out_dtype == FW_BF16) FW_LOW_LAUNCH(N, bf16_t, bf16_t);  \
        else if (w_dtype == FW_F32 && out_dtype == FW_F32) FW_LOW_LAUNCH(N, float, float); \
        else if (w_dtype == FW_F32 && out_dtype == FW_BF16) FW_LOW_LAUNCH(N, float, bf16_t); \
        else FW_REQUIRE(false, "selective_scan_low_rank: unsupported dtypes w=%d out=%d", w_dtype, out_dtype); \
    }
    if (states <= 8) FW_LOW_BY_DTYPE(8)
    else if (states <= 16) FW_LOW_BY_DTYPE(16)
    else if (states <= 24) FW_LOW_BY_DTYPE(24)
    else if (states <= 32) FW_LOW_BY_DTYPE(32)
    else if (states <= 64) FW_LOW_BY_DTYPE(64)
    else FW_LOW_BY_DTYPE(128)
#undef FW_LOW_BY_DTYPE
#undef FW_LOW_LAUNCH
    FW_LAUNCH_CHECK("selective_scan_low_rank");
    return 0;
}
