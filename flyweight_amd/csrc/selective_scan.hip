// The selective scan: a linear recurrence per channel and state whose decay, input and read-out the token itself forms
// (Mamba: Gu and Dao, "Mamba: Linear-Time Sequence Modeling with Selective State Spaces"). Per channel c and state n,
// with the step size dt = softplus(z_c):
//     S[n] <- exp(dt A[n]) S[n] + dt x B[n];   y = sum_n S[n] C[n] + D x;   out = y * silu(gate)
// All float32; only `out` is rounded. State [slot][n][channel], zero at a request's start.
#include "fw_common.h"
#include "fw_kernels.h"

#define SS_TOKENS 16
#define SS_MAX_STATE 128

__device__ __forceinline__ float ss_softplus(float x) { return x > 20.0f ? x : log1pf(expf(x)); }
__device__ __forceinline__ float ss_silu(float z) { return z / (1.0f + expf(-z)); }

// A thread per (segment, channel), its N states in registers (N: the template's size, the model's states of it used; the
// others have A = B = C = 0 and stay zero). A's rows come times log2(e): exp(dt A) = 2^(dt A'). B and C of SS_TOKENS tokens
// at a time are staged in LDS, where all lanes read the same word.
template <int N, typename TO>
__global__ __launch_bounds__(64) void selective_scan_step_kernel(
    const float* __restrict__ x, int x_stride, const float* __restrict__ z, int z_stride, const float* __restrict__ bc, int bc_stride,
    const float* __restrict__ gate, int gate_stride, const float* __restrict__ A2, const float* __restrict__ D, float* __restrict__ state,
    TO* __restrict__ out, const int32_t* __restrict__ seg_row0, const int32_t* __restrict__ seg_slot, int channels, int states) {
    __shared__ __attribute__((aligned(16))) float staged[SS_TOKENS * 2 * N];
    const int seg = blockIdx.x;
    const int c = blockIdx.y * 64 + threadIdx.x;
    const bool live = c < channels;
    const int at = live ? c : channels - 1;
    const int first = seg_row0[seg], count = seg_row0[seg + 1] - first;
    float* mine = state + (size_t)seg_slot[seg] * states * channels + at;
    float S[N], a[N];
#pragma unroll
    for (int n = 0; n < N; ++n) {
        S[n] = n < states ? mine[(size_t)n * channels] : 0.0f;
        a[n] = n < states ? A2[(size_t)n * channels + at] : 0.0f;
    }
    const float d = D[at];
    for (int base = 0; base < count; base += SS_TOKENS) {
        const int tokens = count - base < SS_TOKENS ? count - base : SS_TOKENS;
        __syncthreads();
        for (int i = threadIdx.x; i < tokens * 2 * N; i += 64) {
            const int token = i / (2 * N), j = i % (2 * N), n = j % N;
            staged[i] = n < states ? bc[(size_t)(first + base + token) * bc_stride + (j < N ? n : states + n)] : 0.0f;
        }
        __syncthreads();
        for (int token = 0; token < tokens; ++token) {
            const size_t row = (size_t)(first + base + token);
            const float xx = x[row * x_stride + at], g = gate[row * gate_stride + at];
            const float dt = ss_softplus(z[row * z_stride + at]);
            const float dx = dt * xx;
            const float* B = staged + token * 2 * N;
            float y = 0.0f;
#pragma unroll
            for (int n = 0; n < N; ++n) {
                S[n] = fmaf(__builtin_amdgcn_exp2f(dt * a[n]), S[n], dx * B[n]);
                y = fmaf(S[n], B[N + n], y);
            }
            y = fmaf(d, xx, y);
            if (live) store_from_float(out, row * channels + c, y * ss_silu(g));
        }
    }
    if (live)
#pragma unroll
        for (int n = 0; n < N; ++n)
            if (n < states) mine[(size_t)n * channels] = S[n];
}

extern "C" int fw_selective_scan(const float* x, int x_stride, const float* z, int z_stride, const float* bc, int bc_stride, const float* gate,
                                 int gate_stride, const float* A2, const float* D, float* state, int slots, void* out, int out_dtype,
                                 const int32_t* seg_row0, const int32_t* seg_slot, int rows, int segments, int channels, int states, void* stream) {
    FW_REQUIRE(rows >= 0 && segments >= 0 && channels > 0 && slots > 0, "selective_scan: bad sizes rows=%d segments=%d channels=%d", rows, segments, channels);
    FW_REQUIRE(states >= 1 && states <= SS_MAX_STATE, "selective_scan: %d states a channel (1..%d)", states, SS_MAX_STATE);
    FW_REQUIRE(x_stride >= channels && z_stride >= channels && gate_stride >= channels && bc_stride >= 2 * states,
               "selective_scan: rows of %d / %d / %d / %d values do not hold %d channels and %d states", x_stride, z_stride, gate_stride, bc_stride, channels, states);
    FW_REQUIRE(out_dtype == FW_F32 || out_dtype == FW_BF16, "selective_scan: unknown dtype %d", out_dtype);
    if (rows == 0 || segments == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid(segments, fw_ceil_div(channels, 64));
#define FW_SCAN_LAUNCH(N)                                                                                                              \
    {                                                                                                                                  \
        if (out_dtype == FW_F32) selective_scan_step_kernel<N, float><<<grid, 64, 0, s>>>(x, x_stride, z, z_stride, bc, bc_stride, gate, \
            gate_stride, A2, D, state, (float*)out, seg_row0, seg_slot, channels, states);                                             \
        else selective_scan_step_kernel<N, bf16_t><<<grid, 64, 0, s>>>(x, x_stride, z, z_stride, bc, bc_stride, gate, gate_stride, A2, \
            D, state, (bf16_t*)out, seg_row0, seg_slot, channels, states);                                                             \
    }
    if (states <= 8) FW_SCAN_LAUNCH(8)
    else if (states <= 16) FW_SCAN_LAUNCH(16)
    else if (states <= 24) FW_SCAN_LAUNCH(24)
    else if (states <= 32) FW_SCAN_LAUNCH(32)
    else if (states <= 64) FW_SCAN_LAUNCH(64)
    else FW_SCAN_LAUNCH(128)
#undef FW_SCAN_LAUNCH
    FW_LAUNCH_CHECK("selective_scan");
    return 0;
}
