// A linear recurrence over a matrix state per head with one fixed decay per head ("lightning attention"). Per head, a
// token brings q, k (dim channels) and v (vdim channels), each the silu of a projection:
//     S <- decay S + k v^T;   o = S^T q
// (the read-out sees the token's own write). State [slot][head][dim][vdim] float32, zero at a request's start.
//
// All arithmetic is float32, whatever the run's dtype.
#include "fw_common.h"
#include "fw_kernels.h"

__device__ __forceinline__ float dr_silu(float z) { return z / (1.0f + expf(-z)); }

// ---- token by token ---------------------------------------------------------------------------------------------
// Workgroup (segment, head, block of 64 value channels): a lane owns a value channel, the four waves share the key
// channels out (RPT neighbouring ones each, the state's columns of them in registers). DR_TOKENS tokens at a time are
// staged in LDS, silu applied; a wave's part of a token's read-out goes to LDS and the four parts are added, in order,
// once per chunk. Segments of more than `long_rows` rows are left alone (long_rows > 0).
#define DR_TOKENS 16
template <int RPT>
__global__ __launch_bounds__(256) void decay_recurrence_step_kernel(
    const float* __restrict__ q, const float* __restrict__ k, const float* __restrict__ v, int stride, const float* __restrict__ decay,
    float* __restrict__ state, float* __restrict__ out, const int32_t* __restrict__ seg_row0, const int32_t* __restrict__ seg_slot, int heads,
    int dim, int vdim, int long_rows) {
    constexpr int DP = 4 * RPT;
    __shared__ __attribute__((aligned(16))) float staged_q[DR_TOKENS * DP];
    __shared__ __attribute__((aligned(16))) float staged_k[DR_TOKENS * DP];
    __shared__ float staged_v[DR_TOKENS * 64];
    __shared__ float parts[DR_TOKENS * 4 * 64];
    const int seg = blockIdx.x, head = blockIdx.y, block = blockIdx.z;
    const int first = seg_row0[seg], count = seg_row0[seg + 1] - first;
    if (long_rows > 0 && count > long_rows) return;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int column = block * 64 + lane;
    const bool live = column < vdim;
    float* mine = state + ((size_t)seg_slot[seg] * heads + head) * dim * vdim + (live ? column : 0);
    const float g = decay[head];
    float S[RPT];
#pragma unroll
    for (int t = 0; t < RPT; ++t) {
        const int key = wave * RPT + t;
        S[t] = mine[(size_t)(key < dim ? key : 0) * vdim];
    }
    for (int base = 0; base < count; base += DR_TOKENS) {
        const int tokens = count - base < DR_TOKENS ? count - base : DR_TOKENS;
        for (int i = threadIdx.x; i < tokens * DP; i += 256) {
            const int token = i / DP, c = i % DP;
            const size_t at = (size_t)(first + base + token) * stride + (size_t)head * dim + (c < dim ? c : 0);
            const float zq = q[at], zk = k[at];
            staged_q[i] = c < dim ? dr_silu(zq) : 0.0f;
            staged_k[i] = c < dim ? dr_silu(zk) : 0.0f;
        }
        for (int i = threadIdx.x; i < tokens * 64; i += 256) {
            const int token = i / 64, c = block * 64 + i % 64;
            staged_v[i] = c < vdim ? dr_silu(v[(size_t)(first + base + token) * stride + (size_t)head * vdim + c]) : 0.0f;
        }
        __syncthreads();
        for (int token = 0; token < tokens; ++token) {
            const float value = staged_v[token * 64 + lane];
            float read = 0.0f;
#pragma unroll
            for (int t = 0; t < RPT; ++t) {
                S[t] = fmaf(g, S[t], staged_k[token * DP + wave * RPT + t] * value);
                read = fmaf(S[t], staged_q[token * DP + wave * RPT + t], read);
            }
            parts[(token * 4 + wave) * 64 + lane] = read;
        }
        __syncthreads();
        for (int i = threadIdx.x; i < tokens * 64; i += 256) {
            const int token = i / 64, c = i % 64;
            if (block * 64 + c < vdim) {
                const float* p = parts + token * 256 + c;
                out[((size_t)(first + base + token) * heads + head) * vdim + block * 64 + c] = ((p[0] + p[64]) + p[128]) + p[192];
            }
        }
    }
    if (live) {
#pragma unroll
        for (int t = 0; t < RPT; ++t) {
            const int key = wave * RPT + t;
            if (key < dim) mine[(size_t)key * vdim] = S[t];
        }
    }
}

extern "C" int fw_decay_recurrence(const float* q, const float* k, const float* v, int stride, const float* decay, float* state, int slots,
                                   float* out, const int32_t* seg_row0, const int32_t* seg_slot, int rows, int segments, int heads, int dim,
                                   int vdim, void* stream) {
    FW_REQUIRE(rows >= 0 && segments >= 0 && heads > 0 && heads <= 65535 && slots > 0, "decay_recurrence: bad sizes rows=%d segments=%d heads=%d",
               rows, segments, heads);
    FW_REQUIRE(dim >= 1 && dim <= 256 && vdim >= 1 && vdim <= 1 << 20, "decay_recurrence: heads of %d (1..256) and %d channels", dim, vdim);
    FW_REQUIRE(stride >= heads * dim && stride >= heads * vdim, "decay_recurrence: rows of %d values do not hold %d heads of %d / %d", stride, heads, dim, vdim);
    if (rows == 0 || segments == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid(segments, heads, fw_ceil_div(vdim, 64));
#define FW_DECAY_LAUNCH(RPT) \
    decay_recurrence_step_kernel<RPT><<<grid, 256, 0, s>>>(q, k, v, stride, decay, state, out, seg_row0, seg_slot, heads, dim, vdim, 0)
    if (dim <= 16) FW_DECAY_LAUNCH(4);
    else if (dim <= 32) FW_DECAY_LAUNCH(8);
    else if (dim <= 64) FW_DECAY_LAUNCH(16);
    else if (dim <= 128) FW_DECAY_LAUNCH(32);
    else FW_DECAY_LAUNCH(64);
#undef FW_DECAY_LAUNCH
    FW_LAUNCH_CHECK("decay_recurrence");
    return 0;
}
