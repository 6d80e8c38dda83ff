// A linear recurrence over a matrix state per head with one fixed decay per head ("lightning attention"). Per head, a
// token brings q, k (dim channels) and v (vdim channels), each the silu of a projection:
//     S <- decay S + k v^T;   o = S^T q
// (the read-out sees the token's own write). State [slot][head][dim][vdim] float32, zero at a request's start.
//
// All arithmetic is float32, whatever the run's dtype. powers [head][DR_CHUNK + 1]: decay^0 .. decay^DR_CHUNK.
#include "fw_common.h"
#include "fw_kernels.h"

#define DR_CHUNK 64

__device__ __forceinline__ float dr_silu(float z) { return z / (1.0f + expf(-z)); }

// ---- token by token ---------------------------------------------------------------------------------------------
// Workgroup (segment, head, block of 64 value channels): a lane owns a value channel, the four waves share the key
// channels out (RPT neighbouring ones each, the state's columns of them in registers). DR_TOKENS tokens at a time are
// staged in LDS, silu applied; a wave's part of a token's read-out goes to LDS and the four parts are added, in order,
// once per chunk. Segments of more than `long_rows` rows are left alone (long_rows > 0).
#define DR_TOKENS 16
template <int RPT>
__global__ __launch_bounds__(256) void decay_recurrence_step_kernel(
    const float* __restrict__ q, const float* __restrict__ k, const float* __restrict__ v, int stride, const float* __restrict__ powers,
    float* __restrict__ state, float* __restrict__ out, const int32_t* __restrict__ seg_row0, const int32_t* __restrict__ seg_slot, int heads,
    int dim, int vdim, int long_rows) {
    constexpr int DP = 4 * RPT;
    __shared__ __attribute__((aligned(16))) float staged_q[DR_TOKENS * DP];
    __shared__ __attribute__((aligned(16))) float staged_k[DR_TOKENS * DP];
    __shared__ float staged_v[DR_TOKENS * 64];
    __shared__ float parts[DR_TOKENS * 4 * 64];
    const int seg = blockIdx.x, head = blockIdx.y, block = blockIdx.z;
    const int first = seg_row0[seg], count = seg_row0[seg + 1] - first;
    if (long_rows > 0 && count > long_rows) return;     // the chunked kernels take it
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int column = block * 64 + lane;
    const bool live = column < vdim;
    float* mine = state + ((size_t)seg_slot[seg] * heads + head) * dim * vdim + (live ? column : 0);
    const float g = powers[head * (DR_CHUNK + 1) + 1];
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

// ---- in chunks --------------------------------------------------------------------------------------------------
// Long segments are cut into chunks of DR_CHUNK rows (chunk_seg, chunk_row0: the chunks of all long segments, those of a
// segment side by side; seg_chunk0 [segments + 1]: where a segment's chunks begin, an empty range for a short one). With a
// chunk's n rows counted from 0 and S_in the state ahead of it,
//     o_i = decay^(i + 1) S_in^T q_i + sum_{j <= i} decay^(i - j) (q_i . k_j) v_j
//     S_out = decay^n S_in + sum_j decay^(n - 1 - j) k_j v_j^T
// in three launches: every chunk's own sum of S_out (side by side), the states ahead of the chunks (a thread per element of
// a head's state walks the chunks), and the read-outs (side by side). The products run on the matrix cores in float32
// (v_mfma_f32_32x32x2f32: exact products, float32 sums), so both run dtypes share the kernels.
typedef __attribute__((ext_vector_type(16))) float dr_f32x16;
typedef __attribute__((ext_vector_type(4))) float dr_f32x4;

__device__ __forceinline__ float dr_silu_quick(float z) { return z * __builtin_amdgcn_rcpf(1.0f + __expf(-z)); }

// Copies a chunk's rows of one head's q and k (or k alone: q null) into LDS rows `pitch` apart, silu applied; what lies past the
// chunk's last row, and past dim up to `width`, is zero. 256 threads; eight elements of each are asked for before any is used.
template <bool BOTH>
__device__ __forceinline__ void dr_stage(const float* __restrict__ q, const float* __restrict__ k, int stride, int tokens, int dim, int width,
                                         int pitch, float* lq, float* lk, const float* weight) {
    const int shift = width <= 32 ? 5 : width <= 64 ? 6 : width <= 128 ? 7 : 8;     // columns are numbered in a power of two
    for (int base = threadIdx.x; base < (DR_CHUNK << shift); base += 256 * 8) {
        float zq[8], zk[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            const int i = base + 256 * u;
            const int token = i >> shift, c = i & ((1 << shift) - 1);
            const int at = (token < tokens ? token : tokens - 1) * stride + (c < dim ? c : dim - 1);
            if (BOTH) zq[u] = q[at];
            zk[u] = k[at];
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            const int i = base + 256 * u;
            const int token = i >> shift, c = i & ((1 << shift) - 1);
            if (token >= DR_CHUNK || c >= width) continue;
            const bool there = token < tokens && c < dim;
            if (BOTH) lq[token * pitch + c] = there ? dr_silu_quick(zq[u]) : 0.0f;
            lk[token * pitch + c] = there ? dr_silu_quick(zk[u]) * (weight ? weight[tokens - 1 - token] : 1.0f) : 0.0f;
        }
    }
}

__device__ __forceinline__ dr_f32x16 dr_zero() {
    dr_f32x16 acc;
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[r] = 0.0f;
    return acc;
}

// The chunk's own sum, [dim][vdim] to local[chunk][head]. A wave owns 32 value channels at a time and up to 128 key
// channels of them; k (times its decay) lies in LDS, [token][dim padded to 32], v comes straight from memory: only this
// wave reads it. The product's inner dimension is the token: lanes 0..31 hold the even token of a step, lanes 32..63
// the odd one.
__global__ __launch_bounds__(256, 2) void decay_chunk_sum_kernel(const float* __restrict__ k, const float* __restrict__ v, int stride,
                                                              const float* __restrict__ powers, float* __restrict__ local,
                                                              const int32_t* __restrict__ chunk_seg, const int32_t* __restrict__ chunk_row0,
                                                              const int32_t* __restrict__ seg_row0, int heads, int dim, int vdim) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int chunk = blockIdx.x, head = blockIdx.y;
    const int row0 = chunk_row0[chunk], end = seg_row0[chunk_seg[chunk] + 1];
    const int tokens = end - row0 < DR_CHUNK ? end - row0 : DR_CHUNK;
    const int dp = (dim + 31) & ~31;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, half = lane >> 5, column = lane & 31;
    const float* p = powers + head * (DR_CHUNK + 1);
    dr_stage<false>(nullptr, k + (size_t)row0 * stride + (size_t)head * dim, stride, tokens, dim, dp, dp, nullptr, lds, p);
    __syncthreads();
    float* to = local + ((size_t)chunk * heads + head) * dim * vdim;
    for (int col0 = wave * 32; col0 < vdim; col0 += 128) {
        const int col = col0 + column;
        const float* from = v + (size_t)row0 * stride + (size_t)head * vdim + (col < vdim ? col : vdim - 1);
        float value[DR_CHUNK / 2];
#pragma unroll
        for (int t = 0; t < DR_CHUNK / 2; ++t) {
            const int token = 2 * t + half;
            value[t] = from[(size_t)(token < tokens ? token : tokens - 1) * stride];
        }
#pragma unroll
        for (int t = 0; t < DR_CHUNK / 2; ++t) value[t] = dr_silu_quick(value[t]);      // (a row past the chunk's end meets k = 0)
        for (int key0 = 0; key0 < dp; key0 += 128) {
            const int tiles = (dp - key0) / 32 < 4 ? (dp - key0) / 32 : 4;
            dr_f32x16 acc[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) acc[i] = dr_zero();
#pragma unroll 8
            for (int t = 0; t < DR_CHUNK / 2; ++t) {
                const float* row = lds + (2 * t + half) * dp + key0 + column;
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (i < tiles) acc[i] = __builtin_amdgcn_mfma_f32_32x32x2f32(row[32 * i], value[t], acc[i], 0, 0, 0);
            }
            fw_mfma_drain();
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int r = 0; r < 16; ++r) {
                    const int key = key0 + 32 * i + 8 * (r >> 2) + 4 * half + (r & 3);
                    if (i < tiles && key < dim && col < vdim) to[(size_t)key * vdim + col] = acc[i][r];
                }
        }
    }
}

// local[chunk] becomes the state ahead of the chunk; the slot moves on to the state behind the segment. A thread per
// element of (segment, head): nothing but loads and one multiply-add per chunk.
__global__ __launch_bounds__(256) void decay_chunk_state_kernel(const float* __restrict__ powers, float* __restrict__ local, float* __restrict__ state,
                                                                const int32_t* __restrict__ seg_chunk0, const int32_t* __restrict__ seg_row0,
                                                                const int32_t* __restrict__ seg_slot, int heads, int size) {
    const int seg = blockIdx.x, head = blockIdx.y;
    const int begin = seg_chunk0[seg], chunks = seg_chunk0[seg + 1] - begin;
    const int i = blockIdx.z * 256 + threadIdx.x;
    if (chunks <= 0 || i >= size) return;
    const int count = seg_row0[seg + 1] - seg_row0[seg];
    const float* p = powers + head * (DR_CHUNK + 1);
    const float whole = p[DR_CHUNK], last = p[count - (chunks - 1) * DR_CHUNK];
    float* slot = state + ((size_t)seg_slot[seg] * heads + head) * size + i;
    float* at = local + ((size_t)begin * heads + head) * size + i;
    const size_t step = (size_t)heads * size;
    float S = *slot;
    for (int c = 0; c < chunks; c += 8) {
        float own[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) own[u] = at[(size_t)(c + u < chunks ? c + u : chunks - 1) * step];
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            if (c + u >= chunks) break;
            at[(size_t)(c + u) * step] = S;
            S = fmaf(c + u == chunks - 1 ? last : whole, S, own[u]);
        }
    }
    *slot = S;
}

// The read-outs of a chunk and head. q and k lie in LDS (rows of dim padded to 8, and four more: the 16-byte reads of 32
// rows then spread over the banks); the scores take k's place once they are formed. A wave owns 32 value channels at a
// time: S_in and v come straight from memory, only this wave reads them. A step of a product over channels takes eight of them:
// lanes 0..31 the first four, lanes 32..63 the next four, one per instruction.
__global__ __launch_bounds__(256, 2) void decay_chunk_read_kernel(const float* __restrict__ q, const float* __restrict__ k, const float* __restrict__ v,
                                                               int stride, const float* __restrict__ powers, const float* __restrict__ local,
                                                               float* __restrict__ out, const int32_t* __restrict__ chunk_seg,
                                                               const int32_t* __restrict__ chunk_row0, const int32_t* __restrict__ seg_row0,
                                                               int heads, int dim, int vdim) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int chunk = blockIdx.x, head = blockIdx.y;
    const int row0 = chunk_row0[chunk], end = seg_row0[chunk_seg[chunk] + 1];
    const int tokens = end - row0 < DR_CHUNK ? end - row0 : DR_CHUNK;
    const int dp = (dim + 7) & ~7, pitch = dp + 4;
    constexpr int SCORES = DR_CHUNK + 4;                // a row of scores
    float* lq = lds;
    float* lk = lds + DR_CHUNK * pitch;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, half = lane >> 5, within = lane & 31;
    const float* p = powers + head * (DR_CHUNK + 1);
    const size_t at = (size_t)row0 * stride + (size_t)head * dim;
    dr_stage<true>(q + at, k + at, stride, tokens, dim, dp, pitch, lq, lk, nullptr);
    __syncthreads();
    // scores: a 32 x 32 tile a wave; the tile above the diagonal is zero
    const int ti = wave >> 1, tj = wave & 1;
    dr_f32x16 scores = dr_zero();
    if (tj <= ti) {
        const float* rq = lq + (ti * 32 + within) * pitch + 4 * half;
        const float* rk = lk + (tj * 32 + within) * pitch + 4 * half;
#pragma unroll 4
        for (int c = 0; c < dp; c += 8) {
            const dr_f32x4 a = *reinterpret_cast<const dr_f32x4*>(rq + c), b = *reinterpret_cast<const dr_f32x4*>(rk + c);
#pragma unroll
            for (int e = 0; e < 4; ++e) scores = __builtin_amdgcn_mfma_f32_32x32x2f32(a[e], b[e], scores, 0, 0, 0);
        }
    }
    fw_mfma_drain();
    __syncthreads();                                    // k has been read by all
    float* ls = lk;
#pragma unroll
    for (int r = 0; r < 16; ++r) {
        const int i = ti * 32 + 8 * (r >> 2) + 4 * half + (r & 3), j = tj * 32 + within;
        ls[i * SCORES + j] = j <= i ? scores[r] * p[i - j] : 0.0f;
    }
    __syncthreads();
    const float* S_in = local + ((size_t)chunk * heads + head) * dim * vdim;
    for (int col0 = wave * 32; col0 < vdim; col0 += 128) {
        const int col = col0 + within, safe = col < vdim ? col : vdim - 1;
        dr_f32x16 acc[2] = {dr_zero(), dr_zero()};
        const float* rq = lq + within * pitch + 4 * half;
#pragma unroll 4
        for (int c = 0; c < dp; c += 8) {
            const dr_f32x4 a0 = *reinterpret_cast<const dr_f32x4*>(rq + c), a1 = *reinterpret_cast<const dr_f32x4*>(rq + 32 * pitch + c);
            float b[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int key = c + 4 * half + e;       // (channels past dim meet q = 0; they are read at the last one)
                b[e] = S_in[(size_t)(key < dim ? key : dim - 1) * vdim + safe];
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                acc[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(a0[e], b[e], acc[0], 0, 0, 0);
                acc[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(a1[e], b[e], acc[1], 0, 0, 0);
            }
        }
        fw_mfma_drain();
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int r = 0; r < 16; ++r) acc[i][r] *= p[i * 32 + 8 * (r >> 2) + 4 * half + (r & 3) + 1];
        const float* from = v + (size_t)row0 * stride + (size_t)head * vdim + safe;
#pragma unroll
        for (int t = 0; t < DR_CHUNK; t += 8) {
            float b[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int token = t + 4 * half + e;
                b[e] = dr_silu_quick(from[(size_t)(token < tokens ? token : tokens - 1) * stride]);     // (its scores are zero)
            }
            const dr_f32x4 a1 = *reinterpret_cast<const dr_f32x4*>(ls + (32 + within) * SCORES + t + 4 * half);
            if (t < 32) {
                const dr_f32x4 a0 = *reinterpret_cast<const dr_f32x4*>(ls + within * SCORES + t + 4 * half);
#pragma unroll
                for (int e = 0; e < 4; ++e) acc[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(a0[e], b[e], acc[0], 0, 0, 0);
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) acc[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(a1[e], b[e], acc[1], 0, 0, 0);
        }
        fw_mfma_drain();
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                const int token = i * 32 + 8 * (r >> 2) + 4 * half + (r & 3);
                if (token < tokens && col < vdim) out[((size_t)(row0 + token) * heads + head) * vdim + col] = acc[i][r];
            }
    }
}

extern "C" int fw_decay_chunk_rows(void) { return DR_CHUNK; }

extern "C" int fw_decay_recurrence(const float* q, const float* k, const float* v, int stride, const float* powers, float* state, int slots,
                                   float* out, const int32_t* seg_row0, const int32_t* seg_slot, int rows, int segments, int heads, int dim,
                                   int vdim, const int32_t* chunk_seg, const int32_t* chunk_row0, const int32_t* seg_chunk0, int chunks,
                                   int long_rows, int all_long, float* workspace, void* stream) {
    FW_REQUIRE(rows >= 0 && segments >= 0 && heads > 0 && heads <= 65535 && slots > 0, "decay_recurrence: bad sizes rows=%d segments=%d heads=%d",
               rows, segments, heads);
    FW_REQUIRE(dim >= 1 && dim <= 256 && vdim >= 1 && vdim <= 65536, "decay_recurrence: heads of %d (1..256) and %d channels", dim, vdim);
    FW_REQUIRE(stride <= 1 << 24, "decay_recurrence: rows of %d values", stride);
    FW_REQUIRE(stride >= heads * dim && stride >= heads * vdim, "decay_recurrence: rows of %d values do not hold %d heads of %d / %d", stride, heads, dim, vdim);
    FW_REQUIRE(chunks >= 0 && (chunks == 0 || (chunk_seg && chunk_row0 && seg_chunk0 && workspace && long_rows > 0)),
               "decay_recurrence: chunks come with their places, a workspace and the length from which they are used");
    if (rows == 0 || segments == 0) return 0;
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid(segments, heads, fw_ceil_div(vdim, 64));
    if (chunks == 0 || !all_long) {
#define FW_DECAY_LAUNCH(RPT)                                                                                                             \
        decay_recurrence_step_kernel<RPT><<<grid, 256, 0, s>>>(q, k, v, stride, powers, state, out, seg_row0, seg_slot, heads, dim, vdim, \
                                                               chunks > 0 ? long_rows : 0)
        if (dim <= 16) FW_DECAY_LAUNCH(4);
        else if (dim <= 32) FW_DECAY_LAUNCH(8);
        else if (dim <= 64) FW_DECAY_LAUNCH(16);
        else if (dim <= 128) FW_DECAY_LAUNCH(32);
        else FW_DECAY_LAUNCH(64);
#undef FW_DECAY_LAUNCH
        FW_LAUNCH_CHECK("decay_recurrence");
    }
    if (chunks == 0) return 0;
    const int sum_bytes = DR_CHUNK * ((dim + 31) & ~31) * 4;
    const int read_width = ((dim + 7) & ~7) + 4;
    const int read_bytes = DR_CHUNK * (read_width + (read_width > DR_CHUNK + 4 ? read_width : DR_CHUNK + 4)) * 4;
    static bool configured = false;
    if (!configured) {
        hipError_t status = hipFuncSetAttribute((const void*)decay_chunk_sum_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, DR_CHUNK * 256 * 4);
        if (status == hipSuccess)
            status = hipFuncSetAttribute((const void*)decay_chunk_read_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, DR_CHUNK * 2 * 260 * 4);
        FW_REQUIRE(status == hipSuccess, "decay_recurrence: cannot reserve LDS: %s", hipGetErrorString(status));
        configured = true;
    }
    const dim3 by_chunk(chunks, heads);
    decay_chunk_sum_kernel<<<by_chunk, 256, sum_bytes, s>>>(k, v, stride, powers, workspace, chunk_seg, chunk_row0, seg_row0, heads, dim, vdim);
    FW_LAUNCH_CHECK("decay_recurrence (chunks)");
    const dim3 by_element(segments, heads, fw_ceil_div((long long)dim * vdim, 256));
    decay_chunk_state_kernel<<<by_element, 256, 0, s>>>(powers, workspace, state, seg_chunk0, seg_row0, seg_slot, heads, dim * vdim);
    FW_LAUNCH_CHECK("decay_recurrence (states)");
    decay_chunk_read_kernel<<<by_chunk, 256, read_bytes, s>>>(q, k, v, stride, powers, workspace, out, chunk_seg, chunk_row0, seg_row0, heads, dim, vdim);
    FW_LAUNCH_CHECK("decay_recurrence (read)");
    return 0;
}
