// Shared device helpers for the gfx950 kernels: storage types, conversions, wave64
// reductions, and the error channel behind the flat C ABI.
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

// dtype codes used across the C ABI
#define FW_F32 0
#define FW_BF16 1

// ---- error channel: every entry point returns 0 or -1 and leaves a message ---------
void fw_set_error(const char* format, ...);
// A workgroup barrier that orders LDS traffic only. __syncthreads() also waits for every global
// load in flight (its fence covers global memory), which empties a prefetch pipeline at each
// barrier; use this one where waves hand data to each other through LDS alone.
__device__ __forceinline__ void fw_lds_barrier() {
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
    __builtin_amdgcn_s_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
}

// Reductions over the four lanes l, l ^ 16, l ^ 32, l ^ 48 of a wave (every lane gets the result)
// with the row-swap instructions of gfx950 instead of two trips through the LDS crossbar
// (__shfl_xor). v_permlane16_swap exchanges rows 1 and 3 of its first register with rows 0 and 2
// of its second; v_permlane32_swap the upper half of the first with the lower half of the second.
// Given one value in two registers, the two results of a swap are the two partners of a lane.
// The second copy is made opaque: given one value twice the compiler may name one register
// twice, and the instruction then swaps rows inside that register. The results are taken as
// scalars before they are reinterpreted (a bit cast straight from the builtin's vector result
// lost its second element at compile time).
__device__ __forceinline__ void fw_quad_partners16(float x, float& mine, float& partner) {
    uint32_t u = __float_as_uint(x), copy = u;
    asm volatile("" : "+v"(copy));
    const auto swapped = __builtin_amdgcn_permlane16_swap(u, copy, false, false);
    const uint32_t first = swapped[0], second = swapped[1];
    mine = __uint_as_float(first);
    partner = __uint_as_float(second);
}
__device__ __forceinline__ void fw_quad_partners32(float x, float& mine, float& partner) {
    uint32_t u = __float_as_uint(x), copy = u;
    asm volatile("" : "+v"(copy));
    const auto swapped = __builtin_amdgcn_permlane32_swap(u, copy, false, false);
    const uint32_t first = swapped[0], second = swapped[1];
    mine = __uint_as_float(first);
    partner = __uint_as_float(second);
}
__device__ __forceinline__ float fw_quad_max(float x) {
    float a, b;
    fw_quad_partners16(x, a, b);
    fw_quad_partners32(fmaxf(a, b), a, b);
    return fmaxf(a, b);
}
__device__ __forceinline__ float fw_quad_sum(float x) {
    float a, b;
    fw_quad_partners16(x, a, b);
    fw_quad_partners32(a + b, a, b);
    return a + b;
}

// Lets the matrix pipe finish what was issued before control goes on. Inside one basic block the
// compiler keeps a product and the first read of its result far enough apart; where the read is
// the target of a taken branch it has been seen one instruction behind the product, reading the
// registers the product writes last before they were written (seen in the attention kernel with
// head sizes below the template's: two of four components stale). Called once behind a loop of
// products, before branches that lead to code reading the accumulators. 24 wait states cover the
// longest product (16 passes).
__device__ __forceinline__ void fw_mfma_drain() {
    __builtin_amdgcn_sched_barrier(0);
    asm volatile("s_nop 15\n\ts_nop 7");
    __builtin_amdgcn_sched_barrier(0);
}

#define FW_REQUIRE(cond, ...)                    \
    do {                                         \
        if (!(cond)) {                           \
            fw_set_error(__VA_ARGS__);           \
            return -1;                           \
        }                                        \
    } while (0)
#define FW_LAUNCH_CHECK(name)                                                     \
    do {                                                                          \
        hipError_t fw_status__ = hipGetLastError();                               \
        if (fw_status__ != hipSuccess) {                                          \
            fw_set_error("%s: launch failed: %s", name, hipGetErrorString(fw_status__)); \
            return -1;                                                            \
        }                                                                         \
    } while (0)

// ---- bfloat16 as raw bits ----------------------------------------------------------
struct bf16_t {
    uint16_t bits;
};

__device__ __forceinline__ float bf16_to_float(bf16_t v) {
    return __uint_as_float(((uint32_t)v.bits) << 16);
}
__device__ __forceinline__ float bf16_bits_to_float(uint32_t bits) {
    return __uint_as_float(bits << 16);
}
// round to nearest, ties to even; NaN stays NaN
__device__ __forceinline__ uint16_t float_to_bf16_bits(float f) {
    uint32_t u = __float_as_uint(f);
    if ((u & 0x7fffffffu) > 0x7f800000u) return (uint16_t)((u >> 16) | 0x0040u);
    u += 0x7fffu + ((u >> 16) & 1u);
    return (uint16_t)(u >> 16);
}
__device__ __forceinline__ bf16_t float_to_bf16(float f) {
    bf16_t r;
    r.bits = float_to_bf16_bits(f);
    return r;
}

template <typename T> __device__ __forceinline__ float load_as_float(const T* p, size_t i);
template <> __device__ __forceinline__ float load_as_float<float>(const float* p, size_t i) { return p[i]; }
template <> __device__ __forceinline__ float load_as_float<bf16_t>(const bf16_t* p, size_t i) {
    return bf16_to_float(p[i]);
}
template <typename T> __device__ __forceinline__ void store_from_float(T* p, size_t i, float v);
template <> __device__ __forceinline__ void store_from_float<float>(float* p, size_t i, float v) { p[i] = v; }
template <> __device__ __forceinline__ void store_from_float<bf16_t>(bf16_t* p, size_t i, float v) {
    p[i] = float_to_bf16(v);
}
// the value a store of this type would leave behind (used where a value is both kept
// in registers and written, so later reads from memory see the same number)
template <typename T> __device__ __forceinline__ float round_through(float v);
template <> __device__ __forceinline__ float round_through<float>(float v) { return v; }
template <> __device__ __forceinline__ float round_through<bf16_t>(float v) {
    return bf16_bits_to_float(float_to_bf16_bits(v));
}

// ---- wave64 reductions (fixed butterfly order: the result does not depend on
//      anything but the 64 inputs) -----------------------------------------------------
__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int offset = 32; offset > 0; offset >>= 1) v += __shfl_xor(v, offset, 64);
    return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
    for (int offset = 32; offset > 0; offset >>= 1) v = fmaxf(v, __shfl_xor(v, offset, 64));
    return v;
}

// block-wide sum for blocks of up to 1024 threads; every thread gets the result
__device__ __forceinline__ float block_sum(float v, float* scratch /* >= 16 floats */) {
    const int lane = threadIdx.x & 63;
    const int wave = threadIdx.x >> 6;
    const int waves = (blockDim.x + 63) >> 6;
    v = wave_sum(v);
    __syncthreads();
    if (lane == 0) scratch[wave] = v;
    __syncthreads();
    float total = 0.0f;
    for (int i = 0; i < waves; ++i) total += scratch[i];
    return total;
}

// The same over 256 threads, the waves meeting over LDS alone (loads and stores on the way stay on the way);
// the parts are added in the same order. Every sum of a kernel has four floats of its own.
__device__ __forceinline__ float block_sum_by_lds(float v, float* scratch) {
    v = wave_sum(v);
    if ((threadIdx.x & 63) == 0) scratch[threadIdx.x >> 6] = v;
    fw_lds_barrier();
    return ((scratch[0] + scratch[1]) + scratch[2]) + scratch[3];
}

// The tanh form of gelu, 0.5 z (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3))), is z * sigmoid of this
// (0.5 (1 + tanh(y)) = sigmoid(2 y)).
__device__ __forceinline__ float fw_gelu_tanh_argument(float z) { return 1.5957691216057308f * z * fmaf(0.044715f * z, z, 1.0f); }
// ... for results that are rounded to bfloat16
__device__ __forceinline__ float fw_gelu_tanh_quick(float z) { return z * __builtin_amdgcn_rcpf(1.0f + __expf(-fw_gelu_tanh_argument(z))); }

// A gated unit behind a product that holds gate and up of one feature: silu(g) * u (limit 0), gelu_tanh(g) * u (limit < 0), or
// with clamped halves g' = min(g, limit), u' = clamp(u, -limit, limit): g' * sigmoid(alpha g') * (u' + shift).
// `silu` is the product's own form of silu(g) * u, so that the plain unit's results stay what they were.
template <typename Silu>
__device__ __forceinline__ float fw_gated_unit(float g, float u, float limit, float alpha, float shift, Silu silu) {
    if (limit < 0.0f) return fw_gelu_tanh_quick(g) * u;
    if (limit == 0.0f) return silu(g) * u;
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    const float z = alpha * g;
    const float e = __expf(z >= 0.0f ? -z : z);
    return g * (z >= 0.0f ? 1.0f / (1.0f + e) : e / (1.0f + e)) * (u + shift);
}

// z Phi(z), Phi the normal distribution's cumulative function: the exact gelu
__device__ __forceinline__ float fw_gelu(float z) { return 0.5f * z * (1.0f + erff(z * 0.70710678118654752f)); }

// The exact gelu for results that are rounded to bfloat16: the complement of the error function as a polynomial in 1 / (1 + p x)
// times e^(-x^2) (Abramowitz and Stegun, Handbook of Mathematical Functions, 7.1.26: within 1.5e-7), which gives the
// lower half of Phi without a difference of nearly equal numbers.
__device__ __forceinline__ float fw_gelu_quick(float z) {
    const float x = fabsf(z) * 0.70710678118654752f;
    const float t = __builtin_amdgcn_rcpf(fmaf(0.3275911f, x, 1.0f));
    float poly = fmaf(1.061405429f, t, -1.453152027f);
    poly = fmaf(poly, t, 1.421413741f);
    poly = fmaf(poly, t, -0.284496736f);
    poly = fmaf(poly, t, 0.254829592f);
    const float lower = 0.5f * poly * t * __builtin_amdgcn_exp2f(-x * x * 1.4426950408889634f);      // Phi(-|z|)
    return z * (z < 0.0f ? lower : 1.0f - lower);
}

// A product that stores gelu(sum) in bfloat16 is the storing product with this output type (dtype code
// FW_BF16_GELU): the unit is formed from the float32 sum and rounded once.
#define FW_BF16_GELU 2
struct gelu_bf16_t {
    uint16_t bits;
};
template <> __device__ __forceinline__ float load_as_float<gelu_bf16_t>(const gelu_bf16_t* p, size_t i) { return bf16_bits_to_float(p[i].bits); }
template <> __device__ __forceinline__ void store_from_float<gelu_bf16_t>(gelu_bf16_t* p, size_t i, float v) {
    p[i].bits = float_to_bf16_bits(fw_gelu_quick(v));
}
// what a store of this output type does to a float32 sum before it is rounded (for stores that pack several values)
template <typename T> __device__ __forceinline__ float fw_before_store(float v) { return v; }
template <> __device__ __forceinline__ float fw_before_store<gelu_bf16_t>(float v) { return fw_gelu_quick(v); }

// The gated product (gate rows, then up rows) with this output type (dtype code FW_BF16_GEGLU) stores gelu_tanh(gate) * up in
// bfloat16 in place of silu(gate) * up.
#define FW_BF16_GEGLU 3
struct geglu_bf16_t {
    uint16_t bits;
};
template <> __device__ __forceinline__ void store_from_float<geglu_bf16_t>(geglu_bf16_t* p, size_t i, float v) { p[i].bits = float_to_bf16_bits(v); }
template <> __device__ __forceinline__ float load_as_float<geglu_bf16_t>(const geglu_bf16_t* p, size_t i) { return bf16_bits_to_float(p[i].bits); }
// what the gate passes, by the output's type; `silu` is the product's own form of silu
template <typename T, typename Silu> struct fw_gate {
    static __device__ __forceinline__ float of(float g, Silu silu) { return silu(g); }
};
template <typename Silu> struct fw_gate<geglu_bf16_t, Silu> {
    static __device__ __forceinline__ float of(float g, Silu) { return fw_gelu_tanh_quick(g); }
};
template <typename T, typename Silu> __device__ __forceinline__ float fw_gate_of(float g, Silu silu) { return fw_gate<T, Silu>::of(g, silu); }

// The first key that a row at position `pos` may see: with a window the last `window` keys (itself
// among them), with a chunk only the keys of its own chunk (chunks counted from position 0 of the
// sequence); 0 switches either off. Never falls as the position rises.
__host__ __device__ __forceinline__ int fw_first_visible(int pos, int window, int chunk) {
    int first = window > 0 && pos - window + 1 > 0 ? pos - window + 1 : 0;
    if (chunk > 0) {
        const int start = pos - pos % chunk;
        first = start > first ? start : first;
    }
    return first;
}

static inline int fw_ceil_div(long long a, long long b) { return (int)((a + b - 1) / b); }

// Eight bfloat16 of a weight matrix that a decode step reads once: with `streamed` the load says
// so (nontemporal), which keeps a stream of weights from pushing the step's activations out of the
// caches and, on whole 1 KB pieces per wave, reads faster (a read-only kernel over 268 MB: 39.5 against
// 43.7 us). Weights in row-major order are loaded as they always were.
typedef __attribute__((ext_vector_type(8))) __bf16 fw_bf16x8;
typedef __attribute__((ext_vector_type(4))) uint32_t fw_u32x4;
template <bool STREAMED>
__device__ __forceinline__ fw_bf16x8 fw_load_weights(const uint16_t* from) {
    const fw_u32x4* at = reinterpret_cast<const fw_u32x4*>(from);
    const fw_u32x4 v = STREAMED ? __builtin_nontemporal_load(at) : *at;
    return __builtin_bit_cast(fw_bf16x8, v);
}

// ---- candidates for the next token ----------------------------------------------------
// A candidate is ordered by (value descending, id ascending); NaN sorts last. The key packs both
// so that one 64-bit comparison orders two candidates (a greater key comes first) and ties go to
// the lowest id, as the reference's fused LM-head argmax does
// (native/include/flyweight_v2_qwen_kernels.hpp:2391-2405).
__device__ __forceinline__ unsigned long long candidate_key(float value, int id) {
    uint32_t bits = value == 0.0f ? 0u : __float_as_uint(value);        // -0 and +0 are one value: the lower id first
    uint32_t ordered;
    if (value != value) ordered = 0u;                                   // NaN: below everything
    else ordered = (bits & 0x80000000u) ? ~bits : (bits | 0x80000000u); // monotone in value
    return ((unsigned long long)ordered << 32) | (unsigned long long)(0xffffffffu - (uint32_t)id);
}
__device__ __forceinline__ int candidate_id(unsigned long long key) { return (int)(0xffffffffu - (uint32_t)(key & 0xffffffffull)); }

