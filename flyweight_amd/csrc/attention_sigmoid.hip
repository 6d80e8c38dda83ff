// Attention over the paged cache whose weights are sigmoids and whose heads mix their weights:
//     a_g(i, j) = sigmoid(q_g . k * scale + bias[g])            (each visible key on its own: no sum over keys)
//     out_h(i)  = gate . sum_j (sum_g mix[h][g] a_g(i, j)) v_j  (v of h's own key/value head; gate = sigmoid(raw))
// The mix needs every head's weight of one (row, key) pair at once, so a workgroup works on all heads.
// There is no running maximum and nothing to rescale: parts of a row's keys simply add up. Scores,
// sigmoids, the mix and every sum are float32. A sliding window bounds the keys (0: every earlier key).
//
// Cache layout as in attention_generic.hip: K [page][kv_head][64][head_dim], V [page][kv_head][v_dim][64].
#include "fw_common.h"
#include "fw_kernels.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) float f32x4;
typedef __attribute__((ext_vector_type(4))) uint32_t u32x4;
typedef __attribute__((ext_vector_type(2))) uint32_t u32x2;
typedef __attribute__((ext_vector_type(2))) float f32x2;
typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2;

#define PAGE 64
#define SG_MAX_HEADS 256            // of the plain kernel
#define SG_MAX_DIM 1024
#define SG_TILE_HEADS 16            // of the matrix-core kernels
#define LOG2E_F 1.4426950408889634f

__device__ __forceinline__ uint32_t sg_pack(float lo, float hi) {
    const f32x2 v = {lo, hi};
    return __builtin_bit_cast(uint32_t, __builtin_convertvector(v, bf16x2));
}
// a factor on an output channel: sigmoid of the gate's raw value
__device__ __forceinline__ float sg_gate(float z) { return 1.0f / (1.0f + expf(-z)); }
// the same by the hardware's 2^x and reciprocal (about 1e-7 of the result), for results that are rounded to bfloat16
__device__ __forceinline__ float sg_gate_quick(float z) { return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-z * LOG2E_F)); }

// ---- the plain kernel: any sizes, float32 arithmetic ------------------------------------------------
// A workgroup per (row, run of output heads). Per page: a wave's lanes are the page's keys and its heads
// every fourth one; the weights of all heads meet in LDS, the mix for the workgroup's own heads is formed
// there, and every thread adds the page to its outputs. Sums run over the keys in order.
#define SG_HELD 16
template <typename T>
__global__ __launch_bounds__(256) void sigmoid_attention_generic_kernel(
    const T* __restrict__ q, T* __restrict__ out, const T* __restrict__ k_pages, const T* __restrict__ v_pages,
    const int32_t* __restrict__ block_table, int table_stride, const int32_t* __restrict__ row_seg,
    const int32_t* __restrict__ row_pos, int num_heads, int num_kv_heads, int head_dim, int v_dim, float scale, int window,
    const float* __restrict__ bias, const float* __restrict__ mix, const float* __restrict__ gate, int gate_stride, int heads_per_block) {
    extern __shared__ float sg_lds[];
    float* weights = sg_lds;                                // [heads][64]
    float* mixed = sg_lds + num_heads * PAGE;               // [heads of the workgroup][64]
    const int row = blockIdx.x, head0 = blockIdx.y * heads_per_block;
    const int heads_here = num_heads - head0 < heads_per_block ? num_heads - head0 : heads_per_block;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int group = num_heads / num_kv_heads;
    const int pos = row_pos[row];
    const int first = fw_first_visible(pos, window, 0);
    const int32_t* table = block_table + (size_t)row_seg[row] * table_stride;
    float acc[SG_HELD];
#pragma unroll
    for (int u = 0; u < SG_HELD; ++u) acc[u] = 0.0f;
    for (int tile = first / PAGE; tile <= pos / PAGE; ++tile) {
        const int page = table[tile];
        const int t = tile * PAGE + lane;
        const bool seen = t >= first && t <= pos;
        for (int g = wave; g < num_heads; g += 4) {
            float a = 0.0f;
            if (seen) {
                const T* key = k_pages + (((size_t)page * num_kv_heads + g / group) * PAGE + lane) * head_dim;
                const T* query = q + ((size_t)row * num_heads + g) * head_dim;
                float dot = 0.0f;
                for (int d = 0; d < head_dim; ++d) dot = fmaf(load_as_float(query, d), load_as_float(key, d), dot);
                a = 1.0f / (1.0f + expf(-fmaf(dot, scale, bias[g])));
            }
            weights[g * PAGE + lane] = a;
        }
        __syncthreads();
        for (int h = wave; h < heads_here; h += 4) {
            const float* row_of_mix = mix + (size_t)(head0 + h) * num_heads;
            float sum = 0.0f;
            for (int g = 0; g < num_heads; ++g) sum = fmaf(row_of_mix[g], weights[g * PAGE + lane], sum);
            mixed[h * PAGE + lane] = sum;
        }
        __syncthreads();
        const int lo = first - tile * PAGE > 0 ? first - tile * PAGE : 0;
        const int hi = pos - tile * PAGE < PAGE - 1 ? pos - tile * PAGE : PAGE - 1;
#pragma unroll
        for (int u = 0; u < SG_HELD; ++u) {
            const int item = threadIdx.x + 256 * u;
            if (item < heads_here * v_dim) {
                const int h = item / v_dim, d = item % v_dim;
                const T* value = v_pages + (((size_t)page * num_kv_heads + (head0 + h) / group) * v_dim + d) * PAGE;
                float sum = 0.0f;
                for (int s = lo; s <= hi; ++s) sum = fmaf(mixed[h * PAGE + s], load_as_float(value, s), sum);
                acc[u] += sum;
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int u = 0; u < SG_HELD; ++u) {
        const int item = threadIdx.x + 256 * u;
        if (item < heads_here * v_dim) {
            const size_t channel = (size_t)head0 * v_dim + item;
            const float factor = gate ? sg_gate(gate[(size_t)row * gate_stride + channel]) : 1.0f;
            store_from_float(out, (size_t)row * num_heads * v_dim + channel, acc[u] * factor);
        }
    }
}

static int sg_check(const char* name, int rows, int num_heads, int num_kv_heads, int head_dim, int v_dim, int window, const float* bias,
                    const float* mix, const float* gate, int gate_stride, int page_size, int num_pages, int table_stride) {
    FW_REQUIRE(rows >= 0 && rows <= 1 << 20 && num_heads > 0 && num_kv_heads > 0 && num_heads % num_kv_heads == 0,
               "%s: rows %d; heads %d must be a positive multiple of kv heads %d", name, rows, num_heads, num_kv_heads);
    FW_REQUIRE(head_dim > 0 && v_dim > 0, "%s: head sizes %d and %d must be positive", name, head_dim, v_dim);
    FW_REQUIRE(window >= 0, "%s: window must be 0 (all keys) or positive, got %d", name, window);
    FW_REQUIRE(bias && mix, "%s: the scores' biases and the heads' mix are needed", name);
    FW_REQUIRE(gate == nullptr || gate_stride >= num_heads * v_dim, "%s: the gates' rows (%d wide) do not hold %d x %d", name, gate_stride,
               num_heads, v_dim);
    FW_REQUIRE(page_size == PAGE, "%s: page size must be %d, got %d", name, PAGE, page_size);
    FW_REQUIRE(num_pages > 0 && table_stride > 0, "%s: empty cache (pages=%d, table stride=%d)", name, num_pages, table_stride);
    return 0;
}

extern "C" int fw_sigmoid_attention_generic(const void* q, void* out, int dtype, const void* k_pages, const void* v_pages,
                                            const int32_t* block_table, int table_stride, const int32_t* row_seg, const int32_t* row_pos,
                                            int rows, int num_heads, int num_kv_heads, int head_dim, int v_dim, float scale, int window,
                                            const float* bias, const float* mix, const float* gate, int gate_stride, int page_size,
                                            int num_pages, void* stream) {
    if (sg_check("sigmoid_attention", rows, num_heads, num_kv_heads, head_dim, v_dim, window, bias, mix, gate, gate_stride, page_size,
                 num_pages, table_stride)) return -1;
    FW_REQUIRE(num_heads <= SG_MAX_HEADS && head_dim <= SG_MAX_DIM && v_dim <= SG_MAX_DIM,
               "sigmoid_attention: %d heads of %d / %d channels exceed the limits of %d heads and %d channels", num_heads, head_dim, v_dim,
               SG_MAX_HEADS, SG_MAX_DIM);
    if (rows == 0) return 0;
    int per_block = 256 * SG_HELD / v_dim;
    if (per_block > num_heads) per_block = num_heads;
    const int lds_bytes = (num_heads + per_block) * PAGE * (int)sizeof(float);
    dim3 grid(rows, (num_heads + per_block - 1) / per_block);
#define SG_LAUNCH(T)                                                                                                                \
    {                                                                                                                              \
        static int configured = 0;                                                                                                 \
        if (lds_bytes > 48 * 1024 && lds_bytes > configured) {                                                                      \
            hipError_t status = hipFuncSetAttribute((const void*)sigmoid_attention_generic_kernel<T>,                               \
                                                    hipFuncAttributeMaxDynamicSharedMemorySize, lds_bytes);                        \
            FW_REQUIRE(status == hipSuccess, "sigmoid_attention: cannot reserve %d bytes of LDS", lds_bytes);                       \
            configured = lds_bytes;                                                                                                \
        }                                                                                                                          \
        sigmoid_attention_generic_kernel<T><<<grid, 256, lds_bytes, (hipStream_t)stream>>>(                                         \
            (const T*)q, (T*)out, (const T*)k_pages, (const T*)v_pages, block_table, table_stride, row_seg, row_pos, num_heads,     \
            num_kv_heads, head_dim, v_dim, scale, window, bias, mix, gate, gate_stride, per_block);                                 \
    }
    if (dtype == FW_F32) SG_LAUNCH(float)
    else if (dtype == FW_BF16) SG_LAUNCH(bf16_t)
    else FW_REQUIRE(false, "sigmoid_attention: unknown dtype %d", dtype);
#undef SG_LAUNCH
    FW_LAUNCH_CHECK("sigmoid_attention");
    return 0;
}

// ---- prompt portions on the matrix cores --------------------------------------------------------------
// A workgroup of eight waves takes 16 query rows of one segment, all heads, and walks the visible keys
// 128 at a time. Of those a wave first takes 16: per head g it forms S^T[key][row] = K Q^T
// (v_mfma_f32_16x16x32_bf16, the key/value head's keys loaded once per group straight into operand registers, one
// key/value head ahead of the work, the queries from LDS), so that a lane holds the scores of 4 keys x 1 row of EVERY
// head, turns them into sigmoids, and mixes the heads where they are: v_mfma_f32_4x4x1f32 multiplies a 4 x 1 column
// of the mix (4 output heads, one g) by 64 lanes' weights of g, sixteen blocks side by side, which is a mix in exact
// float32 that moves nothing between lanes and leaves the vector unit to the sigmoids. The mixed
// weights, rounded to bfloat16, go to LDS [head][row][128 keys]; behind a barrier the waves share out
// the heads (and, with few heads, the halves of their channels) and add V^T P^T (v_mfma_f32_16x16x32_bf16, values
// straight from the cache, one run of tiles ahead) to accumulators that stay in registers to the end, where the gate joins.
// gridDim.y workgroups share the steps of 128 keys of a tile where the tiles alone would not fill the chip: parts
// of a row's keys add up, so each leaves its float32 sums and the one that arrives last (a ticket per tile; nobody
// waits) adds them in the order of the keys.
// HB: heads in fours (num_heads <= 4 HB; heads beyond have a zero column and row in the mix and are not stored). GS: a
// divisor of the heads on one key/value head (4, 2 or 1); the scores of that many heads are formed side by side.
// What is the same for a whole wave is kept in scalar registers (its number, pages, heads), and a lane's place
// in a page as one 32-bit offset: the vector registers are all taken by what is in flight.
#define SG_WAVES 8
#define SG_STEP 128
#define SG_PAD 8
template <int HD, int HB, int GS>
__global__ __launch_bounds__(64 * SG_WAVES) void sigmoid_attention_prefill_kernel(
    const uint16_t* __restrict__ q, uint16_t* __restrict__ out, float* partial, int* tickets, const uint16_t* __restrict__ k_pages,
    const uint16_t* __restrict__ v_pages, const int32_t* __restrict__ block_table, int table_stride,
    const int32_t* __restrict__ tile_seg, const int32_t* __restrict__ tile_row0, const int32_t* __restrict__ seg_row0,
    const int32_t* __restrict__ row_pos, int num_heads, int num_kv_heads, int head_dim, int v_dim, float scale_log2, int window,
    const float* __restrict__ bias, const float* __restrict__ mix, const float* __restrict__ gate, int gate_stride) {
    constexpr int HP = 4 * HB;                          // heads with padding
    constexpr int SLOTS = (HB + 1) / 2;                 // heads of a wave in the weighted sums
    constexpr int HALVES = HB == 1 ? 1 : 2;             // halves of a head's channels a wave takes
    constexpr int TILES = HD / 32;                      // tiles of 16 channels in a half
    constexpr bool AHEAD = HD <= 128;                   // values are asked for a run of tiles ahead where registers allow
    constexpr int Q_STRIDE = HD + SG_PAD, P_STRIDE = SG_STEP + SG_PAD;
    extern __shared__ __attribute__((aligned(16))) unsigned char sg_raw[];
    uint16_t* lds_q = reinterpret_cast<uint16_t*>(sg_raw);                          // [heads][16 rows][Q_STRIDE]
    uint16_t* lds_p = lds_q + (size_t)num_heads * 16 * Q_STRIDE;                    // [heads][16 rows][P_STRIDE]
    // the mix as the lanes read it: [4 output heads][4 g's][output head % 4][g % 4]
    float* lds_mix = reinterpret_cast<float*>(lds_p + (size_t)num_heads * 16 * P_STRIDE);
    float* lds_bias = lds_mix + HP * HP;                                            // [HP], times log2(e)
    int* ticket_shared = reinterpret_cast<int*>(lds_bias + HP);

    const int tile = blockIdx.x >> 2, sub = blockIdx.x & 3;
    const int seg = tile_seg[tile];
    const int row0 = tile_row0[tile] + sub * 16;
    const int seg_end = seg_row0[seg + 1];
    if (row0 >= seg_end) return;                // the whole workgroup
    const int rows = seg_end - row0 < 16 ? seg_end - row0 : 16;
    const int pos_lo = row_pos[row0], pos_hi = row_pos[row0 + rows - 1];
    const int all_first = fw_first_visible(pos_lo, window, 0) / PAGE, last_block = pos_hi / PAGE;
    // this workgroup's share of the tile's steps
    const int all_steps = (last_block - all_first) / 2 + 1;
    const int share = (all_steps + (int)gridDim.y - 1) / (int)gridDim.y, parts = (all_steps + share - 1) / share;
    const int first_block = all_first + (int)blockIdx.y * share * 2;
    if (first_block > last_block) return;       // the whole workgroup
    const int end_block = first_block + 2 * share - 1 < last_block ? first_block + 2 * share - 1 : last_block;
    const int tid = threadIdx.x, lane = tid & 63, i16 = lane & 15, g4 = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int group = num_heads / num_kv_heads;
    const int32_t* table = block_table + (size_t)seg * table_stride;
    auto page_of = [&](int block) { return table[block <= end_block ? block : end_block]; };

    // A lane's place in a head's page of keys, in bytes. Channels past head_dim (whole runs of 32, or the last
    // run's upper half: head_dim is a multiple of 16) are read from channels that are there, and are zero by the time
    // they are used.
    const uint32_t key_offset = (uint32_t)(((wave & 3) * 16 + i16) * head_dim + g4 * 8) * 2u;
    const uint32_t key_offset_tail = g4 >= 2 ? key_offset - 32u : key_offset;
    const int whole_runs = head_dim / 32;
    auto load_keys = [&](u32x4 (&kf)[HD / 32], int page, int kvh) {
        const char* keys = reinterpret_cast<const char*>(k_pages + ((size_t)page * num_kv_heads + kvh) * PAGE * head_dim);
#pragma unroll
        for (int dc = 0; dc < HD / 32; ++dc) {
            const char* from = keys + (dc * 32 < head_dim ? dc * 64 : 0);
            kf[dc] = *reinterpret_cast<const u32x4*>(from + (dc < whole_runs ? key_offset : key_offset_tail));
        }
    };
    u32x4 kf_next[HD / 32];
    bf16x8 kf[HD / 32];
    auto take_keys = [&]() {
#pragma unroll
        for (int dc = 0; dc < HD / 32; ++dc) {
            u32x4 bits = kf_next[dc];
            if (dc >= whole_runs) {             // uniform, and never with a full head_dim
                const bool in = dc * 32 + g4 * 8 < head_dim;
                bits = u32x4{in ? bits[0] : 0u, in ? bits[1] : 0u, in ? bits[2] : 0u, in ? bits[3] : 0u};
            }
            kf[dc] = __builtin_bit_cast(bf16x8, bits);
        }
    };
    int page_a = page_of(first_block), page_b = page_of(first_block + 1);       // the step's two pages
    load_keys(kf_next, wave >> 2 ? page_b : page_a, 0);

    // queries of the 16 rows, head by head; channels past head_dim and rows past the end are zero
    for (int run = tid; run < num_heads * 16 * (HD / 8); run += 64 * SG_WAVES) {
        const int at = run % (HD / 8), r = run / (HD / 8) % 16, h = run / (HD / 8) / 16;
        u32x4 v = {0u, 0u, 0u, 0u};
        if (r < rows && at * 8 < head_dim) v = *reinterpret_cast<const u32x4*>(q + ((size_t)(row0 + r) * num_heads + h) * head_dim + at * 8);
        *reinterpret_cast<u32x4*>(lds_q + ((size_t)h * 16 + r) * Q_STRIDE + at * 8) = v;
    }
    for (int item = tid; item < HP * HP; item += 64 * SG_WAVES) {
        const int g = (item / 16 % HB) * 4 + item % 4, h = item / (16 * HB) * 4 + item / 4 % 4;
        lds_mix[item] = (h < num_heads && g < num_heads) ? mix[(size_t)h * num_heads + g] : 0.0f;
    }
    if (tid < HP) lds_bias[tid] = tid < num_heads ? bias[tid] * LOG2E_F : 0.0f;
    fw_lds_barrier();

    const bool row_there = i16 < rows;
    const int my_pos = row_pos[row0 + (row_there ? i16 : 0)];
    const int my_first = fw_first_visible(my_pos, window, 0);
    // the heads of this wave's weighted sums (one past the last computes along and is not stored)
    int head_of[SLOTS], kv_of[SLOTS];
#pragma unroll
    for (int n = 0; n < SLOTS; ++n) {
        const int head = HB == 1 ? wave >> 1 : wave * SLOTS + n;
        head_of[n] = head < num_heads ? head : num_heads - 1;
        kv_of[n] = head_of[n] / group;
    }
    const int half0 = HB == 1 ? (wave & 1) : 0;
    // (v_dim is a multiple of 16: a tile of channels is there or not; one past the last is the last again, not stored)
    const uint32_t value_offset = (uint32_t)(i16 * PAGE + g4 * 8) * 2u;
    const int last_tile = v_dim / 16 - 1;
    auto load_values = [&](u32x4 (&v)[TILES], int page, int kb, int half, int kvh) {
        const char* values = reinterpret_cast<const char*>(v_pages + ((size_t)page * num_kv_heads + kvh) * v_dim * PAGE + (kb & 1) * 32);
#pragma unroll
        for (int t = 0; t < TILES; ++t) {
            const int at = (half0 + half) * TILES + t, there = at < last_tile ? at : last_tile;
            v[t] = *reinterpret_cast<const u32x4*>(values + (size_t)there * 16 * PAGE * 2 + value_offset);
        }
    };

    f32x4 acc[SLOTS][HALVES][TILES];
#pragma unroll
    for (int n = 0; n < SLOTS; ++n)
#pragma unroll
        for (int half = 0; half < HALVES; ++half)
#pragma unroll
            for (int t = 0; t < TILES; ++t) acc[n][half][t] = f32x4{0.f, 0.f, 0.f, 0.f};

    for (int block0 = first_block; block0 <= end_block; block0 += 2) {
        // -- weights of this wave's 16 keys, every head
        const int my_block = block0 + (wave >> 2);
        const int key0 = my_block * PAGE + (wave & 3) * 16;
        const int next_a = page_of(block0 + 2), next_b = page_of(block0 + 3);
        float w[HP][4];
        int kvh = -1, left = 0;                 // heads left on this key/value head
#pragma unroll
        for (int g0 = 0; g0 < HP; g0 += GS) {
            if (left == 0 && g0 < num_heads) {  // uniform: the next key/value head's keys, and the ones after them asked for
                ++kvh;
                left = group;
                take_keys();
                const bool last = kvh + 1 >= num_kv_heads;
                load_keys(kf_next, wave >> 2 ? (last ? next_b : page_b) : (last ? next_a : page_a), last ? 0 : kvh + 1);
            }
            left -= GS;
            f32x4 s[GS];
#pragma unroll
            for (int u = 0; u < GS; ++u) s[u] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int dc = 0; dc < HD / 32; ++dc)
#pragma unroll
                for (int u = 0; u < GS; ++u) {
                    const int head = g0 + u < num_heads ? g0 + u : num_heads - 1;
                    const bf16x8 query = *reinterpret_cast<const bf16x8*>(lds_q + ((size_t)head * 16 + i16) * Q_STRIDE + g4 * 8 + dc * 32);
                    s[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[dc], query, s[u], 0, 0, 0);
                }
#pragma unroll
            for (int u = 0; u < GS; ++u) {
                const float b = lds_bias[g0 + u];
#pragma unroll
                for (int r = 0; r < 4; ++r)     // sigmoid by the hardware's 2^x and reciprocal; 2^x = infinity gives 0
                    w[g0 + u][r] = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-fmaf(s[u][r], scale_log2, b)));
            }
        }
        u32x4 v[TILES], v_next[AHEAD ? TILES : 1];
        if constexpr (AHEAD) load_values(v_next, page_a, 0, 0, kv_of[0]);        // they travel while the heads are mixed
        // all of the wave's keys seen by all of its rows (all but the pages at the window's edge and the diagonal): no mask
        const bool whole = __all(row_there && key0 >= my_first && key0 + 15 <= my_pos) && my_block <= end_block;
        if (!whole) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int key = key0 + g4 * 4 + r;
                const bool seen = row_there && key >= my_first && key <= my_pos && my_block <= end_block;
#pragma unroll
                for (int g = 0; g < HP; ++g) w[g][r] = seen ? w[g][r] : 0.0f;
            }
        }
        // -- the heads mixed, and stored as the next product reads them
#pragma unroll
        for (int hb = 0; hb < HB; ++hb) {
            f32x4 m[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) m[r] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int gb = 0; gb < HB; ++gb) {
                const f32x4 t = *reinterpret_cast<const f32x4*>(lds_mix + ((hb * HB + gb) * 4 + (lane & 3)) * 4);
#pragma unroll
                for (int g = 0; g < 4; ++g)
#pragma unroll
                    for (int r = 0; r < 4; ++r) m[r] = __builtin_amdgcn_mfma_f32_4x4x1f32(t[g], w[gb * 4 + g][r], m[r], 0, 0, 0);
            }
#pragma unroll
            for (int x = 0; x < 4; ++x) {
                const u32x2 packed = {sg_pack(m[0][x], m[1][x]), sg_pack(m[2][x], m[3][x])};
                if (hb * 4 + x < num_heads)
                    *reinterpret_cast<u32x2*>(lds_p + ((size_t)(hb * 4 + x) * 16 + i16) * P_STRIDE + wave * 16 + g4 * 4) = packed;
            }
        }
        fw_lds_barrier();
        // -- the weighted sums of this wave's heads
#pragma unroll
        for (int kb = 0; kb < 4; ++kb) {
            // values of keys nobody has written yet must not meet a weight of 0 as they are
            const int last_written = pos_hi - (block0 + (kb >> 1)) * PAGE - (kb & 1) * 32 - g4 * 8;     // in this lane's eight keys
            uint32_t keep[4];
#pragma unroll
            for (int word = 0; word < 4; ++word)
                keep[word] = 2 * word + 1 <= last_written ? 0xffffffffu : (2 * word <= last_written ? 0xffffu : 0u);
            bf16x8 pf[SLOTS];
#pragma unroll
            for (int n = 0; n < SLOTS; ++n)
                pf[n] = *reinterpret_cast<const bf16x8*>(lds_p + ((size_t)head_of[n] * 16 + i16) * P_STRIDE + kb * 32 + g4 * 8);
#pragma unroll
            for (int half = 0; half < HALVES; ++half) {
                if constexpr (AHEAD) {
#pragma unroll
                    for (int t = 0; t < TILES; ++t) v[t] = v_next[t];
                    if (kb < 3 || half + 1 < HALVES) {
                        const int kb_next = half + 1 < HALVES ? kb : kb + 1;
                        load_values(v_next, kb_next >> 1 ? page_b : page_a, kb_next, half + 1 < HALVES ? half + 1 : 0, kv_of[0]);
                    }
                } else {
                    load_values(v, kb >> 1 ? page_b : page_a, kb, half, kv_of[0]);
                }
#pragma unroll
                for (int n = 0; n < SLOTS; ++n) {
                    if (n > 0 && kv_of[n] != kv_of[n - 1]) load_values(v, kb >> 1 ? page_b : page_a, kb, half, kv_of[n]);    // uniform
#pragma unroll
                    for (int t = 0; t < TILES; ++t) {
                        const u32x4 clean = {v[t][0] & keep[0], v[t][1] & keep[1], v[t][2] & keep[2], v[t][3] & keep[3]};
                        acc[n][half][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, clean), pf[n], acc[n][half][t], 0, 0, 0);
                    }
                }
            }
        }
        fw_mfma_drain();
        fw_lds_barrier();       // the weights are read: the next step may store its own
        page_a = next_a;
        page_b = next_b;
    }
    const int channels = num_heads * v_dim;
    if (parts > 1) {
        // [tile of 16 rows][part][register][thread]: device-scope stores, which pass the caches that workgroups on other
        // dies do not share
        constexpr int HELD = SLOTS * HALVES * TILES * 4;
        float* mine = partial + ((size_t)blockIdx.x * gridDim.y + blockIdx.y) * HELD * 512 + tid;
#pragma unroll
        for (int n = 0; n < SLOTS; ++n)
#pragma unroll
            for (int half = 0; half < HALVES; ++half)
#pragma unroll
                for (int t = 0; t < TILES; ++t)
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        __hip_atomic_store(mine + (size_t)(((n * HALVES + half) * TILES + t) * 4 + r) * 512, acc[n][half][t][r], __ATOMIC_RELAXED,
                                           __HIP_MEMORY_SCOPE_AGENT);
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
        if (tid == 0) *ticket_shared = __hip_atomic_fetch_add(tickets + blockIdx.x, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        __syncthreads();
        if (*ticket_shared != parts - 1) return;
        if (tid == 0) __hip_atomic_store(tickets + blockIdx.x, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
#pragma unroll
        for (int n = 0; n < SLOTS; ++n)
#pragma unroll
            for (int half = 0; half < HALVES; ++half)
#pragma unroll
                for (int t = 0; t < TILES; ++t) acc[n][half][t] = f32x4{0.f, 0.f, 0.f, 0.f};
        for (int part = 0; part < parts; ++part) {
            const float* from = partial + ((size_t)blockIdx.x * gridDim.y + part) * HELD * 512 + tid;
#pragma unroll
            for (int n = 0; n < SLOTS; ++n)
#pragma unroll
                for (int half = 0; half < HALVES; ++half)
#pragma unroll
                    for (int t = 0; t < TILES; ++t)
#pragma unroll
                        for (int r = 0; r < 4; ++r)
                            acc[n][half][t][r] += __hip_atomic_load(from + (size_t)(((n * HALVES + half) * TILES + t) * 4 + r) * 512, __ATOMIC_RELAXED,
                                                                    __HIP_MEMORY_SCOPE_AGENT);
        }
    }
    if (!row_there) return;
#pragma unroll
    for (int n = 0; n < SLOTS; ++n) {
        const int head = HB == 1 ? wave >> 1 : wave * SLOTS + n;
        if (head >= num_heads) continue;
#pragma unroll
        for (int half = 0; half < HALVES; ++half)
#pragma unroll
            for (int t = 0; t < TILES; ++t) {
                const int channel = (half0 + half) * (HD / 2) + t * 16 + g4 * 4;
                if (channel >= v_dim) continue;     // v_dim is a multiple of 16
                f32x4 o = acc[n][half][t];
                if (gate) {
                    const float* z = gate + (size_t)(row0 + i16) * gate_stride + (size_t)head * v_dim + channel;
#pragma unroll
                    for (int r = 0; r < 4; ++r) o[r] *= sg_gate_quick(z[r]);
                }
                *reinterpret_cast<u32x2*>(out + (size_t)(row0 + i16) * channels + (size_t)head * v_dim + channel) =
                    u32x2{sg_pack(o[0], o[1]), sg_pack(o[2], o[3])};
            }
    }
}

static int sg_tiled_check(const char* name, int num_heads, int head_dim, int v_dim) {
    FW_REQUIRE(num_heads <= SG_TILE_HEADS, "%s: at most %d heads, got %d", name, SG_TILE_HEADS, num_heads);
    FW_REQUIRE(head_dim % 16 == 0 && v_dim % 16 == 0 && head_dim <= 256 && v_dim <= 256,
               "%s: head sizes %d and %d must be multiples of 16 up to 256", name, head_dim, v_dim);
    return 0;
}
static int sg_prefill_lds(int num_heads, int widest_class) {
    const int heads_padded = (num_heads + 3) / 4 * 4;
    return num_heads * 16 * (widest_class + SG_PAD + SG_STEP + SG_PAD) * 2 + (heads_padded * heads_padded + heads_padded + 1) * 4;
}
static int sg_class(int head_dim, int v_dim) {
    const int widest = head_dim > v_dim ? head_dim : v_dim;
    return widest <= 32 ? 32 : widest <= 64 ? 64 : widest <= 128 ? 128 : 256;
}
#define SG_LDS_LIMIT (160 * 1024)
#define SG_MAX_PARTS 8
#define SG_FILL 256                 // workgroups that fill the chip (one to a compute unit at many heads)

// 1 if the matrix-core kernels take these sizes (bfloat16): up to 16 heads, sizes in steps of 16 up to 256, and
// the queries and weights of 16 rows of all heads within a compute unit's LDS
extern "C" int fw_sigmoid_attention_fits(int num_heads, int head_dim, int v_dim) {
    if (num_heads < 1 || num_heads > SG_TILE_HEADS || head_dim < 16 || v_dim < 16 || head_dim % 16 || v_dim % 16) return 0;
    if (head_dim > 256 || v_dim > 256) return 0;
    return sg_prefill_lds(num_heads, sg_class(head_dim, v_dim)) <= SG_LDS_LIMIT ? 1 : 0;
}

// Floats of workspace that a tile of 16 rows leaves per part (all of a workgroup's accumulators)
static int sg_part_floats(int num_heads, int width) {
    const int fours = (num_heads + 3) / 4;
    return (fours + 1) / 2 * (fours == 1 ? 1 : 2) * (width / 32) * 4 * 512;
}

// What `tiles` tiles of 64 rows that see at most `max_keys` keys each need for `parts` workgroups to a tile of 16 rows: floats
// of workspace (0: none) and zeroed counters. parts <= 0: as many as fill the chip; the number used is returned.
extern "C" int fw_sigmoid_attention_prefill_plan(int tiles, int num_heads, int head_dim, int v_dim, int window, int max_context, int parts,
                                                 long long* workspace_floats, int* counters) {
    long long keys = max_context;
    if (window > 0 && window + 16 < keys) keys = window + 16;
    const int steps = (int)((keys + PAGE - 2) / PAGE + 1) / 2 + 1;
    if (parts <= 0) parts = tiles > 0 ? SG_FILL / (tiles * 4) : 1;
    if (parts > steps) parts = steps;
    if (parts > SG_MAX_PARTS) parts = SG_MAX_PARTS;
    if (parts < 1) parts = 1;
    *workspace_floats = parts > 1 ? (long long)tiles * 4 * parts * sg_part_floats(num_heads, sg_class(head_dim, v_dim)) : 0;
    *counters = parts > 1 ? tiles * 4 : 0;
    return parts;
}

extern "C" int fw_sigmoid_attention_prefill(const void* q, void* out, float* partial, long long partial_floats, int* tickets,
                                            int tickets_len, int parts, const void* k_pages, const void* v_pages,
                                            const int32_t* block_table, int table_stride, const int32_t* tile_seg,
                                            const int32_t* tile_row0, int tiles, const int32_t* seg_row0, const int32_t* row_pos, int rows,
                                            int num_heads, int num_kv_heads, int head_dim, int v_dim, float scale, int window,
                                            const float* bias, const float* mix, const float* gate, int gate_stride, int page_size,
                                            int num_pages, void* stream) {
    if (sg_check("sigmoid_attention_prefill", rows, num_heads, num_kv_heads, head_dim, v_dim, window, bias, mix, gate, gate_stride, page_size,
                 num_pages, table_stride)) return -1;
    if (sg_tiled_check("sigmoid_attention_prefill", num_heads, head_dim, v_dim)) return -1;
    FW_REQUIRE(tiles >= 0 && tiles <= rows, "sigmoid_attention_prefill: %d tiles for %d rows", tiles, rows);
    const int width = sg_class(head_dim, v_dim), fours = (num_heads + 3) / 4;
    const int lds_bytes = sg_prefill_lds(num_heads, width);
    FW_REQUIRE(lds_bytes <= SG_LDS_LIMIT, "sigmoid_attention_prefill: %d heads of %d / %d channels need %d bytes of LDS", num_heads, head_dim,
               v_dim, lds_bytes);
    if (rows == 0 || tiles == 0) return 0;
    FW_REQUIRE(parts >= 1 && parts <= SG_MAX_PARTS, "sigmoid_attention_prefill: %d parts (1..%d)", parts, SG_MAX_PARTS);
    FW_REQUIRE(parts == 1 || (partial && tickets && partial_floats >= (long long)tiles * 4 * parts * sg_part_floats(num_heads, width) &&
                              tickets_len >= tiles * 4), "sigmoid_attention_prefill: %d parts of %d tiles need more workspace or counters", parts, tiles);
    dim3 grid((unsigned)tiles * 4, (unsigned)parts);
#define SG_LAUNCH(HD, HB, GS)                                                                                                         \
    {                                                                                                                               \
        static int configured = 0;                                                                                                  \
        if (lds_bytes > configured) {                                                                                               \
            hipError_t status = hipFuncSetAttribute((const void*)sigmoid_attention_prefill_kernel<HD, HB, GS>,                       \
                                                    hipFuncAttributeMaxDynamicSharedMemorySize, lds_bytes);                         \
            FW_REQUIRE(status == hipSuccess, "sigmoid_attention_prefill: cannot reserve %d bytes of LDS", lds_bytes);                \
            configured = lds_bytes;                                                                                                 \
        }                                                                                                                           \
        sigmoid_attention_prefill_kernel<HD, HB, GS><<<grid, 64 * SG_WAVES, lds_bytes, (hipStream_t)stream>>>(                       \
            (const uint16_t*)q, (uint16_t*)out, partial, tickets, (const uint16_t*)k_pages, (const uint16_t*)v_pages, block_table, table_stride, \
            tile_seg, tile_row0, seg_row0, row_pos, num_heads, num_kv_heads, head_dim, v_dim, scale * LOG2E_F, window, bias, mix,    \
            gate, gate_stride);                                                                                                     \
    }
#define SG_BY_GROUP(HD, HB)                                                                                                         \
    if (group % 4 == 0) SG_LAUNCH(HD, HB, 4) else if (group % 2 == 0) SG_LAUNCH(HD, HB, 2) else SG_LAUNCH(HD, HB, 1)
#define SG_BY_HEADS(HD)                                                                                                             \
    if (fours == 1) { SG_BY_GROUP(HD, 1) } else if (fours == 2) { SG_BY_GROUP(HD, 2) } else if (fours == 3) { SG_BY_GROUP(HD, 3) } else { SG_BY_GROUP(HD, 4) }
    const int group = num_heads / num_kv_heads;
    if (width == 32) { SG_BY_HEADS(32) }
    else if (width == 64) { SG_BY_HEADS(64) }
    else if (width == 128) { SG_BY_HEADS(128) }
    else { if (fours == 1) SG_LAUNCH(256, 1, 1) else if (fours == 2) SG_LAUNCH(256, 2, 1) else SG_LAUNCH(256, 3, 1) }
#undef SG_BY_HEADS
#undef SG_BY_GROUP
#undef SG_LAUNCH
    FW_LAUNCH_CHECK("sigmoid_attention_prefill");
    return 0;
}

// ---- decoding on the matrix cores -----------------------------------------------------------------------
// grid (rows, splits): a workgroup of four waves takes one row, all heads and `pages_per_split` pages of the
// row's visible keys. Per page a wave forms S[head][key] of 16 keys (all heads as the first operand's rows, one
// product per key/value head, of which each lane keeps the rows whose group it is), the sigmoids, and the
// mix as v_mfma_f32_16x16x4_f32 (its second operand is the lane's four weights as they stand); the mixed
// weights meet in LDS, and the waves share out the channel tiles of the weighted sum, in which the weights of
// heads outside a key/value head's group are zero. Parts of a row add up: a workgroup leaves its sums, and the
// one that arrives last (a ticket per row; nobody waits) adds them in the order of the keys and
// applies the gate.
// `fused.qkv`: the step's raw projections (float32 rows of `width`: q | k | v). The workgroup then forms its
// queries itself (each head divided by its root mean square), and the one whose pages include the row's own
// position first stores the new key (likewise normed) and value there.
struct SigmoidFused {
    const float* qkv;
    int width, qk_norm, write_kv;
    float eps;
};

// one vector of `dim` channels by one wave: v / sqrt(mean(v^2) + eps) if normed; store(d, value)
template <typename Store>
__device__ __forceinline__ void sg_unit_vector(const float* __restrict__ source, int dim, int normed, float eps, Store store) {
    const int lane = threadIdx.x & 63;
    float v[4], sum = 0.0f;             // dim <= 256
#pragma unroll
    for (int u = 0; u < 4; ++u) {
        v[u] = lane + 64 * u < dim ? source[lane + 64 * u] : 0.0f;
        sum += v[u] * v[u];
    }
    const float inv = normed ? rsqrtf(wave_sum(sum) / (float)dim + eps) : 1.0f;
#pragma unroll
    for (int u = 0; u < 4; ++u)
        if (lane + 64 * u < dim) store(lane + 64 * u, v[u] * inv);
}

template <int HD, bool FUSED>
__global__ __launch_bounds__(256) void sigmoid_attention_decode_kernel(
    const uint16_t* __restrict__ q, uint16_t* __restrict__ out, float* partial, int* tickets, uint16_t* k_pages, uint16_t* v_pages,
    const int32_t* __restrict__ block_table, int table_stride, const int32_t* __restrict__ row_seg, const int32_t* __restrict__ row_pos,
    int num_heads, int num_kv_heads, int head_dim, int v_dim, float scale_log2, int window, const float* __restrict__ bias,
    const float* __restrict__ mix, const float* __restrict__ gate, int gate_stride, int pages_per_split, const SigmoidFused fused) {
    constexpr int TILES = (HD / 16 + 3) / 4;            // channel tiles of a wave
    constexpr int KV_AT_ONCE = HD <= 128 ? 4 : 2;
    __shared__ __attribute__((aligned(16))) uint16_t lds_q[16][HD + SG_PAD];
    __shared__ __attribute__((aligned(16))) uint16_t lds_p[2][16][PAGE + SG_PAD];
    __shared__ int ticket_shared;
    const int row = blockIdx.x, split = blockIdx.y;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, i16 = lane & 15, g4 = lane >> 4;
    const int group = num_heads / num_kv_heads;
    const int pos = row_pos[row], segment = row_seg[row];
    const int first = fw_first_visible(pos, window, 0);
    const int first_block = first / PAGE, last_block = pos / PAGE;
    const int block0 = first_block + split * pages_per_split;
    if (block0 > last_block) return;                    // the whole workgroup
    const int block_end = block0 + pages_per_split - 1 < last_block ? block0 + pages_per_split - 1 : last_block;
    const int32_t* table = block_table + (size_t)segment * table_stride;

    if (FUSED) {
        const float* projections = fused.qkv + (size_t)row * fused.width;
        const bool stores = fused.write_kv && block_end == last_block;
        const int vectors = 16 + (stores ? 2 * num_kv_heads : 0);
        const int own_page = stores ? table[last_block] : 0, slot = pos % PAGE;
        for (int v = wave; v < vectors; v += 4) {
            if (v < 16) {
                uint16_t* dest = lds_q[v];
                if (v < num_heads)
                    sg_unit_vector(projections + (size_t)v * head_dim, head_dim, fused.qk_norm, fused.eps,
                                   [&](int d, float value) { dest[d] = float_to_bf16_bits(value); });
                for (int d = (v < num_heads ? head_dim : 0) + lane; d < HD; d += 64) dest[d] = 0;
            } else if (v < 16 + num_kv_heads) {
                const int c = v - 16;
                uint16_t* dest = k_pages + (((size_t)own_page * num_kv_heads + c) * PAGE + slot) * head_dim;
                sg_unit_vector(projections + (size_t)(num_heads + c) * head_dim, head_dim, fused.qk_norm, fused.eps,
                               [&](int d, float value) { dest[d] = float_to_bf16_bits(value); });
            } else {
                const int c = v - 16 - num_kv_heads;
                const float* value = projections + (size_t)(num_heads + num_kv_heads) * head_dim + (size_t)c * v_dim;
                uint16_t* dest = v_pages + ((size_t)own_page * num_kv_heads + c) * v_dim * PAGE + slot;
                for (int d = lane; d < v_dim; d += 64) dest[(size_t)d * PAGE] = float_to_bf16_bits(value[d]);
            }
        }
        // the page is read below by this workgroup's own waves: its stores have to be done first
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    } else {
        for (int run = tid; run < 16 * (HD / 8); run += 256) {
            const int at = run % (HD / 8), h = run / (HD / 8);
            u32x4 v = {0u, 0u, 0u, 0u};
            if (h < num_heads && at * 8 < head_dim) v = *reinterpret_cast<const u32x4*>(q + ((size_t)row * num_heads + h) * head_dim + at * 8);
            *reinterpret_cast<u32x4*>(&lds_q[h][at * 8]) = v;
        }
    }
    __syncthreads();
    bf16x8 qf[HD / 32];         // first operand: head i16, channels 32 dc + 8 g4 ..
#pragma unroll
    for (int dc = 0; dc < HD / 32; ++dc) qf[dc] = *reinterpret_cast<const bf16x8*>(&lds_q[i16][dc * 32 + g4 * 8]);
    // this lane's rows of the scores are heads 4 g4 + r; its first operand of the mix is mix[i16][4 g4 + s]
    float head_bias[4], mix_row[4];
    int kv_of[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int h = g4 * 4 + r;
        head_bias[r] = h < num_heads ? bias[h] * LOG2E_F : 0.0f;
        kv_of[r] = h < num_heads ? h / group : -1;
        mix_row[r] = (i16 < num_heads && h < num_heads) ? mix[(size_t)i16 * num_heads + h] : 0.0f;
    }
    const int my_kv = i16 < num_heads ? i16 / group : -1;
    f32x4 acc[TILES];
#pragma unroll
    for (int t = 0; t < TILES; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};

    for (int block = block0; block <= block_end; ++block) {
        const int page = table[block];
        const int buffer = (block - block0) & 1;
        f32x4 s = {0.f, 0.f, 0.f, 0.f};
        const uint16_t* key = k_pages + ((size_t)page * num_kv_heads * PAGE + wave * 16 + i16) * head_dim + g4 * 8;
        // a few key/value heads at a time, their keys asked for together (one past the last: the last one's again, not used)
        for (int c0 = 0; c0 < num_kv_heads; c0 += KV_AT_ONCE) {
            bf16x8 kf[KV_AT_ONCE][HD / 32];
#pragma unroll
            for (int u = 0; u < KV_AT_ONCE; ++u) {
                const int c = c0 + u < num_kv_heads ? c0 + u : num_kv_heads - 1;
#pragma unroll
                for (int dc = 0; dc < HD / 32; ++dc) {
                    kf[u][dc] = bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
                    if (dc * 32 + g4 * 8 < head_dim) kf[u][dc] = *reinterpret_cast<const bf16x8*>(key + (size_t)c * PAGE * head_dim + dc * 32);
                }
            }
            f32x4 of_kv[KV_AT_ONCE];
#pragma unroll
            for (int u = 0; u < KV_AT_ONCE; ++u) {
                of_kv[u] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int dc = 0; dc < HD / 32; ++dc) of_kv[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[dc], kf[u][dc], of_kv[u], 0, 0, 0);
            }
            fw_mfma_drain();
#pragma unroll
            for (int u = 0; u < KV_AT_ONCE; ++u)
#pragma unroll
                for (int r = 0; r < 4; ++r) s[r] = kv_of[r] == c0 + u ? of_kv[u][r] : s[r];
        }
        const int key_at = block * PAGE + wave * 16 + i16;
        const bool seen = key_at >= first && key_at <= pos;
        f32x4 mixed = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const float a = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-fmaf(s[r], scale_log2, head_bias[r])));
            s[r] = seen && kv_of[r] >= 0 ? a : 0.0f;
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) mixed = __builtin_amdgcn_mfma_f32_16x16x4f32(mix_row[r], s[r], mixed, 0, 0, 0);
        fw_mfma_drain();
#pragma unroll
        for (int r = 0; r < 4; ++r) lds_p[buffer][g4 * 4 + r][wave * 16 + i16] = float_to_bf16_bits(mixed[r]);
        fw_lds_barrier();       // two buffers: nobody stores into this one again before everybody has passed the next barrier
        const int last_written = pos - block * PAGE;
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) {
            const u32x4 pw = *reinterpret_cast<const u32x4*>(&lds_p[buffer][i16][kb * 32 + g4 * 8]);
            const int in_lane = last_written - kb * 32 - g4 * 8;
            uint32_t keep[4];
#pragma unroll
            for (int word = 0; word < 4; ++word)
                keep[word] = 2 * word + 1 <= in_lane ? 0xffffffffu : (2 * word <= in_lane ? 0xffffu : 0u);
            const uint16_t* value = v_pages + (size_t)page * num_kv_heads * v_dim * PAGE + kb * 32 + g4 * 8;
            for (int c0 = 0; c0 < num_kv_heads; c0 += KV_AT_ONCE) {
                u32x4 v[KV_AT_ONCE][TILES];
#pragma unroll
                for (int u = 0; u < KV_AT_ONCE; ++u) {
                    const int c = c0 + u < num_kv_heads ? c0 + u : num_kv_heads - 1;
#pragma unroll
                    for (int t = 0; t < TILES; ++t) {
                        const int channel = (t * 4 + wave) * 16 + i16;
                        v[u][t] = *reinterpret_cast<const u32x4*>(value + ((size_t)c * v_dim + (channel < v_dim ? channel : v_dim - 1)) * PAGE);
                    }
                }
#pragma unroll
                for (int u = 0; u < KV_AT_ONCE; ++u) {
                    const uint32_t mine = my_kv == c0 + u ? 0xffffffffu : 0u;
                    const u32x4 pm = {pw[0] & mine, pw[1] & mine, pw[2] & mine, pw[3] & mine};
#pragma unroll
                    for (int t = 0; t < TILES; ++t) {
                        const u32x4 clean = {v[u][t][0] & keep[0], v[u][t][1] & keep[1], v[u][t][2] & keep[2], v[u][t][3] & keep[3]};
                        acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, clean), __builtin_bit_cast(bf16x8, pm), acc[t], 0, 0, 0);
                    }
                }
            }
        }
    }
    fw_mfma_drain();
    const int row_splits = (last_block - first_block + pages_per_split) / pages_per_split;
    const int channels = num_heads * v_dim;
    if (i16 < num_heads) {
#pragma unroll
        for (int t = 0; t < TILES; ++t) {
            const int channel = (t * 4 + wave) * 16 + g4 * 4;
            if (channel >= v_dim) break;
            const size_t at = (size_t)i16 * v_dim + channel;
            if (row_splits == 1) {
                f32x4 o = acc[t];
                if (gate) {
#pragma unroll
                    for (int r = 0; r < 4; ++r) o[r] *= sg_gate_quick(gate[(size_t)row * gate_stride + at + r]);
                }
                *reinterpret_cast<u32x2*>(out + (size_t)row * channels + at) = u32x2{sg_pack(o[0], o[1]), sg_pack(o[2], o[3])};
            } else {
                // device-scope stores: they pass the caches that workgroups on other dies do not share
                float* dest = partial + ((size_t)row * gridDim.y + split) * channels + at;
#pragma unroll
                for (int r = 0; r < 4; ++r) __hip_atomic_store(dest + r, acc[t][r], __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
            }
        }
    }
    if (row_splits == 1) return;
    // every wave waits for its own stores to be acknowledged, the workgroup meets, one thread takes the ticket
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (tid == 0) ticket_shared = __hip_atomic_fetch_add(tickets + row, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    __syncthreads();
    if (ticket_shared != row_splits - 1) return;
    if (tid == 0) __hip_atomic_store(tickets + row, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    const float* parts = partial + (size_t)row * gridDim.y * channels;
    for (int item0 = tid; item0 < channels; item0 += 256 * 4) {
        float sum[4] = {0.f, 0.f, 0.f, 0.f};
        for (int sp0 = 0; sp0 < row_splits; sp0 += 8) {
            float v[4][8];
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const int sp = sp0 + e < row_splits ? sp0 + e : row_splits - 1;
#pragma unroll
                for (int u = 0; u < 4; ++u) {
                    const int item = item0 + 256 * u < channels ? item0 + 256 * u : channels - 1;
                    v[u][e] = __hip_atomic_load(parts + (size_t)sp * channels + item, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
                }
            }
#pragma unroll
            for (int e = 0; e < 8; ++e)
                if (sp0 + e < row_splits) {
#pragma unroll
                    for (int u = 0; u < 4; ++u) sum[u] += v[u][e];
                }
        }
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int item = item0 + 256 * u;
            if (item < channels) {
                const float factor = gate ? sg_gate_quick(gate[(size_t)row * gate_stride + item]) : 1.0f;
                out[(size_t)row * channels + item] = float_to_bf16_bits(sum[u] * factor);
            }
        }
    }
}

// One row per request. q: finished bfloat16 queries, or null with `qkv` (float32 [rows][qkv_stride]: q | k | v as the
// projections leave them; qk_norm: q and k of a head are brought to unit RMS; write_kv: the new key
// and value are stored). partial: float32 workspace of rows * max_splits * heads * v_dim; tickets: a zeroed int32 per row, left
// zero. max_context: no row's position reaches it; max_splits * pages_per_split covers the pages such a row sees.
extern "C" int fw_sigmoid_attention_decode(const void* q, const float* qkv, int qkv_stride, int qk_norm, float eps, int write_kv, void* out,
                                           float* partial, int max_splits, int pages_per_split, int max_context, int* tickets,
                                           int tickets_len, void* k_pages, void* v_pages, const int32_t* block_table, int table_stride,
                                           const int32_t* row_seg, const int32_t* row_pos, int rows, int num_heads, int num_kv_heads,
                                           int head_dim, int v_dim, float scale, int window, const float* bias, const float* mix,
                                           const float* gate, int gate_stride, int page_size, int num_pages, void* stream) {
    if (sg_check("sigmoid_attention_decode", rows, num_heads, num_kv_heads, head_dim, v_dim, window, bias, mix, gate, gate_stride, page_size,
                 num_pages, table_stride)) return -1;
    if (sg_tiled_check("sigmoid_attention_decode", num_heads, head_dim, v_dim)) return -1;
    FW_REQUIRE((q == nullptr) != (qkv == nullptr), "sigmoid_attention_decode: either finished queries or the raw projections");
    FW_REQUIRE(qkv == nullptr || qkv_stride >= (num_heads + num_kv_heads) * head_dim + num_kv_heads * v_dim,
               "sigmoid_attention_decode: projections %d wide do not hold q, k and v", qkv_stride);
    FW_REQUIRE(pages_per_split >= 1 && max_splits >= 1 && max_splits <= 65535 && max_context >= 1, "sigmoid_attention_decode: %d splits of %d pages, context %d",
               max_splits, pages_per_split, max_context);
    int blocks = (max_context + PAGE - 1) / PAGE;
    FW_REQUIRE(blocks <= table_stride, "sigmoid_attention_decode: a context of %d tokens exceeds the block table (%d pages)", max_context, table_stride);
    if (window > 0 && (window + PAGE - 2) / PAGE + 1 < blocks) blocks = (window + PAGE - 2) / PAGE + 1;
    FW_REQUIRE((long long)max_splits * pages_per_split >= blocks, "sigmoid_attention_decode: %d splits of %d pages do not cover %d pages", max_splits,
               pages_per_split, blocks);
    FW_REQUIRE(max_splits == 1 || (partial != nullptr && tickets != nullptr && tickets_len >= rows), "sigmoid_attention_decode: %d rows need as many ticket counters", rows);
    if (rows == 0) return 0;
    const SigmoidFused fused = {qkv, qkv_stride, qk_norm, write_kv, eps};
    dim3 grid(rows, max_splits);
#define SG_LAUNCH(HD, FUSED)                                                                                                             \
    sigmoid_attention_decode_kernel<HD, FUSED><<<grid, 256, 0, (hipStream_t)stream>>>(                                                    \
        (const uint16_t*)q, (uint16_t*)out, partial, tickets, (uint16_t*)k_pages, (uint16_t*)v_pages, block_table, table_stride, row_seg, \
        row_pos, num_heads, num_kv_heads, head_dim, v_dim, scale * LOG2E_F, window, bias, mix, gate, gate_stride, pages_per_split, fused)
#define SG_BY_FORM(HD) if (qkv) SG_LAUNCH(HD, true); else SG_LAUNCH(HD, false)
    const int width = sg_class(head_dim, v_dim);
    if (width == 32) { SG_BY_FORM(32); }
    else if (width == 64) { SG_BY_FORM(64); }
    else if (width == 128) { SG_BY_FORM(128); }
    else { SG_BY_FORM(256); }
#undef SG_BY_FORM
#undef SG_LAUNCH
    FW_LAUNCH_CHECK("sigmoid_attention_decode");
    return 0;
}
