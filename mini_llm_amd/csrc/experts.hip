// Routed experts that run for the rows that picked them, and for no others: the lists of rows by expert that the grouped products of
// many rows walk (gemm_stream.h), and the two products of few rows (decoding), which find their rows themselves.
//
// A router leaves picks [rows, top] (expert ids, -1 for none) and their weights. Entry p = row * top + k is row `row` with its k-th
// pick. An expert's matrices: the gate and up rows of the up matrix in turns of 32, [2 * units, width], and the down matrix [width,
// units], both packed, one expert behind the other; units a multiple of 64 (zero rows and columns fill it up), the down matrix's rows
// whole sixteens. The down product of a row's k-th pick goes to plane k of out [top, rows, width]: whoever reads the branch adds the
// planes up, in that order.
#include "common.h"
#include "gate_unit.h"

namespace {

constexpr int MAX_EXPERTS = 1024;

// The lists, a block an expert, without an atomic that could order them: entries of an expert in the order of their rows, experts behind
// each other. Every block counts all experts' entries (so that it knows where its own begin) and places its own: wave w counts a
// contiguous share of the entries, 64 at a time by ballots (of up to 64 experts: lane e keeps expert e's count; of more: by LDS counters,
// which so many addresses seldom make wait for each other), and places its share behind those of the waves before it.
constexpr int LIST_WAVES = 16;

__global__ __launch_bounds__(64 * LIST_WAVES) void expert_lists_kernel(const int* __restrict__ picks, const float* __restrict__ pick_weights, int n_rows, int top,
                                                                       int n_experts, int tile_rows, int* __restrict__ a_row, int* __restrict__ out_row,
                                                                       float* __restrict__ weight, int4* __restrict__ tiles, int* __restrict__ n_tiles) {
    __shared__ int counts[MAX_EXPERTS];
    __shared__ int mine_before[LIST_WAVES], start, first_tile;
    const int expert = blockIdx.x, tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE;
    const int entries = n_rows * top, chunks = (entries + WAVE - 1) / WAVE;
    const int share = (chunks + LIST_WAVES - 1) / LIST_WAVES, chunk0 = min(chunks, wave * share), chunk1 = min(chunks, chunk0 + share);
    for (int e = tid; e < n_experts; e += 64 * LIST_WAVES) counts[e] = 0;
    __syncthreads();
    int mine = 0, of_lane = 0;
    constexpr int AHEAD = 4;
    for (int c0 = chunk0; c0 < chunk1; c0 += AHEAD) {
        int pick[AHEAD];
#pragma unroll
        for (int u = 0; u < AHEAD; u++) {
            const int p = (c0 + u) * WAVE + lane;
            pick[u] = c0 + u < chunk1 && p < entries ? picks[p] : -1;
        }
#pragma unroll
        for (int u = 0; u < AHEAD; u++) {
            mine += __popcll(__ballot(pick[u] == expert));
            if (n_experts <= WAVE) {
                for (int e = 0; e < n_experts; e++) {
                    const int n = __popcll(__ballot(pick[u] == e));
                    of_lane += lane == e ? n : 0;
                }
            } else if (pick[u] >= 0 && pick[u] < n_experts) {
                atomicAdd(&counts[pick[u]], 1);
            }
        }
    }
    if (n_experts <= WAVE && lane < n_experts && of_lane > 0) atomicAdd(&counts[lane], of_lane);
    if (lane == 0) mine_before[wave] = mine;
    __syncthreads();
    if (wave == 0) {
        int before = 0, tiles_before = 0;
        for (int e = lane; e < expert; e += WAVE) {
            before += counts[e];
            tiles_before += (counts[e] + tile_rows - 1) / tile_rows;
        }
#pragma unroll
        for (int offset = WAVE / 2; offset > 0; offset >>= 1) {
            before += __shfl_xor(before, offset, WAVE);
            tiles_before += __shfl_xor(tiles_before, offset, WAVE);
        }
        if (lane == 0) {
            start = before;
            first_tile = tiles_before;
        }
    }
    __syncthreads();
    const int total = counts[expert], my_tiles = (total + tile_rows - 1) / tile_rows, first = start;
    for (int t = tid; t < my_tiles; t += 64 * LIST_WAVES) tiles[first_tile + t] = make_int4(expert, first + t * tile_rows, first + total, 0);
    if (expert == n_experts - 1 && tid == 0) *n_tiles = first_tile + my_tiles;
    if (mine == 0) return;   // (uniform over the wave)
    int placed = first;
    for (int w = 0; w < wave; w++) placed += mine_before[w];
    for (int c0 = chunk0; c0 < chunk1; c0 += AHEAD) {
        int pick[AHEAD];
        float its_weight[AHEAD];
#pragma unroll
        for (int u = 0; u < AHEAD; u++) {
            const int p = (c0 + u) * WAVE + lane, inside = min(p, entries - 1);
            pick[u] = picks[inside];
            its_weight[u] = pick_weights[inside];
            if (c0 + u >= chunk1 || p >= entries) pick[u] = -1;
        }
#pragma unroll
        for (int u = 0; u < AHEAD; u++) {
            const unsigned long long ballot = __ballot(pick[u] == expert);
            if (pick[u] == expert) {
                const int at = placed + __popcll(ballot & ((1ull << lane) - 1)), p = (c0 + u) * WAVE + lane, row = p / top;
                a_row[at] = row;
                out_row[at] = (p - row * top) * n_rows + row;
                weight[at] = its_weight[u];
            }
            placed += __popcll(ballot);
        }
    }
}

constexpr int FEW_ROWS = 64;

// This block's expert: the entries that picked it, and their weights, in LDS (a row picks an expert at most once, so there are at most
// FEW_ROWS). Returns how many; called by all threads.
__device__ __forceinline__ int gather_entries(const int* __restrict__ picks, const float* __restrict__ pick_weights, int entries, int expert, int* list,
                                              float* weights, int* count) {
    if (threadIdx.x < WAVE) {
        int found = 0;
        for (int p0 = 0; p0 < entries; p0 += WAVE) {
            const int p = p0 + threadIdx.x, inside = min(p, entries - 1);
            const int pick = picks[inside];
            const float weight = pick_weights ? pick_weights[inside] : 0.0f;
            const bool here = p < entries && pick == expert;
            const unsigned long long ballot = __ballot(here);
            const int at = found + __popcll(ballot & ((1ull << threadIdx.x) - 1));
            if (here && at < FEW_ROWS) {
                list[at] = p;
                weights[at] = weight;
            }
            found += __popcll(ballot);
        }
        if (threadIdx.x == 0) *count = min(found, FEW_ROWS);
    }
    __syncthreads();
    return *count;
}

// A step of K of one 16 x 16 tile of sums: 32 of bfloat16, 16 of float (the true 32-bit product), from 16 bytes a lane of either operand.
template <typename T>
__device__ __forceinline__ void multiply(const Vec16& w, const Vec16& x, f32x4& acc) {
    if constexpr (sizeof(T) == 2) {
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(&w), *reinterpret_cast<const bf16x8*>(&x), acc, 0, 0, 0);
    } else {
#pragma unroll
        for (int c = 0; c < 4; c++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32((*reinterpret_cast<const f32x4*>(&w))[c], (*reinterpret_cast<const f32x4*>(&x))[c], acc, 0, 0, 0);
    }
}

// hidden[p, units] = the gate unit of entry p's row with its expert's matrices. A block takes 16 units of an expert: its gate and up rows
// stream from memory once, straight into matrix-core operands (out^T = W . x^T, W the 16-row operand), for up to MT times 16 rows at a
// time; the waves take the steps along the width in turns and their sums meet in LDS, where the gate unit is. Rows of x are whole 16-byte
// pieces; a piece beyond their end is the last one again, and meets the zeros that fill the packed matrix.
template <typename T, int MT, int KSPLIT>
__global__ __launch_bounds__(64 * KSPLIT) void experts_few_up_kernel(const T* __restrict__ x, const T* __restrict__ W, T* __restrict__ hidden,
                                                                     const int* __restrict__ picks, const float* __restrict__ pick_weights, int n_rows, int top,
                                                                     int units, int width, GateUnit unit, int weigh_input) {
    constexpr int UNROLL = MT == 4 ? 4 : 8, VEC = 16 / (int)sizeof(T), KSTEP = 4 * VEC;
    __shared__ float sums[KSPLIT][2 * MT * 4][WAVE];
    __shared__ int list[FEW_ROWS], count;
    __shared__ float weights[FEW_ROWS];
    const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE, row16 = lane % 16, quad = lane / 16;
    const int expert = blockIdx.y, u0 = blockIdx.x * 16;
    const int n = gather_entries(picks, pick_weights, n_rows * top, expert, list, weights, &count);
    if (n == 0) return;   // nobody picked this expert (uniform over the block)
    const int steps = packed_k_steps<T>(width);
    const int gate_tile = expert * (2 * units / 16) + u0 / 32 * 4 + u0 / 16 % 2;   // 32 gate rows, 32 up rows in turn
    const T* x_row[MT];
#pragma unroll
    for (int i = 0; i < MT; i++) x_row[i] = x + (size_t)(list[min(i * 16 + row16, n - 1)] / top) * width;   // beyond the last: never stored
    f32x4 gate[MT], up[MT];
#pragma unroll
    for (int i = 0; i < MT; i++) gate[i] = up[i] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    for (int step0 = wave * UNROLL; step0 < steps; step0 += KSPLIT * UNROLL) {
        Vec16 g_op[UNROLL], u_op[UNROLL], x_op[UNROLL][MT];
#pragma unroll
        for (int u = 0; u < UNROLL; u++) {
            const int step = min(step0 + u, steps - 1);   // beyond the end: the last step again, not used
            g_op[u] = *reinterpret_cast<const Vec16*>(W + packed_offset<T>(gate_tile, step, steps, lane));
            u_op[u] = *reinterpret_cast<const Vec16*>(W + packed_offset<T>(gate_tile + 2, step, steps, lane));
#pragma unroll
            for (int i = 0; i < MT; i++) x_op[u][i] = *reinterpret_cast<const Vec16*>(x_row[i] + min(step * KSTEP + quad * VEC, width - VEC));
        }
#pragma unroll
        for (int u = 0; u < UNROLL; u++) {
            if (step0 + u >= steps) break;
#pragma unroll
            for (int i = 0; i < MT; i++) {
                multiply<T>(g_op[u], x_op[u][i], gate[i]);
                multiply<T>(u_op[u], x_op[u][i], up[i]);
            }
        }
    }
    // gate[i][r] belongs to entry i * 16 + lane % 16, unit u0 + 4 * (lane / 16) + r
#pragma unroll
    for (int i = 0; i < MT; i++)
#pragma unroll
        for (int r = 0; r < 4; r++) {
            sums[wave][i * 4 + r][lane] = gate[i][r];
            sums[wave][(MT + i) * 4 + r][lane] = up[i][r];
        }
    __syncthreads();
    // a thread finishes whole units: entry index / 16, unit index % 16
    for (int index = threadIdx.x; index < n * 16; index += 64 * KSPLIT) {
        const int entry = index / 16, unit_at = index % 16, i = entry / 16;
        const int l = (unit_at / 4) * 16 + entry % 16, r = unit_at % 4;
        float g = 0.0f, u = 0.0f;
#pragma unroll
        for (int w = 0; w < KSPLIT; w++) {   // the same order for every element
            g += sums[w][i * 4 + r][l];
            u += sums[w][(MT + i) * 4 + r][l];
        }
        const float weight = weights[entry];
        const float value = weigh_input ? gated(g * weight, u * weight, unit) : gated(g, u, unit) * weight;
        hidden[(size_t)list[entry] * units + u0 + unit_at] = from_float<T>(value);
    }
}

// out[k, row, :] = hidden[row * top + k, units] . its expert's down matrix^T, 32-bit; a block takes 16 columns of an expert.
template <typename T, int MT, int KSPLIT>
__global__ __launch_bounds__(64 * KSPLIT) void experts_few_down_kernel(const T* __restrict__ hidden, const T* __restrict__ W, float* __restrict__ out,
                                                                       const int* __restrict__ picks, int n_rows, int top, int units, int width) {
    constexpr int UNROLL = MT == 4 ? 4 : 8, VEC = 16 / (int)sizeof(T), KSTEP = 4 * VEC;
    __shared__ float sums[KSPLIT][MT * 4][WAVE];
    __shared__ int list[FEW_ROWS], count;
    __shared__ float weights[FEW_ROWS];
    const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE, row16 = lane % 16, quad = lane / 16;
    const int expert = blockIdx.y, n0 = blockIdx.x * 16;
    const int n = gather_entries(picks, nullptr, n_rows * top, expert, list, weights, &count);
    if (n == 0) return;
    const int steps = units / KSTEP, tile = expert * ((width + 15) / 16) + blockIdx.x;   // (the units are whole steps)
    const T* h_row[MT];
#pragma unroll
    for (int i = 0; i < MT; i++) h_row[i] = hidden + (size_t)list[min(i * 16 + row16, n - 1)] * units + quad * VEC;
    f32x4 acc[MT];
#pragma unroll
    for (int i = 0; i < MT; i++) acc[i] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    for (int step0 = wave * UNROLL; step0 < steps; step0 += KSPLIT * UNROLL) {
        Vec16 w_op[UNROLL], h_op[UNROLL][MT];
#pragma unroll
        for (int u = 0; u < UNROLL; u++) {
            const int step = min(step0 + u, steps - 1);
            w_op[u] = *reinterpret_cast<const Vec16*>(W + packed_offset<T>(tile, step, steps, lane));
#pragma unroll
            for (int i = 0; i < MT; i++) h_op[u][i] = *reinterpret_cast<const Vec16*>(h_row[i] + step * KSTEP);
        }
#pragma unroll
        for (int u = 0; u < UNROLL; u++) {
            if (step0 + u >= steps) break;
#pragma unroll
            for (int i = 0; i < MT; i++) multiply<T>(w_op[u], h_op[u][i], acc[i]);
        }
    }
#pragma unroll
    for (int i = 0; i < MT; i++)
#pragma unroll
        for (int r = 0; r < 4; r++) sums[wave][i * 4 + r][lane] = acc[i][r];
    __syncthreads();
    for (int index = threadIdx.x; index < n * 16; index += 64 * KSPLIT) {
        const int entry = index / 16, column = index % 16, i = entry / 16;
        const int l = (column / 4) * 16 + entry % 16, r = column % 4;
        if (n0 + column >= width) continue;
        float value = 0.0f;
#pragma unroll
        for (int w = 0; w < KSPLIT; w++) value += sums[w][i * 4 + r][l];
        const int p = list[entry], row = p / top;
        out[((size_t)(p - row * top) * n_rows + row) * width + n0 + column] = value;
    }
}

bool few_sizes(int n_rows, int top, int n_experts, int units, int width, int dtype) {
    const int vec = dtype == MLLM_F32 ? 4 : 8;
    return (dtype == MLLM_F32 || dtype == MLLM_BF16) && n_rows >= 0 && n_rows <= FEW_ROWS && top >= 1 && n_experts >= 1 && n_experts <= MAX_EXPERTS && top <= n_experts &&
           units >= 64 && units % 64 == 0 && width >= vec && width % vec == 0;
}

}  // namespace

// Rows up to which the products of few rows take the experts (0: rows of this width are not whole 16-byte pieces).
MLLM_API int mllm_experts_few_rows(int width, int dtype) { return few_sizes(0, 1, 1, 64, width, dtype) ? FEW_ROWS : 0; }

// picks, pick_weights [n_rows, top] -> the lists: a_row, out_row, weight [n_rows * top] (as many entries as picks that name an expert), tiles [up to
// n_rows * top / tile_rows + min(n_experts, n_rows * top)] of four integers each, n_tiles [1].
MLLM_API int mllm_expert_lists(const int* picks, const float* pick_weights, int n_rows, int top, int n_experts, int tile_rows, int* a_row, int* out_row, float* weight,
                               int* tiles, int* n_tiles, hipStream_t stream) {
    MLLM_REQUIRE(n_rows >= 0 && top >= 1 && n_experts >= 1 && n_experts <= MAX_EXPERTS && tile_rows >= 1 && (long long)n_rows * top < (1LL << 30), "expert_lists: bad sizes");
    MLLM_REQUIRE(picks && pick_weights && a_row && out_row && weight && tiles && n_tiles && ((uintptr_t)tiles & 15) == 0, "expert_lists: a missing operand");
    mllm_count_kernel(MLLM_K_EXPERT_LISTS);
    expert_lists_kernel<<<n_experts, 64 * LIST_WAVES, 0, stream>>>(picks, pick_weights, n_rows, top, n_experts, tile_rows, a_row, out_row, weight, (int4*)tiles, n_tiles);
    return mllm_check_launch("expert_lists");
}

// STEPS: the steps of K; four waves share them, eight where they are many
#define MLLM_FEW_CASES(KERNEL, T, GRID, STEPS, ...)                                                    \
    do {                                                                                               \
        if ((STEPS) <= 32) {                                                                           \
            if (n_rows <= 16) KERNEL<T, 1, 4><<<GRID, 256, 0, stream>>>(__VA_ARGS__);                  \
            else if (n_rows <= 32) KERNEL<T, 2, 4><<<GRID, 256, 0, stream>>>(__VA_ARGS__);             \
            else KERNEL<T, 4, 4><<<GRID, 256, 0, stream>>>(__VA_ARGS__);                               \
        } else {                                                                                       \
            if (n_rows <= 16) KERNEL<T, 1, 8><<<GRID, 512, 0, stream>>>(__VA_ARGS__);                  \
            else if (n_rows <= 32) KERNEL<T, 2, 8><<<GRID, 512, 0, stream>>>(__VA_ARGS__);             \
            else KERNEL<T, 4, 4><<<GRID, 256, 0, stream>>>(__VA_ARGS__);   /* (its sums take 32 KB of LDS as it is) */ \
        }                                                                                              \
    } while (0)

// x [n_rows, width], hidden [n_rows * top, units] (rows of picks that name no expert are left alone), W packed [n_experts * 2 * units, width].
MLLM_API int mllm_experts_few_up(const void* x, const void* W, void* hidden, const int* picks, const float* pick_weights, int n_rows, int top, int n_experts, int units,
                                 int width, float limit, float alpha, float shift, int weigh_input, int dtype, hipStream_t stream) {
    MLLM_REQUIRE(few_sizes(n_rows, top, n_experts, units, width, dtype), "experts_few_up: no kernel for %d rows, %d of %d experts, %d units, width %d", n_rows, top, n_experts, units, width);
    MLLM_REQUIRE(x && W && hidden && picks && pick_weights && limit > 0.0f && ((uintptr_t)x & 15) == 0, "experts_few_up: a missing operand");
    if (n_rows == 0) return 0;
    mllm_count_kernel(MLLM_K_EXPERTS_FEW);
    const dim3 grid(units / 16, n_experts);
    const GateUnit unit{limit, alpha, shift};
    if (dtype == MLLM_F32)
        MLLM_FEW_CASES(experts_few_up_kernel, float, grid, packed_k_steps<float>(width), (const float*)x, (const float*)W, (float*)hidden, picks, pick_weights, n_rows, top,
                       units, width, unit, weigh_input);
    else
        MLLM_FEW_CASES(experts_few_up_kernel, bf16_t, grid, packed_k_steps<bf16_t>(width), (const bf16_t*)x, (const bf16_t*)W, (bf16_t*)hidden, picks, pick_weights, n_rows,
                       top, units, width, unit, weigh_input);
    return mllm_check_launch("experts_few_up");
}

// out [top, n_rows, width] (rows of picks that name no expert are left alone), W packed, every expert's [width, units] filled up to whole sixteens of rows.
MLLM_API int mllm_experts_few_down(const void* hidden, const void* W, float* out, const int* picks, int n_rows, int top, int n_experts, int units, int width, int dtype,
                                   hipStream_t stream) {
    MLLM_REQUIRE(few_sizes(n_rows, top, n_experts, units, width, dtype), "experts_few_down: no kernel for %d rows, %d of %d experts, %d units, width %d", n_rows, top, n_experts, units, width);
    MLLM_REQUIRE(hidden && W && out && picks && ((uintptr_t)hidden & 15) == 0, "experts_few_down: a missing operand");
    if (n_rows == 0) return 0;
    mllm_count_kernel(MLLM_K_EXPERTS_FEW);
    const dim3 grid(ceil_div(width, 16), n_experts);
    if (dtype == MLLM_F32)
        MLLM_FEW_CASES(experts_few_down_kernel, float, grid, units / 16, (const float*)hidden, (const float*)W, out, picks, n_rows, top, units, width);
    else
        MLLM_FEW_CASES(experts_few_down_kernel, bf16_t, grid, units / 32, (const bf16_t*)hidden, (const bf16_t*)W, out, picks, n_rows, top, units, width);
    return mllm_check_launch("experts_few_down");
}
