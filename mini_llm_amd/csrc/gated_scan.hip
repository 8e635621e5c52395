// A gated recurrence whose gate and candidate depend on the current row alone (minGRU), so that a whole portion is a scan of
// first-order maps: with sums p = W_z h + b_z and u = W_x h + b_x, z = sigmoid(p), candidate c = u + shift where u >= 0 and sigmoid(u)
// where u < 0, S_t = (1 - z) S_(t-1) + z c element by element, and the result S_t * silu(g). State, gates and sums are 32-bit.
//
// A row is the map S -> A S + B with A = 1 - z, B = z c; a run of rows is one such map too (A = A2 A1, B = A2 B1 + B2 for run 1 before
// run 2), which is what lets a portion's chunks run side by side.
#include "common.h"

namespace {

constexpr int SCAN_WAVES = 4, SCAN_ROWS = 16, SCAN_CHUNK = SCAN_WAVES * SCAN_ROWS;   // a wave takes 64 elements of 16 rows
constexpr int SCAN_ROW_BY_ROW = 16;   // portions up to so many rows go row by row, a thread an element

// The columns of the fused product a row holds its sums in.
struct ScanColumns {
    const float* rows;
    int stride, z_at, x_at, g_at;
};

__device__ __forceinline__ void row_map(float p, float u, float shift, float& keep, float& add) {
    const float small = expf(-fabsf(p)), over = 1.0f / (1.0f + small);   // sigmoid of |p| and of -|p|, neither by a difference
    const float z = p >= 0.0f ? over : small * over;
    keep = p >= 0.0f ? small * over : over;
    float candidate = u + shift;
    if (u < 0.0f) {
        const float e = expf(u);
        candidate = e / (1.0f + e);
    }
    add = z * candidate;
}

__device__ __forceinline__ float silu(float g) { return g / (1.0f + expf(-g)); }

// Row by row: a thread an element of a request. The next row's sums are asked for before the current ones are used.
template <typename T>
__global__ __launch_bounds__(256) void scan_rows_kernel(ScanColumns in, float* __restrict__ state, long long state_stride, const int* __restrict__ q_starts,
                                                        const int* __restrict__ state_slots, T* __restrict__ out, int out_stride, int width, float shift) {
    const int request = blockIdx.y, channel = blockIdx.x * blockDim.x + threadIdx.x;
    const int slot = state_slots[request];
    if (slot < 0 || channel >= width) return;
    const int first = q_starts[request], end = q_starts[request + 1];
    if (first >= end) return;
    float s = state[slot * state_stride + channel];
    const float* at = in.rows + (size_t)first * in.stride + channel;
    float p = at[in.z_at], u = at[in.x_at], g = at[in.g_at];
    for (int row = first; row < end; row++) {
        const float* next = in.rows + (size_t)min(row + 1, end - 1) * in.stride + channel;
        const float p1 = next[in.z_at], u1 = next[in.x_at], g1 = next[in.g_at];
        float keep, add;
        row_map(p, u, shift, keep, add);
        s = keep * s + add;
        out[(size_t)row * out_stride + channel] = from_float<T>(s * silu(g));
        p = p1;
        u = u1;
        g = g1;
    }
    state[slot * state_stride + channel] = s;
}

// Where the record (A [width], B [width]) of a request's chunk lies: behind those of the requests before it.
__device__ __forceinline__ size_t record_at(int first, int request, int chunk, int width) {
    return ((size_t)(first / SCAN_CHUNK) + request + chunk) * 2 * width;
}

// The rows of this wave in registers, as maps; rows beyond the portion are the identity.
struct WaveRows {
    float keep[SCAN_ROWS], add[SCAN_ROWS];
};
__device__ __forceinline__ void load_rows(const ScanColumns& in, int row0, int end, int channel, float shift, WaveRows& rows) {
    float p[SCAN_ROWS], u[SCAN_ROWS];
#pragma unroll
    for (int t = 0; t < SCAN_ROWS; t++) {
        const float* at = in.rows + (size_t)min(row0 + t, end - 1) * in.stride + channel;
        p[t] = at[in.z_at];
        u[t] = at[in.x_at];
    }
#pragma unroll
    for (int t = 0; t < SCAN_ROWS; t++) {
        row_map(p[t], u[t], shift, rows.keep[t], rows.add[t]);
        if (row0 + t >= end) rows.keep[t] = 1.0f, rows.add[t] = 0.0f;
    }
}
__device__ __forceinline__ void run_map(const WaveRows& rows, float& a, float& b) {
    a = 1.0f;
    b = 0.0f;
#pragma unroll
    for (int t = 0; t < SCAN_ROWS; t++) {
        a *= rows.keep[t];
        b = rows.keep[t] * b + rows.add[t];
    }
}

// The map of every chunk of the portions that have more than one. The first chunk's record holds the state the portion starts from
// (in A's place) and the state behind the chunk (in B's): the last chunk of the next kernel overwrites the state slot while others
// still need what was in it.
__global__ __launch_bounds__(64 * SCAN_WAVES) void scan_chunks_kernel(ScanColumns in, const float* __restrict__ state, long long state_stride,
                                                                      const int* __restrict__ q_starts, const int* __restrict__ state_slots,
                                                                      float* __restrict__ records, int width, float shift) {
    __shared__ float maps[SCAN_WAVES][2][WAVE];
    const int request = blockIdx.z, chunk = blockIdx.y, lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
    const int slot = state_slots[request];
    if (slot < 0) return;
    const int first = q_starts[request], end = q_starts[request + 1];
    if (end - first <= SCAN_CHUNK || first + (chunk + 1) * SCAN_CHUNK >= end) return;   // one chunk alone, and the last one, need no record
    const int channel = blockIdx.x * WAVE + lane, inside = min(channel, width - 1);
    WaveRows rows;
    load_rows(in, first + chunk * SCAN_CHUNK + wave * SCAN_ROWS, end, inside, shift, rows);
    float a, b;
    run_map(rows, a, b);
    maps[wave][0][lane] = a;
    maps[wave][1][lane] = b;
    __syncthreads();
    if (wave != 0 || channel >= width) return;
    for (int w = 1; w < SCAN_WAVES; w++) {
        b = maps[w][0][lane] * b + maps[w][1][lane];
        a *= maps[w][0][lane];
    }
    float* record = records + record_at(first, request, chunk, width) + channel;
    if (chunk == 0) {
        const float start = state[slot * state_stride + channel];
        b = a * start + b;
        a = start;
    }
    record[0] = a;
    record[width] = b;
}

// The chunks once more, now from the state each starts at: the records of the chunks before it, a quarter of them to each wave.
template <typename T>
__global__ __launch_bounds__(64 * SCAN_WAVES) void scan_out_kernel(ScanColumns in, float* __restrict__ state, long long state_stride, const int* __restrict__ q_starts,
                                                                   const int* __restrict__ state_slots, const float* __restrict__ records,
                                                                   T* __restrict__ out, int out_stride, int width, float shift) {
    __shared__ float before[SCAN_WAVES][2][WAVE], maps[SCAN_WAVES][2][WAVE];
    const int request = blockIdx.z, chunk = blockIdx.y, lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
    const int slot = state_slots[request];
    if (slot < 0) return;
    const int first = q_starts[request], end = q_starts[request + 1];
    const int chunk0 = first + chunk * SCAN_CHUNK;
    if (chunk0 >= end) return;
    const int channel = blockIdx.x * WAVE + lane, inside = min(channel, width - 1);
    const bool lone = end - first <= SCAN_CHUNK;
    const int row0 = chunk0 + wave * SCAN_ROWS;
    WaveRows rows;
    float g[SCAN_ROWS];
#pragma unroll
    for (int t = 0; t < SCAN_ROWS; t++) g[t] = in.rows[(size_t)min(row0 + t, end - 1) * in.stride + in.g_at + inside];
    load_rows(in, row0, end, inside, shift, rows);
    // what the first chunk's record (or the slot) gives to start from, and the chunks 1 .. chunk - 1 behind it
    float start = 0.0f;
    if (lone) start = state[slot * state_stride + inside];
    else start = records[record_at(first, request, 0, width) + (chunk == 0 ? 0 : width) + inside];
    const int between = max(chunk - 1, 0), share = (between + SCAN_WAVES - 1) / SCAN_WAVES;
    const int lo = 1 + min(between, wave * share), hi = 1 + min(between, (wave + 1) * share);
    float a = 1.0f, b = 0.0f;
#pragma unroll 4
    for (int k = lo; k < hi; k++) {
        const float* record = records + record_at(first, request, k, width) + inside;
        const float ka = record[0], kb = record[width];
        b = ka * b + kb;
        a *= ka;
    }
    before[wave][0][lane] = a;
    before[wave][1][lane] = b;
    run_map(rows, a, b);
    maps[wave][0][lane] = a;
    maps[wave][1][lane] = b;
    __syncthreads();
    float s = start;
#pragma unroll
    for (int w = 0; w < SCAN_WAVES; w++) s = before[w][0][lane] * s + before[w][1][lane];
    for (int w = 0; w < wave; w++) s = maps[w][0][lane] * s + maps[w][1][lane];
    if (channel >= width) return;
#pragma unroll
    for (int t = 0; t < SCAN_ROWS; t++) {
        s = rows.keep[t] * s + rows.add[t];
        if (row0 + t < end) out[(size_t)(row0 + t) * out_stride + channel] = from_float<T>(s * silu(g[t]));
    }
    if (chunk0 + SCAN_CHUNK >= end && wave == SCAN_WAVES - 1) state[slot * state_stride + channel] = s;   // rows beyond the end kept it
}

template <typename T>
void launch_scan(const ScanColumns& in, float* state, long long state_stride, const int* q_starts, const int* state_slots, T* out, int out_stride,
                 int n_requests, int width, float shift, int max_q_len, float* records, hipStream_t stream) {
    if (max_q_len <= SCAN_ROW_BY_ROW) {
        dim3 grid(ceil_div(width, 256), n_requests);
        scan_rows_kernel<T><<<grid, 256, 0, stream>>>(in, state, state_stride, q_starts, state_slots, out, out_stride, width, shift);
        return;
    }
    dim3 grid(ceil_div(width, WAVE), ceil_div(max_q_len, SCAN_CHUNK), n_requests);
    if (max_q_len > SCAN_CHUNK)
        scan_chunks_kernel<<<grid, 64 * SCAN_WAVES, 0, stream>>>(in, state, state_stride, q_starts, state_slots, records, width, shift);
    scan_out_kernel<T><<<grid, 64 * SCAN_WAVES, 0, stream>>>(in, state, state_stride, q_starts, state_slots, records, out, out_stride, width, shift);
}

}  // namespace

// Rows of a chunk: a batch of n rows in r requests needs (n / this + r + 1) * 2 * width floats for its records.
MLLM_API int mllm_gated_scan_chunk_rows() { return SCAN_CHUNK; }

// rows: [n_rows, stride] 32-bit sums holding the gate's, the candidate's and the output gate's columns (`width` each). q_starts
// [n_requests + 1], state_slots [n_requests] (negative: the request is passed by and its rows of out are left alone); state: a row of
// `width` floats a slot, state_stride apart. max_q_len: the longest portion, or a bound on it.
MLLM_API int mllm_gated_scan(const float* rows, int stride, int z_at, int x_at, int g_at, float* state, long long state_stride, const int* q_starts,
                             const int* state_slots, void* out, int out_stride, int n_rows, int n_requests, int width, float shift, int max_q_len,
                             float* records, long long record_floats, int dtype, hipStream_t stream) {
    MLLM_REQUIRE(n_rows >= 0 && n_requests >= 0 && n_requests <= 65535 && width > 0 && max_q_len >= 0, "gated_scan: bad sizes");
    MLLM_REQUIRE(rows && state && q_starts && state_slots && out, "gated_scan: a missing operand");
    MLLM_REQUIRE(z_at >= 0 && x_at >= 0 && g_at >= 0 && z_at + width <= stride && x_at + width <= stride && g_at + width <= stride && state_stride >= width &&
                     out_stride >= width, "gated_scan: columns beyond the rows");
    MLLM_REQUIRE(dtype == MLLM_F32 || dtype == MLLM_BF16, "gated_scan: unknown dtype %d", dtype);
    MLLM_REQUIRE(ceil_div(max_q_len, SCAN_CHUNK) <= 65535, "gated_scan: portions of %d rows", max_q_len);
    MLLM_REQUIRE(max_q_len <= SCAN_CHUNK || (records && record_floats >= ((long long)n_rows / SCAN_CHUNK + n_requests + 1) * 2 * width),
                 "gated_scan: no room for the chunks' records");
    if (n_rows == 0 || n_requests == 0) return 0;
    mllm_count_kernel(MLLM_K_GATED_SCAN);
    const ScanColumns in{rows, stride, z_at, x_at, g_at};
    if (dtype == MLLM_F32) launch_scan<float>(in, state, state_stride, q_starts, state_slots, (float*)out, out_stride, n_requests, width, shift, max_q_len, records, stream);
    else launch_scan<bf16_t>(in, state, state_stride, q_starts, state_slots, (bf16_t*)out, out_stride, n_requests, width, shift, max_q_len, records, stream);
    return mllm_check_launch("gated_scan");
}
