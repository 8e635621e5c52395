// A matrix per head and request whose rows fade at a pace of their own (gated linear attention): S_t = diag(alpha_t) S_(t-1) + k_t v_t^T, o_t =
// S_t^T q_t, with a decay per key channel, alpha = sigmoid(z)^(1 / tau), z = up^T low + bias from a few 32-bit sums `low` a row. Behind it every
// head's o is divided by its root mean square, multiplied by a gain vector that all heads share and by silu of a gate row.
// Everything is 32-bit up to the result. Decays are kept as logarithms to the base of two, so that a decay is one 2^x; sums of them over
// stretches of rows are taken in the direction in which no large terms cancel.
//
// Two ways through a portion: row by row (decoding and short portions), and chunk by chunk in three kernels (long portions).
#include "common.h"

#include <math.h>

namespace {

constexpr float LOG2E = 1.4426950408889634f;
constexpr int THREADS = 512, WAVES = THREADS / WAVE, SUB = 16;

// Where a batch's operands lie: columns of the float32 rows of one fused product.
struct MemoryRows {
    const float* rows;
    int stride, q_at, k_at, v_at, g_at, low_at;
    const float* up;     // [rank, n_heads * dim]
    const float* bias;   // [n_heads * dim]
    int rank;
    float inverse_tau, q_scale;
    const float* gain;   // [vdim]
    float eps;
    const int* q_starts;
    const int* state_slots;
    int dim, vdim;
};

__device__ __forceinline__ float exp2_of(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float silu_of(float z) { return z / (1.0f + expf(-z)); }
// log2 of sigmoid(z)^(1 / tau)
__device__ __forceinline__ float log2_decay(float z, float inverse_tau) {
    return -(fmaxf(-z, 0.0f) + log1pf(expf(-fabsf(z)))) * (LOG2E * inverse_tau);
}

// ---- row by row ---------------------------------------------------------------------------------------------------------------------
// A block takes one (request, head, tile of VT value columns) and walks the request's rows of this step in order; thread (part p, column j)
// keeps S[p R .. p R + R - 1, j] in registers. Rows are taken TB at a time: q, k, v, the decays and the gates are staged in LDS, every thread
// moves its piece of S on row by row and leaves its share of each row's output. NORMS: the tile holds all of the head's values, and a wave a
// row adds the shares up, norms and gates them into `out`; else the sums go to `sums` as they are.
template <typename T, int R, bool NORMS>
__global__ __launch_bounds__(THREADS) void memory_rows_kernel(MemoryRows op, float* __restrict__ state, long long state_stride, T* __restrict__ out,
                                                              float* __restrict__ sums, int P, int VT, int TB) {
    extern __shared__ float lds[];
    const int request = blockIdx.x, head = blockIdx.y, n_heads = gridDim.y, dim = op.dim, vdim = op.vdim;
    const int slot = op.state_slots[request];
    const int first_row = op.q_starts[request], rows = op.q_starts[request + 1] - first_row;
    if (slot < 0 || rows <= 0) return;   // the whole block: a padding request, or one that brings nothing
    const int dim_pad = P * R;
    float* sq = lds;                     // [TB][dim_pad]
    float* sk = sq + TB * dim_pad;       // [TB][dim_pad]
    float* sa = sk + TB * dim_pad;       // [TB][dim_pad] decays
    float* sv = sa + TB * dim_pad;       // [TB][VT]
    float* sg = sv + TB * VT;            // [TB][VT] gain times silu of the gate
    float* part = sg + TB * VT;          // [TB][P][VT]
    const int tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE, n_waves = blockDim.x / WAVE;
    const int p = tid / VT, jt = tid % VT, j0 = blockIdx.z * VT, j = j0 + jt;
    const bool works = p < P, column = works && j < vdim;
    const int i0 = p * R;
    float* S_at = state + (size_t)slot * state_stride + (size_t)head * dim * vdim;
    float S[R];
#pragma unroll
    for (int r = 0; r < R; r++) S[r] = column && i0 + r < dim ? S_at[(size_t)(i0 + r) * vdim + j] : 0.0f;
    for (int t0 = 0; t0 < rows; t0 += TB) {
        const int n_valid = min(TB, rows - t0);
        // an element of the values and one of the channels a thread: all of an element's loads are under way before the first is used
        for (int e = tid; e < n_valid * max(dim_pad, VT); e += blockDim.x) {
            const bool is_value = e < n_valid * VT, is_channel = e < n_valid * dim_pad;
            float value = 0.0f, gate = 0.0f, gain = 0.0f;
            if (is_value) {
                const int t = e / VT, c = min(j0 + e % VT, vdim - 1);
                const float* row = op.rows + (size_t)(first_row + t0 + t) * op.stride + head * vdim + c;
                value = row[op.v_at];
                if (NORMS) gate = row[op.g_at], gain = op.gain[c];
            }
            if (is_channel) {
                const int t = e / dim_pad, i = e % dim_pad, channel = head * dim + min(i, dim - 1);
                const float* row = op.rows + (size_t)(first_row + t0 + t) * op.stride;
                const float qv = row[op.q_at + channel] * op.q_scale, kv = row[op.k_at + channel];
                float z = op.bias[channel];
                const float* low = row + op.low_at;
                const float* up = op.up + channel;
#pragma unroll 16
                for (int r = 0; r < op.rank; r++) z = __builtin_fmaf(low[r], up[(size_t)r * n_heads * dim], z);
                const bool counts = i < dim;
                sq[e] = counts ? qv : 0.0f;
                sk[e] = counts ? kv : 0.0f;
                sa[e] = counts ? exp2_of(log2_decay(z, op.inverse_tau)) : 0.0f;
            }
            if (is_value) {
                sv[e] = j0 + e % VT < vdim ? value : 0.0f;
                if (NORMS) sg[e] = gain * silu_of(gate);
            }
        }
        __syncthreads();
        if (works) {
            for (int t = 0; t < n_valid; t++) {
                const float vv = sv[t * VT + jt];
                const float *at = sa + t * dim_pad + i0, *kt = sk + t * dim_pad + i0, *qt = sq + t * dim_pad + i0;
                float sum = 0.0f;
#pragma unroll
                for (int r = 0; r < R; r++) {
                    S[r] = __builtin_fmaf(at[r], S[r], kt[r] * vv);
                    sum = __builtin_fmaf(S[r], qt[r], sum);
                }
                part[(t * P + p) * VT + jt] = sum;
            }
        }
        __syncthreads();
        if (NORMS) {
            for (int t = wave; t < n_valid; t += n_waves) {   // VT <= 128: two columns a lane
                float o[2], squares = 0.0f;
#pragma unroll
                for (int u = 0; u < 2; u++) {
                    const int c = lane + u * WAVE;
                    o[u] = 0.0f;
                    if (c < vdim)
                        for (int pp = 0; pp < P; pp++) o[u] += part[(t * P + pp) * VT + c];
                    squares += o[u] * o[u];
                }
                const float factor = 1.0f / sqrtf(wave_total(squares) / (float)vdim + op.eps);
#pragma unroll
                for (int u = 0; u < 2; u++) {
                    const int c = lane + u * WAVE;
                    if (c < vdim) out[(size_t)(first_row + t0 + t) * n_heads * vdim + head * vdim + c] = from_float<T>(o[u] * factor * sg[t * VT + c]);
                }
            }
        } else {
            for (int e = tid; e < n_valid * VT; e += blockDim.x) {
                const int t = e / VT, c = e % VT;
                if (j0 + c >= vdim) continue;
                float sum = 0.0f;
                for (int pp = 0; pp < P; pp++) sum += part[(t * P + pp) * VT + c];
                sums[(size_t)(first_row + t0 + t) * n_heads * vdim + head * vdim + j0 + c] = sum;
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int r = 0; r < R; r++)
        if (column && i0 + r < dim) S_at[(size_t)(i0 + r) * vdim + j] = S[r];
}

struct Plan {
    int R, P, VT, TB, threads, tiles, norms;
    size_t lds_bytes;
};

// How a head of dim x vdim is laid over a block: all value columns where there are at most 128 of them and a thread then holds at most 32 rows
// of S (the block can norm), else tiles of up to 64 columns; as many parts along dim as 512 threads allow.
bool plan_for(int dim, int vdim, Plan& plan) {
    auto rows_of = [&](int columns) {
        int parts = THREADS / columns;
        if (parts > dim) parts = dim;
        int R = 1;
        while (R * parts < dim) R *= 2;
        return R;
    };
    plan.norms = vdim <= 128 && rows_of(vdim) <= 32;
    plan.VT = plan.norms || vdim <= 64 ? vdim : 64;
    plan.R = rows_of(plan.VT);
    if (plan.R > 64) return false;
    plan.tiles = ceil_div(vdim, plan.VT);
    plan.P = ceil_div(dim, plan.R);
    plan.threads = ceil_div(plan.P * plan.VT, 64) * 64;
    for (plan.TB = 8;; plan.TB /= 2) {
        plan.lds_bytes = (size_t)plan.TB * (3 * plan.P * plan.R + 2 * plan.VT + plan.P * plan.VT) * sizeof(float);
        if (plan.lds_bytes <= 60 * 1024 || plan.TB == 1) break;
    }
    return plan.lds_bytes <= 64 * 1024;
}

// ---- chunk by chunk -----------------------------------------------------------------------------------------------------------------
// Inside a chunk of L rows that starts from the state S0, with b_t[i] the sum of channel i's log decays up to and with row t:
//     o_t = (q_t 2^(b_t))^T S0 + sum_{s <= t} [sum_i q_t[i] k_s[i] 2^(b_t[i] - b_s[i])] v_s
// and the state behind it is diag(2^B) S0 + U with U = sum_s (k_s 2^(B - b_s)) v_s^T, B the whole chunk's sums. Three kernels: (1) every
// chunk's U and 2^B, all chunks at once; (2) per (request, head) the chunks in order, each U replaced by the state at its chunk's start,
// and the request's slot moved on; (3) every chunk's outputs, all chunks at once.
// 2^(b_t - b_s) is split over stretches of 16 rows: with the decays from the start of t's stretch to t, from s to the end of s's stretch, and
// over the whole stretches between, all factors are at most 1. Inside one stretch it is 2^(c_t) 2^(-c_s), c counted from the stretch's
// start, as long as no channel of the chunk fades by more than 2^-32 within a stretch; else that chunk takes these pairs one by one.
// Scratch: a record of dim * vdim + dim floats per (chunk, head); chunk c of request r whose first row in the batch is f has record f / L + r.
constexpr float LEAST_STRETCH = -32.0f;

template <int L, int DPT>
struct Chunk {
    static constexpr int DP = 16 * DPT, NS = L / SUB;   // the head's key channels filled up to sixteens; stretches of a chunk
    static constexpr int RPW = L / WAVES, CB = (DP + WAVE - 1) / WAVE;
    static_assert(DP * NS <= THREADS, "a thread takes a channel of a stretch");
};

__device__ __forceinline__ size_t record_of(int first_row, int chunk_rows, int request) { return (size_t)(first_row / chunk_rows + request); }
__device__ __forceinline__ f32x4 multiply_add(float a, float b, f32x4 sums) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, sums, 0, 0, 0); }

// What a thread needs of 16 of the decays' rank, asked for at once (from clamped places), early in a kernel.
template <int L, int DPT>
struct DecayPiece {
    using C = Chunk<L, DPT>;
    static constexpr int LOWS = L * 16 / THREADS;
    float w[C::CB][16], low[LOWS];
    __device__ __forceinline__ void ask(const MemoryRows& op, int chunk_first, int n_valid, int head, int n_heads, int r0) {
        const int tid = threadIdx.x, lane = tid % WAVE, columns = n_heads * op.dim;
#pragma unroll
        for (int u = 0; u < LOWS; u++) {
            const int e = tid + u * THREADS, r = r0 + e % 16;
            low[u] = op.rows[(size_t)(chunk_first + min(e / 16, n_valid - 1)) * op.stride + op.low_at + min(r, op.rank - 1)];
            if (r >= op.rank) low[u] = 0.0f;
        }
#pragma unroll
        for (int cb = 0; cb < C::CB; cb++)
#pragma unroll
            for (int r = 0; r < 16; r++) w[cb][r] = op.up[(size_t)min(r0 + r, op.rank - 1) * columns + head * op.dim + min(cb * WAVE + lane, op.dim - 1)];
    }
};

// The log decays of a chunk's rows for one head into la[s * la_stride + i] (0 beyond n_valid rows and dim channels); `low` [L][16] holds 16 of
// the rank at a time, `piece` brings the first. A lane a channel, a wave every eighth row. Ends with a barrier.
template <int L, int DPT>
__device__ __forceinline__ void chunk_decays(const MemoryRows& op, DecayPiece<L, DPT>& piece, int chunk_first, int n_valid, int head, int n_heads, float* la, int la_stride,
                                             float* low) {
    using C = Chunk<L, DPT>;
    const int tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE;
    float z[C::CB][C::RPW];
#pragma unroll
    for (int cb = 0; cb < C::CB; cb++) {
        const float bias = op.bias[head * op.dim + min(cb * WAVE + lane, op.dim - 1)];
#pragma unroll
        for (int u = 0; u < C::RPW; u++) z[cb][u] = bias;
    }
    for (int r0 = 0; r0 < op.rank; r0 += 16) {
        if (r0 > 0) {
            piece.ask(op, chunk_first, n_valid, head, n_heads, r0);
            __syncthreads();
        }
#pragma unroll
        for (int u = 0; u < DecayPiece<L, DPT>::LOWS; u++) low[tid + u * THREADS] = piece.low[u];
        __syncthreads();
#pragma unroll
        for (int u = 0; u < C::RPW; u++) {
            const f32x4* row = reinterpret_cast<const f32x4*>(low + (wave + u * WAVES) * 16);
#pragma unroll
            for (int r4 = 0; r4 < 4; r4++) {
                const f32x4 four = row[r4];
#pragma unroll
                for (int cb = 0; cb < C::CB; cb++)
#pragma unroll
                    for (int e = 0; e < 4; e++) z[cb][u] = __builtin_fmaf(four[e], piece.w[cb][r4 * 4 + e], z[cb][u]);
            }
        }
    }
#pragma unroll
    for (int cb = 0; cb < C::CB; cb++) {
        const int i = cb * WAVE + lane;
        if (i >= C::DP) continue;
#pragma unroll
        for (int u = 0; u < C::RPW; u++) {
            const int s = wave + u * WAVES;
            la[s * la_stride + i] = s < n_valid && i < op.dim ? log2_decay(z[cb][u], op.inverse_tau) : 0.0f;
        }
    }
    __syncthreads();
}

constexpr int SUM_TILE = 64;   // value columns a block of the first kernel takes

template <int L, int DPT>
__global__ __launch_bounds__(THREADS) void memory_sums_kernel(MemoryRows op, float* __restrict__ records, int tiles) {
    using C = Chunk<L, DPT>;
    constexpr int DP = C::DP, KS = DP % 32 == 0 ? DP + 16 : DP, VS = SUM_TILE + 16;   // rows two apart on the same banks, neighbours on others
    extern __shared__ __align__(16) float lds[];
    float* K = lds;                  // [L][KS] log decays, then the faded keys
    float* V = K + L * KS;           // [L][VS]
    float* low = V + L * VS;         // [L][16]
    float* total = low + L * 16;     // [NS][DP] the stretches' log decays
    const int request = blockIdx.x, head = blockIdx.y, n_heads = gridDim.y, chunk = blockIdx.z / tiles, tile = blockIdx.z % tiles;
    const int first_row = op.q_starts[request], rows = op.q_starts[request + 1] - first_row;
    if (op.state_slots[request] < 0 || chunk * L >= rows) return;
    const int n_valid = min(L, rows - chunk * L), chunk_first = first_row + chunk * L, dim = op.dim, vdim = op.vdim;
    const int tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE;
    float* record = records + (record_of(chunk_first, L, request) * n_heads + head) * ((size_t)dim * vdim + dim);
    // a thread's keys (channel i of the 16 rows of stretch n) and values are asked for before the decays are made
    const int i = tid % DP, n = tid / DP;
    const bool works = n < C::NS;
    float keys[SUB];
#pragma unroll
    for (int s = 0; s < SUB; s++) {
        const int row = min((works ? n : 0) * SUB + s, n_valid - 1);
        keys[s] = op.rows[(size_t)(chunk_first + row) * op.stride + op.k_at + head * dim + min(i, dim - 1)];
    }
    constexpr int VPER = L * SUM_TILE / THREADS;
    const int column = tile * SUM_TILE + lane;
    float values[VPER];
#pragma unroll
    for (int u = 0; u < VPER; u++)
        values[u] = op.rows[(size_t)(chunk_first + min(wave + u * WAVES, n_valid - 1)) * op.stride + op.v_at + head * vdim + min(column, vdim - 1)];
    DecayPiece<L, DPT> piece;
    piece.ask(op, chunk_first, n_valid, head, n_heads, 0);
    chunk_decays<L, DPT>(op, piece, chunk_first, n_valid, head, n_heads, K, KS, low);
#pragma unroll
    for (int u = 0; u < VPER; u++) V[(wave + u * WAVES) * VS + lane] = wave + u * WAVES < n_valid && column < vdim ? values[u] : 0.0f;
    float la[SUB];
    if (works) {
        float sum = 0.0f;
#pragma unroll
        for (int s = 0; s < SUB; s++) {
            la[s] = K[(n * SUB + s) * KS + i];
            sum += la[s];
        }
        total[n * DP + i] = sum;
    }
    __syncthreads();
    if (works) {
        float later = 0.0f;   // the decays behind the row, up to the chunk's end
        for (int m = n + 1; m < C::NS; m++) later += total[m * DP + i];
#pragma unroll
        for (int s = SUB - 1; s >= 0; s--) {
            K[(n * SUB + s) * KS + i] = n * SUB + s < n_valid && i < dim ? keys[s] * exp2_of(later) : 0.0f;
            later += la[s];
        }
        if (n == 0 && tile == 0 && i < dim) record[(size_t)dim * vdim + i] = exp2_of(later);
    }
    __syncthreads();
    // U = (faded keys)^T V: a wave 16 columns j, every second tile of 16 channels i
    const int l16 = lane % 16, quad = lane / 16, jt = wave % 4;
    for (int it = wave / 4; it < DPT; it += 2) {
        f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int step = 0; step < L / 4; step++) {   // (rows beyond the chunk's are zeros)
            const int s = step * 4 + quad;
            acc = multiply_add(K[s * KS + it * 16 + l16], V[s * VS + jt * 16 + l16], acc);
        }
        const int j = tile * SUM_TILE + jt * 16 + l16;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int channel = it * 16 + quad * 4 + r;
            if (channel < dim && j < vdim) record[(size_t)channel * vdim + j] = acc[r];
        }
    }
}

// The chunks of one (request, head) in order, 1,024 elements of the matrix a block (four a thread); eight chunks asked for at a time.
__global__ __launch_bounds__(256) void memory_scan_kernel(const int* __restrict__ q_starts, const int* __restrict__ state_slots, float* __restrict__ records,
                                                          float* __restrict__ state, long long state_stride, int dim, int vdim, int chunk_rows) {
    constexpr int PER = 4, AHEAD = 8;
    const int request = blockIdx.x, head = blockIdx.y, n_heads = gridDim.y, tid = threadIdx.x;
    const int slot = state_slots[request];
    const int first_row = q_starts[request], rows = q_starts[request + 1] - first_row;
    if (slot < 0 || rows <= 0) return;
    const int n_chunks = (rows + chunk_rows - 1) / chunk_rows, elements = dim * vdim, base = blockIdx.z * 256 * PER;
    float* S_at = state + (size_t)slot * state_stride + (size_t)head * elements;
    auto record = [&](int c) { return records + (record_of(first_row + c * chunk_rows, chunk_rows, request) * n_heads + head) * ((size_t)elements + dim); };
    float S[PER];
    int at[PER], channel[PER];
#pragma unroll
    for (int u = 0; u < PER; u++) {
        at[u] = min(base + u * 256 + tid, elements - 1);
        channel[u] = elements + at[u] / vdim;
        S[u] = S_at[at[u]];
    }
    for (int c0 = 0; c0 < n_chunks; c0 += AHEAD) {
        float sums[AHEAD][PER], keeps[AHEAD][PER];
#pragma unroll
        for (int d = 0; d < AHEAD; d++) {
            const float* from = record(min(c0 + d, n_chunks - 1));
#pragma unroll
            for (int u = 0; u < PER; u++) sums[d][u] = from[at[u]], keeps[d][u] = from[channel[u]];
        }
#pragma unroll
        for (int d = 0; d < AHEAD; d++) {
            if (c0 + d >= n_chunks) break;
            float* to = record(c0 + d);
#pragma unroll
            for (int u = 0; u < PER; u++) {
                if (base + u * 256 + tid < elements) to[at[u]] = S[u];
                S[u] = __builtin_fmaf(keeps[d][u], S[u], sums[d][u]);
            }
        }
    }
#pragma unroll
    for (int u = 0; u < PER; u++)
        if (base + u * 256 + tid < elements) S_at[at[u]] = S[u];
}

template <int L, int DPT>
struct OutputLds {
    using C = Chunk<L, DPT>;
    static constexpr int QS = C::DP + 4, AS = L + 4;                  // rows of whole 16-byte pieces, four banks apart
    static constexpr int Q = 0, K = Q + L * QS, D = K + L * QS, A = D + L * QS, TOTAL = A + L * AS;
    static constexpr int FROM_START = TOTAL + C::NS * C::DP;          // [NS][DP]: the decay from the chunk's start to the stretch's
    static constexpr int BETWEEN = FROM_START + C::NS * C::DP;        // [NS][NS][DP] (first, second): the stretches between the two
    static constexpr int SQUARES = BETWEEN + (C::NS > 2 ? C::NS * C::NS * C::DP : 0);
    static constexpr int FACTOR = SQUARES + WAVES * L, V = FACTOR + L;
    static int value_stride(int vdim) { return ceil_div(vdim, 16) % 2 == 0 ? ceil_div(vdim, 16) * 16 + 16 : ceil_div(vdim, 16) * 16; }
};

template <typename T, int L, int DPT>
__global__ __launch_bounds__(THREADS) void memory_output_kernel(MemoryRows op, const float* __restrict__ records, T* __restrict__ out, int v_at_lds, int VS) {
    using C = Chunk<L, DPT>;
    using Lds = OutputLds<L, DPT>;
    constexpr int DP = C::DP, NS = C::NS, QS = Lds::QS, AS = Lds::AS;
    extern __shared__ __align__(16) float lds[];
    float *Q = lds + Lds::Q, *K = lds + Lds::K, *D = lds + Lds::D, *A = lds + Lds::A, *total = lds + Lds::TOTAL, *from_start = lds + Lds::FROM_START,
          *between = lds + Lds::BETWEEN, *squares_lds = lds + Lds::SQUARES, *factor_lds = lds + Lds::FACTOR, *V = lds + v_at_lds;
    const bool v_early = v_at_lds >= Lds::V;   // the values have a place of their own; else they take the keys' and the decays' when those are through
    const int request = blockIdx.x, head = blockIdx.y, n_heads = gridDim.y, chunk = blockIdx.z;
    const int first_row = op.q_starts[request], rows = op.q_starts[request + 1] - first_row;
    if (op.state_slots[request] < 0 || chunk * L >= rows) return;
    const int n_valid = min(L, rows - chunk * L), chunk_first = first_row + chunk * L, dim = op.dim, vdim = op.vdim;
    const int tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE, l16 = lane % 16, quad = lane / 16;
    const float* record = records + (record_of(chunk_first, L, request) * n_heads + head) * ((size_t)dim * vdim + dim);
    const int value_tiles = ceil_div(vdim, 16);

    // Everything the block reads from memory is asked for here, from clamped places, and waits in registers for its turn: queries and keys, the
    // decays' operands, the values of the first 128 columns, the state the chunk starts from and the gates (in the order of their use).
    constexpr int QPER = L * DP / THREADS, VROWS = L / WAVES, VBLOCKS = 2, ITEMS = 2;
    float q_mine[QPER], k_mine[QPER];
#pragma unroll
    for (int u = 0; u < QPER; u++) {
        const int e = tid + u * THREADS, s = e / DP, i = e % DP;
        const float* row = op.rows + (size_t)(chunk_first + min(s, n_valid - 1)) * op.stride + head * dim + min(i, dim - 1);
        q_mine[u] = row[op.q_at], k_mine[u] = row[op.k_at];
    }
    DecayPiece<L, DPT> piece;
    piece.ask(op, chunk_first, n_valid, head, n_heads, 0);
    float v_mine[VBLOCKS][VROWS];   // column block * 64 + lane of every eighth row
    auto ask_values = [&](int block, float (&mine)[VROWS]) {
#pragma unroll
        for (int u = 0; u < VROWS; u++)
            mine[u] = op.rows[(size_t)(chunk_first + min(wave + u * WAVES, n_valid - 1)) * op.stride + op.v_at + head * vdim + min(block * WAVE + lane, vdim - 1)];
    };
    auto leave_values = [&](int block, const float (&mine)[VROWS]) {
        const int c = block * WAVE + lane;
        if (c >= value_tiles * 16) return;
#pragma unroll
        for (int u = 0; u < VROWS; u++) V[(wave + u * WAVES) * VS + c] = wave + u * WAVES < n_valid && c < vdim ? mine[u] : 0.0f;
    };
#pragma unroll
    for (int block = 0; block < VBLOCKS; block++) ask_values(block, v_mine[block]);
    auto load_values = [&]() {
#pragma unroll
        for (int block = 0; block < VBLOCKS; block++) leave_values(block, v_mine[block]);
        for (int block = VBLOCKS; block * WAVE < vdim; block++) {
            float more[VROWS];
            ask_values(block, more);
            leave_values(block, more);
        }
    };
    // outputs: 16 value columns a wave (up to ITEMS such tiles), all rows or, where there are few columns, half of them
    const bool halves = value_tiles <= WAVES / 2 && NS >= 2;
    constexpr int EARLY = DPT <= 4 ? ITEMS : DPT * L <= 256 ? 1 : 0;   // tiles whose states wait in registers (more of them would not fit)
    auto ask_state = [&](int j, float (&mine)[DPT][4]) {
#pragma unroll
        for (int step = 0; step < DPT; step++)
#pragma unroll
            for (int e = 0; e < 4; e++) mine[step][e] = record[(size_t)min(step * 16 + quad * 4 + e, dim - 1) * vdim + j];
    };
    float start[ITEMS][DPT][4], gates[ITEMS][NS][4], gain[ITEMS];
#pragma unroll
    for (int u = 0; u < ITEMS; u++) {
        const int item = wave + u * WAVES, jt = halves ? item / 2 : item, j = min(jt * 16 + l16, vdim - 1);
        if (jt >= value_tiles) continue;
        if (u < EARLY) ask_state(j, start[u]);
#pragma unroll
        for (int t = 0; t < NS; t++)
#pragma unroll
            for (int r = 0; r < 4; r++)
                gates[u][t][r] = op.rows[(size_t)(chunk_first + min(t * SUB + quad * 4 + r, n_valid - 1)) * op.stride + op.g_at + head * vdim + j];
        gain[u] = op.gain[j];
    }
#pragma unroll
    for (int u = 0; u < QPER; u++) {
        const int e = tid + u * THREADS, s = e / DP, i = e % DP;
        const bool counts = s < n_valid && i < dim;
        Q[s * QS + i] = counts ? q_mine[u] * op.q_scale : 0.0f;
        K[s * QS + i] = counts ? k_mine[u] : 0.0f;
    }
    for (int e = tid; e < WAVES * L; e += THREADS) squares_lds[e] = 0.0f;
    chunk_decays<L, DPT>(op, piece, chunk_first, n_valid, head, n_heads, D, QS, A);
    if (v_early) load_values();

    // ---- decays inside the stretches: thread (channel i, stretch n) ----
    const int i = tid % DP, n = tid / DP;
    const bool works = n < NS;
    float la[SUB], whole = 0.0f;
#pragma unroll
    for (int s = 0; s < SUB; s++) {
        la[s] = works ? D[(n * SUB + s) * QS + i] : 0.0f;
        whole += la[s];
    }
    if (works) total[n * DP + i] = whole;
    const bool mild = __syncthreads_and(whole >= LEAST_STRETCH);
    if (!mild) {   // pairs inside the stretches one by one, from exact differences of logarithms
        float c = 0.0f;
#pragma unroll
        for (int s = 0; s < SUB; s++) {
            c += la[s];
            if (works) D[(n * SUB + s) * QS + i] = c;
        }
        __syncthreads();
        for (int e = tid; e < NS * SUB * SUB; e += THREADS) {
            const int t = e / SUB, s = t / SUB * SUB + e % SUB;
            float sum = 0.0f;
            if (s <= t)
                for (int d = 0; d < DP; d++) sum += Q[t * QS + d] * K[s * QS + d] * exp2_of(D[t * QS + d] - D[s * QS + d]);
            A[t * AS + s] = sum;
        }
        __syncthreads();
    }
    if (works) {
        float c = 0.0f;
#pragma unroll
        for (int s = 0; s < SUB; s++) {   // queries faded from the stretch's start; keys grown back to it
            c += la[s];
            const int at = (n * SUB + s) * QS + i;
            if (mild) D[at] = K[at] * exp2_of(-c);
            Q[at] *= exp2_of(c);
        }
        float behind = 0.0f;
#pragma unroll
        for (int s = SUB - 1; s >= 0; s--) {   // keys faded to the stretch's end
            K[(n * SUB + s) * QS + i] *= exp2_of(behind);
            behind += la[s];
        }
        float before = 0.0f;
        for (int m = 0; m < n; m++) before += total[m * DP + i];
        from_start[n * DP + i] = exp2_of(before);
        if constexpr (NS > 2) {
            float gap = 0.0f;
            for (int m = n - 1; m >= 0; m--) {
                between[(m * NS + n) * DP + i] = exp2_of(gap);
                gap += total[m * DP + i];
            }
        }
    }
    __syncthreads();

    // ---- scores: tiles of 16 queries x 16 keys, a wave each ----
    for (int item = wave; item < NS * (NS + 1) / 2; item += WAVES) {
        int query = 0, key = item;
        while (key > query) key -= ++query;   // item = query (query + 1) / 2 + key
        if (!mild && query == key) continue;
        f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
        const float* q_row = Q + (query * SUB + l16) * QS + quad * 4;
        const float* k_row = (query == key ? D : K) + (key * SUB + l16) * QS + quad * 4;
        const bool gap = NS > 2 && query - key >= 2;
#pragma unroll
        for (int step = 0; step < DPT; step++) {
            const f32x4 qs = *reinterpret_cast<const f32x4*>(q_row + step * 16);
            f32x4 ks = *reinterpret_cast<const f32x4*>(k_row + step * 16);
            if (gap) {
                const f32x4 fade = *reinterpret_cast<const f32x4*>(between + (key * NS + query) * DP + step * 16 + quad * 4);
#pragma unroll
                for (int e = 0; e < 4; e++) ks[e] *= fade[e];
            }
#pragma unroll
            for (int e = 0; e < 4; e++) acc = multiply_add(qs[e], ks[e], acc);
        }
#pragma unroll
        for (int r = 0; r < 4; r++) A[(query * SUB + quad * 4 + r) * AS + key * SUB + l16] = query > key || l16 <= quad * 4 + r ? acc[r] : 0.0f;
    }
    __syncthreads();
    if (!v_early) {
        load_values();
        __syncthreads();
    }

    // ---- outputs ----
    f32x4 acc[ITEMS][NS];
#pragma unroll
    for (int u = 0; u < ITEMS; u++) {
#pragma unroll
        for (int t = 0; t < NS; t++) acc[u][t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
        const int item = wave + u * WAVES, jt = halves ? item / 2 : item;
        if (jt >= value_tiles) continue;
        const int t_first = halves && item % 2 ? NS / 2 : 0, t_last = halves && item % 2 == 0 ? NS / 2 : NS;
        if (u >= EARLY) ask_state(min(jt * 16 + l16, vdim - 1), start[u]);
#pragma unroll
        for (int block = 0; block < NS; block++) {
            if (block >= t_last) continue;
            float values[4];
#pragma unroll
            for (int e = 0; e < 4; e++) values[e] = V[(block * SUB + quad * 4 + e) * VS + jt * 16 + l16];
#pragma unroll
            for (int t = block; t < NS; t++) {
                if (t < t_first || t >= t_last) continue;
                const f32x4 scores = *reinterpret_cast<const f32x4*>(A + (t * SUB + l16) * AS + block * SUB + quad * 4);
#pragma unroll
                for (int e = 0; e < 4; e++) acc[u][t] = multiply_add(scores[e], values[e], acc[u][t]);
            }
        }
#pragma unroll
        for (int t = 0; t < NS; t++) {
            if (t < t_first || t >= t_last) continue;
#pragma unroll
            for (int step = 0; step < DPT; step++) {
                f32x4 qs = *reinterpret_cast<const f32x4*>(Q + (t * SUB + l16) * QS + step * 16 + quad * 4);
                if (t > 0) {
                    const f32x4 fade = *reinterpret_cast<const f32x4*>(from_start + t * DP + step * 16 + quad * 4);
#pragma unroll
                    for (int e = 0; e < 4; e++) qs[e] *= fade[e];
                }
#pragma unroll
                for (int e = 0; e < 4; e++) acc[u][t] = multiply_add(qs[e], start[u][step][e], acc[u][t]);
            }
        }
        // (a lane's sums: rows t * 16 + 4 * quad + r of column jt * 16 + l16)
#pragma unroll
        for (int t = 0; t < NS; t++) {
            if (t < t_first || t >= t_last) continue;
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const float mine = jt * 16 + l16 < vdim ? acc[u][t][r] : 0.0f;
                const float sum = lanes_sum<16>(mine * mine);
                if (l16 == 0) squares_lds[wave * L + t * SUB + quad * 4 + r] += sum;   // this wave's own place
            }
        }
    }
    __syncthreads();
    if (tid < L) {
        float sum = 0.0f;
        for (int w = 0; w < WAVES; w++) sum += squares_lds[w * L + tid];
        factor_lds[tid] = 1.0f / sqrtf(sum / (float)vdim + op.eps);
    }
    __syncthreads();
#pragma unroll
    for (int u = 0; u < ITEMS; u++) {
        const int item = wave + u * WAVES, jt = halves ? item / 2 : item, j = jt * 16 + l16;
        if (j >= vdim) continue;
        const int t_first = halves && item % 2 ? NS / 2 : 0, t_last = halves && item % 2 == 0 ? NS / 2 : NS;
#pragma unroll
        for (int t = 0; t < NS; t++) {
            if (t < t_first || t >= t_last) continue;
#pragma unroll
            for (int r = 0; r < 4; r++) {
                const int row = t * SUB + quad * 4 + r;
                if (row < n_valid) out[(size_t)(chunk_first + row) * n_heads * vdim + head * vdim + j] = from_float<T>(acc[u][t][r] * factor_lds[row] * gain[u] * silu_of(gates[u][t][r]));
            }
        }
    }
}

constexpr size_t LDS_MOST = 156 * 1024;

template <int L, int DPT>
size_t output_lds_floats(int vdim, int& v_at, int& v_stride) {
    using Lds = OutputLds<L, DPT>;
    v_stride = Lds::value_stride(vdim);
    const int values = L * v_stride, freed = 2 * L * Lds::QS;   // keys and decays lie behind each other
    v_at = Lds::V;
    if (((size_t)Lds::V + values) * sizeof(float) <= LDS_MOST || values > freed) return (size_t)Lds::V + values;
    v_at = Lds::K;
    return Lds::V;
}

// What fits a block's LDS with all of a head's values.
int chunk_rows_for(int dim, int vdim) { return dim <= 64 || (dim <= 128 && vdim <= 128) ? 64 : 32; }

template <typename T, int L, int DPT>
int launch_chunks(const MemoryRows& op, float* state, long long state_stride, T* out, int n_requests, int n_heads, int chunks, float* records, hipStream_t stream) {
    using C = Chunk<L, DPT>;
    constexpr int KS = C::DP % 32 == 0 ? C::DP + 16 : C::DP;
    constexpr size_t sums_bytes = (L * (KS + SUM_TILE + 16) + L * 16 + C::NS * C::DP) * sizeof(float);
    int v_at, v_stride;
    const size_t output_bytes = output_lds_floats<L, DPT>(op.vdim, v_at, v_stride) * sizeof(float);
    MLLM_REQUIRE(output_bytes <= LDS_MOST, "channel_memory: heads of %d x %d do not fit a block", op.dim, op.vdim);
    static bool raised = false;   // per instantiation: the limit on dynamic LDS is a property of the kernel
    if (!raised) {
        MLLM_REQUIRE(hipFuncSetAttribute((const void*)memory_sums_kernel<L, DPT>, hipFuncAttributeMaxDynamicSharedMemorySize, sums_bytes) == hipSuccess &&
                         hipFuncSetAttribute((const void*)memory_output_kernel<T, L, DPT>, hipFuncAttributeMaxDynamicSharedMemorySize, LDS_MOST) == hipSuccess,
                     "channel_memory: the kernels cannot have the LDS they need");
        raised = true;
    }
    const int tiles = ceil_div(op.vdim, SUM_TILE);
    MLLM_REQUIRE((long long)chunks * tiles <= 65535, "channel_memory: too many chunks for one launch");
    mllm_count_kernel(MLLM_K_CHANNEL_MEMORY);
    memory_sums_kernel<L, DPT><<<dim3(n_requests, n_heads, chunks * tiles), THREADS, sums_bytes, stream>>>(op, records, tiles);
    mllm_count_kernel(MLLM_K_CHANNEL_MEMORY);
    memory_scan_kernel<<<dim3(n_requests, n_heads, ceil_div(op.dim * op.vdim, 1024)), 256, 0, stream>>>(op.q_starts, op.state_slots, records, state, state_stride, op.dim, op.vdim, L);
    mllm_count_kernel(MLLM_K_CHANNEL_MEMORY);
    memory_output_kernel<T, L, DPT><<<dim3(n_requests, n_heads, chunks), THREADS, output_bytes, stream>>>(op, records, out, v_at, v_stride);
    return mllm_check_launch("channel_memory");
}

template <typename T>
int launch_rows(const MemoryRows& op, float* state, long long state_stride, T* out, float* sums, int n_requests, int n_heads, const Plan& plan, hipStream_t stream) {
    const dim3 grid(n_requests, n_heads, plan.tiles);
    mllm_count_kernel(MLLM_K_CHANNEL_MEMORY);
#define ROWS(R)                                                                                                                                             \
    do {                                                                                                                                                    \
        if (plan.norms) memory_rows_kernel<T, (R <= 32 ? R : 32), true><<<grid, plan.threads, plan.lds_bytes, stream>>>(op, state, state_stride, out, sums, plan.P, plan.VT, plan.TB); \
        else memory_rows_kernel<T, R, false><<<grid, plan.threads, plan.lds_bytes, stream>>>(op, state, state_stride, out, sums, plan.P, plan.VT, plan.TB);  \
    } while (0)
    switch (plan.R) {
        case 1: ROWS(1); break;
        case 2: ROWS(2); break;
        case 4: ROWS(4); break;
        case 8: ROWS(8); break;
        case 16: ROWS(16); break;
        case 32: ROWS(32); break;
        default: ROWS(64); break;
    }
#undef ROWS
    return mllm_check_launch("channel_memory");
}

template <typename T>
int launch_memory(const MemoryRows& op, float* state, long long state_stride, T* out, float* sums, int n_requests, int n_heads, int longest, float* records,
                  int chunk_rows, hipStream_t stream) {
    if (chunk_rows) {
        const int chunks = ceil_div(longest, chunk_rows);
#define CHUNKS(L, DPT) return launch_chunks<T, L, DPT>(op, state, state_stride, out, n_requests, n_heads, chunks, records, stream)
        if (op.dim <= 32) CHUNKS(64, 2);
        if (op.dim <= 64) CHUNKS(64, 4);
        if (op.dim <= 96 && chunk_rows == 64) CHUNKS(64, 6);
        if (op.dim <= 128 && chunk_rows == 64) CHUNKS(64, 8);
        if (op.dim <= 96) CHUNKS(32, 6);
        if (op.dim <= 128) CHUNKS(32, 8);
        if (op.dim <= 192) CHUNKS(32, 12);
        CHUNKS(32, 16);
#undef CHUNKS
    }
    Plan plan;
    MLLM_REQUIRE(plan_for(op.dim, op.vdim, plan), "channel_memory: heads of %d x %d are larger than the kernel takes", op.dim, op.vdim);
    MLLM_REQUIRE(plan.norms || sums != nullptr, "channel_memory: heads of %d x %d need a place for their sums", op.dim, op.vdim);
    return launch_rows<T>(op, state, state_stride, out, sums, n_requests, n_heads, plan, stream);
}

}  // namespace

// The rows a chunk of long portions holds for heads of these sizes (0: only row by row).
MLLM_API int mllm_channel_memory_chunk_rows(int dim, int vdim) { return dim >= 1 && dim <= 256 && vdim >= 1 && vdim <= 256 ? chunk_rows_for(dim, vdim) : 0; }

// 1 if the row by row kernel norms and gates by itself, 0 if it leaves its sums for a norm behind it, -1 if it does not take such heads.
MLLM_API int mllm_channel_memory_norms(int dim, int vdim) {
    Plan plan;
    return dim > 0 && vdim > 0 && plan_for(dim, vdim, plan) ? plan.norms : -1;
}

// rows: [n_rows, stride] float32; chunk_rows 0: row by row, else the number above, with records for (n_rows / chunk_rows + n_requests + 1) chunks
// of n_heads * (dim * vdim + dim) floats. longest: the longest portion, or a bound on it. sums: see mllm_channel_memory_norms.
MLLM_API int mllm_channel_memory(const float* rows, int stride, int q_at, int k_at, int v_at, int g_at, int low_at, const float* up, const float* bias, int rank,
                                 float inverse_tau, float q_scale, const float* gain, float eps, float* state, long long state_stride, const int* q_starts,
                                 const int* state_slots, void* out, float* sums, int n_rows, int n_requests, int n_heads, int dim, int vdim, int longest,
                                 float* records, long long record_floats, int chunk_rows, int dtype, hipStream_t stream) {
    MLLM_REQUIRE(n_rows >= 0 && n_requests >= 0 && n_heads > 0 && dim > 0 && vdim > 0 && rank > 0 && longest >= 0, "channel_memory: bad sizes");
    const int qw = n_heads * dim, vw = n_heads * vdim;
    MLLM_REQUIRE(q_at >= 0 && q_at + qw <= stride && k_at >= 0 && k_at + qw <= stride && v_at >= 0 && v_at + vw <= stride && g_at >= 0 && g_at + vw <= stride && low_at >= 0 &&
                     low_at + rank <= stride,
                 "channel_memory: columns lie beyond the rows");
    MLLM_REQUIRE(rows && up && bias && gain && state && q_starts && state_slots && out && state_stride >= (long long)qw * vdim, "channel_memory: a missing operand, or a state that is too small");
    MLLM_REQUIRE(inverse_tau > 0.0f && eps > 0.0f && (dtype == MLLM_F32 || dtype == MLLM_BF16), "channel_memory: tau and eps must be positive, the result of a known type");
    MLLM_REQUIRE(n_heads <= 65535, "channel_memory: too many heads for one launch");
    if (chunk_rows) {
        MLLM_REQUIRE(chunk_rows == mllm_channel_memory_chunk_rows(dim, vdim), "channel_memory: chunks of %d rows for heads of %d x %d", chunk_rows, dim, vdim);
        MLLM_REQUIRE(records != nullptr && record_floats >= ((long long)n_rows / chunk_rows + n_requests + 1) * n_heads * ((long long)dim * vdim + dim),
                     "channel_memory: the records' memory is too small");
    }
    if (n_requests == 0 || n_rows == 0 || longest == 0) return 0;
    const MemoryRows op{rows, stride, q_at, k_at, v_at, g_at, low_at, up, bias, rank, inverse_tau, q_scale, gain, eps, q_starts, state_slots, dim, vdim};
    if (dtype == MLLM_F32) return launch_memory<float>(op, state, state_stride, (float*)out, sums, n_requests, n_heads, longest, records, chunk_rows, stream);
    return launch_memory<bf16_t>(op, state, state_stride, (bf16_t*)out, sums, n_requests, n_heads, longest, records, chunk_rows, stream);
}
