// The sum of a layer's branches with the stream and what the layer norms (or RMS norms) that read the sum next make of it, from one
// launch; and the cap of a model's logits.
#include "common.h"

#include <math.h>

namespace {

constexpr int JOIN_WAVES = 4;   // rows a block

struct JoinOperands {
    const float* x;                                       // the stream [rows, width]
    const float* a; int n_a; long long a_stride;          // a branch (null: none): [n_a, rows, width], partial products that are added up
    const float* a_bias;                                  // [width] or null
    const float* b; int n_b; long long b_stride;
    const float* b_bias;
    const float* vector;                                  // [width] or null: joins every row
    float* total;                                         // the sum (null: not written; then there is nothing but x)
    const float *gain_1, *offset_1, *gain_2, *offset_2;   // [width]; a null gain: no such norm; a null offset: none
    int centred, one_plus;
    float eps;
    int n_rows, width;
};

// A wave a row. A lane owns VEC neighbouring elements in each of CHUNKS pieces of the row; they stay in registers between the sum, the mean,
// the centred squares and the normed rows. What is absent is asked for nowhere (the same branches for all lanes); partial products are
// asked for two at a time behind the first loads.
template <typename T, int VEC, int CHUNKS>
__global__ __launch_bounds__(64 * JOIN_WAVES) void join_norms_kernel(JoinOperands op, T* __restrict__ rows_1, T* __restrict__ rows_2) {
    struct Piece {
        float v[VEC];
    };
    const int lane = threadIdx.x % WAVE;
    const int row = blockIdx.x * JOIN_WAVES + threadIdx.x / WAVE;
    if (row >= op.n_rows) return;
    const size_t at = (size_t)row * op.width;
    const int last = op.width - VEC;
    auto piece = [](const float* from) {
        Piece out;
        if constexpr (VEC == 4) {
            const f32x4 loaded = *reinterpret_cast<const f32x4*>(from);
#pragma unroll
            for (int e = 0; e < 4; e++) out.v[e] = loaded[e];
        } else {
            out.v[0] = *from;
        }
        return out;
    };
    auto place = [&](int c) { return min((c * WAVE + lane) * VEC, last); };   // beyond the row: its last piece, masked where it counts
    Piece sums[CHUNKS], gains_1[CHUNKS], offsets_1[CHUNKS], gains_2[CHUNKS], offsets_2[CHUNKS];
#pragma unroll
    for (int c = 0; c < CHUNKS; c++) sums[c] = piece(op.x + at + place(c));
    auto add = [&](const float* from) {
        Piece more[CHUNKS];
#pragma unroll
        for (int c = 0; c < CHUNKS; c++) more[c] = piece(from + place(c));
#pragma unroll
        for (int c = 0; c < CHUNKS; c++)
#pragma unroll
            for (int e = 0; e < VEC; e++) sums[c].v[e] += more[c].v[e];
    };
    auto add_two = [&](const float* from, const float* then) {
        Piece more[CHUNKS], again[CHUNKS];
#pragma unroll
        for (int c = 0; c < CHUNKS; c++) more[c] = piece(from + place(c)), again[c] = piece(then + place(c));
#pragma unroll
        for (int c = 0; c < CHUNKS; c++)
#pragma unroll
            for (int e = 0; e < VEC; e++) sums[c].v[e] += more[c].v[e] + again[c].v[e];
    };
    if (op.gain_1) {
#pragma unroll
        for (int c = 0; c < CHUNKS; c++) {
            gains_1[c] = piece(op.gain_1 + place(c));
            offsets_1[c] = piece((op.offset_1 ? op.offset_1 : op.gain_1) + place(c));
        }
    }
    if (op.gain_2) {
#pragma unroll
        for (int c = 0; c < CHUNKS; c++) {
            gains_2[c] = piece(op.gain_2 + place(c));
            offsets_2[c] = piece((op.offset_2 ? op.offset_2 : op.gain_2) + place(c));
        }
    }
    if (op.a && op.b) add_two(op.a + at, op.b + at);
    else if (op.a) add(op.a + at);
    else if (op.b) add(op.b + at);
    auto more_of = [&](const float* branch, int n, long long stride) {
        for (int p = 1; p < n; p += 2) {
            if (p + 1 < n) add_two(branch + (size_t)p * stride + at, branch + (size_t)(p + 1) * stride + at);
            else add(branch + (size_t)p * stride + at);
        }
    };
    if (op.a) more_of(op.a, op.n_a, op.a_stride);
    if (op.b) more_of(op.b, op.n_b, op.b_stride);
    if (op.a_bias) add(op.a_bias);
    if (op.b_bias) add(op.b_bias);
    if (op.vector) add(op.vector);
    if (op.total) {
#pragma unroll
        for (int c = 0; c < CHUNKS; c++) {
            const int d = (c * WAVE + lane) * VEC;
            if (d > last) continue;
            if constexpr (VEC == 4) *reinterpret_cast<f32x4*>(op.total + at + d) = f32x4{sums[c].v[0], sums[c].v[1], sums[c].v[2], sums[c].v[3]};
            else op.total[at + d] = sums[c].v[0];
        }
    }
    if (op.gain_1 == nullptr) return;
    float mean = 0.0f;
    if (op.centred) {
#pragma unroll
        for (int c = 0; c < CHUNKS; c++)
#pragma unroll
            for (int e = 0; e < VEC; e++) mean += (c * WAVE + lane) * VEC <= last ? sums[c].v[e] : 0.0f;
        mean = wave_total(mean) / (float)op.width;
    }
    float squares = 0.0f;
#pragma unroll
    for (int c = 0; c < CHUNKS; c++)
#pragma unroll
        for (int e = 0; e < VEC; e++) {
            sums[c].v[e] -= mean;
            squares += (c * WAVE + lane) * VEC <= last ? sums[c].v[e] * sums[c].v[e] : 0.0f;
        }
    const float factor = 1.0f / sqrtf(wave_total(squares) / (float)op.width + op.eps), plus = op.one_plus ? 1.0f : 0.0f;
    auto leave = [&](T* rows, const Piece (&gains)[CHUNKS], const Piece (&offsets)[CHUNKS], bool has_offset) {
#pragma unroll
        for (int c = 0; c < CHUNKS; c++) {
            const int d = (c * WAVE + lane) * VEC;
            if (d > last) continue;
            float made[VEC];
#pragma unroll
            for (int e = 0; e < VEC; e++) made[e] = sums[c].v[e] * factor * (plus + gains[c].v[e]) + (has_offset ? offsets[c].v[e] : 0.0f);
            if constexpr (VEC == 4 && sizeof(T) == 4) *reinterpret_cast<f32x4*>(rows + at + d) = f32x4{made[0], made[1], made[2], made[3]};
            else if constexpr (VEC == 4) *reinterpret_cast<bf16x4*>(rows + at + d) = bf16x4{from_float<T>(made[0]), from_float<T>(made[1]), from_float<T>(made[2]), from_float<T>(made[3])};
            else rows[at + d] = from_float<T>(made[0]);
        }
    };
    leave(rows_1, gains_1, offsets_1, op.offset_1 != nullptr);
    if (op.gain_2) leave(rows_2, gains_2, offsets_2, op.offset_2 != nullptr);
}

// The same for rows of any width, element by element: the sum is made once into `total` (or is x), and read again by the lane that made it.
template <typename T>
__global__ __launch_bounds__(64 * JOIN_WAVES) void join_norms_any_kernel(JoinOperands op, T* __restrict__ rows_1, T* __restrict__ rows_2) {
    const int lane = threadIdx.x % WAVE;
    const int row = blockIdx.x * JOIN_WAVES + threadIdx.x / WAVE;
    if (row >= op.n_rows) return;
    const size_t at = (size_t)row * op.width;
    const float* made = op.total ? op.total : op.x;
    float mean = 0.0f, squares = 0.0f;
    for (int d = lane; d < op.width; d += WAVE) {
        float sum = op.x[at + d];
        for (int p = 0; op.a && p < op.n_a; p++) sum += op.a[(size_t)p * op.a_stride + at + d];
        for (int p = 0; op.b && p < op.n_b; p++) sum += op.b[(size_t)p * op.b_stride + at + d];
        if (op.a_bias) sum += op.a_bias[d];
        if (op.b_bias) sum += op.b_bias[d];
        if (op.vector) sum += op.vector[d];
        if (op.total) op.total[at + d] = sum;
        mean += sum;
    }
    if (op.gain_1 == nullptr) return;
    mean = op.centred ? wave_sum(mean) / (float)op.width : 0.0f;
    for (int d = lane; d < op.width; d += WAVE) {
        const float centred = made[at + d] - mean;
        squares += centred * centred;
    }
    const float factor = 1.0f / sqrtf(wave_sum(squares) / (float)op.width + op.eps), plus = op.one_plus ? 1.0f : 0.0f;
    for (int d = lane; d < op.width; d += WAVE) {
        const float normed = (made[at + d] - mean) * factor;
        rows_1[at + d] = from_float<T>(normed * (plus + op.gain_1[d]) + (op.offset_1 ? op.offset_1[d] : 0.0f));
        if (op.gain_2) rows_2[at + d] = from_float<T>(normed * (plus + op.gain_2[d]) + (op.offset_2 ? op.offset_2[d] : 0.0f));
    }
}

__global__ __launch_bounds__(256) void soft_cap_kernel(const float* x, float* out, long long n, float cap) {
    const long long i = (long long)blockIdx.x * 256 + threadIdx.x;
    if (i < n) out[i] = cap * tanhf(x[i] / cap);
}

template <typename T>
void launch_join(const JoinOperands& op, void* rows_1, void* rows_2, bool pieces, hipStream_t stream) {
    const int blocks = ceil_div(op.n_rows, JOIN_WAVES), chunks = ceil_div(op.width, pieces ? 256 : 64);
#define JOIN(VEC, CHUNKS) join_norms_kernel<T, VEC, CHUNKS><<<blocks, 64 * JOIN_WAVES, 0, stream>>>(op, (T*)rows_1, (T*)rows_2)
    if (pieces && chunks <= 1) JOIN(4, 1);
    else if (pieces && chunks <= 2) JOIN(4, 2);
    else if (pieces && chunks <= 3) JOIN(4, 3);
    else if (pieces && chunks <= 4) JOIN(4, 4);
    else if (pieces && chunks <= 8) JOIN(4, 8);
    else if (!pieces && chunks <= 4) JOIN(1, 4);
    else join_norms_any_kernel<T><<<blocks, 64 * JOIN_WAVES, 0, stream>>>(op, (T*)rows_1, (T*)rows_2);
#undef JOIN
}

}  // namespace

// total = x + sum of a's and of b's partial products (+ biases) + vector; rows_i = norm(total) gain_i + offset_i. See JoinOperands.
MLLM_API int mllm_join_norms(const float* x, const float* a, int n_a, long long a_stride, const float* a_bias, const float* b, int n_b, long long b_stride,
                             const float* b_bias, const float* vector, float* total, const float* gain_1, const float* offset_1, void* rows_1,
                             const float* gain_2, const float* offset_2, void* rows_2, int centred, int one_plus, float eps, int rows_dtype, int n_rows,
                             int width, hipStream_t stream) {
    MLLM_REQUIRE(n_rows >= 0 && width > 0 && x != nullptr, "join_norms: bad sizes rows=%d width=%d, or no stream", n_rows, width);
    MLLM_REQUIRE((a == nullptr || n_a >= 1) && (b == nullptr || n_b >= 1), "join_norms: a branch without rows");
    MLLM_REQUIRE((n_a <= 1 || a_stride >= (long long)n_rows * width) && (n_b <= 1 || b_stride >= (long long)n_rows * width), "join_norms: partial products lie a whole matrix apart");
    MLLM_REQUIRE(total != x && (total != nullptr || (a == nullptr && b == nullptr && a_bias == nullptr && b_bias == nullptr && vector == nullptr)),
                 "join_norms: a sum needs a place of its own");
    MLLM_REQUIRE((gain_1 == nullptr || rows_1 != nullptr) && (gain_2 == nullptr || (gain_1 != nullptr && rows_2 != nullptr)), "join_norms: a norm needs rows to write");
    MLLM_REQUIRE(gain_1 == nullptr || ((rows_dtype == MLLM_F32 || rows_dtype == MLLM_BF16) && eps > 0.0f), "join_norms: normed rows of a known type, with a positive eps");
    if (n_rows == 0) return 0;
    mllm_count_kernel(MLLM_K_JOIN_NORMS);
    const JoinOperands op{x, a, n_a, a_stride, a_bias, b, n_b, b_stride, b_bias, vector, total, gain_1, offset_1, gain_2, offset_2, centred, one_plus, eps, n_rows, width};
    auto whole = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
    const bool pieces = width % 4 == 0 && a_stride % 4 == 0 && b_stride % 4 == 0 && whole(x) && whole(a) && whole(a_bias) && whole(b) && whole(b_bias) && whole(vector) &&
                        whole(total) && whole(gain_1) && whole(offset_1) && whole(rows_1) && whole(gain_2) && whole(offset_2) && whole(rows_2);
    if (gain_1 == nullptr || rows_dtype == MLLM_F32) launch_join<float>(op, rows_1, rows_2, pieces, stream);
    else launch_join<bf16_t>(op, rows_1, rows_2, pieces, stream);
    return mllm_check_launch("join_norms");
}

// out = cap tanh(x / cap); out may be x.
MLLM_API int mllm_soft_cap(const float* x, float* out, long long n, float cap, hipStream_t stream) {
    MLLM_REQUIRE(n >= 0 && cap > 0.0f && x != nullptr && out != nullptr, "soft_cap: bad sizes or a missing operand");
    MLLM_REQUIRE((n + 255) / 256 <= 0x7fffffffLL, "soft_cap: too many elements for one launch");
    if (n == 0) return 0;
    mllm_count_kernel(MLLM_K_SOFT_CAP);
    soft_cap_kernel<<<(int)((n + 255) / 256), 256, 0, stream>>>(x, out, n, cap);
    return mllm_check_launch("soft_cap");
}
