// A feed-forward made of many small ones ("experts") of which a router picks a few per row, and the two gate units of feed-forwards
// whose activation is more than one function of one number.
//
// The routed experts run as ONE up product over all experts' matrices laid behind each other and ONE down product over their down
// matrices laid side by side: between the two, `expert_unit` multiplies every expert's hidden units by the row's weight for that
// expert, which is zero for the experts the router did not pick, so the down product's sum over all hidden units is the weighted sum
// over the picked experts. Nothing is planned on the host and no row's result depends on the other rows of the batch.
#include "common.h"
#include "gate_unit.h"

#include <math.h>

namespace {

constexpr int ROUTE_MAX_EXPERTS = 1024, ROUTE_FEW_EXPERTS = 64;

// (value, index) a is picked before b: the larger value, among equals the smaller index.
__device__ __forceinline__ bool picked_before(float a, int ia, float b, int ib) { return a > b || (a == b && ia < ib); }

// What a router does with a row's sums: scores s = softmax over all n_experts, or with `sigmoid` 1 / (1 + e^-z); choice c = s + correction
// (null: none). The experts form n_groups equal groups of neighbours; a group's rank goes by the largest c in it, and only experts of
// the best `keep` groups can be picked (the others count as minus infinity). The `top` experts of largest c are picked; a picked
// expert's weight is s_e / (sum of the picked experts' s + floor), without `renormalise` s_e itself. (Softmax scores without a correction
// are compared by the sums themselves: the same order, also where scores vanish in 32 bits.)
struct Choice {
    const float* correction;
    int n_experts, top, n_groups, keep;
    float floor;
    int sigmoid, renormalise;
    int always;   // so many experts n_experts, n_experts + 1, ... that every row uses stand behind its own picks, with weight 1
};
// Where it goes, each optional: weights [row, n_experts] (rows `stride` apart, 0 for the experts that were not picked); picks and
// pick_weights [row, top + always], the picked experts in the order of their choice scores (-1 where sums that are no numbers left none to pick).
struct Routed {
    float* weights;
    int stride;
    int* picks;
    float* pick_weights;
};

// One wave; `score` holds the row's sums.
__device__ void route_row(const Choice& how, const Routed& to, size_t row, float* score, float* choice, float* group_best, int lane) {
    const int n_experts = how.n_experts;
    const int places = how.top + how.always;
    if (to.picks)
        for (int k = lane; k < places; k += WAVE) {
            to.picks[row * places + k] = k < how.top ? -1 : n_experts + k - how.top;
            if (k >= how.top) to.pick_weights[row * places + k] = 1.0f;
        }
    float largest = -INFINITY;
    for (int e = lane; e < n_experts; e += WAVE) largest = fmaxf(largest, score[e]);
    largest = wave_max(largest);
    float total = 0.0f;
    for (int e = lane; e < n_experts; e += WAVE) {
        const float z = score[e], p = how.sigmoid ? 1.0f / (1.0f + expf(-z)) : expf(z - largest);
        score[e] = p;
        choice[e] = z;
        total += p;
    }
    total = how.sigmoid ? 1.0f : wave_sum(total);
    for (int e = lane; e < n_experts; e += WAVE) {
        const float s = score[e] / total;
        score[e] = s;
        if (how.sigmoid || how.correction) choice[e] = s + (how.correction ? how.correction[e] : 0.0f);
    }
    __builtin_amdgcn_wave_barrier();
    __threadfence_block();
    if (how.n_groups > 1) {
        const int size = n_experts / how.n_groups;
        for (int g = lane; g < how.n_groups; g += WAVE) {
            float best = -INFINITY;
            for (int e = g * size; e < (g + 1) * size; e++) best = fmaxf(best, choice[e]);
            group_best[g] = best;
        }
        __builtin_amdgcn_wave_barrier();
        __threadfence_block();
        for (int g = lane; g < how.n_groups; g += WAVE) {   // a group is kept if fewer than `keep` groups come before it
            const float mine = group_best[g];
            int before = 0;
            for (int o = 0; o < how.n_groups; o++) before += picked_before(group_best[o], o, mine, g) ? 1 : 0;
            if (before >= how.keep)
                for (int e = g * size; e < (g + 1) * size; e++) choice[e] = -INFINITY;
        }
        __builtin_amdgcn_wave_barrier();
        __threadfence_block();
    }
    float picked_sum = 0.0f;
    for (int e = lane; e < n_experts; e += WAVE) {
        const float mine = choice[e];
        int before = 0;
        for (int o = 0; o < n_experts; o++) before += picked_before(choice[o], o, mine, e) ? 1 : 0;
        const bool picked = before < how.top && mine > -INFINITY;
        picked_sum += picked ? score[e] : 0.0f;
        group_best[e] = picked ? (float)before : -1.0f;   // every lane reads and writes its own experts' entries only from here on
    }
    picked_sum = how.renormalise ? wave_sum(picked_sum) + how.floor : 1.0f;
    for (int e = lane; e < n_experts; e += WAVE) {
        const int place = (int)group_best[e];
        const float weight = place >= 0 ? score[e] / picked_sum : 0.0f;
        if (to.weights) to.weights[row * to.stride + e] = weight;
        if (to.picks && place >= 0) {
            to.picks[row * places + place] = e;
            to.pick_weights[row * places + place] = weight;
        }
    }
}

// One wave a row. logits: the router's 32-bit sums [row, n_experts] (rows `stride` apart).
__global__ __launch_bounds__(WAVE) void route_kernel(const float* __restrict__ logits, int stride, Choice how, Routed to) {
    __shared__ float score[ROUTE_MAX_EXPERTS], choice[ROUTE_MAX_EXPERTS], group_best[ROUTE_MAX_EXPERTS];
    const int lane = threadIdx.x;
    const size_t row = blockIdx.x;
    for (int e = lane; e < how.n_experts; e += WAVE) score[e] = logits[row * stride + e];
    route_row(how, to, row, score, choice, group_best, lane);
}

// The router's product and its choice in one: four waves share a row's experts, a wave an expert at a time (16-byte pieces of x and of
// the expert's row of the router's matrix [n_experts, K], sums in 32-bit), then the first wave chooses. For routers of few outputs: the
// matrix is read once a row.
template <typename T>
__global__ __launch_bounds__(256) void route_rows_kernel(const T* __restrict__ x, const T* __restrict__ router, int K, Choice how, Routed to) {
    __shared__ float score[ROUTE_FEW_EXPERTS], choice[ROUTE_FEW_EXPERTS], group_best[ROUTE_FEW_EXPERTS];
    constexpr int VEC = 16 / (int)sizeof(T);
    const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE;
    const size_t row = blockIdx.x;
    const T* x_row = x + row * K;
    for (int e0 = wave; e0 < how.n_experts; e0 += 8) {   // two experts of a wave at a time
        const int e1 = min(e0 + 4, how.n_experts - 1);
        float sum0 = 0.0f, sum1 = 0.0f;
        for (int k = lane * VEC; k < K; k += WAVE * VEC) {
            const Vec16 xs = *reinterpret_cast<const Vec16*>(x_row + k), a = *reinterpret_cast<const Vec16*>(router + (size_t)e0 * K + k),
                        b = *reinterpret_cast<const Vec16*>(router + (size_t)e1 * K + k);
            const T *xe = reinterpret_cast<const T*>(&xs), *ae = reinterpret_cast<const T*>(&a), *be = reinterpret_cast<const T*>(&b);
#pragma unroll
            for (int j = 0; j < VEC; j++) {
                sum0 = __builtin_fmaf(to_float(xe[j]), to_float(ae[j]), sum0);
                sum1 = __builtin_fmaf(to_float(xe[j]), to_float(be[j]), sum1);
            }
        }
        sum0 = wave_total(sum0);
        sum1 = wave_total(sum1);
        if (lane == 0) {
            score[e0] = sum0;
            if (e0 + 4 < how.n_experts) score[e0 + 4] = sum1;
        }
    }
    __syncthreads();
    if (wave == 0) route_row(how, to, row, score, choice, group_best, lane);
}

// up: [rows, n_routed * ff + shared] hidden units before their activation, expert by expert, then `shared` units of an expert that
// every row uses. out = relu(up)^2 * weights[row, expert] (shared units: relu(up)^2). Behind the `unit_blocks` blocks of the hidden units
// the grid goes on over `width` columns of `carried` (null: none): carried[row, :] = h[row, :] * (the sum of weights[row, n_routed ..
// n_routed + n_identity)), the share of the experts that hand their input on as it is. PIECES: a thread takes 16 bytes of units (ff and
// shared are multiples of that many units, so a piece lies in one expert).
template <typename T, bool PIECES>
__global__ __launch_bounds__(256) void expert_unit_kernel(const T* __restrict__ up, T* __restrict__ out, const float* __restrict__ weights, int weights_stride,
                                                          int n_routed, int ff, int shared, const T* __restrict__ h, float* __restrict__ carried,
                                                          int n_identity, int width, int unit_blocks) {
    constexpr int VEC = PIECES ? 16 / (int)sizeof(T) : 1;
    const int inner = n_routed * ff + shared;
    const size_t row = blockIdx.y;
    const float* w = weights + row * weights_stride;
    if ((int)blockIdx.x >= unit_blocks) {
        const int j = ((int)blockIdx.x - unit_blocks) * blockDim.x + threadIdx.x;
        if (carried == nullptr || j >= width) return;
        float share = 0.0f;
        for (int e = 0; e < n_identity; e++) share += w[n_routed + e];
        carried[row * width + j] = to_float(h[row * width + j]) * share;
        return;
    }
    const int j = (blockIdx.x * blockDim.x + threadIdx.x) * VEC;
    if (j >= inner) return;
    const float weight = j < n_routed * ff ? w[j / ff] : 1.0f;
    if constexpr (PIECES) {
        const Vec16 in = *reinterpret_cast<const Vec16*>(up + row * inner + j);
        Vec16 result;
        const T* ie = reinterpret_cast<const T*>(&in);
        T* re = reinterpret_cast<T*>(&result);
#pragma unroll
        for (int e = 0; e < VEC; e++) {
            const float u = fmaxf(to_float(ie[e]), 0.0f);
            re[e] = from_float<T>(u * u * weight);
        }
        *reinterpret_cast<Vec16*>(out + row * inner + j) = result;
    } else {
        const float u = fmaxf(to_float(up[row * inner + j]), 0.0f);
        out[row * inner + j] = from_float<T>(u * u * weight);
    }
}

// both: [rows, 2 * inner], a gate half and an up half; out = their gate unit (gate_unit.h). PIECES: a thread takes 16 bytes of each half.
template <typename T, bool PIECES>
__global__ __launch_bounds__(256) void gate_unit_kernel(const T* __restrict__ both, T* __restrict__ out, int inner, GateUnit unit) {
    constexpr int VEC = PIECES ? 16 / (int)sizeof(T) : 1;
    const int j = (blockIdx.x * blockDim.x + threadIdx.x) * VEC;
    if (j >= inner) return;
    const size_t row = blockIdx.y;
    const T* g_at = both + row * 2 * inner + j;
    const T* u_at = g_at + inner;
    T* out_at = out + row * inner + j;
    if constexpr (PIECES) {
        const Vec16 gs = *reinterpret_cast<const Vec16*>(g_at), us = *reinterpret_cast<const Vec16*>(u_at);
        Vec16 result;
        const T* ge = reinterpret_cast<const T*>(&gs);
        const T* ue = reinterpret_cast<const T*>(&us);
        T* re = reinterpret_cast<T*>(&result);
#pragma unroll
        for (int e = 0; e < VEC; e++) {
            re[e] = from_float<T>(gated(to_float(ge[e]), to_float(ue[e]), unit));
        }
        *reinterpret_cast<Vec16*>(out_at) = result;
    } else {
        *out_at = from_float<T>(gated(to_float(*g_at), to_float(*u_at), unit));
    }
}

template <typename T>
void launch_expert_unit(const void* up, void* out, const float* weights, int weights_stride, int rows, int n_routed, int ff, int shared, const void* h,
                        float* carried, int n_identity, int width, hipStream_t stream) {
    constexpr int VEC = 16 / (int)sizeof(T);
    const int inner = n_routed * ff + shared;
    const bool pieces = ff % VEC == 0 && shared % VEC == 0 && ((uintptr_t)up & 15) == 0 && ((uintptr_t)out & 15) == 0;
    const int unit_blocks = ceil_div(pieces ? inner / VEC : inner, 256);
    dim3 grid(unit_blocks + (carried != nullptr ? ceil_div(width, 256) : 0), rows);
    if (pieces)
        expert_unit_kernel<T, true><<<grid, 256, 0, stream>>>((const T*)up, (T*)out, weights, weights_stride, n_routed, ff, shared, (const T*)h, carried, n_identity,
                                                              width, unit_blocks);
    else
        expert_unit_kernel<T, false><<<grid, 256, 0, stream>>>((const T*)up, (T*)out, weights, weights_stride, n_routed, ff, shared, (const T*)h, carried, n_identity,
                                                               width, unit_blocks);
}

template <typename T>
void launch_gate_unit(const void* both, void* out, int rows, int inner, GateUnit unit, hipStream_t stream) {
    constexpr int VEC = 16 / (int)sizeof(T);
    if (inner % VEC == 0 && ((uintptr_t)both & 15) == 0 && ((uintptr_t)out & 15) == 0) {
        dim3 grid(ceil_div(inner / VEC, 256), rows);
        gate_unit_kernel<T, true><<<grid, 256, 0, stream>>>((const T*)both, (T*)out, inner, unit);
    } else {
        dim3 grid(ceil_div(inner, 256), rows);
        gate_unit_kernel<T, false><<<grid, 256, 0, stream>>>((const T*)both, (T*)out, inner, unit);
    }
}

}  // namespace

namespace {
int check_choice(int n_rows, const Choice& how, const Routed& to) {
    MLLM_REQUIRE(n_rows >= 0 && how.n_experts > 0 && how.n_experts <= ROUTE_MAX_EXPERTS, "route: %d experts (the kernel takes up to %d)", how.n_experts, ROUTE_MAX_EXPERTS);
    MLLM_REQUIRE(how.n_groups >= 1 && how.n_experts % how.n_groups == 0 && how.keep >= 1 && how.keep <= how.n_groups, "route: %d experts in %d groups of which %d are kept",
                 how.n_experts, how.n_groups, how.keep);
    MLLM_REQUIRE(how.top >= 1 && how.top <= how.keep * (how.n_experts / how.n_groups), "route: %d experts to pick among %d groups of %d", how.top, how.keep,
                 how.n_experts / how.n_groups);
    MLLM_REQUIRE((to.weights != nullptr || to.picks != nullptr) && (to.picks == nullptr) == (to.pick_weights == nullptr), "route: nowhere to leave the choice");
    MLLM_REQUIRE(how.always >= 0 && (how.always == 0 || to.picks != nullptr) && how.n_experts + how.always <= ROUTE_MAX_EXPERTS, "route: %d experts behind the picks", how.always);
    MLLM_REQUIRE(to.weights == nullptr || to.stride >= how.n_experts, "route: the weights' rows are too short");
    return 0;
}
}  // namespace

MLLM_API int mllm_route(const float* logits, int stride, const float* correction, float* weights, int weights_stride, int* picks, float* pick_weights, int n_rows,
                        int n_experts, int top, int n_groups, int keep, float floor, int sigmoid, int renormalise, int always, hipStream_t stream) {
    const Choice how{correction, n_experts, top, n_groups, keep, floor, sigmoid, renormalise, always};
    const Routed to{weights, weights_stride, picks, pick_weights};
    if (int status = check_choice(n_rows, how, to)) return status;
    MLLM_REQUIRE(stride >= n_experts && logits != nullptr, "route: rows are too short or missing");
    if (n_rows == 0) return 0;
    mllm_count_kernel(MLLM_K_ROUTE);
    route_kernel<<<n_rows, WAVE, 0, stream>>>(logits, stride, how, to);
    return mllm_check_launch("route");
}

// Whether the router's product rides in the choice's kernel (mllm_route_rows): few outputs, rows of whole 16-byte pieces.
MLLM_API int mllm_route_rows_supported(int n_experts, int K, int dtype) {
    const int vec = dtype == MLLM_F32 ? 4 : 8;
    return n_experts >= 1 && n_experts <= ROUTE_FEW_EXPERTS && K >= vec && K % vec == 0;
}

MLLM_API int mllm_route_rows(const void* x, const void* router, int K, const float* correction, float* weights, int weights_stride, int* picks,
                             float* pick_weights, int n_rows, int n_experts, int top, int n_groups, int keep, float floor, int sigmoid, int renormalise,
                             int always, int dtype, hipStream_t stream) {
    const Choice how{correction, n_experts, top, n_groups, keep, floor, sigmoid, renormalise, always};
    const Routed to{weights, weights_stride, picks, pick_weights};
    if (int status = check_choice(n_rows, how, to)) return status;
    MLLM_REQUIRE(dtype == MLLM_F32 || dtype == MLLM_BF16, "route_rows: unknown dtype %d", dtype);
    MLLM_REQUIRE(mllm_route_rows_supported(n_experts, K, dtype), "route_rows: no kernel for %d outputs over rows of %d", n_experts, K);
    MLLM_REQUIRE(((uintptr_t)x & 15) == 0 && ((uintptr_t)router & 15) == 0 && x && router, "route_rows: rows and matrix must start on 16 bytes");
    if (n_rows == 0) return 0;
    mllm_count_kernel(MLLM_K_ROUTE);
    if (dtype == MLLM_F32) route_rows_kernel<float><<<n_rows, 256, 0, stream>>>((const float*)x, (const float*)router, K, how, to);
    else route_rows_kernel<bf16_t><<<n_rows, 256, 0, stream>>>((const bf16_t*)x, (const bf16_t*)router, K, how, to);
    return mllm_check_launch("route_rows");
}

MLLM_API int mllm_expert_unit(const void* up, void* out, const float* weights, int weights_stride, int n_rows, int n_routed, int ff, int shared, const void* h,
                              float* carried, int n_identity, int width, int dtype, hipStream_t stream) {
    MLLM_REQUIRE(n_rows >= 0 && n_routed >= 0 && ff > 0 && shared >= 0 && n_identity >= 0, "expert_unit: bad sizes");
    MLLM_REQUIRE(weights_stride >= n_routed + n_identity && up != nullptr && out != nullptr && weights != nullptr, "expert_unit: a missing operand or short weights");
    MLLM_REQUIRE(carried == nullptr || (h != nullptr && width > 0), "expert_unit: the rows that are handed on need the input rows");
    MLLM_REQUIRE(dtype == MLLM_F32 || dtype == MLLM_BF16, "expert_unit: unknown dtype %d", dtype);
    if (n_rows == 0) return 0;
    mllm_count_kernel(MLLM_K_EXPERT_UNIT);
    const long long inner = (long long)n_routed * ff + shared;
    const size_t element = dtype == MLLM_F32 ? 4 : 2;
    for (int row0 = 0; row0 < n_rows; row0 += 65535) {   // the grid's second dimension holds 65,535 rows
        const int rows = n_rows - row0 < 65535 ? n_rows - row0 : 65535;
        const char* up_at = (const char*)up + (size_t)row0 * inner * element;
        char* out_at = (char*)out + (size_t)row0 * inner * element;
        const char* h_at = h == nullptr ? nullptr : (const char*)h + (size_t)row0 * width * element;
        float* carried_at = carried == nullptr ? nullptr : carried + (size_t)row0 * width;
        const float* weights_at = weights + (size_t)row0 * weights_stride;
        if (dtype == MLLM_F32) launch_expert_unit<float>(up_at, out_at, weights_at, weights_stride, rows, n_routed, ff, shared, h_at, carried_at, n_identity, width, stream);
        else launch_expert_unit<bf16_t>(up_at, out_at, weights_at, weights_stride, rows, n_routed, ff, shared, h_at, carried_at, n_identity, width, stream);
    }
    return mllm_check_launch("expert_unit");
}

MLLM_API int mllm_gate_unit(const void* both, void* out, int n_rows, int inner, float limit, float alpha, float shift, int dtype, hipStream_t stream) {
    MLLM_REQUIRE(n_rows >= 0 && inner > 0, "gate_unit: bad sizes");
    MLLM_REQUIRE(limit > 0.0f, "gate_unit: the limit must be positive (infinite: none)");
    MLLM_REQUIRE(dtype == MLLM_F32 || dtype == MLLM_BF16, "gate_unit: unknown dtype %d", dtype);
    if (n_rows == 0) return 0;
    mllm_count_kernel(MLLM_K_GATE_UNIT);
    const size_t element = dtype == MLLM_F32 ? 4 : 2;
    for (int row0 = 0; row0 < n_rows; row0 += 65535) {
        const int rows = n_rows - row0 < 65535 ? n_rows - row0 : 65535;
        const char* in_at = (const char*)both + (size_t)row0 * 2 * inner * element;
        char* out_at = (char*)out + (size_t)row0 * inner * element;
        if (dtype == MLLM_F32) launch_gate_unit<float>(in_at, out_at, rows, inner, GateUnit{limit, alpha, shift}, stream);
        else launch_gate_unit<bf16_t>(in_at, out_at, rows, inner, GateUnit{limit, alpha, shift}, stream);
    }
    return mllm_check_launch("gate_unit");
}
