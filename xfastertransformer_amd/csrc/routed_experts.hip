// Routing of layer plans' expert feed-forwards: scores, choices and weights of every token, the lists of tokens by expert that
// the grouped products read, and the weighted sum behind them.  Router outputs past the experts hand the input through.
#include "plan_dev.h"

namespace xfthip {

namespace {

constexpr int kMaxRoutes = 1024, kMaxTop = 64;

struct RouteParams {
    const float *logits;
    const float *correction;
    int ld, T, experts, routes, top;
    int groups, keep; // groups 0: softmax and correction
    float scale;
    RouteBuffers b;
};

__device__ inline float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// Sigmoid scores, the choice within the best groups of neighbouring experts; one token a wave, a group a lane (in turns of 64) for
// the groups' scores.  Equal groups: the lower one first.
template <int CH>
__device__ inline void route_groups(const RouteParams &p, int t, int lane) {
    const float *logits = p.logits + (size_t)t * p.ld;
    const int n = p.routes / p.groups;
    float z[CH], choice[CH], group[CH];
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int e = i * 64 + lane;
        z[i] = e < p.routes ? sigmoid(logits[e]) : 0.0f;
        choice[i] = -INFINITY;
        group[i] = -INFINITY;
        if (e < p.groups) { // (at most as many groups as outputs)
            const float *g = logits + (size_t)e * n;
            float a = g[0], b = -INFINITY;
#pragma unroll 4
            for (int k = 1; k < n; ++k) {
                const float x = g[k];
                b = fmaxf(b, fminf(a, x)), a = fmaxf(a, x);
            }
            group[i] = sigmoid(a) + (n > 1 ? sigmoid(b) : 0.0f);
        }
    }
    for (int k = 0; k < p.keep; ++k) {
        float best = group[0];
#pragma unroll
        for (int i = 1; i < CH; ++i) best = fmaxf(best, group[i]);
        best = wave_largest(best);
        int chosen = p.groups - 1;
        bool open = true;
#pragma unroll
        for (int i = 0; i < CH; ++i) {
            const unsigned long long at = open ? __ballot(group[i] == best) : 0ull;
            if (at == 0ull) continue;
            const int who = __ffsll(at) - 1;
            open = false, chosen = i * 64 + who;
            if (lane == who) group[i] = -INFINITY;
        }
#pragma unroll
        for (int i = 0; i < CH; ++i) {
            const int e = i * 64 + lane;
            if (e < p.routes && e / n == chosen) choice[i] = z[i];
        }
    }
    float sum = 0.0f;
    for (int k = 0; k < p.top; ++k) {
        float best = choice[0];
#pragma unroll
        for (int i = 1; i < CH; ++i) best = fmaxf(best, choice[i]);
        best = wave_largest(best);
        int e = p.routes - 1; // (scores that are not numbers equal nothing)
        bool open = true;
#pragma unroll
        for (int i = 0; i < CH; ++i) {
            const unsigned long long at = open ? __ballot(choice[i] == best) : 0ull;
            if (at == 0ull) continue;
            const int who = __ffsll(at) - 1;
            open = false, e = i * 64 + who;
            if (lane == who) choice[i] = -INFINITY;
        }
        sum += best;
        if (lane == 0) p.b.sel[(size_t)t * p.top + k] = e < p.routes ? e : p.routes - 1;
        if (lane == 0) p.b.weight[(size_t)t * p.top + k] = best;
    }
    const float f = p.scale / (sum + 1e-20f);
    if (lane == 0)
        for (int k = 0; k < p.top; ++k) p.b.weight[(size_t)t * p.top + k] *= f;
}

// One token a wave: CH router outputs a lane.  The choice scores give way one by one, the lower index first among equals.
template <int CH>
__device__ inline void route_one(const RouteParams &p, int t, int lane) {
    if (p.groups > 0) return route_groups<CH>(p, t, lane);
    float z[CH], choice[CH], mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int e = i * 64 + lane;
        z[i] = e < p.routes ? p.logits[(size_t)t * p.ld + e] : -INFINITY;
        choice[i] = e < p.routes ? p.correction[e] : 0.0f;
        mx = fmaxf(mx, z[i]);
    }
    mx = wave_largest(mx);
    float sum = 0.0f;
#pragma unroll
    for (int i = 0; i < CH; ++i) z[i] = i * 64 + lane < p.routes ? expf(z[i] - mx) : 0.0f, sum += z[i];
    sum = wave_total(sum);
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        z[i] /= sum;
        choice[i] = i * 64 + lane < p.routes ? z[i] + choice[i] : -INFINITY;
    }
    for (int k = 0; k < p.top; ++k) {
        float best = choice[0];
#pragma unroll
        for (int i = 1; i < CH; ++i) best = fmaxf(best, choice[i]);
        best = wave_largest(best);
        // (scores that are not numbers equal nothing: the last output then, with a weight that is none either)
        int e = p.routes - 1;
        float score = sum;
        bool open = true;
#pragma unroll
        for (int i = 0; i < CH; ++i) {
            const unsigned long long at = open ? __ballot(choice[i] == best) : 0ull;
            if (at == 0ull) continue;
            const int who = __ffsll(at) - 1;
            open = false, e = i * 64 + who, score = __shfl(z[i], who, 64);
            if (lane == who) choice[i] = -INFINITY;
        }
        if (lane == 0) p.b.sel[(size_t)t * p.top + k] = e < p.routes ? e : p.routes - 1, p.b.weight[(size_t)t * p.top + k] = score;
    }
}

// lists of tokens by expert, in one workgroup: count, lay the lists back to back, fill
__device__ inline void build_lists(const RouteParams &p, int *count, int *first) {
    const int n = p.T * p.top;
    for (int e = threadIdx.x; e < p.experts; e += blockDim.x) count[e] = 0;
    __syncthreads();
    for (int i = threadIdx.x; i < n; i += blockDim.x) {
        const int e = p.b.sel[i];
        p.b.slot_row[i] = e < p.experts ? atomicAdd(&count[e], 1) : -1;
    }
    __syncthreads();
    if (threadIdx.x < 64) {
        const int per = (p.experts + 63) / 64, e0 = threadIdx.x * per;
        int own = 0;
        for (int e = e0; e < e0 + per && e < p.experts; ++e) own += count[e];
        int upto = own;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const int o = __shfl_up(upto, off, 64);
            if ((int)threadIdx.x >= off) upto += o;
        }
        int at = upto - own;
        for (int e = e0; e < e0 + per && e < p.experts; ++e) {
            first[e] = at;
            p.b.group_rows[3 * e] = count[e], p.b.group_rows[3 * e + 1] = at, p.b.group_rows[3 * e + 2] = at;
            at += count[e];
        }
    }
    __syncthreads();
    for (int i = threadIdx.x; i < n; i += blockDim.x) {
        const int e = p.b.sel[i];
        if (e >= p.experts) continue;
        const int row = first[e] + p.b.slot_row[i];
        p.b.slot_row[i] = row;
        p.b.row_token[row] = i / p.top;
    }
}

template <int CH>
__global__ __launch_bounds__(256) void route_kernel(RouteParams p) {
    const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (t < p.T) route_one<CH>(p, t, threadIdx.x & 63);
}
__global__ __launch_bounds__(1024) void route_lists_kernel(RouteParams p) {
    __shared__ int count[kMaxRoutes], first[kMaxRoutes];
    build_lists(p, count, first);
}
// few tokens: both at once
template <int CH>
__global__ __launch_bounds__(1024) void route_few_kernel(RouteParams p) {
    __shared__ int count[kMaxRoutes], first[kMaxRoutes];
    for (int t = threadIdx.x >> 6; t < p.T; t += 16) route_one<CH>(p, t, threadIdx.x & 63);
    __syncthreads();
    build_lists(p, count, first);
}

struct CombineParams {
    const float *base, *outputs;
    const void *h;
    int top;
    const float *weight;
    const int *slot_row;
    float *dst;
    void *narrow;
    int hidden;
};

// grid (tokens, column chunks of 1024)
template <bool BF16>
__global__ __launch_bounds__(256) void combine_experts_kernel(CombineParams p) {
    const int t = blockIdx.x, c = (blockIdx.y * 256 + threadIdx.x) * 4;
    if (c >= p.hidden) return;
    const size_t at = (size_t)t * p.hidden + c;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    if (p.base) acc = *(const f32x4 *)(p.base + at);
    for (int k = 0; k < p.top; ++k) {
        const int row = p.slot_row[t * p.top + k];
        const float w = p.weight[t * p.top + k];
        f32x4 y;
        if (row >= 0) {
            y = *(const f32x4 *)(p.outputs + (size_t)row * p.hidden + c);
        } else if constexpr (BF16) {
            const uint2 u = *(const uint2 *)((const uint16_t *)p.h + at);
            y = f32x4 {u2f(u.x << 16), u2f(u.x & 0xFFFF0000u), u2f(u.y << 16), u2f(u.y & 0xFFFF0000u)};
        } else {
            y = *(const f32x4 *)((const float *)p.h + at);
        }
        acc += y * w;
    }
    *(f32x4 *)(p.dst + at) = acc;
    if (p.narrow) put4<BF16>(p.narrow, at, acc);
}

template <int CH>
int launch_route(const RouteParams &p, hipStream_t st) {
    if (p.T <= 32) {
        hipLaunchKernelGGL(route_few_kernel<CH>, dim3(1), dim3(1024), 0, st, p);
    } else {
        hipLaunchKernelGGL(route_kernel<CH>, dim3((p.T + 3) / 4), dim3(256), 0, st, p);
        hipLaunchKernelGGL(route_lists_kernel, dim3(1), dim3(1024), 0, st, p);
    }
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

} // namespace

int route_tokens(const float *logits, int ld, const RouteRule &r, int T, const RouteBuffers &b, hipStream_t st) {
    const int routes = r.routes;
    XFT_REQUIRE(T > 0 && r.experts > 0 && routes >= r.experts && routes <= kMaxRoutes && r.top > 0 && r.top <= routes && r.top <= kMaxTop && ld >= routes
                    && (r.groups > 0 ? routes == r.experts && routes % r.groups == 0 && r.keep > 0 && r.keep <= r.groups : r.correction != nullptr),
            "route_tokens: %d of %d + %d outputs", r.top, r.experts, routes - r.experts);
    const RouteParams p = {logits, r.correction, ld, T, r.experts, routes, r.top, r.groups, r.keep, r.scale, b};
    if (routes <= 64) return launch_route<1>(p, st);
    if (routes <= 128) return launch_route<2>(p, st);
    if (routes <= 256) return launch_route<4>(p, st);
    return launch_route<16>(p, st);
}

int combine_experts(int act, const float *base, const float *outputs, const void *h, int top, const RouteBuffers &b, float *dst, void *narrow, int T,
        int hidden, hipStream_t st) {
    XFT_REQUIRE(T > 0 && dst && hidden % 4 == 0, "combine_experts: bad argument");
    const CombineParams p = {base, outputs, h, top, b.weight, b.slot_row, dst, narrow, hidden};
    const dim3 grid(T, (hidden + 1023) / 1024);
    if (act == XFTHIP_BF16) hipLaunchKernelGGL(combine_experts_kernel<true>, grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL(combine_experts_kernel<false>, grid, dim3(256), 0, st, p);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

} // namespace xfthip
