// The gated linear recurrence of layer plans: a causal filter a channel (unit_filter), the products of both gates (tile_gemm, block by
// block), and S = a S + sqrt(1 - a^2) i u with a = exp(-8 r softplus(lambda)), times gelu(y) (unit_scan).  Channels do not interact.
// Behind the filter everything is fp32.
#include "plan_dev.h"

namespace xfthip {

namespace {

constexpr int kFilterTokens = 16; // tokens a thread of the filter walks
constexpr int kChunk = 64; // tokens a thread of the scan walks
constexpr int kAhead = 8; // tokens (or chunk ends) whose operands are requested together

struct FilterParams {
    StepView v;
    const void *in;
    int ld, channels, taps;
    const float *filter, *bias;
    void *u, *conv_state;
};

// One thread a channel and kFilterTokens tokens of a segment; grid (channels / 256, token tiles, segments).  A sequence's single new
// token shifts the inputs in place (nobody else reads this channel of the slot); longer segments leave that to conv_tail.
template <bool BF16>
__global__ __launch_bounds__(256) void unit_filter_kernel(FilterParams p) {
    const int ch = blockIdx.x * 256 + threadIdx.x, seg = blockIdx.z, n = p.v.seg_len[seg], i0 = blockIdx.y * kFilterTokens;
    if (ch >= p.channels || i0 >= n) return;
    const int off = p.v.seg_off[seg], start = p.v.seg_pos[seg], end = i0 + kFilterTokens < n ? i0 + kFilterTokens : n;
    const size_t hist = (size_t)p.v.seg_row[seg] * (p.taps - 1) * p.channels + ch;
    const float bias = p.bias[ch];
    auto input = [&](int i) { // local index; negative: what earlier steps left, before the sequence's start: zero
        if (start + i < 0) return 0.0f;
        return i >= 0 ? ldact<BF16>(p.in, (size_t)(off + i) * p.ld + ch) : ldact<BF16>(p.conv_state, hist + (size_t)(p.taps - 1 + i) * p.channels);
    };
    for (int i = i0; i < end; ++i) {
        float acc = bias;
        for (int j = 0; j < p.taps; ++j) acc = fmaf(p.filter[(size_t)ch * p.taps + j], input(i - (p.taps - 1) + j), acc);
        stact<BF16>(p.u, (size_t)(off + i) * p.channels + ch, acc);
    }
    if (n == 1) {
        for (int s = 0; s + 1 < p.taps - 1; ++s) stact<BF16>(p.conv_state, hist + (size_t)s * p.channels, ldact<BF16>(p.conv_state, hist + (size_t)(s + 1) * p.channels));
        if (p.taps > 1) stact<BF16>(p.conv_state, hist + (size_t)(p.taps - 2) * p.channels, ldact<BF16>(p.in, (size_t)off * p.ld + ch));
    }
}

// The same for filters of up to 4 taps and two channels a thread (channels and ld are even): the window of inputs stays in registers.
// grid (channels / 512, token tiles, segments)
template <bool BF16, int TAPS>
__global__ __launch_bounds__(256) void unit_filter_tiled_kernel(FilterParams p) {
    const int ch = (blockIdx.x * 256 + threadIdx.x) * 2, seg = blockIdx.z, n = p.v.seg_len[seg], i0 = blockIdx.y * kFilterTokens;
    if (ch >= p.channels || i0 >= n) return;
    const int off = p.v.seg_off[seg], start = p.v.seg_pos[seg], end = i0 + kFilterTokens < n ? i0 + kFilterTokens : n;
    const size_t hist = (size_t)p.v.seg_row[seg] * (TAPS - 1) * p.channels + ch;
    const float2 bias = *(const float2 *)(p.bias + ch);
    float2 w[TAPS], x[TAPS - 1 + kFilterTokens];
#pragma unroll
    for (int t = 0; t < TAPS; ++t) w[t] = make_float2(p.filter[(size_t)ch * TAPS + t], p.filter[(size_t)(ch + 1) * TAPS + t]);
#pragma unroll
    for (int t = 0; t < TAPS - 1; ++t) {
        const int i = i0 - (TAPS - 1) + t;
        x[t] = start + i < 0 ? make_float2(0.0f, 0.0f)
                             : (i >= 0 ? load2<BF16>(p.in, (size_t)(off + i) * p.ld + ch) : load2<BF16>(p.conv_state, hist + (size_t)(TAPS - 1 + i) * p.channels));
    }
#pragma unroll
    for (int k = 0; k < kFilterTokens; ++k) x[TAPS - 1 + k] = i0 + k < end ? load2<BF16>(p.in, (size_t)(off + i0 + k) * p.ld + ch) : make_float2(0.0f, 0.0f);
#pragma unroll
    for (int k = 0; k < kFilterTokens; ++k) {
        float2 a = bias;
#pragma unroll
        for (int t = 0; t < TAPS; ++t) a.x = fmaf(w[t].x, x[k + t].x, a.x), a.y = fmaf(w[t].y, x[k + t].y, a.y);
        if (i0 + k < end) store2<BF16>(p.u, (size_t)(off + i0 + k) * p.channels + ch, a);
    }
    if (n == 1) {
#pragma unroll
        for (int s = 0; s < TAPS - 1; ++s) store2<BF16>(p.conv_state, hist + (size_t)s * p.channels, x[s + 1]);
    }
}

struct UnitParams {
    StepView v;
    const void *u;
    const float *gates, *gate_bias, *lambda;
    const void *y; // rows of pitch ld
    int ld;
    void *out; // rows of pitch out_ld
    int out_ld, channels, D;
    float mul;
    float *state;
    float2 *carry; // see carry_row
};

// a and b of S = a S + b; FAST (bf16 activations): the hardware's exponential, reciprocal and square root
template <bool FAST>
__device__ inline float2 recurrence(float r, float i, float u, float lambda) {
    if constexpr (FAST) {
        const float log_a = -lambda * __builtin_amdgcn_rcpf(1.0f + fast_exp(-r)), a = fast_exp(log_a), t = 2.0f * log_a;
        // 1 - exp(t), by its series where the difference would cancel (t^7 / 8! is below 2e-7 there)
        float series = 1.0f;
#pragma unroll
        for (int k = 7; k > 1; --k) series = fmaf(series, t * (1.0f / k), 1.0f);
        const float rest = t > -0.5f ? -t * series : fmaf(-a, a, 1.0f);
        return make_float2(a, __builtin_amdgcn_sqrtf(rest) * u * __builtin_amdgcn_rcpf(1.0f + fast_exp(-i)));
    } else {
        const float log_a = -lambda / (1.0f + expf(-r));
        return make_float2(expf(log_a), sqrtf(-expm1f(2.0f * log_a)) * u / (1.0f + expf(-i)));
    }
}

// 0.5 (1 + tanh(x)) = 1 / (1 + exp(-2 x))
template <bool FAST>
__device__ inline float gelu_of(float z) {
    if constexpr (FAST) return z * __builtin_amdgcn_rcpf(1.0f + fast_exp(-1.5957691216057308f * (z + 0.044715f * z * z * z)));
    else return gelu_tanh(z);
}

// rows of a segment in the carry buffer: the state in front of it, then a pair (product of a, end from zero) a chunk
__device__ inline size_t carry_row(const UnitParams &p, int seg) { return ((size_t)p.v.seg_off[seg] / kChunk + 2 * (size_t)seg) * p.channels; }

// One thread a channel and chunk; grid (channels / 256, chunks, segments).  FIRST: what a chunk does to the state that enters it.
// Otherwise: the outputs, behind the chunks before it (a segment of one chunk needs no first pass).
template <bool BF16, bool FIRST>
__global__ __launch_bounds__(256) void unit_scan_kernel(UnitParams p) {
    const int ch = blockIdx.x * 256 + threadIdx.x, seg = blockIdx.z, n = p.v.seg_len[seg], i0 = blockIdx.y * kChunk;
    if (ch >= p.channels || i0 >= n || (FIRST && n <= kChunk)) return;
    const int off = p.v.seg_off[seg], end = i0 + kChunk < n ? i0 + kChunk : n;
    float *state = p.state + (size_t)p.v.seg_row[seg] * p.channels + ch;
    float2 *carry = p.carry + carry_row(p, seg) + ch;
    const int block = ch / p.D, gc = (2 * block) * p.D + ch % p.D;
    const float rb = p.gate_bias[gc], ib = p.gate_bias[gc + p.D], lambda = p.lambda[ch];
    const size_t gpitch = (size_t)2 * p.channels;
    struct Operands {
        float r, i, u, y;
    };
    auto request = [&](int i) {
        const float *g = p.gates + (size_t)(off + i) * gpitch + gc;
        return Operands {g[0], g[p.D], ldact<BF16>(p.u, (size_t)(off + i) * p.channels + ch), FIRST ? 0.0f : ldact<BF16>(p.y, (size_t)(off + i) * p.ld + ch)};
    };
    float a = 1.0f, s = 0.0f;
    auto token = [&](int i, const Operands &q) {
        const float2 x = recurrence<BF16>(q.r + rb, q.i + ib, q.u, lambda);
        s = fmaf(x.x, s, x.y);
        if constexpr (FIRST) a *= x.x;
        else stact<BF16>(p.out, (size_t)(off + i) * p.out_ld + ch, s * gelu_of<BF16>(q.y) * p.mul);
    };
    if constexpr (!FIRST) {
        if (n <= kChunk) {
            if (p.v.seg_pos[seg] > 0) s = *state;
        } else {
            for (int c0 = 0; c0 <= (int)blockIdx.y; c0 += kAhead) {
                float2 x[kAhead];
#pragma unroll
                for (int k = 0; k < kAhead; ++k) x[k] = c0 + k <= (int)blockIdx.y ? carry[(size_t)(c0 + k) * p.channels] : make_float2(1.0f, 0.0f);
#pragma unroll
                for (int k = 0; k < kAhead; ++k) s = fmaf(x[k].x, s, x[k].y);
            }
        }
    }
    int i = i0;
    if (end - i >= kAhead) {
        Operands next[kAhead];
#pragma unroll
        for (int k = 0; k < kAhead; ++k) next[k] = request(i + k);
        for (; i + kAhead <= end; i += kAhead) {
            Operands now[kAhead];
            const bool more = i + 2 * kAhead <= end;
#pragma unroll
            for (int k = 0; k < kAhead; ++k) now[k] = next[k];
            if (more) {
#pragma unroll
                for (int k = 0; k < kAhead; ++k) next[k] = request(i + kAhead + k);
            }
#pragma unroll
            for (int k = 0; k < kAhead; ++k) token(i + k, now[k]);
        }
    }
    for (; i < end; ++i) token(i, request(i));
    if constexpr (FIRST) {
        carry[(size_t)(blockIdx.y + 1) * p.channels] = make_float2(a, s);
        if (blockIdx.y == 0) carry[0] = make_float2(0.0f, p.v.seg_pos[seg] > 0 ? *state : 0.0f);
    } else if (end == n) {
        *state = s;
    }
}

} // namespace

size_t unit_carry_floats(const PlanLayer &L, size_t tokens, size_t segments) { return (tokens / kChunk + 2 * segments + 2) * L.channels() * 2; }

int unit_filter(int act, const PlanLayer &L, const StepView &v, const UnitBuffers &b, hipStream_t st) {
    const int C = L.channels();
    const void *x = (const char *)b.in + (size_t)(L.in_col + C) * (act == XFTHIP_BF16 ? 2 : 4);
    const FilterParams p = {v, x, L.in_ld, C, L.s.taps, L.conv, L.conv_bias, b.u, b.conv_state};
    const unsigned tiles = (v.longest + kFilterTokens - 1) / kFilterTokens;
    const dim3 grid((C + 255) / 256, tiles, v.B), pairs((C / 2 + 255) / 256, tiles, v.B);
    const bool paired = C % 2 == 0 && L.in_ld % 2 == 0 && (L.in_col + C) % 2 == 0;
    auto launch = [&](void (*kernel)(FilterParams), const dim3 &g) { hipLaunchKernelGGL(kernel, g, dim3(256), 0, st, p); };
    const int form = paired && p.taps >= 2 && p.taps <= 4 ? p.taps : 0;
    if (act == XFTHIP_BF16) {
        if (form == 2) launch(unit_filter_tiled_kernel<true, 2>, pairs);
        else if (form == 3) launch(unit_filter_tiled_kernel<true, 3>, pairs);
        else if (form == 4) launch(unit_filter_tiled_kernel<true, 4>, pairs);
        else launch(unit_filter_kernel<true>, grid);
    } else {
        if (form == 2) launch(unit_filter_tiled_kernel<false, 2>, pairs);
        else if (form == 3) launch(unit_filter_tiled_kernel<false, 3>, pairs);
        else if (form == 4) launch(unit_filter_tiled_kernel<false, 4>, pairs);
        else launch(unit_filter_kernel<false>, grid);
    }
    XFT_CHECK_HIP(hipGetLastError());
    return conv_tail(act, v, x, L.in_ld, C, L.s.taps, b.conv_state, st);
}

int unit_scan(int act, const PlanLayer &L, const StepView &v, const UnitBuffers &b, hipStream_t st) {
    const int C = L.channels();
    const size_t esz = act == XFTHIP_BF16 ? 2 : 4;
    const UnitParams p = {v, b.u, b.gates, L.gate_bias, L.lambda, (const char *)b.in + (size_t)L.in_col * esz, L.in_ld, (char *)b.out + (size_t)L.out_col * esz, L.out_ld,
            C, L.D, L.mix_scale, b.state, (float2 *)b.carry};
    const dim3 grid((C + 255) / 256, (v.longest + kChunk - 1) / kChunk, v.B);
    if (act == XFTHIP_BF16) {
        if (v.longest > kChunk) hipLaunchKernelGGL((unit_scan_kernel<true, true>), grid, dim3(256), 0, st, p);
        hipLaunchKernelGGL((unit_scan_kernel<true, false>), grid, dim3(256), 0, st, p);
    } else {
        if (v.longest > kChunk) hipLaunchKernelGGL((unit_scan_kernel<false, true>), grid, dim3(256), 0, st, p);
        hipLaunchKernelGGL((unit_scan_kernel<false, false>), grid, dim3(256), 0, st, p);
    }
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

} // namespace xfthip
