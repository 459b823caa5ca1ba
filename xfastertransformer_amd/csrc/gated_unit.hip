// The gated linear recurrence of layer plans: a causal filter a channel (unit_filter), the products of both gates (tile_gemm, block by
// block), and S = a S + sqrt(1 - a^2) i u with a = exp(-8 r softplus(lambda)), times gelu(y) (unit_scan).  Channels do not interact.
// Behind the filter everything is fp32.
#include "plan_dev.h"

namespace xfthip {

namespace {

constexpr int kFilterTokens = 16; // tokens a thread of the filter walks
constexpr int kChunk = 64; // tokens a thread of the scan walks

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

// a and b of S = a S + b
__device__ inline float2 recurrence(float r, float i, float u, float lambda) {
    const float log_a = -lambda / (1.0f + expf(-r));
    return make_float2(expf(log_a), sqrtf(-expm1f(2.0f * log_a)) * u / (1.0f + expf(-i)));
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
    auto at = [&](int i) {
        const float *g = p.gates + (size_t)(off + i) * gpitch + gc;
        return recurrence(g[0] + rb, g[p.D] + ib, ldact<BF16>(p.u, (size_t)(off + i) * p.channels + ch), lambda);
    };
    if constexpr (FIRST) {
        float a = 1.0f, s = 0.0f;
#pragma unroll 4
        for (int i = i0; i < end; ++i) {
            const float2 x = at(i);
            a *= x.x, s = fmaf(x.x, s, x.y);
        }
        carry[(size_t)(blockIdx.y + 1) * p.channels] = make_float2(a, s);
        if (blockIdx.y == 0) carry[0] = make_float2(0.0f, p.v.seg_pos[seg] > 0 ? *state : 0.0f);
        return;
    }
    float s = 0.0f;
    if (n <= kChunk) {
        if (p.v.seg_pos[seg] > 0) s = *state;
    } else {
        for (int c = 0; c <= (int)blockIdx.y; ++c) {
            const float2 x = carry[(size_t)c * p.channels];
            s = fmaf(x.x, s, x.y);
        }
    }
#pragma unroll 4
    for (int i = i0; i < end; ++i) {
        const float2 x = at(i);
        s = fmaf(x.x, s, x.y);
        const float y = ldact<BF16>(p.y, (size_t)(off + i) * p.ld + ch);
        stact<BF16>(p.out, (size_t)(off + i) * p.out_ld + ch, s * gelu_tanh(y) * p.mul);
    }
    if (end == n) *state = s;
}

} // namespace

size_t unit_carry_floats(const PlanLayer &L, size_t tokens, size_t segments) { return (tokens / kChunk + 2 * segments + 2) * L.channels() * 2; }

int unit_filter(int act, const PlanLayer &L, const StepView &v, const UnitBuffers &b, hipStream_t st) {
    const int C = L.channels();
    const void *x = (const char *)b.in + (size_t)(L.in_col + C) * (act == XFTHIP_BF16 ? 2 : 4);
    const FilterParams p = {v, x, L.in_ld, C, L.s.taps, L.conv, L.conv_bias, b.u, b.conv_state};
    const dim3 grid((C + 255) / 256, (v.longest + kFilterTokens - 1) / kFilterTokens, v.B);
    if (act == XFTHIP_BF16) hipLaunchKernelGGL(unit_filter_kernel<true>, grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL(unit_filter_kernel<false>, grid, dim3(256), 0, st, p);
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
