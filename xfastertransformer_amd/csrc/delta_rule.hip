// The gated delta-rule recurrence of layer plans: short convolutions, unit norms, decays and step sizes (delta_prepare), the
// walk over the tokens with the state in registers (delta_scan), the gated per-head norm behind it (delta_output).
// Everything between the projections' outputs and the output projection's input is fp32.
#include "plan.h"

namespace xfthip {

namespace {

__device__ inline float wave_total(float v) {
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off, 64);
    return v;
}

struct PrepParams {
    StepView v;
    DeltaBuffers b;
    const float *conv, *decay, *dt_bias;
    int H, KH, KD, VD, taps, ld, channels, beta_col, gcols;
    float qscale;
};

// One wave a (token, head): its value channels, decay and step size, and (heads below KH) the query and key channels of
// key head `head`.  A channel is touched by one lane of one wave only, so that a sequence's single new token can shift the
// convolution's inputs in place; longer segments leave that to conv_tail_kernel.
template <bool BF16>
__global__ __launch_bounds__(256) void delta_prepare_kernel(PrepParams p) {
    const int lane = threadIdx.x & 63, t = blockIdx.x, head = blockIdx.y * 4 + (threadIdx.x >> 6);
    if (head >= p.H) return;
    constexpr int DT = BF16 ? XFTHIP_BF16 : XFTHIP_F32;
    const int seg = p.v.tok_seg[t], pos = p.v.tok_pos[t];
    const int off = p.v.seg_off[seg], row = p.v.seg_row[seg];
    const bool alone = p.v.seg_len[seg] == 1;
    const int local = t - off;
    const size_t hist = (size_t)row * (p.taps - 1) * p.channels;
    auto conv = [&](int ch) {
        float acc = 0.0f;
        for (int j = 0; j < p.taps; ++j) {
            const int back = p.taps - 1 - j;
            if (pos < back) continue;
            const float in = local >= back ? load_as_f32(p.b.in, DT, (size_t)(t - back) * p.ld + ch)
                                           : load_as_f32(p.b.conv_state, DT, hist + (size_t)(p.taps - 1 + local - back) * p.channels + ch);
            acc = fmaf(p.conv[(size_t)ch * p.taps + j], in, acc);
        }
        if (alone) {
            for (int s = 0; s + 1 < p.taps - 1; ++s)
                store_from_f32(p.b.conv_state, DT, hist + (size_t)s * p.channels + ch, load_as_f32(p.b.conv_state, DT, hist + (size_t)(s + 1) * p.channels + ch));
            if (p.taps > 1)
                store_from_f32(p.b.conv_state, DT, hist + (size_t)(p.taps - 2) * p.channels + ch, load_as_f32(p.b.in, DT, (size_t)t * p.ld + ch));
        }
        return acc / (1.0f + expf(-acc));
    };
    if (head < p.KH) {
        float q[4], k[4], sq = 0.0f, sk = 0.0f, dot = 0.0f;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int c = i * 64 + lane;
            q[i] = k[i] = 0.0f;
            if (c < p.KD) {
                q[i] = conv(head * p.KD + c);
                k[i] = conv((p.KH + head) * p.KD + c);
            }
            sq = fmaf(q[i], q[i], sq), sk = fmaf(k[i], k[i], sk);
        }
        sq = 1.0f / sqrtf(wave_total(sq) + 1e-6f) * p.qscale;
        sk = 1.0f / sqrtf(wave_total(sk) + 1e-6f);
        const size_t at = ((size_t)t * p.KH + head) * p.KD;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int c = i * 64 + lane;
            q[i] *= sq, k[i] *= sk;
            dot = fmaf(q[i], k[i], dot);
            if (c < p.KD) p.b.q[at + c] = q[i], p.b.k[at + c] = k[i];
        }
        dot = wave_total(dot);
        if (lane == 0) p.b.qk[(size_t)t * p.KH + head] = dot;
    }
    for (int c = lane; c < p.VD; c += 64) p.b.v[((size_t)t * p.H + head) * p.VD + c] = conv(2 * p.KH * p.KD + head * p.VD + c);
    const float a = p.decay[head];
    for (int c = lane; c < p.KD; c += 64) {
        const float x = p.b.gates[(size_t)t * 2 * p.gcols + head * p.KD + c] + p.dt_bias[head * p.KD + c];
        const float sp = x > 20.0f ? x : log1pf(expf(x));
        p.b.g[((size_t)t * p.H + head) * p.KD + c] = expf(-a * sp);
    }
    if (lane == 0) p.b.beta[(size_t)t * p.H + head] = 1.0f / (1.0f + expf(-load_as_f32(p.b.in, DT, (size_t)t * p.ld + p.beta_col + head)));
}

// the last taps - 1 inputs of a segment of several tokens; one thread a channel
template <bool BF16>
__global__ __launch_bounds__(256) void conv_tail_kernel(PrepParams p) {
    constexpr int DT = BF16 ? XFTHIP_BF16 : XFTHIP_F32;
    const int seg = blockIdx.y, n = p.v.seg_len[seg], ch = blockIdx.x * 256 + threadIdx.x;
    if (n <= 1 || ch >= p.channels) return;
    const size_t hist = (size_t)p.v.seg_row[seg] * (p.taps - 1) * p.channels;
    const int off = p.v.seg_off[seg];
    for (int s = 0; s < p.taps - 1; ++s) { // ascending: slot s is read (as a later source) only by slots below it
        const int from = n - (p.taps - 1) + s;
        const float x = from >= 0 ? load_as_f32(p.b.in, DT, (size_t)(off + from) * p.ld + ch)
                                  : load_as_f32(p.b.conv_state, DT, hist + (size_t)(s + n) * p.channels + ch);
        store_from_f32(p.b.conv_state, DT, hist + (size_t)s * p.channels + ch, x);
    }
}

template <int CTRL>
__device__ inline float dpp_add(float v) {
    return v + __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xF, 0xF, true));
}
// sum over aligned groups of L lanes, the same in all of them
template <int L>
__device__ inline float group_sum(float v) {
    v = dpp_add<0xB1>(v); // quad_perm 1 0 3 2
    v = dpp_add<0x4E>(v); // quad_perm 2 3 0 1
    if constexpr (L >= 8) v = dpp_add<0x141>(v); // row_half_mirror
    if constexpr (L >= 16) v = dpp_add<0x140>(v); // row_mirror
    if constexpr (L >= 32) v += __shfl_xor(v, 16, 64);
    return v;
}

struct ScanParams {
    StepView v;
    DeltaBuffers b;
    int H, KH, VD;
};

// The state's columns (value channels) do not interact: a column is held by L = KD / 8 lanes, 8 key rows each.  With
// S' = g S the step is a = S'^T k, b = S'^T q, u = beta (v - a), S = S' + k u^T, o = b + (q . k) u: both sums over the key
// rows run side by side and the read-out needs none of its own.  q, k, g of CT tokens are staged in LDS, the next CT on
// their way through registers.  grid (segments, heads, column groups of 256 / L).
template <int L>
__global__ __launch_bounds__(256) void delta_scan_kernel(ScanParams p) {
    constexpr int KD = 8 * L, COLS = 256 / L, CT = L == 32 ? 8 : 16; // CT: tokens staged in LDS at a time
    constexpr int CHUNK4 = CT * KD / 4; // float4 of one array and chunk
    constexpr int PER = (3 * CHUNK4 + 255) / 256, PERV = (CT * COLS + 255) / 256;
    __shared__ float lds[2][3 * CT * KD];
    __shared__ float vlds[2][CT * COLS];
    __shared__ float sc[2][2 * CT];
    __shared__ float olds[CT * COLS];
    const int seg = blockIdx.x, head = blockIdx.y, kvh = head / (p.H / p.KH);
    const int n = p.v.seg_len[seg], off = p.v.seg_off[seg];
    const int li = threadIdx.x % L, lc = threadIdx.x / L;
    const int col0 = blockIdx.z * COLS, col = col0 + lc;
    const bool own = col < p.VD;
    float *state = p.b.state + (((size_t)p.v.seg_row[seg] * p.H + head) * p.VD + (own ? col : 0)) * KD;
    f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = s0;
    if (p.v.seg_pos[seg] > 0) s0 = *(const f32x4 *)(state + 4 * li), s1 = *(const f32x4 *)(state + 4 * (L + li));

    f32x4 stage[PER];
    float vstage[PERV], cstage = 0.0f;
    auto fetch = [&](int c0) {
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = i * 256 + threadIdx.x;
            const int arr = e / CHUNK4, r = e % CHUNK4, tok = r / (KD / 4), d = (r % (KD / 4)) * 4;
            const int t = off + (c0 + tok < n ? c0 + tok : n - 1);
            if (e < 3 * CHUNK4) {
                const float *src = arr == 2 ? p.b.g + ((size_t)t * p.H + head) * KD : (arr ? p.b.k : p.b.q) + ((size_t)t * p.KH + kvh) * KD;
                stage[i] = *(const f32x4 *)(src + d);
            }
        }
#pragma unroll
        for (int i = 0; i < PERV; ++i) {
            const int e = i * 256 + threadIdx.x, tok = e / COLS, c = col0 + e % COLS;
            const int t = off + (c0 + tok < n ? c0 + tok : n - 1);
            if (e < CT * COLS) vstage[i] = p.b.v[((size_t)t * p.H + head) * p.VD + (c < p.VD ? c : p.VD - 1)];
        }
        if (threadIdx.x < 2 * CT) {
            const int tok = threadIdx.x % CT, t = off + (c0 + tok < n ? c0 + tok : n - 1);
            cstage = threadIdx.x < CT ? p.b.beta[(size_t)t * p.H + head] : p.b.qk[(size_t)t * p.KH + kvh];
        }
    };
    auto stash = [&](int buf) {
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = i * 256 + threadIdx.x;
            if (e < 3 * CHUNK4) *(f32x4 *)(&lds[buf][4 * e]) = stage[i];
        }
#pragma unroll
        for (int i = 0; i < PERV; ++i) {
            const int e = i * 256 + threadIdx.x;
            if (e < CT * COLS) vlds[buf][e] = vstage[i];
        }
        if (threadIdx.x < 2 * CT) sc[buf][threadIdx.x] = cstage;
    };
    fetch(0);
    stash(0);
    __syncthreads();
    int buf = 0;
    for (int c0 = 0; c0 < n; c0 += CT, buf ^= 1) {
        const int m = n - c0 < CT ? n - c0 : CT;
        if (c0 + CT < n) fetch(c0 + CT);
        const float *lq = lds[buf] + 4 * li, *lk = lq + CT * KD, *lg = lk + CT * KD;
        for (int i = 0; i < m; ++i) {
            const f32x4 q0 = *(const f32x4 *)(lq + i * KD), q1 = *(const f32x4 *)(lq + i * KD + 4 * L);
            const f32x4 k0 = *(const f32x4 *)(lk + i * KD), k1 = *(const f32x4 *)(lk + i * KD + 4 * L);
            const f32x4 g0 = *(const f32x4 *)(lg + i * KD), g1 = *(const f32x4 *)(lg + i * KD + 4 * L);
            const float vv = vlds[buf][i * COLS + lc], beta = sc[buf][i], qk = sc[buf][CT + i];
            float a = 0.0f, b = 0.0f;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                s0[r] *= g0[r], s1[r] *= g1[r];
                a = fmaf(k0[r], s0[r], a), b = fmaf(q0[r], s0[r], b);
            }
#pragma unroll
            for (int r = 0; r < 4; ++r) a = fmaf(k1[r], s1[r], a), b = fmaf(q1[r], s1[r], b);
            a = group_sum<L>(a), b = group_sum<L>(b);
            const float u = beta * (vv - a);
#pragma unroll
            for (int r = 0; r < 4; ++r) s0[r] = fmaf(k0[r], u, s0[r]), s1[r] = fmaf(k1[r], u, s1[r]);
            if (li == 0) olds[i * COLS + lc] = fmaf(qk, u, b);
        }
        if (c0 + CT < n) stash(buf ^ 1); // (the other buffer was last read before the barrier below, one chunk ago)
        __syncthreads();
        for (int e = threadIdx.x; e < m * COLS; e += 256) {
            const int c = col0 + e % COLS;
            if (c < p.VD) p.b.o[((size_t)(off + c0 + e / COLS) * p.H + head) * p.VD + c] = olds[e];
        }
        __syncthreads();
    }
    if (own) *(f32x4 *)(state + 4 * li) = s0, *(f32x4 *)(state + 4 * (L + li)) = s1;
}

struct OutParams {
    const float *o, *gates, *norm;
    void *on;
    int H, VD, vdim, gcols, T;
    float eps;
};

// per-head RMS norm times the sigmoid gate; one wave a (token, head)
template <bool BF16>
__global__ __launch_bounds__(256) void delta_output_kernel(OutParams p) {
    const int lane = threadIdx.x & 63;
    const size_t idx = (size_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (idx >= (size_t)p.T * p.H) return;
    const int t = (int)(idx / p.H), head = (int)(idx % p.H);
    const float *o = p.o + idx * p.VD;
    const float *gate = p.gates + (size_t)t * 2 * p.gcols + p.gcols + head * p.VD;
    float sq = 0.0f;
    for (int c = lane; c < p.VD; c += 64) sq = fmaf(o[c], o[c], sq);
    const float r = 1.0f / sqrtf(wave_total(sq) / (float)p.vdim + p.eps);
    for (int c = lane; c < p.VD; c += 64)
        store_from_f32(p.on, BF16 ? XFTHIP_BF16 : XFTHIP_F32, idx * p.VD + c, o[c] * r * p.norm[c] / (1.0f + expf(-gate[c])));
}

PrepParams prep_params(const PlanLayer &L, const StepView &v, const DeltaBuffers &b) {
    PrepParams p;
    p.v = v, p.b = b;
    p.conv = L.conv, p.decay = L.decay, p.dt_bias = L.dt_bias;
    p.H = L.s.heads, p.KH = L.s.kv_heads, p.KD = L.KD, p.VD = L.VD, p.taps = L.s.taps;
    p.ld = L.row_in(), p.channels = L.channels(), p.beta_col = L.channels(), p.gcols = L.gcols;
    p.qscale = 1.0f / sqrtf((float)L.s.dim);
    return p;
}

} // namespace

int delta_prepare(int act, const PlanLayer &L, const StepView &v, const DeltaBuffers &b, hipStream_t st) {
    const PrepParams p = prep_params(L, v, b);
    const dim3 grid(v.T, (p.H + 3) / 4), tail((p.channels + 255) / 256, v.B);
    const bool long_segments = v.longest > 1 && p.taps > 1;
    if (act == XFTHIP_BF16) {
        hipLaunchKernelGGL(delta_prepare_kernel<true>, grid, dim3(256), 0, st, p);
        if (long_segments) hipLaunchKernelGGL(conv_tail_kernel<true>, tail, dim3(256), 0, st, p);
    } else {
        hipLaunchKernelGGL(delta_prepare_kernel<false>, grid, dim3(256), 0, st, p);
        if (long_segments) hipLaunchKernelGGL(conv_tail_kernel<false>, tail, dim3(256), 0, st, p);
    }
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

int delta_scan(const PlanLayer &L, const StepView &v, const DeltaBuffers &b, hipStream_t st) {
    ScanParams p;
    p.v = v, p.b = b, p.H = L.s.heads, p.KH = L.s.kv_heads, p.VD = L.VD;
    const int lanes = L.KD / 8, cols = 256 / lanes;
    const dim3 grid(v.B, p.H, (L.VD + cols - 1) / cols);
    switch (lanes) {
        case 4: hipLaunchKernelGGL(delta_scan_kernel<4>, grid, dim3(256), 0, st, p); break;
        case 8: hipLaunchKernelGGL(delta_scan_kernel<8>, grid, dim3(256), 0, st, p); break;
        case 16: hipLaunchKernelGGL(delta_scan_kernel<16>, grid, dim3(256), 0, st, p); break;
        case 32: hipLaunchKernelGGL(delta_scan_kernel<32>, grid, dim3(256), 0, st, p); break;
        default: set_error("delta_scan: key dimension %d of a head is above 256", L.s.dim); return 2;
    }
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

int delta_output(int act, const PlanLayer &L, const StepView &v, const DeltaBuffers &b, float eps, hipStream_t st) {
    const OutParams p = {b.o, b.gates, L.out_norm, b.on, L.s.heads, L.VD, L.s.vdim, L.gcols, v.T, eps};
    const unsigned blocks = (unsigned)(((size_t)v.T * L.s.heads + 3) / 4);
    if (act == XFTHIP_BF16)
        hipLaunchKernelGGL(delta_output_kernel<true>, dim3(blocks), dim3(256), 0, st, p);
    else
        hipLaunchKernelGGL(delta_output_kernel<false>, dim3(blocks), dim3(256), 0, st, p);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

} // namespace xfthip
