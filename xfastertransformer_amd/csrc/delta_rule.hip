// The gated delta-rule recurrence of layer plans: short convolutions, unit norms, decays and step sizes (delta_prepare), the
// walk over the tokens with the state in registers (delta_scan), the gated per-head norm behind it (delta_output).
// Everything between the projections' outputs and the output projection's input is fp32.
#include "plan_dev.h"

namespace xfthip {

namespace {

template <bool BF16>
__device__ inline float ldb(const void *p, size_t i) {
    if constexpr (BF16) return bf16_to_f32(((const uint16_t *)p)[i]);
    else return ((const float *)p)[i];
}

struct PrepParams {
    StepView v;
    DeltaBuffers b;
    const float *conv, *decay, *dt_bias;
    int H, KH, KD, VD, taps, ld, channels, beta_col, decay_col, gcols; // decay_col: one decay a head, in the row (or -1)
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
    if (p.decay_col >= 0) {
        const float x = load_as_f32(p.b.in, DT, (size_t)t * p.ld + p.decay_col + head) + p.dt_bias[head];
        if (lane == 0) p.b.g[(size_t)t * p.H + head] = expf(-a * (x > 20.0f ? x : log1pf(expf(x))));
    }
    for (int c = lane; c < p.KD && p.decay_col < 0; c += 64) {
        const float x = p.b.gates[(size_t)t * 2 * p.gcols + head * p.KD + c] + p.dt_bias[head * p.KD + c];
        const float sp = x > 20.0f ? x : log1pf(expf(x));
        p.b.g[((size_t)t * p.H + head) * p.KD + c] = expf(-a * sp);
    }
    if (lane == 0) p.b.beta[(size_t)t * p.H + head] = 1.0f / (1.0f + expf(-load_as_f32(p.b.in, DT, (size_t)t * p.ld + p.beta_col + head)));
}

// The same for the usual shapes (TAPS taps, head widths of at most 256): a wave walks TT consecutive tokens of one segment and
// head, two neighbouring channels a lane, the convolutions' last inputs in registers - every input is read once and every
// result leaves as a pair.  grid (token tiles of a segment, ceil(heads / 4), segments)
constexpr int kPrepTokens = 8;

template <bool BF16, int TAPS, int J> // J: turns of 128 channels that cover a head's width
__global__ __launch_bounds__(256) void delta_prepare_tiled_kernel(PrepParams p) {
    const int lane = threadIdx.x & 63, head = blockIdx.y * 4 + (threadIdx.x >> 6), seg = blockIdx.z;
    const int n = p.v.seg_len[seg], i0 = blockIdx.x * kPrepTokens;
    if (head >= p.H || i0 >= n) return;
    const int off = p.v.seg_off[seg], row = p.v.seg_row[seg], start = p.v.seg_pos[seg];
    const int cnt = n - i0 < kPrepTokens ? n - i0 : kPrepTokens;
    const bool qk_head = head < p.KH;
    const size_t hist = (size_t)row * (TAPS - 1) * p.channels;
    const int vbase = 2 * p.KH * p.KD + head * p.VD;
    // input of channel pair c at local index i (negative: what earlier steps left; before the sequence's start: zero)
    auto input = [&](int c, int i) {
        if (start + i < 0) return make_float2(0.0f, 0.0f);
        return i >= 0 ? load2<BF16>(p.b.in, (size_t)(off + i) * p.ld + c) : load2<BF16>(p.b.conv_state, hist + (size_t)(TAPS - 1 + i) * p.channels + c);
    };
    struct Window {
        float2 w[TAPS]; // filter of either channel, tap by tap
        float2 x[TAPS > 1 ? TAPS - 1 : 1];
    };
    Window q[J], k[J], v[J];
    auto open = [&](Window &win, int c) {
#pragma unroll
        for (int t = 0; t < TAPS; ++t) win.w[t] = make_float2(p.conv[(size_t)c * TAPS + t], p.conv[(size_t)(c + 1) * TAPS + t]);
#pragma unroll
        for (int t = 0; t < TAPS - 1; ++t) win.x[t] = input(c, i0 - (TAPS - 1) + t);
    };
    auto advance = [&](Window &win, float2 in) { // silu of the filtered inputs; the window moves on by one token
        float2 a = make_float2(0.0f, 0.0f);
#pragma unroll
        for (int t = 0; t < TAPS - 1; ++t) a.x = fmaf(win.w[t].x, win.x[t].x, a.x), a.y = fmaf(win.w[t].y, win.x[t].y, a.y);
        a.x = fmaf(win.w[TAPS - 1].x, in.x, a.x), a.y = fmaf(win.w[TAPS - 1].y, in.y, a.y);
#pragma unroll
        for (int t = 0; t + 1 < TAPS - 1; ++t) win.x[t] = win.x[t + 1];
        if constexpr (TAPS > 1) win.x[TAPS - 2] = in;
        return make_float2(silu_of<BF16>(a.x), silu_of<BF16>(a.y));
    };
    float2 dtb[J];
#pragma unroll
    for (int j = 0; j < J; ++j) {
        const int c = j * 128 + lane * 2;
        if (qk_head && c < p.KD) open(q[j], head * p.KD + c), open(k[j], (p.KH + head) * p.KD + c);
        if (c < p.VD) open(v[j], vbase + c);
        dtb[j] = c < p.KD && p.decay_col < 0 ? *(const float2 *)(p.dt_bias + head * p.KD + c) : make_float2(0.0f, 0.0f);
    }
    const float decay = p.decay[head], head_dt = p.decay_col >= 0 ? p.dt_bias[head] : 0.0f;
    float2 nq[J], nk[J], nv[J], ng[J]; // the next token's values, requested a token ahead
    float nb = 0.0f, nd = 0.0f;
    auto request = [&](int i) {
        const int t = off + i;
        const size_t in_row = (size_t)t * p.ld;
#pragma unroll
        for (int j = 0; j < J; ++j) {
            const int c = j * 128 + lane * 2;
            nq[j] = nk[j] = nv[j] = ng[j] = make_float2(0.0f, 0.0f);
            if (qk_head && c < p.KD) nq[j] = load2<BF16>(p.b.in, in_row + head * p.KD + c), nk[j] = load2<BF16>(p.b.in, in_row + (p.KH + head) * p.KD + c);
            if (c < p.VD) nv[j] = load2<BF16>(p.b.in, in_row + vbase + c);
            if (c < p.KD && p.decay_col < 0) ng[j] = *(const float2 *)(p.b.gates + (size_t)t * 2 * p.gcols + head * p.KD + c);
        }
        nb = ldb<BF16>(p.b.in, in_row + p.beta_col + head);
        if (p.decay_col >= 0) nd = ldb<BF16>(p.b.in, in_row + p.decay_col + head);
    };
    request(i0);
    for (int i = i0; i < i0 + cnt; ++i) {
        const int t = off + i;
        float2 xq[J], xk[J], xv[J], xg[J];
#pragma unroll
        for (int j = 0; j < J; ++j) xq[j] = nq[j], xk[j] = nk[j], xv[j] = nv[j], xg[j] = ng[j];
        const float bl = nb, dl = nd;
        if (i + 1 < i0 + cnt) request(i + 1);
        float sq = 0.0f, sk = 0.0f, dot = 0.0f;
#pragma unroll
        for (int j = 0; j < J; ++j) {
            const int c = j * 128 + lane * 2;
            if (qk_head && c < p.KD) {
                xq[j] = advance(q[j], xq[j]), xk[j] = advance(k[j], xk[j]);
                sq = fmaf(xq[j].x, xq[j].x, fmaf(xq[j].y, xq[j].y, sq));
                sk = fmaf(xk[j].x, xk[j].x, fmaf(xk[j].y, xk[j].y, sk));
                dot = fmaf(xq[j].x, xk[j].x, fmaf(xq[j].y, xk[j].y, dot));
            }
            if (c < p.VD) *(float2 *)(p.b.v + ((size_t)t * p.H + head) * p.VD + c) = advance(v[j], xv[j]);
            if (c < p.KD && p.decay_col < 0) {
                *(float2 *)(p.b.g + ((size_t)t * p.H + head) * p.KD + c) = make_float2(exp_of<BF16>(-decay * softplus_of<BF16>(xg[j].x + dtb[j].x)),
                        exp_of<BF16>(-decay * softplus_of<BF16>(xg[j].y + dtb[j].y)));
            }
        }
        if (qk_head) { // (the same for the whole wave)
            sq = 1.0f / sqrtf(wave_total(sq) + 1e-6f) * p.qscale, sk = 1.0f / sqrtf(wave_total(sk) + 1e-6f);
            dot = wave_total(dot) * sq * sk;
            const size_t at = ((size_t)t * p.KH + head) * p.KD;
#pragma unroll
            for (int j = 0; j < J; ++j) {
                const int c = j * 128 + lane * 2;
                if (c < p.KD) {
                    *(float2 *)(p.b.q + at + c) = make_float2(xq[j].x * sq, xq[j].y * sq);
                    *(float2 *)(p.b.k + at + c) = make_float2(xk[j].x * sk, xk[j].y * sk);
                }
            }
            if (lane == 0) p.b.qk[(size_t)t * p.KH + head] = dot;
        }
        if (lane == 0) {
            p.b.beta[(size_t)t * p.H + head] = sigmoid_of<BF16>(bl);
            if (p.decay_col >= 0) p.b.g[(size_t)t * p.H + head] = exp_of<BF16>(-decay * softplus_of<BF16>(dl + head_dt));
        }
    }
    if (n == 1 && TAPS > 1) { // a single new token: nobody else reads these channels of the slot
        auto keep = [&](const Window &win, int c) {
#pragma unroll
            for (int t = 0; t < TAPS - 1; ++t) store2<BF16>(p.b.conv_state, hist + (size_t)t * p.channels + c, win.x[t]);
        };
#pragma unroll
        for (int j = 0; j < J; ++j) {
            const int c = j * 128 + lane * 2;
            if (qk_head && c < p.KD) keep(q[j], head * p.KD + c), keep(k[j], (p.KH + head) * p.KD + c);
            if (c < p.VD) keep(v[j], vbase + c);
        }
    }
}

struct TailParams {
    StepView v;
    const void *in;
    int ld, channels, taps;
    void *conv_state;
};
// the last taps - 1 inputs of a segment of several tokens; one thread a channel
template <bool BF16>
__global__ __launch_bounds__(256) void conv_tail_kernel(TailParams p) {
    constexpr int DT = BF16 ? XFTHIP_BF16 : XFTHIP_F32;
    const int seg = blockIdx.y, n = p.v.seg_len[seg], ch = blockIdx.x * 256 + threadIdx.x;
    if (n <= 1 || ch >= p.channels) return;
    const size_t hist = (size_t)p.v.seg_row[seg] * (p.taps - 1) * p.channels;
    const int off = p.v.seg_off[seg];
    for (int s = 0; s < p.taps - 1; ++s) { // ascending: slot s is read (as a later source) only by slots below it
        const int from = n - (p.taps - 1) + s;
        const float x = from >= 0 ? load_as_f32(p.in, DT, (size_t)(off + from) * p.ld + ch)
                                  : load_as_f32(p.conv_state, DT, hist + (size_t)(s + n) * p.channels + ch);
        store_from_f32(p.conv_state, DT, hist + (size_t)s * p.channels + ch, x);
    }
}

struct ScanParams {
    StepView v;
    DeltaBuffers b;
    int H, KH, VD;
};

// The state's columns (value channels) do not interact.  L lanes hold C neighbouring columns, 4 RV key rows each (KD = 4 L RV).
// With S' = g S the step is a = S'^T k, b = S'^T q, u = beta (v - a), S = S' + k u^T, o = b + (q . k) u: both sums over the key
// rows run side by side and the read-out needs none of its own.  q, k, g of CT tokens are staged in LDS, the next CT on
// their way through registers.  grid (segments, heads, column groups of COLS).
// ONE: one decay a head, a scalar beside beta.
// One prompt of 32 heads is one wave a SIMD: the time is about 75 vector instructions a token and the latency of the
// reductions in them.  (KD = 128 as 32 lanes x 4 rows x 2 columns, half the LDS reads: 510 us for 2048 tokens against 440 as
// 16 x 8 x 1.)
template <int L, int RV, int C, bool ONE>
__global__ __launch_bounds__(256) void delta_scan_kernel(ScanParams p) {
    constexpr int KD = 4 * L * RV, GROUPS = 256 / L, COLS = GROUPS * C, CT = KD > 128 ? 8 : 16;
    constexpr int CHUNK4 = CT * KD / 4; // float4 of one array and chunk
    constexpr int ARRAYS = ONE ? 2 : 3, SCALARS = ONE ? 3 : 2; // q, k(, g); beta, q . k(, g)
    constexpr int PER = (ARRAYS * CHUNK4 + 255) / 256, PERV = (CT * COLS + 255) / 256;
    __shared__ float lds[2][ARRAYS * CT * KD];
    __shared__ float vlds[2][CT * COLS];
    __shared__ float sc[2][SCALARS * CT];
    __shared__ float olds[2][CT * COLS];
    const int seg = blockIdx.x, head = blockIdx.y, kvh = head / (p.H / p.KH);
    const int n = p.v.seg_len[seg], off = p.v.seg_off[seg];
    const int li = threadIdx.x % L, lc = threadIdx.x / L * C;
    const int col0 = blockIdx.z * COLS, col = col0 + lc;
    const bool own = col < p.VD; // (VD is a multiple of 32: C neighbouring columns are in it or not together)
    float *state = p.b.state + (((size_t)p.v.seg_row[seg] * p.H + head) * p.VD + (own ? col : 0)) * KD + 4 * li;
    f32x4 s[C][RV];
#pragma unroll
    for (int c = 0; c < C; ++c)
#pragma unroll
        for (int r = 0; r < RV; ++r) s[c][r] = p.v.seg_pos[seg] > 0 ? *(const f32x4 *)(state + c * KD + r * 4 * L) : f32x4 {0.f, 0.f, 0.f, 0.f};

    f32x4 stage[PER];
    float vstage[PERV], cstage = 0.0f;
    // (threads without a part fetch the last one: a load under a condition would be waited for before the next one goes out)
    auto fetch = [&](int c0) {
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int part = i * 256 + (int)threadIdx.x, e = part < ARRAYS * CHUNK4 ? part : ARRAYS * CHUNK4 - 1;
            const int arr = e / CHUNK4, r = e % CHUNK4, tok = r / (KD / 4), d = (r % (KD / 4)) * 4;
            const int t = off + (c0 + tok < n ? c0 + tok : n - 1);
            const float *src = arr == 2 ? p.b.g + ((size_t)t * p.H + head) * KD : (arr ? p.b.k : p.b.q) + ((size_t)t * p.KH + kvh) * KD;
            stage[i] = *(const f32x4 *)(src + d);
        }
#pragma unroll
        for (int i = 0; i < PERV; ++i) {
            const int part = i * 256 + (int)threadIdx.x, e = part < CT * COLS ? part : CT * COLS - 1, tok = e / COLS, c = col0 + e % COLS;
            const int t = off + (c0 + tok < n ? c0 + tok : n - 1);
            vstage[i] = p.b.v[((size_t)t * p.H + head) * p.VD + (c < p.VD ? c : p.VD - 1)];
        }
        const int tok = threadIdx.x % CT, t = off + (c0 + tok < n ? c0 + tok : n - 1);
        const float *scalar = threadIdx.x < CT ? p.b.beta + (size_t)t * p.H + head : threadIdx.x < 2 * CT || !ONE ? p.b.qk + (size_t)t * p.KH + kvh : p.b.g + (size_t)t * p.H + head;
        cstage = *scalar;
    };
    auto stash = [&](int buf) {
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = i * 256 + threadIdx.x;
            if (e < ARRAYS * CHUNK4) *(f32x4 *)(&lds[buf][4 * e]) = stage[i];
        }
#pragma unroll
        for (int i = 0; i < PERV; ++i) {
            const int e = i * 256 + threadIdx.x;
            if (e < CT * COLS) vlds[buf][e] = vstage[i];
        }
        if (threadIdx.x < SCALARS * CT) sc[buf][threadIdx.x] = cstage;
    };
#pragma unroll
    for (int c = 0; c < C; ++c)
#pragma unroll
        for (int r = 0; r < RV; ++r) arrived(s[c][r]);
    fetch(0);
    stash(0);
    __syncthreads();
    int buf = 0;
    for (int c0 = 0; c0 < n; c0 += CT, buf ^= 1) {
        const int m = n - c0 < CT ? n - c0 : CT;
        if (c0 + CT < n) fetch(c0 + CT);
        const float *lq = lds[buf] + 4 * li;
        struct Operands {
            f32x4 q[RV], k[RV], g[ONE ? 1 : RV];
            float v[C], beta, qk, fade;
        };
        auto read = [&](int i) {
            const float *q = lq + i * KD, *k = q + CT * KD, *g = k + CT * KD;
            Operands x;
#pragma unroll
            for (int r = 0; r < RV; ++r) {
                x.q[r] = *(const f32x4 *)(q + r * 4 * L), x.k[r] = *(const f32x4 *)(k + r * 4 * L);
                if constexpr (!ONE) x.g[r] = *(const f32x4 *)(g + r * 4 * L);
            }
#pragma unroll
            for (int c = 0; c < C; ++c) x.v[c] = vlds[buf][i * COLS + lc + c];
            x.beta = sc[buf][i], x.qk = sc[buf][CT + i];
            if constexpr (ONE) x.fade = sc[buf][2 * CT + i];
            return x;
        };
        // the operands of the next token are on their way from LDS while this one's sums go round
        auto token = [&](const Operands &x, int i) {
            float a[C], b[C], u[C];
#pragma unroll
            for (int c = 0; c < C; ++c) {
                a[c] = b[c] = 0.0f;
#pragma unroll
                for (int r = 0; r < RV; ++r)
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        if constexpr (ONE) s[c][r][e] *= x.fade;
                        else s[c][r][e] *= x.g[r][e];
                        a[c] = fmaf(x.k[r][e], s[c][r][e], a[c]), b[c] = fmaf(x.q[r][e], s[c][r][e], b[c]);
                    }
            }
#pragma unroll
            for (int c = 0; c < C; ++c) a[c] = group_sum<L>(a[c]), b[c] = group_sum<L>(b[c]);
#pragma unroll
            for (int c = 0; c < C; ++c) {
                u[c] = x.beta * (x.v[c] - a[c]);
#pragma unroll
                for (int r = 0; r < RV; ++r)
#pragma unroll
                    for (int e = 0; e < 4; ++e) s[c][r][e] = fmaf(x.k[r][e], u[c], s[c][r][e]);
            }
            if (li == 0) {
#pragma unroll
                for (int c = 0; c < C; ++c) olds[buf][i * COLS + lc + c] = fmaf(x.qk, u[c], b[c]);
            }
        };
        Operands even = read(0), odd;
        for (int i = 0; i < m; i += 2) {
            odd = read(i + 1 < m ? i + 1 : i);
            token(even, i);
            if (i + 1 >= m) break;
            even = read(i + 2 < m ? i + 2 : i + 1);
            token(odd, i + 1);
        }
        if (c0 + CT < n) stash(buf ^ 1); // (the other buffer, and the other results, were last read before or behind this barrier one chunk ago)
        __syncthreads();
        for (int e = threadIdx.x; e < m * COLS; e += 256) {
            const int c = col0 + e % COLS;
            if (c < p.VD) p.b.o[((size_t)(off + c0 + e / COLS) * p.H + head) * p.VD + c] = olds[buf][e];
        }
    }
    if (own) {
#pragma unroll
        for (int c = 0; c < C; ++c)
#pragma unroll
            for (int r = 0; r < RV; ++r) *(f32x4 *)(state + c * KD + r * 4 * L) = s[c][r];
    }
}

// The same step for segments of one token: nothing to stage, the kernel is a read and a write of the state.
template <int L, bool ONE>
__global__ __launch_bounds__(256) void delta_step_kernel(ScanParams p) {
    constexpr int KD = 8 * L, COLS = 256 / L;
    const int seg = blockIdx.x, head = blockIdx.y, kvh = head / (p.H / p.KH), t = p.v.seg_off[seg];
    const int li = threadIdx.x % L, col = blockIdx.z * COLS + threadIdx.x / L;
    if (col >= p.VD) return; // (whole groups of L lanes)
    float *state = p.b.state + (((size_t)p.v.seg_row[seg] * p.H + head) * p.VD + col) * KD;
    f32x4 s0 = *(const f32x4 *)(state + 4 * li), s1 = *(const f32x4 *)(state + 4 * (L + li));
    const float *q = p.b.q + ((size_t)t * p.KH + kvh) * KD + 4 * li, *k = p.b.k + ((size_t)t * p.KH + kvh) * KD + 4 * li;
    f32x4 g0, g1;
    if constexpr (ONE) {
        const float fade = p.b.g[(size_t)t * p.H + head];
        g0 = g1 = f32x4 {fade, fade, fade, fade};
    } else {
        const float *g = p.b.g + ((size_t)t * p.H + head) * KD + 4 * li;
        g0 = *(const f32x4 *)g, g1 = *(const f32x4 *)(g + 4 * L);
    }
    const f32x4 q0 = *(const f32x4 *)q, q1 = *(const f32x4 *)(q + 4 * L), k0 = *(const f32x4 *)k, k1 = *(const f32x4 *)(k + 4 * L);
    const float v = p.b.v[((size_t)t * p.H + head) * p.VD + col], beta = p.b.beta[(size_t)t * p.H + head], qk = p.b.qk[(size_t)t * p.KH + kvh];
    if (p.v.seg_pos[seg] == 0) s0 = s1 = f32x4 {0.f, 0.f, 0.f, 0.f};
    float a = 0.0f, b = 0.0f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        s0[r] *= g0[r], s1[r] *= g1[r];
        a = fmaf(k0[r], s0[r], a), b = fmaf(q0[r], s0[r], b);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) a = fmaf(k1[r], s1[r], a), b = fmaf(q1[r], s1[r], b);
    a = group_sum<L>(a), b = group_sum<L>(b);
    const float u = beta * (v - a);
#pragma unroll
    for (int r = 0; r < 4; ++r) s0[r] = fmaf(k0[r], u, s0[r]), s1[r] = fmaf(k1[r], u, s1[r]);
    *(f32x4 *)(state + 4 * li) = s0, *(f32x4 *)(state + 4 * (L + li)) = s1;
    if (li == 0) p.b.o[((size_t)t * p.H + head) * p.VD + col] = fmaf(qk, u, b);
}

struct OutParams {
    const float *o, *gates, *norm;
    const void *row_gate; // the gate in the rows of the input product (pitch ld), through a silu; or null
    int ld;
    void *out; // rows of pitch out_ld
    int out_ld;
    int H, VD, vdim, gcols, T;
    float eps, mul;
};

// per-head RMS norm times the gate; one wave a (token, head)
template <bool BF16>
__global__ __launch_bounds__(256) void delta_output_kernel(OutParams p) {
    const int lane = threadIdx.x & 63;
    const size_t idx = (size_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (idx >= (size_t)p.T * p.H) return;
    const int t = (int)(idx / p.H), head = (int)(idx % p.H);
    const float *o = p.o + idx * p.VD;
    const float *gate = p.gates + (size_t)t * 2 * p.gcols + p.gcols + head * p.VD;
    float sq = 0.0f;
    for (int c = lane * 2; c < p.VD; c += 128) {
        const float2 x = *(const float2 *)(o + c);
        sq = fmaf(x.x, x.x, fmaf(x.y, x.y, sq));
    }
    const float r = 1.0f / sqrtf(wave_total(sq) / (float)p.vdim + p.eps);
    const float f = r * p.mul;
    for (int c = lane * 2; c < p.VD; c += 128) {
        const float2 x = *(const float2 *)(o + c), w = *(const float2 *)(p.norm + c);
        float2 z;
        if (p.row_gate) {
            z = load2<BF16>(p.row_gate, (size_t)t * p.ld + head * p.VD + c);
            z.x = silu_of<BF16>(z.x), z.y = silu_of<BF16>(z.y);
        } else {
            z = *(const float2 *)(gate + c);
            z.x = sigmoid_of<BF16>(z.x), z.y = sigmoid_of<BF16>(z.y);
        }
        store2<BF16>(p.out, (size_t)t * p.out_ld + head * p.VD + c, make_float2(x.x * f * w.x * z.x, x.y * f * w.y * z.y));
    }
}

PrepParams prep_params(int act, const PlanLayer &L, const StepView &v, const DeltaBuffers &b) {
    PrepParams p;
    p.v = v, p.b = b;
    p.b.in = (char *)b.in + (size_t)L.in_col * (act == XFTHIP_BF16 ? 2 : 4);
    p.conv = L.conv, p.decay = L.decay, p.dt_bias = L.dt_bias;
    p.H = L.s.heads, p.KH = L.s.kv_heads, p.KD = L.KD, p.VD = L.VD, p.taps = L.s.taps;
    p.ld = L.in_ld, p.channels = L.channels(), p.beta_col = L.channels(), p.decay_col = L.head_decay() ? p.beta_col + L.beta_cols() : -1, p.gcols = L.gcols;
    p.qscale = 1.0f / sqrtf((float)L.s.dim);
    return p;
}

int launch_output(int act, const PlanLayer &L, int T, OutParams p, float eps, hipStream_t st) {
    p.out = (char *)p.out + (size_t)L.out_col * (act == XFTHIP_BF16 ? 2 : 4), p.out_ld = L.out_ld;
    p.H = L.s.heads, p.VD = L.VD, p.vdim = L.s.vdim, p.gcols = L.gcols, p.T = T, p.eps = eps, p.mul = L.mix_scale;
    const unsigned blocks = (unsigned)(((size_t)T * p.H + 3) / 4);
    if (act == XFTHIP_BF16) hipLaunchKernelGGL(delta_output_kernel<true>, dim3(blocks), dim3(256), 0, st, p);
    else hipLaunchKernelGGL(delta_output_kernel<false>, dim3(blocks), dim3(256), 0, st, p);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

} // namespace

int delta_prepare(int act, const PlanLayer &L, const StepView &v, const DeltaBuffers &b, hipStream_t st) {
    const PrepParams p = prep_params(act, L, v, b);
    const dim3 grid(v.T, (p.H + 3) / 4);
    const int width = p.KD > p.VD ? p.KD : p.VD;
    const bool tiled = p.taps >= 2 && p.taps <= 4 && width <= 256;
    if (tiled) {
        const dim3 tiles((v.longest + kPrepTokens - 1) / kPrepTokens, (p.H + 3) / 4, v.B);
        const int key = (act == XFTHIP_BF16 ? 0 : 10) + p.taps + (width > 128 ? 100 : 0);
        switch (key) {
            case 2: hipLaunchKernelGGL((delta_prepare_tiled_kernel<true, 2, 1>), tiles, dim3(256), 0, st, p); break;
            case 3: hipLaunchKernelGGL((delta_prepare_tiled_kernel<true, 3, 1>), tiles, dim3(256), 0, st, p); break;
            case 4: hipLaunchKernelGGL((delta_prepare_tiled_kernel<true, 4, 1>), tiles, dim3(256), 0, st, p); break;
            case 12: hipLaunchKernelGGL((delta_prepare_tiled_kernel<false, 2, 1>), tiles, dim3(256), 0, st, p); break;
            case 13: hipLaunchKernelGGL((delta_prepare_tiled_kernel<false, 3, 1>), tiles, dim3(256), 0, st, p); break;
            case 14: hipLaunchKernelGGL((delta_prepare_tiled_kernel<false, 4, 1>), tiles, dim3(256), 0, st, p); break;
            case 102: hipLaunchKernelGGL((delta_prepare_tiled_kernel<true, 2, 2>), tiles, dim3(256), 0, st, p); break;
            case 103: hipLaunchKernelGGL((delta_prepare_tiled_kernel<true, 3, 2>), tiles, dim3(256), 0, st, p); break;
            case 104: hipLaunchKernelGGL((delta_prepare_tiled_kernel<true, 4, 2>), tiles, dim3(256), 0, st, p); break;
            case 112: hipLaunchKernelGGL((delta_prepare_tiled_kernel<false, 2, 2>), tiles, dim3(256), 0, st, p); break;
            case 113: hipLaunchKernelGGL((delta_prepare_tiled_kernel<false, 3, 2>), tiles, dim3(256), 0, st, p); break;
            default: hipLaunchKernelGGL((delta_prepare_tiled_kernel<false, 4, 2>), tiles, dim3(256), 0, st, p); break;
        }
    }
    if (!tiled) {
        if (act == XFTHIP_BF16) hipLaunchKernelGGL(delta_prepare_kernel<true>, grid, dim3(256), 0, st, p);
        else hipLaunchKernelGGL(delta_prepare_kernel<false>, grid, dim3(256), 0, st, p);
    }
    XFT_CHECK_HIP(hipGetLastError());
    return conv_tail(act, v, p.b.in, p.ld, p.channels, p.taps, b.conv_state, st);
}

int conv_tail(int act, const StepView &v, const void *in, int ld, int channels, int taps, void *conv_state, hipStream_t st) {
    if (v.longest <= 1 || taps <= 1) return 0;
    const TailParams p = {v, in, ld, channels, taps, conv_state};
    const dim3 grid((channels + 255) / 256, v.B);
    if (act == XFTHIP_BF16) hipLaunchKernelGGL(conv_tail_kernel<true>, grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL(conv_tail_kernel<false>, grid, dim3(256), 0, st, p);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

int delta_scan(const PlanLayer &L, const StepView &v, const DeltaBuffers &b, hipStream_t st) {
    ScanParams p;
    p.v = v, p.b = b, p.H = L.s.heads, p.KH = L.s.kv_heads, p.VD = L.VD;
    const int lanes = L.KD / 8, cols = 256 / lanes;
    const bool one = L.head_decay();
    const dim3 grid(v.B, p.H, (L.VD + cols - 1) / cols);
    auto launch = [&](auto several, auto single) {
        if (one) hipLaunchKernelGGL(single, grid, dim3(256), 0, st, p);
        else hipLaunchKernelGGL(several, grid, dim3(256), 0, st, p);
    };
    const int key = (v.longest == 1 ? 0 : 1000) + L.KD; // (both forms: 256 / lanes columns a workgroup)
    switch (key) {
        case 32: launch(delta_step_kernel<4, false>, delta_step_kernel<4, true>); break;
        case 64: launch(delta_step_kernel<8, false>, delta_step_kernel<8, true>); break;
        case 128: launch(delta_step_kernel<16, false>, delta_step_kernel<16, true>); break;
        case 256: launch(delta_step_kernel<32, false>, delta_step_kernel<32, true>); break;
        case 1032: launch(delta_scan_kernel<4, 2, 1, false>, delta_scan_kernel<4, 2, 1, true>); break;
        case 1064: launch(delta_scan_kernel<8, 2, 1, false>, delta_scan_kernel<8, 2, 1, true>); break;
        case 1128: launch(delta_scan_kernel<16, 2, 1, false>, delta_scan_kernel<16, 2, 1, true>); break;
        case 1256: launch(delta_scan_kernel<32, 2, 1, false>, delta_scan_kernel<32, 2, 1, true>); break;
        default: set_error("delta_scan: key dimension %d of a head is above 256", L.s.dim); return 2;
    }
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

int delta_output(int act, const PlanLayer &L, const StepView &v, const DeltaBuffers &b, float eps, hipStream_t st) {
    if (L.silu_gate()) return gated_head_norm(act, L, v.T, b.o, b.in, b.out, eps, st);
    return launch_output(act, L, v.T, {b.o, b.gates, L.out_norm, nullptr, L.in_ld, b.out}, eps, st);
}

int gated_head_norm(int act, const PlanLayer &L, int T, const float *o, const void *in, void *out, float eps, hipStream_t st) {
    return launch_output(act, L, T, {o, nullptr, L.out_norm, (const char *)in + (size_t)L.out_gate_col() * (act == XFTHIP_BF16 ? 2 : 4), L.in_ld, out}, eps, st);
}

} // namespace xfthip
