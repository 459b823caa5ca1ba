// Gated linear attention of layer plans: per head S = diag(alpha) S + k v^T and o = S^T q, alpha a decay of every key channel, then the norm of
// every head and a silu gate.  Queries, keys and values are read from the rows of the input product, the decays come out of their product's
// epilogue; between those and the output projection's input everything is fp32.
#include "plan_dev.h"

namespace xfthip {

namespace {

struct LinearParams {
    StepView v;
    const void *in; // q | k | v of a row
    int ld;
    const float *alpha; // [T][H][KD]
    float *o; // [T][H][VD]
    float *state;
    int H, VD;
    float qscale;
    // single tokens: what follows the recurrence
    const void *gate; // in the rows
    const float *norm;
    void *out;
    int out_ld, vdim;
    float eps, mul;
};

// sums of two values over aligned groups of 32 lanes: of `a` in the first 16 of them, of `b` in the others
__device__ inline float two_sums(float a, float b) {
    const auto x = __builtin_amdgcn_permlane16_swap(f2u(a), f2u(b), false, false);
    return group_sum<16>(u2f(x[0]) + u2f(x[1]));
}

// A walk over a segment's tokens with the state in registers.  The state's columns (value channels) do not interact: L lanes hold C neighbouring
// columns, 4 RV key rows each (KD = 4 L RV).  A token is S = g S + k v and a sum over the key rows that nothing waits for.  q, k, g of
// CT tokens are staged in LDS, the next CT on their way through registers.  grid (segments, heads, column groups of COLS)
template <bool BF16, int L, int RV, int C>
__global__ __launch_bounds__(256) void linear_scan_kernel(LinearParams p) {
    constexpr int KD = 4 * L * RV, COLS = 256 / L * C, CT = KD > 128 ? 8 : 16;
    constexpr int QK8 = 2 * CT * KD / 8, G4 = CT * KD / 4; // groups of eight of q and k, float4 of the decays of a chunk
    constexpr int PERQ = (QK8 + 255) / 256, PERG = (G4 + 255) / 256, PERV = (CT * COLS + 255) / 256;
    __shared__ float lds[2][3 * CT * KD];
    __shared__ float vlds[2][CT * COLS];
    __shared__ float olds[2][CT * COLS];
    const int seg = blockIdx.x, head = blockIdx.y, n = p.v.seg_len[seg], off = p.v.seg_off[seg];
    const int li = threadIdx.x % L, lc = threadIdx.x / L * C, col0 = blockIdx.z * COLS, col = col0 + lc;
    const bool own = col < p.VD; // (VD is a multiple of 32: C neighbouring columns are in it or not together)
    float *state = p.state + (((size_t)p.v.seg_row[seg] * p.H + head) * p.VD + (own ? col : 0)) * KD + 4 * li;
    const int vcol = 2 * p.H * KD + head * p.VD;
    f32x4 s[C][RV];
#pragma unroll
    for (int c = 0; c < C; ++c)
#pragma unroll
        for (int r = 0; r < RV; ++r) s[c][r] = p.v.seg_pos[seg] > 0 ? *(const f32x4 *)(state + c * KD + r * 4 * L) : f32x4 {0.f, 0.f, 0.f, 0.f};

    constexpr int WORDS = BF16 ? 1 : 2; // of 16 bytes that hold eight activations
    u32x4 qk[PERQ][WORDS];
    f32x4 g[PERG];
    float vs[PERV];
    auto token_at = [&](int i) { return off + (i < n ? i : n - 1); };
    auto fetch = [&](int c0) {
#pragma unroll
        for (int i = 0; i < PERQ; ++i) {
            const int e = i * 256 + threadIdx.x, k = e / (QK8 / 2), r = e % (QK8 / 2);
            if (e >= QK8) continue;
            const size_t at = (size_t)token_at(c0 + r / (KD / 8)) * p.ld + (size_t)(k * p.H + head) * KD + r % (KD / 8) * 8;
            const u32x4 *src = (const u32x4 *)((const char *)p.in + at * (BF16 ? 2 : 4));
#pragma unroll
            for (int w = 0; w < WORDS; ++w) qk[i][w] = src[w];
        }
#pragma unroll
        for (int i = 0; i < PERG; ++i) {
            const int e = i * 256 + threadIdx.x;
            if (e < G4) g[i] = *(const f32x4 *)(p.alpha + ((size_t)token_at(c0 + e / (KD / 4)) * p.H + head) * KD + e % (KD / 4) * 4);
        }
#pragma unroll
        for (int i = 0; i < PERV; ++i) {
            const int e = i * 256 + threadIdx.x, c = col0 + e % COLS;
            if (e < CT * COLS) vs[i] = ldact<BF16>(p.in, (size_t)token_at(c0 + e / COLS) * p.ld + vcol + (c < p.VD ? c : p.VD - 1));
        }
    };
    auto stash = [&](int buf) {
#pragma unroll
        for (int i = 0; i < PERQ; ++i) {
            const int e = i * 256 + threadIdx.x;
            if (e >= QK8) continue;
            const float mul = e < QK8 / 2 ? p.qscale : 1.0f;
            float *dst = &lds[buf][8 * e];
            f32x4 lo, hi;
            if constexpr (BF16) {
#pragma unroll
                for (int k = 0; k < 2; ++k) {
                    lo[2 * k] = u2f(qk[i][0][k] << 16), lo[2 * k + 1] = u2f(qk[i][0][k] & 0xFFFF0000u);
                    hi[2 * k] = u2f(qk[i][0][2 + k] << 16), hi[2 * k + 1] = u2f(qk[i][0][2 + k] & 0xFFFF0000u);
                }
            } else {
                lo = __builtin_bit_cast(f32x4, qk[i][0]), hi = __builtin_bit_cast(f32x4, qk[i][WORDS - 1]);
            }
            *(f32x4 *)dst = lo * mul, *(f32x4 *)(dst + 4) = hi * mul;
        }
#pragma unroll
        for (int i = 0; i < PERG; ++i) {
            const int e = i * 256 + threadIdx.x;
            if (e < G4) *(f32x4 *)(&lds[buf][2 * CT * KD + 4 * e]) = g[i];
        }
#pragma unroll
        for (int i = 0; i < PERV; ++i) {
            const int e = i * 256 + threadIdx.x;
            if (e < CT * COLS) vlds[buf][e] = vs[i];
        }
    };
    fetch(0);
    stash(0);
    __syncthreads();
    int buf = 0;
    for (int c0 = 0; c0 < n; c0 += CT, buf ^= 1) {
        const int m = n - c0 < CT ? n - c0 : CT;
        if (c0 + CT < n) fetch(c0 + CT);
        struct Operands {
            f32x4 q[RV], k[RV], g[RV];
            float v[C];
        };
        auto read = [&](int i) {
            const float *q = lds[buf] + i * KD + 4 * li, *k = q + CT * KD, *a = k + CT * KD;
            Operands x;
#pragma unroll
            for (int r = 0; r < RV; ++r)
                x.q[r] = *(const f32x4 *)(q + r * 4 * L), x.k[r] = *(const f32x4 *)(k + r * 4 * L), x.g[r] = *(const f32x4 *)(a + r * 4 * L);
#pragma unroll
            for (int c = 0; c < C; ++c) x.v[c] = vlds[buf][i * COLS + lc + c];
            return x;
        };
        auto token = [&](const Operands &x, int i) {
            float o[C];
#pragma unroll
            for (int c = 0; c < C; ++c) {
                o[c] = 0.0f;
#pragma unroll
                for (int r = 0; r < RV; ++r)
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        s[c][r][e] = fmaf(x.g[r][e], s[c][r][e], x.k[r][e] * x.v[c]);
                        o[c] = fmaf(x.q[r][e], s[c][r][e], o[c]);
                    }
            }
            if constexpr (L == 32 && C == 2) {
                const float sum = two_sums(o[0], o[1]);
                if (li % 16 == 0) olds[buf][i * COLS + lc + li / 16] = sum;
            } else {
#pragma unroll
                for (int c = 0; c < C; ++c) o[c] = group_sum<L>(o[c]);
                if (li == 0) {
#pragma unroll
                    for (int c = 0; c < C; ++c) olds[buf][i * COLS + lc + c] = o[c];
                }
            }
        };
        // the operands of the next token are on their way from LDS while this one's sum goes round
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
            if (c < p.VD) p.o[((size_t)(off + c0 + e / COLS) * p.H + head) * p.VD + c] = olds[buf][e];
        }
    }
    if (own) {
#pragma unroll
        for (int c = 0; c < C; ++c)
#pragma unroll
            for (int r = 0; r < RV; ++r) *(f32x4 *)(state + c * KD + r * 4 * L) = s[c][r];
    }
}

// Segments of one token: a read and a write of a head's state, its norm and gate behind it.  L lanes a column, four key rows each.
// grid (heads, segments)
constexpr int kStepThreads = 512;
template <bool BF16, int L>
__global__ __launch_bounds__(kStepThreads) void linear_step_kernel(LinearParams p) {
    extern __shared__ float os[]; // [VD]
    constexpr int KD = 4 * L, COLS = kStepThreads / L, AHEAD = 4; // columns of a pass, passes whose loads go out together
    const int head = blockIdx.x, seg = blockIdx.y, t = p.v.seg_off[seg], li = threadIdx.x % L, lane = threadIdx.x & 63;
    const bool begins = p.v.seg_pos[seg] == 0;
    float *state = p.state + ((size_t)p.v.seg_row[seg] * p.H + head) * p.VD * KD + 4 * li;
    const size_t row = (size_t)t * p.ld;
    const float2 q0 = load2<BF16>(p.in, row + head * KD + 4 * li), q1 = load2<BF16>(p.in, row + head * KD + 4 * li + 2);
    const float2 k0 = load2<BF16>(p.in, row + (p.H + head) * KD + 4 * li), k1 = load2<BF16>(p.in, row + (p.H + head) * KD + 4 * li + 2);
    const f32x4 q = f32x4 {q0.x, q0.y, q1.x, q1.y} * p.qscale, k = {k0.x, k0.y, k1.x, k1.y};
    const f32x4 g = *(const f32x4 *)(p.alpha + ((size_t)t * p.H + head) * KD + 4 * li);
    const size_t vrow = row + 2 * p.H * KD + head * p.VD;
    for (int c0 = threadIdx.x / L; c0 < p.VD; c0 += AHEAD * COLS) {
        f32x4 s[AHEAD];
        float v[AHEAD];
#pragma unroll
        for (int a = 0; a < AHEAD; ++a) {
            const int c = c0 + a * COLS < p.VD ? c0 + a * COLS : c0; // (past the end: the first once more, unused)
            s[a] = begins ? f32x4 {0.f, 0.f, 0.f, 0.f} : *(const f32x4 *)(state + (size_t)c * KD);
            v[a] = ldact<BF16>(p.in, vrow + c);
        }
#pragma unroll
        for (int a = 0; a < AHEAD; ++a) {
            const int c = c0 + a * COLS;
            float o = 0.0f;
#pragma unroll
            for (int e = 0; e < 4; ++e) s[a][e] = fmaf(g[e], s[a][e], k[e] * v[a]), o = fmaf(q[e], s[a][e], o);
            o = group_sum<(L < 32 ? L : 32)>(o);
            if constexpr (L > 32) o += __shfl_xor(o, 32, 64);
            if (c >= p.VD) continue;
            *(f32x4 *)(state + (size_t)c * KD) = s[a];
            if (li == 0) os[c] = o;
        }
    }
    __syncthreads();
    float sq = 0.0f;
    for (int c = lane; c < p.VD; c += 64) sq = fmaf(os[c], os[c], sq);
    const float f = 1.0f / sqrtf(wave_total(sq) / (float)p.vdim + p.eps) * p.mul;
    for (int c = threadIdx.x; c < p.VD; c += kStepThreads)
        stact<BF16>(p.out, (size_t)t * p.out_ld + head * p.VD + c, os[c] * f * p.norm[c] * silu_of<BF16>(ldact<BF16>(p.gate, row + head * p.VD + c)));
}

template <bool BF16>
int launch_scan(int KD, const LinearParams &p, hipStream_t st) {
    auto launch = [&](void (*kernel)(LinearParams), int cols) {
        hipLaunchKernelGGL(kernel, dim3(p.v.B, p.H, (p.VD + cols - 1) / cols), dim3(256), 0, st, p);
    };
    switch (KD) {
        case 32: launch(linear_scan_kernel<BF16, 8, 1, 2>, 64); break;
        case 64: launch(linear_scan_kernel<BF16, 16, 1, 2>, 32); break;
        case 128: launch(linear_scan_kernel<BF16, 32, 1, 2>, 16); break;
        default: launch(linear_scan_kernel<BF16, 32, 2, 2>, 16); break;
    }
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

template <bool BF16>
int launch_step(int KD, const LinearParams &p, hipStream_t st) {
    auto launch = [&](void (*kernel)(LinearParams)) { hipLaunchKernelGGL(kernel, dim3(p.H, p.v.B), dim3(kStepThreads), (size_t)p.VD * 4, st, p); };
    switch (KD) {
        case 32: launch(linear_step_kernel<BF16, 8>); break;
        case 64: launch(linear_step_kernel<BF16, 16>); break;
        case 128: launch(linear_step_kernel<BF16, 32>); break;
        default: launch(linear_step_kernel<BF16, 64>); break;
    }
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

} // namespace

int linear_attention(int act, const PlanLayer &L, const StepView &v, const LinearBuffers &b, float eps, hipStream_t st) {
    const size_t esz = act == XFTHIP_BF16 ? 2 : 4;
    XFT_REQUIRE(L.KD <= 256 && (L.KD & (L.KD - 1)) == 0 && L.VD % 32 == 0, "linear_attention: heads of %d / %d values", L.s.dim, L.s.vdim);
    const LinearParams p = {v, (const char *)b.in + L.in_col * esz, L.in_ld, b.alpha, b.o, b.state, L.s.heads, L.VD, 1.0f / sqrtf((float)L.s.dim),
            (const char *)b.in + L.out_gate_col() * esz, L.out_norm, (char *)b.out + L.out_col * esz, L.out_ld, L.s.vdim, eps, L.mix_scale};
    if (v.longest == 1) return act == XFTHIP_BF16 ? launch_step<true>(L.KD, p, st) : launch_step<false>(L.KD, p, st);
    if (int rc = act == XFTHIP_BF16 ? launch_scan<true>(L.KD, p, st) : launch_scan<false>(L.KD, p, st)) return rc;
    return gated_head_norm(act, L, v.T, b.o, b.in, b.out, eps, st);
}

} // namespace xfthip
