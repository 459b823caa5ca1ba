// Gated linear attention of layer plans: per head S = diag(alpha) S + k v^T and o = S^T q, alpha a decay of every key channel, then the norm of
// every head and a silu gate.  Queries, keys and values are read from the rows of the input product, the decays come out of their product's
// epilogue; between those and the output projection's input everything is fp32.
#include <type_traits>

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

// A walk over a segment's tokens with the state in registers.  The state's columns (value channels) do not interact: L lanes hold two
// neighbouring columns, E key rows each (KD = E L).  A token is S = g S + k v and a sum over the key rows that nothing waits for.  q, k, g, v
// of CT tokens are staged in LDS, the next CT on their way through registers.  grid (segments, heads, column groups of COLS)
// (one prompt of 32 heads of 128 is one wave a SIMD: the time is that of the 52 instructions a token)
template <int L, int E>
struct ScanShape {
    static constexpr int KD = E * L, COLS = 256 / L * 2, CT = KD > 128 ? 16 : 32;
    static constexpr size_t lds_floats = 2 * (3 * CT * KD + 2 * CT * COLS);
};
template <bool BF16, int L, int E>
__global__ __launch_bounds__(256) void linear_scan_kernel(LinearParams p) {
    typedef float Rows __attribute__((ext_vector_type(E)));
    typedef typename std::conditional<BF16, uint16_t, float>::type Act;
    constexpr int KD = ScanShape<L, E>::KD, COLS = ScanShape<L, E>::COLS, CT = ScanShape<L, E>::CT;
    constexpr int QK8 = 2 * CT * KD / 8, G4 = CT * KD / 4; // groups of eight of q and k, float4 of the decays of a chunk
    constexpr int PERQ = (QK8 + 255) / 256, PERG = (G4 + 255) / 256, PERV = (CT * COLS + 255) / 256;
    extern __shared__ __align__(16) float scan_lds[]; // twice: q, k, g [CT][KD], v, o [CT][COLS]
    constexpr int HALF = 3 * CT * KD + 2 * CT * COLS, V0 = 3 * CT * KD, O0 = V0 + CT * COLS;
    const int seg = blockIdx.x, head = blockIdx.y, n = p.v.seg_len[seg], off = p.v.seg_off[seg];
    const int li = threadIdx.x % L, lc = threadIdx.x / L * 2, col0 = blockIdx.z * COLS, col = col0 + lc;
    const bool own = col < p.VD; // (VD is a multiple of 32: neighbouring columns are in it or not together)
    float *state = p.state + (((size_t)p.v.seg_row[seg] * p.H + head) * p.VD + (own ? col : 0)) * KD + E * li;
    const int vcol = 2 * p.H * KD + head * p.VD;
    Rows s[2];
#pragma unroll
    for (int c = 0; c < 2; ++c) {
        s[c] = p.v.seg_pos[seg] > 0 ? *(const Rows *)(state + c * KD) : (Rows)0.0f;
        arrived(s[c]);
    }

    constexpr int WORDS = BF16 ? 1 : 2; // of 16 bytes that hold eight activations
    u32x4 qk[PERQ][WORDS];
    f32x4 g[PERG];
    Act vs[PERV];
    auto token_at = [&](int i) { return off + (i < n ? i : n - 1); };
    // (threads without a part take the last one too: a load under a condition would be waited for before the next one goes out)
    auto fetch = [&](int c0) {
#pragma unroll
        for (int i = 0; i < PERQ; ++i) {
            const int part = i * 256 + (int)threadIdx.x, e = part < QK8 ? part : QK8 - 1, k = e / (QK8 / 2), r = e % (QK8 / 2);
            const size_t at = (size_t)token_at(c0 + r / (KD / 8)) * p.ld + (size_t)(k * p.H + head) * KD + r % (KD / 8) * 8;
            const u32x4 *src = (const u32x4 *)((const char *)p.in + at * (BF16 ? 2 : 4));
#pragma unroll
            for (int w = 0; w < WORDS; ++w) qk[i][w] = src[w];
        }
#pragma unroll
        for (int i = 0; i < PERG; ++i) {
            const int part = i * 256 + (int)threadIdx.x, e = part < G4 ? part : G4 - 1;
            g[i] = *(const f32x4 *)(p.alpha + ((size_t)token_at(c0 + e / (KD / 4)) * p.H + head) * KD + e % (KD / 4) * 4);
        }
#pragma unroll
        for (int i = 0; i < PERV; ++i) {
            const int part = i * 256 + (int)threadIdx.x, e = part < CT * COLS ? part : CT * COLS - 1, c = col0 + e % COLS;
            vs[i] = ((const Act *)p.in)[(size_t)token_at(c0 + e / COLS) * p.ld + vcol + (c < p.VD ? c : p.VD - 1)];
        }
    };
    auto stash = [&](int c0, float *lds) { // (a token past the end: decays of one, a key of zero)
#pragma unroll
        for (int i = 0; i < PERQ; ++i) {
            const int part = i * 256 + (int)threadIdx.x, e = part < QK8 ? part : QK8 - 1;
            const float mul = e < QK8 / 2 ? p.qscale : c0 + e % (QK8 / 2) / (KD / 8) < n ? 1.0f : 0.0f;
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
            *(f32x4 *)(lds + 8 * e) = lo * mul, *(f32x4 *)(lds + 8 * e + 4) = hi * mul;
        }
#pragma unroll
        for (int i = 0; i < PERG; ++i) {
            const int part = i * 256 + (int)threadIdx.x, e = part < G4 ? part : G4 - 1;
            *(f32x4 *)(lds + 2 * CT * KD + 4 * e) = c0 + e / (KD / 4) < n ? g[i] : f32x4 {1.f, 1.f, 1.f, 1.f};
        }
#pragma unroll
        for (int i = 0; i < PERV; ++i) {
            const int part = i * 256 + (int)threadIdx.x, e = part < CT * COLS ? part : CT * COLS - 1;
            if constexpr (BF16) lds[V0 + e] = bf16_to_f32(vs[i]);
            else lds[V0 + e] = vs[i];
        }
    };
    fetch(0);
    stash(0, scan_lds);
    __syncthreads();
    int buf = 0;
    for (int c0 = 0; c0 < n; c0 += CT, buf ^= 1) {
        float *lds = scan_lds + buf * HALF;
        const int m = n - c0 < CT ? n - c0 : CT;
        fetch(c0 + CT);
        struct Operands {
            Rows q, k, g;
            float2 v;
        };
        auto read = [&](Operands (&x)[2], int i) {
#pragma unroll
            for (int b = 0; b < 2; ++b) {
                const float *q = lds + (i + b) * KD + E * li, *k = q + CT * KD, *a = k + CT * KD;
                x[b] = Operands {*(const Rows *)q, *(const Rows *)k, *(const Rows *)a, *(const float2 *)(lds + V0 + (i + b) * COLS + lc)};
            }
        };
        float o[4][2];
        auto tokens = [&](const Operands (&x)[2], int first) {
#pragma unroll
            for (int b = 0; b < 2; ++b)
#pragma unroll
                for (int c = 0; c < 2; ++c) {
                    const float v = c ? x[b].v.y : x[b].v.x;
                    float sum = 0.0f;
#pragma unroll
                    for (int e = 0; e < E; ++e) {
                        s[c][e] = fmaf(x[b].g[e], s[c][e], x[b].k[e] * v);
                        sum = fmaf(x[b].q[e], s[c][e], sum);
                    }
                    o[first + b][c] = sum;
                }
        };
        // Four tokens at a time, whose sums go round side by side; a pair's operands are asked for a pair ahead (more reads in flight than
        // the hardware counts would be waited for).  Tokens past the segment's end change nothing: stash.
        Operands even[2], odd[2];
        read(even, 0), read(odd, 2);
        for (int i = 0; i < m; i += 4) {
            const int next = i + 4 < CT ? i + 4 : 0;
            tokens(even, 0);
            read(even, next);
            __builtin_amdgcn_sched_barrier(0);
            tokens(odd, 2);
            read(odd, next + 2);
            __builtin_amdgcn_sched_barrier(0);
            float *dst = lds + O0 + i * COLS + lc;
            if constexpr (L == 32) {
                float sum[4];
#pragma unroll
                for (int b = 0; b < 4; ++b) sum[b] = two_sums(o[b][0], o[b][1]);
                if (li % 16 == 0) {
#pragma unroll
                    for (int b = 0; b < 4; ++b) dst[b * COLS + li / 16] = sum[b];
                }
            } else {
#pragma unroll
                for (int b = 0; b < 4; ++b) o[b][0] = group_sum<L>(o[b][0]), o[b][1] = group_sum<L>(o[b][1]);
                if (li == 0) {
#pragma unroll
                    for (int b = 0; b < 4; ++b) *(float2 *)(dst + b * COLS) = make_float2(o[b][0], o[b][1]);
                }
            }
        }
        stash(c0 + CT, scan_lds + (buf ^ 1) * HALF); // (the other buffer, and the other results, were last read before or behind this barrier one chunk ago)
        __syncthreads();
        float y[PERV];
#pragma unroll
        for (int i = 0; i < PERV; ++i) y[i] = lds[O0 + (i * 256 + (int)threadIdx.x) % (CT * COLS)];
#pragma unroll
        for (int i = 0; i < PERV; ++i) {
            const int e = i * 256 + (int)threadIdx.x, c = col0 + e % COLS;
            if (e < m * COLS && c < p.VD) p.o[((size_t)(off + c0 + e / COLS) * p.H + head) * p.VD + c] = y[i];
        }
    }
    if (own) {
#pragma unroll
        for (int c = 0; c < 2; ++c) *(Rows *)(state + c * KD) = s[c];
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

template <bool BF16, int L, int E>
int launch_scan_shape(const LinearParams &p, hipStream_t st) {
    using S = ScanShape<L, E>;
    static const hipError_t attr = hipFuncSetAttribute((const void *)linear_scan_kernel<BF16, L, E>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    XFT_CHECK_HIP(attr);
    hipLaunchKernelGGL((linear_scan_kernel<BF16, L, E>), dim3(p.v.B, p.H, (p.VD + S::COLS - 1) / S::COLS), dim3(256), S::lds_floats * 4, st, p);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}
template <bool BF16>
int launch_scan(int KD, const LinearParams &p, hipStream_t st) {
    switch (KD) {
        case 32: return launch_scan_shape<BF16, 8, 4>(p, st);
        case 64: return launch_scan_shape<BF16, 16, 4>(p, st);
        case 128: return launch_scan_shape<BF16, 32, 4>(p, st);
        default: return launch_scan_shape<BF16, 32, 8>(p, st);
    }
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
