// Embedding and norms of layer plans: the norm behind a sublayer, the residual sum, the embedding output that joins in
// front of a further pass of a loop, and the norms in front of the next sublayers are one kernel; the gate of the side embedding.
#include "plan_dev.h"

namespace xfthip {

namespace {

__global__ void plan_embed_kernel(EmbedTables e, StepView v, const int *__restrict__ ids, const int *__restrict__ last_token, float *__restrict__ x) {
    const int t = blockIdx.x, seg = v.tok_seg[t];
    const int prev = v.tok_pos[t] == 0 ? -1 : t > v.seg_off[seg] ? ids[t - 1] : last_token[v.seg_row[seg]];
    embed_token(e, ids[t], v.tok_pos[t] == 0, prev, x + (size_t)t * e.hidden);
}

__global__ __launch_bounds__(256) void plan_softcap_kernel(float *z, size_t n, float cap) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i < n) z[i] = cap * tanhf(z[i] / cap);
}

template <int NT>
__device__ inline float block_sum(float v, float *part) {
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off, 64);
    if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = v;
    __syncthreads();
    float s = 0.0f;
#pragma unroll
    for (int w = 0; w < NT / 64; ++w) s += part[w];
    return s;
}

// one token a workgroup of NT threads; the row stays in registers (CH float4 a thread), every load is requested before the first use
template <bool BF16, int CH, int NT>
__global__ __launch_bounds__(NT) void plan_norm_kernel(PlanNormArgs p) {
    __shared__ float part[2 * NT / 64];
    const int t = blockIdx.x;
    const float *xr = p.x + (size_t)(p.rows ? p.rows[t] : t) * p.hidden;
    f32x4 x[CH], y[CH], wpost[CH], wpre[CH];
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int c = 0; c < CH; ++c) {
        const int col = (c * NT + threadIdx.x) * 4;
        const bool in = col < p.hidden;
        x[c] = in ? *(const f32x4 *)(xr + col) : zero;
        y[c] = in && p.y ? *(const f32x4 *)(p.y + (size_t)t * p.hidden + col) : zero;
        wpost[c] = in && p.post ? *(const f32x4 *)(p.post + col) : zero;
        wpre[c] = in && p.pre.w && !p.pre.b ? *(const f32x4 *)(p.pre.w + col) : zero;
    }
    if (p.table) {
        int id = p.ids[t];
        id = id < 0 ? 0 : (id >= p.vocab ? p.vocab - 1 : id);
        const uint16_t *row = p.table + (size_t)id * p.hidden;
        float sq = 0.0f;
#pragma unroll
        for (int c = 0; c < CH; ++c)
#pragma unroll
            for (int i = 0; i < 4; ++i) sq = fmaf(y[c][i], y[c][i], sq);
        const float r = p.y ? 1.0f / sqrtf(block_sum<NT>(sq, part) / (float)p.width + p.eps) : 0.0f;
#pragma unroll
        for (int c = 0; c < CH; ++c) {
            const int col = (c * NT + threadIdx.x) * 4;
            if (col >= p.hidden) continue;
            const uint2 e = *(const uint2 *)(row + col);
            const f32x4 emb = {u2f(e.x << 16), u2f(e.x & 0xFFFF0000u), u2f(e.y << 16), u2f(e.y & 0xFFFF0000u)};
            x[c] = (x[c] + y[c] * r * wpost[c]) + emb;
        }
    } else if (p.y && !p.post) {
#pragma unroll
        for (int c = 0; c < CH; ++c) x[c] = x[c] + y[c] * p.mul;
    } else if (p.y) {
        float sq = 0.0f;
#pragma unroll
        for (int c = 0; c < CH; ++c)
#pragma unroll
            for (int i = 0; i < 4; ++i) sq = fmaf(y[c][i], y[c][i], sq);
        const float r = 1.0f / sqrtf(block_sum<NT>(sq, part) / (float)p.width + p.eps);
#pragma unroll
        for (int c = 0; c < CH; ++c) x[c] = x[c] + y[c] * r * wpost[c];
    }
    if (p.y || p.table) {
#pragma unroll
        for (int c = 0; c < CH; ++c) {
            const int col = (c * NT + threadIdx.x) * 4;
            if (col < p.hidden) *(f32x4 *)(p.x + (size_t)t * p.hidden + col) = x[c];
        }
    }
    if (!p.pre.w) return;
    if (p.pre.b) { // tanh norms: one value at a time, up to two of them
#pragma unroll
        for (int k = 0; k < 2; ++k) {
            const PlanNorm &n = k ? p.pre2 : p.pre;
            if (!n.w) break;
#pragma unroll
            for (int c = 0; c < CH; ++c) {
                const int col = (c * NT + threadIdx.x) * 4;
                if (col >= p.hidden) continue;
                const f32x4 w = *(const f32x4 *)(n.w + col), b = *(const f32x4 *)(n.b + col);
                f32x4 v;
#pragma unroll
                for (int i = 0; i < 4; ++i) v[i] = fmaf(tanhf(n.alpha * x[c][i]), w[i], b[i]);
                put4<BF16>(k ? p.xn2 : p.xn, (size_t)t * p.hidden + col, v);
            }
        }
        return;
    }
    float sq = 0.0f;
#pragma unroll
    for (int c = 0; c < CH; ++c)
#pragma unroll
        for (int i = 0; i < 4; ++i) sq = fmaf(x[c][i], x[c][i], sq);
    const float r = 1.0f / sqrtf(block_sum<NT>(sq, part + NT / 64) / (float)p.width + p.eps);
#pragma unroll
    for (int c = 0; c < CH; ++c) {
        const int col = (c * NT + threadIdx.x) * 4;
        if (col >= p.hidden) continue;
        const f32x4 v = x[c] * r * wpre[c];
        put4<BF16>(p.xn, (size_t)t * p.hidden + col, v);
    }
}

// Factors 1 / sqrt(mean + eps) of the groups a thread's values belong to.  `unit` lanes (a power of two) add the squares of their
// neighbouring values up before the sums meet in LDS; unit 0: groups that are no whole number of float4, by value.
template <int CH, int NT>
__device__ inline void group_factors(const f32x4 (&v)[CH], const PlanNormArgs &p, int unit, float *sums, f32x4 (&r)[CH]) {
    const int size = p.width / p.groups;
    __syncthreads(); // (the sums of an earlier norm have been read)
#pragma unroll
    for (int c = 0; c < CH; ++c) {
        const int at = c * NT + threadIdx.x; // float4 of the row
        const f32x4 q = v[c] * v[c];
        if (unit == 0) {
            if (at * 4 < p.hidden) *(f32x4 *)(sums + at * 4) = q;
            continue;
        }
        float s = (q[0] + q[1]) + (q[2] + q[3]);
        for (int off = 1; off < unit; off <<= 1) s += __shfl_xor(s, off, 64);
        if (at % unit == 0 && at * 4 < p.hidden) sums[at / unit] = s;
    }
    __syncthreads();
#pragma unroll
    for (int c = 0; c < CH; ++c) {
        const int col = (c * NT + threadIdx.x) * 4;
        r[c] = f32x4 {0.f, 0.f, 0.f, 0.f};
        if (unit > 0) {
            if (col >= p.width) continue;
            const int n = size / (4 * unit);
            const float *part = sums + (size_t)(col / size) * n;
            float s = 0.0f;
            for (int k = 0; k < n; ++k) s += part[k];
            const float f = 1.0f / sqrtf(s / (float)size + p.eps);
            r[c] = f32x4 {f, f, f, f};
        } else {
            for (int i = 0; i < 4; ++i) {
                if (col + i >= p.width) break;
                const float *part = sums + (size_t)((col + i) / size) * size;
                float s = 0.0f;
                for (int k = 0; k < size; ++k) s += part[k];
                r[c][i] = 1.0f / sqrtf(s / (float)size + p.eps);
            }
        }
    }
}

// The same steps with norms in groups and with the results of two mixers that meet here: y = rms(y) mix1 + rms(y2) mix2, x += norm(y) post,
// xn = norm(x) pre
template <bool BF16, int CH, int NT>
__global__ __launch_bounds__(NT) void plan_group_norm_kernel(PlanNormArgs p, int unit) {
    extern __shared__ float sums[];
    __shared__ float part[2][NT / 64];
    const int t = blockIdx.x;
    const float *xr = p.x + (size_t)(p.rows ? p.rows[t] : t) * p.hidden;
    f32x4 x[CH], y[CH], z[CH], wpost[CH], wpre[CH], r[CH];
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int c = 0; c < CH; ++c) {
        const int col = (c * NT + threadIdx.x) * 4;
        const bool in = col < p.hidden;
        x[c] = in ? *(const f32x4 *)(xr + col) : zero;
        y[c] = in && p.y ? *(const f32x4 *)(p.y + (size_t)t * p.hidden + col) : zero;
        z[c] = in && p.y2 ? *(const f32x4 *)(p.y2 + (size_t)t * p.hidden + col) : zero;
        wpost[c] = in && p.post ? *(const f32x4 *)(p.post + col) : zero;
        wpre[c] = in && p.pre.w ? *(const f32x4 *)(p.pre.w + col) : zero;
    }
    if (p.y2) {
        float s1 = 0.0f, s2 = 0.0f;
#pragma unroll
        for (int c = 0; c < CH; ++c)
#pragma unroll
            for (int i = 0; i < 4; ++i) s1 = fmaf(y[c][i], y[c][i], s1), s2 = fmaf(z[c][i], z[c][i], s2);
        s1 = wave_total(s1), s2 = wave_total(s2);
        if ((threadIdx.x & 63) == 0) part[0][threadIdx.x >> 6] = s1, part[1][threadIdx.x >> 6] = s2;
        __syncthreads();
        s1 = s2 = 0.0f;
#pragma unroll
        for (int w = 0; w < NT / 64; ++w) s1 += part[0][w], s2 += part[1][w];
        const float r1 = 1.0f / sqrtf(s1 / (float)p.width + p.eps), r2 = 1.0f / sqrtf(s2 / (float)p.width + p.eps);
#pragma unroll
        for (int c = 0; c < CH; ++c) {
            const int col = (c * NT + threadIdx.x) * 4;
            if (col >= p.hidden) continue;
            y[c] = y[c] * r1 * *(const f32x4 *)(p.mix1 + col) + z[c] * r2 * *(const f32x4 *)(p.mix2 + col);
        }
    }
    if (p.y) {
        if (p.post) {
            group_factors<CH, NT>(y, p, unit, sums, r);
#pragma unroll
            for (int c = 0; c < CH; ++c) x[c] = x[c] + y[c] * r[c] * wpost[c];
        } else {
#pragma unroll
            for (int c = 0; c < CH; ++c) x[c] = x[c] + y[c] * p.mul;
        }
#pragma unroll
        for (int c = 0; c < CH; ++c) {
            const int col = (c * NT + threadIdx.x) * 4;
            if (col < p.hidden) *(f32x4 *)(p.x + (size_t)t * p.hidden + col) = x[c];
        }
    }
    if (!p.pre.w) return;
    group_factors<CH, NT>(x, p, unit, sums, r);
#pragma unroll
    for (int c = 0; c < CH; ++c) {
        const int col = (c * NT + threadIdx.x) * 4;
        if (col < p.hidden) put4<BF16>(p.xn, (size_t)t * p.hidden + col, x[c] * r[c] * wpre[c]);
    }
}

struct SideParams {
    const float *z;
    const uint16_t *table;
    int ld, first;
    const int *ids;
    int vocab, T, width;
    void *out;
};
template <bool BF16>
__global__ __launch_bounds__(256) void side_gate_kernel(SideParams p) {
    const size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * 4;
    if (i >= (size_t)p.T * p.width) return;
    const int t = (int)(i / p.width), c = (int)(i % p.width);
    int id = p.ids[t];
    id = id < 0 ? 0 : (id >= p.vocab ? p.vocab - 1 : id);
    const f32x4 z = *(const f32x4 *)(p.z + i);
    const uint2 e = *(const uint2 *)(p.table + (size_t)id * p.ld + p.first + c);
    const f32x4 emb = {u2f(e.x << 16), u2f(e.x & 0xFFFF0000u), u2f(e.y << 16), u2f(e.y & 0xFFFF0000u)};
    f32x4 v;
#pragma unroll
    for (int k = 0; k < 4; ++k) v[k] = gelu_tanh(z[k]) * emb[k];
    put4<BF16>(p.out, i, v);
}

template <bool BF16>
int launch_group_norm(const PlanNormArgs &p, int T, hipStream_t st) {
    const int ch = (p.hidden + 1023) / 1024, size = p.width / p.groups;
    XFT_REQUIRE(ch <= 16, "plan_norm: hidden size %d above 16384", p.hidden);
    int unit = 0;
    if (size % 4 == 0)
        for (unit = 1; unit < 64 && size % (8 * unit) == 0;) unit *= 2;
    const size_t smem = unit ? (size_t)p.hidden / (4 * unit) * 4 + 16 : (size_t)p.hidden * 4;
    auto launch = [&](void (*kernel)(PlanNormArgs, int), int threads) { hipLaunchKernelGGL(kernel, dim3(T), dim3(threads), smem, st, p, unit); };
    if (T <= 64 && ch > 1) {
        if (ch <= 4) launch(plan_group_norm_kernel<BF16, 1, 1024>, 1024);
        else launch(plan_group_norm_kernel<BF16, 4, 1024>, 1024);
    } else if (ch <= 1) launch(plan_group_norm_kernel<BF16, 1, 256>, 256);
    else if (ch <= 2) launch(plan_group_norm_kernel<BF16, 2, 256>, 256);
    else if (ch <= 4) launch(plan_group_norm_kernel<BF16, 2, 512>, 512);
    else if (ch <= 8) launch(plan_group_norm_kernel<BF16, 4, 512>, 512);
    else launch(plan_group_norm_kernel<BF16, 4, 1024>, 1024);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

template <bool BF16>
int launch_norm(const PlanNormArgs &p, int T, hipStream_t st) {
    const int ch = (p.hidden + 1023) / 1024;
    XFT_REQUIRE(ch <= 16, "plan_norm: hidden size %d above 16384", p.hidden);
    // few rows: the kernel is one chain of latencies, shorter with the row spread over more threads
    if (T <= 64 && ch > 1) {
        if (ch <= 4) hipLaunchKernelGGL((plan_norm_kernel<BF16, 1, 1024>), dim3(T), dim3(1024), 0, st, p);
        else hipLaunchKernelGGL((plan_norm_kernel<BF16, 4, 1024>), dim3(T), dim3(1024), 0, st, p);
    } else if (ch <= 1) hipLaunchKernelGGL((plan_norm_kernel<BF16, 1, 256>), dim3(T), dim3(256), 0, st, p);
    else if (ch <= 2) hipLaunchKernelGGL((plan_norm_kernel<BF16, 2, 256>), dim3(T), dim3(256), 0, st, p);
    else if (ch <= 4) hipLaunchKernelGGL((plan_norm_kernel<BF16, 4, 256>), dim3(T), dim3(256), 0, st, p);
    else if (ch <= 8) hipLaunchKernelGGL((plan_norm_kernel<BF16, 8, 256>), dim3(T), dim3(256), 0, st, p);
    else hipLaunchKernelGGL((plan_norm_kernel<BF16, 16, 256>), dim3(T), dim3(256), 0, st, p);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

} // namespace

int plan_embed(const EmbedTables &e, const StepView &v, const int *ids, const int *last_token, float *x, hipStream_t st) {
    hipLaunchKernelGGL(plan_embed_kernel, dim3(v.T), dim3(256), 0, st, e, v, ids, last_token, x);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

int plan_softcap(float *logits, size_t n, float cap, hipStream_t st) {
    XFT_REQUIRE(n > 0 && cap > 0.0f, "plan_softcap: bad argument");
    hipLaunchKernelGGL(plan_softcap_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, st, logits, n, cap);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

int plan_norm(int act, const PlanNormArgs &p, int T, hipStream_t st) {
    XFT_REQUIRE(T > 0 && p.x && p.hidden % 4 == 0 && p.width <= p.hidden && (!p.rows || (!p.y && !p.table)) && (!p.pre2.w || p.pre.b)
                    && (!p.table || !p.y || p.post),
            "plan_norm: bad argument");
    if (p.groups > 1 || p.y2) {
        XFT_REQUIRE(p.width % p.groups == 0 && !p.table && !p.pre.b && !p.pre2.w && (!p.y2 || (p.y && p.mix1 && p.mix2)), "plan_norm: options that do not go together");
        return act == XFTHIP_BF16 ? launch_group_norm<true>(p, T, st) : launch_group_norm<false>(p, T, st);
    }
    return act == XFTHIP_BF16 ? launch_norm<true>(p, T, st) : launch_norm<false>(p, T, st);
}

int plan_side_gate(int act, const float *z, const uint16_t *table, int ld, int first, const int *ids, int vocab, void *out, int T, int width,
        hipStream_t st) {
    XFT_REQUIRE(T > 0 && width % 4 == 0 && ld % 4 == 0 && first % 4 == 0, "plan_side_gate: bad argument");
    const SideParams p = {z, table, ld, first, ids, vocab, T, width, out};
    const dim3 grid((unsigned)(((size_t)T * width / 4 + 255) / 256));
    if (act == XFTHIP_BF16) hipLaunchKernelGGL(side_gate_kernel<true>, grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL(side_gate_kernel<false>, grid, dim3(256), 0, st, p);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

} // namespace xfthip
