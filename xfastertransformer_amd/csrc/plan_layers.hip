// Embedding and norms of layer plans: the norm behind a sublayer, the residual sum, the embedding output that joins in
// front of a further pass of a loop, and the norm in front of the next sublayer are one kernel.
#include "plan.h"

namespace xfthip {

namespace {

__global__ void plan_embed_kernel(const uint16_t *__restrict__ table, const int *__restrict__ ids, float *__restrict__ x, int hidden, int vocab) {
    int id = ids[blockIdx.x];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
    const uint16_t *row = table + (size_t)id * hidden;
    for (int c = threadIdx.x; c < hidden; c += blockDim.x) x[(size_t)blockIdx.x * hidden + c] = bf16_to_f32(row[c]);
}

struct NormParams {
    float *x;
    const float *y, *post;
    const uint16_t *table;
    const int *ids, *rows;
    int vocab;
    const float *pre;
    void *xn;
    int hidden, width;
    float eps;
};

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
__global__ __launch_bounds__(NT) void plan_norm_kernel(NormParams p) {
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
        wpost[c] = in && p.y ? *(const f32x4 *)(p.post + col) : zero;
        wpre[c] = in && p.pre ? *(const f32x4 *)(p.pre + col) : zero;
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
    if (!p.pre) return;
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
        const size_t at = (size_t)t * p.hidden + col;
        if constexpr (BF16)
            *(uint2 *)((uint16_t *)p.xn + at) = make_uint2(f32_to_bf16_ref(v[0]) | ((uint32_t)f32_to_bf16_ref(v[1]) << 16),
                    f32_to_bf16_ref(v[2]) | ((uint32_t)f32_to_bf16_ref(v[3]) << 16));
        else
            *(f32x4 *)((float *)p.xn + at) = v;
    }
}

template <bool BF16>
int launch_norm(const NormParams &p, int T, hipStream_t st) {
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

int plan_embed(const uint16_t *table, const int *ids, float *x, int T, int hidden, int vocab, hipStream_t st) {
    hipLaunchKernelGGL(plan_embed_kernel, dim3(T), dim3(256), 0, st, table, ids, x, hidden, vocab);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

int plan_norm(int act, float *x, const float *y, const float *post, const uint16_t *table, const int *ids, int vocab, const float *pre, void *xn,
        const int *rows, int T, int hidden, int width, float eps, hipStream_t st) {
    XFT_REQUIRE(T > 0 && x && hidden % 4 == 0 && width <= hidden && (!rows || (!y && !table)), "plan_norm: bad argument");
    const NormParams p = {x, y, post, table, ids, rows, vocab, pre, xn, hidden, width, eps};
    return act == XFTHIP_BF16 ? launch_norm<true>(p, T, st) : launch_norm<false>(p, T, st);
}

} // namespace xfthip
