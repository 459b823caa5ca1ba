// Latent attention of layer plans: keys and values of all heads are linear images of one normalised latent a token, which is
// what the cache holds, beside one rotated key part shared by the heads.
//
// Absorbed form: a query is carried into the latent space by its head's W_uk turned round, scores are products with the
// cached rows themselves, and the weighted sum of latents is carried to the value space by W_uv behind the softmax.  All
// heads of a token then read the same cache rows.
#include "plan.h"

namespace xfthip {

namespace {

__device__ inline float wave_total(float v) {
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) v += __shfl_xor(v, off, 64);
    return v;
}
__device__ inline float wave_largest(float v) {
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) v = fmaxf(v, __shfl_xor(v, off, 64));
    return v;
}

template <bool BF16>
__device__ inline float ldact(const void *p, size_t i) {
    if constexpr (BF16) return bf16_to_f32(((const uint16_t *)p)[i]);
    else return ((const float *)p)[i];
}
template <bool BF16>
__device__ inline void stact(void *p, size_t i, float v) {
    if constexpr (BF16) ((uint16_t *)p)[i] = f32_to_bf16_ref(v);
    else ((float *)p)[i] = v;
}

// cache row of position `pos` of slot `row`
__device__ inline size_t cache_row(const StepView &v, int row, int pos) {
    return (size_t)v.table[(size_t)row * v.table_stride + pos / kPageTokens] * kPageTokens + pos % kPageTokens;
}

struct PrepareParams {
    StepView v;
    const void *a;
    void *cq;
    LatentCacheView cache;
    const float *q_norm, *kv_norm, *cosT, *sinT;
    int QR, RD, q_rank, kv_rank, rot, interleaved;
    float eps;
};

template <bool BF16>
__global__ __launch_bounds__(256) void latent_prepare_kernel(PrepareParams p) {
    __shared__ float part[2][4];
    const int t = blockIdx.x, R = p.cache.R;
    const size_t base = (size_t)t * (p.QR + R + p.RD);
    float sq = 0.0f, sk = 0.0f;
    for (int c = threadIdx.x; c < p.QR; c += 256) {
        const float x = ldact<BF16>(p.a, base + c);
        sq = fmaf(x, x, sq);
    }
    for (int c = threadIdx.x; c < R; c += 256) {
        const float x = ldact<BF16>(p.a, base + p.QR + c);
        sk = fmaf(x, x, sk);
    }
    sq = wave_total(sq), sk = wave_total(sk);
    if ((threadIdx.x & 63) == 0) part[0][threadIdx.x >> 6] = sq, part[1][threadIdx.x >> 6] = sk;
    __syncthreads();
    sq = (part[0][0] + part[0][1]) + (part[0][2] + part[0][3]), sk = (part[1][0] + part[1][1]) + (part[1][2] + part[1][3]);
    const float rq = 1.0f / sqrtf(sq / (float)p.q_rank + p.eps), rk = 1.0f / sqrtf(sk / (float)p.kv_rank + p.eps);
    for (int c = threadIdx.x; c < p.QR; c += 256) stact<BF16>(p.cq, (size_t)t * p.QR + c, ldact<BF16>(p.a, base + c) * rq * p.q_norm[c]);
    const int seg = p.v.tok_seg[t], pos = p.v.tok_pos[t];
    const size_t dst = cache_row(p.v, p.v.seg_row[seg], pos) * (R + p.RD);
    for (int c = threadIdx.x; c < R; c += 256) stact<BF16>(p.cache.pool, dst + c, ldact<BF16>(p.a, base + p.QR + c) * rk * p.kv_norm[c]);
    const int half = p.rot / 2;
    for (int c = threadIdx.x; c < p.RD; c += 256) {
        float y = 0.0f;
        if (c < p.rot) {
            const int i = p.interleaved ? c >> 1 : (c < half ? c : c - half);
            const bool second = p.interleaved ? (c & 1) != 0 : c >= half;
            const float u = ldact<BF16>(p.a, base + p.QR + R + (p.interleaved ? 2 * i : i));
            const float w = ldact<BF16>(p.a, base + p.QR + R + (p.interleaved ? 2 * i + 1 : i + half));
            const float cs = p.cosT[(size_t)pos * half + i], sn = p.sinT[(size_t)pos * half + i];
            y = second ? fmaf(w, cs, u * sn) : fmaf(u, cs, -(w * sn));
        }
        stact<BF16>(p.cache.pool, dst + R + c, y);
    }
}

// one thread a rotated pair
template <bool BF16>
__global__ __launch_bounds__(256) void rotate_q_kernel(StepView v, void *q, int T, int H, int D, int RD, int half, int interleaved, const float *cosT,
        const float *sinT) {
    const size_t idx = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (idx >= (size_t)T * H * half) return;
    const int i = (int)(idx % half);
    const size_t th = idx / half;
    const int pos = v.tok_pos[th / H];
    const size_t at = th * (D + RD) + D;
    const size_t iu = at + (interleaved ? 2 * i : i), iw = at + (interleaved ? 2 * i + 1 : i + half);
    const float u = ldact<BF16>(q, iu), w = ldact<BF16>(q, iw);
    const float cs = cosT[(size_t)pos * half + i], sn = sinT[(size_t)pos * half + i];
    stact<BF16>(q, iu, fmaf(u, cs, -(w * sn)));
    stact<BF16>(q, iw, fmaf(w, cs, u * sn));
}

struct AttendParams {
    StepView v;
    const void *qa, *q;
    void *out;
    LatentCacheView cache;
    const float *sink; // or null
    int H, D, window;
    float scale;
};

// Any type, any size: one workgroup a (token, head), 256 keys at a time, a key a thread for the scores and a latent
// dimension a thread for the weighted sum.
template <bool BF16>
__global__ __launch_bounds__(256) void latent_attend_kernel(AttendParams p) {
    extern __shared__ float smem[];
    const int R = p.cache.R, RD = p.cache.RD, row_len = R + RD;
    float *qs = smem, *ps = qs + row_len, *o = ps + 256, *part = o + R;
    size_t *kr = (size_t *)(part + 8); // (8-byte aligned: R, RD are multiples of 32)
    const int t = blockIdx.x, h = blockIdx.y;
    const int seg = p.v.tok_seg[t], pos = p.v.tok_pos[t], slot = p.v.seg_row[seg];
    for (int c = threadIdx.x; c < R; c += 256) qs[c] = ldact<BF16>(p.qa, ((size_t)t * p.H + h) * R + c), o[c] = 0.0f;
    for (int c = threadIdx.x; c < RD; c += 256) qs[R + c] = ldact<BF16>(p.q, ((size_t)t * p.H + h) * (p.D + RD) + p.D + c);
    const int first = p.window > 0 && pos + 1 > p.window ? pos + 1 - p.window : 0;
    float m = p.sink ? p.sink[h] : -INFINITY, l = p.sink ? 1.0f : 0.0f; // the sink has no key and no value
    __syncthreads();
    for (int k0 = first; k0 <= pos; k0 += 256) {
        const int j = k0 + threadIdx.x;
        float s = -INFINITY;
        if (j <= pos) {
            const size_t at = cache_row(p.v, slot, j) * row_len;
            kr[threadIdx.x] = at;
            float acc = 0.0f;
            for (int c = 0; c < row_len; ++c) acc = fmaf(qs[c], ldact<BF16>(p.cache.pool, at + c), acc);
            s = acc * p.scale;
        }
        float mx = wave_largest(s);
        if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = mx;
        __syncthreads();
        const float m_new = fmaxf(fmaxf(fmaxf(part[0], part[1]), fmaxf(part[2], part[3])), m);
        const float alpha = expf(m - m_new); // (0 while nothing has been seen)
        const float e = j <= pos ? expf(s - m_new) : 0.0f;
        ps[threadIdx.x] = e;
        const float sum = wave_total(e);
        if ((threadIdx.x & 63) == 0) part[4 + (threadIdx.x >> 6)] = sum;
        __syncthreads();
        l = l * alpha + ((part[4] + part[5]) + (part[6] + part[7]));
        m = m_new;
        const int n = pos - k0 + 1 < 256 ? pos - k0 + 1 : 256;
        for (int c = threadIdx.x; c < R; c += 256) {
            float acc = o[c] * alpha;
            for (int i = 0; i < n; ++i) acc = fmaf(ps[i], ldact<BF16>(p.cache.pool, kr[i] + c), acc);
            o[c] = acc;
        }
        __syncthreads();
    }
    for (int c = threadIdx.x; c < R; c += 256) stact<BF16>(p.out, ((size_t)t * p.H + h) * R + c, o[c] / l);
}

} // namespace

int latent_prepare(int act, const PlanLayer &L, const StepView &v, const void *a, void *cq, const LatentCacheView &cache, float eps, hipStream_t st) {
    const PrepareParams p = {v, a, cq, cache, L.q_norm, L.kv_norm, L.cosT, L.sinT, L.QR, L.RD, L.s.q_rank, L.s.kv_rank, L.s.rot_dim,
            L.s.rot_interleaved, eps};
    if (act == XFTHIP_BF16)
        hipLaunchKernelGGL(latent_prepare_kernel<true>, dim3(v.T), dim3(256), 0, st, p);
    else
        hipLaunchKernelGGL(latent_prepare_kernel<false>, dim3(v.T), dim3(256), 0, st, p);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

int latent_rotate_q(int act, const PlanLayer &L, const StepView &v, void *q, hipStream_t st) {
    const int half = L.s.rot_dim / 2;
    if (half == 0) return 0;
    const unsigned blocks = (unsigned)(((size_t)v.T * L.s.heads * half + 255) / 256);
    if (act == XFTHIP_BF16)
        hipLaunchKernelGGL(rotate_q_kernel<true>, dim3(blocks), dim3(256), 0, st, v, q, v.T, L.s.heads, L.D, L.RD, half, L.s.rot_interleaved, L.cosT, L.sinT);
    else
        hipLaunchKernelGGL(rotate_q_kernel<false>, dim3(blocks), dim3(256), 0, st, v, q, v.T, L.s.heads, L.D, L.RD, half, L.s.rot_interleaved, L.cosT, L.sinT);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

int latent_split_count(const PlanLayer &, int, int, int) { return 1; }

int latent_attention(int act, const PlanLayer &L, const StepView &v, const void *qa, const void *q, void *out, const LatentCacheView &cache, int hint,
        float *part, size_t part_floats, hipStream_t st) {
    (void)hint, (void)part, (void)part_floats;
    const AttendParams p = {v, qa, q, out, cache, L.sink, L.s.heads, L.D, L.s.window, L.s.scale};
    const size_t smem = (size_t)(2 * L.R + L.RD + 256 + 8) * 4 + 256 * 8;
    XFT_REQUIRE(smem <= 64 * 1024, "latent_attention: latent of %d values too wide", L.R);
    if (act == XFTHIP_BF16)
        hipLaunchKernelGGL(latent_attend_kernel<true>, dim3(v.T, L.s.heads), dim3(256), smem, st, p);
    else
        hipLaunchKernelGGL(latent_attend_kernel<false>, dim3(v.T, L.s.heads), dim3(256), smem, st, p);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

} // namespace xfthip
