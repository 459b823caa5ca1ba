// Latent attention of layer plans: keys and values of all heads are linear images of one normalised latent a token, which is
// what the cache holds, beside one rotated key part shared by the heads.
//
// Absorbed form: a query is carried into the latent space by its head's W_uk turned round, scores are products with the
// cached rows themselves, and the weighted sum of latents is carried to the value space by W_uv behind the softmax.  All
// heads of a token then read the same cache rows.  Expanded form: keys and values of every head are made from the latents of
// the whole context first, which pays when many tokens attend to them.
#include "plan_dev.h"

namespace xfthip {

namespace {

struct PrepareParams {
    StepView v;
    const void *a;
    void *cq;
    LatentCacheView cache;
    const float *q_norm, *kv_norm, *cosT, *sinT;
    int QR, RD, q_rank, kv_rank, rot, interleaved;
    float eps;
};

// One token a workgroup, 8 neighbouring values a thread and turn; the row and the norm weights are in registers (CH turns)
// before the sums meet.
template <bool BF16, int CH>
__global__ __launch_bounds__(256) void latent_prepare_kernel(PrepareParams p) {
    __shared__ float part[2][4];
    const int t = blockIdx.x, R = p.cache.R, len = p.QR + R + p.RD;
    const size_t base = (size_t)t * len;
    const int seg = p.v.tok_seg[t], pos = p.v.tok_pos[t];
    float x[CH][8], w[CH][8], sq = 0.0f, sk = 0.0f;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (i * 256 + (int)threadIdx.x) * 8;
        if (c >= p.QR + R) continue;
        load8<BF16>(p.a, base + c, x[i]);
        load8<false>(c < p.QR ? p.q_norm : p.kv_norm - p.QR, c, w[i]);
    }
    const size_t dst = cache_row(p.v, p.v.seg_row[seg], pos) * (R + p.RD);
    // the shared key part: one value a thread, its partner read beside it
    const int half = p.rot / 2;
    for (int c = threadIdx.x; c < p.RD; c += 256) {
        float y = 0.0f;
        if (c < p.rot) {
            const int i = p.interleaved ? c >> 1 : (c < half ? c : c - half);
            const bool second = p.interleaved ? (c & 1) != 0 : c >= half;
            const float u = ldact<BF16>(p.a, base + p.QR + R + (p.interleaved ? 2 * i : i));
            const float z = ldact<BF16>(p.a, base + p.QR + R + (p.interleaved ? 2 * i + 1 : i + half));
            const float cs = p.cosT[(size_t)pos * half + i], sn = p.sinT[(size_t)pos * half + i];
            y = second ? fmaf(z, cs, u * sn) : fmaf(u, cs, -(z * sn));
        }
        stact<BF16>(p.cache.pool, dst + R + c, y);
    }
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (i * 256 + (int)threadIdx.x) * 8;
        if (c >= p.QR + R) continue;
        float s = 0.0f;
#pragma unroll
        for (int k = 0; k < 8; ++k) s = fmaf(x[i][k], x[i][k], s);
        (c < p.QR ? sq : sk) += s;
    }
    sq = wave_total(sq), sk = wave_total(sk);
    if ((threadIdx.x & 63) == 0) part[0][threadIdx.x >> 6] = sq, part[1][threadIdx.x >> 6] = sk;
    __syncthreads();
    sq = (part[0][0] + part[0][1]) + (part[0][2] + part[0][3]), sk = (part[1][0] + part[1][1]) + (part[1][2] + part[1][3]);
    const float rq = 1.0f / sqrtf(sq / (float)p.q_rank + p.eps), rk = 1.0f / sqrtf(sk / (float)p.kv_rank + p.eps);
#pragma unroll
    for (int i = 0; i < CH; ++i) {
        const int c = (i * 256 + (int)threadIdx.x) * 8;
        if (c >= p.QR + R) continue;
        const float r = c < p.QR ? rq : rk;
#pragma unroll
        for (int k = 0; k < 8; ++k) x[i][k] = x[i][k] * r * w[i][k];
        if (c < p.QR) store8<BF16>(p.cq, (size_t)t * p.QR + c, x[i]);
        else store8<BF16>(p.cache.pool, dst + c - p.QR, x[i]);
    }
}

// One thread eight rotated values: four neighbouring pairs (interleaved), or four pairs of either half.
template <bool BF16>
__global__ __launch_bounds__(256) void rotate_q_kernel(StepView v, void *q, int T, int H, int D, int RD, int half, int interleaved, const float *cosT,
        const float *sinT) {
    const int per = (half + 3) / 4;
    const size_t idx = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (idx >= (size_t)T * H * per) return;
    const int i0 = (int)(idx % per) * 4;
    const size_t th = idx / per;
    const int pos = v.tok_pos[th / H];
    const size_t at = th * (D + RD) + D;
    const float *cs = cosT + (size_t)pos * half, *sn = sinT + (size_t)pos * half;
    if ((half & 3) == 0) {
        const f32x4 c = *(const f32x4 *)(cs + i0), s = *(const f32x4 *)(sn + i0);
        if (interleaved) {
            float x[8], y[8];
            load8<BF16>(q, at + 2 * i0, x);
#pragma unroll
            for (int k = 0; k < 4; ++k) {
                y[2 * k] = fmaf(x[2 * k], c[k], -(x[2 * k + 1] * s[k]));
                y[2 * k + 1] = fmaf(x[2 * k + 1], c[k], x[2 * k] * s[k]);
            }
            store8<BF16>(q, at + 2 * i0, y);
        } else {
            f32x4 a, b;
            if constexpr (BF16) {
                const uint2 ua = *(const uint2 *)((const uint16_t *)q + at + i0), ub = *(const uint2 *)((const uint16_t *)q + at + half + i0);
                a = f32x4 {u2f(ua.x << 16), u2f(ua.x & 0xFFFF0000u), u2f(ua.y << 16), u2f(ua.y & 0xFFFF0000u)};
                b = f32x4 {u2f(ub.x << 16), u2f(ub.x & 0xFFFF0000u), u2f(ub.y << 16), u2f(ub.y & 0xFFFF0000u)};
            } else {
                a = *(const f32x4 *)((const float *)q + at + i0), b = *(const f32x4 *)((const float *)q + at + half + i0);
            }
            f32x4 ya, yb;
#pragma unroll
            for (int k = 0; k < 4; ++k) ya[k] = fmaf(a[k], c[k], -(b[k] * s[k])), yb[k] = fmaf(b[k], c[k], a[k] * s[k]);
            if constexpr (BF16) {
                *(uint2 *)((uint16_t *)q + at + i0) = make_uint2(pack_pair(ya[0], ya[1]), pack_pair(ya[2], ya[3]));
                *(uint2 *)((uint16_t *)q + at + half + i0) = make_uint2(pack_pair(yb[0], yb[1]), pack_pair(yb[2], yb[3]));
            } else {
                *(f32x4 *)((float *)q + at + i0) = ya, *(f32x4 *)((float *)q + at + half + i0) = yb;
            }
        }
        return;
    }
    for (int i = i0; i < i0 + 4 && i < half; ++i) {
        const size_t iu = at + (interleaved ? 2 * i : i), iw = at + (interleaved ? 2 * i + 1 : i + half);
        const float u = ldact<BF16>(q, iu), w = ldact<BF16>(q, iw);
        stact<BF16>(q, iu, fmaf(u, cs[i], -(w * sn[i])));
        stact<BF16>(q, iw, fmaf(w, cs[i], u * sn[i]));
    }
}

struct AttendParams {
    StepView v;
    const void *qa, *q;
    void *out;
    LatentCacheView cache;
    const float *sink; // or null
    int H, D, window, max_len; // segments longer than max_len are somebody else's
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
    if (p.v.seg_len[seg] > p.max_len) return;
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

typedef __attribute__((ext_vector_type(4))) short s16x4;
typedef __attribute__((ext_vector_type(8))) short s16x8;
#define LDS_PTR(type, p) ((__attribute__((address_space(3))) type *)(p))

// Two transposing LDS reads: within 16 lanes, lane i names token row i / 4 and dims 4 (i % 4) of a block of 4 tokens x 16 dims
// and receives the four tokens of dim i.  `second` lies where the lane's other four tokens start.
__device__ inline bf16x8 transposed_pair(const unsigned char *first, const unsigned char *second) {
    const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16(LDS_PTR(s16x4, first)), b = __builtin_amdgcn_ds_read_tr16_b64_v4i16(LDS_PTR(s16x4, second));
    return __builtin_bit_cast(bf16x8, __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7));
}

struct MfmaParams {
    AttendParams a;
    int RD, nsplit, max_len;
    float *part; // [units][nsplit][32][R] outputs, behind them [units][nsplit][32][2] maxima and sums
    size_t part_ml;
};

// BF16, absorbed form: 32 columns (neighbouring (token, head) pairs of one segment, which all read the same cache rows) a
// workgroup, the context split over gridDim.z.  32 tokens at a time go through LDS: a wave scores 16 of them for 16 columns
// (A = cached rows, B = the columns' queries in registers), the scores meet in LDS, every wave turns them into
// probabilities and adds up its own quarter of the latent dimensions (A = the same rows read transposed).
// DT: 16-dim tiles of a wave (R <= 64 DT); KSMAX: most 32-dim steps of a row; EXACT: R = 64 DT and a row is KSMAX steps, so
// that the loops over them are straight-line code.
template <int DT, int KSMAX, bool EXACT>
__global__ __launch_bounds__(256, 2) void latent_mfma_kernel(MfmaParams p) {
    extern __shared__ unsigned char lds[];
    const StepView &v = p.a.v;
    const int seg = blockIdx.y, n = v.seg_len[seg], H = p.a.H, R = EXACT ? 64 * DT : p.a.cache.R, RD = p.RD;
    const int c0 = blockIdx.x * 32, ncols = n * H;
    if (n > p.max_len || c0 >= ncols) return;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, i16 = lane & 15;
    const int off = v.seg_off[seg], start = v.seg_pos[seg];
    const int *table = v.table + (size_t)v.seg_row[seg] * v.table_stride;
    const int last = c0 + 31 < ncols ? c0 + 31 : ncols - 1;
    const int lo = start + c0 / H, hi = start + last / H; // positions of the first and the last column's token
    const int first_vis = p.a.window > 0 && lo + 1 > p.a.window ? lo + 1 - p.a.window : 0;
    const int b0 = first_vis >> 5, b1 = (hi >> 5) + 1;
    const int per = (b1 - b0 + p.nsplit - 1) / p.nsplit;
    const int bb = b0 + (int)blockIdx.z * per, be = bb + per < b1 ? bb + per : b1;
    const int row_len = EXACT ? KSMAX * 32 : R + RD, ks_n = row_len / 32, row_chunks = row_len / 8, chunks = 32 * row_chunks;
    const int pitch = row_len * 2 + 16;
    float *sc = (float *)(lds + 2 * 32 * pitch); // [32 columns][36]

    const int ct_s = wave >> 1, tt = wave & 1; // this wave's score tile
    bf16x8 qf[KSMAX];
    {
        const int c = c0 + 16 * ct_s + i16;
        const size_t at = (size_t)off * H + (c < ncols ? c : ncols - 1);
        const uint16_t *qa = (const uint16_t *)p.a.qa + at * R + 8 * g;
        const uint16_t *qr = (const uint16_t *)p.a.q + at * (p.a.D + RD) + p.a.D + 8 * g - R;
#pragma unroll
        for (int ks = 0; ks < KSMAX; ++ks)
            if (EXACT || ks < ks_n) qf[ks] = *(const bf16x8 *)((ks * 32 < R ? qa : qr) + ks * 32);
    }
    // this lane's column of either column tile: position, running maximum (log2 domain) and this lane's part of the sum
    int cpos[2];
    float m[2], l[2];
    f32x4 o[DT][2];
#pragma unroll
    for (int ct = 0; ct < 2; ++ct) {
        const int c = c0 + 16 * ct + i16;
        cpos[ct] = c < ncols ? start + c / H : -1;
        m[ct] = kUnseen, l[ct] = 0.0f;
#pragma unroll
        for (int d = 0; d < DT; ++d) o[d][ct] = f32x4 {0.f, 0.f, 0.f, 0.f};
    }
    const float scale2 = p.a.scale * kLog2e;

    constexpr int PER = (KSMAX + 1) / 2;
    u32x4 stage[PER];
    auto fetch = [&](int blk, int page) {
        const u32x4 *src = (const u32x4 *)((const uint16_t *)p.a.cache.pool + ((size_t)page * kPageTokens + (blk & 1) * 32) * row_len);
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const int e = i * 256 + threadIdx.x;
            stage[i] = src[e < chunks ? e : chunks - 1]; // (past the block: its last chunk once more)
        }
    };
    int lds_off[PER]; // chunk e of a block: 16 bytes of padding behind every row before it
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        int e = i * 256 + threadIdx.x;
        e = e < chunks ? e : chunks - 1;
        lds_off[i] = (e + e / row_chunks) * 16;
    }
    if (bb < be) fetch(bb, table[bb >> 1]);
    int page = bb + 1 < be ? table[(bb + 1) >> 1] : 0;
    int buf = 0;
    for (int blk = bb; blk < be; ++blk, buf ^= 1) {
        unsigned char *kv = lds + buf * 32 * pitch;
#pragma unroll
        for (int i = 0; i < PER; ++i) *(u32x4 *)(kv + lds_off[i]) = stage[i];
        __syncthreads();
        if (blk + 1 < be) fetch(blk + 1, page);
        if (blk + 2 < be) page = table[(blk + 2) >> 1];
        f32x4 s = {0.f, 0.f, 0.f, 0.f}, s1 = s; // (two chains of products)
        const unsigned char *krow = kv + (16 * tt + i16) * pitch + 16 * g;
#pragma unroll
        for (int ks = 0; ks < KSMAX; ++ks)
            if (EXACT || ks < ks_n) (ks & 1 ? s1 : s) = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8 *)(krow + ks * 64), qf[ks], ks & 1 ? s1 : s, 0, 0, 0);
        *(f32x4 *)(sc + (16 * ct_s + i16) * 36 + 16 * tt + 4 * g) = s + s1;
        __syncthreads();
        // a lane group takes tokens 4 g .. 4 g + 3 and 16 + 4 g .. of the block: the transposed reads below then touch eight
        // neighbouring rows at a time, which the row pitch spreads over the banks
        bf16x8 pf[2];
        float alpha[2];
        const bool open = blk * 32 + 31 <= lo && (p.a.window <= 0 || blk * 32 > hi - p.a.window); // every column sees the whole block
#pragma unroll
        for (int ct = 0; ct < 2; ++ct) {
            const float *row = sc + (16 * ct + i16) * 36 + 4 * g;
            const f32x4 x0 = *(const f32x4 *)row * scale2, x1 = *(const f32x4 *)(row + 16) * scale2;
            float x[8], bm = kUnseen;
#pragma unroll
            for (int j = 0; j < 8; ++j) x[j] = j < 4 ? x0[j & 3] : x1[j & 3];
            if (!open) {
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    const int t = blk * 32 + 4 * g + (j & 3) + (j < 4 ? 0 : 16);
                    x[j] = t <= cpos[ct] && (p.a.window <= 0 || t > cpos[ct] - p.a.window) ? x[j] : kUnseen;
                }
            }
#pragma unroll
            for (int j = 0; j < 8; ++j) bm = fmaxf(bm, x[j]);
            bm = fmaxf(bm, __shfl_xor(bm, 16, 64));
            bm = fmaxf(bm, __shfl_xor(bm, 32, 64));
            const float m_new = fmaxf(m[ct], bm);
            alpha[ct] = __builtin_amdgcn_exp2f(m[ct] - m_new);
            m[ct] = m_new;
            float sum = 0.0f;
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                // (a column that has seen no key has its reference point at the masked score)
                const float e = __builtin_amdgcn_exp2f(x[j] - m_new);
                x[j] = open || x[j] > 0.5f * kUnseen ? e : 0.0f;
                sum += x[j];
            }
            l[ct] = l[ct] * alpha[ct] + sum;
            pf[ct] = pack_bf16x8(x);
        }
        if (__builtin_amdgcn_ballot_w64(alpha[0] != 1.0f || alpha[1] != 1.0f) != 0) {
#pragma unroll
            for (int d = 0; d < DT; ++d) o[d][0] *= alpha[0], o[d][1] *= alpha[1];
        }
        const unsigned char *vrow = kv + (4 * g + (i16 >> 2)) * pitch + 8 * (i16 & 3);
#pragma unroll
        for (int d = 0; d < DT; ++d) {
            const int tile = wave * DT + d;
            if (EXACT || tile * 16 < R) {
                const bf16x8 a = transposed_pair(vrow + tile * 32, vrow + tile * 32 + 16 * pitch);
                o[d][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, pf[0], o[d][0], 0, 0, 0);
                o[d][1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, pf[1], o[d][1], 0, 0, 0);
            }
        }
    }
#pragma unroll
    for (int ct = 0; ct < 2; ++ct) {
        l[ct] += __shfl_xor(l[ct], 16, 64);
        l[ct] += __shfl_xor(l[ct], 32, 64);
        const int c = c0 + 16 * ct + i16;
        if (p.nsplit > 1) {
            const size_t slot = (((size_t)seg * gridDim.x + blockIdx.x) * p.nsplit + blockIdx.z) * 32 + 16 * ct + i16;
            if (wave == 0 && g == 0) *(float2 *)(p.part + p.part_ml + slot * 2) = make_float2(m[ct], l[ct]);
            if (bb < be && c < ncols) {
#pragma unroll
                for (int d = 0; d < DT; ++d) {
                    const int tile = wave * DT + d;
                    if (EXACT || tile * 16 < R) *(f32x4 *)(p.part + slot * R + tile * 16 + 4 * g) = o[d][ct];
                }
            }
        } else if (c < ncols) {
            float den = l[ct], mul = 1.0f;
            if (p.a.sink) {
                const float s2 = p.a.sink[c % H] * kLog2e, mt = fmaxf(m[ct], s2);
                mul = __builtin_amdgcn_exp2f(m[ct] - mt);
                den = den * mul + __builtin_amdgcn_exp2f(s2 - mt);
            }
            mul /= den;
            uint16_t *dst = (uint16_t *)p.a.out + ((size_t)off * H + c) * R;
#pragma unroll
            for (int d = 0; d < DT; ++d) {
                const int tile = wave * DT + d;
                if (EXACT || tile * 16 < R) {
                    const f32x4 y = o[d][ct] * mul;
                    *(uint2 *)(dst + tile * 16 + 4 * g) = make_uint2(pack_pair(y[0], y[1]), pack_pair(y[2], y[3]));
                }
            }
        }
    }
}

// sum of a column's splits; grid (column groups, segments, 32 columns).  The splits' weights are worked out once, side by
// side, and the outputs are added four splits at a time.
constexpr int kMaxSplits = 64;
__global__ __launch_bounds__(128) void latent_merge_kernel(MfmaParams p) {
    __shared__ float w[kMaxSplits];
    __shared__ float inv_den;
    const StepView &v = p.a.v;
    const int seg = blockIdx.y, n = v.seg_len[seg], H = p.a.H, R = p.a.cache.R;
    const int c = blockIdx.x * 32 + blockIdx.z;
    if (n > p.max_len || c >= n * H) return;
    const size_t unit = ((size_t)seg * gridDim.x + blockIdx.x) * p.nsplit;
    if (threadIdx.x < 64) {
        float2 ml = make_float2(kUnseen, 0.0f);
        if ((int)threadIdx.x < p.nsplit) ml = *(const float2 *)(p.part + p.part_ml + ((unit + threadIdx.x) * 32 + blockIdx.z) * 2);
        const float s2 = p.a.sink ? p.a.sink[c % H] * kLog2e : kUnseen;
        const float mt = fmaxf(wave_largest(ml.x), s2);
        const float e = ml.x > 0.5f * kUnseen ? __builtin_amdgcn_exp2f(ml.x - mt) : 0.0f;
        const float den = wave_total(ml.y * e) + (p.a.sink ? __builtin_amdgcn_exp2f(s2 - mt) : 0.0f);
        w[threadIdx.x] = e;
        if (threadIdx.x == 0) inv_den = 1.0f / den;
    }
    __syncthreads();
    const float inv = inv_den;
    uint16_t *dst = (uint16_t *)p.a.out + ((size_t)v.seg_off[seg] * H + c) * R;
    const float *src = p.part + (unit * 32 + blockIdx.z) * R;
    for (int d = threadIdx.x * 4; d < R; d += 512) {
        f32x4 acc[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[i] = f32x4 {0.f, 0.f, 0.f, 0.f};
        for (int s0 = 0; s0 < p.nsplit; s0 += 4) {
            f32x4 x[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) x[i] = *(const f32x4 *)(src + (size_t)(s0 + i < p.nsplit ? s0 + i : p.nsplit - 1) * 32 * R + d);
            // (a part nobody wrote has weight 0 and may hold anything)
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (s0 + i < p.nsplit && w[s0 + i] > 0.0f) acc[i] += x[i] * w[s0 + i];
        }
        const f32x4 y = ((acc[0] + acc[1]) + (acc[2] + acc[3])) * inv;
        *(uint2 *)(dst + d) = make_uint2(pack_pair(y[0], y[1]), pack_pair(y[2], y[3]));
    }
}

// cache rows of positions [base, base + rows) of a slot, side by side
__global__ __launch_bounds__(256) void latent_gather_kernel(StepView v, int slot, int base, const uint16_t *pool, int row_len, uint16_t *out) {
    const size_t src = cache_row(v, slot, base + blockIdx.x) * row_len;
    for (int c = threadIdx.x * 8; c < row_len; c += 2048) *(u32x4 *)(out + (size_t)blockIdx.x * row_len + c) = *(const u32x4 *)(pool + src + c);
}

struct ExpandedParams {
    const uint16_t *q, *k, *vv, *rows; // queries [T][H][D + RD]; keys [ctx][H D], values [ctx][H V]; cache rows [ctx][R + RD]
    uint16_t *out; // [T][H V]
    const float *sink;
    int off, start, n, base, H, D, RD, V, R, window;
    float scale;
};

// BF16, expanded form, for long segments: keys and values of every head made from the latents beforehand.  A workgroup takes
// 128 query tokens of one head (32 a wave) and walks the visible context in blocks of 32 tokens, on 32 x 32 tiles:
//   S^T = K Q^T (A = keys from LDS, B = the wave's queries in registers), O^T += V^T P^T (A = values from LDS read
// transposed, B = probabilities straight from the score registers: half h of the wave holds tokens 8 q + 4 h + s of a block,
// and the value operand takes its tokens in that order).
// KSM: most 16-dim steps of a query; VTM: most 32-dim tiles of a value; EXACT: as many.  grid (heads, query blocks)
template <int KSM, int VTM, bool EXACT>
__global__ __launch_bounds__(256, 2) void latent_expanded_kernel(ExpandedParams p) {
    extern __shared__ unsigned char lds[];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), h = lane >> 5, cl = lane & 31;
    const int head = blockIdx.x, q0 = ((int)gridDim.y - 1 - (int)blockIdx.y) * 128; // the blocks with the longest contexts first
    const int Dq = EXACT ? KSM * 16 : p.D + p.RD, ks_n = Dq / 16, V = EXACT ? VTM * 32 : p.V, vt_n = V / 32;
    const int kpitch = Dq * 2 + 16, vpitch = V * 2 + 16, bufb = 32 * (kpitch + vpitch);
    const int qi = q0 + wave * 32 + cl;
    const int pos = p.start + (qi < p.n ? qi : p.n - 1);
    const int wlo = p.start + q0 + wave * 32, whi_q = q0 + wave * 32 + 31;
    const int whi = p.start + (whi_q < p.n ? whi_q : p.n - 1); // last position of the wave's queries
    const bool wave_on = q0 + wave * 32 < p.n;
    bf16x8 qf[KSM];
    {
        const uint16_t *row = p.q + ((size_t)(p.off + (qi < p.n ? qi : p.n - 1)) * p.H + head) * Dq + 8 * h;
#pragma unroll
        for (int ks = 0; ks < KSM; ++ks)
            if (EXACT || ks < ks_n) qf[ks] = *(const bf16x8 *)(row + ks * 16);
    }
    f32x16 o[VTM];
#pragma unroll
    for (int d = 0; d < VTM; ++d)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[d][r] = 0.0f;
    float m = kUnseen, l = 0.0f;
    const float scale2 = p.scale * kLog2e;
    const int first = p.window > 0 && p.start + q0 + 1 > p.window ? p.start + q0 + 1 - p.window : 0;
    const int last_q = q0 + 127 < p.n ? q0 + 127 : p.n - 1;
    const int b0 = first >> 5, b1 = ((p.start + last_q) >> 5) + 1;
    const int wfirst = p.window > 0 && wlo + 1 > p.window ? wlo + 1 - p.window : 0;

    constexpr int PER = (16 * KSM + 32 * VTM + 63) / 64;
    const int kd = p.D / 8, kr = p.RD / 8, kv8 = V / 8;
    u32x4 stage[PER];
    // chunk e of a block: 32 rows of unrotated keys, of rotated parts, of values (past them: the last one once more)
    const uint16_t *src[PER];
    uint32_t step[PER];
    int dst[PER];
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        int e = i * 256 + threadIdx.x;
        if (e < 32 * kd) {
            const int r = e / kd, c = e % kd;
            step[i] = (uint32_t)(p.H * p.D), src[i] = p.k + (size_t)r * step[i] + (size_t)head * p.D + c * 8, dst[i] = r * kpitch + c * 16;
        } else if ((e -= 32 * kd) < 32 * kr) {
            const int r = e / kr, c = e % kr;
            step[i] = (uint32_t)(p.R + p.RD), src[i] = p.rows + (size_t)r * step[i] + p.R + c * 8, dst[i] = r * kpitch + p.D * 2 + c * 16;
        } else {
            e -= 32 * kr;
            e = e < 32 * kv8 ? e : 32 * kv8 - 1;
            const int r = e / kv8, c = e % kv8;
            step[i] = (uint32_t)(p.H * V), src[i] = p.vv + (size_t)r * step[i] + (size_t)head * V + c * 8, dst[i] = 32 * kpitch + r * vpitch + c * 16;
        }
    }
    // (rows behind the segment's end lie inside the buffers, which hold whole blocks)
    auto fetch = [&](int blk) {
#pragma unroll
        for (int i = 0; i < PER; ++i) stage[i] = *(const u32x4 *)(src[i] + (size_t)(uint32_t)(blk * 32 - p.base) * step[i]);
    };
    fetch(b0);
    int buf = 0;
    for (int blk = b0; blk < b1; ++blk, buf ^= 1) {
        unsigned char *kb = lds + buf * bufb, *vb = kb + 32 * kpitch;
#pragma unroll
        for (int i = 0; i < PER; ++i) *(u32x4 *)(kb + dst[i]) = stage[i];
        __syncthreads();
        if (blk + 1 < b1) fetch(blk + 1);
        const int t0 = blk * 32;
        if (!wave_on || t0 > whi || t0 + 31 < wfirst) continue; // (the same for the whole wave; the barriers above are all there are)
        f32x16 s;
#pragma unroll
        for (int r = 0; r < 16; ++r) s[r] = 0.0f;
        const unsigned char *krow = kb + cl * kpitch + 16 * h;
#pragma unroll
        for (int ks = 0; ks < KSM; ++ks)
            if (EXACT || ks < ks_n) s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*(const bf16x8 *)(krow + ks * 32), qf[ks], s, 0, 0, 0);
        const bool masked = t0 + 31 > wlo || (p.window > 0 && t0 + p.window <= whi);
        float bm = kUnseen;
#pragma unroll
        for (int r = 0; r < 16; ++r) s[r] *= scale2;
        if (masked) {
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                const int t = t0 + 8 * (r >> 2) + 4 * h + (r & 3);
                s[r] = t <= pos && (p.window <= 0 || t > pos - p.window) ? s[r] : kUnseen;
            }
        }
#pragma unroll
        for (int r = 0; r < 16; ++r) bm = fmaxf(bm, s[r]);
        bm = fmaxf(bm, __shfl_xor(bm, 32, 64));
        const float m_new = bm > m + 8.0f ? bm : m; // (the reference point moves only when it has to)
        const float alpha = __builtin_amdgcn_exp2f(m - m_new);
        m = m_new;
        float sum = 0.0f;
#pragma unroll
        for (int r = 0; r < 16; ++r) s[r] = __builtin_amdgcn_exp2f(s[r] - m_new);
        if (masked) {
            // (a column that has seen no key yet has its reference point at the masked score)
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                const int t = t0 + 8 * (r >> 2) + 4 * h + (r & 3);
                s[r] = t <= pos && (p.window <= 0 || t > pos - p.window) ? s[r] : 0.0f;
            }
        }
#pragma unroll
        for (int r = 0; r < 16; ++r) sum += s[r];
        l = l * alpha + sum;
        if (__builtin_amdgcn_ballot_w64(alpha != 1.0f) != 0) {
#pragma unroll
            for (int d = 0; d < VTM; ++d) o[d] *= alpha;
        }
#pragma unroll
        for (int t = 0; t < 2; ++t) {
            float pr[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) pr[j] = s[8 * t + j];
            const bf16x8 pf = pack_bf16x8(pr);
            const unsigned char *vrow = vb + (16 * t + 4 * h + ((lane & 15) >> 2)) * vpitch + 32 * ((lane >> 4) & 1) + 8 * (lane & 3);
#pragma unroll
            for (int d = 0; d < VTM; ++d)
                if (EXACT || d < vt_n) o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(transposed_pair(vrow + d * 64, vrow + d * 64 + 8 * vpitch), pf, o[d], 0, 0, 0);
        }
    }
    l += __shfl_xor(l, 32, 64);
    if (qi >= p.n) return;
    float mul = 1.0f;
    if (p.sink) {
        const float s2 = p.sink[head] * kLog2e, mt = fmaxf(m, s2);
        mul = __builtin_amdgcn_exp2f(m - mt);
        l = l * mul + __builtin_amdgcn_exp2f(s2 - mt);
    }
    mul /= l;
    uint16_t *out = p.out + (size_t)(p.off + qi) * p.H * p.V + (size_t)head * p.V;
#pragma unroll
    for (int d = 0; d < VTM; ++d)
        if (EXACT || d < vt_n) {
#pragma unroll
            for (int q = 0; q < 4; ++q)
                *(uint2 *)(out + d * 32 + 8 * q + 4 * h) =
                        make_uint2(pack_pair(o[d][4 * q] * mul, o[d][4 * q + 1] * mul), pack_pair(o[d][4 * q + 2] * mul, o[d][4 * q + 3] * mul));
        }
}

template <int DT, int KSMAX, bool EXACT>
int launch_mfma(const MfmaParams &p, dim3 grid, size_t smem, hipStream_t st) {
    static const hipError_t attr = hipFuncSetAttribute((const void *)latent_mfma_kernel<DT, KSMAX, EXACT>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    XFT_CHECK_HIP(attr);
    hipLaunchKernelGGL((latent_mfma_kernel<DT, KSMAX, EXACT>), grid, dim3(256), smem, st, p);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}
template <int KSM, int VTM, bool EXACT>
int launch_expanded(const ExpandedParams &p, dim3 grid, size_t smem, hipStream_t st) {
    static const hipError_t attr = hipFuncSetAttribute((const void *)latent_expanded_kernel<KSM, VTM, EXACT>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    XFT_CHECK_HIP(attr);
    hipLaunchKernelGGL((latent_expanded_kernel<KSM, VTM, EXACT>), grid, dim3(256), smem, st, p);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

// does the matrix-unit form of the absorbed attention take this layer
bool mfma_takes(const PlanLayer &L) {
    const int ks = (L.R + L.RD) / 32;
    return (L.R <= 64 && ks <= 6) || (L.R <= 128 && ks <= 8) || (L.R <= 256 && ks <= 12) || (L.R <= 512 && ks <= 20);
}

} // namespace

int latent_prepare(int act, const PlanLayer &L, const StepView &v, const void *a, void *cq, const LatentCacheView &cache, float eps, hipStream_t st) {
    const PrepareParams p = {v, a, cq, cache, L.q_norm, L.kv_norm, L.cosT, L.sinT, L.QR, L.RD, L.s.q_rank, L.s.kv_rank, L.s.rot_dim,
            L.s.rot_interleaved, eps};
    const int ch = (L.QR + L.R + 2047) / 2048;
    XFT_REQUIRE(ch <= 4, "latent_prepare: latents of %d + %d values too wide", L.QR, L.R);
    if (act == XFTHIP_BF16) {
        if (ch == 1) hipLaunchKernelGGL((latent_prepare_kernel<true, 1>), dim3(v.T), dim3(256), 0, st, p);
        else hipLaunchKernelGGL((latent_prepare_kernel<true, 4>), dim3(v.T), dim3(256), 0, st, p);
    } else {
        if (ch == 1) hipLaunchKernelGGL((latent_prepare_kernel<false, 1>), dim3(v.T), dim3(256), 0, st, p);
        else hipLaunchKernelGGL((latent_prepare_kernel<false, 4>), dim3(v.T), dim3(256), 0, st, p);
    }
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

int latent_rotate_q(int act, const PlanLayer &L, const StepView &v, void *q, hipStream_t st) {
    const int half = L.s.rot_dim / 2;
    if (half == 0) return 0;
    const unsigned blocks = (unsigned)(((size_t)v.T * L.s.heads * ((half + 3) / 4) + 255) / 256);
    if (act == XFTHIP_BF16)
        hipLaunchKernelGGL(rotate_q_kernel<true>, dim3(blocks), dim3(256), 0, st, v, q, v.T, L.s.heads, L.D, L.RD, half, L.s.rot_interleaved, L.cosT, L.sinT);
    else
        hipLaunchKernelGGL(rotate_q_kernel<false>, dim3(blocks), dim3(256), 0, st, v, q, v.T, L.s.heads, L.D, L.RD, half, L.s.rot_interleaved, L.cosT, L.sinT);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

// Parts a context of `hint` tokens is split into: as many as give every compute unit a workgroup, blocks of 32 tokens permitting.
int latent_split_count(const PlanLayer &L, int B, int longest, int hint) {
    if (!mfma_takes(L)) return 1;
    const long units = (long)B * ((longest * L.s.heads + 31) / 32);
    const int ctx = L.s.window > 0 && L.s.window + longest < hint ? L.s.window + longest : hint;
    const int blocks = (ctx + 31) / 32;
    long want = device_cu_count() / units; // (two a compute unit: no faster, and twice the merge)
    want = want < blocks ? want : blocks;
    want = want < kMaxSplits / 2 ? want : kMaxSplits / 2; // (more parts cost more in the merge than they save)
    return want < 1 ? 1 : (int)want;
}

size_t latent_part_floats(const PlanLayer &L) { return mfma_takes(L) ? (size_t)device_cu_count() * 32 * (L.R + 2) : 0; }

int latent_attention(int act, const PlanLayer &L, const StepView &v, int longest, const void *qa, const void *q, void *out, const LatentCacheView &cache,
        int hint, float *part, size_t part_floats, hipStream_t st) {
    const AttendParams a = {v, qa, q, out, cache, L.sink, L.s.heads, L.D, L.s.window, longest, L.s.scale};
    if (act == XFTHIP_BF16 && mfma_takes(L)) {
        MfmaParams p = {a, L.RD, latent_split_count(L, v.B, longest, hint), longest, part, 0};
        const unsigned groups = (unsigned)((longest * L.s.heads + 31) / 32);
        const size_t slots = (size_t)v.B * groups * p.nsplit * 32;
        p.part_ml = slots * L.R;
        XFT_REQUIRE(p.nsplit == 1 || slots * (L.R + 2) <= part_floats, "latent_attention: workspace too small for %zu partial columns", slots);
        const dim3 grid(groups, v.B, p.nsplit);
        const size_t smem = (size_t)2 * 32 * ((L.R + L.RD) * 2 + 16) + 32 * 36 * 4;
        const int ks = (L.R + L.RD) / 32;
        int rc;
        if (L.R == 512 && ks == 18) rc = launch_mfma<8, 18, true>(p, grid, smem, st);
        else if (L.R == 512 && ks == 17) rc = launch_mfma<8, 17, true>(p, grid, smem, st);
        else if (L.R == 256 && ks == 10) rc = launch_mfma<4, 10, true>(p, grid, smem, st);
        else if (L.R == 256 && ks == 9) rc = launch_mfma<4, 9, true>(p, grid, smem, st);
        else if (L.R == 128 && ks == 6) rc = launch_mfma<2, 6, true>(p, grid, smem, st);
        else if (L.R == 128 && ks == 5) rc = launch_mfma<2, 5, true>(p, grid, smem, st);
        else if (L.R == 64 && ks == 3) rc = launch_mfma<1, 3, true>(p, grid, smem, st);
        else if (L.R <= 64 && ks <= 6) rc = launch_mfma<1, 6, false>(p, grid, smem, st);
        else if (L.R <= 128 && ks <= 8) rc = launch_mfma<2, 8, false>(p, grid, smem, st);
        else if (L.R <= 256 && ks <= 12) rc = launch_mfma<4, 12, false>(p, grid, smem, st);
        else rc = launch_mfma<8, 20, false>(p, grid, smem, st);
        if (rc || p.nsplit == 1) return rc;
        hipLaunchKernelGGL(latent_merge_kernel, dim3(groups, v.B, 32), dim3(128), 0, st, p);
        XFT_CHECK_HIP(hipGetLastError());
        return 0;
    }
    const size_t smem = (size_t)(2 * L.R + L.RD + 256 + 8) * 4 + 256 * 8;
    XFT_REQUIRE(smem <= 64 * 1024, "latent_attention: latent of %d values too wide", L.R);
    if (act == XFTHIP_BF16)
        hipLaunchKernelGGL(latent_attend_kernel<true>, dim3(v.T, L.s.heads), dim3(256), smem, st, a);
    else
        hipLaunchKernelGGL(latent_attend_kernel<false>, dim3(v.T, L.s.heads), dim3(256), smem, st, a);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

bool latent_expanded_takes(int act, const PlanLayer &L, int n, int ctx) {
    if (act != XFTHIP_BF16 || n < 32) return false;
    const int ks = (L.D + L.RD) / 16, vt = L.V / 32;
    if (!((ks <= 4 && vt <= 2) || (ks <= 8 && vt <= 4) || (ks <= 12 && vt <= 4))) return false;
    // what the narrower products save against making keys and values of the context that came before
    return (double)n * ctx * (2.0 * L.R - L.D - L.V) >= (double)(ctx - n) * L.R * (L.D + L.V);
}

int latent_gather(const StepView &v, int slot, int base, int rows, const LatentCacheView &cache, void *out, hipStream_t st) {
    hipLaunchKernelGGL(latent_gather_kernel, dim3(rows), dim3(256), 0, st, v, slot, base, (const uint16_t *)cache.pool, cache.R + cache.RD, (uint16_t *)out);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

int latent_expanded(const PlanLayer &L, int off, int start, int n, int base, const void *q, const void *k, const void *values, const void *rows, void *out,
        hipStream_t st) {
    const ExpandedParams p = {(const uint16_t *)q, (const uint16_t *)k, (const uint16_t *)values, (const uint16_t *)rows, (uint16_t *)out, L.sink, off, start, n,
            base, L.s.heads, L.D, L.RD, L.V, L.R, L.s.window, L.s.scale};
    const dim3 grid(L.s.heads, (n + 127) / 128);
    const size_t smem = (size_t)2 * 32 * ((L.D + L.RD) * 2 + 16 + L.V * 2 + 16);
    const int ks = (L.D + L.RD) / 16, vt = L.V / 32;
    if (ks == 12 && vt == 4) return launch_expanded<12, 4, true>(p, grid, smem, st);
    if (ks == 10 && vt == 4) return launch_expanded<10, 4, true>(p, grid, smem, st);
    if (ks == 8 && vt == 4) return launch_expanded<8, 4, true>(p, grid, smem, st);
    if (ks == 6 && vt == 2) return launch_expanded<6, 2, true>(p, grid, smem, st);
    if (ks == 4 && vt == 1) return launch_expanded<4, 1, true>(p, grid, smem, st);
    if (ks <= 4 && vt <= 2) return launch_expanded<4, 2, false>(p, grid, smem, st);
    if (ks <= 8 && vt <= 4) return launch_expanded<8, 4, false>(p, grid, smem, st);
    return launch_expanded<12, 4, false>(p, grid, smem, st);
}

} // namespace xfthip
