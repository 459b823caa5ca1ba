// Grouped attention of layer plans: every key / value head serves a group of query heads; keys and values live in pages.
//
// A page holds, head after head, 64 keys [64][D] and two blocks of 32 tokens of values with the tokens innermost, [V][32]:
// both are then operands of the matrix units as they lie in memory.
//
// Short form (decoded tokens, short portions): 16 columns - neighbouring (token, query head) pairs of one key / value head - a
// workgroup, straight from memory, the context split over the four waves and over workgroups.  Long form: 128 columns a
// workgroup, blocks of 32 tokens through LDS.  Scores come out as S^T = K Q^T with the tokens along the registers, in an order
// chosen (by the row of the key operand a token is put in) so that a lane's probabilities are those of eight neighbouring
// tokens: the operand of O^T += V^T P^T, whose other side is one 16-byte read.
//
// What a window leaves out but a position sees all the same - the first tokens of the sequence, or the means of whole blocks of tokens,
// which have pages of their own - is a number of blocks in front of the window's: both forms walk them like the others.
// The two values of a rotated pair are neighbours (PlanLayer::head_place).
#include "plan_dev.h"

namespace xfthip {

namespace {

// first element of a head's part of the page that holds position `pos`
__device__ inline size_t head_page(const int *table, int pos, int G, int g, int D, int V) {
    return ((size_t)table[pos / kPageTokens] * G + g) * kPageTokens * (D + V);
}
// element of a value behind a head's keys: token `i` of the page, dimension d
__device__ inline size_t value_at(int D, int V, int i, int d) { return (size_t)kPageTokens * D + ((size_t)(i >> 5) * V + d) * 32 + (i & 31); }

struct PrepareParams {
    StepView v;
    GroupedBuffers b;
    const float *q_norm, *k_norm, *cosT, *sinT; // norms may be null
    const float *cosV, *sinV; // rotation of the values, or null
    const uint16_t *filter; // [taps][channels] bf16, or null
    int taps, channels;
    int normed; // heads are divided by their root mean square (with or without weights)
    int pool; // tokens of a block whose mean is kept, or 0
    int ld, value_col; // pitch of a's rows, first column of the values
    int H, G, D, V, dim, vdim, rot, lanes; // lanes a head takes (a power of two, 8 values each)
    int h0, h1; // heads to move, key heads behind the query heads
    int all; // norms over all query heads, all key heads: a workgroup a token
    int v_blocks, seg_blocks, keep; // keep: write first_values
    float share, eps; // share of first_values in the values
};

// Eight neighbouring channels of token t's row from c on, behind their filter.  TAPS: of the filter (0: none, -1: any number).  The only new
// token of a sequence shifts the filter's inputs in place: a channel belongs to one thread.  (longer segments: conv_tail)
template <bool BF16, int TAPS>
__device__ inline void filtered8(const PrepareParams &p, int t, int c, float (&x)[8]) {
    load8<BF16>(p.b.a, (size_t)t * p.ld + c, x);
    if constexpr (TAPS == 0) return;
    const int seg = p.v.tok_seg[t], pos = p.v.tok_pos[t], local = t - p.v.seg_off[seg], keep = TAPS > 0 ? TAPS - 1 : p.taps - 1;
    const size_t hist = (size_t)p.v.seg_row[seg] * keep * p.channels + c;
    const bool alone = p.v.seg_len[seg] == 1;
    // the input `back` tokens before this one: of the step, or kept from earlier ones (nothing in front of the sequence, but something to read)
    auto input = [&](int back, float (&in)[8]) {
        const bool here = local >= back;
        load8<BF16>(here ? p.b.a : p.b.conv_state, here ? (size_t)(t - back) * p.ld + c : hist + (size_t)(keep + local - back) * p.channels, in);
    };
    float y[8];
    if constexpr (TAPS > 0) {
        float in[TAPS][8], w[TAPS][8];
#pragma unroll
        for (int back = 0; back < TAPS; ++back) {
            if (back > 0) input(back, in[back]);
            load8<true>(p.filter, (size_t)(keep - back) * p.channels + c, w[back]);
        }
#pragma unroll
        for (int k = 0; k < 8; ++k) in[0][k] = x[k], y[k] = w[0][k] * x[k];
#pragma unroll
        for (int back = 1; back < TAPS; ++back)
#pragma unroll
            for (int k = 0; k < 8; ++k) y[k] = fmaf(w[back][k], back <= pos ? in[back][k] : 0.0f, y[k]);
        if (alone) {
#pragma unroll
            for (int s = 0; s < TAPS - 1; ++s) store8<BF16>(p.b.conv_state, hist + (size_t)s * p.channels, in[TAPS - 2 - s]);
        }
    } else {
        float in[8], w[8];
        load8<true>(p.filter, (size_t)keep * p.channels + c, w);
#pragma unroll
        for (int k = 0; k < 8; ++k) y[k] = w[k] * x[k];
        for (int back = 1; back <= keep && back <= pos; ++back) {
            input(back, in);
            load8<true>(p.filter, (size_t)(keep - back) * p.channels + c, w);
#pragma unroll
            for (int k = 0; k < 8; ++k) y[k] = fmaf(w[k], in[k], y[k]);
        }
        if (alone && keep > 0) {
            for (int s = 0; s + 1 < keep; ++s) {
                load8<BF16>(p.b.conv_state, hist + (size_t)(s + 1) * p.channels, in);
                store8<BF16>(p.b.conv_state, hist + (size_t)s * p.channels, in);
            }
            store8<BF16>(p.b.conv_state, hist + (size_t)(keep - 1) * p.channels, x);
        }
    }
#pragma unroll
    for (int k = 0; k < 8; ++k) x[k] = y[k];
}

// N / 2 neighbouring pairs from dimension c (a multiple of N) on, turned by the angles of their tables' row (or back)
template <int N, bool BACK, class X>
__device__ inline void turn_pairs(X &x, const float *cs, const float *sn, int c, int half) {
    const int first = c / 2;
    if (first >= half) return;
    float cc[N / 2], ss[N / 2];
    if (N == 8 && half % 4 == 0) {
        const f32x4 a = *(const f32x4 *)(cs + first), b = *(const f32x4 *)(sn + first);
#pragma unroll
        for (int k = 0; k < N / 2; ++k) cc[k] = a[k], ss[k] = b[k];
    } else {
#pragma unroll
        for (int k = 0; k < N / 2; ++k) { // (past the rotated part: its last pair's, unused)
            const int i = first + k < half ? first + k : half - 1;
            cc[k] = cs[i], ss[k] = sn[i];
        }
    }
#pragma unroll
    for (int k = 0; k < N / 2; ++k) {
        const float u = x[2 * k], z = x[2 * k + 1], turn = BACK ? -ss[k] : ss[k];
        const bool on = first + k < half;
        x[2 * k] = on ? fmaf(u, cc[k], -(z * turn)) : u, x[2 * k + 1] = on ? fmaf(z, cc[k], u * turn) : z;
    }
}

template <bool BF16>
__device__ inline float stored(float x) { // as memory holds it
    if constexpr (BF16) return bf16_to_f32(f32_to_bf16_ref(x));
    else return x;
}

// Eight values of a head from c on, normed (r: factor of the norm, or 1) and rotated, to q or into the page
template <bool BF16>
__device__ inline void move_values(const PrepareParams &p, int t, int hh, int c, float (&x)[8], float r) {
    const int D = p.D, H = p.H, G = p.G;
    const float *norm = hh < H ? p.q_norm : p.k_norm;
    if (norm && p.all) norm += (size_t)(hh < H ? hh : hh - H) * D;
    float w[8];
#pragma unroll
    for (int k = 0; k < 8; ++k) w[k] = 1.0f;
    if (norm) load8<false>(norm, c, w);
#pragma unroll
    for (int k = 0; k < 8; ++k) x[k] = x[k] * r * w[k];
    const int pos = p.v.tok_pos[t], half = p.rot / 2;
    turn_pairs<8, false>(x, p.cosT + (size_t)pos * half, p.sinT + (size_t)pos * half, c, half);
    if (hh < H) {
        store8<BF16>(p.b.q, ((size_t)t * H + hh) * D + c, x);
        return;
    }
    const int seg = p.v.tok_seg[t], slot = p.v.seg_row[seg];
    const int *table = p.v.table + (size_t)slot * p.v.table_stride;
    store8<BF16>(p.b.pool, head_page(table, pos, G, hh - H, D, p.V) + (size_t)(pos % kPageTokens) * D + c, x);
    if (p.pool == 0 || p.v.seg_len[seg] != 1 || (pos + 1) % p.pool != 0) return;
    // the only new token of a sequence, and its block is full: the others of the block are there already
#pragma unroll
    for (int k = 0; k < 8; ++k) x[k] = stored<BF16>(x[k]);
    for (int j = pos - p.pool + 1; j < pos; ++j) {
        load8<BF16>(p.b.pool, head_page(table, j, G, hh - H, D, p.V) + (size_t)(j % kPageTokens) * D + c, w);
#pragma unroll
        for (int k = 0; k < 8; ++k) x[k] += w[k];
    }
#pragma unroll
    for (int k = 0; k < 8; ++k) x[k] /= (float)p.pool;
    const int block = pos / p.pool;
    store8<BF16>(p.b.means, head_page(p.b.means_table + (size_t)slot * p.b.means_stride, block, G, hh - H, D, p.V) + (size_t)(block % kPageTokens) * D + c, x);
}

// One launch, two kinds of workgroups.  The first v_blocks: one head's values of up to 32 tokens (a block of the cache), turned round through
// LDS (the longer way, so they go first).  The others: a group of `lanes` threads one query or key head of a token (norms over all heads: a
// workgroup a token).
template <bool BF16, int TAPS>
__global__ __launch_bounds__(256) void grouped_prepare_kernel(PrepareParams p) {
    const int D = p.D, V = p.V, H = p.H, G = p.G;
    if ((int)blockIdx.x >= p.v_blocks && p.all) {
        __shared__ float part[8];
        const int t = (int)blockIdx.x - p.v_blocks, q_end = H * D, end = p.h1 * D; // (h0 is 0)
        const size_t row = (size_t)t * p.ld;
        float sq = 0.0f, sk = 0.0f;
        for (int e = threadIdx.x * 8; e < end; e += 2048) {
            float x[8], sum = 0.0f;
            load8<BF16>(p.b.a, row + e, x);
#pragma unroll
            for (int k = 0; k < 8; ++k) sum = fmaf(x[k], x[k], sum);
            if (e < q_end) sq += sum;
            else sk += sum;
        }
        sq = wave_total(sq), sk = wave_total(sk);
        if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = sq, part[4 + (threadIdx.x >> 6)] = sk;
        __syncthreads();
        const float rq = 1.0f / sqrtf(((part[0] + part[1]) + (part[2] + part[3])) / (float)(H * p.dim) + p.eps);
        const float rk = 1.0f / sqrtf(((part[4] + part[5]) + (part[6] + part[7])) / (float)(G * p.dim) + p.eps);
        for (int e = threadIdx.x * 8; e < end; e += 2048) {
            float x[8];
            load8<BF16>(p.b.a, row + e, x);
            move_values<BF16>(p, t, e / D, e % D, x, e < q_end ? rq : rk);
        }
        return;
    }
    if ((int)blockIdx.x >= p.v_blocks) {
        const size_t idx = (size_t)((int)blockIdx.x - p.v_blocks) * 256 + threadIdx.x;
        const size_t item = idx / p.lanes;
        const int c = (int)(idx % p.lanes) * 8, heads = p.h1 - p.h0;
        const bool on = item < (size_t)p.v.T * heads && c < D;
        const int t = on ? (int)(item / heads) : 0, hh = on ? (int)(item % heads) + p.h0 : p.h0;
        float x[8];
#pragma unroll
        for (int k = 0; k < 8; ++k) x[k] = 0.0f;
        if (on) filtered8<BF16, TAPS>(p, t, hh * D + c, x);
        float r = 1.0f;
        if (p.normed) {
            float sq = 0.0f;
#pragma unroll
            for (int k = 0; k < 8; ++k) sq = fmaf(x[k], x[k], sq);
            for (int off = p.lanes / 2; off > 0; off >>= 1) sq += __shfl_xor(sq, off, 64);
            r = 1.0f / sqrtf(sq / (float)p.dim + p.eps);
        }
        if (on) move_values<BF16>(p, t, hh, c, x, r);
        return;
    }
    __shared__ float tile[32][129];
    int job = blockIdx.x;
    const int g = job % G;
    job /= G;
    const int seg = job / p.seg_blocks, start = p.v.seg_pos[seg], n = p.v.seg_len[seg], off = p.v.seg_off[seg];
    const int b0 = ((start >> 5) + job % p.seg_blocks) * 32; // positions b0 .. b0 + 31
    if (b0 >= start + n) return;
    const int lo = start > b0 ? start : b0, hi = start + n < b0 + 32 ? start + n : b0 + 32;
    const int *table = p.v.table + (size_t)p.v.seg_row[seg] * p.v.table_stride;
    const size_t dst = head_page(table, b0, G, g, D, V);
    for (int d0 = 0; d0 < V; d0 += 128) {
        const int slice = V - d0 < 128 ? V - d0 : 128;
        if (d0) __syncthreads();
        for (int i = threadIdx.x; i < (hi - lo) * (slice / 8); i += 256) {
            const int tok = lo + i / (slice / 8), c = i % (slice / 8) * 8, t = off + tok - start;
            const size_t first = ((size_t)t * G + g) * V + d0 + c;
            float x[8];
            filtered8<BF16, TAPS>(p, t, p.value_col + g * V + d0 + c, x);
            if (p.cosV) {
                const size_t row = (size_t)tok * (p.vdim / 2);
                turn_pairs<8, false>(x, p.cosV + row, p.sinV + row, d0 + c, p.vdim / 2);
            }
            if (p.keep) {
                store8<BF16>(p.b.first_values, first, x);
            } else if (p.share != 0.0f) {
                float y[8];
                load8<BF16>(p.b.first_values, first, y);
#pragma unroll
                for (int k = 0; k < 8; ++k) x[k] = (1.0f - p.share) * x[k] + p.share * y[k];
            }
#pragma unroll
            for (int k = 0; k < 8; ++k) tile[tok - b0][c + k] = x[k];
        }
        __syncthreads();
        for (int i = threadIdx.x; i < slice * 4; i += 256) {
            const int d = i >> 2, t8 = (i & 3) * 8;
            if (b0 + t8 >= hi || b0 + t8 + 8 <= lo) continue;
            const size_t at = dst + value_at(D, V, (b0 & 32) + t8, d0 + d);
            if (b0 + t8 >= lo && b0 + t8 + 8 <= hi) {
                float x[8];
#pragma unroll
                for (int k = 0; k < 8; ++k) x[k] = tile[t8 + k][d];
                store8<BF16>(p.b.pool, at, x);
            } else {
                for (int k = 0; k < 8; ++k)
                    if (b0 + t8 + k >= lo && b0 + t8 + k < hi) stact<BF16>(p.b.pool, at + k, tile[t8 + k][d]);
            }
        }
        if (p.pool == 0 || n != 1 || (start + 1) % p.pool != 0) continue; // (as for keys)
        for (int d = threadIdx.x; d < slice; d += 256) {
            float sum = stored<BF16>(tile[start - b0][d]);
            for (int j = start - p.pool + 1; j < start; ++j)
                sum += ldact<BF16>(p.b.pool, head_page(table, j, G, g, D, V) + value_at(D, V, j % kPageTokens, d0 + d));
            const int block = start / p.pool;
            stact<BF16>(p.b.means, head_page(p.b.means_table + (size_t)p.v.seg_row[seg] * p.b.means_stride, block, G, g, D, V)
                    + value_at(D, V, block % kPageTokens, d0 + d), sum / (float)p.pool);
        }
    }
}

// Means of the blocks that segments of several tokens fill: a workgroup one block of one head.  grid (heads * blocks, segments)
template <bool BF16>
__global__ __launch_bounds__(256) void grouped_means_kernel(PrepareParams p) {
    const int D = p.D, V = p.V, G = p.G, seg = blockIdx.y, n = p.v.seg_len[seg], start = p.v.seg_pos[seg], g = blockIdx.x % G;
    const int block = start / p.pool + (int)(blockIdx.x / G);
    if (n == 1 || (block + 1) * p.pool > start + n) return;
    const int *table = p.v.table + (size_t)p.v.seg_row[seg] * p.v.table_stride;
    const size_t dst = head_page(p.b.means_table + (size_t)p.v.seg_row[seg] * p.b.means_stride, block, G, g, D, V);
    const int first = block * p.pool, end = first + p.pool;
    const float inv = 1.0f / (float)p.pool;
    // keys: p.lanes threads a token, the sets of threads take turns; values: a thread a dimension
    __shared__ float sums[256 * 8];
    const int sets = 256 / p.lanes, set = (int)threadIdx.x / p.lanes, c = (int)threadIdx.x % p.lanes * 8;
    float x[8] = {0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f};
    for (int j = first + set; j < end && c < D; j += sets) {
        float w[8];
        load8<BF16>(p.b.pool, head_page(table, j, G, g, D, V) + (size_t)(j % kPageTokens) * D + c, w);
#pragma unroll
        for (int k = 0; k < 8; ++k) x[k] += w[k];
    }
#pragma unroll
    for (int k = 0; k < 8; ++k) sums[k * 256 + threadIdx.x] = x[k];
    for (int d = threadIdx.x; d < V; d += 256) {
        float sum = 0.0f;
        for (int j = first; j < end;) { // (runs of tokens of a value block, eight at a time where they are whole)
            const size_t at = head_page(table, j, G, g, D, V) + value_at(D, V, j % kPageTokens, d);
            if (j % 8 == 0 && j + 8 <= end) {
                float w[8];
                load8<BF16>(p.b.pool, at, w);
                sum += ((w[0] + w[1]) + (w[2] + w[3])) + ((w[4] + w[5]) + (w[6] + w[7]));
                j += 8;
            } else {
                sum += ldact<BF16>(p.b.pool, at);
                ++j;
            }
        }
        stact<BF16>(p.b.means, dst + value_at(D, V, block % kPageTokens, d), sum * inv);
    }
    __syncthreads();
    if (set > 0 || c >= D) return;
#pragma unroll
    for (int k = 0; k < 8; ++k) {
        x[k] = 0.0f;
        for (int t = 0; t < sets && t < p.pool; ++t) x[k] += sums[k * 256 + t * p.lanes + threadIdx.x];
        x[k] *= inv;
    }
    store8<BF16>(p.b.means, dst + (size_t)(block % kPageTokens) * D + c, x);
}

struct AttendParams {
    StepView v;
    const void *q, *pool;
    int q_ld; // pitch of a token's queries
    void *out; // rows of pitch out_ld
    int out_ld;
    const float *sink; // or null
    // the output: times out_scale, times sigmoid(gate) of every element or head (rows of pitch gate_ld, of the activation type)
    const void *gate;
    int gate_kind, gate_ld;
    float out_scale;
    float softcap; // or 0
    int distance_bias;
    int H, G, D, V, window, chunk;
    // in front of the window: first tokens that stay visible, or means of blocks of `block` tokens
    int keep_first, block;
    const void *means;
    const int *means_table;
    int means_stride;
    const float *cosV, *sinV; // outputs are turned back by their position, or null
    int vhalf;
    int min_len, max_len; // segments of other lengths are somebody else's
    float scale;
    int nsplit, groups; // context splits; column groups of the longest segment
    float *part; // [segments][G * groups][nsplit][16][V] outputs, behind them as many [2] maxima and sums
    size_t part_ml;
};

// first position that position `pos` sees
__device__ inline int first_seen(const AttendParams &p, int pos) {
    if (p.chunk > 0) return pos - pos % p.chunk;
    return p.window > 0 && pos + 1 > p.window ? pos + 1 - p.window : 0;
}
// entries in front of the window that position `pos` sees (kept first tokens: those that the window does not reach)
__device__ inline int front_seen(const AttendParams &p, int pos) {
    if (p.block == 0) return p.keep_first;
    return pos + 1 - p.window >= p.block ? (pos + 1 - p.window) / p.block : 0;
}
// a position's outputs from dimension d on, turned back
template <int N, class X>
__device__ inline void turn_back(const AttendParams &p, int pos, int d, X &x) {
    if (p.cosV) turn_pairs<N, true>(x, p.cosV + (size_t)pos * p.vhalf, p.sinV + (size_t)pos * p.vhalf, d, p.vhalf);
}
// what a token of distance costs head h
__device__ inline float head_slope(const AttendParams &p, int h) { return p.distance_bias ? exp2f(-8.0f * (float)(h + 1) / (float)p.H) : 0.0f; }

// factors on four neighbouring outputs of a bf16 row
__device__ inline f32x4 output_gate(const AttendParams &p, int t, int head, int d) {
    f32x4 f = {p.out_scale, p.out_scale, p.out_scale, p.out_scale};
    const uint16_t *row = (const uint16_t *)p.gate + (size_t)t * p.gate_ld;
    if (p.gate_kind == XFTHIP_GATE_ELEMENT) {
        const uint2 u = *(const uint2 *)(row + (size_t)head * p.V + d);
        const f32x4 z = {u2f(u.x << 16), u2f(u.x & 0xFFFF0000u), u2f(u.y << 16), u2f(u.y & 0xFFFF0000u)};
#pragma unroll
        for (int k = 0; k < 4; ++k) f[k] *= __builtin_amdgcn_rcpf(1.0f + fast_exp(-z[k]));
    } else if (p.gate_kind == XFTHIP_GATE_HEAD) {
        f *= __builtin_amdgcn_rcpf(1.0f + fast_exp(-bf16_to_f32(row[head])));
    }
    return f;
}

// Scores that are more than a scaled product, in units of log2: a cap and a cost of distance
struct ScoreRule {
    float twice, cap2, slope2; // 2 log2(e) scale / cap, cap log2(e), slope log2(e)
    __device__ inline float operator()(float s, float scale2, float distance) const {
        // cap tanh(x / cap) = cap (1 - 2 / (exp(2 x / cap) + 1))
        const float x = cap2 > 0.0f ? cap2 * fmaf(-2.0f, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s * twice) + 1.0f), 1.0f) : s * scale2;
        return fmaf(-slope2, distance, x);
    }
    // N scores of a column; value r stands ahead(r) tokens closer than `distance`
    template <int N, class S, class F>
    __device__ inline void all(S &s, float scale2, float distance, F ahead) const {
        const float far = -slope2 * distance;
        if (cap2 > 0.0f) {
#pragma unroll
            for (int r = 0; r < N; ++r)
                s[r] = fmaf(-2.0f * cap2, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s[r] * twice) + 1.0f), fmaf(slope2, ahead(r), cap2 + far));
        } else {
#pragma unroll
            for (int r = 0; r < N; ++r) s[r] = fmaf(s[r], scale2, fmaf(slope2, ahead(r), far));
        }
    }
};
__device__ inline ScoreRule score_rule(const AttendParams &p, int head) {
    const bool cap = p.softcap > 0.0f;
    return ScoreRule {cap ? 2.0f * kLog2e * p.scale / p.softcap : 0.0f, cap ? p.softcap * kLog2e : 0.0f, head_slope(p, head) * kLog2e};
}

// Any type, any size: one workgroup a (token, head), 256 keys at a time, a key a thread for the scores and a value
// dimension a thread for the weighted sum.
template <bool BF16>
__global__ __launch_bounds__(256) void grouped_attend_kernel(AttendParams p) {
    extern __shared__ float smem[];
    const int D = p.D, V = p.V;
    float *qs = smem, *ps = qs + D, *o = ps + 256, *part = o + V;
    const int t = blockIdx.x, h = blockIdx.y, g = h / (p.H / p.G);
    const int seg = p.v.tok_seg[t], pos = p.v.tok_pos[t];
    const int *table = p.v.table + (size_t)p.v.seg_row[seg] * p.v.table_stride;
    for (int c = threadIdx.x; c < D; c += 256) qs[c] = ldact<BF16>(p.q, (size_t)t * p.q_ld + (size_t)h * D + c);
    for (int c = threadIdx.x; c < V; c += 256) o[c] = 0.0f;
    const int first = first_seen(p, pos);
    const float slope = head_slope(p, h);
    float m = p.sink ? p.sink[h] : -INFINITY, l = p.sink ? 1.0f : 0.0f; // the sink has no key and no value
    __syncthreads();
    // the entries in front of the window, then the window's
    const int front = front_seen(p, pos), ahead = p.block == 0 && front > first ? first : front;
    for (int stretch = 0; stretch < 2; ++stretch) {
        const bool mean = stretch == 0 && p.block > 0;
        const int begin = stretch ? first : 0, end = stretch ? pos : ahead - 1;
        const void *pool = mean ? p.means : p.pool;
        const int *pages = mean ? p.means_table + (size_t)p.v.seg_row[seg] * p.means_stride : table;
        for (int k0 = begin; k0 <= end; k0 += 256) {
            const int j = k0 + threadIdx.x;
            float s = -INFINITY;
            if (j <= end) {
                const size_t at = head_page(pages, j, p.G, g, D, V) + (size_t)(j % kPageTokens) * D;
                float acc = 0.0f;
                for (int c = 0; c < D; c += 8) {
                    float k[8];
                    load8<BF16>(pool, at + c, k);
    #pragma unroll
                    for (int i = 0; i < 8; ++i) acc = fmaf(qs[c + i], k[i], acc);
                }
                s = acc * p.scale;
                if (p.softcap > 0.0f) s = p.softcap * tanhf(s / p.softcap);
                s -= slope * (float)(pos - j);
            }
            const float mx = wave_largest(s);
            if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = mx;
            __syncthreads();
            const float m_new = fmaxf(fmaxf(fmaxf(part[0], part[1]), fmaxf(part[2], part[3])), m);
            const float alpha = expf(m - m_new); // (0 while nothing has been seen)
            const float e = j <= end ? expf(s - m_new) : 0.0f;
            ps[threadIdx.x] = e;
            const float sum = wave_total(e);
            if ((threadIdx.x & 63) == 0) part[4 + (threadIdx.x >> 6)] = sum;
            __syncthreads();
            l = l * alpha + ((part[4] + part[5]) + (part[6] + part[7]));
            m = m_new;
            const int n = end - k0 + 1 < 256 ? end - k0 + 1 : 256;
            for (int c = threadIdx.x; c < V; c += 256) {
                float acc = o[c] * alpha;
                for (int i = 0; i < n;) {
                    // the run of tokens up to the end of a value block
                    const int at = k0 + i, run = 32 - (at & 31) < n - i ? 32 - (at & 31) : n - i;
                    const size_t src = head_page(pages, at, p.G, g, D, V) + value_at(D, V, at % kPageTokens, c);
                    for (int k = 0; k < run; ++k) acc = fmaf(ps[i + k], ldact<BF16>(pool, src + k), acc);
                    i += run;
                }
                o[c] = acc;
            }
            __syncthreads();
        }
    }
    for (int c = threadIdx.x; c < V; c += 256) {
        float y[2] = {o[c & ~1], o[c | 1]}; // (V is even)
        turn_back<2>(p, pos, c & ~1, y);
        y[0] = (c & 1 ? y[1] : y[0]) / l * p.out_scale;
        if (p.gate_kind) y[0] /= 1.0f + expf(-ldact<BF16>(p.gate, (size_t)t * p.gate_ld + (p.gate_kind == XFTHIP_GATE_HEAD ? h : h * V + c)));
        stact<BF16>(p.out, (size_t)t * p.out_ld + (size_t)h * V + c, y[0]);
    }
}

// What the kernels know beforehand: plain scores; scores that are capped or pay for distance; entries in front of a window, with either
// kind of score, and outputs that are turned back
enum { kPlain, kRule, kFront };

// The blocks of 32 entries that columns of positions lo .. hi see: those in front of the window, then the window's.  For `kFront`
struct FrontBlocks {
    int n, seen_lo, keep; // blocks; entries that the first column sees; kept first tokens (0: means)
    const uint16_t *means;
    const int *table;
};
__device__ inline FrontBlocks front_blocks(const AttendParams &p, int slot, int lo, int hi) {
    FrontBlocks f;
    if (p.block > 0) {
        f.n = (front_seen(p, hi) + 31) >> 5, f.seen_lo = front_seen(p, lo), f.keep = 0;
    } else {
        const int b0 = first_seen(p, lo) >> 5, n = (p.keep_first + 31) >> 5;
        f.n = n < b0 ? n : b0, f.seen_lo = f.keep = p.keep_first;
    }
    f.means = (const uint16_t *)p.means, f.table = p.means_table + (size_t)slot * p.means_stride;
    return f;
}

// BF16, short form.  KS: most 32-dim steps of a key; VT: most 16-dim tiles of a value; EXACT: as many; FORM: see above.
// grid (splits, G * column groups, segments)
template <int KS, int VT, bool EXACT, int FORM>
__global__ __launch_bounds__(256, (KS <= 4 && VT <= 8) ? 3 : 1) void grouped_short_kernel(AttendParams p) {
    constexpr bool FRONT = FORM == kFront;
    extern __shared__ float merge[]; // [4 waves][16][2] maxima and sums, [4][16][V + 4] outputs
    const StepView &v = p.v;
    const int seg = blockIdx.z, n = v.seg_len[seg];
    const int G = p.G, gs = p.H / G, g = blockIdx.y / p.groups, c0 = (blockIdx.y - g * p.groups) * 16, ncols = n * gs;
    if (n < p.min_len || n > p.max_len || c0 >= ncols) return;
    const int D = EXACT ? KS * 32 : p.D, V = EXACT ? VT * 16 : p.V, ks_n = D / 32, vt_n = V / 16;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lg = lane >> 4, i16 = lane & 15;
    const int off = v.seg_off[seg], start = v.seg_pos[seg];
    const int *table = v.table + (size_t)v.seg_row[seg] * v.table_stride;
    const int last = c0 + 15 < ncols ? c0 + 15 : ncols - 1;
    const int lo = start + c0 / gs, hi = start + last / gs; // positions of the first and the last column's token
    const int first_lo = first_seen(p, lo), first_hi = first_seen(p, hi);
    const int b1 = (hi >> 5) + 1;
    FrontBlocks front {};
    if constexpr (FRONT) front = front_blocks(p, v.seg_row[seg], lo, hi);
    const int b0 = (first_lo >> 5) - front.n; // (blocks in front have numbers from b0 on, as if they were neighbours of the window's)
    const int per = (b1 - b0 + p.nsplit - 1) / p.nsplit;
    int wb = b0 + (int)blockIdx.x * per, we = wb + per < b1 ? wb + per : b1;
    const int wper = (we - wb + 3) / 4; // this wave's blocks
    const int bb = wb + wave * wper, be = bb + wper < we ? bb + wper : we;

    const int c = c0 + i16, cv = c < ncols ? c : ncols - 1;
    const int cpos = c < ncols ? start + c / gs : -1, cfirst = first_seen(p, cpos < 0 ? 0 : cpos);
    const int cfront = FRONT && p.block > 0 ? front_seen(p, cpos) : p.keep_first;
    const bool ruled = FORM == kRule || (FRONT && (p.softcap > 0.0f || p.distance_bias));
    ScoreRule rule;
    if constexpr (FORM != kPlain) rule = score_rule(p, g * gs + cv % gs);
    bf16x8 qf[KS];
    {
        const uint16_t *row = (const uint16_t *)p.q + (size_t)(off + cv / gs) * p.q_ld + (size_t)(g * gs + cv % gs) * D + 8 * lg;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
            if (EXACT || ks < ks_n) qf[ks] = *(const bf16x8 *)(row + ks * 32);
    }
    f32x4 o[VT];
#pragma unroll
    for (int d = 0; d < VT; ++d) o[d] = f32x4 {0.f, 0.f, 0.f, 0.f};
    float m = kUnseen, l = 0.0f;
    const float scale2 = p.scale * kLog2e;

    // row i16 of key tile tt is token 8 (i16 / 4) + 4 tt + i16 % 4 of the block
    const int krow = (8 * (i16 >> 2) + (i16 & 3)) * D + 8 * lg, vrow = i16 * 32 + 8 * lg;
    const uint16_t *pool = (const uint16_t *)p.pool;
    const size_t page_len = (size_t)kPageTokens * (D + V);
    bf16x8 kf[2][KS], vf[VT];
    // block `at` of the walk: its number among those in front of the window or of all, where its page begins
    auto in_front = [&](int at) { return FRONT && at < b0 + front.n; };
    auto number = [&](int at) { return in_front(at) ? at - b0 : at; };
    auto page_of = [&](int at) {
        const int n = number(at) >> 1;
        if (FRONT && front.keep == 0 && in_front(at)) return front.means + ((size_t)front.table[n] * G + g) * page_len;
        return pool + ((size_t)table[n] * G + g) * page_len;
    };
    auto load_keys = [&](int at, const uint16_t *page) {
        const uint16_t *k = page + (number(at) & 1) * 32 * D + krow;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
            if (EXACT || ks < ks_n) kf[0][ks] = *(const bf16x8 *)(k + ks * 32), kf[1][ks] = *(const bf16x8 *)(k + 4 * D + ks * 32);
    };
    auto load_values = [&](int at, const uint16_t *page) {
        const uint16_t *w = page + (size_t)kPageTokens * D + (number(at) & 1) * 32 * V + vrow;
#pragma unroll
        for (int d = 0; d < VT; ++d)
            if (EXACT || d < vt_n) vf[d] = *(const bf16x8 *)(w + d * 512);
    };
    const uint16_t *page = bb < be ? page_of(bb) : pool;
    if (bb < be) load_keys(bb, page), load_values(bb, page);
    for (int at = bb; at < be; ++at) {
        const bool more = at + 1 < be;
        if (more) page = page_of(at + 1);
        const int t0 = number(at) * 32;
        f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = s0;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
            if (EXACT || ks < ks_n) {
                s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[0][ks], qf[ks], s0, 0, 0, 0);
                s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[1][ks], qf[ks], s1, 0, 0, 0);
            }
        if (more) load_keys(at + 1, page);
        if (!ruled) s0 *= scale2, s1 *= scale2;
        float x[8], bm = kUnseen;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            x[j] = j < 4 ? s0[j & 3] : s1[j & 3];
            if (ruled) x[j] = rule(x[j], scale2, (float)(cpos - (t0 + 8 * lg + j)));
        }
        const bool open = in_front(at) ? t0 + 31 < front.seen_lo : t0 + 31 <= lo && t0 >= first_hi; // every column sees the whole block
        if (!open) {
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const int t = t0 + 8 * lg + j;
                const bool seen = in_front(at) ? t < cfront : t <= cpos && (t >= cfirst || (FRONT && t < front.keep));
                x[j] = seen ? x[j] : kUnseen;
            }
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) bm = fmaxf(bm, x[j]);
        bm = fmaxf(bm, __shfl_xor(bm, 16, 64));
        bm = fmaxf(bm, __shfl_xor(bm, 32, 64));
        const float m_new = fmaxf(m, bm);
        const float alpha = __builtin_amdgcn_exp2f(m - m_new);
        m = m_new;
        float sum = 0.0f;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            // (a column that has seen no key has its reference point at the masked score)
            const float e = __builtin_amdgcn_exp2f(x[j] - m_new);
            x[j] = open || x[j] > 0.5f * kUnseen ? e : 0.0f;
            sum += x[j];
        }
        l = l * alpha + sum;
        const bf16x8 pf = pack_bf16x8(x);
        if (__builtin_amdgcn_ballot_w64(alpha != 1.0f) != 0) {
#pragma unroll
            for (int d = 0; d < VT; ++d) o[d] *= alpha;
        }
#pragma unroll
        for (int d = 0; d < VT; ++d)
            if (EXACT || d < vt_n) o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[d], pf, o[d], 0, 0, 0);
        if (more) load_values(at + 1, page);
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    // the four waves' parts meet in LDS
    float *ml = merge, *outs = merge + 4 * 16 * 2;
    const int pitch = V + 4;
    if (lg == 0) ml[(wave * 16 + i16) * 2] = m, ml[(wave * 16 + i16) * 2 + 1] = l;
#pragma unroll
    for (int d = 0; d < VT; ++d)
        if (EXACT || d < vt_n) *(f32x4 *)(outs + (wave * 16 + i16) * pitch + d * 16 + 4 * lg) = o[d];
    __syncthreads();
    const size_t slot0 = (((size_t)seg * gridDim.y + blockIdx.y) * p.nsplit + blockIdx.x) * 16;
    for (int i = threadIdx.x; i < 16 * (V / 4); i += 256) {
        const int col = i / (V / 4), d = i % (V / 4) * 4, cc = c0 + col;
        if (cc >= ncols) continue;
        float mt = kUnseen, den = 0.0f;
#pragma unroll
        for (int w = 0; w < 4; ++w) mt = fmaxf(mt, ml[(w * 16 + col) * 2]);
        const float s2 = p.sink && p.nsplit == 1 ? p.sink[g * gs + cc % gs] * kLog2e : kUnseen;
        mt = fmaxf(mt, s2);
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < 4; ++w) {
            const float mw = ml[(w * 16 + col) * 2], e = mw > 0.5f * kUnseen ? __builtin_amdgcn_exp2f(mw - mt) : 0.0f;
            den += ml[(w * 16 + col) * 2 + 1] * e;
            acc += *(const f32x4 *)(outs + (w * 16 + col) * pitch + d) * e;
        }
        if (p.nsplit > 1) {
            *(f32x4 *)(p.part + (slot0 + col) * V + d) = acc;
            if (d == 0) *(float2 *)(p.part + p.part_ml + (slot0 + col) * 2) = make_float2(mt, den);
        } else {
            if (p.sink) den += __builtin_amdgcn_exp2f(s2 - mt);
            const int t = off + cc / gs, head = g * gs + cc % gs;
            if constexpr (FRONT) turn_back<4>(p, start + cc / gs, d, acc);
            acc *= output_gate(p, t, head, d) * (1.0f / den);
            uint16_t *dst = (uint16_t *)p.out + (size_t)t * p.out_ld + (size_t)head * V + d;
            *(uint2 *)dst = make_uint2(pack_pair(acc[0], acc[1]), pack_pair(acc[2], acc[3]));
        }
    }
}

// sum of a column's splits; grid (G * column groups, segments, 16 columns).  Four neighbouring dimensions a thread, the splits
// dealt out to as many sets of threads as a workgroup holds.
constexpr int kMaxSplits = 64;
__global__ __launch_bounds__(256) void grouped_merge_kernel(AttendParams p) {
    __shared__ float w[kMaxSplits], inv_den;
    __shared__ f32x4 sums[256];
    const StepView &v = p.v;
    const int seg = blockIdx.y, n = v.seg_len[seg], gs = p.H / p.G, V = p.V;
    const int g = blockIdx.x / p.groups, c = (blockIdx.x - g * p.groups) * 16 + blockIdx.z;
    if (n < p.min_len || n > p.max_len || c >= n * gs) return;
    const int head = g * gs + c % gs, per = V / 4, sets = 256 / per;
    const int set = (int)threadIdx.x / per, d = (int)threadIdx.x % per * 4;
    const size_t slot0 = ((size_t)seg * gridDim.x + blockIdx.x) * p.nsplit * 16 + blockIdx.z;
    // the first outputs are on their way while the weights are worked out
    const float *src = p.part + slot0 * V + d;
    const size_t step = (size_t)16 * V;
    f32x4 x[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int s = set + i * sets;
        x[i] = *(const f32x4 *)(src + (s < p.nsplit ? s : 0) * step);
    }
    if (threadIdx.x < 64) {
        float2 ml = make_float2(kUnseen, 0.0f);
        if ((int)threadIdx.x < p.nsplit) ml = *(const float2 *)(p.part + p.part_ml + (slot0 + (size_t)threadIdx.x * 16) * 2);
        const float s2 = p.sink ? p.sink[head] * kLog2e : kUnseen;
        const float mt = fmaxf(wave_largest(ml.x), s2);
        const float e = ml.x > 0.5f * kUnseen ? __builtin_amdgcn_exp2f(ml.x - mt) : 0.0f;
        const float den = wave_total(ml.y * e) + (p.sink ? __builtin_amdgcn_exp2f(s2 - mt) : 0.0f);
        w[threadIdx.x] = e;
        if (threadIdx.x == 0) inv_den = 1.0f / den;
    }
    __syncthreads();
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    if (set < sets) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (set + i * sets < p.nsplit) acc += x[i] * w[set + i * sets];
        for (int s = set + 4 * sets; s < p.nsplit; s += sets) acc += *(const f32x4 *)(src + s * step) * w[s];
    }
    sums[threadIdx.x] = acc;
    __syncthreads();
    if (set > 0) return;
    for (int s = 1; s < sets; ++s) acc += sums[s * per + threadIdx.x];
    const int t = v.seg_off[seg] + c / gs;
    turn_back<4>(p, v.seg_pos[seg] + c / gs, d, acc);
    acc *= output_gate(p, t, head, d) * inv_den;
    uint16_t *dst = (uint16_t *)p.out + (size_t)t * p.out_ld + (size_t)head * V + d;
    *(uint2 *)dst = make_uint2(pack_pair(acc[0], acc[1]), pack_pair(acc[2], acc[3]));
}

// BF16, long form: 128 columns a workgroup (32 a wave), the visible context in blocks of 32 tokens through LDS, on 32 x 32 tiles.
// KSM: most 16-dim steps of a key; VTM: most 32-dim tiles of a value; EXACT, FORM as above.  grid (G, column groups, segments)
template <int KSM, int VTM, bool EXACT, int FORM>
__global__ __launch_bounds__(256, (KSM <= 8 && VTM <= 4) ? 2 : 1) void grouped_long_kernel(AttendParams p) {
    constexpr bool FRONT = FORM == kFront;
    extern __shared__ unsigned char lds[];
    const StepView &v = p.v;
    const int seg = blockIdx.z, n = v.seg_len[seg];
    const int G = p.G, gs = p.H / G, g = blockIdx.x, ncols = n * gs;
    const int c0 = ((int)gridDim.y - 1 - (int)blockIdx.y) * 128; // the columns with the longest contexts first
    if (n < p.min_len || n > p.max_len || c0 >= ncols) return;
    const int D = EXACT ? KSM * 16 : p.D, V = EXACT ? VTM * 32 : p.V, ks_n = D / 16, vt_n = V / 32;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), h = lane >> 5, cl = lane & 31;
    const int off = v.seg_off[seg], start = v.seg_pos[seg];
    const int *table = v.table + (size_t)v.seg_row[seg] * v.table_stride;
    const int kpitch = D * 2 + 16, vpitch = 80, bufb = 32 * kpitch + V * vpitch;
    const int c = c0 + wave * 32 + cl, cv = c < ncols ? c : ncols - 1;
    const int pos = start + cv / gs;
    const int wc0 = c0 + wave * 32, wc1 = wc0 + 31 < ncols ? wc0 + 31 : ncols - 1;
    const int wlo = start + wc0 / gs, whi = start + wc1 / gs; // positions of the wave's first and last column
    const bool wave_on = wc0 < ncols;
    const int head = g * gs + cv % gs;
    const int token = off + cv / gs, pos_first = first_seen(p, pos);
    const bool ruled = FORM == kRule || (FRONT && (p.softcap > 0.0f || p.distance_bias));
    ScoreRule rule;
    if constexpr (FORM != kPlain) rule = score_rule(p, head);
    bf16x8 qf[KSM];
    {
        const uint16_t *row = (const uint16_t *)p.q + (size_t)token * p.q_ld + (size_t)head * D + 8 * h;
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
    const int lo = start + c0 / gs, last = c0 + 127 < ncols ? c0 + 127 : ncols - 1, hi = start + last / gs;
    FrontBlocks front {};
    if constexpr (FRONT) front = front_blocks(p, v.seg_row[seg], lo, hi);
    const int b0 = (first_seen(p, lo) >> 5) - front.n, b1 = (hi >> 5) + 1; // (numbers as in the short form)
    int pos_front = 0, wfront_lo = 0, wfront_hi = 0; // entries in front that the column, the wave's first and its last column see
    if constexpr (FRONT) pos_front = front_seen(p, pos), wfront_lo = front_seen(p, wlo), wfront_hi = front_seen(p, whi);
    const int wfirst = first_seen(p, wlo), wfirst_hi = first_seen(p, whi);

    constexpr int PER = KSM / 4 + VTM / 2 + 1; // 16-byte chunks of a block a thread carries (at least D / 64 + V / 64)
    const int kch = D * 4, chunks = kch + V * 4; // of keys, of both
    u32x4 stage[PER];
    int src[PER], step[PER], dst[PER]; // element behind the head's page, way to the second block of the page, byte in LDS
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        int e = i * 256 + threadIdx.x;
        e = e < chunks ? e : chunks - 1; // (past the block: its last chunk once more)
        if (e < kch) {
            src[i] = e * 8, step[i] = 32 * D, dst[i] = (e + e / (D / 8)) * 16; // 16 bytes of padding behind every row before it
        } else {
            e -= kch; // four chunks a value row
            src[i] = kPageTokens * D + e * 8, step[i] = 32 * V, dst[i] = 32 * kpitch + (e >> 2) * vpitch + (e & 3) * 16;
        }
    }
    const uint16_t *pool = (const uint16_t *)p.pool;
    auto in_front = [&](int at) { return FRONT && at < b0 + front.n; };
    auto number = [&](int at) { return in_front(at) ? at - b0 : at; };
    auto page_of = [&](int at) { return FRONT && front.keep == 0 && in_front(at) ? front.table[number(at) >> 1] : table[number(at) >> 1]; };
    auto fetch = [&](int at, int page) {
        const uint16_t *base = (FRONT && front.keep == 0 && in_front(at) ? front.means : pool) + ((size_t)page * G + g) * kPageTokens * (D + V);
#pragma unroll
        for (int i = 0; i < PER; ++i)
            if (i * 256 < chunks) stage[i] = *(const u32x4 *)(base + src[i] + (number(at) & 1) * step[i]);
    };
    // row cl of the key operand is the token with bits 2 and 3 swapped: register 8 t + j of half h is then token 16 t + 8 h + j
    const int ktok = (cl & 19) | ((cl & 4) << 1) | ((cl & 8) >> 1);
    fetch(b0, page_of(b0));
    int page = b0 + 1 < b1 ? page_of(b0 + 1) : 0;
    int buf = 0;
    for (int at = b0; at < b1; ++at, buf ^= 1) {
        unsigned char *kb = lds + buf * bufb, *vb = kb + 32 * kpitch;
#pragma unroll
        for (int i = 0; i < PER; ++i)
            if (i * 256 < chunks) *(u32x4 *)(kb + dst[i]) = stage[i];
        __syncthreads();
        if (at + 1 < b1) fetch(at + 1, page);
        if (at + 2 < b1) page = page_of(at + 2);
        const int t0 = number(at) * 32;
        const bool none = in_front(at) ? t0 >= wfront_hi : t0 > whi || (t0 + 31 < wfirst && !(FRONT && t0 < front.keep));
        if (!wave_on || none) continue; // (the same for the whole wave; the barrier above is all there is)
        f32x16 s;
#pragma unroll
        for (int r = 0; r < 16; ++r) s[r] = 0.0f;
        const unsigned char *krow = kb + ktok * kpitch + 16 * h;
#pragma unroll
        for (int ks = 0; ks < KSM; ++ks)
            if (EXACT || ks < ks_n) s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*(const bf16x8 *)(krow + ks * 32), qf[ks], s, 0, 0, 0);
        const bool masked = in_front(at) ? t0 + 31 >= wfront_lo : t0 + 31 > wlo || t0 < wfirst_hi;
        float bm = kUnseen;
        if (ruled) {
            rule.all<16>(s, scale2, (float)(pos - (t0 + 8 * h)), [](int r) { return (float)(16 * (r >> 3) + (r & 7)); });
        } else {
#pragma unroll
            for (int r = 0; r < 16; ++r) s[r] *= scale2;
        }
        if (masked) {
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                const int t = t0 + 16 * (r >> 3) + 8 * h + (r & 7);
                const bool seen = in_front(at) ? t < pos_front : t <= pos && (t >= pos_first || (FRONT && t < front.keep));
                s[r] = seen ? s[r] : kUnseen;
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
        for (int r = 0; r < 16; ++r) {
            const float e = __builtin_amdgcn_exp2f(s[r] - m_new);
            // (a column that has seen no key yet has its reference point at the masked score)
            s[r] = !masked || s[r] > 0.5f * kUnseen ? e : 0.0f;
            sum += s[r];
        }
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
            const unsigned char *vrow = vb + cl * vpitch + t * 32 + h * 16;
#pragma unroll
            for (int d = 0; d < VTM; ++d)
                if (EXACT || d < vt_n) o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(*(const bf16x8 *)(vrow + d * 32 * vpitch), pf, o[d], 0, 0, 0);
        }
    }
    l += __shfl_xor(l, 32, 64);
    if (c >= ncols) return;
    float mul = 1.0f;
    if (p.sink) {
        const float s2 = p.sink[head] * kLog2e, mt = fmaxf(m, s2);
        mul = __builtin_amdgcn_exp2f(m - mt);
        l = l * mul + __builtin_amdgcn_exp2f(s2 - mt);
    }
    mul /= l;
    uint16_t *out = (uint16_t *)p.out + (size_t)token * p.out_ld + (size_t)head * V;
#pragma unroll
    for (int d = 0; d < VTM; ++d)
        if (EXACT || d < vt_n) {
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                const int at = d * 32 + 8 * q + 4 * h;
                const f32x4 f = output_gate(p, token, head, at) * mul;
                f32x4 y = {o[d][4 * q], o[d][4 * q + 1], o[d][4 * q + 2], o[d][4 * q + 3]};
                if constexpr (FRONT) turn_back<4>(p, pos, at, y);
                y *= f;
                *(uint2 *)(out + at) = make_uint2(pack_pair(y[0], y[1]), pack_pair(y[2], y[3]));
            }
        }
}

template <int KS, int VT, bool EXACT, int FORM>
int launch_short_form(const AttendParams &p, hipStream_t st) {
    static const hipError_t attr = hipFuncSetAttribute((const void *)grouped_short_kernel<KS, VT, EXACT, FORM>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    XFT_CHECK_HIP(attr);
    const size_t smem = (size_t)4 * 16 * (2 + p.V + 4) * 4;
    hipLaunchKernelGGL((grouped_short_kernel<KS, VT, EXACT, FORM>), dim3(p.nsplit, p.G * p.groups, p.v.B), dim3(256), smem, st, p);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}
template <int KSM, int VTM, bool EXACT, int FORM>
int launch_long_form(const AttendParams &p, hipStream_t st) {
    static const hipError_t attr = hipFuncSetAttribute((const void *)grouped_long_kernel<KSM, VTM, EXACT, FORM>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    XFT_CHECK_HIP(attr);
    const size_t smem = (size_t)2 * (32 * (p.D * 2 + 16) + p.V * 80);
    hipLaunchKernelGGL((grouped_long_kernel<KSM, VTM, EXACT, FORM>), dim3(p.G, (p.v.longest * (p.H / p.G) + 127) / 128, p.v.B), dim3(256), smem, st, p);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}
int form_of(const AttendParams &p) { return p.keep_first > 0 || p.block > 0 || p.cosV ? kFront : p.softcap > 0.0f || p.distance_bias ? kRule : kPlain; }
template <int KS, int VT, bool EXACT>
int launch_short(const AttendParams &p, hipStream_t st) {
    switch (form_of(p)) {
        case kFront: return launch_short_form<KS, VT, EXACT, kFront>(p, st);
        case kRule: return launch_short_form<KS, VT, EXACT, kRule>(p, st);
        default: return launch_short_form<KS, VT, EXACT, kPlain>(p, st);
    }
}
template <int KSM, int VTM, bool EXACT>
int launch_long(const AttendParams &p, hipStream_t st) {
    switch (form_of(p)) {
        case kFront: return launch_long_form<KSM, VTM, EXACT, kFront>(p, st);
        case kRule: return launch_long_form<KSM, VTM, EXACT, kRule>(p, st);
        default: return launch_long_form<KSM, VTM, EXACT, kPlain>(p, st);
    }
}

bool mfma_takes(const PlanLayer &L) { return L.D <= 256 && L.V <= 256; }
constexpr int kShortTokens = 16; // longest segment of the short form

} // namespace

int grouped_prepare(int act, const PlanLayer &L, const StepView &v, const GroupedBuffers &b0, float eps, hipStream_t st) {
    const xfthip_plan_layer &s = L.s;
    const bool own = L.kv_from < 0;
    GroupedBuffers b = b0;
    b.a = (const char *)b.a + (size_t)L.in_col * (act == XFTHIP_BF16 ? 2 : 4);
    PrepareParams p = {v, b, L.q_norm, L.kv_norm, L.cosT, L.sinT, L.cosV, L.sinV, L.filter, s.taps, L.channels(), s.qk_norm != 0, s.pool, L.in_ld, L.value_col(),
            s.heads, s.kv_heads, L.D, L.V, s.dim, s.vdim, s.rot_dim, 4, L.moves_queries() ? 0 : s.heads, own ? s.heads + s.kv_heads : s.heads, s.qk_norm == XFTHIP_QK_NORM_ALL ? 1 : 0, 0, 0, L.first_values ? 1 : 0,
            s.v_mix && !L.first_values ? L.value_share : 0.0f, eps};
    while (p.lanes * 8 < L.D) p.lanes *= 2;
    XFT_REQUIRE(p.lanes <= 64, "grouped_prepare: heads of %d values too wide", L.D);
    const int qk_blocks = p.h0 >= p.h1 ? 0 : p.all ? v.T : (int)(((size_t)v.T * (p.h1 - p.h0) * p.lanes + 255) / 256);
    p.seg_blocks = own ? (v.longest + 62) / 32 : 0; // blocks of 32 positions a segment of that length can touch
    p.v_blocks = v.B * s.kv_heads * p.seg_blocks;
    const dim3 grid(p.v_blocks + qk_blocks);
    if (grid.x == 0) return 0;
    auto launch = [&](void (*bf16)(PrepareParams), void (*f32)(PrepareParams)) {
        if (act == XFTHIP_BF16) hipLaunchKernelGGL(bf16, grid, dim3(256), 0, st, p);
        else hipLaunchKernelGGL(f32, grid, dim3(256), 0, st, p);
    };
    switch (L.filters() ? s.taps : 0) {
        case 0: launch(grouped_prepare_kernel<true, 0>, grouped_prepare_kernel<false, 0>); break;
        case 2: launch(grouped_prepare_kernel<true, 2>, grouped_prepare_kernel<false, 2>); break;
        case 3: launch(grouped_prepare_kernel<true, 3>, grouped_prepare_kernel<false, 3>); break;
        case 4: launch(grouped_prepare_kernel<true, 4>, grouped_prepare_kernel<false, 4>); break;
        default: launch(grouped_prepare_kernel<true, -1>, grouped_prepare_kernel<false, -1>);
    }
    XFT_CHECK_HIP(hipGetLastError());
    if (L.filters())
        if (int rc = conv_tail(act, v, b.a, L.in_ld, L.channels(), s.taps, b.conv_state, st)) return rc;
    if (s.pool > 0 && v.longest > 1) {
        const dim3 blocks(s.kv_heads * (v.longest / s.pool + 1), v.B);
        if (act == XFTHIP_BF16) hipLaunchKernelGGL(grouped_means_kernel<true>, blocks, dim3(256), 0, st, p);
        else hipLaunchKernelGGL(grouped_means_kernel<false>, blocks, dim3(256), 0, st, p);
        XFT_CHECK_HIP(hipGetLastError());
    }
    return 0;
}

// Parts a context of `hint` tokens is split into: as many as give every compute unit a workgroup, every wave a block permitting.
int grouped_split_count(const PlanLayer &L, int B, int longest, int hint) {
    if (!mfma_takes(L)) return 1;
    longest = longest < kShortTokens ? longest : kShortTokens;
    const long units = (long)B * L.s.kv_heads * ((longest * (L.s.heads / L.s.kv_heads) + 15) / 16);
    const int span = L.s.chunk > 0 ? L.s.chunk : L.s.window;
    const int ahead = L.s.pool > 0 ? hint / L.s.pool : L.s.keep_first; // entries in front of a window
    const int ctx = span > 0 && span + ahead + longest < hint ? span + ahead + longest : hint;
    const int most = (ctx + 127) / 128;
    long want = device_cu_count() / units;
    want = want < most ? want : most;
    want = want < kMaxSplits / 2 ? want : kMaxSplits / 2;
    return want < 1 ? 1 : (int)want;
}

// (splits times units never exceed the compute units, or nothing is split)
size_t grouped_part_floats(const PlanLayer &L) {
    return mfma_takes(L) ? (size_t)device_cu_count() * 16 * (L.V + 2) : 0;
}

int grouped_attention(int act, const PlanLayer &L, const StepView &v, const GroupedBuffers &b, void *out, int hint, float *part, size_t part_floats,
        hipStream_t st) {
    const xfthip_plan_layer &s = L.s;
    const size_t esz = act == XFTHIP_BF16 ? 2 : 4;
    const char *rows = (const char *)b.a + L.in_col * esz;
    AttendParams p = {v, L.moves_queries() ? b.q : rows, b.pool, L.moves_queries() ? s.heads * L.D : L.in_ld, (char *)out + L.out_col * esz, L.out_ld, L.sink,
            rows + L.gate_col() * esz, s.out_gate, L.in_ld, L.mix_scale, s.softcap, s.distance_bias, s.heads, s.kv_heads, L.D, L.V, s.window, s.chunk, s.keep_first, s.pool,
            b.means, b.means_table, b.means_stride, L.cosV, L.sinV, s.vdim / 2, 0, 1 << 30, s.scale, 1, 1, part, 0};
    if (act != XFTHIP_BF16 || !mfma_takes(L)) {
        const size_t smem = (size_t)(L.D + 256 + L.V + 8) * 4;
        if (act == XFTHIP_BF16) hipLaunchKernelGGL(grouped_attend_kernel<true>, dim3(v.T, s.heads), dim3(256), smem, st, p);
        else hipLaunchKernelGGL(grouped_attend_kernel<false>, dim3(v.T, s.heads), dim3(256), smem, st, p);
        XFT_CHECK_HIP(hipGetLastError());
        return 0;
    }
    const int ks = L.D / 32, vt = L.V / 16, gs = s.heads / s.kv_heads;
    int rc = 0;
    if (v.longest > kShortTokens) {
        p.min_len = kShortTokens + 1;
        if (ks == 4 && vt == 8) rc = launch_long<8, 4, true>(p, st);
        else if (ks == 6 && vt == 8) rc = launch_long<12, 4, true>(p, st);
        else if (ks == 2 && vt == 4) rc = launch_long<4, 2, true>(p, st);
        else if (ks <= 4 && vt <= 8) rc = launch_long<8, 4, false>(p, st);
        else rc = launch_long<16, 8, false>(p, st);
        if (rc || v.T == v.longest) return rc; // (a batch of one long segment)
    }
    p.min_len = 0, p.max_len = kShortTokens;
    const int longest = v.longest < kShortTokens ? v.longest : kShortTokens;
    p.groups = (longest * gs + 15) / 16;
    p.nsplit = grouped_split_count(L, v.B, longest, hint);
    const size_t slots = (size_t)v.B * s.kv_heads * p.groups * p.nsplit * 16;
    p.part_ml = slots * L.V;
    XFT_REQUIRE(p.nsplit == 1 || slots * (L.V + 2) <= part_floats, "grouped_attention: workspace too small for %zu partial columns", slots);
    if (ks == 4 && vt == 8) rc = launch_short<4, 8, true>(p, st);
    else if (ks == 6 && vt == 8) rc = launch_short<6, 8, true>(p, st);
    else if (ks == 2 && vt == 4) rc = launch_short<2, 4, true>(p, st);
    else if (ks <= 4 && vt <= 8) rc = launch_short<4, 8, false>(p, st);
    else rc = launch_short<8, 16, false>(p, st);
    if (rc || p.nsplit == 1) return rc;
    hipLaunchKernelGGL(grouped_merge_kernel, dim3(s.kv_heads * p.groups, v.B, 16), dim3(256), 0, st, p);
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

} // namespace xfthip
