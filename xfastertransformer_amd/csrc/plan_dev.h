// Device helpers of the layer plans' attention kernels: activations of either type, the page lookup, packed bf16 operands.
#pragma once
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

typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2;
// two values -> packed bf16 pair, round to nearest even (v_cvt_pk_bf16_f32)
__device__ inline uint32_t pack_pair(float lo, float hi) { return __builtin_bit_cast(uint32_t, bf16x2 {(__bf16)lo, (__bf16)hi}); }

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

// neighbouring pairs
template <bool BF16>
__device__ inline float2 load2(const void *p, size_t i) {
    if constexpr (BF16) {
        const uint32_t u = *(const uint32_t *)((const uint16_t *)p + i);
        return make_float2(u2f(u << 16), u2f(u & 0xFFFF0000u));
    } else {
        return *(const float2 *)((const float *)p + i);
    }
}
template <bool BF16>
__device__ inline void store2(void *p, size_t i, float2 v) {
    if constexpr (BF16) *(uint32_t *)((uint16_t *)p + i) = f32_bits_to_bf16_sel(f2u(v.x)) | (f32_bits_to_bf16_sel(f2u(v.y)) << 16);
    else *(float2 *)((float *)p + i) = v;
}

// cache row of position `pos` of slot `row`
__device__ inline size_t cache_row(const StepView &v, int row, int pos) {
    return (size_t)v.table[(size_t)row * v.table_stride + pos / kPageTokens] * kPageTokens + pos % kPageTokens;
}

template <bool BF16>
__device__ inline void load8(const void *p, size_t i, float (&v)[8]) {
    if constexpr (BF16) {
        const uint4 q = *(const uint4 *)((const uint16_t *)p + i);
        const uint32_t w[4] = {q.x, q.y, q.z, q.w};
#pragma unroll
        for (int k = 0; k < 4; ++k) v[2 * k] = u2f(w[k] << 16), v[2 * k + 1] = u2f(w[k] & 0xFFFF0000u);
    } else {
        const f32x4 x = *(const f32x4 *)((const float *)p + i), y = *(const f32x4 *)((const float *)p + i + 4);
#pragma unroll
        for (int k = 0; k < 4; ++k) v[k] = x[k], v[4 + k] = y[k];
    }
}
template <bool BF16>
__device__ inline void store8(void *p, size_t i, const float (&v)[8]) {
    if constexpr (BF16) {
        uint32_t w[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) w[k] = pack_pair(v[2 * k], v[2 * k + 1]);
        *(uint4 *)((uint16_t *)p + i) = make_uint4(w[0], w[1], w[2], w[3]);
    } else {
        *(f32x4 *)((float *)p + i) = f32x4 {v[0], v[1], v[2], v[3]};
        *(f32x4 *)((float *)p + i + 4) = f32x4 {v[4], v[5], v[6], v[7]};
    }
}

template <bool BF16>
__device__ inline void put4(void *p, size_t i, f32x4 v) {
    if constexpr (BF16) *(uint2 *)((uint16_t *)p + i) = make_uint2(pack_pair(v[0], v[1]), pack_pair(v[2], v[3]));
    else *(f32x4 *)((float *)p + i) = v;
}

// exp, x / (1 + exp(-x)), 1 / (1 + exp(-x)) and log(1 + exp(x)): the library functions with 32-bit activations; with bf16
// ones the hardware's exp2 / log2 / reciprocal, each good to a few units in the last place (log(1 + y) through
// y log(u) / (u - 1), u = 1 + y rounded, which keeps small y exact)
template <bool FAST>
__device__ inline float exp_of(float x) {
    if constexpr (FAST) return fast_exp(x);
    else return expf(x);
}
template <bool FAST>
__device__ inline float sigmoid_of(float x) {
    if constexpr (FAST) return __builtin_amdgcn_rcpf(1.0f + fast_exp(-x));
    else return 1.0f / (1.0f + expf(-x));
}
template <bool FAST>
__device__ inline float silu_of(float x) {
    if constexpr (FAST) return x * __builtin_amdgcn_rcpf(1.0f + fast_exp(-x));
    else return x / (1.0f + expf(-x));
}
template <bool FAST>
__device__ inline float softplus_of(float x) {
    if (x > 20.0f) return x;
    if constexpr (FAST) {
        const float y = fast_exp(x), u = 1.0f + y, d = u - 1.0f;
        return d > 0.0f ? y * (__logf(u) * __builtin_amdgcn_rcpf(d)) : y;
    } else {
        return log1pf(expf(x));
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

// The value is in its register from here on.  What is loaded in front of a loop and changed in it would otherwise be waited for inside, and
// with it the loads that the loop has just sent ahead.
template <class V>
__device__ inline void arrived(V &v) {
    asm volatile("" : "+v"(v));
}

// tanh form of the Gaussian error linear unit
__device__ inline float gelu_tanh(float z) { return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z))); }

// a row of the residual from a token and the one before it (prev: any value in front of a sequence's first token)
__device__ inline void embed_token(const EmbedTables &e, int id, bool first, int prev, float *x) {
    id = id < 0 ? 0 : (id >= e.vocab ? e.vocab - 1 : id);
    prev = prev < 0 ? 0 : (prev >= e.vocab ? e.vocab - 1 : prev);
    const uint16_t *row = e.table + (size_t)id * e.hidden;
    const uint16_t *pair = e.pairs;
    if (pair) pair += (size_t)(first ? e.buckets : (prev * e.mul_prev + id * e.mul_cur) % e.buckets) * e.hidden;
    for (int c = threadIdx.x * 4; c < e.hidden; c += blockDim.x * 4) { // (rows are whole 32-value groups)
        const uint2 a = *(const uint2 *)(row + c), b = pair ? *(const uint2 *)(pair + c) : make_uint2(0, 0);
        const f32x4 v = {u2f(a.x << 16), u2f(a.x & 0xFFFF0000u), u2f(a.y << 16), u2f(a.y & 0xFFFF0000u)};
        const f32x4 w = {u2f(b.x << 16), u2f(b.x & 0xFFFF0000u), u2f(b.y << 16), u2f(b.y & 0xFFFF0000u)};
        *(f32x4 *)(x + c) = v * e.scale + w;
    }
}

typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
constexpr float kUnseen = -1.0e30f; // score of a masked key, maximum of a column that has seen none
constexpr float kLog2e = 1.4426950408889634f;

__device__ inline bf16x8 pack_bf16x8(const float (&v)[8]) {
    u32x4 u;
#pragma unroll
    for (int i = 0; i < 4; ++i) u[i] = pack_pair(v[2 * i], v[2 * i + 1]);
    return __builtin_bit_cast(bf16x8, u);
}

} // namespace

} // namespace xfthip
