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
