// Matrix products of layer plans that the weight-only GEMMs do not cover: 32-bit activations (true fp32 products on the
// fp32 matrix units), and heads side by side (every block of output columns multiplies its own slice of the activation
// row, the per-head products of latent attention and the two gates of the delta rule), also for the weights of a group in one
// launch (experts).  BF16 weights in the packed layout of common.h.
#include "plan_dev.h"

namespace xfthip {

namespace {

struct TileGemm {
    const uint8_t *packed;
    int KT, ktiles, NTILES, N, M;
    const void *A;
    int lda, tiles_per_block, a_block_stride;
    void *C;
    int ldc, c_dtype, glu, add;
    float glu_limit, glu_alpha;
    const float *bias;
    float decay; // 1 / decay_tau, or 0
    const uint16_t *side;
    int side_ld, side_vocab;
    const int *side_ids;
    const GroupWeight *group;
    const int *group_rows, *a_rows;
};

__device__ inline float precise_glu(float gate, float up, float limit, float alpha) {
    if (alpha == 0.0f) return gate / (1.0f + expf(-gate)) * up; // no limits
    const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
    return g / (1.0f + expf(-alpha * g)) * (u + 1.0f);
}

// sigmoid(z)^power.  (FAST: log(1 + exp(-z)) may be off by a rounding of 1, which is a rounding of the result)
template <bool FAST>
__device__ inline float decay_of(float z, float power) {
    if constexpr (FAST) {
        const float x = -kLog2e * z;
        return __builtin_amdgcn_exp2f(-power * (x > 80.0f ? x : __builtin_amdgcn_logf(1.0f + __builtin_amdgcn_exp2f(x))));
    } else {
        return expf(-power * softplus_of<false>(-z));
    }
}

// A wave: TW column tiles (16 weight columns each; two, or one in the 16-wave form) x MT row tiles (16 activation rows each).  The weight tile is the MFMA
// A operand, the activation rows the B operand: a lane ends up with four neighbouring columns of one row.  With fp32
// activations step j of a 32-row weight tile multiplies rows 8 g + j of the four lane groups g.
// KS > 1 (few rows): KS waves of a workgroup take a part of K each of the same column tiles, for as many workgroups and as short
// chains of loads as the weight allows (16 where there are few columns); their sums meet in LDS.
template <bool F32, int MT, int KS>
__global__ __launch_bounds__(KS > 4 ? 64 * KS : 256) void tile_gemm_kernel(TileGemm p) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int g = lane >> 4, ml = lane & 15;
    constexpr int TW = KS > 4 ? 1 : 2;
    const int nt0 = (KS > 1 ? blockIdx.x : blockIdx.x * 4 + wave) * TW;
    if (nt0 >= p.NTILES) return; // (KS > 1: the whole workgroup or nobody)
    const int kper = (p.ktiles + KS - 1) / KS, k0 = KS > 1 ? wave * kper : 0;
    const int k1 = k0 + kper < p.ktiles ? k0 + kper : p.ktiles;
    const int m0 = blockIdx.y * 16 * MT;
    int a_first = 0;
    if (p.group) { // blockIdx.z: the weight
        const int *rec = p.group_rows + 3 * blockIdx.z;
        p.packed = p.group[blockIdx.z].packed;
        p.M = rec[0] < p.M ? rec[0] : p.M;
        a_first = rec[1];
        p.C = (char *)p.C + (size_t)rec[2] * p.ldc * (p.c_dtype == XFTHIP_F32 ? 4 : 2);
        if (m0 >= p.M) return; // (the whole workgroup)
    }
    const uint8_t *w[TW];
    int aofs[2] = {0, 0};
#pragma unroll
    for (int t = 0; t < TW; ++t) {
        const int nt = nt0 + t < p.NTILES ? nt0 + t : p.NTILES - 1;
        w[t] = p.packed + (size_t)nt * p.KT * 1024 + lane * 16;
        aofs[t] = p.tiles_per_block ? nt / p.tiles_per_block * p.a_block_stride : 0;
    }
    const bool same = TW == 1 || aofs[0] == aofs[1];
    size_t row[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        const int r = m0 + m * 16 + ml;
        const int ra = a_first + (r < p.M ? r : p.M - 1);
        row[m] = (size_t)(p.a_rows ? p.a_rows[ra] : ra) * p.lda + 8 * g;
    }
    // the 16-wave form: one result a thread, and what the side embedding says about it is fetched at once
    float side_value = 1.0f;
    if constexpr (KS > 4) {
        const int r = m0 + (int)(threadIdx.x >> 8) * 16 + (int)((threadIdx.x >> 2) & 15), n = nt0 * 16 + 4 * (int)((threadIdx.x >> 6) & 3) + (int)(threadIdx.x & 3);
        if (p.side && (int)threadIdx.x < MT * 256 && r < p.M && n < p.N) {
            int id = p.side_ids[r];
            id = id < 0 ? 0 : (id >= p.side_vocab ? p.side_vocab - 1 : id);
            side_value = bf16_to_f32(p.side[(size_t)id * p.side_ld + n]);
        }
    }
    f32x4 acc[TW][MT];
#pragma unroll
    for (int t = 0; t < TW; ++t)
#pragma unroll
        for (int m = 0; m < MT; ++m) acc[t][m] = f32x4 {0.f, 0.f, 0.f, 0.f};

    if constexpr (F32) {
        for (int kt = k0; kt < k1; ++kt) {
            u32x4 wq[TW];
#pragma unroll
            for (int t = 0; t < TW; ++t) wq[t] = *(const u32x4 *)(w[t] + (size_t)kt * 1024);
            const float *A = (const float *)p.A;
#pragma unroll
            for (int m = 0; m < MT; ++m) {
                f32x4 a[2][2];
                a[0][0] = *(const f32x4 *)(A + row[m] + aofs[0] + kt * 32), a[0][1] = *(const f32x4 *)(A + row[m] + aofs[0] + kt * 32 + 4);
                if (same) {
                    a[1][0] = a[0][0], a[1][1] = a[0][1];
                } else {
                    a[1][0] = *(const f32x4 *)(A + row[m] + aofs[1] + kt * 32), a[1][1] = *(const f32x4 *)(A + row[m] + aofs[1] + kt * 32 + 4);
                }
#pragma unroll
                for (int t = 0; t < TW; ++t)
#pragma unroll
                    for (int j = 0; j < 8; ++j) {
                        const uint32_t pair = wq[t][j >> 1];
                        const float wv = u2f((j & 1) ? (pair & 0xFFFF0000u) : (pair << 16));
                        acc[t][m] = __builtin_amdgcn_mfma_f32_16x16x4f32(wv, a[t][j >> 2][j & 3], acc[t][m], 0, 0, 0);
                    }
            }
        }
    } else {
        // few rows: the loads of UN steps go out together, the chain of round trips is that much shorter
        constexpr int UN = KS > 1 ? 4 : 1;
        const uint16_t *A = (const uint16_t *)p.A;
        for (int kb = k0; kb < k1; kb += UN) {
            u32x4 wq[UN][TW], a0[UN][MT], a1[UN][MT];
#pragma unroll
            for (int u = 0; u < UN; ++u) {
                const int kt = kb + u < k1 ? kb + u : k1 - 1; // (past the end: the last step's once more, unused)
#pragma unroll
                for (int t = 0; t < TW; ++t) wq[u][t] = *(const u32x4 *)(w[t] + (size_t)kt * 1024);
#pragma unroll
                for (int m = 0; m < MT; ++m) {
                    a0[u][m] = *(const u32x4 *)(A + row[m] + aofs[0] + kt * 32);
                    a1[u][m] = a0[u][m];
                    if (TW > 1 && !same) a1[u][m] = *(const u32x4 *)(A + row[m] + aofs[1] + kt * 32);
                }
            }
#pragma unroll
            for (int u = 0; u < UN; ++u) {
                if (UN > 1 && kb + u >= k1) break;
#pragma unroll
                for (int m = 0; m < MT; ++m) {
                    acc[0][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, wq[u][0]), __builtin_bit_cast(bf16x8, a0[u][m]), acc[0][m], 0, 0, 0);
                    if constexpr (TW > 1)
                        acc[TW - 1][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, wq[u][TW - 1]), __builtin_bit_cast(bf16x8, a1[u][m]), acc[TW - 1][m], 0, 0, 0);
                }
            }
        }
    }

    if constexpr (KS > 4) {
        __shared__ f32x4 sums[KS][MT][64];
#pragma unroll
        for (int m = 0; m < MT; ++m) sums[wave][m][lane] = acc[0][m];
        __syncthreads();
        if ((int)threadIdx.x >= MT * 256) return;
        const float *part = (const float *)sums + threadIdx.x;
        float y = 0.0f;
#pragma unroll
        for (int w = 0; w < KS; ++w) y += part[w * MT * 256];
        const int r = m0 + (int)(threadIdx.x >> 8) * 16 + (int)((threadIdx.x >> 2) & 15), n = nt0 * 16 + 4 * (int)((threadIdx.x >> 6) & 3) + (int)(threadIdx.x & 3);
        if (r >= p.M || n >= p.N) return;
        const size_t at = (size_t)r * p.ldc + n;
        if (p.bias) y += p.bias[n];
        if (p.decay > 0.0f) y = decay_of<!F32>(y, p.decay);
        if (p.side) y = gelu_tanh(y) * side_value;
        if (p.add) y += ((const float *)p.C)[at];
        store_from_f32(p.C, p.c_dtype, at, y);
        return;
    } else {
        if constexpr (KS > 1) {
            __shared__ f32x4 sums[KS - 1][2 * MT][64];
            if (wave > 0) {
#pragma unroll
                for (int t = 0; t < 2; ++t)
#pragma unroll
                    for (int m = 0; m < MT; ++m) sums[wave - 1][t * MT + m][lane] = acc[t][m];
            }
            __syncthreads();
            if (wave > 0) return;
#pragma unroll
            for (int w = 0; w < KS - 1; ++w)
#pragma unroll
                for (int t = 0; t < 2; ++t)
#pragma unroll
                    for (int m = 0; m < MT; ++m) acc[t][m] += sums[w][t * MT + m][lane];
        }
#pragma unroll
        for (int m = 0; m < MT; ++m) {
            const int r = m0 + m * 16 + ml;
            if (r >= p.M) continue;
            if (p.glu) { // tile pairs: 16 gate columns, the matching 16 up columns
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int n = (nt0 >> 1) * 16 + 4 * g + i;
                    if (n >= p.N / 2) continue;
                    const float gate = acc[0][m][i] + (p.bias ? p.bias[n] : 0.0f), up = acc[1][m][i] + (p.bias ? p.bias[p.N / 2 + n] : 0.0f);
                    store_from_f32(p.C, p.c_dtype, (size_t)r * p.ldc + n, precise_glu(gate, up, p.glu_limit, p.glu_alpha));
                }
                continue;
            }
            const uint16_t *side = nullptr;
            if (p.side) {
                int id = p.side_ids[r];
                id = id < 0 ? 0 : (id >= p.side_vocab ? p.side_vocab - 1 : id);
                side = p.side + (size_t)id * p.side_ld;
            }
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                const int n = (nt0 + t) * 16 + 4 * g;
                if (side || p.add || p.bias || p.decay > 0.0f) {
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        if (n + i >= p.N) continue;
                        if (p.bias) acc[t][m][i] += p.bias[n + i];
                        if (p.decay > 0.0f) acc[t][m][i] = decay_of<!F32>(acc[t][m][i], p.decay);
                        if (side) acc[t][m][i] = gelu_tanh(acc[t][m][i]) * bf16_to_f32(side[n + i]);
                        if (p.add) acc[t][m][i] += ((const float *)p.C)[(size_t)r * p.ldc + n + i];
                    }
                }
                const size_t at = (size_t)r * p.ldc + n;
                if (n + 4 <= p.N && (p.ldc & 3) == 0) {
                    if (p.c_dtype == XFTHIP_F32)
                        *(f32x4 *)((float *)p.C + at) = acc[t][m];
                    else
                        *(uint2 *)((uint16_t *)p.C + at) = make_uint2(f32_to_bf16_ref(acc[t][m][0]) | ((uint32_t)f32_to_bf16_ref(acc[t][m][1]) << 16),
                                f32_to_bf16_ref(acc[t][m][2]) | ((uint32_t)f32_to_bf16_ref(acc[t][m][3]) << 16));
                } else {
#pragma unroll
                    for (int i = 0; i < 4; ++i)
                        if (n + i < p.N) store_from_f32(p.C, p.c_dtype, at + i, acc[t][m][i]);
                }
            }
        }
    }
}

} // namespace

int tile_gemm(xfthip_weight_t w, int act_in, const TileGemmArgs &a, hipStream_t st) {
    XFT_REQUIRE(w && a.A && a.C && a.M > 0, "tile_gemm: null argument");
    const PackedWeight &pw = w->pw;
    const int M = a.M;
    XFT_REQUIRE(pw.kind == XFTHIP_W_BF16 && pw.K % 32 == 0, "tile_gemm: BF16 weights with K a multiple of 32 (K=%d)", pw.K);
    XFT_REQUIRE(a.block_cols % 16 == 0 && a.lda % 8 == 0 && a.a_block_stride % 8 == 0 && ((uintptr_t)a.A & 15) == 0, "tile_gemm: unaligned operands");
    const int blocks = a.block_cols ? (pw.N + a.block_cols - 1) / a.block_cols : 1;
    XFT_REQUIRE((long)(blocks - 1) * a.a_block_stride + pw.K <= a.lda, "tile_gemm: %d blocks of K=%d reach past the row (%d)", blocks, pw.K, a.lda);
    XFT_REQUIRE(a.ldc >= (a.glu ? pw.N / 2 : pw.N) && a.glu == ((pw.flags & XFTHIP_WF_GATEUP) != 0), "tile_gemm: ldc=%d N=%d glu=%d", a.ldc, pw.N, a.glu);
    XFT_REQUIRE(!a.bias || !a.group, "tile_gemm: no bias in groups");
    XFT_REQUIRE(a.decay_tau >= 0.0f && (a.decay_tau == 0.0f || (!a.glu && !a.add && !a.side && !a.group)), "tile_gemm: decays of plain products only");
    XFT_REQUIRE((!a.add || (a.c_dtype == XFTHIP_F32 && !a.glu)) && (!a.side || (!a.glu && !a.group && a.side_ids)) && (!a.group || a.group_rows),
            "tile_gemm: options that do not go together");
    const TileGemm p = {pw.packed, pw.KT, pw.K / 32, pw.NTILES, pw.N, M, a.A, a.lda, a.block_cols / 16, a.a_block_stride, a.C, a.ldc, a.c_dtype, a.glu, a.add,
            a.glu_limit, a.glu_alpha, a.bias, a.decay_tau > 0.0f ? 1.0f / a.decay_tau : 0.0f, a.side, a.side_ld, a.side_vocab, a.side_ids, a.group, a.group_rows, a.a_rows};
    const unsigned gz = a.group ? (unsigned)a.group_n : 1;
    const unsigned gx = (unsigned)((pw.NTILES + 7) / 8), gx1 = (unsigned)((pw.NTILES + 1) / 2);
    const bool f32 = act_in == XFTHIP_F32;
    auto launch = [&](auto kernel, unsigned x, unsigned y) { hipLaunchKernelGGL(kernel, dim3(x, y, gz), dim3(256), 0, st, p); };
    auto launch16 = [&](auto kernel, unsigned x, unsigned y) { hipLaunchKernelGGL(kernel, dim3(x, y, gz), dim3(1024), 0, st, p); };
    const bool deep = pw.NTILES <= 64 && pw.K >= 1024 && !a.block_cols && !a.glu && !a.group; // few columns against a deep K
    if (!f32 && deep && M <= 32) {
        launch16(tile_gemm_kernel<false, 1, 16>, (unsigned)pw.NTILES, (unsigned)((M + 15) / 16));
    } else if (M <= 16) {
        if (f32) launch(tile_gemm_kernel<true, 1, 4>, gx1, 1);
        else launch(tile_gemm_kernel<false, 1, 4>, gx1, 1);
    } else if (!f32 && a.decay_tau > 0.0f) { // (a shallow K and a long epilogue: smaller tiles.  2048 rows x 4096 columns, K = 64: 24 us against 30)
        if (M <= 32) launch(tile_gemm_kernel<false, 1, 4>, gx1, 2);
        else launch(tile_gemm_kernel<false, 2, 1>, gx, (unsigned)((M + 31) / 32));
    } else if (M <= 32) {
        if (f32) launch(tile_gemm_kernel<true, 2, 4>, gx1, 1);
        else launch(tile_gemm_kernel<false, 2, 4>, gx1, 1);
    } else if ((long)gx * ((M + 63) / 64) < 2L * device_cu_count() && !a.group) {
        if (f32) launch(tile_gemm_kernel<true, 1, 1>, gx, (unsigned)((M + 15) / 16));
        else launch(tile_gemm_kernel<false, 1, 1>, gx, (unsigned)((M + 15) / 16));
    } else {
        if (f32) launch(tile_gemm_kernel<true, 4, 1>, gx, (unsigned)((M + 63) / 64));
        else launch(tile_gemm_kernel<false, 4, 1>, gx, (unsigned)((M + 63) / 64));
    }
    XFT_CHECK_HIP(hipGetLastError());
    return 0;
}

} // namespace xfthip
