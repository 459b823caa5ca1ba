// Driver of layer plans: the plan's weights (composed, padded and packed from the model's tensors), the page pool and the
// state slots, and the order of kernels a step runs.  One step is a ragged batch: segments of any length, each the next
// tokens of one sequence; a decode step is the same with one token a segment and everything position-dependent read from
// device memory, so that it can be recorded.
#include <math.h>
#include <string.h>

#include <algorithm>
#include <map>

#include "model_impl.h"
#include "plan_dev.h"

namespace xfthip {

namespace {

int pad32(int n) { return (n + 31) / 32 * 32; }

float bf16_value(uint16_t b) {
    const uint32_t u = (uint32_t)b << 16;
    float f;
    memcpy(&f, &u, 4);
    return f;
}

using Tensor = xfthip_plan::Tensor;

struct Matrix { // [K][N] bf16, zero where nothing is placed
    int K, N;
    std::vector<uint16_t> w;
    Matrix(int k, int n) : K(k), N(n), w((size_t)k * n, 0) {}
    // rows [r0, r0 + rows) and columns [c0, c0 + cols) of an [out, in] tensor to columns n0 .. / rows k0 ..
    void place(const Tensor &t, int r0, int rows, int c0, int cols, int k0, int n0) {
        for (int cb = 0; cb < cols; cb += 32)
            for (int rb = 0; rb < rows; rb += 32)
                for (int c = cb; c < cols && c < cb + 32; ++c)
                    for (int r = rb; r < rows && r < rb + 32; ++r) w[(size_t)(k0 + c) * N + n0 + r] = t.data[(size_t)(r0 + r) * t.cols + c0 + c];
    }
    // the same block turned round: tensor rows along K
    void place_turned(const Tensor &t, int r0, int rows, int c0, int cols, int k0, int n0) {
        for (int r = 0; r < rows; ++r) memcpy(&w[(size_t)(k0 + r) * N + n0], &t.data[(size_t)(r0 + r) * t.cols + c0], (size_t)cols * 2);
    }
};

__global__ void plan_decode_begin_kernel(EmbedTables e, const int *dec_rows, const int *pos, const int *ids, float *x, int *last_token, int *tok_seg,
        int *tok_pos, int *tok_ids, int *seg, int seg_cap, int *log, const int *step, int max_seq) {
    const int b = blockIdx.x, row = dec_rows[b], id = ids[row], prev = last_token[row];
    int at = pos[row];
    at = at < 0 ? 0 : (at >= max_seq ? max_seq - 1 : at);
    __syncthreads(); // (all have read the token before)
    if (threadIdx.x == 0) {
        log[(size_t)step[0] * gridDim.x + b] = id;
        tok_seg[b] = b, tok_pos[b] = at, tok_ids[b] = id;
        seg[b] = row, seg[seg_cap + b] = b, seg[2 * seg_cap + b] = 1, seg[3 * seg_cap + b] = at;
        last_token[row] = id;
    }
    embed_token(e, id, at == 0, prev, x + (size_t)b * e.hidden);
}

// behind a step: where its sequences stand, and the last token of each
__global__ void plan_advance_kernel(const int *seg, int seg_cap, int n, const int *ids, int *pos, int *last_token) {
    const int b = blockIdx.x * blockDim.x + threadIdx.x;
    if (b >= n) return;
    pos[seg[b]] = seg[3 * seg_cap + b] + seg[2 * seg_cap + b];
    last_token[seg[b]] = ids[seg[seg_cap + b] + seg[2 * seg_cap + b] - 1];
}

__global__ void plan_fill_kernel(int *p, int n, int v) {
    const int i = blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) p[i] = v;
}

// Frequency of pair i of a rotation and the factor on cos and sin.  Context extension: pairs that turn fewer than `slow` times
// within the original context have their frequency divided by the factor, those above `fast` keep it, a ramp over i between.
double rotation_frequency(const xfthip_plan_layer &s, int i) {
    const double f = pow(s.rot_base, -2.0 * i / s.rot_dim);
    if (s.rot_factor <= 0.0) return f;
    auto pair_at = [&](double turns) { return s.rot_dim * log(s.rot_original / (2.0 * M_PI * turns)) / (2.0 * log(s.rot_base)); };
    const double lo = std::max(floor(pair_at(s.rot_fast)), 0.0), hi = std::min(ceil(pair_at(s.rot_slow)), s.rot_dim - 1.0);
    const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
    return f / s.rot_factor * ramp + f * (1.0 - ramp);
}
double rotation_magnitude(const xfthip_plan_layer &s) { return s.rot_factor > 0.0 ? 0.1 * log(s.rot_factor) + 1.0 : 1.0; }

// rotation tables [positions][rot_dim / 2]: angles in double, as far apart as positions can be
int rotation_tables(const xfthip_plan_layer &s, int positions, float **cosT, float **sinT) {
    const int half = s.rot_dim / 2;
    const double mul = rotation_magnitude(s);
    std::vector<float> c((size_t)positions * half), sn((size_t)positions * half);
    for (int i = 0; i < half; ++i) {
        const double f = rotation_frequency(s, i);
        for (int p = 0; p < positions; ++p) c[(size_t)p * half + i] = (float)(cos(p * f) * mul), sn[(size_t)p * half + i] = (float)(sin(p * f) * mul);
    }
    XFT_CHECK_HIP(hipMalloc((void **)cosT, c.size() * 4 + 16));
    XFT_CHECK_HIP(hipMalloc((void **)sinT, sn.size() * 4 + 16));
    XFT_CHECK_HIP(hipMemcpy(*cosT, c.data(), c.size() * 4, hipMemcpyHostToDevice));
    XFT_CHECK_HIP(hipMemcpy(*sinT, sn.data(), sn.size() * 4, hipMemcpyHostToDevice));
    return 0;
}

int plan_gemm(xfthip_model *m, xfthip_weight_t w, int M, const void *A, int lda, void *C, int ldc, int c_dtype, hipStream_t st, const float *bias = nullptr) {
    // (few rows against few columns: the form with the most waves along K)
    if (m->plan->act == XFTHIP_F32 || (M <= 32 && w->pw.N <= 256 && w->pw.K >= 1024)) {
        TileGemmArgs a;
        a.M = M, a.A = A, a.lda = lda, a.C = C, a.ldc = ldc, a.c_dtype = c_dtype, a.bias = bias;
        return tile_gemm(w, m->plan->act, a, st);
    }
    return xfthip_gemm(w, M, A, lda, C, ldc, c_dtype, bias ? XFTHIP_EPI_BIAS : XFTHIP_EPI_NONE, bias, nullptr, 0, XFTHIP_F32, 1.0f, st);
}

// the product in front of a layer's mixers -> a
int plan_gemm_in(xfthip_model *m, const PlanLayer &L, int T, hipStream_t st) {
    const PlanState &p = *m->plan;
    return plan_gemm(m, L.in, T, p.xn, m->cfg.hidden, p.a, L.in_ld, p.act, st, L.in_bias);
}

// a sublayer's last product: into y, or, in parallel blocks, added to the residual
int plan_gemm_out(xfthip_model *m, xfthip_weight_t w, int M, const void *A, int lda, const float *bias, hipStream_t st) {
    const PlanState &p = *m->plan;
    const int hidden = m->cfg.hidden;
    if (p.plan->cfg.block != XFTHIP_BLOCK_PARALLEL) return plan_gemm(m, w, M, A, lda, p.y, hidden, XFTHIP_F32, st, bias);
    if (p.act == XFTHIP_F32) {
        TileGemmArgs a;
        a.M = M, a.A = A, a.lda = lda, a.C = m->x, a.ldc = hidden, a.add = true, a.bias = bias;
        return tile_gemm(w, XFTHIP_F32, a, st);
    }
    return xfthip_gemm(w, M, A, lda, m->x, hidden, XFTHIP_F32, XFTHIP_EPI_RESIDENTIAL, bias, m->x, hidden, XFTHIP_F32, 1.0f, st);
}

// heads side by side (block_cols output columns a head, a_block_stride input columns apart)
int plan_gemm_heads(int act, xfthip_weight_t w, int M, const void *A, int lda, int block_cols, int a_block_stride, void *C, int ldc, int c_dtype, hipStream_t st) {
    TileGemmArgs a;
    a.M = M, a.A = A, a.lda = lda, a.block_cols = block_cols, a.a_block_stride = a_block_stride, a.C = C, a.ldc = ldc, a.c_dtype = c_dtype;
    return tile_gemm(w, act, a, st);
}

int run_latent(xfthip_model *m, const PlanLayer &L, int run, const StepView &v, hipStream_t st) {
    PlanState &p = *m->plan;
    const int T = v.T, H = L.s.heads, act = p.act;
    const int qcols = H * (L.D + L.RD);
    const LatentCacheView cache = {p.cache[run], L.R, L.RD};
    int rc;
    if ((rc = plan_gemm_in(m, L, T, st))) return rc;
    if ((rc = latent_prepare(act, L, v, p.a, p.cq, cache, m->cfg.rms_eps, st))) return rc;
    if ((rc = plan_gemm(m, L.uq, T, p.cq, L.QR, p.q, qcols, act, st))) return rc;
    if ((rc = latent_rotate_q(act, L, v, p.q, st))) return rc;
    // long segments one by one in the expanded form; the others, as far as they are neighbours, together in the absorbed one
    const size_t B = p.seg_len_host.size();
    const char *q = (const char *)p.q;
    int longest = 0, short_from = -1;
    auto absorb = [&](int from, int to) {
        return plan_gemm_heads(act, L.absorb, to - from, q + (size_t)from * qcols * p.esz, qcols, L.R, L.D + L.RD, (char *)p.qa + (size_t)from * H * L.R * p.esz,
                H * L.R, act, st);
    };
    auto to_values = [&](int from, int to) {
        return plan_gemm_heads(act, L.uv, to - from, (char *)p.oc + (size_t)from * H * L.R * p.esz, H * L.R, L.V, L.R,
                (char *)p.ov + (size_t)from * H * L.V * p.esz, H * L.V, act, st);
    };
    std::vector<std::pair<int, int>> spans; // token ranges of the absorbed form
    for (size_t i = 0; i < B; ++i) {
        const int n = p.seg_len_host[i], off = p.seg_off_host[i], start = p.seg_pos_host[i];
        const int from = L.s.window > 0 && start + 1 > L.s.window ? (start + 1 - L.s.window) & ~31 : 0, rows = start + n - from;
        const bool expand = p.kx != nullptr && latent_expanded_takes(act, L, n, rows);
        if (!expand) {
            longest = std::max(longest, n);
            if (short_from < 0) short_from = off;
        }
        if (short_from >= 0 && (expand || i + 1 == B)) {
            spans.push_back({short_from, expand ? off : off + n});
            short_from = -1;
        }
        if (!expand) continue;
        if ((rc = latent_gather(v, p.seg_row_host[i], from, rows, cache, p.rows, st))) return rc;
        if ((rc = xfthip_gemm(L.uk, rows, p.rows, L.R + L.RD, p.kx, H * L.D, XFTHIP_BF16, XFTHIP_EPI_NONE, nullptr, nullptr, 0, XFTHIP_F32, 1.0f, st))) return rc;
        if ((rc = xfthip_gemm(L.uv, rows, p.rows, L.R + L.RD, p.vx, H * L.V, XFTHIP_BF16, XFTHIP_EPI_NONE, nullptr, nullptr, 0, XFTHIP_F32, 1.0f, st))) return rc;
        if ((rc = latent_expanded(L, off, start, n, from, p.q, p.kx, p.vx, p.rows, p.ov, st))) return rc;
    }
    if (!spans.empty()) {
        for (auto &s : spans)
            if ((rc = absorb(s.first, s.second))) return rc;
        if ((rc = latent_attention(act, L, v, longest, p.qa, p.q, p.oc, cache, m->len_hint, p.part, p.part_floats, st))) return rc;
        for (auto &s : spans)
            if ((rc = to_values(s.first, s.second))) return rc;
    }
    return plan_gemm_out(m, L.o, T, p.ov, H * L.V, nullptr, st);
}

int mix_delta(xfthip_model *m, const PlanLayer &L, int store, const StepView &v, hipStream_t st) {
    PlanState &p = *m->plan;
    const int act = p.act;
    int rc;
    const DeltaBuffers b = {p.a, p.gates, p.dq, p.dk, p.dqk, p.dg, p.dv, p.dbeta, p.do_, p.ov, p.state[store], p.conv_state[store]};
    if (L.gates) {
        const int first = L.in_col + L.channels() + L.beta_cols();
        if ((rc = plan_gemm_heads(act, L.gates, v.T, (const char *)p.a + (size_t)first * p.esz, L.in_ld, L.gcols, L.rank, p.gates, 2 * L.gcols, XFTHIP_F32, st)))
            return rc;
    }
    if ((rc = delta_prepare(act, L, v, b, st))) return rc;
    if ((rc = delta_scan(L, v, b, st))) return rc;
    return delta_output(act, L, v, b, m->cfg.rms_eps, st);
}

int mix_grouped(xfthip_model *m, const PlanLayer &L, int store, const StepView &v, hipStream_t st) {
    PlanState &p = *m->plan;
    int rc;
    const PageTable &t = p.tables[L.means_table];
    const GroupedBuffers b = {p.a, p.q, p.cache[p.reads[store]], p.first_values, p.conv_state[store], p.means[store], p.table + t.at, t.stride};
    if ((rc = grouped_prepare(p.act, L, v, b, m->cfg.rms_eps, st))) return rc;
    return grouped_attention(p.act, L, v, b, p.ov, m->len_hint, p.part, p.part_floats, st);
}

int mix_unit(xfthip_model *m, const PlanLayer &L, int store, const StepView &v, hipStream_t st) {
    PlanState &p = *m->plan;
    int rc;
    const UnitBuffers b = {p.a, p.u, p.gates, p.carry, p.ov, p.state[store], p.conv_state[store]};
    if ((rc = unit_filter(p.act, L, v, b, st))) return rc;
    if ((rc = plan_gemm_heads(p.act, L.gates, v.T, p.u, L.channels(), 2 * L.D, L.D, p.gates, 2 * L.channels(), XFTHIP_F32, st))) return rc;
    return unit_scan(p.act, L, v, b, st);
}

int mix_linear(xfthip_model *m, const PlanLayer &L, int store, const StepView &v, hipStream_t st) {
    PlanState &p = *m->plan;
    TileGemmArgs a; // the decays
    a.M = v.T, a.A = (const char *)p.a + (size_t)(L.in_col + L.channels()) * p.esz, a.lda = L.in_ld, a.block_cols = L.s.heads * L.KD, a.C = p.gates;
    a.ldc = L.s.heads * L.KD, a.bias = L.dt_bias, a.decay_tau = L.s.tau;
    if (int rc = tile_gemm(L.gates, p.act, a, st)) return rc;
    return linear_attention(p.act, L, v, {p.a, p.gates, p.do_, p.ov, p.state[store]}, m->cfg.rms_eps, st);
}

// between the input and the output product of a mixer
int mix(xfthip_model *m, const PlanLayer &L, int store, const StepView &v, hipStream_t st) {
    switch (L.s.mixer) {
        case XFTHIP_MIXER_GROUPED: return mix_grouped(m, L, store, v, st);
        case XFTHIP_MIXER_UNIT: return mix_unit(m, L, store, v, st);
        case XFTHIP_MIXER_LINEAR: return mix_linear(m, L, store, v, st);
        default: return mix_delta(m, L, store, v, st);
    }
}

int run_mixers(xfthip_model *m, int run, const StepView &v, hipStream_t st) {
    PlanState &p = *m->plan;
    const LayerRun &r = p.plan->runs[run];
    const PlanLayer &L = p.layers[r.layer];
    if (L.s.mixer == XFTHIP_MIXER_LATENT) return run_latent(m, L, run, v, st);
    int rc;
    if ((rc = plan_gemm_in(m, L, v.T, st))) return rc;
    if ((rc = mix(m, L, run, v, st))) return rc;
    if (r.beside >= 0 && (rc = mix(m, p.layers[r.beside], r.beside_store, v, st))) return rc;
    if (L.result_norm) { // the results meet behind norms of their own
        const PlanLayer &S = p.layers[r.beside];
        if ((rc = plan_gemm(m, S.o, v.T, (const char *)p.ov + (size_t)S.out_col * p.esz, S.out_ld, p.y2, m->cfg.hidden, XFTHIP_F32, st, S.o_bias))) return rc;
    }
    return plan_gemm_out(m, L.o, v.T, p.ov, L.out_ld, L.o_bias, st);
}

// gate and up projections of a dense or shared feed-forward, combined -> h
int run_gateup(xfthip_model *m, const PlanLayer &L, int T, const void *in, hipStream_t st) {
    PlanState &p = *m->plan;
    const int hidden = m->cfg.hidden;
    if (p.act != XFTHIP_F32 && L.s.glu_alpha == 0.0f) return xfthip_gemm_gateup_silu_bias(L.gateup, T, in, hidden, p.h, L.ff, XFTHIP_BF16, L.gateup_bias, st);
    if (p.act != XFTHIP_F32) return xfthip_gemm_gateup_clamped(L.gateup, T, in, hidden, p.h, L.ff, XFTHIP_BF16, L.s.glu_limit, L.s.glu_alpha, st);
    TileGemmArgs a;
    a.M = T, a.A = in, a.lda = hidden, a.C = p.h, a.ldc = L.ff, a.c_dtype = XFTHIP_F32, a.glu = true, a.glu_limit = L.s.glu_limit, a.glu_alpha = L.s.glu_alpha;
    a.bias = L.gateup_bias;
    return tile_gemm(L.gateup, XFTHIP_F32, a, st);
}

// the products of all chosen experts: in -> eh -> expert_out, rows by the lists of the routing
int run_experts(xfthip_model *m, const PlanLayer &L, int T, const void *in, hipStream_t st) {
    PlanState &p = *m->plan;
    const xfthip_plan_layer &s = L.s;
    const int hidden = m->cfg.hidden, E = s.experts;
    const int most = s.top < E ? s.top : E; // choices of a token that reach an expert
    const RouteBuffers &r = p.route;
    int rc;
    if (p.act != XFTHIP_F32) {
        if ((rc = gemm_grouped_rows_dev(L.egateup.data(), E, L.etable, most * T, T, r.group_rows, 3, in, hidden, p.eh, L.eff, XFTHIP_BF16, st, r.row_token,
                     s.expert_limit, s.glu_alpha)))
            return rc;
        return gemm_grouped_rows_dev(L.edown.data(), E, L.etable + E, most * T, T, r.group_rows, 3, p.eh, L.eff, p.expert_out, hidden, XFTHIP_F32, st);
    }
    TileGemmArgs a;
    a.M = T, a.A = in, a.lda = hidden, a.C = p.eh, a.ldc = L.eff, a.c_dtype = XFTHIP_F32, a.glu = true, a.glu_limit = s.expert_limit, a.glu_alpha = s.glu_alpha;
    a.group = L.etable, a.group_n = E, a.group_rows = r.group_rows, a.a_rows = r.row_token;
    if ((rc = tile_gemm(L.egateup[0], XFTHIP_F32, a, st))) return rc;
    TileGemmArgs d;
    d.M = T, d.A = p.eh, d.lda = L.eff, d.C = p.expert_out, d.ldc = hidden, d.group = L.etable + E, d.group_n = E, d.group_rows = r.group_rows;
    return tile_gemm(L.edown[0], XFTHIP_F32, d, st);
}

// The feed-forward: dense, or routed experts beside an optional shared one.  Its result goes where plan_gemm_out puts results; in
// (activation type) is its input, narrow (or null) receives the residual behind a parallel block, of the activation type.
int run_feed_forward(xfthip_model *m, const PlanLayer &L, int T, const void *in, void *narrow, hipStream_t st) {
    PlanState &p = *m->plan;
    const bool parallel = p.plan->cfg.block == XFTHIP_BLOCK_PARALLEL;
    const int hidden = m->cfg.hidden;
    int rc;
    if (L.ff > 0) {
        if ((rc = run_gateup(m, L, T, in, st))) return rc;
        if ((rc = plan_gemm_out(m, L.down, T, p.h, L.ff, L.down_bias, st))) return rc;
    }
    float *dst = parallel ? m->x : p.y;
    if (L.s.experts > 0) {
        const int ld = pad32(L.routes());
        const RouteRule rule = {L.s.experts, L.routes(), L.s.top, L.correction, L.s.router == XFTHIP_ROUTE_SIGMOID_GROUPS ? L.s.route_groups : 0, L.s.route_keep,
                L.s.route_scale};
        if ((rc = plan_gemm(m, L.router, T, in, hidden, p.router_logits, ld, XFTHIP_F32, st))) return rc;
        if ((rc = route_tokens(p.router_logits, ld, rule, T, p.route, st))) return rc;
        if ((rc = run_experts(m, L, T, in, st))) return rc;
        return combine_experts(p.act, parallel || L.ff > 0 ? dst : nullptr, p.expert_out, in, L.s.top, p.route, dst, narrow, T, hidden, st);
    }
    return narrow ? combine_experts(p.act, dst, nullptr, nullptr, 0, p.route, dst, narrow, T, hidden, st) : 0;
}

// y = P (gelu(G x) * e) of the token's side embedding; x: the residual in the activation type
int run_side(xfthip_model *m, const PlanLayer &L, int layer, int T, const void *x, hipStream_t st) {
    PlanState &p = *m->plan;
    const xfthip_plan &plan = *p.plan;
    const int hidden = m->cfg.hidden, pad = plan.side_pad, ld = pad * plan.cfg.layers;
    int rc;
    if (p.act == XFTHIP_F32 || T <= 32) { // the gate in the product's epilogue
        TileGemmArgs a;
        a.M = T, a.A = x, a.lda = hidden, a.C = p.side, a.ldc = pad, a.c_dtype = p.act;
        a.side = plan.side_embedding + (size_t)layer * pad, a.side_ld = ld, a.side_ids = p.ids, a.side_vocab = m->cfg.vocab;
        if ((rc = tile_gemm(L.side_gate, p.act, a, st))) return rc;
    } else {
        if ((rc = plan_gemm(m, L.side_gate, T, x, hidden, p.side_z, pad, XFTHIP_F32, st))) return rc;
        if ((rc = plan_side_gate(p.act, p.side_z, plan.side_embedding, ld, layer * pad, p.ids, m->cfg.vocab, p.side, T, pad, st))) return rc;
    }
    return plan_gemm(m, L.side_proj, T, p.side, pad, p.y, hidden, XFTHIP_F32, st);
}

// all layer runs over the step's tokens, whose embeddings are in m->x
int plan_layers(xfthip_model *m, const StepView &v, hipStream_t st) {
    PlanState &p = *m->plan;
    const xfthip_plan &plan = *p.plan;
    const int T = v.T, hidden = m->cfg.hidden;
    const bool parallel = plan.cfg.block == XFTHIP_BLOCK_PARALLEL;
    const int nruns = (int)plan.runs.size();
    int rc;
    // next: the layer whose first norms follow, or null
    // pair: the layer whose mixers' results meet here, or null
    auto norm = [&](const float *y, const float *post, bool again, const PlanNorm &pre, const PlanNorm &pre2, const PlanLayer *pair) {
        PlanNormArgs a = {m->x, y, post, again ? plan.embedding : nullptr, p.ids, m->cfg.vocab, pre, pre2, p.xn, p.xn2, nullptr, hidden, plan.cfg.hidden,
                m->cfg.rms_eps, plan.cfg.residual_mult, plan.cfg.norm_groups};
        if (pair && pair->result_norm) a.y2 = p.y2, a.mix1 = pair->result_norm, a.mix2 = p.layers[pair->beside].result_norm;
        return plan_norm(p.act, a, T, st);
    };
    const PlanNorm none;
    auto enter = [&](const float *y, const float *post, bool again, const PlanLayer *next) {
        return norm(y, post, again, next ? next->pre1 : none, next && parallel ? next->pre2 : none, nullptr);
    };
    if ((rc = enter(nullptr, nullptr, plan.runs[0].add_embedding, &p.layers[plan.runs[0].layer]))) return rc;
    for (int r = 0; r < nruns; ++r) {
        const PlanLayer &L = p.layers[plan.runs[r].layer];
        const bool last = r + 1 == nruns;
        // (a traced run keeps the embedding of a further pass apart, so that the trace shows the layer's own result)
        const bool again = !last && plan.runs[r + 1].add_embedding, join = again && !p.trace;
        const PlanLayer *next = last ? nullptr : &p.layers[plan.runs[r + 1].layer], *then = p.trace ? nullptr : next;
        if ((rc = run_mixers(m, r, v, st))) return rc;
        const bool ff = L.feeds_forward(), side = plan.cfg.side_dim > 0;
        const void *narrow = p.act == XFTHIP_F32 ? (const void *)m->x : p.narrow; // what the side embedding's gate reads
        void *narrow_out = side && p.act != XFTHIP_F32 ? p.narrow : nullptr;
        if (parallel) {
            if ((ff || narrow_out) && (rc = run_feed_forward(m, L, T, p.xn2, narrow_out, st))) return rc;
            if (side && (rc = run_side(m, L, plan.runs[r].layer, T, narrow, st))) return rc;
            if (!last || side)
                if ((rc = enter(side ? p.y : nullptr, L.side_post, join, then))) return rc;
        } else {
            if ((rc = norm(p.y, L.post1, !ff && join, ff ? L.pre2 : then ? then->pre1 : none, none, &L))) return rc;
            if (ff) {
                if ((rc = run_feed_forward(m, L, T, p.xn, nullptr, st))) return rc;
                if ((rc = enter(p.y, L.post2, join, then))) return rc;
            }
        }
        if (p.trace) {
            XFT_CHECK_HIP(hipMemcpyAsync(p.trace_buf + (size_t)r * T * hidden, m->x, (size_t)T * hidden * 4, hipMemcpyDeviceToDevice, st));
            if (!last && (rc = enter(nullptr, nullptr, again, next))) return rc;
        }
    }
    return 0;
}

int upload_table(PlanState &p, hipStream_t st) {
    if (!p.table_dirty) return 0;
    memcpy(p.table_pinned, p.table_host.data(), p.table_host.size() * 4);
    XFT_CHECK_HIP(hipMemcpyAsync(p.table, p.table_pinned, p.table_host.size() * 4, hipMemcpyHostToDevice, st));
    p.table_dirty = false;
    return 0;
}

StepView view_of(const xfthip_model *m, int B, int T, int longest) {
    const PlanState &p = *m->plan;
    const int cap = p.slots;
    return StepView {B, T, longest, p.tok_seg, p.tok_pos, p.seg, p.seg + cap, p.seg + 2 * cap, p.seg + 3 * cap, p.table, p.tables[0].stride};
}

EmbedTables embed_tables(const xfthip_model *m) {
    const xfthip_plan &plan = *m->plan->plan;
    const xfthip_plan_config &c = plan.cfg;
    return EmbedTables {plan.embedding, plan.pair_embedding, m->cfg.hidden, m->cfg.vocab, c.embed_scale, c.bigram_buckets, c.bigram_mul_prev, c.bigram_mul_cur};
}

} // namespace

int plan_reserve(xfthip_model *m, int row, int tokens) {
    PlanState &p = *m->plan;
    for (PageTable &t : p.tables) {
        const int need = t.pages_for(tokens);
        XFT_REQUIRE(need <= t.stride, "the sequence of slot %d is longer than the model's %d positions", row, m->cfg.max_seq);
        while ((int)t.held[row].size() < need) {
            XFT_REQUIRE(!t.free_pages.empty(), "the page pool (%d pages of %d entries, %d tokens each) is exhausted", t.pages, kPageTokens, t.unit);
            const int page = t.free_pages.back();
            t.free_pages.pop_back();
            p.table_host[t.at + (size_t)row * t.stride + t.held[row].size()] = page;
            t.held[row].push_back(page);
            p.table_dirty = true;
        }
    }
    return 0;
}

void plan_release(xfthip_model *m, int row) {
    for (PageTable &t : m->plan->tables) {
        for (size_t i = t.held[row].size(); i-- > 0;) t.free_pages.push_back(t.held[row][i]);
        t.held[row].clear();
    }
}

int plan_run(xfthip_model *m, int n, const int *rows, const int *lens, const int *ids, hipStream_t st) {
    PlanState &p = *m->plan;
    const xfthip_model_config &c = m->cfg;
    XFT_REQUIRE(n > 0 && n <= p.slots, "a step of %d entries; the model has %d slots", n, p.slots);
    std::vector<char> seen(p.slots, 0);
    long T = 0;
    int longest = 0, deepest = 0;
    for (int i = 0; i < n; ++i) {
        XFT_REQUIRE(rows[i] >= 0 && rows[i] < p.slots && !seen[rows[i]], "slot %d listed twice or outside the model's %d", rows[i], p.slots);
        seen[rows[i]] = 1;
        const int at = m->row_pos[rows[i]] < 0 ? 0 : m->row_pos[rows[i]];
        XFT_REQUIRE(lens[i] > 0 && at + lens[i] <= c.max_seq, "slot %d: %d tokens at position %d exceed the model's %d positions", rows[i], lens[i], at, c.max_seq);
        T += lens[i];
        longest = std::max(longest, lens[i]);
        deepest = std::max(deepest, at + lens[i]);
    }
    XFT_REQUIRE(T <= c.max_tokens, "a step of %ld tokens; the model takes %d", T, c.max_tokens);
    for (int i = 0; i < n; ++i)
        if (int rc = plan_reserve(m, rows[i], std::max(m->row_pos[rows[i]], 0) + lens[i])) return rc;
    if (int rc = upload_table(p, st)) return rc;
    // the description: tok_seg | tok_pos | ids | seg (4 arrays of `slots`), one copy each way
    const int cap = p.slots, mt = c.max_tokens;
    int *hs = p.desc_host, *hp = hs + mt, *hi = hp + mt, *hg = hi + mt;
    int t = 0;
    p.seg_off_host.resize(n), p.seg_len_host.assign(lens, lens + n), p.seg_pos_host.resize(n), p.seg_row_host.assign(rows, rows + n);
    for (int i = 0; i < n; ++i) {
        const int at = std::max(m->row_pos[rows[i]], 0);
        p.seg_off_host[i] = t, p.seg_pos_host[i] = at;
        hg[i] = rows[i], hg[cap + i] = t, hg[2 * cap + i] = lens[i], hg[3 * cap + i] = at;
        for (int k = 0; k < lens[i]; ++k, ++t) hs[t] = i, hp[t] = at + k, hi[t] = ids[t];
    }
    XFT_CHECK_HIP(hipMemcpyAsync(p.tok_seg, hs, (size_t)T * 4, hipMemcpyHostToDevice, st));
    XFT_CHECK_HIP(hipMemcpyAsync(p.tok_pos, hp, (size_t)T * 4, hipMemcpyHostToDevice, st));
    XFT_CHECK_HIP(hipMemcpyAsync(p.ids, hi, (size_t)T * 4, hipMemcpyHostToDevice, st));
    XFT_CHECK_HIP(hipMemcpyAsync(p.seg, hg, (size_t)4 * cap * 4, hipMemcpyHostToDevice, st));
    const StepView view = view_of(m, n, (int)T, longest);
    if (int rc = plan_embed(embed_tables(m), view, p.ids, p.last_token, m->x, st)) return rc;
    m->len_hint = deepest;
    if (p.trace) {
        const size_t need = p.plan->runs.size() * (size_t)T * c.hidden;
        if (need > p.trace_floats) {
            XFT_CHECK_HIP(hipStreamSynchronize(st));
            if (p.trace_buf) (void)hipFree(p.trace_buf);
            p.trace_buf = nullptr, p.trace_floats = 0;
            XFT_CHECK_HIP(hipMalloc((void **)&p.trace_buf, need * 4));
            p.trace_floats = need;
        }
        p.trace_tokens = (int)T;
    }
    if (int rc = plan_layers(m, view, st)) return rc;
    hipLaunchKernelGGL(plan_advance_kernel, dim3((n + 63) / 64), dim3(64), 0, st, p.seg, cap, n, p.ids, m->pos, p.last_token);
    XFT_CHECK_HIP(hipGetLastError());
    for (int i = 0; i < n; ++i) m->row_pos[rows[i]] = std::max(m->row_pos[rows[i]], 0) + lens[i];
    return 0;
}

int plan_head(xfthip_model *m, const int *rows_dev, int n, int at, hipStream_t st) {
    PlanState &p = *m->plan;
    const xfthip_plan &plan = *p.plan;
    const xfthip_model_config &c = m->cfg;
    const PlanNormArgs a = {m->x, nullptr, nullptr, nullptr, nullptr, c.vocab, plan.final_norm, {}, p.xn, nullptr, rows_dev, c.hidden, plan.cfg.hidden, c.rms_eps, 0.0f,
            plan.cfg.norm_groups};
    if (int rc = plan_norm(p.act, a, n, st)) return rc;
    float *logits = m->logits + (size_t)at * c.vocab;
    if (int rc = plan_gemm(m, plan.head, n, p.xn, c.hidden, logits, c.vocab, XFTHIP_F32, st)) return rc;
    return plan.cfg.logit_softcap > 0.0f ? plan_softcap(logits, (size_t)n * c.vocab, plan.cfg.logit_softcap, st) : 0;
}

int plan_logits(xfthip_model *m, const int *list, int n, float *logits_host, hipStream_t st) {
    PlanState &p = *m->plan;
    const size_t vocab = m->cfg.vocab;
    for (int i = 0; i < n; i += p.logit_rows) {
        const int k = std::min(n - i, p.logit_rows);
        memcpy(p.want_host, list + i, (size_t)k * 4);
        XFT_CHECK_HIP(hipMemcpyAsync(p.want, p.want_host, (size_t)k * 4, hipMemcpyHostToDevice, st));
        if (int rc = plan_head(m, p.want, k, 0, st)) return rc;
        XFT_CHECK_HIP(hipMemcpyAsync(p.logits_pinned, m->logits, (size_t)k * vocab * 4, hipMemcpyDeviceToHost, st));
        XFT_CHECK_HIP(hipStreamSynchronize(st));
        memcpy(logits_host + (size_t)i * vocab, p.logits_pinned, (size_t)k * vocab * 4);
    }
    return 0;
}

int plan_prompt_pass(xfthip_model *m, const int *rows, int B, int S, const int *ids, float *logits_host, hipStream_t st) {
    PlanState &p = *m->plan;
    const xfthip_model_config &c = m->cfg;
    std::vector<int> lens(B, S);
    if (int rc = plan_run(m, B, rows, lens.data(), ids, st)) return rc;
    for (int b = 0; b < B; ++b) p.want_host[b] = (b + 1) * S - 1;
    XFT_CHECK_HIP(hipMemcpyAsync(p.want, p.want_host, (size_t)B * 4, hipMemcpyHostToDevice, st));
    // (the prompts of one call sit in neighbouring slots)
    if (int rc = plan_head(m, p.want, B, rows[0], st)) return rc;
    if (int rc = argmax_rows(m->logits + (size_t)rows[0] * c.vocab, B, c.vocab, m->ids, p.seg, nullptr, nullptr, st)) return rc;
    hipLaunchKernelGGL(plan_fill_kernel, dim3(1), dim3(64), 0, st, m->step, 1, 0);
    XFT_CHECK_HIP(hipGetLastError());
    if (logits_host)
        XFT_CHECK_HIP(hipMemcpyAsync(p.logits_pinned, m->logits + (size_t)rows[0] * c.vocab, (size_t)B * c.vocab * 4, hipMemcpyDeviceToHost, st));
    XFT_CHECK_HIP(hipStreamSynchronize(st));
    if (logits_host) memcpy(logits_host, p.logits_pinned, (size_t)B * c.vocab * 4);
    for (int b = 0; b < B; ++b) p.logit_of_row[rows[b]] = rows[0] + b;
    return 0;
}

int plan_decode_begin(xfthip_model *m, int steps, hipStream_t st) {
    PlanState &p = *m->plan;
    for (int r : p.dec_list)
        if (int rc = plan_reserve(m, r, m->row_pos[r] + steps)) return rc;
    if (int rc = upload_table(p, st)) return rc;
    memcpy(p.dec_host, p.dec_list.data(), p.dec_list.size() * 4);
    XFT_CHECK_HIP(hipMemcpyAsync(p.dec_rows, p.dec_host, p.dec_list.size() * 4, hipMemcpyHostToDevice, st));
    for (size_t b = 0; b < p.dec_list.size(); ++b) p.logit_of_row[p.dec_list[b]] = (int)b;
    return 0;
}

int plan_decode_step(xfthip_model *m, int B, hipStream_t st) {
    PlanState &p = *m->plan;
    const xfthip_model_config &c = m->cfg;
    hipLaunchKernelGGL(plan_decode_begin_kernel, dim3(B), dim3(256), 0, st, embed_tables(m), p.dec_rows, m->pos, m->ids, m->x, p.last_token, p.tok_seg,
            p.tok_pos, p.ids, p.seg, p.slots, m->idlog, m->step, c.max_seq);
    XFT_CHECK_HIP(hipGetLastError());
    const bool trace = p.trace;
    p.trace = false;
    // (lengths and offsets only: where the segments stand is known on the device)
    p.seg_off_host.resize(B), p.seg_len_host.assign(B, 1), p.seg_pos_host.assign(B, 0), p.seg_row_host.assign(B, 0);
    for (int b = 0; b < B; ++b) p.seg_off_host[b] = b;
    int rc = plan_layers(m, view_of(m, B, B, 1), st);
    p.trace = trace;
    if (rc) return rc;
    if ((rc = plan_head(m, nullptr, B, 0, st))) return rc;
    return argmax_rows(m->logits, B, c.vocab, m->ids, p.dec_rows, m->pos, m->step, st);
}

int plan_decode_splits(xfthip_model *m, int B, int hint) {
    int s = 0; // the split counts of the attentions, as far as a recorded step depends on them
    for (auto &L : m->plan->layers)
        if (L.s.mixer == XFTHIP_MIXER_LATENT) s = s * 31 + latent_split_count(L, B, 1, hint);
        else if (L.s.mixer == XFTHIP_MIXER_GROUPED) s = s * 31 + grouped_split_count(L, B, 1, hint);
    return s;
}

// Slot dst[i] becomes a copy of slot src[i]: pages, recurrent state, convolution inputs.  Everything is read before anything
// is written (through a staging buffer, run by run).
int plan_reorder(xfthip_model *m, const int *dst, const int *src, int n, hipStream_t st) {
    PlanState &p = *m->plan;
    XFT_CHECK_HIP(hipStreamSynchronize(st));
    std::vector<std::vector<std::vector<int>>> from(p.tables.size()); // pages of the sources, by table
    for (size_t t = 0; t < p.tables.size(); ++t) {
        PageTable &pt = p.tables[t];
        for (int i = 0; i < n; ++i) from[t].push_back(pt.held[src[i]]);
        for (int i = 0; i < n; ++i)
            while (pt.held[dst[i]].size() > from[t][i].size()) {
                pt.free_pages.push_back(pt.held[dst[i]].back());
                pt.held[dst[i]].pop_back();
            }
    }
    // (a slot whose pages another one reads keeps them: it is a destination itself only if it is listed, with as many or more pages)
    // what a record keeps: pages of some table, and so many bytes a slot
    struct Kept {
        char *base;
        int table; // or -1: by slot
        size_t bytes; // of a page or a slot
    };
    auto kept = [&](size_t r) {
        const PlanLayer &L = p.layers[p.store_layer[r]];
        std::vector<Kept> k;
        if (L.kv_from >= 0) return k; // (what it reads is another record's)
        const size_t page = kPageTokens * L.token_elems() * p.esz;
        if (L.paged()) k.push_back({(char *)p.cache[r], 0, page});
        if (L.means_table) k.push_back({(char *)p.means[r], L.means_table, page});
        if (L.state_floats()) k.push_back({(char *)p.state[r], -1, L.state_floats() * 4});
        if (L.history()) k.push_back({(char *)p.conv_state[r], -1, L.history() * p.esz});
        return k;
    };
    size_t bytes = (size_t)n * 4;
    const size_t stores = p.store_layer.size();
    for (size_t r = 0; r < stores; ++r)
        for (const Kept &k : kept(r)) {
            size_t need = 0;
            for (int i = 0; i < n; ++i) need += k.bytes * (k.table < 0 ? 1 : from[k.table][i].size());
            bytes = std::max(bytes, need);
        }
    char *stage = nullptr;
    XFT_CHECK_HIP(hipMalloc((void **)&stage, bytes + 16));
    int rc = 0;
    for (int i = 0; i < n && rc == 0; ++i) rc = plan_reserve(m, dst[i], (int)from[0][i].size() * kPageTokens);
    if (rc == 0) rc = upload_table(p, st);
    hipError_t e = hipSuccess;
    auto copy = [&](void *d, const void *s, size_t b) {
        if (e == hipSuccess && b) e = hipMemcpyAsync(d, s, b, hipMemcpyDeviceToDevice, st);
    };
    for (int write = 0; write < 2 && rc == 0; ++write)
        for (int i = 0; i < n; ++i) {
            if (write) copy(p.last_token + dst[i], stage + 4 * (size_t)i, 4);
            else copy(stage + 4 * (size_t)i, p.last_token + src[i], 4);
        }
    for (size_t r = 0; r < stores && rc == 0; ++r)
        for (const Kept &k : kept(r))
            for (int write = 0; write < 2; ++write) {
                size_t at = 0;
                for (int i = 0; i < n; ++i) {
                    const size_t count = k.table < 0 ? 1 : from[k.table][i].size();
                    for (size_t j = 0; j < count; ++j, at += k.bytes) {
                        const int place = k.table < 0 ? (write ? dst[i] : src[i]) : write ? p.tables[k.table].held[dst[i]][j] : from[k.table][i][j];
                        char *there = k.base + (size_t)place * k.bytes;
                        if (write) copy(there, stage + at, k.bytes);
                        else copy(stage + at, there, k.bytes);
                    }
                }
            }
    if (e == hipSuccess) e = hipStreamSynchronize(st);
    (void)hipFree(stage);
    if (rc) return rc;
    XFT_CHECK_HIP(e);
    return 0;
}

void plan_state_destroy(PlanState *p) {
    for (void *b : p->owned) (void)hipFree(b);
    if (p->trace_buf) (void)hipFree(p->trace_buf);
    if (p->desc_host) (void)hipHostFree(p->desc_host);
    if (p->logits_pinned) (void)hipHostFree(p->logits_pinned);
    delete p;
}

} // namespace xfthip

using namespace xfthip;

extern "C" {

int xfthip_plan_create(const xfthip_plan_config *cfg, const xfthip_plan_layer *layers, xfthip_plan_t *out) {
    XFT_REQUIRE(cfg && layers && out, "xfthip_plan_create: null argument");
    const xfthip_plan_config &c = *cfg;
    XFT_REQUIRE(c.layers > 0 && c.hidden > 0 && c.hidden <= 16384 && c.vocab > 0, "xfthip_plan_create: bad sizes");
    const bool loop = c.loop_times > 1 && c.loop_start != c.loop_stop; // (a loop over nothing is none)
    XFT_REQUIRE((c.block == XFTHIP_BLOCK_SANDWICH && (c.norm == XFTHIP_NORM_RMS_ABOUT_ONE || c.norm == XFTHIP_NORM_RMS) && c.side_dim == 0)
                    || (c.block == XFTHIP_BLOCK_PARALLEL && c.norm == XFTHIP_NORM_DYNAMIC_TANH && c.side_dim >= 0)
                    || (c.block == XFTHIP_BLOCK_SERIAL && c.norm == XFTHIP_NORM_RMS && c.side_dim == 0 && !loop),
            "xfthip_plan_create: block arrangement %d with norm %d and side width %d is not served", c.block, c.norm, c.side_dim);
    XFT_REQUIRE(!loop || (c.loop_start >= 0 && c.loop_start < c.loop_stop && c.loop_stop <= c.layers), "xfthip_plan_create: loop over layers %d .. %d of %d",
            c.loop_start, c.loop_stop, c.layers);
    XFT_REQUIRE(c.bigram_buckets >= 0 && c.bigram_buckets < (1ll << 31) - 1 && (c.embed_scale == 0.0f || c.embed_scale == 1.0f || !loop) && c.logit_softcap >= 0.0f,
            "xfthip_plan_create: bad embedding or logit constants");
    XFT_REQUIRE(c.norm_groups >= 0 && (c.norm_groups <= 1 || (c.norm == XFTHIP_NORM_RMS && c.hidden % c.norm_groups == 0 && !loop)),
            "xfthip_plan_create: %d groups of a norm over %d values", c.norm_groups, c.hidden);
    xfthip_plan *p = new xfthip_plan();
    p->cfg = c;
    if (c.embed_scale == 0.0f) p->cfg.embed_scale = 1.0f;
    if (c.norm_groups == 0) p->cfg.norm_groups = 1;
    p->hidden = pad32(c.hidden);
    p->side_pad = pad32(c.side_dim);
    int first_mix = -1; // the first layer with mixed values
    for (int i = 0; i < c.layers; ++i) {
        PlanLayer L;
        L.s = layers[i];
        const xfthip_plan_layer &s = L.s;
        bool ok = s.heads > 0 && s.dim > 0 && s.vdim > 0 && s.inter >= 0;
        if (s.mixer == XFTHIP_MIXER_LATENT) {
            ok = ok && s.rot_dim > 0 && s.rot_dim % 2 == 0 && s.kv_rank > 0 && s.kv_rank <= 1024 && s.q_rank > 0 && s.window >= 0;
            L.D = pad32(s.dim), L.RD = pad32(s.rot_dim), L.V = pad32(s.vdim), L.R = pad32(s.kv_rank), L.QR = pad32(s.q_rank);
        } else if (s.mixer == XFTHIP_MIXER_DELTA) {
            ok = ok && s.kv_heads > 0 && s.heads % s.kv_heads == 0 && s.dim <= 256 && s.taps >= 1 && s.decay_rank >= 0 && s.gate_rank >= 0
                    && (s.decay_rank > 0) == (s.gate_rank > 0);
            L.KD = 32;
            while (L.KD < s.dim) L.KD *= 2;
            L.VD = pad32(s.vdim);
            L.rank = pad32(std::max(s.decay_rank, s.gate_rank));
            if (L.rank > 0) L.gcols = s.heads * std::max(L.KD, L.VD);
        } else if (s.mixer == XFTHIP_MIXER_GROUPED) {
            ok = ok && s.kv_heads > 0 && s.heads % s.kv_heads == 0 && s.dim <= 512 && s.vdim <= 512 && s.rot_dim >= 0 && s.rot_dim <= s.dim && s.rot_dim % 2 == 0
                    && s.window >= 0 && s.chunk >= 0 && !(s.window > 0 && s.chunk > 0) && s.softcap >= 0.0f && s.qk_norm >= 0 && s.qk_norm <= XFTHIP_QK_NORM_UNIT
                    && s.out_gate >= 0 && s.out_gate <= XFTHIP_GATE_HEAD && (!s.key_values || (s.dim == s.vdim && !s.v_mix)) && (s.rot_factor <= 0.0 || (s.rot_original > 0.0 && s.rot_fast > 0.0 && s.rot_slow > 0.0));
            ok = ok && s.taps >= 0 && (s.taps == 0 || (s.qk_norm != XFTHIP_QK_NORM_ALL && !s.v_mix && !s.key_values && s.kv_from == 0))
                    && s.keep_first >= 0 && s.pool >= 0 && ((s.keep_first == 0 && s.pool == 0) || s.window > 0) && !(s.keep_first > 0 && s.pool > 0) && !(s.pool > 0 && s.distance_bias)
                    && !(s.pool > 0 && s.kv_from != 0) && (!s.v_rot || (s.vdim % 2 == 0 && s.rot_base > 0.0 && !s.key_values && !s.v_mix && s.kv_from == 0));
            L.D = pad32(s.dim), L.V = pad32(s.vdim);
            if (ok && s.v_mix) {
                L.first_values = first_mix < 0;
                if (first_mix < 0) first_mix = i;
                const xfthip_plan_layer &f = layers[first_mix];
                ok = f.kv_heads == s.kv_heads && f.vdim == s.vdim; // values of the same shape
            }
            if (ok && s.kv_from != 0) { // a record before this one with keys and values of its own and of the same shape
                ok = s.kv_from > 0 && s.kv_from <= i && !loop && !s.v_mix;
                const xfthip_plan_layer &f = layers[ok ? s.kv_from - 1 : 0];
                ok = ok && f.mixer == XFTHIP_MIXER_GROUPED && f.kv_from == 0 && f.kv_heads == s.kv_heads && f.dim == s.dim && f.vdim == s.vdim && !f.v_rot;
                const bool moved = s.rot_dim > 0 && !s.rot_interleaved, f_moved = f.rot_dim > 0 && !f.rot_interleaved; // (and the same order of dimensions)
                ok = ok && moved == f_moved && (!moved || s.rot_dim == f.rot_dim);
                if (ok) L.kv_from = s.kv_from - 1;
            }
        } else if (s.mixer == XFTHIP_MIXER_UNIT) {
            ok = ok && s.taps >= 1;
            L.D = pad32(s.dim);
        } else if (s.mixer == XFTHIP_MIXER_LINEAR) {
            ok = ok && s.dim <= 256 && s.taps <= 1 && s.decay_rank > 0 && s.gate_rank == 0 && s.tau > 0.0f;
            L.KD = 32;
            while (L.KD < s.dim) L.KD *= 2;
            L.VD = pad32(s.vdim), L.rank = pad32(s.decay_rank);
        } else {
            ok = false;
        }
        ok = ok && (!s.o_bias || (s.mixer == XFTHIP_MIXER_GROUPED && (!s.beside || s.result_norm))) && (!s.mlp_bias || (s.inter > 0 && s.experts == 0 && s.glu_alpha == 0.0f))
                && (!s.result_norm || c.block != XFTHIP_BLOCK_PARALLEL);
        L.ff = pad32(s.inter);
        if (s.experts > 0) {
            ok = ok && s.identity >= 0 && s.top > 0 && s.top <= L.routes() && s.top <= 64 && L.routes() <= 1024 && s.expert_inter > 0 && s.glu_alpha >= 0.0f;
            if (ok && s.router == XFTHIP_ROUTE_SIGMOID_GROUPS)
                ok = s.identity == 0 && s.route_groups > 0 && s.experts % s.route_groups == 0 && s.route_keep > 0 && s.route_keep <= s.route_groups
                        && s.top <= s.route_keep * (s.experts / s.route_groups);
            else ok = ok && s.router == XFTHIP_ROUTE_SOFTMAX;
            L.eff = pad32(s.expert_inter);
        }
        if (s.scaled && !s.result_norm) L.mix_scale = s.mix_scale;
        L.in_ld = L.row_in(), L.out_ld = L.out_cols();
        if (s.beside) { // joins the layer before it, whose projections it continues
            ok = ok && i > 0 && !loop && !layers[i - 1].beside && layers[i - 1].mixer != XFTHIP_MIXER_LATENT && s.mixer != XFTHIP_MIXER_LATENT && s.inter == 0
                    && s.experts == 0 && !s.result_norm == !layers[i - 1].result_norm && (s.result_norm || !layers[i - 1].o_bias);
            if (ok) {
                PlanLayer &f = p->layers[i - 1];
                f.beside = i;
                L.in_col = f.in_ld, L.out_col = f.out_ld;
                f.in_ld = L.in_ld += f.in_ld, f.out_ld = L.out_ld += f.out_ld;
            }
        }
        if (s.result_norm && !s.beside) ok = ok && i + 1 < c.layers && layers[i + 1].beside;
        if (!ok) {
            delete p;
            XFT_REQUIRE(false, "xfthip_plan_create: layer %d has sizes this library does not serve", i);
        }
        p->layers.push_back(L);
    }
    auto add = [&](int from, int to, bool again) {
        for (int i = from; i < to; ++i)
            if (!p->layers[i].s.beside) p->runs.push_back({i, again && i == from, p->layers[i].beside});
    };
    add(0, loop ? c.loop_start : c.layers, false);
    if (loop) {
        for (int t = 0; t < c.loop_times; ++t) add(c.loop_start, c.loop_stop, t > 0);
        add(c.loop_stop, c.layers, false);
    }
    int stores = (int)p->runs.size();
    for (LayerRun &r : p->runs)
        if (r.beside >= 0) r.beside_store = stores++;
    *out = p;
    return 0;
}

int xfthip_plan_destroy(xfthip_plan_t p) {
    if (!p) return 0;
    for (PlanLayer &L : p->layers) {
        for (xfthip_weight_t w : {L.in, L.o, L.gateup, L.down, L.uq, L.absorb, L.uk, L.uv, L.gates, L.router, L.side_gate, L.side_proj}) xfthip_weight_destroy(w);
        for (auto *list : {&L.egateup, &L.edown})
            for (xfthip_weight_t w : *list) xfthip_weight_destroy(w);
        for (float *f : {L.q_norm, L.kv_norm, L.sink, L.conv, L.decay, L.dt_bias, L.out_norm, L.pre1.w, L.pre1.b, L.pre2.w, L.pre2.b, L.post1, L.post2, L.correction,
                     L.side_post, L.in_bias, L.conv_bias, L.lambda, L.gate_bias, L.o_bias, L.gateup_bias, L.down_bias, L.result_norm})
            if (f) (void)hipFree(f);
        if (L.filter) (void)hipFree(L.filter);
        if (L.etable) (void)hipFree(L.etable);
    }
    xfthip_weight_destroy(p->head);
    if (p->embedding) (void)hipFree(p->embedding);
    for (void *b : {(void *)p->final_norm.w, (void *)p->final_norm.b, (void *)p->side_embedding, (void *)p->pair_embedding})
        if (b) (void)hipFree(b);
    delete p;
    return 0;
}

int xfthip_plan_set_tensor(xfthip_plan_t p, int layer, const char *name, const uint16_t *data_host, int rows, int cols) {
    XFT_REQUIRE(p && name && data_host && rows > 0 && cols > 0, "xfthip_plan_set_tensor: bad argument");
    XFT_REQUIRE(!p->finished, "xfthip_plan_set_tensor: the plan is finished");
    XFT_REQUIRE(layer >= -1 && layer < p->cfg.layers, "xfthip_plan_set_tensor: layer %d out of range", layer);
    Tensor t;
    t.rows = rows, t.cols = cols;
    t.data.assign(data_host, data_host + (size_t)rows * cols);
    p->pending.emplace_back((layer < 0 ? std::string() : std::to_string(layer) + "/") + name, std::move(t));
    return 0;
}

int xfthip_plan_finish(xfthip_plan_t p) {
    XFT_REQUIRE(p && !p->finished, "xfthip_plan_finish: bad plan");
    std::map<std::string, Tensor> all;
    for (auto &kv : p->pending) all[kv.first] = std::move(kv.second);
    p->pending.clear();
    std::string prefix, missing;
    static const Tensor empty;
    auto get = [&](const char *name, int rows, int cols) -> const Tensor & {
        auto it = all.find(prefix + name);
        if (it == all.end() || it->second.rows != rows || it->second.cols != cols) {
            if (missing.empty()) {
                missing = prefix + name + ": ";
                missing += it == all.end() ? std::string("missing")
                                           : "[" + std::to_string(it->second.rows) + ", " + std::to_string(it->second.cols) + "] instead of ["
                                + std::to_string(rows) + ", " + std::to_string(cols) + "]";
            }
            return empty;
        }
        return it->second;
    };
    int rc = 0;
    auto upload = [&](const std::vector<float> &v, float **dst) {
        if (rc) return;
        if (hipMalloc((void **)dst, v.size() * 4 + 16) != hipSuccess || hipMemcpy(*dst, v.data(), v.size() * 4, hipMemcpyHostToDevice) != hipSuccess) {
            set_error("xfthip_plan_finish: upload failed");
            rc = 1;
        }
    };
    auto pack = [&](const Matrix &w, int flags, xfthip_weight_t *dst) {
        if (rc) return;
        rc = xfthip_weight_create(XFTHIP_W_BF16, w.K, w.N, w.w.data(), nullptr, nullptr, flags, dst);
        if (rc == 0) p->weight_bytes += xfthip_weight_bytes(*dst);
    };
    auto values = [&](const Tensor &t, int n) {
        std::vector<float> v(n, 0.0f);
        for (int i = 0; i < t.rows * t.cols && i < n; ++i) v[i] = bf16_value(t.data[i]);
        return v;
    };
    const int W = p->cfg.hidden, Wp = p->hidden, V = p->cfg.vocab;
    // rows x (parts * width) bf16 -> device, every part padded to `pad` columns
    auto upload_embedding = [&](const Tensor &t, int parts, int width, int pad, uint16_t **dst) {
        if (rc) return;
        std::vector<uint16_t> table((size_t)t.rows * parts * pad, 0);
        for (int v = 0; v < t.rows; ++v)
            for (int k = 0; k < parts; ++k) memcpy(&table[((size_t)v * parts + k) * pad], &t.data[((size_t)v * parts + k) * width], (size_t)width * 2);
        if (hipMalloc((void **)dst, table.size() * 2 + 16) != hipSuccess || hipMemcpy(*dst, table.data(), table.size() * 2, hipMemcpyHostToDevice) != hipSuccess) {
            set_error("xfthip_plan_finish: upload failed");
            rc = 1;
        }
    };
    auto upload_bits = [&](const std::vector<uint16_t> &v, uint16_t **dst) {
        if (rc) return;
        if (hipMalloc((void **)dst, v.size() * 2 + 16) != hipSuccess || hipMemcpy(*dst, v.data(), v.size() * 2, hipMemcpyHostToDevice) != hipSuccess) {
            set_error("xfthip_plan_finish: upload failed");
            rc = 1;
        }
    };
    auto one_plus = [&](const Tensor &t, const Tensor *scale) {
        std::vector<float> v(Wp, 0.0f);
        for (int i = 0; i < t.rows; ++i) v[i] = (1.0f + bf16_value(t.data[i])) * (scale ? bf16_value(scale->data[i]) : 1.0f);
        return v;
    };
#define NEED(var, name, r, c)                 \
    const Tensor &var = get(name, r, c);      \
    if (!missing.empty()) break
    const bool tanh_norm = p->cfg.norm == XFTHIP_NORM_DYNAMIC_TANH, sandwich = p->cfg.block == XFTHIP_BLOCK_SANDWICH;
    // a norm in front of something; mul multiplies its result
    auto front = [&](const std::string &name, float mul, PlanNorm *dst) {
        const Tensor &w = get(name.c_str(), W, 1);
        if (!missing.empty()) return;
        if (!tanh_norm) {
            std::vector<float> v = p->cfg.norm == XFTHIP_NORM_RMS ? values(w, Wp) : one_plus(w, nullptr);
            for (float &f : v) f *= mul;
            upload(v, &dst->w);
            return;
        }
        const Tensor &alpha = get((name + ".alpha").c_str(), 1, 1), &b = get((name + ".b").c_str(), W, 1);
        if (!missing.empty()) return;
        std::vector<float> vw = values(w, Wp), vb = values(b, Wp);
        for (float &f : vw) f *= mul;
        for (float &f : vb) f *= mul;
        upload(vw, &dst->w), upload(vb, &dst->b);
        dst->alpha = bf16_value(alpha.data[0]);
    };
    auto gate_up = [&](const Tensor &gate, const Tensor &up, int ff, int pad, xfthip_weight_t *dst) {
        Matrix gu(Wp, 2 * pad);
        gu.place(gate, 0, ff, 0, W, 0, 0);
        gu.place(up, 0, ff, 0, W, 0, pad);
        pack(gu, XFTHIP_WF_GATEUP, dst);
    };
    // [rows, cols] tensor -> weight of `k` inputs and `n` outputs
    auto plain = [&](const Tensor &t, int k, int n, xfthip_weight_t *dst) {
        Matrix w(k, n);
        w.place(t, 0, t.rows, 0, t.cols, 0, 0);
        pack(w, XFTHIP_WF_NONE, dst);
    };
    // a mixer's part of the layer's two products, and its own tensors
    auto mixer = [&](PlanLayer &L, Matrix &in, Matrix &mo, std::vector<float> &bias, bool &biased) {
        const xfthip_plan_layer &s = L.s;
        const int H = s.heads, c0 = L.in_col, r0 = L.out_col;
        do {
            if (s.mixer == XFTHIP_MIXER_LATENT) {
                const int d = s.dim, r = s.rot_dim, dv = s.vdim, R = s.kv_rank;
                NEED(dq, "mix.dq", s.q_rank, W);
                NEED(dqn, "mix.dq.norm", s.q_rank, 1);
                NEED(uq, "mix.uq", H * (d + r), s.q_rank);
                NEED(dkv, "mix.dkv", R + r, W);
                NEED(dkvn, "mix.dkv.norm", R, 1);
                NEED(uk, "mix.uk", H * d, R);
                NEED(uv, "mix.uv", H * dv, R);
                NEED(o, "mix.o", W, H * dv);
                in.place(dq, 0, s.q_rank, 0, W, 0, c0);
                in.place(dkv, 0, R, 0, W, 0, c0 + L.QR);
                in.place(dkv, R, r, 0, W, 0, c0 + L.QR + L.R);
                Matrix mq(L.QR, H * (L.D + L.RD)), ma(L.D, H * L.R), mk(L.R, H * L.D), mv(L.R, H * L.V);
                for (int h = 0; h < H; ++h) {
                    mq.place(uq, h * (d + r), d, 0, s.q_rank, 0, h * (L.D + L.RD));
                    mq.place(uq, h * (d + r) + d, r, 0, s.q_rank, 0, h * (L.D + L.RD) + L.D);
                    ma.place_turned(uk, h * d, d, 0, R, 0, h * L.R);
                    mk.place(uk, h * d, d, 0, R, 0, h * L.D);
                    mv.place(uv, h * dv, dv, 0, R, 0, h * L.V);
                    mo.place(o, 0, W, h * dv, dv, r0 + h * L.V, 0);
                }
                pack(mq, XFTHIP_WF_NONE, &L.uq);
                pack(ma, XFTHIP_WF_NONE, &L.absorb);
                pack(mk, XFTHIP_WF_NONE, &L.uk);
                pack(mv, XFTHIP_WF_NONE, &L.uv);
                upload(values(dqn, L.QR), &L.q_norm);
                upload(values(dkvn, L.R), &L.kv_norm);
                if (s.has_sink) {
                    NEED(sink, "mix.sink", H, 1);
                    upload(values(sink, H), &L.sink);
                }
            } else if (s.mixer == XFTHIP_MIXER_GROUPED) {
                const int G = s.kv_heads, d = s.dim, dv = s.vdim, k0 = c0 + H * L.D, v0 = c0 + L.value_col(), g0 = c0 + L.gate_col();
                const bool own = L.kv_from < 0;
                // where the dimensions of a head are kept
                std::vector<int> same, head, value;
                for (int x = 0; x < std::max(d, dv); ++x) same.push_back(x), head.push_back(L.head_place(x)), value.push_back(L.value_place(x));
                std::vector<uint16_t> filter(L.filters() ? (size_t)s.taps * L.channels() : 0, 0);
                // a projection of n heads of width w, each padded to `pad` columns from c on, with its bias and filters
                auto project = [&](const char *name, int n, int w, int pad, int c, const std::vector<int> &place, bool with_bias, bool with_filter) {
                    const Tensor &t = get(name, n * w, W);
                    if (!missing.empty()) return;
                    const bool in_order = std::equal(place.begin(), place.begin() + w, same.begin());
                    for (int h = 0; h < n && in_order; ++h) in.place(t, h * w, w, 0, W, 0, c + h * pad);
                    for (int x = 0; x < n * w && !in_order; ++x) in.place(t, x, 1, 0, W, 0, c + x / w * pad + place[x % w]);
                    if (with_bias) {
                        const Tensor &b = get((std::string(name) + ".b").c_str(), n * w, 1);
                        if (!missing.empty()) return;
                        for (int x = 0; x < n * w; ++x) bias[c + x / w * pad + place[x % w]] = bf16_value(b.data[x]);
                        biased = true;
                    }
                    if (with_filter) {
                        const Tensor &f = get((std::string(name) + ".conv").c_str(), n * w, s.taps);
                        if (!missing.empty()) return;
                        for (int x = 0; x < n * w; ++x)
                            for (int j = 0; j < s.taps; ++j) filter[(size_t)j * L.channels() + c - c0 + x / w * pad + place[x % w]] = f.data[(size_t)x * s.taps + j];
                    }
                };
                project("mix.q", H, d, L.D, c0, head, s.qkv_bias, L.filters());
                if (own) project("mix.k", G, d, L.D, k0, head, s.qkv_bias, L.filters());
                if (own && !s.key_values) project("mix.v", G, dv, L.V, v0, value, s.qkv_bias, L.filters());
                if (s.out_gate == XFTHIP_GATE_ELEMENT) project("mix.g", H, dv, L.V, g0, value, false, false);
                if (s.out_gate == XFTHIP_GATE_HEAD) project("mix.g", H, 1, 1, g0, same, false, false);
                NEED(o, "mix.o", W, H * dv);
                for (int h = 0; h < H; ++h)
                    for (int x = 0; x < dv; ++x) mo.place(o, 0, W, h * dv + x, 1, r0 + h * L.V + value[x], 0);
                auto spread = [&](const Tensor &t, int n) {
                    std::vector<float> v((size_t)n * L.D, 0.0f);
                    for (int x = 0; x < n * d; ++x) v[(size_t)(x / d) * L.D + head[x % d]] = bf16_value(t.data[x]);
                    return v;
                };
                if (L.filters()) upload_bits(filter, &L.filter);
                if (s.o_bias) {
                    NEED(ob, "mix.o.b", W, 1);
                    std::vector<float> v = values(ob, Wp);
                    for (float &f : v) f *= L.mix_scale;
                    upload(v, &L.o_bias);
                }
                if (s.qk_norm == XFTHIP_QK_NORM_HEAD) {
                    NEED(qn, "mix.q.norm", d, 1);
                    NEED(kn, "mix.k.norm", d, 1);
                    upload(spread(qn, 1), &L.q_norm);
                    upload(spread(kn, 1), &L.kv_norm);
                } else if (s.qk_norm == XFTHIP_QK_NORM_ALL) {
                    NEED(qn, "mix.q.norm", H * d, 1);
                    upload(spread(qn, H), &L.q_norm);
                    if (own) {
                        NEED(kn, "mix.k.norm", G * d, 1);
                        upload(spread(kn, G), &L.kv_norm);
                    }
                }
                if (s.has_sink) {
                    NEED(sink, "mix.sink", H, 1);
                    upload(values(sink, H), &L.sink);
                }
                if (s.v_mix && !L.first_values) {
                    NEED(share, "mix.vmix", 1, 1);
                    L.value_share = bf16_value(share.data[0]);
                }
            } else if (s.mixer == XFTHIP_MIXER_UNIT) {
                const int B = s.heads, d = s.dim, n = s.taps, C = B * d, P = B * L.D;
                NEED(y, "mix.y", C, W);
                NEED(yb, "mix.y.b", C, 1);
                NEED(x, "mix.x", C, W);
                NEED(xb, "mix.x.b", C, 1);
                NEED(cv, "mix.conv", C, n);
                NEED(cb, "mix.conv.b", C, 1);
                NEED(ra, "mix.ra", B, d * d);
                NEED(rab, "mix.ra.b", B, d);
                NEED(ri, "mix.ri", B, d * d);
                NEED(rib, "mix.ri.b", B, d);
                NEED(lam, "mix.lam", C, 1);
                NEED(o, "mix.o", W, C);
                std::vector<float> conv((size_t)P * n, 0.0f), conv_bias(P, 0.0f), lambda(P, 0.0f), gate_bias((size_t)2 * P, 0.0f);
                Matrix gt(L.D, 2 * P);
                for (int b = 0; b < B; ++b) {
                    in.place(y, b * d, d, 0, W, 0, c0 + b * L.D);
                    in.place(x, b * d, d, 0, W, 0, c0 + P + b * L.D);
                    mo.place(o, 0, W, b * d, d, r0 + b * L.D, 0);
                    for (int e = 0; e < d; ++e) {
                        const int from = b * d + e, to = b * L.D + e;
                        bias[c0 + to] = bf16_value(yb.data[from]), bias[c0 + P + to] = bf16_value(xb.data[from]);
                        for (int k = 0; k < n; ++k) conv[(size_t)to * n + k] = bf16_value(cv.data[(size_t)from * n + k]);
                        conv_bias[to] = bf16_value(cb.data[from]);
                        const double z = bf16_value(lam.data[from]);
                        lambda[to] = (float)(8.0 * (z > 0.0 ? z + log1p(exp(-z)) : log1p(exp(z))));
                        gate_bias[(size_t)2 * b * L.D + e] = bf16_value(rab.data[from]), gate_bias[(size_t)(2 * b + 1) * L.D + e] = bf16_value(rib.data[from]);
                        for (int k = 0; k < d; ++k) { // (square matrices [out, in])
                            gt.w[(size_t)k * gt.N + 2 * b * L.D + e] = ra.data[((size_t)b * d + e) * d + k];
                            gt.w[(size_t)k * gt.N + (2 * b + 1) * L.D + e] = ri.data[((size_t)b * d + e) * d + k];
                        }
                    }
                }
                biased = true;
                pack(gt, XFTHIP_WF_NONE, &L.gates);
                upload(conv, &L.conv), upload(conv_bias, &L.conv_bias), upload(lambda, &L.lambda), upload(gate_bias, &L.gate_bias);
            } else if (s.mixer == XFTHIP_MIXER_LINEAR) {
                const int d = s.dim, dv = s.vdim, k0 = H * L.KD, v0 = 2 * H * L.KD, a0 = c0 + L.channels(), g0 = a0 + L.rank;
                NEED(q, "mix.q", H * d, W);
                NEED(k, "mix.k", H * d, W);
                NEED(v, "mix.v", H * dv, W);
                NEED(g, "mix.g", H * dv, W);
                NEED(a1, "mix.a1", s.decay_rank, W);
                NEED(a2, "mix.a2", H * d, s.decay_rank);
                NEED(ab, "mix.a2.b", H * d, 1);
                NEED(nm, "mix.norm", dv, 1);
                NEED(o, "mix.o", W, H * dv);
                std::vector<float> ab_values((size_t)H * L.KD, 0.0f);
                Matrix gt(L.rank, H * L.KD);
                for (int h = 0; h < H; ++h) {
                    in.place(q, h * d, d, 0, W, 0, c0 + h * L.KD);
                    in.place(k, h * d, d, 0, W, 0, c0 + k0 + h * L.KD);
                    in.place(v, h * dv, dv, 0, W, 0, c0 + v0 + h * L.VD);
                    in.place(g, h * dv, dv, 0, W, 0, g0 + h * L.VD);
                    mo.place(o, 0, W, h * dv, dv, r0 + h * L.VD, 0);
                    gt.place(a2, h * d, d, 0, s.decay_rank, 0, h * L.KD);
                    for (int e = 0; e < d; ++e) ab_values[(size_t)h * L.KD + e] = bf16_value(ab.data[(size_t)h * d + e]);
                }
                in.place(a1, 0, s.decay_rank, 0, W, 0, a0);
                pack(gt, XFTHIP_WF_NONE, &L.gates);
                upload(ab_values, &L.dt_bias);
                upload(values(nm, L.VD), &L.out_norm);
            } else {
                const int KH = s.kv_heads, d = s.dim, dv = s.vdim, n = s.taps;
                NEED(q, "mix.q", KH * d, W);
                NEED(k, "mix.k", KH * d, W);
                NEED(v, "mix.v", H * dv, W);
                NEED(qc, "mix.q.conv", KH * d, n);
                NEED(kc, "mix.k.conv", KH * d, n);
                NEED(vc, "mix.v.conv", H * dv, n);
                NEED(b, "mix.b", H, W);
                NEED(al, "mix.A_log", H, 1);
                NEED(nm, "mix.norm", dv, 1);
                NEED(o, "mix.o", W, H * dv);
                std::vector<float> conv((size_t)L.channels() * n, 0.0f), dec(H);
                const int k0 = KH * L.KD, v0 = 2 * KH * L.KD, b0 = c0 + L.channels(), a0 = b0 + L.beta_cols(), g0 = a0 + (L.head_decay() ? L.beta_cols() : L.rank);
                auto filters = [&](const Tensor &t, int from, int count, int to) {
                    for (int i2 = 0; i2 < count * n; ++i2) conv[(size_t)to * n + i2] = bf16_value(t.data[(size_t)from * n + i2]);
                };
                for (int h = 0; h < KH; ++h) {
                    in.place(q, h * d, d, 0, W, 0, c0 + h * L.KD);
                    in.place(k, h * d, d, 0, W, 0, c0 + k0 + h * L.KD);
                    filters(qc, h * d, d, h * L.KD);
                    filters(kc, h * d, d, k0 + h * L.KD);
                }
                for (int h = 0; h < H; ++h) {
                    in.place(v, h * dv, dv, 0, W, 0, c0 + v0 + h * L.VD);
                    filters(vc, h * dv, dv, v0 + h * L.VD);
                    mo.place(o, 0, W, h * dv, dv, r0 + h * L.VD, 0);
                    dec[h] = expf(bf16_value(al.data[h]));
                }
                in.place(b, 0, H, 0, W, 0, b0);
                if (L.head_decay()) {
                    NEED(ad, "mix.a", H, W);
                    NEED(dt, "mix.dt_bias", H, 1);
                    NEED(g, "mix.g", H * dv, W);
                    in.place(ad, 0, H, 0, W, 0, a0);
                    for (int h = 0; h < H; ++h) in.place(g, h * dv, dv, 0, W, 0, g0 + h * L.VD);
                    upload(values(dt, H), &L.dt_bias);
                } else {
                    NEED(a1, "mix.a1", s.decay_rank, W);
                    NEED(a2, "mix.a2", H * d, s.decay_rank);
                    NEED(dt, "mix.dt_bias", H * d, 1);
                    NEED(g1, "mix.g1", s.gate_rank, W);
                    NEED(g2, "mix.g2", H * dv, s.gate_rank);
                    std::vector<float> dtb((size_t)H * L.KD, 0.0f);
                    Matrix gt(L.rank, 2 * L.gcols);
                    for (int h = 0; h < H; ++h) {
                        gt.place(a2, h * d, d, 0, s.decay_rank, 0, h * L.KD);
                        gt.place(g2, h * dv, dv, 0, s.gate_rank, 0, L.gcols + h * L.VD);
                        for (int e = 0; e < d; ++e) dtb[(size_t)h * L.KD + e] = bf16_value(dt.data[(size_t)h * d + e]);
                    }
                    in.place(a1, 0, s.decay_rank, 0, W, 0, a0);
                    in.place(g1, 0, s.gate_rank, 0, W, 0, g0);
                    pack(gt, XFTHIP_WF_NONE, &L.gates);
                    upload(dtb, &L.dt_bias);
                }
                upload(conv, &L.conv);
                upload(dec, &L.decay);
                upload(values(nm, L.VD), &L.out_norm);
            }
            if (s.result_norm) {
                NEED(rn, "mix.out", W, 1);
                std::vector<float> v = values(rn, Wp);
                for (float &f : v) f *= s.scaled ? s.mix_scale : 1.0f;
                upload(v, &L.result_norm);
            }
        } while (false);
    };
    do {
        NEED(embed, "embed", V, W);
        upload_embedding(embed, 1, W, Wp, &p->embedding);
        front("final.norm", p->cfg.logit_scale, &p->final_norm); // the logits are linear in the normed row
        if (p->cfg.bigram_buckets > 0) {
            NEED(pairs, "bigram", (int)p->cfg.bigram_buckets + 1, W);
            upload_embedding(pairs, 1, W, Wp, &p->pair_embedding);
        }
        if (p->cfg.side_dim > 0) {
            NEED(side, "side.embed", V, p->cfg.layers * p->cfg.side_dim);
            upload_embedding(side, p->cfg.layers, p->cfg.side_dim, p->side_pad, &p->side_embedding);
        }
        NEED(head, p->cfg.tied_head ? "embed" : "head", V, W);
        Matrix hm(Wp, V);
        hm.place(head, 0, V, 0, W, 0, 0);
        pack(hm, XFTHIP_WF_NONE, &p->head);
    } while (false);
    for (int i = 0; i < p->cfg.layers && missing.empty() && rc == 0; ++i) do {
        PlanLayer &L = p->layers[i];
        const xfthip_plan_layer &s = L.s;
        if (s.beside) break; // (with the layer before it)
        prefix = std::to_string(i) + "/";
        front("norm1", 1.0f, &L.pre1);
        if (L.feeds_forward()) front("norm2", 1.0f, &L.pre2);
        if (!missing.empty()) break;
        if (sandwich && p->cfg.norm == XFTHIP_NORM_RMS) { // no further scale
            NEED(n1b, "norm1b", W, 1);
            upload(values(n1b, Wp), &L.post1);
            if (L.feeds_forward()) {
                NEED(n2b, "norm2b", W, 1);
                upload(values(n2b, Wp), &L.post2);
            }
        } else if (sandwich) {
            NEED(n1b, "norm1b", W, 1);
            NEED(ls1, "ls1", W, 1);
            upload(one_plus(n1b, &ls1), &L.post1);
            if (L.feeds_forward()) {
                NEED(n2b, "norm2b", W, 1);
                NEED(ls2, "ls2", W, 1);
                upload(one_plus(n2b, &ls2), &L.post2);
            }
        }
        if (s.inter > 0) {
            const std::string at = s.experts > 0 ? "mlp.shared." : "mlp.";
            NEED(gate, (at + "gate").c_str(), s.inter, W);
            NEED(up, (at + "up").c_str(), s.inter, W);
            NEED(down, (at + "down").c_str(), W, s.inter);
            gate_up(gate, up, s.inter, L.ff, &L.gateup);
            plain(down, L.ff, Wp, &L.down);
            if (s.mlp_bias) {
                NEED(gb, (at + "gate.b").c_str(), s.inter, 1);
                NEED(ub, (at + "up.b").c_str(), s.inter, 1);
                NEED(db, (at + "down.b").c_str(), W, 1);
                std::vector<float> v = values(gb, L.ff), u = values(ub, L.ff);
                v.insert(v.end(), u.begin(), u.end());
                upload(v, &L.gateup_bias), upload(values(db, Wp), &L.down_bias);
            }
        }
        if (s.experts > 0) {
            NEED(router, "mlp.router", L.routes(), W);
            plain(router, Wp, L.routes(), &L.router);
            if (s.router == XFTHIP_ROUTE_SOFTMAX) {
                NEED(correction, "mlp.correction", L.routes(), 1);
                upload(values(correction, L.routes()), &L.correction);
            }
            L.egateup.assign(s.experts, nullptr), L.edown.assign(s.experts, nullptr);
            std::vector<GroupWeight> table(2 * (size_t)s.experts);
            for (int e = 0; e < s.experts && rc == 0; ++e) {
                const std::string at = "mlp.e" + std::to_string(e) + ".";
                NEED(gate, (at + "gate").c_str(), s.expert_inter, W);
                NEED(up, (at + "up").c_str(), s.expert_inter, W);
                NEED(down, (at + "down").c_str(), W, s.expert_inter);
                gate_up(gate, up, s.expert_inter, L.eff, &L.egateup[e]);
                plain(down, L.eff, Wp, &L.edown[e]);
                if (rc) break;
                const PackedWeight &g = L.egateup[e]->pw, &d = L.edown[e]->pw;
                table[e] = {g.packed, g.scale, g.zero}, table[s.experts + e] = {d.packed, d.scale, d.zero};
            }
            if (!missing.empty() || rc) break;
            if (hipMalloc((void **)&L.etable, table.size() * sizeof(GroupWeight)) != hipSuccess
                    || hipMemcpy(L.etable, table.data(), table.size() * sizeof(GroupWeight), hipMemcpyHostToDevice) != hipSuccess) {
                set_error("xfthip_plan_finish: upload failed");
                rc = 1;
                break;
            }
        }
        if (p->cfg.side_dim > 0) {
            NEED(gate, "side.gate", p->cfg.side_dim, W);
            NEED(proj, "side.proj", W, p->cfg.side_dim);
            NEED(norm, "side.norm", W, 1);
            plain(gate, Wp, p->side_pad, &L.side_gate);
            plain(proj, p->side_pad, Wp, &L.side_proj);
            upload(values(norm, Wp), &L.side_post);
        }
        // the mixer, or both: one input product, one output product
        Matrix in(Wp, L.in_ld), mo(L.out_ld, Wp);
        std::vector<float> bias(L.in_ld, 0.0f);
        bool biased = false;
        for (int k = i; k >= 0 && missing.empty() && rc == 0; k = k == i ? L.beside : -1) {
            if (k != i) prefix = std::to_string(k) + "/";
            mixer(p->layers[k], in, mo, bias, biased);
        }
        if (!missing.empty() || rc) break;
        pack(in, XFTHIP_WF_NONE, &L.in);
        if (s.result_norm) { // an output product each: rows of the common one
            for (int k : {i, L.beside}) {
                PlanLayer &own = p->layers[k];
                Matrix part(own.out_cols(), Wp);
                memcpy(part.w.data(), &mo.w[(size_t)own.out_col * Wp], part.w.size() * 2);
                pack(part, XFTHIP_WF_NONE, &own.o);
            }
        } else {
            pack(mo, XFTHIP_WF_NONE, &L.o);
        }
        if (biased) upload(bias, &L.in_bias);
    } while (false);
#undef NEED
    XFT_REQUIRE(missing.empty(), "xfthip_plan_finish: tensor %s", missing.c_str());
    p->finished = rc == 0;
    return rc;
}

size_t xfthip_plan_weight_bytes(xfthip_plan_t p) { return p ? p->weight_bytes : 0; }

int xfthip_model_create_from_plan(xfthip_plan_t plan, int act_dtype, int max_batch, int max_seq, int max_tokens, int pool_tokens, xfthip_model_t *out) {
    XFT_REQUIRE(plan && plan->finished && out, "xfthip_model_create_from_plan: needs a finished plan");
    XFT_REQUIRE(act_dtype == XFTHIP_BF16 || act_dtype == XFTHIP_F32, "xfthip_model_create_from_plan: activations are bf16 or fp32");
    XFT_REQUIRE(max_batch > 0 && max_seq > 0 && max_tokens >= max_batch && pool_tokens >= 0, "xfthip_model_create_from_plan: bad limits");
    xfthip_model *m = new xfthip_model();
    memset(&m->cfg, 0, sizeof(m->cfg));
    m->cfg.layers = plan->cfg.layers, m->cfg.hidden = plan->hidden, m->cfg.vocab = plan->cfg.vocab;
    m->cfg.max_batch = max_batch, m->cfg.max_seq = max_seq, m->cfg.max_tokens = max_tokens, m->cfg.max_pos_embed = max_seq;
    m->cfg.rms_eps = plan->cfg.eps;
    m->final_norm = plan->final_norm.w;
    m->lm_head = plan->head;
    m->row_pos.assign(max_batch, -1);
    PlanState *p = new PlanState();
    m->plan = p;
    p->plan = plan, p->layers = plan->layers, p->act = act_dtype, p->esz = act_dtype == XFTHIP_F32 ? 4 : 2, p->slots = max_batch;
    // a table of tokens, and one for every size of block whose means some layer keeps
    auto add_table = [&](int unit) {
        for (size_t t = 1; t < p->tables.size(); ++t)
            if (p->tables[t].unit == unit) return (int)t;
        PageTable t;
        t.unit = unit, t.at = p->table_host.size();
        t.stride = std::max(t.pages_for(max_seq), 1);
        if (p->tables.empty()) t.pages = pool_tokens > 0 ? (pool_tokens + kPageTokens - 1) / kPageTokens : max_batch * t.stride;
        else t.pages = std::min(p->tables[0].pages / unit + max_batch, max_batch * t.stride); // (every slot may end in a part of a page)
        for (int i = t.pages; i-- > 0;) t.free_pages.push_back(i);
        t.held.resize(max_batch);
        p->table_host.resize(t.at + (size_t)max_batch * t.stride, 0);
        p->tables.push_back(t);
        return (int)p->tables.size() - 1;
    };
    add_table(1);
    for (PlanLayer &L : p->layers)
        if (L.s.mixer == XFTHIP_MIXER_GROUPED && L.s.pool > 0) L.means_table = add_table(L.s.pool);
    p->logit_of_row.resize(max_batch);
    for (int r = 0; r < max_batch; ++r) p->logit_of_row[r] = r;
    p->logit_rows = std::max(max_batch, 64);
    bool ok = true;
    auto alloc = [&](void *dst, size_t bytes, bool clear = false) {
        void *b = nullptr;
        if (!ok) return;
        if (hipMalloc(&b, bytes + 256) != hipSuccess || (clear && hipMemset(b, 0, bytes + 256) != hipSuccess)) {
            ok = false;
            return;
        }
        p->owned.push_back(b);
        memcpy(dst, &b, sizeof(b));
    };
    const size_t T = max_tokens, e = p->esz, hidden = plan->hidden;
    bool normed_results = false;
    size_t a = 0, cq = 0, q = 0, qa = 0, ov = 0, h = 0, gates = 0, dk = 0, dqk = 0, dg = 0, dv = 0, heads = 0, fv = 0, u = 0, carry = 0;
    size_t top = 0, experts = 0, routes = 0, eh = 0, eo = 0;
    for (const PlanLayer &L : p->layers) {
        const size_t H = L.s.heads;
        a = std::max(a, (size_t)L.in_ld), ov = std::max(ov, (size_t)L.out_ld);
        h = std::max(h, (size_t)L.ff);
        normed_results = normed_results || L.s.result_norm;
        if (L.s.experts > 0) {
            const size_t most = std::min(L.s.top, L.s.experts);
            top = std::max(top, (size_t)L.s.top), experts = std::max(experts, (size_t)L.s.experts), routes = std::max(routes, (size_t)pad32(L.routes()));
            eh = std::max(eh, most * L.eff), eo = std::max(eo, most * hidden);
        }
        if (L.s.mixer == XFTHIP_MIXER_GROUPED) {
            q = std::max(q, H * L.D);
            if (L.s.v_mix) fv = std::max(fv, (size_t)L.s.kv_heads * L.V);
        } else if (L.s.mixer == XFTHIP_MIXER_UNIT) {
            gates = std::max(gates, (size_t)2 * L.channels()), u = std::max(u, (size_t)L.channels());
            carry = std::max(carry, unit_carry_floats(L, max_tokens, max_batch));
        } else if (L.s.mixer == XFTHIP_MIXER_LINEAR) {
            gates = std::max(gates, H * L.KD), dv = std::max(dv, H * L.VD);
        } else if (L.s.mixer == XFTHIP_MIXER_LATENT) {
            cq = std::max(cq, (size_t)L.QR), q = std::max(q, H * (L.D + L.RD)), qa = std::max(qa, H * L.R);
        } else {
            const size_t KH = L.s.kv_heads;
            gates = std::max(gates, (size_t)2 * L.gcols), dk = std::max(dk, KH * L.KD), dqk = std::max(dqk, KH), dg = std::max(dg, L.head_decay() ? H : H * L.KD);
            dv = std::max(dv, H * L.VD), heads = std::max(heads, H);
        }
    }
    alloc(&p->xn, std::max(T, (size_t)p->logit_rows) * hidden * e);
    alloc(&p->y, T * hidden * 4);
    if (normed_results) alloc(&p->y2, T * hidden * 4);
    alloc(&p->a, T * a * e), alloc(&p->cq, T * cq * e), alloc(&p->q, T * q * e), alloc(&p->qa, T * qa * e), alloc(&p->oc, T * qa * e);
    alloc(&p->ov, T * ov * e), alloc(&p->h, T * h * e), alloc(&p->u, T * u * e);
    alloc(&p->carry, carry * 4), alloc(&p->last_token, (size_t)max_batch * 4, true);
    alloc(&p->gates, T * gates * 4), alloc(&p->dq, T * dk * 4), alloc(&p->dk, T * dk * 4), alloc(&p->dqk, T * dqk * 4), alloc(&p->dg, T * dg * 4);
    alloc(&p->dv, T * dv * 4), alloc(&p->dbeta, T * heads * 4), alloc(&p->do_, T * dv * 4);
    if (plan->cfg.block == XFTHIP_BLOCK_PARALLEL) alloc(&p->xn2, T * hidden * e), alloc(&p->narrow, T * hidden * e);
    alloc(&p->first_values, T * fv * e), alloc(&p->side, T * plan->side_pad * e), alloc(&p->side_z, T * plan->side_pad * 4);
    alloc(&p->router_logits, T * routes * 4), alloc(&p->eh, T * eh * e), alloc(&p->expert_out, T * eo * 4);
    alloc(&p->route.sel, T * top * 4), alloc(&p->route.weight, T * top * 4), alloc(&p->route.slot_row, T * top * 4), alloc(&p->route.row_token, T * top * 4);
    alloc(&p->route.group_rows, experts * 12);
    // the expanded form's context (whole blocks of 32 tokens; cleared: rows behind the end meet zero weights)
    if (act_dtype == XFTHIP_BF16 && max_tokens >= 32) {
        const size_t ctx = pad32(max_seq) + 32;
        size_t kx = 0, vx = 0, rl = 0;
        for (const PlanLayer &L : p->layers)
            if (L.s.mixer == XFTHIP_MIXER_LATENT && latent_expanded_takes(act_dtype, L, 1 << 20, 1 << 20))
                kx = std::max(kx, (size_t)L.s.heads * L.D), vx = std::max(vx, (size_t)L.s.heads * L.V), rl = std::max(rl, (size_t)(L.R + L.RD));
        if (kx) alloc(&p->rows, ctx * rl * e, true), alloc(&p->kx, ctx * kx * e, true), alloc(&p->vx, ctx * vx * e, true);
    }
    for (const PlanLayer &L : p->layers) {
        if (L.s.mixer == XFTHIP_MIXER_LATENT) p->part_floats = std::max(p->part_floats, latent_part_floats(L));
        if (L.s.mixer == XFTHIP_MIXER_GROUPED) p->part_floats = std::max(p->part_floats, grouped_part_floats(L));
    }
    alloc(&p->part, p->part_floats * 4);
    for (const LayerRun &r : plan->runs) p->store_layer.push_back(r.layer);
    for (const LayerRun &r : plan->runs)
        if (r.beside >= 0) p->store_layer.push_back(r.beside);
    for (size_t k = 0; k < p->store_layer.size(); ++k) {
        const PlanLayer &L = p->layers[p->store_layer[k]];
        void *pool = nullptr, *means = nullptr;
        float *state = nullptr;
        void *conv = nullptr;
        int from = (int)k;
        if (L.kv_from >= 0) {
            for (from = 0; p->store_layer[from] != L.kv_from;) ++from;
        } else {
            // cleared: keys that lie behind a sequence's end are multiplied by zero weights and must be numbers
            const size_t page = kPageTokens * L.token_elems() * e;
            if (L.paged()) alloc(&pool, p->tables[0].pages * page, true);
            if (L.means_table) alloc(&means, p->tables[L.means_table].pages * page, true);
            if (L.state_floats()) alloc(&state, (size_t)max_batch * L.state_floats() * 4, true);
            if (L.history()) alloc(&conv, max_batch * L.history() * e, true);
        }
        p->reads.push_back(from), p->cache.push_back(pool), p->state.push_back(state), p->conv_state.push_back(conv), p->means.push_back(means);
    }
    alloc(&p->table, p->table_host.size() * 4, true);
    alloc(&p->desc, (3 * T + 4 * (size_t)max_batch) * 4, true);
    alloc(&p->dec_rows, (size_t)max_batch * 4, true);
    alloc(&p->want, (size_t)p->logit_rows * 4, true);
    std::map<std::vector<double>, std::pair<float *, float *>> rot; // layers of the same rotation share its tables
    auto tables_of = [&](const xfthip_plan_layer &s, float **cosT, float **sinT) {
        const bool extended = s.rot_factor > 0.0;
        auto &t = rot[{s.rot_base, (double)s.rot_dim, extended ? s.rot_factor : 0.0, extended ? s.rot_original : 0.0, extended ? s.rot_fast : 0.0,
                extended ? s.rot_slow : 0.0}];
        if (!t.first) {
            ok = rotation_tables(s, max_seq, &t.first, &t.second) == 0;
            if (t.first) p->owned.push_back(t.first);
            if (t.second) p->owned.push_back(t.second);
        }
        *cosT = t.first, *sinT = t.second;
    };
    for (PlanLayer &L : p->layers) {
        if (!L.paged() || L.s.rot_dim == 0 || !ok) continue;
        tables_of(L.s, &L.cosT, &L.sinT);
    }
    for (PlanLayer &L : p->layers) {
        if (L.s.mixer != XFTHIP_MIXER_GROUPED || !L.s.v_rot || !ok) continue;
        xfthip_plan_layer values = L.s;
        values.rot_dim = L.s.vdim, values.rot_factor = 0.0;
        tables_of(values, &L.cosV, &L.sinV);
    }
    ok = ok && hipHostMalloc((void **)&p->desc_host, (3 * T + 5 * (size_t)max_batch + p->logit_rows + p->table_host.size()) * 4) == hipSuccess
            && hipHostMalloc((void **)&p->logits_pinned, (size_t)p->logit_rows * plan->cfg.vocab * 4) == hipSuccess;
    p->dec_host = p->desc_host + 3 * T + 4 * (size_t)max_batch;
    p->want_host = p->dec_host + max_batch;
    p->table_pinned = p->want_host + p->logit_rows;
    p->tok_seg = p->desc, p->tok_pos = p->desc + T, p->ids = p->desc + 2 * T, p->seg = p->desc + 3 * T;
    const size_t nids = T > 64 ? T : 64;
    m->idlog_cap = max_seq + 1;
    ok = ok && hipMalloc((void **)&m->x, T * hidden * 4) == hipSuccess && hipMalloc((void **)&m->ids, nids * 4) == hipSuccess
            && hipMemset(m->ids, 0, nids * 4) == hipSuccess && hipMalloc((void **)&m->pos, (size_t)max_batch * 4) == hipSuccess
            && hipMemset(m->pos, 0, (size_t)max_batch * 4) == hipSuccess && hipMalloc((void **)&m->step, 64) == hipSuccess
            && hipMemset(m->step, 0, 64) == hipSuccess
            && hipMalloc((void **)&m->logits, (size_t)p->logit_rows * plan->cfg.vocab * 4) == hipSuccess
            && hipMalloc((void **)&m->idlog, (size_t)m->idlog_cap * max_batch * 4) == hipSuccess;
    if (!ok) {
        set_error("xfthip_model_create_from_plan: out of device memory");
        xfthip_model_destroy(m);
        return 1;
    }
    *out = m;
    return 0;
}

int xfthip_model_trace_residual(xfthip_model_t m, int enable) {
    XFT_REQUIRE(m && m->plan, "xfthip_model_trace_residual: only for models from a plan");
    m->plan->trace = enable != 0;
    m->plan->trace_tokens = 0;
    return 0;
}

int xfthip_model_read_residual(xfthip_model_t m, float *out_host, int *runs, int *tokens) {
    XFT_REQUIRE(m && m->plan, "xfthip_model_read_residual: only for models from a plan");
    const PlanState &p = *m->plan;
    const int n = (int)p.plan->runs.size(), T = p.trace_tokens, W = p.plan->cfg.hidden, Wp = p.plan->hidden;
    if (runs) *runs = n;
    if (tokens) *tokens = T;
    if (!out_host) return 0;
    XFT_REQUIRE(T > 0, "xfthip_model_read_residual: nothing traced yet");
    XFT_CHECK_HIP(hipDeviceSynchronize());
    XFT_CHECK_HIP(hipMemcpy2D(out_host, (size_t)W * 4, p.trace_buf, (size_t)Wp * 4, (size_t)W * 4, (size_t)n * T, hipMemcpyDeviceToHost));
    return 0;
}

int xfthip_model_pool_pages(xfthip_model_t m, int *free_pages, int *total_pages) {
    XFT_REQUIRE(m && m->plan, "xfthip_model_pool_pages: only for models from a plan");
    if (free_pages) *free_pages = (int)m->plan->tables[0].free_pages.size();
    if (total_pages) *total_pages = m->plan->tables[0].pages;
    return 0;
}

} // extern "C"
