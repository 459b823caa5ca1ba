// Layer plans: decoder stacks whose layers differ in kind (latent attention, grouped attention, delta-rule recurrence, gated
// linear recurrence, gated linear attention), whose keys live in a page pool shared by all sequences and whose recurrent layers keep a state per sequence
// slot.  Declarations shared by the plan's driver (plan_model.hip) and its kernels (plan_layers.hip, latent_attention.hip,
// grouped_attention.hip, delta_rule.hip, gated_unit.hip, linear_attention.hip, routed_experts.hip, tile_gemm.hip).
//
// Every inner width is padded to whole 32-value groups (the state's key dimension to a power of two) by zero rows and
// columns of the packed weights, so that the kernels see whole MFMA steps whatever sizes a model has.
#pragma once
#include <string>
#include <vector>

#include "common.h"
#include "qgemm.h"

namespace xfthip {

constexpr int kPageTokens = 64; // tokens of a page of the cache

// One step: B segments (one a sequence), T tokens, back to back.  All pointers are device memory.
struct StepView {
    int B, T;
    int longest; // tokens of the longest segment
    const int *tok_seg, *tok_pos; // [T] segment and position of a token
    const int *seg_row, *seg_off, *seg_len, *seg_pos; // [B] slot, first token, tokens, position of the first token
    const int *table; // [slots][table_stride] page numbers
    int table_stride;
};

// what stands in front of a sublayer: an RMS norm with weight w, or, with b set, tanh(alpha x) * w + b
struct PlanNorm {
    float *w = nullptr, *b = nullptr;
    float alpha = 0.0f;
};

struct PlanLayer {
    xfthip_plan_layer s;
    // latent attention: padded widths of a head's unrotated / rotated / value part, of the key and the query latent;
    // grouped attention: D and V, of the query / key and the value part of a head
    int D = 0, RD = 0, V = 0, R = 0, QR = 0;
    // delta rule, linear attention: padded key / value width of a head, padded rank of the gates and columns of one gate; gated unit: D, of
    // a block
    int KD = 0, VD = 0, rank = 0, gcols = 0;
    // Where a mixer finds its projections and puts its result: mixers side by side share the rows of one input product
    // (row_in() columns from in_col on of in_ld) and of one output product (out_cols() from out_col on of out_ld).
    int in_col = 0, in_ld = 0, out_col = 0, out_ld = 0;
    float mix_scale = 1.0f; // of the result
    float *result_norm = nullptr; // weights of the norm of the result (times its scale), or null; then each of a pair has an output product
    int beside = -1; // the record of the mixer next to this one
    int kv_from = -1; // grouped attention: the record whose cache serves
    int ff = 0; // padded
    xfthip_weight_t in = nullptr, o = nullptr, gateup = nullptr, down = nullptr; // (in, o: of both mixers, with the first one)
    float *in_bias = nullptr; // [in_ld] or null
    float *o_bias = nullptr, *gateup_bias = nullptr, *down_bias = nullptr; // [hidden], [2 ff], [hidden] or null
    // latent: queries from their latent; W_uk turned round (query -> latent), W_uk and W_uv (latent -> key / value)
    xfthip_weight_t uq = nullptr, absorb = nullptr, uk = nullptr, uv = nullptr;
    float *q_norm = nullptr, *kv_norm = nullptr, *sink = nullptr; // (grouped attention: weights of the query and the key heads)
    float value_share = 0.0f; // v_mix: lambda
    bool first_values = false; // the layer whose values the others mix in
    float *cosT = nullptr, *sinT = nullptr; // [max positions][rot_dim / 2], shared by layers of the same rotation
    float *cosV = nullptr, *sinV = nullptr; // [max positions][vdim / 2]: of rotated values
    uint16_t *filter = nullptr; // grouped attention: filters [taps][channels], bf16
    int means_table = 0; // grouped attention: the page table of block means, or 0
    // delta rule: both gates' second projections (decay | output gate), filters [channels][taps], exp(A_log), ...
    xfthip_weight_t gates = nullptr;
    float *conv = nullptr, *decay = nullptr, *dt_bias = nullptr, *out_norm = nullptr;
    // gated unit (conv as above, gates: both square products of every block): filter biases, 8 softplus(lambda), biases [blocks][2][D]
    float *conv_bias = nullptr, *lambda = nullptr, *gate_bias = nullptr;
    // routed experts: padded width, weights of one shape by expert and their device table ([experts] gate / up, [experts] down)
    int eff = 0;
    std::vector<xfthip_weight_t> egateup, edown;
    GroupWeight *etable = nullptr;
    xfthip_weight_t router = nullptr;
    float *correction = nullptr;
    // the token's side embedding: into the part's width, back, the norm's weight behind it
    xfthip_weight_t side_gate = nullptr, side_proj = nullptr;
    float *side_post = nullptr;
    // in front of the sublayers (RMS: 1 + w), behind them in sandwich blocks ((1 + w) * layer scale)
    PlanNorm pre1, pre2;
    float *post1 = nullptr, *post2 = nullptr;

    // columns of the input product: latent: query latent | key latent | shared key part; grouped: q | k | v | gate; delta rule: q | k |
    // v | beta | decays | gate; linear attention: q | k | v | decays | gate; gated unit: y | x
    int row_in() const {
        if (s.mixer == XFTHIP_MIXER_LATENT) return QR + R + RD;
        if (s.mixer == XFTHIP_MIXER_GROUPED) return gate_col() + (s.out_gate == XFTHIP_GATE_ELEMENT ? s.heads * V : s.out_gate == XFTHIP_GATE_HEAD ? beta_cols() : 0);
        if (s.mixer == XFTHIP_MIXER_UNIT) return 2 * s.heads * D;
        if (s.mixer == XFTHIP_MIXER_LINEAR) return channels() + rank + s.heads * VD;
        return channels() + beta_cols() + (head_decay() ? beta_cols() : rank) + (silu_gate() ? s.heads * VD : rank);
    }
    int out_cols() const { return s.mixer == XFTHIP_MIXER_UNIT ? s.heads * D : s.heads * (s.mixer == XFTHIP_MIXER_DELTA || s.mixer == XFTHIP_MIXER_LINEAR ? VD : V); }
    // delta rule, linear attention: first column of a gate in the rows
    int out_gate_col() const { return in_col + channels() + (s.mixer == XFTHIP_MIXER_LINEAR ? rank : 2 * beta_cols()); }
    // grouped attention: first columns of values and gate
    int value_col() const { return s.heads * D + (s.key_values ? 0 : s.kv_heads * D); }
    int gate_col() const { return s.heads * D + (kv_from >= 0 ? 0 : s.kv_heads * (D + (s.key_values ? 0 : V))); }
    bool filters() const { return s.mixer == XFTHIP_MIXER_GROUPED && s.taps > 0; }
    bool moves_queries() const { return s.rot_dim > 0 || s.qk_norm || filters(); } // or they stay in the row
    // Grouped attention keeps the two values of a rotated pair side by side, whatever the model's order (the packed weights see to it):
    // where dimension d of a query / key head or of a value head of the model is kept
    int head_place(int d) const { return !s.rot_interleaved && d < s.rot_dim ? beside_partner(d, s.rot_dim / 2) : d; }
    int value_place(int d) const { return s.key_values ? head_place(d) : s.v_rot && !s.rot_interleaved ? beside_partner(d, s.vdim / 2) : d; }
    static int beside_partner(int d, int half) { return d < half ? 2 * d : 2 * (d - half) + 1; }
    bool head_decay() const { return s.decay_rank == 0; }
    bool silu_gate() const { return s.gate_rank == 0; }
    bool paged() const { return s.mixer == XFTHIP_MIXER_LATENT || s.mixer == XFTHIP_MIXER_GROUPED; }
    // elements a token takes in the page pool
    size_t token_elems() const { return s.mixer == XFTHIP_MIXER_LATENT ? R + RD : (size_t)s.kv_heads * (D + V); }
    // floats of a slot's state, channels of the short convolution, elements of a slot's inputs of it
    size_t state_floats() const { return paged() ? 0 : s.mixer == XFTHIP_MIXER_UNIT ? (size_t)s.heads * D : (size_t)s.heads * VD * KD; }
    int channels() const { // (q | k | v; gated unit: x)
        if (s.mixer == XFTHIP_MIXER_UNIT) return s.heads * D;
        if (s.mixer == XFTHIP_MIXER_GROUPED) return s.heads * D + s.kv_heads * (D + V);
        return 2 * (s.mixer == XFTHIP_MIXER_LINEAR ? s.heads : s.kv_heads) * KD + s.heads * VD;
    }
    size_t history() const { return s.mixer != XFTHIP_MIXER_LATENT && s.taps > 1 ? (size_t)(s.taps - 1) * channels() : 0; }
    int routes() const { return s.experts + s.identity; }
    bool feeds_forward() const { return ff > 0 || s.experts > 0; }
    int beta_cols() const { return (s.heads + 31) / 32 * 32; }
};

struct LayerRun {
    int layer;
    bool add_embedding; // the embedding output joins the residual in front of this run
    int beside = -1; // the record of the layer's second mixer, and its place among caches and states
    int beside_store = -1;
};

// ---- kernels -----------------------------------------------------------------------------------------------------
// (act: XFTHIP_BF16 or XFTHIP_F32, the type of activations between kernels; the residual is fp32)

// x = table[id] * scale (bf16 tables, ids clamped to the vocabulary), with a pair table: plus its row of (previous token, token) - the
// row behind the buckets for the first token of a sequence
struct EmbedTables {
    const uint16_t *table, *pairs; // pairs: [buckets + 1][hidden] or null
    int hidden, vocab;
    float scale;
    long long buckets, mul_prev, mul_cur;
};
// the step's tokens; last_token [slots]: of the tokens a slot has seen
int plan_embed(const EmbedTables &e, const StepView &v, const int *ids, const int *last_token, float *x, hipStream_t st);
// logits pass cap * tanh(z / cap)
int plan_softcap(float *logits, size_t n, float cap, hipStream_t st);

// With y2: y = rms(y) * mix1 + rms(y2) * mix2 first, means over the width.  Then
// x += rms(y) * post (y may be null; post null: x += mul * y), then x += table[ids] (table may be null), then xn = pre(x) (pre.w may be null) and
// xn2 = pre2(x) (pre2.w may be null; tanh norms only).  Means over `width` of the `hidden` columns, with groups > 1 over each of so many
// equal parts of them.  rows: xn row i comes from x
// row rows[i] (only without y and table).
struct PlanNormArgs {
    float *x;
    const float *y, *post;
    const uint16_t *table;
    const int *ids;
    int vocab;
    PlanNorm pre, pre2;
    void *xn, *xn2;
    const int *rows;
    int hidden, width;
    float eps;
    float mul;
    int groups = 1;
    const float *y2 = nullptr, *mix1 = nullptr, *mix2 = nullptr;
};
int plan_norm(int act, const PlanNormArgs &p, int T, hipStream_t st);
// out[t][c] = gelu(z[t][c]) * table[ids[t]][first + c] (tanh form of the gelu), c < width; bf16 table [vocab][ld], ids clamped
int plan_side_gate(int act, const float *z, const uint16_t *table, int ld, int first, const int *ids, int vocab, void *out, int T, int width,
        hipStream_t st);

// C[t][n] = sum_k A[t][block(n) * a_block_stride + k] W[k][n], block(n) = n / block_cols: a plain product of 32-bit
// activations (block_cols = 0), or heads side by side.  BF16 weights; act_in / c_dtype XFTHIP_BF16 or XFTHIP_F32.
struct TileGemmArgs {
    int M = 0;
    const void *A = nullptr;
    int lda = 0, block_cols = 0, a_block_stride = 0;
    void *C = nullptr;
    int ldc = 0, c_dtype = XFTHIP_F32;
    bool add = false; // C += (fp32)
    bool glu = false; // the weight holds gate / up pairs (XFTHIP_WF_GATEUP), combined as clamped_glu, or (glu_alpha 0) silu(gate) * up
    float glu_limit = 0, glu_alpha = 0;
    const float *bias = nullptr; // [N], joins the product (glu: of the gates, behind them of the others)
    float decay_tau = 0; // > 0: C = sigmoid(product)^(1 / decay_tau)
    // C = gelu(product) * side[ids[t]][n] (as plan_side_gate)
    const uint16_t *side = nullptr;
    int side_ld = 0;
    const int *side_ids = nullptr;
    int side_vocab = 0;
    // weights of one shape behind one launch, M rows at most each: records {rows, first row of A, first row of C} in device memory;
    // a_rows (or null): row r of A is row a_rows[r]
    const GroupWeight *group = nullptr;
    int group_n = 0;
    const int *group_rows = nullptr, *a_rows = nullptr;
};
int tile_gemm(xfthip_weight_t w, int act_in, const TileGemmArgs &a, hipStream_t st);

// ---- routed experts
struct RouteBuffers {
    int *sel; // [T][top] router output of a choice
    float *weight; // [T][top]
    int *slot_row; // [T][top] row of a choice among the gathered rows; -1: an identity expert
    int *row_token; // [T * top] token of a gathered row
    int *group_rows; // [experts][3] records of the expert products
};
// softmax over a token's `routes` logits (row pitch ld), the `top` largest of score + correction; or (groups > 0) sigmoid scores, the `top`
// largest within the `keep` groups whose two best scores sum highest, divided by their sum and multiplied by `scale`.  Then lists of
// tokens by expert
struct RouteRule {
    int experts, routes, top;
    const float *correction;
    int groups, keep;
    float scale;
};
int route_tokens(const float *logits, int ld, const RouteRule &rule, int T, const RouteBuffers &b, hipStream_t st);
// dst[t] = base[t] + sum over choices of weight * (expert output row, or h[t]); base, dst fp32 (base may be null or dst), h of the
// activation type; narrow (or null): dst once more, of the activation type
int combine_experts(int act, const float *base, const float *outputs, const void *h, int top, const RouteBuffers &b, float *dst, void *narrow, int T,
        int hidden, hipStream_t st);

// ---- grouped attention
struct GroupedBuffers {
    const void *a; // the step's rows of the input product, of the activation type: q | k | v | gate from in_col on
    void *q; // [T][heads][D]: normed, rotated queries
    void *pool; // pages: by key / value head [64][D] keys, then two blocks of 32 tokens [V][32] values
    void *first_values; // [T][kv_heads][V]: written by the layer that says so, read by the others that mix
    void *conv_state; // filters: [slots][taps - 1][channels] of the activation type
    void *means; // pages as the pool's: means of blocks of tokens, a block an entry; their table [slots][means_stride]
    const int *means_table;
    int means_stride;
};
// filters, norms and rotation of queries and keys, mixing or rotation of values, append to the pages, means of the blocks that are full
int grouped_prepare(int act, const PlanLayer &L, const StepView &v, const GroupedBuffers &b, float eps, hipStream_t st);
// out: the step's rows of the output product's input; hint: upper bound of the sequence lengths
int grouped_attention(int act, const PlanLayer &L, const StepView &v, const GroupedBuffers &b, void *out, int hint, float *part, size_t part_floats,
        hipStream_t st);
int grouped_split_count(const PlanLayer &L, int B, int longest, int hint);
size_t grouped_part_floats(const PlanLayer &L);

struct LatentCacheView {
    void *pool; // [pages][kPageTokens][R + RD] of the activation type: normalised latent | rotated shared key part
    int R, RD;
};
// the query latent's norm -> cq; the key latent's norm and the shared key part's rotation -> cache
int latent_prepare(int act, const PlanLayer &L, const StepView &v, const void *a, void *cq, const LatentCacheView &cache, float eps, hipStream_t st);
// rotates the rotated parts of q [T][heads][D + RD] in place
int latent_rotate_q(int act, const PlanLayer &L, const StepView &v, void *q, hipStream_t st);
// absorbed form: qa [T][heads][R] queries in the latent space, q their rotated parts; out [T][heads][R] weighted latents;
// segments of up to `longest` tokens.  part: workspace of part_floats floats (split contexts).  hint: upper bound of the
// sequence lengths
int latent_attention(int act, const PlanLayer &L, const StepView &v, int longest, const void *qa, const void *q, void *out, const LatentCacheView &cache,
        int hint, float *part, size_t part_floats, hipStream_t st);
int latent_split_count(const PlanLayer &L, int B, int longest, int hint);
size_t latent_part_floats(const PlanLayer &L);
// expanded form: should a segment of n tokens that ends at position ctx take it
bool latent_expanded_takes(int act, const PlanLayer &L, int n, int ctx);
// cache rows of positions base .. base + rows - 1 of a slot -> out [rows][R + RD]
int latent_gather(const StepView &v, int slot, int base, int rows, const LatentCacheView &cache, void *out, hipStream_t st);
// one segment: tokens off .. off + n - 1 of the step at positions start .., q [T][heads][D + RD]; keys [ctx][heads D], values
// [ctx][heads V] and gathered cache rows of the positions from base (a multiple of 32) on, whole blocks of 32; out [T][heads V]
int latent_expanded(const PlanLayer &L, int off, int start, int n, int base, const void *q, const void *k, const void *values, const void *rows, void *out,
        hipStream_t st);

struct DeltaBuffers {
    void *in; // rows of the input product, of the activation type: q | k | v | beta | decay (rank) | gate (rank) from in_col on
    float *gates; // [T][2 * gcols]: decay step (before softplus) | output gate (before the sigmoid)
    float *q, *k, *qk; // [T][kv_heads][KD] twice, [T][kv_heads]
    float *g, *v, *beta; // [T][heads][KD] (one decay a head: [T][heads]), [T][heads][VD], [T][heads]
    float *o; // [T][heads][VD]
    void *out; // rows of the output product's input, of the activation type
    float *state; // [slots][heads][VD][KD]
    void *conv_state; // [slots][taps - 1][channels] of the activation type
};
// the last taps - 1 inputs of segments of several tokens: in [T] rows of pitch ld -> conv_state
int conv_tail(int act, const StepView &v, const void *in, int ld, int channels, int taps, void *conv_state, hipStream_t st);
int delta_prepare(int act, const PlanLayer &L, const StepView &v, const DeltaBuffers &b, hipStream_t st);
int delta_scan(const PlanLayer &L, const StepView &v, const DeltaBuffers &b, hipStream_t st);
int delta_output(int act, const PlanLayer &L, const StepView &v, const DeltaBuffers &b, float eps, hipStream_t st);

// ---- gated linear attention: S = diag(alpha) S + k v^T, o = S^T q
struct LinearBuffers {
    const void *in; // rows of the input product, of the activation type: q | k | v | decays (rank) | gate from in_col on
    const float *alpha; // [T][heads][KD]
    float *o; // [T][heads][VD]
    void *out; // rows of the output product's input, of the activation type
    float *state; // [slots][heads][VD][KD]
};
// the recurrence, the norm of every head and the gate
int linear_attention(int act, const PlanLayer &L, const StepView &v, const LinearBuffers &b, float eps, hipStream_t st);
// norm of every head of o [T][heads][VD] and silu gate (delta_output behind other recurrences)
int gated_head_norm(int act, const PlanLayer &L, int T, const float *o, const void *in, void *out, float eps, hipStream_t st);

// ---- gated linear recurrence: S = a S + sqrt(1 - a^2) i u by channel, a and i gated by the filtered input u itself
struct UnitBuffers {
    const void *in; // rows of the input product, of the activation type: y | x from in_col on
    void *u; // [T][channels] of the activation type
    float *gates; // [T][blocks][2][D]: r | i before their biases and sigmoids
    float *carry; // unit_carry_floats()
    void *out; // rows of the output product's input, of the activation type
    float *state; // [slots][channels]
    void *conv_state; // [slots][taps - 1][channels] of the activation type
};
int unit_filter(int act, const PlanLayer &L, const StepView &v, const UnitBuffers &b, hipStream_t st);
int unit_scan(int act, const PlanLayer &L, const StepView &v, const UnitBuffers &b, hipStream_t st);
size_t unit_carry_floats(const PlanLayer &L, size_t tokens, size_t segments);

} // namespace xfthip

struct xfthip_plan {
    xfthip_plan_config cfg;
    std::vector<xfthip::PlanLayer> layers;
    std::vector<xfthip::LayerRun> runs;
    int hidden = 0; // width padded to whole 32-value groups
    uint16_t *embedding = nullptr; // [vocab][hidden] bf16
    xfthip::PlanNorm final_norm; // times the logit scale
    uint16_t *pair_embedding = nullptr; // [bigram_buckets + 1][hidden] bf16
    uint16_t *side_embedding = nullptr; // [vocab][layers * side_pad] bf16
    int side_pad = 0;
    xfthip_weight_t head = nullptr;
    struct Tensor {
        std::vector<uint16_t> data;
        int rows = 0, cols = 0;
    };
    std::vector<std::pair<std::string, Tensor>> pending; // tensors given so far, until the plan is finished
    bool finished = false;
    size_t weight_bytes = 0;
};

namespace xfthip {

// Pages of 64 entries, `unit` tokens an entry (1: keys and values of tokens; more: means of blocks of tokens): free ones, those of every slot
// in position order, and the table [slots][stride], of which `at` is the place in the tables' common buffers.
struct PageTable {
    int unit = 1, pages = 0, stride = 0;
    size_t at = 0;
    std::vector<int> free_pages;
    std::vector<std::vector<int>> held;
    int pages_for(int tokens) const { return (tokens / unit + kPageTokens - 1) / kPageTokens; }
};

// What a model from a plan adds to xfthip_model: the page pool and the state slots, scratch, the step's description.
struct PlanState {
    xfthip_plan *plan = nullptr;
    std::vector<PlanLayer> layers; // the plan's, with this model's rotation tables
    int act = XFTHIP_BF16, esz = 2;
    int slots = 0;
    // by layer run, second mixers behind all of them: the record, page pool of an attention, state and convolution inputs of a
    // recurrence; which page pool an attention reads
    std::vector<int> store_layer, reads;
    std::vector<void *> cache;
    std::vector<float *> state;
    std::vector<void *> conv_state, means;
    std::vector<PageTable> tables; // the first: of tokens
    std::vector<int> table_host; // all tables, and on the device
    int *table = nullptr;
    bool table_dirty = true;
    // step description on the device, its host image (pinned) and the views into it
    int *desc = nullptr, *desc_host = nullptr;
    // pinned images of what else a step copies: the rows whose logits are wanted, a decode call's slots, the page table, logits
    int *want_host = nullptr, *dec_host = nullptr, *table_pinned = nullptr;
    float *logits_pinned = nullptr;
    int *tok_seg = nullptr, *tok_pos = nullptr, *ids = nullptr, *seg = nullptr, *dec_rows = nullptr, *want = nullptr;
    std::vector<int> seg_off_host, seg_len_host, seg_pos_host, seg_row_host; // the step's segments
    std::vector<int> dec_list; // slots of the decode call in flight
    std::vector<int> logit_of_row; // which row of the logits a slot's last ones are in
    int logit_rows = 0;
    // scratch (activation type unless float)
    void *xn = nullptr, *a = nullptr, *cq = nullptr, *q = nullptr, *qa = nullptr, *oc = nullptr, *ov = nullptr, *h = nullptr, *u = nullptr;
    float *y = nullptr, *y2 = nullptr, *gates = nullptr, *dq = nullptr, *dk = nullptr, *dqk = nullptr, *dg = nullptr, *dv = nullptr, *dbeta = nullptr, *do_ = nullptr, *carry = nullptr;
    int *last_token = nullptr; // [slots]
    void *xn2 = nullptr, *first_values = nullptr, *side = nullptr, *narrow = nullptr;
    float *router_logits = nullptr, *expert_out = nullptr, *side_z = nullptr;
    void *eh = nullptr;
    RouteBuffers route {};
    void *rows = nullptr, *kx = nullptr, *vx = nullptr; // gathered latents, keys and values of a long segment's context
    float *part = nullptr; // split contexts
    size_t part_floats = 0;
    std::vector<void *> owned; // every device buffer above
    bool trace = false;
    float *trace_buf = nullptr;
    size_t trace_floats = 0;
    int trace_tokens = 0;
};

// pages for the first `tokens` positions of a slot
int plan_reserve(xfthip_model *m, int row, int tokens);
void plan_release(xfthip_model *m, int row);
// residual rows of a step: entry i = the next lens[i] tokens of slot rows[i] (m->row_pos says where they stand; it moves on)
int plan_run(xfthip_model *m, int n, const int *rows, const int *lens, const int *ids, hipStream_t st);
// final norm and head of the residual rows rows_dev[0 .. n) (null: rows 0 .. n - 1) into m->logits + at * vocab
int plan_head(xfthip_model *m, const int *rows_dev, int n, int at, hipStream_t st);
// final norm and head of the residual rows list[0 .. n) (host), logits to host memory, as many rows at a time as fit
int plan_logits(xfthip_model *m, const int *list, int n, float *logits_host, hipStream_t st);
// upload of what a decode call of the slots in dec_list needs, for `steps` steps
int plan_decode_begin(xfthip_model *m, int steps, hipStream_t st);
// one decode step of the slots in dec_rows (recordable): positions and input ids from m->pos / m->ids
int plan_decode_step(xfthip_model *m, int B, hipStream_t st);
int plan_decode_splits(xfthip_model *m, int B, int hint);
int plan_prompt_pass(xfthip_model *m, const int *rows, int B, int S, const int *ids, float *logits_host, hipStream_t st);
int plan_reorder(xfthip_model *m, const int *dst, const int *src, int n, hipStream_t st);
void plan_state_destroy(PlanState *p);

// model.hip: first-maximum arg-max of n rows of logits; entry b goes to ids[rows ? rows[b] : b] (and bumps advance_pos there)
int argmax_rows(const float *logits, int n, int cols, int *ids, const int *rows, int *advance_pos, int *advance_step, hipStream_t st);

} // namespace xfthip
