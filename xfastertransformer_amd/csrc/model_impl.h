// The device model: weights by reference, caches, activation scratch and decode state of one decoder stack.
// Shared by the drivers (model.hip for uniform Llama-family stacks, plan_model.hip for layer plans).
#pragma once
#include <vector>

#include "attention_dev.h"
#include "kvcache.h"
#include "qgemm.h"

namespace xfthip {

struct LayerW {
    xfthip_weight_t qkv = nullptr, o = nullptr, gateup = nullptr, down = nullptr;
    // optional second set used by the prompt pass only (the reference's HybridModel: one weight type for the
    // first token, another for the following ones, src/models/hybrid_model.h:25-84)
    xfthip_weight_t first_qkv = nullptr, first_o = nullptr, first_gateup = nullptr, first_down = nullptr;
    float *ln1 = nullptr, *ln2 = nullptr, *qkv_bias = nullptr, *o_bias = nullptr;
    // set: the layer's two norms are LayerNorms with these shifts (NormType::LN of the layer API) instead of RMSNorms
    float *ln1_beta = nullptr, *ln2_beta = nullptr;
    // set: the layer's MLP is this sparse one (MixtralMLP; it carries its own norm weight and router), not gateup / down
    xfthip_moe_t moe = nullptr;
};

struct PlanState; // plan.h

} // namespace xfthip

struct xfthip_model {
    xfthip_model_config cfg;
    // set: the layers follow a plan (several kinds of layers, paged cache and recurrent state); layers / caches stay empty
    xfthip::PlanState *plan = nullptr;
    std::vector<xfthip::LayerW> layers;
    std::vector<xfthip_kvcache_t> caches;
    // INT8 KV: the first-token pass attends over unquantised keys/values, as the reference's
    // flash path does on its bf16 copies (src/layers/attention.h:1121-1188); they live here
    xfthip_kvcache_t prefill_cache = nullptr;
    xfthip::AttnWorkspace attn_ws; // split-KV partials and tickets of this model's attention launches
    // W8A8 layers: int8 activation rows + per-row (scale, zero, sum), and the [tokens, 2 * inter]
    // bf16 result of the gate/up projection (which runs as a plain GEMM for this kind)
    int8_t *w8a8_qa = nullptr;
    size_t w8a8_qa_bytes = 0;
    float *w8a8_stat = nullptr;
    uint16_t *gu = nullptr;
    float *cosT = nullptr, *sinT = nullptr;
    // scratch
    uint16_t *xn = nullptr, *qkv = nullptr, *att = nullptr, *h = nullptr;
    float *x = nullptr, *xlast = nullptr, *logits = nullptr;
    int *ids = nullptr, *pos = nullptr, *step = nullptr, *idlog = nullptr;
    int idlog_cap = 0;
    // head
    uint16_t *embedding = nullptr;
    float *final_norm = nullptr;
    xfthip_weight_t lm_head = nullptr;
    // decode state
    int cur_B = 0, cur_pos = 0;
    int prompt_rows = 0; // rows of `x` that hold the last layer's output of the most recent prompt pass (0 after a decode step)
    int prefix_len = 0; // positions [0, prefix_len) of cache row 0 hold a shared prefix (xfthip_model_set_prefix)
    // continuous batching: sequences live in cache rows of their own, each at its own position
    int row0 = 0; // cache row of the first sequence of the forward call in flight
    bool ragged = false; // rows may differ in position or sit out a step (set by the xfthip_model_seq_* calls)
    int *active = nullptr; // device [max_batch]: rows taking part in the next decode call
    int *prompt_ids = nullptr; // device [max_tokens]: prompt of a single-sequence prefill
    std::vector<int> row_pos; // host copy of every row's position (-1 = free row)
    unsigned char *kv_stage = nullptr; // staging buffer of xfthip_model_seq_reorder (grown on demand)
    size_t kv_stage_bytes = 0;
    int *reorder_rows = nullptr; // device [2 * max_batch]: source rows, destination rows
    hipGraphExec_t graph = nullptr;
    int graph_B = 0;
    int graph_nsplit = 0; // attention split count the captured step was built with
    bool graph_ragged = false; // the captured step's last node holds the `active` mask only in this mode
    int len_hint = 0; // upper bound of the sequence length during the current decode call (0 = unknown)
    hipStream_t graph_stream = nullptr;
    bool use_graph = true;
    bool fuse_decode = true; // RMSNorm prologue / RoPE + cache-append epilogue inside the decode GEMVs
};
