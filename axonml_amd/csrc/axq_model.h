// The decode model's state, shared by the LLaMA-shape layers (axq_decode.hip) and the described layers (axq_stack.hip).
#pragma once
#include <vector>

#include "axq_internal.h"

struct axq_stack;

struct axq_model {
    axq_ctx *ctx;
    axq_model_config cfg;
    int qkv_rows, q_dim, kv_dim;
    // weights
    uint16_t *emb;                  // f16 [vocab, hidden], or
    float *emb32 = nullptr;         // f32 [vocab, hidden] as the reference keeps it (one of the two is set)
    float *norm_attn, *norm_ffn;    // [layers, hidden]
    float *norm_final;              // [hidden]
    std::vector<axq_weight *> w_qkv, w_o, w_gu, w_down;
    // q, k or v of a layer whose block type differs from the fused weight's (GGUF files that keep attn_v at six bits
    // beside four-bit attn_q and attn_k): a weight of its own, multiplied after the fused one into its rows of qkv
    std::vector<axq_weight *> w_sep[3];
    axq_weight *w_head;
    std::vector<uint32_t> set_mask; // per layer: bit per axq_linear_id that has been set
    bool head_set;
    float *rope_cos, *rope_sin;     // [max_pos, head_dim / 2]
    uint16_t *kcache, *vcache;      // f16 [layers, kv_heads, max_pos, head_dim]
    // activations
    float *h, *xn, *qkv, *att, *gu, *act, *logits;
    float *att_part;                // [kv_heads][max_splits][rep][head_dim + 2] partial attention results
    float *pb_h, *pb_xn, *pb_qkv, *pb_att, *pb_gu, *pb_act; // the same activations for pb_cap prompt tokens at a time
    int pb_cap;
    int n_seq;                      // sequences the caches and the per-sequence state hold (axq_model_set_batch)
    size_t seq_stride;              // cache elements of one sequence: layers * kv_heads * max_pos * head_dim
    size_t part_stride;             // floats of att_part per sequence
    std::vector<int> seq_pos;       // host mirror of pos[s] for the batched calls (sequence 0: host_pos)
    int32_t *bprompt, *boffsets, *bout; // prompts, their offsets and the generated ids of a batched generate
    hipGraphExec_t graph_b, graph_bf; // batched step: split attention / one attention workgroup per head (short contexts)
    bool graph_b_ok, graph_bf_ok;
    int max_splits;
    // device-side state
    int32_t *pos, *tok, *next, *gen, *prompt, *out;
    int32_t *hist;                  // every token fed so far, by position (what a repetition penalty looks at)
    void *sample_scratch;           // scratch of the sampler, allocated when one is set
    bool sampling;                  // next token by axq_sampling_config instead of the plain argmax
    axq_sampling_config sampler;
    uint64_t sample_seed;
    int prompt_cap, out_cap;
    int host_pos;
    hipGraphExec_t graph;           // the one-token step with the attention split over the positions
    bool graph_ok;
    hipGraphExec_t graph_f;         // the same with one attention workgroup per head (short contexts)
    bool graph_f_ok;
    int fused_max;                  // contexts up to this many positions take graph_f
    int prompt_chunk;               // most prompt rows per pass through the layers
    bool attn_mfma;                 // prompt attention of many rows on the matrix pipe (development knob AXQ_ATTN_MFMA=0: off)
    axq_stack *stack = nullptr;     // layers described one by one (axq_model_create_stack) instead of the LLaMA shape above
};

// axq_decode.hip: the buffers every model has (token, position, history, prompt, output, logits), for one sequence.
int axq_model_alloc_common(axq_model *m);
void axq_model_drop_graphs(axq_model *m);

// axq_stack.hip: what the stepping functions of axq_decode.hip call for a model with m->stack set.
// One token (m->tok at position *m->pos) through the layers to m->logits; fit for graph capture.
int axq_stack_step(axq_model *m);
// nb tokens at positions pos0 .. pos0 + nb - 1; afterwards axq_stack_logits_rows can be asked for any of them.
int axq_stack_rows(axq_model *m, const int32_t *toks, int nb, int pos0);
// logits of `n` rows (indices within the last axq_stack_rows, on the host) -> host memory
int axq_stack_logits_rows(axq_model *m, const int32_t *rows, int n, float *logits);
// where the residual stream after every layer run of the coming axq_stack_rows goes (host; NULL: nowhere)
void axq_stack_trace(axq_model *m, float *layers, int total_rows, int row0);
int axq_stack_layer_runs(const axq_model *m);
int axq_stack_ready(axq_model *m);
bool axq_stack_recurrent(const axq_model *m); // state that cannot be rewound
int axq_stack_random_init(axq_model *m, float std, uint64_t seed);
void axq_stack_free(axq_model *m);
