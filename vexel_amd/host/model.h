// The model behind vh_model: block pool, caches, device mirrors, weights; shared by the host runtime's files.
#pragma once

#include <stdint.h>

#include <algorithm>
#include <map>
#include <memory>
#include <mutex>
#include <string>
#include <unordered_map>
#include <vector>

#include "vexel_host.h"

namespace vh {

}  // namespace vh

extern "C" void vh_set_error(const char *text);

namespace vh {

int fail(const char *fmt, ...);  // sets vh_last_error(), returns VH_ERR

#define VXC(expr)                                                         \
    do {                                                                  \
        int _rc = (expr);                                                 \
        if (_rc != VX_OK) return fail("%s: %s", #expr, vx_last_error());  \
    } while (0)
#define VHC(expr)                      \
    do {                               \
        if ((expr) != VH_OK) return VH_ERR; \
    } while (0)

struct SeqState {
    std::vector<int32_t> table;  // logical block -> physical block (same for every layer)
    int seq_len = 0;
    int slot = -1;               // row in the device block-table matrix
    bool dirty = true;           // device row differs from `table`
};

struct Fragment {                 // kv/fragment.go:9-16
    int num_tokens = 0;
    std::vector<int32_t> blocks;  // the cached sequence's table (the same for every layer), one reference each
};

struct BlockPool {
    int block_size = 16, max_blocks = 0;
    std::map<std::string, Fragment> fragments;    // kv/fragment.go:19-23
    std::vector<int32_t> free_list;               // gpu_block_pool.go:110-116
    std::unordered_map<int32_t, int> ref_counts;  // gpu_block_pool.go:42-43
    std::map<int64_t, SeqState> seqs;
    std::mutex mu;                                // gpu_block_pool.go:46
    std::vector<int> free_slots;
    bool free_dirty = true;

    int alloc_block(int32_t *out) {               // gpu_block_pool.go:200-209
        if (free_list.empty()) return fail("no free blocks (max=%d)", max_blocks);
        *out = free_list.back();
        free_list.pop_back();
        ref_counts[*out] = 1;
        free_dirty = true;
        return VH_OK;
    }
    void release_block(int32_t b) {               // gpu_block_pool.go:211-219
        auto it = ref_counts.find(b);
        int rc = it == ref_counts.end() ? 0 : it->second;
        if (rc <= 1) {
            if (it != ref_counts.end()) ref_counts.erase(it);
            free_list.push_back(b);
            free_dirty = true;
        } else {
            it->second = rc - 1;
        }
    }
    int ensure_blocks(SeqState &s, int end_pos) {  // gpu_block_pool.go:234-245
        if (end_pos <= 0) return VH_OK;
        int last = (end_pos - 1) / block_size;
        while ((int)s.table.size() <= last) {
            int32_t b;
            VHC(alloc_block(&b));
            s.table.push_back(b);
            s.dirty = true;
        }
        return VH_OK;
    }
};

// ---- mixer programs: layers whose sublayers are described one by one (layers.cpp) ----

struct Linear {       // packed bfloat16 weights (vx_linear_pack), padded sizes
    void *w = nullptr;
    int n = 0, k = 0;
};

// vx_attn_ragged; columns are places in the layer's input projection. Keys and values leave for the pool in the projection's
// epilogue, or (by_heads) queries, keys and values pass through vx_heads_store, from a float32 projection.
struct AttnMixer {
    int heads = 0, kv_heads = 0, k_dim = 0, v_dim = 0;
    float scale = 1.f, temp_coef = 0.f;
    int temp_every = 0;
    const float *bias = nullptr;  // [heads][bias_len]
    int bias_len = 0;
    bool gate = false;
    float out_scale = 1.f;
    int q_col = 0, k_col = 0, v_col = 0, g_col = 0;    // v_col < 0: values are keys as projected
    bool by_heads = false, norm = false;
    bool row_norm = false;                             // the norms are over all heads of a row
    int kv_from = -1;                                  // the layer whose pool is read, -1: its own
    const float *slopes = nullptr;                     // [heads], as they are behind the mixing of heads
    const void *talk = nullptr;                        // bfloat16 [heads][heads]
    const float *in_bias = nullptr, *norm_q = nullptr, *norm_k = nullptr;
    int rotation = -1;                                 // index in MixModel::rotations, halves of a head's first dimensions
    int window = 0, chunk = 0;
    float softcap = 0.f;
    const float *sink = nullptr;
    int maps = 1;                                      // 2: differential heads
    float diff_lambda = 0.f, diff_scale = 1.f;
};

// vx_decay_attn and vx_gated_norm. Projection: q | k | v with SiLU, heads padded to dim_pad and v_pad columns; behind them, in float32, the
// gate.
struct DecayMixer {
    int heads = 0, vdim = 0, dim_pad = 0, v_pad = 0;
    int split = 0, g_col = 0;                          // columns of q | k | v; the gate's among the others
    const float *decay = nullptr, *norm = nullptr;     // [heads][2]; [heads * v_pad]
};

// vx_forget_attn and vx_head_norm. Projection: q with SiLU | v, heads padded to dim_pad and v_pad columns; behind them, in float32, one minus
// the gates.
struct ForgetMixer {
    int heads = 0, vdim = 0, dim_pad = 0, v_pad = 0;
    const float *bias = nullptr, *keep = nullptr;      // [heads * dim_pad]: of the gates' projection; one minus their lower bound
    const float *norm = nullptr;                       // [v_pad]
};

// vx_route and vx_linear_experts over the layer's normed input; the router's logits are columns of the input projection's float32 part,
// or a map of their own. Experts: gate|up pairs, or (relu2) up alone.
struct ExpertMlp {
    int experts = 0, top = 0, groups = 1, keep = 1;
    bool shared = false;
    int router_col = 0, ff_pad = 0, shared_pad = 0;
    float limit = 0.f, shared_limit = 0.f, alpha = 0.f, add = 0.f;
    const float *correction = nullptr;
    bool relu2 = false, softmax = false;
    Linear router;
    const float *router_bias = nullptr;
    Linear gate_up, down, shared_gate_up, shared_down; // the experts' one behind the other: n counts one expert's
};

struct ScanMixer {    // vx_conv_silu, the projections of its result, vx_selective_scan
    int channels = 0, states = 0, pad = 0, taps = 0, dt_rank = 0, dt_pad = 0;
    float out_scale = 1.f;
    int x_col = 0, z_col = 0;
    const float *conv_w = nullptr, *conv_b = nullptr;  // [taps][channels], [channels]
    Linear x, dt;                                      // channels -> dt_pad | B | C; dt_pad -> channels
    const float *dt_bias = nullptr, *a2 = nullptr, *d = nullptr;
};

struct Rotation {      // pair i turns by position * freqs[i]; cosine and sine times factor
    std::vector<double> freqs;
    float factor = 1.f;
    const double *d_freqs = nullptr;
};

// Latent attention (vx_latent_store, vx_attn_latent). Prompts' queries meet either the latents themselves (queries carried into
// their space by `absorb`, results out of it by `value`) or, from expand_rows rows of a sequence on, keys and values
// spelled out for the step (`expand`, vx_attn_ragged). Heads of the query projection: dim_pad columns, then the rotated part.
struct LatentMixer {
    int heads = 0, rank = 0, rot_dim = 0, q_rank = 0;
    int dim_pad = 0, head_cols = 0, v_pad = 0, rank_pad = 0, row = 0;
    float scale = 1.f;
    int rotation = -1;                                 // index in MixModel::rotations, -1: nothing is rotated
    int kv_from = -1;                                  // the layer whose pool is read, -1: its own
    int c_col = 0, kr_col = 0, kv_cols = 0;            // in the float32 part of the input projection (q_rank > 0: all of it, the
                                                       // query latent first; else kv_cols columns behind the heads)
    const float *norm_c = nullptr, *norm_q = nullptr, *sink = nullptr;
    Linear q_up;                                       // query latent -> heads (q_rank > 0)
    Linear absorb;                                     // per head: dim_pad -> rank_pad, one behind the other
    Linear expand;                                     // rank_pad -> heads' keys [heads * dim_pad] | values [heads * v_pad]
    int expand_rows = 0;                               // 0: never
};

// x += mult * rms(mixers(rms(x) * norm1)) * norm1b, then the same around the MLP. The mixers of a layer read one input
// projection and write one row, which one output projection takes. In a model with post_norm instead: x = rms(alpha * x +
// mixer(x)) * norm1, x = rms(alpha * x + MLP(x)) * norm2, then the average over the depth. A layer with experts instead: x +=
// mixer(h) + experts(h), h = rms(x) * norm1. In a model with branch_norm: x += ln(mixer(x); norm1, norm1b), x += ln(MLP(x); norm2,
// norm2b), MLP dense or experts.
struct MixLayer {
    const float *norm1 = nullptr, *norm1b = nullptr, *norm2 = nullptr, *norm2b = nullptr;
    bool has_attn = false, has_scan = false, has_latent = false, has_decay = false, has_forget = false, has_mlp = false, has_experts = false;
    AttnMixer attn;
    DecayMixer decay;
    ForgetMixer forget;
    ExpertMlp moe;
    const float *out_bias = nullptr;   // of the output projection, in layers without norm1b
    LatentMixer latent;
    ScanMixer scan;
    Linear in, out;
    Linear gate_up, down;
    int ff = 0, ff_pad = 0;
    bool relu2 = false;            // the MLP is down(relu(up + up_bias)^2) + down_bias, gate_up holds up alone
    const float *up_bias = nullptr, *down_bias = nullptr;
    const float *poly = nullptr;   // set: the MLP is down(poly_norm(up)), gate_up holds up alone (vx_poly_norm)
    const float *depth_avg = nullptr;  // weights of the embedding output and of every result up to this layer's
};

struct LayerRun {     // one pass through a layer; every pass has its own cache and state
    int layer = 0;
    bool add_embedding = false;    // the embedding output is added to the stream first
    void *kv = nullptr;            // paged pool (owned by vh_model::kv, by the run that writes it)
    void *conv = nullptr;          // [max_seqs][taps - 1][channels]
    float *state = nullptr;        // [max_seqs][channels][pad], or [max_seqs][heads][dim_pad][v_pad]
};

struct MixActs {      // a step's activations for up to `rows` rows
    int rows = 0;
    float *x = nullptr, *emb = nullptr, *bc = nullptr, *dt = nullptr, *y = nullptr;
    void *h = nullptr, *proj = nullptr, *cat = nullptr, *xc = nullptr, *dtr = nullptr, *act = nullptr;
    void *qc = nullptr, *qa = nullptr, *lo = nullptr, *z = nullptr;  // query latent; queries and results in the latents' space; up's output
    float *hist = nullptr, *rot = nullptr;                           // results of all layers; angle tables, one after the other
    float *o = nullptr;                                              // what states gave
    void *e_act = nullptr, *e_out = nullptr;                         // by place in the experts' order
    float *e_weights = nullptr;
    int32_t *e_places = nullptr, *e_order = nullptr, *e_tiles = nullptr;
};

// The sequences of a step whose keys and values are spelled out: their tokens, block after block, from row 0 on.
struct MixExpand {
    int rows = 0, max_blocks = 0;
    const int32_t *slots = nullptr;    // [rows] pool slot of every token
    const int32_t *tables = nullptr;   // [n_seqs][max_blocks] blocks of the spelled-out rows
    const int32_t *table_rows = nullptr;  // [n_seqs] 0, 1, ..
    void *kv = nullptr;
};

struct MixModel {
    int act = VX_ACT_BF16;
    float eps = 1e-5f, mult = 1.f;
    bool post_norm = false;
    bool branch_norm = false;
    float alpha = 1.f, softcap = 0.f, logit_mult = 0.f;
    // branch_norm: the embedding is ln(token's + position's; emb_norm, emb_norm_b), the last norm has a bias
    const float *positions = nullptr, *emb_norm = nullptr, *emb_norm_b = nullptr, *final_norm_b = nullptr;
    int max_positions = 0;         // > 0: a sequence holds no more tokens
    bool recurrent = false;        // a sequence is more than its blocks
    int expand_rows = 0;           // the smallest of the layers'
    const float *pairs = nullptr;  // set: the embedding has a table of token pairs (vx_pair_embedding)
    int buckets = 0;
    int64_t mul_prev = 0, mul_cur = 0;
    int32_t *token_pool = nullptr;
    std::vector<Rotation> rotations;
    std::vector<MixLayer> layers;
    std::vector<LayerRun> runs;
    Linear head;
    MixActs perm;                  // for steps of at most max_batch rows
};

// Creates the pool, the device mirrors of its tables and the step buffers every model has (cfg, be set).
int init_common(vh_model *m);
SeqState *find_seq(vh_model *m, int64_t id);
int create_seq_locked(vh_model *m, int64_t id);
int sync_pool_to_device(vh_model *m);

// A model whose mixer program is complete in m->mix (weights included): caches, states, activations.
int mix_finish(vh_model *m);
// Embedding of b.rows tokens -> layer runs -> final norm and head of n_want rows (want: device row numbers, NULL = the
// first n_want) -> logits [n_want, vocab].
int mix_forward(vh_model *m, const vx_ragged &b, const int32_t *d_tokens, const MixActs &a, const MixExpand *ex, const int32_t *want,
                int n_want, float *logits);
// One mixed step (vh_step) of such a model.
int mix_step(vh_model *m, int n_seqs, const int64_t *seq_ids, const int32_t *q_lens, const int32_t *tokens, int n_want,
             const int32_t *want_rows, float *logits_out, int32_t *argmax_out);

}  // namespace vh

struct vh_model {
    vx_backend *be = nullptr;
    vh_config cfg{};
    std::vector<vh_layer_weights> layers;
    const float *embedding = nullptr;
    const float *final_norm = nullptr;
    vh_qweight lm_head{};
    std::vector<void *> adopted;  // device buffers a loader handed over (vh_model_adopt_buffer)
    vh::BlockPool pool;
    std::vector<void *> kv;

    int32_t *d_tables = nullptr, *d_num_blocks = nullptr, *d_free = nullptr, *d_free_count = nullptr;
    int32_t *d_slots = nullptr, *d_positions = nullptr, *d_tokens = nullptr, *d_next = nullptr;
    int32_t *d_cu = nullptr, *d_token_pos = nullptr, *d_slot_map = nullptr, *d_kv_lens = nullptr;
    int32_t *d_pos_in = nullptr;  // positions of a host-driven step, input of the packing kernel
    int32_t *d_status = nullptr, *d_step = nullptr, *d_log = nullptr;
    int log_cap = 0;  // steps the log can hold

    float *x = nullptr, *norm = nullptr, *q = nullptr, *k = nullptr, *v = nullptr, *attn = nullptr;
    float *gate = nullptr, *up = nullptr, *logits = nullptr;

    bool fused = true;  // take the fused decode entry points where the weights allow it

    vh_arch arch{};                       // all zero: the LLaMA arm
    std::vector<vh_layer_extras> extras;  // per layer, all NULL by default
    const float *final_norm_bias = nullptr;
    float *zeros = nullptr;               // [hidden] zeros: the bias of a LayerNorm whose bias tensor is absent
    bool general = false;                 // some switch or extra tensor is set: the one-call-per-operation sequence
    bool fused_ok = true;                 // the layer differs from LLaMA's at most by Q/K/V biases and the RoPE form
    bool attn_fused_ok = true;            // the attention half does (RMSNorm without a bias in front of Q|K|V): its fused block serves it
                                          // (Qwen 2): decode may still take the fused entry points

    std::unique_ptr<vh::MixModel> mix;    // set: the layers are a mixer program (layers.cpp) and the fields of the LLaMA family are unused

    vx_graph *graph = nullptr;
    int graph_batch = 0;
    uint64_t graph_scratch_gen = 0;  // vx_scratch_generation() when the graph was captured
    std::vector<int64_t> dev_seq_ids;  // batch currently loaded in d_slots (device-driven mode)
    std::vector<int32_t> dev_positions;
};
