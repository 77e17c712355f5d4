// Models described layer by layer (pi_model_create_layers): weights in the operators' layouts, one pool of cache cells shared by all
// sequences, steps of any mixture of prompt portions and single tokens, and the captured greedy loop.
#include "engine_internal.hpp"
#include "runtime.hpp"

#include <math.h>
#include <stdlib.h>
#include <string.h>

#include <algorithm>
#include <vector>

#define PI_TRY(expr) do { int _rc = (expr); if (_rc != PI_OK) return _rc; } while (0)

namespace {

constexpr int kOwnSeq = 31;              // the model's own sequence (pi_model_decode / pi_model_generate)
constexpr int kHeadRows = 256;           // rows of logits held at a time
constexpr int kMaxLockstep = 16;
constexpr long long kExpandedValues = 1LL << 29;      // most expanded key and value numbers of one run (1 GiB)
constexpr int kItemRows = 32;             // query rows of an attention work item
constexpr int kAttnItems = 512;          // (work item, part) pairs a split attention aims at: two workgroups per compute unit
constexpr int kWideRows = 64;            // query rows from which a run of grouped-query attention takes the wide work items
constexpr int kTalkCells = 256;          // fewest cells of a part of such an item
constexpr int kTalkItems = 32;           // items from which pi_k_gqa_talk fills enough of the device (fewer: the cells of an item are split)
constexpr int kLinearChunked = 17;       // tokens from which a run of linear attention is worked in chunks
constexpr int kFreshSteps = 4;           // first tokens of a sequence that a norm over every head's sums is sensitive to (see layers_step)

int up_to(int v, int m) { return (v + m - 1) / m * m; }

// the recurrent part of a layer's mixer: rows of the joint projection, sizes and weights
struct Rec {
    int kind = -1, n_head = 0, dim = 0, vdim = 0, dim_ld = 0, vdim_ld = 0, rank = 0, rank_ld = 0;
    int off_q = 0, off_k = 0, off_v = 0, off_g = 0, off_a = 0, off_i = 0, off_f = 0, off_att = 0;      // off_att: column of the mixer's result
    float tau = 0.0f, cap = 0.0f, q_scale = 1.0f, scale = 1.0f;
    bool plain = false, silu = false, per_head = false;           // projections without an activation; gate; norm over every head by itself
    const float *decay = nullptr, *powers = nullptr, *norm = nullptr, *a2_b = nullptr, *i_b = nullptr, *f_b = nullptr;
    const void * a2 = nullptr;
    bool on() const { return kind >= 0; }
};

struct Layer {
    pi_layer_desc d{};
    Rec rec;
    int nq = 0, z_rows = 0, dim_ld = 0, rank_ld = 0, kd = 0, hv_ld = 0, ff_ld = 0, rot = 0, hc = 0;      // rot, hc: index among the model's rotations / kinds of heads
    int off_k = 0, off_v = 0, off_glu = 0, off_score = -1, off_router = 0;      // rows of the joint projection (layers with one norm)
    int off_gate = 0, off_gate_ffn = 0, z2_rows = 0;              // norm after the sum: rows of the residual gates, rows of the feed-forward's projection
    int hd = 0, glu_ld = 0, close_ld = 0;
    bool own_kv = true;
    const void *w_z = nullptr, *uk = nullptr, *uk_t = nullptr, *uv = nullptr, *wo = nullptr, *router = nullptr, *up = nullptr, *down = nullptr;
    const float *norm_a = nullptr, *norm_b = nullptr, *dkv_norm = nullptr, *sink = nullptr, *bias = nullptr;
    const void * w_ffn = nullptr;                                 // norm after the sum: [gate and up rows in turn | residual gate]
    const float *q_norm = nullptr, *k_norm = nullptr, *temp = nullptr, *gate_b = nullptr, *gate_ffn_b = nullptr;
    // norms around the sublayers, convolution of the mixer's input, heads mixed and gated, mixed values
    const float *norm_a_after = nullptr, *norm_b_after = nullptr, *conv = nullptr, *talk = nullptr, *v_mix = nullptr;
    int off_head_gate = -1; size_t conv_floats = 0; bool first_values = false;
    // one per pass of the loop the layer is part of
    std::vector<void *> cache;                         // cells
    std::vector<float *> state;                        // [slots][state_floats()]
    size_t cell_values() const { return d.mixer == PI_MIXER_GROUPED ? (size_t)d.n_kv_head * 2 * hd : d.mixer == PI_MIXER_LATENT && own_kv ? (size_t)kd : 0; }
    // a slot: the recurrent part's state, then the last inputs of the convolution
    size_t rec_floats() const { return rec.on() ? pi_k_linear_slot_floats(rec.kind, rec.n_head, rec.dim, rec.vdim) : 0; }
    size_t state_floats() const { return rec_floats() + conv_floats; }
    bool heads_apart() const { return d.head_mix || d.head_gate; }      // the heads' results are mixed or gated behind the attention
    bool moe() const { return d.ffn == PI_FFN_MOE || d.ffn == PI_FFN_GLU_MOE; }
};

struct LayerRun { int layer, pass; bool starts; };     // starts: a pass of the loop begins with it

struct Rotation {
    int dims; double base;
    int scaling; double factor, original, low, high;
    const double * freq;                               // device, with a scaling
    bool same(const pi_layer_desc & d) const {
        return dims == d.rot_dim && base == d.rot_base && scaling == d.rot_scaling && (!scaling || (factor == d.rot_factor && original == d.rot_original && low == d.rot_low && high == d.rot_high));
    }
    double length() const { return scaling == PI_ROT_RAMP ? 0.1 * log(factor) + 1.0 : 1.0; }
    // what becomes of base^(-2 i / dims)
    std::vector<double> frequencies() const {
        std::vector<double> f(dims / 2);
        const auto pair_of = [&](double turns) { return dims * log(original / (2.0 * M_PI * turns)) / (2.0 * log(base)); };      // the pair that makes so many turns
        const double first = std::max(floor(pair_of(high)), 0.0), last = std::min(ceil(pair_of(low)), dims - 1.0);
        for (int i = 0; i < dims / 2; ++i) {
            f[i] = pow(base, -2.0 * i / dims);
            double kept = 1.0;                         // share of the frequency that stays as it is
            if (scaling == PI_ROT_WAVES) {
                const double turns = original * f[i] / (2.0 * M_PI);
                kept = turns > high ? 1.0 : turns < low ? 0.0 : (turns - low) / (high - low);
            } else if (scaling == PI_ROT_RAMP) kept = 1.0 - std::min(std::max((i - first) / std::max(last - first, 0.001), 0.0), 1.0);
            f[i] = f[i] * kept + f[i] / factor * (1.0 - kept);
        }
        return f;
    }
};
// n_head: of a work item's rows - all heads on a latent, the heads of a group otherwise (n_kv groups, with pi_gqa_attn's all_values pairs of them; kd
// values of a key row)
// window > 0: cells a token sees
// talk_tokens: tokens of an item of pi_k_gqa_talk (0: that does not serve these heads)
// (grouped-query attention: n_head query heads per group, n_kv groups, or pairs of a group and whose values its heads meet)
struct HeadKind {
    int mixer, n_head, n_kv, dim, rot_dim, vdim, rank_ld, kd, window, talk_tokens;
    int value_groups() const { int g = 1; while ((g + 1) * (g + 1) <= n_kv) ++g; return g; }      // (where n_kv counts pairs)
};
enum Family { kTwoNorms, kOneNorm, kPostNorm, kBothNorms };

// where a pass finds its tokens
struct Step {
    int T = 0;
    const int32_t *tokens = nullptr, *pos = nullptr, *cell = nullptr, *n_vis = nullptr, *seq = nullptr;
    struct Work { const int32_t * items = nullptr; int n = 0, parts = 1; };
    struct Run { int tok0, T, seq, n_cells; };
    // per kind of latent head (distinct sizes of the model's layers): the tokens that attend in latent space as work items, and the long
    // runs that attend over expanded keys and values
    std::vector<Work> work;
    std::vector<std::vector<Run>> runs;
    // grouped-query attention: the long runs as wide work items (per kind); linear attention: the runs walked token by token and in chunks;
    // prev: each token's predecessor (carry: the embedding moves it on, for a captured step)
    std::vector<Work> wide;
    // heads mixed behind their attention: the tokens of the long runs for pi_k_gqa_talk (then the wide items are its first pass's), and the others
    std::vector<Work> talk;
    std::vector<Work> apart;
    std::vector<const int32_t *> first;                // per kind: the first cell of each token's window (null: counted back from its last)
    int32_t * prev = nullptr; bool carry = false;
    const int32_t *lin = nullptr, *lin_long = nullptr, *lin_first = nullptr, *lin_chunks = nullptr;
    int n_lin = 0, n_lin_long = 0, n_lin_chunks = 0;
    const int32_t * conv = nullptr; int n_conv = 0;    // items of the convolutions
};

}  // namespace

typedef uint16_t bf16_t;                 // bit patterns

struct LayerState {
    pi_layers_opts opts{};
    std::vector<Layer> layers;
    std::vector<Rotation> rots;
    std::vector<HeadKind> kinds;
    int d_ld = 0, es = 2;
    const float *embd_norm = nullptr, *out_norm = nullptr;
    const void *embed = nullptr, *head = nullptr, *bigram = nullptr;
    const float * loop_step = nullptr;                 // [loop_times][n_embd]
    std::vector<LayerRun> order;                       // the layer runs of a step
    Family family = kTwoNorms;
    bool recurrent = false;
    int n_slots = 0, slot_of[32];                      // slots of recurrent states; -1: the sequence has none
    KvCells kv;
    std::vector<int32_t> cell_tok;                     // the token of every cell
    bool auto_pool = false;                            // sized by the engine (decode, batch_init), not by the caller
    int32_t * lists = nullptr;                         // device [32][kv.n]: a sequence's cells in position order
    std::vector<int32_t> list_cells[32], list_pos[32]; // the same on the host
    int32_t * d_delta = nullptr;
    // step buffers for `cap` tokens (one allocation)
    int cap = 0;
    unsigned char * arena = nullptr;
    float *x = nullptr, *x2 = nullptr, *x0 = nullptr, *z = nullptr, *mix = nullptr, *rl = nullptr, *wts = nullptr, *lin_o = nullptr, *lin_den = nullptr, *lin_gates = nullptr;
    void *lin_q = nullptr, *lin_k = nullptr, *lin_v = nullptr, *lin_states = nullptr;
    void *h_a = nullptr, *h_b = nullptr, *q_un = nullptr, *q_lat = nullptr, *o_lat = nullptr, *att = nullptr, *act = nullptr, *y_exp = nullptr;
    int32_t *ids = nullptr, *perm = nullptr, *inv = nullptr, *off = nullptr, *tiles = nullptr, *n_tiles = nullptr;
    float *heads = nullptr, *v_first = nullptr, *stats = nullptr;        // the heads' results ahead of their mixture, the first values of the step's tokens
    std::vector<float *> cs;                           // per rotation [cap][dims / 2] (cos, sin)
    bf16_t * expanded = nullptr; size_t expanded_cap = 0;      // keys and values of a long run's cells
    float * scratch = nullptr;                         // partial sums of a split attention
    float * logits = nullptr; void * h_head = nullptr; int32_t * d_next = nullptr;
    int32_t * h_in = nullptr, * d_in = nullptr; size_t in_cap = 0;       // a pass's integers: pinned host side and device side
    float * streams = nullptr; size_t streams_cap = 0; int streams_T = 0;
    // lockstep decoding and the greedy loop
    int n_seq = 0;
    int32_t last_tok[32], last_pos[32];
    int32_t *g_tok = nullptr, *g_pos = nullptr, *g_cell = nullptr, *g_vis = nullptr, *g_seq = nullptr, *g_work = nullptr, *g_step = nullptr, *g_out = nullptr, *g_prev = nullptr, *g_lin = nullptr, *g_conv = nullptr;
    int max_steps = 4096;
    hipGraph_t graph = nullptr; hipGraphExec_t exec = nullptr;
    int graph_T = 0, graph_seq0 = -1; std::vector<int> graph_parts;
};

namespace {

__global__ void cells_append_kernel(const int32_t * __restrict__ app, int n, int32_t * __restrict__ lists, size_t ld) {
    const int i = blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) lists[(size_t)app[3 * i] * ld + app[3 * i + 1]] = app[3 * i + 2];
}

bool bf16_mode(const LayerState * s) { return s->opts.compute == PI_TYPE_BF16; }

void drop_graph(LayerState * s) {
    if (s->exec) (void)hipGraphExecDestroy(s->exec);
    if (s->graph) (void)hipGraphDestroy(s->graph);
    s->exec = nullptr; s->graph = nullptr;
}

// ---- weights ---------------------------------------------------------------------------------------------------------------------
int want_tensor(const Tensor & t, int type, int64_t ne0, int64_t ne1, const char * what) {
    if (!t.dev || t.type != type || t.ne0 != ne0 || t.ne1 != ne1) {
        char msg[160];
        snprintf(msg, sizeof msg, "pi_model_finalize: %s must be %s of {%lld, %lld}", what, type == PI_TYPE_BF16 ? "BF16" : "F32", (long long)ne0, (long long)ne1);
        return pi::fail(PI_E_ARG, msg);
    }
    return PI_OK;
}

void release(pi_model * m, Tensor & t) {
    if (t.owned) for (auto & o : m->owned) if (o == t.dev) { pi_free(o); o = nullptr; }
    t.owned = false; t.dev = nullptr;
}

// rows of ld values, the tensor itself when it has that pitch already
int padded(pi_model * m, Tensor & t, int ld, const void ** out) {
    if (t.ne0 == ld) { *out = t.dev; return PI_OK; }
    uint16_t * p = m->alloc<uint16_t>((size_t)t.ne1 * ld);
    if (!p) return PI_E_HIP;
    PI_TRY(pi_k_pad_cols_bf16(t.dev, t.ne1, (int)t.ne0, p, ld, nullptr));
    PI_TRY(pi_sync());
    release(m, t);
    *out = p;
    return PI_OK;
}

// the weights of one of the model's norms with the offset of the design added, times a factor (the logit scale rides on the last norm)
int norm_weights(pi_model * m, const Tensor & t, float offset, float factor, const float ** out) {
    std::vector<float> w((size_t)t.ne0);
    PI_TRY(pi_memcpy_d2h(w.data(), t.dev, sizeof(float) * w.size()));
    for (float & v : w) v = (v + offset) * factor;
    float * p = m->alloc<float>(w.size());
    if (!p) return PI_E_HIP;
    PI_TRY(pi_memcpy_h2d(p, w.data(), sizeof(float) * w.size()));
    *out = p;
    return PI_OK;
}

// a matrix of the tensor's rows inside a larger one: rows row0, row0 + step, .., columns col0 .. col0 + width - 1
int place(pi_model * m, Tensor & t, uint16_t * out, int ld, int col0, int width, int64_t row0, int step) {
    PI_TRY(pi_k_place_bf16(t.dev, t.ne1, (int)t.ne0, out, ld, col0, width, row0, step, nullptr));
    PI_TRY(pi_sync());
    release(m, t);
    return PI_OK;
}

uint16_t * zeroed(pi_model * m, size_t n) {
    uint16_t * p = m->alloc<uint16_t>(n);
    return p && pi_memset(p, 0, n * 2) == PI_OK ? p : nullptr;
}

// a vector of n floats
int vec(pi_model * m, int il, int kind, int64_t n, const char * what, const float ** out) {
    PI_TRY(want_tensor(m->L(il, kind), PI_TYPE_F32, n, 1, what));
    *out = (const float *)m->L(il, kind).dev;
    return PI_OK;
}

// the experts of a layer: gate and up rows in turn
int expert_weights(pi_model * m, int il) {
    LayerState * s = m->lay;
    Layer & L = s->layers[il];
    const pi_layer_desc & d = L.d;
    const int D = m->hp.n_embd;
    const auto want = [&](int kind, int64_t ne0, int64_t ne1, const char * what) { return want_tensor(m->L(il, kind), PI_TYPE_BF16, ne0, ne1, what); };
    const int64_t ne = (int64_t)d.n_expert * d.expert_ff;
    uint16_t * up = zeroed(m, (size_t)2 * ne * s->d_ld);
    if (!up) return PI_E_HIP;
    PI_TRY(want(PI_T_EXPERT_GATE, D, ne, "expert_gate"));
    PI_TRY(want(PI_T_EXPERT_UP, D, ne, "expert_up"));
    PI_TRY(want(PI_T_EXPERT_DOWN, d.expert_ff, (int64_t)d.n_expert * D, "expert_down"));
    PI_TRY(place(m, m->L(il, PI_T_EXPERT_GATE), up, s->d_ld, 0, s->d_ld, 0, 2));
    PI_TRY(place(m, m->L(il, PI_T_EXPERT_UP), up, s->d_ld, 0, s->d_ld, 1, 2));
    L.up = up;
    return padded(m, m->L(il, PI_T_EXPERT_DOWN), L.ff_ld, &L.down);
}

// A layer with one norm: everything that reads the normed input is one matrix - the mixer's projections, gate and up rows of the dense or
// shared feed-forward (in turn), its score row, the router - and what closes the layer is one as well, [W_o | W_down].
int one_norm_weights(pi_model * m, int il) {
    LayerState * s = m->lay;
    Layer & L = s->layers[il];
    const pi_layer_desc & d = L.d;
    const int D = m->hp.n_embd, hv = d.n_head * d.vdim;
    const auto want = [&](int kind, int64_t ne0, int64_t ne1, const char * what) { return want_tensor(m->L(il, kind), PI_TYPE_BF16, ne0, ne1, what); };
    PI_TRY(want_tensor(m->L(il, PI_T_ATTN_NORM), PI_TYPE_F32, D, 1, "attn_norm"));
    PI_TRY(norm_weights(m, m->L(il, PI_T_ATTN_NORM), s->opts.norm_offset, 1.0f, &L.norm_a));
    uint16_t * z = zeroed(m, (size_t)L.z_rows * s->d_ld);
    if (!z) return PI_E_HIP;
    L.w_z = z;
    const auto rows = [&](int kind, int64_t n, int off, int step, const char * what) -> int {
        PI_TRY(want(kind, D, n, what));
        return place(m, m->L(il, kind), z, s->d_ld, 0, s->d_ld, off, step);
    };
    PI_TRY(rows(PI_T_MIX_Q, (int64_t)d.n_head * d.dim, 0, 1, "mix_q"));
    const bool grouped = d.mixer == PI_MIXER_GROUPED;
    const int64_t n_kv = grouped ? d.n_kv_head : d.n_head;
    PI_TRY(rows(PI_T_MIX_K, n_kv * d.dim, grouped ? L.off_k : L.rec.off_k, 1, "mix_k"));
    if (!grouped || L.off_v != L.off_k) PI_TRY(rows(PI_T_MIX_V, n_kv * d.vdim, grouped ? L.off_v : L.rec.off_v, 1, "mix_v"));
    if (L.rec.on()) {
        Rec & r = L.rec;
        PI_TRY(rows(PI_T_MIX_G, hv, r.off_g, 1, "mix_g"));
        PI_TRY(vec(m, il, PI_T_MIX_NORM, hv, "mix_norm", &r.norm));
        PI_TRY(vec(m, il, PI_T_MIX_DECAY, d.n_head, "mix_decay", &r.decay));
        const int C = pi_k_linear_chunk();
        std::vector<float> dec(d.n_head), pw((size_t)d.n_head * (C + 1));
        PI_TRY(pi_memcpy_d2h(dec.data(), r.decay, sizeof(float) * dec.size()));
        for (int h = 0; h < d.n_head; ++h) {
            double v = 1.0;
            for (int k = 0; k <= C; ++k, v *= dec[h]) pw[(size_t)h * (C + 1) + k] = (float)v;
        }
        float * p = m->alloc<float>(pw.size());
        if (!p) return PI_E_HIP;
        PI_TRY(pi_memcpy_h2d(p, pw.data(), sizeof(float) * pw.size()));
        r.powers = p;
    }
    uint16_t * close = zeroed(m, (size_t)D * L.close_ld);
    if (!close) return PI_E_HIP;
    L.wo = close;
    PI_TRY(want(PI_T_WO, hv, D, "wo"));
    PI_TRY(place(m, m->L(il, PI_T_WO), close, L.close_ld, 0, L.hv_ld, 0, 1));
    if (d.glu_ff > 0) {
        PI_TRY(rows(PI_T_GLU_GATE, d.glu_ff, L.off_glu, 2, "glu_gate"));
        PI_TRY(rows(PI_T_GLU_UP, d.glu_ff, L.off_glu + 1, 2, "glu_up"));
        PI_TRY(want(PI_T_GLU_DOWN, d.glu_ff, D, "glu_down"));
        PI_TRY(place(m, m->L(il, PI_T_GLU_DOWN), close, L.close_ld, L.hv_ld, L.glu_ld, 0, 1));
        if (L.off_score >= 0) PI_TRY(rows(PI_T_SHARED_SCORE, 1, L.off_score, 1, "shared_score"));
    }
    if (d.ffn != PI_FFN_GLU_MOE) return PI_OK;
    PI_TRY(rows(PI_T_ROUTER, d.n_expert, L.off_router, 1, "router"));
    return expert_weights(m, il);
}

// sizes and places that follow from the description of a layer with one norm
void one_norm_sizes(Layer & L) {
    const pi_layer_desc & d = L.d;
    int at = 0;
    const auto take = [&](int n) { const int o = at; at = up_to(at + n, 16); return o; };
    take(d.n_head * d.dim);
    if (d.mixer == PI_MIXER_GROUPED) {
        L.off_k = take(d.n_kv_head * d.dim);
        L.off_v = d.values_are_keys ? L.off_k : take(d.n_kv_head * d.vdim);
    } else {
        Rec & r = L.rec;
        r.off_k = take(d.n_head * d.dim);
        r.off_v = take(d.n_head * d.vdim);
        r.off_g = take(d.n_head * d.vdim);
    }
    if (d.glu_ff > 0) {
        L.off_glu = take(2 * d.glu_ff);
        if (d.ffn == PI_FFN_GLU_MOE) L.off_score = take(1);
    }
    if (d.ffn == PI_FFN_GLU_MOE) L.off_router = take(d.n_expert);
    L.z_rows = at;
    L.hv_ld = up_to(d.n_head * d.vdim, 128); L.glu_ld = d.glu_ff > 0 ? up_to(d.glu_ff, 128) : 0; L.close_ld = L.hv_ld + L.glu_ld;
    L.ff_ld = d.ffn == PI_FFN_GLU_MOE ? up_to(d.expert_ff, 64) : 0;
}

// A layer whose norms come after the sums: what the mixer projects and the gate of its residual are one matrix, what closes the mixer is one
// ([W_o | W_o of the memory]), gate and up rows of the feed-forward and the gate of its residual are one.
int post_norm_weights(pi_model * m, int il) {
    LayerState * s = m->lay;
    Layer & L = s->layers[il];
    const pi_layer_desc & d = L.d;
    Rec & r = L.rec;
    const int D = m->hp.n_embd, hv = d.n_head * d.vdim;
    const auto want = [&](int kind, int64_t ne0, int64_t ne1, const char * what) { return want_tensor(m->L(il, kind), PI_TYPE_BF16, ne0, ne1, what); };
    PI_TRY(want_tensor(m->L(il, PI_T_ATTN_NORM), PI_TYPE_F32, D, 1, "attn_norm"));
    PI_TRY(norm_weights(m, m->L(il, PI_T_ATTN_NORM), s->opts.norm_offset, 1.0f, &L.norm_a));
    uint16_t * z = zeroed(m, (size_t)L.z_rows * s->d_ld), * close = zeroed(m, (size_t)D * L.close_ld);
    if (!z || !close) return PI_E_HIP;
    L.w_z = z; L.wo = close;
    const auto rows = [&](uint16_t * to, int kind, int64_t n, int off, int step, const char * what) -> int {
        PI_TRY(want(kind, D, n, what));
        return place(m, m->L(il, kind), to, s->d_ld, 0, s->d_ld, off, step);
    };
    const bool grouped = d.mixer == PI_MIXER_GROUPED;
    PI_TRY(rows(z, PI_T_MIX_Q, (int64_t)d.n_head * d.dim, 0, 1, "mix_q"));
    if (grouped) {
        PI_TRY(rows(z, PI_T_MIX_K, (int64_t)d.n_kv_head * d.dim, L.off_k, 1, "mix_k"));
        if (L.off_v != L.off_k) PI_TRY(rows(z, PI_T_MIX_V, (int64_t)d.n_kv_head * d.vdim, L.off_v, 1, "mix_v"));
        if (d.qk_norm) { PI_TRY(vec(m, il, PI_T_MIX_Q_NORM, d.dim, "mix_q_norm", &L.q_norm)); PI_TRY(vec(m, il, PI_T_MIX_K_NORM, d.dim, "mix_k_norm", &L.k_norm)); }
        if (d.head_temp) PI_TRY(vec(m, il, PI_T_MIX_TEMP, d.n_head, "mix_temp", &L.temp));
    } else {
        PI_TRY(rows(z, PI_T_MIX_K, (int64_t)d.n_head * d.dim, r.off_k, 1, "mix_k"));
        PI_TRY(rows(z, PI_T_MIX_V, hv, r.off_v, 1, "mix_v"));
        PI_TRY(rows(z, PI_T_MIX_G, hv, r.off_g, 1, "mix_g"));
        PI_TRY(rows(z, PI_T_MIX_A1, r.rank, r.off_a, 1, "mix_a1"));
        PI_TRY(want(PI_T_MIX_A2, r.rank, (int64_t)d.n_head * d.dim, "mix_a2"));
        PI_TRY(padded(m, m->L(il, PI_T_MIX_A2), r.rank_ld, &r.a2));
        PI_TRY(vec(m, il, PI_T_MIX_A2_B, (int64_t)d.n_head * d.dim, "mix_a2_b", &r.a2_b));
        PI_TRY(vec(m, il, PI_T_MIX_NORM, hv, "mix_norm", &r.norm));
    }
    PI_TRY(want(PI_T_WO, hv, D, "wo"));
    PI_TRY(place(m, m->L(il, PI_T_WO), close, L.close_ld, 0, L.hv_ld, 0, 1));
    if (grouped && r.on()) {
        const int64_t hk = (int64_t)r.n_head * r.dim, mv = (int64_t)r.n_head * r.vdim;
        PI_TRY(rows(z, PI_T_MEM_Q, hk, r.off_q, 1, "mem_q"));
        PI_TRY(rows(z, PI_T_MEM_K, hk, r.off_k, 1, "mem_k"));
        PI_TRY(rows(z, PI_T_MEM_V, mv, r.off_v, 1, "mem_v"));
        PI_TRY(rows(z, PI_T_MEM_G, mv, r.off_g, 1, "mem_g"));
        PI_TRY(rows(z, PI_T_MEM_I, r.n_head, r.off_i, 1, "mem_i"));
        PI_TRY(rows(z, PI_T_MEM_F, r.n_head, r.off_f, 1, "mem_f"));
        PI_TRY(vec(m, il, PI_T_MEM_I_B, r.n_head, "mem_i_b", &r.i_b));
        PI_TRY(vec(m, il, PI_T_MEM_F_B, r.n_head, "mem_f_b", &r.f_b));
        PI_TRY(vec(m, il, PI_T_MEM_NORM, mv, "mem_norm", &r.norm));
        PI_TRY(want(PI_T_MEM_O, mv, D, "mem_o"));
        PI_TRY(place(m, m->L(il, PI_T_MEM_O), close, L.close_ld, r.off_att, L.close_ld - r.off_att, 0, 1));
    }
    if (d.gated_residual) {
        PI_TRY(rows(z, PI_T_RES_GATE, D, L.off_gate, 1, "res_gate"));
        PI_TRY(vec(m, il, PI_T_RES_GATE_B, D, "res_gate_b", &L.gate_b));
    }
    if (d.ffn == PI_FFN_NONE) return PI_OK;
    PI_TRY(want_tensor(m->L(il, PI_T_FFN_NORM), PI_TYPE_F32, D, 1, "ffn_norm"));
    PI_TRY(norm_weights(m, m->L(il, PI_T_FFN_NORM), s->opts.norm_offset, 1.0f, &L.norm_b));
    uint16_t * f = zeroed(m, (size_t)L.z2_rows * s->d_ld);
    if (!f) return PI_E_HIP;
    L.w_ffn = f;
    PI_TRY(rows(f, PI_T_GLU_GATE, d.glu_ff, 0, 2, "glu_gate"));
    PI_TRY(rows(f, PI_T_GLU_UP, d.glu_ff, 1, 2, "glu_up"));
    if (d.gated_residual) {
        PI_TRY(rows(f, PI_T_RES_GATE_FFN, D, L.off_gate_ffn, 1, "res_gate_ffn"));
        PI_TRY(vec(m, il, PI_T_RES_GATE_FFN_B, D, "res_gate_ffn_b", &L.gate_ffn_b));
    }
    PI_TRY(want(PI_T_GLU_DOWN, d.glu_ff, D, "glu_down"));
    return padded(m, m->L(il, PI_T_GLU_DOWN), L.glu_ld, &L.down);
}

void post_norm_sizes(Layer & L, int D) {
    const pi_layer_desc & d = L.d;
    Rec & r = L.rec;
    int at = 0;
    const auto take = [&](int n) { const int o = at; at = up_to(at + n, 16); return o; };
    take(d.n_head * d.dim);
    L.hv_ld = up_to(d.n_head * d.vdim, 128); L.close_ld = L.hv_ld;
    if (d.mixer == PI_MIXER_GROUPED) {
        L.off_k = take(d.n_kv_head * d.dim);
        L.off_v = d.values_are_keys ? L.off_k : take(d.n_kv_head * d.vdim);
        if (r.on()) r.off_q = take(r.n_head * r.dim);
        r.off_att = L.hv_ld;
        if (r.on()) L.close_ld += up_to(r.n_head * r.vdim, 128);
    }
    if (r.on()) {
        r.off_k = take(r.n_head * r.dim);
        r.off_v = take(r.n_head * r.vdim);
        r.off_g = take(r.n_head * r.vdim);
        if (r.kind == PI_DECAY_KEYED) r.off_a = take(r.rank);
        else { r.off_i = take(r.n_head); r.off_f = take(r.n_head); }
    }
    if (d.gated_residual) L.off_gate = take(D);
    L.z_rows = at;
    if (d.ffn == PI_FFN_NONE) return;
    L.off_gate_ffn = up_to(2 * d.glu_ff, 16);
    L.z2_rows = L.off_gate_ffn + (d.gated_residual ? up_to(D, 16) : 0);
    L.glu_ld = up_to(d.glu_ff, 128);
}

// A layer with norms before and after its sublayers: what the mixer projects and the gates of its heads are one matrix.
int both_norms_weights(pi_model * m, int il) {
    LayerState * s = m->lay;
    Layer & L = s->layers[il];
    const pi_layer_desc & d = L.d;
    const int D = m->hp.n_embd, hv = d.n_head * d.vdim;
    const auto want = [&](int kind, int64_t ne0, int64_t ne1, const char * what) { return want_tensor(m->L(il, kind), PI_TYPE_BF16, ne0, ne1, what); };
    const auto norm = [&](int kind, const char * what, const float ** out) -> int {
        PI_TRY(want_tensor(m->L(il, kind), PI_TYPE_F32, D, 1, what));
        return norm_weights(m, m->L(il, kind), s->opts.norm_offset, 1.0f, out);
    };
    PI_TRY(norm(PI_T_ATTN_NORM, "attn_norm", &L.norm_a));
    PI_TRY(norm(PI_T_ATTN_NORM_AFTER, "attn_norm_after", &L.norm_a_after));
    if (s->opts.conv_taps > 0) {
        PI_TRY(want_tensor(m->L(il, PI_T_MIX_CONV), PI_TYPE_F32, D, s->opts.conv_taps, "mix_conv"));
        L.conv = (const float *)m->L(il, PI_T_MIX_CONV).dev;
    }
    uint16_t * z = zeroed(m, (size_t)L.z_rows * s->d_ld);
    if (!z) return PI_E_HIP;
    L.w_z = z;
    const auto rows = [&](int kind, int64_t n, int off, const char * what) -> int {
        PI_TRY(want(kind, D, n, what));
        return place(m, m->L(il, kind), z, s->d_ld, 0, s->d_ld, off, 1);
    };
    PI_TRY(rows(PI_T_MIX_Q, (int64_t)d.n_head * d.dim, 0, "mix_q"));
    PI_TRY(rows(PI_T_MIX_K, (int64_t)d.n_kv_head * d.dim, L.off_k, "mix_k"));
    if (L.off_v != L.off_k) PI_TRY(rows(PI_T_MIX_V, (int64_t)d.n_kv_head * d.vdim, L.off_v, "mix_v"));
    if (d.head_gate) PI_TRY(rows(PI_T_MIX_HEAD_GATE, d.n_head, L.off_head_gate, "mix_head_gate"));
    if (d.qk_norm) { PI_TRY(vec(m, il, PI_T_MIX_Q_NORM, d.dim, "mix_q_norm", &L.q_norm)); PI_TRY(vec(m, il, PI_T_MIX_K_NORM, d.dim, "mix_k_norm", &L.k_norm)); }
    if (d.head_temp) PI_TRY(vec(m, il, PI_T_MIX_TEMP, d.n_head, "mix_temp", &L.temp));
    if (d.head_sinks) PI_TRY(vec(m, il, PI_T_MIX_SINK, d.n_head, "mix_sink", &L.sink));
    if (d.head_mix) {
        PI_TRY(want_tensor(m->L(il, PI_T_MIX_TALK), PI_TYPE_F32, d.n_head, d.n_head, "mix_talk"));
        L.talk = (const float *)m->L(il, PI_T_MIX_TALK).dev;
    }
    if (d.value_mix && !L.first_values) PI_TRY(vec(m, il, PI_T_MIX_VALUE, 1, "mix_value", &L.v_mix));
    PI_TRY(want(PI_T_WO, hv, D, "wo"));
    PI_TRY(padded(m, m->L(il, PI_T_WO), L.close_ld, &L.wo));
    if (d.ffn == PI_FFN_NONE) return PI_OK;
    PI_TRY(norm(PI_T_FFN_NORM, "ffn_norm", &L.norm_b));
    PI_TRY(norm(PI_T_FFN_NORM_AFTER, "ffn_norm_after", &L.norm_b_after));
    PI_TRY(want(PI_T_ROUTER, D, d.n_expert, "router"));
    PI_TRY(padded(m, m->L(il, PI_T_ROUTER), s->d_ld, &L.router));
    return expert_weights(m, il);
}

void both_norms_sizes(Layer & L) {
    const pi_layer_desc & d = L.d;
    int at = 0;
    const auto take = [&](int n) { const int o = at; at = up_to(at + n, 16); return o; };
    take(d.n_head * d.dim);
    L.off_k = take(d.n_kv_head * d.dim);
    L.off_v = d.values_are_keys ? L.off_k : take(d.n_kv_head * d.vdim);
    if (d.head_gate) L.off_head_gate = take(d.n_head);
    L.z_rows = at;
    L.hv_ld = L.close_ld = up_to(d.n_head * d.vdim, 128);
    L.ff_ld = d.ffn == PI_FFN_GLU_MOE ? up_to(d.expert_ff, 64) : 0;
}

// the recurrent part that a description asks for
Rec recurrent_part(const pi_layer_desc & d) {
    Rec r;
    if (d.mixer == PI_MIXER_LINEAR || d.mixer == PI_MIXER_KEYED) { r.n_head = d.n_head; r.dim = d.dim; r.vdim = d.vdim; }
    if (d.mixer == PI_MIXER_LINEAR) r.kind = PI_DECAY_CONST;
    if (d.mixer == PI_MIXER_KEYED) {
        r.kind = PI_DECAY_KEYED;
        r.rank = d.decay_rank; r.rank_ld = up_to(d.decay_rank, 8); r.tau = d.decay_tau; r.silu = true;
    }
    if (d.mixer == PI_MIXER_GROUPED && d.mem_heads > 0) {
        r.kind = PI_DECAY_GATED;
        r.n_head = d.mem_heads; r.dim = d.mem_dim; r.vdim = d.mem_vdim; r.cap = d.mem_cap; r.scale = d.mem_scale;
    }
    r.plain = r.per_head = r.kind > PI_DECAY_CONST;
    if (r.plain) r.q_scale = 1.0f / sqrtf((float)r.dim);
    r.dim_ld = up_to(r.dim, 32); r.vdim_ld = up_to(r.vdim, 64);
    return r;
}

int layer_weights(pi_model * m, int il) {
    LayerState * s = m->lay;
    Layer & L = s->layers[il];
    const pi_layer_desc & d = L.d;
    const int D = m->hp.n_embd;
    PI_TRY(want_tensor(m->L(il, PI_T_ATTN_NORM), PI_TYPE_F32, D, 1, "attn_norm"));
    PI_TRY(norm_weights(m, m->L(il, PI_T_ATTN_NORM), s->opts.norm_offset, 1.0f, &L.norm_a));
    Tensor & q = m->L(il, PI_T_MIX_Q); Tensor & dkv = m->L(il, PI_T_MIX_DKV);
    PI_TRY(want_tensor(q, PI_TYPE_BF16, D, L.nq, "mix_q"));
    if (L.own_kv) {
        PI_TRY(want_tensor(dkv, PI_TYPE_BF16, D, d.kv_rank + d.rot_dim, "mix_dkv"));
        PI_TRY(want_tensor(m->L(il, PI_T_MIX_DKV_NORM), PI_TYPE_F32, d.kv_rank, 1, "mix_dkv_norm"));
        L.dkv_norm = (const float *)m->L(il, PI_T_MIX_DKV_NORM).dev;
        // one matrix, so that one mat-mul gives the queries and the cell
        uint16_t * w = m->alloc<uint16_t>((size_t)L.z_rows * s->d_ld);
        if (!w) return PI_E_HIP;
        PI_TRY(pi_k_pad_cols_bf16(q.dev, q.ne1, D, w, s->d_ld, nullptr));
        PI_TRY(pi_k_pad_cols_bf16(dkv.dev, dkv.ne1, D, w + (size_t)L.nq * s->d_ld, s->d_ld, nullptr));
        PI_TRY(pi_sync());
        release(m, q); release(m, dkv);
        L.w_z = w;
    } else {
        PI_TRY(padded(m, q, s->d_ld, &L.w_z));
    }
    Tensor & uk = m->L(il, PI_T_MIX_UK); Tensor & uv = m->L(il, PI_T_MIX_UV);
    PI_TRY(want_tensor(uk, PI_TYPE_BF16, d.kv_rank, (int64_t)d.n_head * d.dim, "mix_uk"));
    PI_TRY(want_tensor(uv, PI_TYPE_BF16, d.kv_rank, (int64_t)d.n_head * d.vdim, "mix_uv"));
    uint16_t * ukt = m->alloc<uint16_t>((size_t)d.n_head * d.kv_rank * L.dim_ld);
    if (!ukt) return PI_E_HIP;
    PI_TRY(pi_k_transpose_pad_bf16(uk.dev, d.n_head, d.dim, d.kv_rank, ukt, L.dim_ld, nullptr));
    PI_TRY(pi_sync());
    L.uk_t = ukt;
    PI_TRY(padded(m, uk, L.rank_ld, &L.uk));         // as it is, for the expanded keys of long prompt portions
    PI_TRY(padded(m, uv, L.rank_ld, &L.uv));
    PI_TRY(want_tensor(m->L(il, PI_T_MIX_SINK), PI_TYPE_F32, d.n_head, 1, "mix_sink"));
    L.sink = (const float *)m->L(il, PI_T_MIX_SINK).dev;
    PI_TRY(want_tensor(m->L(il, PI_T_WO), PI_TYPE_BF16, (int64_t)d.n_head * d.vdim, D, "wo"));
    PI_TRY(padded(m, m->L(il, PI_T_WO), L.hv_ld, &L.wo));
    if (d.ffn == PI_FFN_NONE) return PI_OK;
    PI_TRY(want_tensor(m->L(il, PI_T_FFN_NORM), PI_TYPE_F32, D, 1, "ffn_norm"));
    PI_TRY(norm_weights(m, m->L(il, PI_T_FFN_NORM), s->opts.norm_offset, 1.0f, &L.norm_b));
    PI_TRY(want_tensor(m->L(il, PI_T_ROUTER), PI_TYPE_BF16, D, d.n_expert, "router"));
    PI_TRY(want_tensor(m->L(il, PI_T_ROUTER_BIAS), PI_TYPE_F32, d.n_expert, 1, "router_bias"));
    PI_TRY(want_tensor(m->L(il, PI_T_EXPERT_UP), PI_TYPE_BF16, D, (int64_t)d.n_expert * d.expert_ff, "expert_up"));
    PI_TRY(want_tensor(m->L(il, PI_T_EXPERT_DOWN), PI_TYPE_BF16, d.expert_ff, (int64_t)d.n_expert * D, "expert_down"));
    L.bias = (const float *)m->L(il, PI_T_ROUTER_BIAS).dev;
    PI_TRY(padded(m, m->L(il, PI_T_ROUTER), s->d_ld, &L.router));
    PI_TRY(padded(m, m->L(il, PI_T_EXPERT_UP), s->d_ld, &L.up));
    PI_TRY(padded(m, m->L(il, PI_T_EXPERT_DOWN), L.ff_ld, &L.down));
    return PI_OK;
}

// ---- step buffers ----------------------------------------------------------------------------------------------------------------
int ensure_capacity(pi_model * m, int T) {
    LayerState * s = m->lay;
    if (T <= s->cap) return PI_OK;
    int cap = 64;
    while (cap < T) cap *= 2;
    const size_t es = s->es, D = m->hp.n_embd;
    size_t z = 0, qu = 0, ql = 0, ol = 0, at = 0, E = 0, top = 0, ff = 0, lq = 0, lv = 0, lo = 0, ls = 0, ln = 0, lg = 0, hr = 0, vf = 0, sh = 0;
    const size_t chunks = s->recurrent && bf16_mode(s) ? (size_t)cap / pi_k_linear_chunk() + 32 : 0;        // every run of a pass ends with a part of one
    for (const Layer & L : s->layers) {
        const pi_layer_desc & d = L.d;
        if (s->family != kTwoNorms) {
            z = std::max({z, (size_t)L.z_rows, (size_t)L.z2_rows}); at = std::max({at, (size_t)L.close_ld, (size_t)L.glu_ld});
            if (d.mixer == PI_MIXER_GROUPED) ql = std::max(ql, (size_t)d.n_head * L.hd);
            if (L.heads_apart()) hr = std::max(hr, (size_t)d.n_head * d.n_kv_head * d.vdim);
            if (L.heads_apart()) sh = std::max(sh, (size_t)d.n_head);
            if (d.value_mix) vf = std::max(vf, (size_t)d.n_kv_head * d.vdim);
            const Rec & r = L.rec;
            if (r.on()) {
                lo = std::max(lo, (size_t)r.n_head * r.vdim);
                if (r.kind == PI_DECAY_GATED) ln = std::max(ln, (size_t)r.n_head);
                if (chunks) {
                    lq = std::max(lq, (size_t)r.n_head * r.dim_ld); lv = std::max(lv, (size_t)r.n_head * r.vdim_ld);
                    ls = std::max(ls, pi_k_linear_states_bytes((int)chunks, r.n_head, r.dim_ld, r.vdim_ld));
                    lg = std::max(lg, pi_k_linear_gate_floats(r.kind, cap, (int)chunks, r.n_head, r.dim_ld));
                }
            }
            if (L.moe()) { E = std::max(E, (size_t)d.n_expert); top = std::max(top, (size_t)d.n_top); ff = std::max(ff, (size_t)d.n_top * L.ff_ld); }
            continue;
        }
        z = std::max(z, (size_t)L.z_rows); qu = std::max(qu, (size_t)d.n_head * L.dim_ld); ql = std::max(ql, (size_t)d.n_head * L.kd);
        ol = std::max(ol, (size_t)d.n_head * L.rank_ld); at = std::max(at, (size_t)L.hv_ld);
        if (d.ffn == PI_FFN_MOE) { E = std::max(E, (size_t)d.n_expert); top = std::max(top, (size_t)d.n_top); ff = std::max(ff, (size_t)d.n_top * L.ff_ld); }
    }
    PI_HIP_TRY(hipStreamSynchronize(m->stream));
    drop_graph(s);
    if (s->arena) { pi_free(s->arena); s->arena = nullptr; s->cap = 0; }
    // carved twice: once to learn the size, once to hand out addresses
    size_t used = 0;
    auto carve = [&](auto *& p, size_t bytes) {
        using P = std::remove_reference_t<decltype(p)>;
        p = reinterpret_cast<P>(s->arena ? s->arena + used : nullptr);
        used += (bytes + 255) / 256 * 256;
    };
    auto lay_out = [&]() {
        used = 0;
        const size_t n = cap;
        carve(s->x, n * D * 4); carve(s->x2, n * D * 4); carve(s->mix, n * D * 4); carve(s->z, n * z * 4);
        carve(s->h_a, n * s->d_ld * es); carve(s->h_b, n * s->d_ld * es);
        carve(s->q_un, n * qu * es); carve(s->q_lat, n * ql * es); carve(s->o_lat, n * ol * es); carve(s->att, n * at * es);
        carve(s->rl, n * E * 4); carve(s->wts, n * top * 4); carve(s->ids, n * top * 4); carve(s->perm, n * top * 4); carve(s->inv, n * top * 4);
        carve(s->off, (E + 1) * 4); carve(s->act, n * ff * es); carve(s->y_exp, n * top * D * es);
        carve(s->tiles, (n * top / 64 + E + 1) * 8); carve(s->n_tiles, 4);
        carve(s->x0, s->opts.loop_times > 0 ? n * D * 4 : 0);
        carve(s->lin_o, n * lo * 4); carve(s->lin_q, n * lq * 2); carve(s->lin_k, n * lq * 2); carve(s->lin_v, n * lv * 2); carve(s->lin_states, ls);
        carve(s->lin_den, n * ln * 4); carve(s->lin_gates, lg * 4); carve(s->heads, n * hr * 4); carve(s->v_first, n * vf * 4); carve(s->stats, n * sh * 4);
        s->cs.resize(s->rots.size());
        for (size_t r = 0; r < s->rots.size(); ++r) carve(s->cs[r], n * s->rots[r].dims * 4);
    };
    lay_out();
    s->arena = (unsigned char *)pi_malloc(used);
    if (!s->arena) return PI_E_HIP;
    lay_out();
    PI_TRY(pi_memset(s->arena, 0, used));           // the padding columns of the operands stay zero or finite from here on
    PI_TRY(pi_sync());
    s->cap = cap;
    return PI_OK;
}

int ensure_inputs(pi_model * m, size_t n) {
    LayerState * s = m->lay;
    if (n <= s->in_cap) return PI_OK;
    PI_HIP_TRY(hipStreamSynchronize(m->stream));
    if (s->h_in) { (void)hipHostFree(s->h_in); s->h_in = nullptr; }
    if (s->d_in) { pi_free(s->d_in); s->d_in = nullptr; }
    s->in_cap = 0;
    size_t c = 4096;
    while (c < n) c *= 2;
    PI_HIP_TRY(hipHostMalloc((void **)&s->h_in, c * 4, hipHostMallocDefault));
    s->d_in = (int32_t *)pi_malloc(c * 4);
    if (!s->d_in) return PI_E_HIP;
    s->in_cap = c;
    return PI_OK;
}

// room for the expanded keys and values of a pass's longest run
int ensure_expanded(pi_model * m, const Step & in) {
    LayerState * s = m->lay;
    size_t need = 0;
    for (size_t k = 0; k < in.runs.size(); ++k)
        for (const Step::Run & r : in.runs[k]) need = std::max(need, (size_t)r.n_cells * s->kinds[k].n_head * (s->kinds[k].dim + s->kinds[k].vdim) + 128);
    if (need <= s->expanded_cap) return PI_OK;
    PI_HIP_TRY(hipStreamSynchronize(m->stream));
    if (s->expanded) { pi_free(s->expanded); s->expanded = nullptr; s->expanded_cap = 0; }
    need += need / 4;                                              // a prompt that grows portion by portion asks again less often
    s->expanded = (bf16_t *)pi_malloc(need * sizeof(bf16_t));
    if (!s->expanded) return PI_E_HIP;
    s->expanded_cap = need;
    return PI_OK;
}

// ---- one pass over the layers ----------------------------------------------------------------------------------------------------
// y [T][rows] = W x, x rows of `cols` values.  bf16: the mat-muls the other models run (steps of up to 16 tokens, LDS tiles, and
// hipBLASLt plans for large products)
int dense(pi_model * m, const void * W, int rows, int cols, const void * x, int T, float * y) {
    LayerState * s = m->lay;
    hipStream_t st = m->stream;
    if (!bf16_mode(s)) {
        pi_group_gemm g{};
        g.W = W; g.rows = rows; g.cols = cols; g.ldw = cols; g.n_group = 1; g.x = x; g.ldx = cols; g.T = T; g.y = y; g.ldy = rows; g.y_f32 = 1; g.alpha = 1.0f;
        return pi_k_group_gemm(s->opts.compute, &g, st);
    }
    if (T <= 16) return pi_k_gemm_bf16(W, rows, cols, x, T, PI_EPI_NONE, nullptr, nullptr, y, nullptr, st);
    const char * own = getenv("PI_PREFILL_GEMM");
    if (T >= 256 && rows >= 1024 && cols >= 1024 && !(own && !strcmp(own, "own"))) {
        if (!m->gemm_lib) {
            m->gemm_lib = pi_gemm_lib_create((size_t)64 << 20);
            if (!m->gemm_lib) return PI_E_HIP;
        }
        const int rc = pi_gemm_lib_bf16(m->gemm_lib, W, rows, cols, x, T, PI_EPI_NONE, nullptr, nullptr, y, nullptr, st);
        if (rc != PI_E_UNSUPPORTED) return rc;
    }
    return pi_k_gemm_tile_bf16(W, rows, cols, x, T, PI_EPI_NONE, nullptr, nullptr, y, nullptr, 0, st);
}

int grouped(LayerState * s, const pi_group_gemm & g, int tile_n, hipStream_t st) {
    return bf16_mode(s) && g.T > 16 ? pi_k_group_gemm_tile(&g, tile_n, st) : pi_k_group_gemm(s->opts.compute, &g, st);
}

pi_latent_prep prep_args(pi_model * m, const Layer & L, const Step & in) {
    LayerState * s = m->lay;
    const pi_layer_desc & d = L.d;
    pi_latent_prep p{};
    p.z = s->z; p.ldz = L.z_rows; p.T = in.T; p.n_head = d.n_head; p.dim = d.dim; p.dim_ld = L.dim_ld; p.rot_dim = d.rot_dim; p.kv_rank = d.kv_rank;
    p.rank_ld = L.rank_ld; p.kd = L.kd; p.cs = s->cs[L.rot]; p.norm_w = L.dkv_norm; p.eps = m->hp.norm_eps; p.q_un = s->q_un; p.q_lat = s->q_lat;
    p.cache = L.own_kv ? L.cache[0] : nullptr; p.cell = in.cell;
    return p;
}

pi_latent_attn attn_args(pi_model * m, const Layer & L, const Layer & src, const Step & in) {
    LayerState * s = m->lay;
    const pi_layer_desc & d = L.d;
    pi_latent_attn a{};
    a.q_lat = s->q_lat; a.cache = src.cache[0]; a.lists = s->lists; a.list_ld = s->kv.n; a.work = bf16_mode(s) ? in.work[L.hc].items : in.seq; a.n_vis = in.n_vis;
    a.n_work = in.work[L.hc].n; a.T = in.T; a.n_head = d.n_head; a.kv_rank = d.kv_rank; a.rank_ld = L.rank_ld; a.kd = L.kd; a.n_parts = in.work[L.hc].parts; a.scale = d.scale;
    a.sink = L.sink; a.scratch = s->scratch; a.out_lat = s->o_lat;
    return a;
}

int attend_latent(pi_model * m, const Layer & L, const Layer & src, const Step & in) {
    LayerState * s = m->lay;
    const pi_layer_desc & d = L.d;
    const int type = s->opts.compute, T = in.T;
    hipStream_t st = m->stream;
    pi_group_gemm g{};                              // each head's query in latent coordinates
    g.W = L.uk_t; g.w_gs = (size_t)d.kv_rank * L.dim_ld; g.rows = d.kv_rank; g.cols = L.dim_ld; g.ldw = L.dim_ld; g.n_group = d.n_head; g.alpha = 1.0f;
    g.x = s->q_un; g.x_gs = L.dim_ld; g.ldx = d.n_head * L.dim_ld; g.T = T; g.y = s->q_lat; g.y_gs = L.kd; g.ldy = d.n_head * L.kd;
    PI_TRY(grouped(s, g, T > 64 ? 128 : 64, st));
    const pi_latent_attn a = attn_args(m, L, src, in);
    PI_TRY(pi_k_latent_attn(type, &a, st));
    pi_group_gemm v{};                              // each head's value from its weighted latent
    v.W = L.uv; v.w_gs = (size_t)d.vdim * L.rank_ld; v.rows = d.vdim; v.cols = L.rank_ld; v.ldw = L.rank_ld; v.n_group = d.n_head; v.alpha = 1.0f;
    v.x = s->o_lat; v.x_gs = L.rank_ld; v.ldx = d.n_head * L.rank_ld; v.T = T; v.y = s->att; v.y_gs = d.vdim; v.ldy = L.hv_ld;
    return grouped(s, v, T > 64 ? 128 : 64, st);
}

// one long run over the expanded keys and values of its cells
int attend_expanded(pi_model * m, const Layer & L, const Layer & src, const Step & in, const Step::Run & r) {
    LayerState * s = m->lay;
    const pi_layer_desc & d = L.d;
    hipStream_t st = m->stream;
    const int32_t * list = s->lists + (size_t)r.seq * s->kv.n;
    const size_t nk = (size_t)d.n_head * d.dim, nv = (size_t)d.n_head * d.vdim, keys = ((size_t)r.n_cells * nk + 127) / 128 * 128;
    bf16_t * k = s->expanded, * v = s->expanded + keys;
    pi_group_gemm g{};
    g.W = L.uk; g.rows = (int)nk; g.cols = L.rank_ld; g.ldw = L.rank_ld; g.n_group = 1; g.x = src.cache[0]; g.ldx = L.kd; g.T = r.n_cells; g.y = k; g.ldy = (int)nk;
    g.alpha = 1.0f; g.gather = list; g.gather_div = 1;
    PI_TRY(pi_k_group_gemm_tile(&g, 128, st));
    g.W = L.uv; g.rows = (int)nv; g.y = v; g.ldy = (int)nv;
    PI_TRY(pi_k_group_gemm_tile(&g, 128, st));
    pi_latent_expanded a{};
    a.q_un = s->q_un; a.q_lat = s->q_lat; a.keys = k; a.values = v; a.cache = src.cache[0]; a.list = list; a.n_vis = in.n_vis; a.sink = L.sink; a.att = s->att;
    a.tok0 = r.tok0; a.T = r.T; a.n_head = d.n_head; a.dim = d.dim; a.dim_ld = L.dim_ld; a.rot_dim = d.rot_dim; a.vdim = d.vdim; a.rank_ld = L.rank_ld; a.kd = L.kd;
    a.ld_att = L.hv_ld; a.scale = d.scale;
    return pi_k_latent_attn_expanded(&a, st);
}

int mix_latent(pi_model * m, Layer & L, const Step & in) {
    LayerState * s = m->lay;
    const pi_layer_desc & d = L.d;
    const int type = s->opts.compute, T = in.T;
    hipStream_t st = m->stream;
    Layer & src = L.own_kv ? L : s->layers[d.kv_from];
    PI_TRY(dense(m, L.w_z, L.z_rows, s->d_ld, s->h_a, T, s->z));
    const pi_latent_prep p = prep_args(m, L, in);
    PI_TRY(pi_k_latent_prep(type, &p, st));
    if (in.work[L.hc].n > 0) PI_TRY(attend_latent(m, L, src, in));
    if (bf16_mode(s)) for (const Step::Run & r : in.runs[L.hc]) PI_TRY(attend_expanded(m, L, src, in, r));
    return dense(m, L.wo, m->hp.n_embd, L.hv_ld, s->att, T, s->mix);
}

// the experts of the chosen pairs (s->ids): relu^2 or, with a gate, clamped GLU in between; s->y_exp holds a row per pair, in expert order
int experts(pi_model * m, Layer & L, const void * h, const Step & in) {
    LayerState * s = m->lay;
    const pi_layer_desc & d = L.d;
    const int T = in.T, D = m->hp.n_embd, per = d.ffn == PI_FFN_GLU_MOE ? 2 : 1;
    hipStream_t st = m->stream;
    const int tile_n = (long long)T * d.n_top > 96LL * d.n_expert ? 128 : 64;       // tokens per tile, by the tokens an expert has on average
    PI_TRY(pi_k_moe_sort(s->ids, T * d.n_top, d.n_expert, s->off, s->perm, s->inv, tile_n, s->tiles, s->n_tiles, st));
    pi_group_gemm g{};
    g.W = L.up; g.w_gs = (size_t)per * d.expert_ff * s->d_ld; g.rows = per * d.expert_ff; g.cols = s->d_ld; g.ldw = s->d_ld; g.n_group = d.n_expert; g.alpha = 1.0f;
    if (per == 2) { g.glu = 1; g.glu_limit = d.expert_limit; g.glu_gain = d.glu_gain; g.glu_plain_up = d.glu_plain_up; }
    else g.relu2 = 1;
    g.x = h; g.ldx = s->d_ld; g.T = T; g.y = s->act; g.ldy = L.ff_ld; g.off = s->off; g.gather = s->perm; g.gather_div = d.n_top;
    g.tiles = s->tiles; g.n_tiles = s->n_tiles; g.max_tiles = T * d.n_top / tile_n + d.n_expert;
    g.pair_w = d.weigh_input ? s->wts : nullptr;
    PI_TRY(grouped(s, g, tile_n, st));
    pi_group_gemm w{};
    w.W = L.down; w.w_gs = (size_t)D * L.ff_ld; w.rows = D; w.cols = L.ff_ld; w.ldw = L.ff_ld; w.n_group = d.n_expert; w.alpha = 1.0f;
    w.x = s->act; w.ldx = L.ff_ld; w.T = T; w.y = s->y_exp; w.ldy = D; w.off = s->off; w.tiles = s->tiles; w.n_tiles = s->n_tiles; w.max_tiles = g.max_tiles;
    return grouped(s, w, tile_n, st);
}

int ffn_moe(pi_model * m, Layer & L, const Step & in) {
    LayerState * s = m->lay;
    const pi_layer_desc & d = L.d;
    PI_TRY(dense(m, L.router, d.n_expert, s->d_ld, s->h_b, in.T, s->rl));
    PI_TRY(pi_k_route(s->rl, in.T, d.n_expert, d.n_top, d.n_group, d.n_group_keep, L.bias, s->ids, s->wts, m->stream));
    return experts(m, L, s->h_b, in);
}

// grouped-query attention over one list of work items
pi_gqa_attn gqa_args(pi_model * m, const Layer & L, int pass, const Step & in, const Step::Work & w, int wide) {
    LayerState * s = m->lay;
    const pi_layer_desc & d = L.d;
    pi_gqa_attn a{};
    a.q = s->q_lat; a.cache = L.cache[pass]; a.lists = s->lists; a.list_ld = s->kv.n; a.work = bf16_mode(s) ? w.items : in.seq; a.n_vis = in.n_vis; a.n_work = w.n; a.T = in.T;
    a.n_head = d.n_head; a.n_kv = d.n_kv_head; a.dim = d.dim; a.vdim = d.vdim; a.hd = L.hd; a.n_parts = w.parts; a.wide = wide; a.scale = d.scale; a.sink = d.sink;
    a.scratch = s->scratch; a.att = s->att; a.ld_att = L.close_ld; a.out_scale = s->family == kPostNorm ? d.out_scale : 1.0f; a.window = d.window; a.first = in.first[L.hc];
    a.softcap = d.softcap; a.sinks = d.head_sinks ? L.sink : nullptr;
    if (L.heads_apart()) { a.all_values = 1; a.att = s->heads; }
    return a;
}

pi_gqa_prep gqa_prep_args(pi_model * m, const Layer & L, int pass, const Step & in) {
    LayerState * s = m->lay;
    const pi_layer_desc & d = L.d;
    pi_gqa_prep p{};
    p.z = s->z; p.ldz = L.z_rows; p.T = in.T; p.n_head = d.n_head; p.n_kv = d.n_kv_head; p.dim = d.dim; p.vdim = d.vdim; p.rot_dim = d.rot_dim; p.off_k = L.off_k; p.off_v = L.off_v;
    p.hd = L.hd; p.unit = d.unit_qk; p.cs = L.rot >= 0 ? s->cs[L.rot] : s->x; p.eps = m->hp.norm_eps; p.q = s->q_lat; p.cache = L.cache[pass]; p.cell = in.cell;
    p.rot_pairs = d.rot_pairs; p.unit_v = d.unit_v; p.q_norm = L.q_norm; p.k_norm = L.k_norm; p.temp = L.temp;
    if (d.value_mix) { p.ld_first = d.n_kv_head * d.vdim; if (L.first_values) p.v_keep = s->v_first; else { p.v_first = s->v_first; p.v_mix = L.v_mix; } }
    return p;
}

// step: the parts of a split attention stay unmerged (parts says which)
int attend_grouped(pi_model * m, const Layer & L, int pass, const Step & in, bool step, pi_gqa_attn & parts) {
    LayerState * s = m->lay;
    const int type = s->opts.compute;
    if (bf16_mode(s) && in.wide[L.hc].n > 0 && in.talk[L.hc].n == 0) {
        const pi_gqa_attn a = gqa_args(m, L, pass, in, in.wide[L.hc], 1);
        PI_TRY(pi_k_gqa_attn(type, &a, m->stream));
    }
    if (in.work[L.hc].n == 0) return PI_OK;
    const pi_gqa_attn a = gqa_args(m, L, pass, in, in.work[L.hc], 0);
    if (!step) return pi_k_gqa_attn(type, &a, m->stream);
    if (a.n_parts > 1) parts = a;
    return pi_k_gqa_attn_parts(&a, m->stream);
}

pi_linear linear_args(pi_model * m, const Layer & L, int pass, const Step & in) {
    LayerState * s = m->lay;
    const Rec & r = L.rec;
    pi_linear p{};
    p.z = s->z; p.ldz = L.z_rows; p.T = in.T; p.n_head = r.n_head; p.dim = r.dim; p.vdim = r.vdim; p.off_q = r.off_q; p.off_k = r.off_k; p.off_v = r.off_v; p.decay = r.decay; p.powers = r.powers;
    p.state = L.state[pass]; p.runs = in.lin; p.n_runs = in.n_lin; p.o = s->lin_o; p.q = s->lin_q; p.k = s->lin_k; p.v = s->lin_v; p.states = s->lin_states;
    p.dim_ld = r.dim_ld; p.vdim_ld = r.vdim_ld; p.decay_kind = r.kind; p.plain = r.plain; p.q_scale = r.q_scale; p.slot_ld = L.state_floats();
    p.a2 = r.a2; p.a2_b = r.a2_b; p.off_a = r.off_a; p.rank = r.rank; p.rank_ld = r.rank_ld; p.tau = r.tau;
    p.i_b = r.i_b; p.f_b = r.f_b; p.off_i = r.off_i; p.off_f = r.off_f; p.cap = r.cap; p.den = s->lin_den; p.gates = s->lin_gates;
    p.n_chunks = in.n_lin_chunks; p.chunks = in.lin_chunks; p.first_chunk = in.lin_first;
    return p;
}

// the recurrent part of a mixer, short runs token by token and long ones in chunks; front or beside in a launch of it where there is one
int recur(pi_model * m, const Layer & L, int pass, const Step & in, const pi_ffn_front * front, const pi_gqa_prep * beside) {
    LayerState * s = m->lay;
    const int type = s->opts.compute;
    hipStream_t st = m->stream;
    pi_linear p = linear_args(m, L, pass, in);
    if (in.n_lin_long == 0) return beside ? pi_k_linear_step_beside(type, &p, beside, st) : pi_k_linear_step(type, &p, front, st);
    PI_TRY(pi_k_linear_prep(type, &p, front, st));
    if (beside) PI_TRY(pi_k_gqa_prep(type, beside, nullptr, st));
    if (in.n_lin > 0) PI_TRY(pi_k_linear_step(type, &p, nullptr, st));
    p.runs = in.lin_long; p.n_runs = in.n_lin_long;
    return pi_k_linear_chunks(&p, st);
}

pi_gate_norm gate_norm_args(pi_model * m, const Layer & L, int T) {
    LayerState * s = m->lay;
    const Rec & r = L.rec;
    pi_gate_norm g{};
    g.o = s->lin_o; g.z = s->z; g.w = r.norm; g.ldz = L.z_rows; g.off_gate = r.off_g; g.n = r.n_head * r.vdim; g.T = T; g.eps = m->hp.norm_eps;
    g.att = (unsigned char *)s->att + (size_t)r.off_att * s->es; g.ld_att = L.close_ld; g.scale = r.scale; g.heads = r.per_head ? r.n_head : 0; g.silu = r.silu;
    g.den = r.kind == PI_DECAY_GATED ? s->lin_den : nullptr;
    return g;
}

// A layer with one norm.  Steps of up to 16 tokens (bf16): norm, joint projection, what lies behind it (queries and cells or the state's step,
// beside the dense or shared feed-forward's activation and the choice of experts), attention, merge or gated norm beside the experts'
// first matrices, and what closes the layer.  Longer steps run the same parts one by one.
int one_norm_layer(pi_model * m, Layer & L, const LayerRun & r, const Step & in, float * keep) {
    LayerState * s = m->lay;
    const pi_layer_desc & d = L.d;
    const int T = in.T, D = m->hp.n_embd, type = s->opts.compute;
    const bool moe = L.moe(), step = bf16_mode(s) && pi_k_layer_step_supported(T, moe ? d.n_expert : 0, moe ? d.n_top : 0), linear = d.mixer == PI_MIXER_LINEAR;
    hipStream_t st = m->stream;
    PI_TRY(pi_k_layer_norm(type, s->x, nullptr, T, D, m->hp.norm_eps, L.norm_a, r.starts && r.pass > 0 ? s->x0 : nullptr, r.starts ? s->loop_step + (size_t)r.pass * D : nullptr,
                           s->h_a, s->d_ld, step, st));
    if (step) PI_TRY(pi_k_gemm_bf16_ol(L.w_z, L.z_rows, s->d_ld, s->h_a, T, PI_EPI_NONE, nullptr, nullptr, s->z, nullptr, st));
    else PI_TRY(dense(m, L.w_z, L.z_rows, s->d_ld, s->h_a, T, s->z));
    pi_ffn_front f{};
    f.off_glu = L.off_glu; f.ff = d.glu_ff; f.ff_ld = L.glu_ld; f.off_score = L.off_score; f.limit = d.glu_limit; f.gain = d.glu_gain;
    f.act = (unsigned char *)s->att + (size_t)L.hv_ld * s->es; f.ld_act = L.close_ld; f.off_router = L.off_router; f.n_expert = moe ? d.n_expert : 0; f.n_top = d.n_top;
    f.ids = s->ids; f.weights = s->wts;
    pi_gqa_attn parts{};
    pi_gate_norm gate{};
    if (linear) {
        PI_TRY(recur(m, L, r.pass, in, &f, nullptr));
        gate = gate_norm_args(m, L, T);
        if (!step) PI_TRY(pi_k_gate_norm(type, &gate, st));
    } else {
        const pi_gqa_prep p = gqa_prep_args(m, L, r.pass, in);
        PI_TRY(pi_k_gqa_prep(type, &p, &f, st));
        PI_TRY(attend_grouped(m, L, r.pass, in, step, parts));
    }
    if (step) {
        if (moe || linear || parts.n_parts > 1)
            PI_TRY(pi_k_mix_up_step(parts.n_parts > 1 ? &parts : nullptr, linear ? &gate : nullptr, L.up, d.n_expert, d.expert_ff, s->d_ld, d.expert_limit, d.glu_gain, s->h_a, T,
                                    moe ? s->ids : nullptr, s->wts, d.n_top, s->act, L.ff_ld, st));
        pi_layer_out o{};
        o.x = s->x; o.wo = L.wo; o.att = s->att; o.rows = D; o.ld_att = L.close_ld; o.T = T; o.out = s->x2; o.keep = keep;
        if (moe) { o.down = L.down; o.act = s->act; o.ids = s->ids; o.ld_act = L.ff_ld; o.top = d.n_top; o.n_expert = d.n_expert; }
        return pi_k_layer_out_step(&o, st);
    }
    PI_TRY(dense(m, L.wo, D, L.close_ld, s->att, T, s->mix));
    if (moe) PI_TRY(experts(m, L, s->h_a, in));
    return pi_k_moe_combine(type, s->x, s->mix, s->y_exp, s->inv, moe ? s->wts : nullptr, moe ? d.n_top : 0, T, D, s->x2, keep, st);
}

// A layer whose norms come after the sums.  Steps of up to 16 tokens (bf16): joint projection, what lies behind it (queries and cells beside the
// state's step), attention, merge and gated norm, the mixer's closing product with the gated sum, norm; gate and up rows with their
// GLU beside the second residual gate, closing product with the gated sum, norm.
int post_norm_layer(pi_model * m, Layer & L, const LayerRun & r, const Step & in, float * keep) {
    LayerState * s = m->lay;
    const pi_layer_desc & d = L.d;
    const int T = in.T, D = m->hp.n_embd, type = s->opts.compute;
    const bool step = bf16_mode(s) && pi_k_layer_step_supported(T, 0, 0), grouped = d.mixer == PI_MIXER_GROUPED;
    hipStream_t st = m->stream;
    if (step) PI_TRY(pi_k_gemm_bf16_ol(L.w_z, L.z_rows, s->d_ld, s->h_a, T, PI_EPI_NONE, nullptr, nullptr, s->z, nullptr, st));
    else PI_TRY(dense(m, L.w_z, L.z_rows, s->d_ld, s->h_a, T, s->z));
    pi_gqa_attn parts{};
    if (grouped) {
        const pi_gqa_prep p = gqa_prep_args(m, L, r.pass, in);
        if (L.rec.on()) PI_TRY(recur(m, L, r.pass, in, nullptr, &p));
        else PI_TRY(pi_k_gqa_prep(type, &p, nullptr, st));
        PI_TRY(attend_grouped(m, L, r.pass, in, step, parts));
    } else PI_TRY(recur(m, L, r.pass, in, nullptr, nullptr));
    const pi_gate_norm gate = L.rec.on() ? gate_norm_args(m, L, T) : pi_gate_norm{};
    if (step) {
        if (L.rec.on() || parts.n_parts > 1)
            PI_TRY(pi_k_mix_up_step(parts.n_parts > 1 ? &parts : nullptr, L.rec.on() ? &gate : nullptr, nullptr, 0, 0, 0, 0.0f, 0.0f, nullptr, T, nullptr, nullptr, 0, nullptr, 0, st));
    } else if (L.rec.on()) PI_TRY(pi_k_gate_norm(type, &gate, st));
    // x = norm(alpha x + gate * W att), with the next product's operand
    const auto close = [&](const void * W, int ld, const float * gz, int ld_gate, int off_gate, const float * gb, const float * w, float * kept) -> int {
        pi_res_norm n{};
        n.w = w; n.T = T; n.cols = D; n.alpha = s->opts.residual_alpha; n.eps = m->hp.norm_eps; n.out = s->x; n.keep = kept; n.h = s->h_a; n.ld = s->d_ld; n.ol = step;
        if (step) {
            pi_layer_out o{};
            o.x = s->x; o.wo = W; o.att = s->att; o.rows = D; o.ld_att = ld; o.T = T; o.out = s->x2; o.scaled = 1; o.alpha = n.alpha;
            o.gate_z = gz; o.ld_gate = ld_gate; o.off_gate = off_gate; o.gate_b = gb;
            PI_TRY(pi_k_layer_out_step(&o, st));
            n.x = s->x2;
        } else {
            PI_TRY(dense(m, W, D, ld, s->att, T, s->mix));
            n.x = s->x; n.mix = s->mix; n.gate_z = gz; n.ld_gate = ld_gate; n.off_gate = off_gate; n.gate_b = gb;
        }
        return pi_k_res_norm(type, &n, st);
    };
    const bool gated = d.gated_residual != 0, ffn = d.ffn == PI_FFN_GLU;
    PI_TRY(close(L.wo, L.close_ld, gated ? s->z : nullptr, L.z_rows, L.off_gate, L.gate_b, L.norm_a, ffn ? nullptr : keep));
    if (!ffn) return PI_OK;
    if (step) {
        const uint16_t * W = (const uint16_t *)L.w_ffn;
        PI_TRY(pi_k_gemm_bf16_ol_glu(W, d.glu_ff, s->h_a, d.glu_limit, d.glu_gain, d.glu_plain_up ? 0.0f : 1.0f, s->att, L.glu_ld, gated ? W + (size_t)L.off_gate_ffn * s->d_ld : nullptr, D,
                                     s->z, s->d_ld, T, st));
        return close(L.down, L.glu_ld, gated ? s->z : nullptr, D, 0, L.gate_ffn_b, L.norm_b, keep);
    }
    PI_TRY(dense(m, L.w_ffn, L.z2_rows, s->d_ld, s->h_a, T, s->z));
    pi_ffn_front f{};
    f.ff = d.glu_ff; f.ff_ld = L.glu_ld; f.off_score = -1; f.limit = d.glu_limit; f.gain = d.glu_gain; f.plain_up = d.glu_plain_up; f.act = s->att; f.ld_act = L.glu_ld;
    PI_TRY(pi_k_ffn_front(type, s->z, L.z2_rows, T, &f, st));
    return close(L.down, L.glu_ld, gated ? s->z : nullptr, L.z2_rows, L.off_gate_ffn, L.gate_ffn_b, L.norm_b, keep);
}

// A layer with norms before and after its sublayers.  Steps of up to 16 tokens (bf16) stream the weights past operands in the matrix cores' layout; the
// sum that closes a sublayer and the norm ahead of the feed-forward are one launch, the norm ahead of the mixer and its convolution another.
int both_norms_layer(pi_model * m, Layer & L, const LayerRun & r, const Step & in, float * keep) {
    LayerState * s = m->lay;
    const pi_layer_desc & d = L.d;
    const int T = in.T, D = m->hp.n_embd, type = s->opts.compute;
    const bool moe = L.moe(), step = bf16_mode(s) && pi_k_layer_step_supported(T, moe ? d.n_expert : 0, moe ? d.n_top : 0);
    hipStream_t st = m->stream;
    if (L.conv) {
        pi_conv_norm c{};
        c.x = s->x; c.w = L.norm_a; c.taps_w = L.conv; c.T = T; c.cols = D; c.groups = s->opts.norm_groups; c.taps = s->opts.conv_taps; c.eps = m->hp.norm_eps;
        c.state = L.conv_floats ? L.state[r.pass] + L.rec_floats() : nullptr; c.slot_ld = L.state_floats(); c.items = in.conv; c.n_items = in.n_conv; c.h = s->h_a; c.ld = s->d_ld; c.ol = step;
        PI_TRY(pi_k_conv_norm(type, &c, st));
    } else {
        pi_sum_norm n{};
        n.x = s->x; n.w_next = L.norm_a; n.T = T; n.cols = D; n.groups = s->opts.norm_groups; n.eps = m->hp.norm_eps; n.h = s->h_a; n.ld = s->d_ld; n.ol = step;
        PI_TRY(pi_k_sum_norm(type, &n, st));
    }
    const auto product = [&](const void * W, int rows, const void * h, float * y) -> int {
        return step ? pi_k_gemm_bf16_ol(W, rows, s->d_ld, h, T, PI_EPI_NONE, nullptr, nullptr, y, nullptr, st) : dense(m, W, rows, s->d_ld, h, T, y);
    };
    PI_TRY(product(L.w_z, L.z_rows, s->h_a, s->z));
    const pi_gqa_prep p = gqa_prep_args(m, L, r.pass, in);
    PI_TRY(pi_k_gqa_prep(type, &p, nullptr, st));
    pi_gqa_attn parts{};
    PI_TRY(attend_grouped(m, L, r.pass, in, step, parts));
    if (parts.n_parts > 1) PI_TRY(pi_k_mix_up_step(&parts, nullptr, nullptr, 0, 0, 0, 0.0f, 0.0f, nullptr, T, nullptr, nullptr, 0, nullptr, 0, st));
    if (L.heads_apart()) {
        const Step::Work & talk = in.talk[L.hc], & apart = in.apart[L.hc];
        pi_gqa_mix x{};
        x.a = s->heads; x.talk = L.talk; x.z = s->z; x.ldz = L.z_rows; x.off_gate = L.off_head_gate; x.T = T; x.n_head = d.n_head; x.n_kv = d.n_kv_head; x.vdim = d.vdim;
        x.att = s->att; x.ld_att = L.close_ld;
        if (talk.n > 0) { x.tokens = apart.items; x.n_tokens = apart.n; }
        if (talk.n == 0 || apart.n > 0) PI_TRY(pi_k_gqa_mix(type, &x, st));
        if (talk.n > 0) {
            if (talk.parts > d.n_kv_head) return pi::fail(PI_E_ARG, "attention: more parts than there is room for");
            const pi_gqa_attn a = gqa_args(m, L, r.pass, in, in.wide[L.hc], 1);
            x.tokens = nullptr; x.n_tokens = 0; x.parts = s->heads; x.n_parts = talk.parts;      // (s->heads has room for n_kv parts, and is free again)
            PI_TRY(pi_k_gqa_stats(&a, s->stats, st));
            PI_TRY(pi_k_gqa_talk(&a, &x, s->stats, talk.items, talk.n, st));
        }
    }
    pi_layer_out o{};
    o.rows = D; o.T = T; o.out = s->mix;
    if (step) { o.wo = L.wo; o.att = s->att; o.ld_att = L.close_ld; PI_TRY(pi_k_layer_out_step(&o, st)); }
    else PI_TRY(dense(m, L.wo, D, L.close_ld, s->att, T, s->mix));
    pi_sum_norm n{};
    n.x = s->x; n.mix = s->mix; n.w = L.norm_a_after; n.mult = s->opts.residual_mult; n.T = T; n.cols = D; n.groups = s->opts.norm_groups; n.eps = m->hp.norm_eps;
    n.ld = s->d_ld; n.ol = step;
    if (moe) { n.h = s->h_b; n.w_next = L.norm_b; } else n.keep = keep;
    PI_TRY(pi_k_sum_norm(type, &n, st));
    if (!moe) return PI_OK;
    PI_TRY(product(L.router, d.n_expert, s->h_b, s->rl));
    PI_TRY(pi_k_route_scores(s->rl, T, d.n_expert, d.n_top, s->ids, s->wts, st));
    n.w = L.norm_b_after; n.w_next = nullptr; n.h = nullptr; n.keep = keep;
    if (step) {
        PI_TRY(pi_k_expert_up_step(L.up, d.n_expert, d.expert_ff, s->d_ld, d.expert_limit, d.glu_gain, d.glu_plain_up, d.weigh_input, s->h_b, T, s->ids, s->wts, d.n_top, s->act, L.ff_ld, st));
        o.wo = nullptr; o.down = L.down; o.act = s->act; o.ids = s->ids; o.ld_act = L.ff_ld; o.top = d.n_top; o.n_expert = d.n_expert;
        PI_TRY(pi_k_layer_out_step(&o, st));
    } else {
        PI_TRY(experts(m, L, s->h_b, in));
        n.mix = nullptr; n.y = s->y_exp; n.inv = s->inv; n.top = d.n_top; n.y_w = d.weigh_input ? nullptr : s->wts;
    }
    return pi_k_sum_norm(type, &n, st);
}

// a layer of a step of up to 16 tokens (bf16): six launches
int step_layer(pi_model * m, Layer & L, const Step & in, float * keep) {
    LayerState * s = m->lay;
    const pi_layer_desc & d = L.d;
    const int T = in.T, D = m->hp.n_embd;
    const bool moe = d.ffn == PI_FFN_MOE;
    hipStream_t st = m->stream;
    Layer & src = L.own_kv ? L : s->layers[d.kv_from];
    PI_TRY(pi_k_norm_pair(PI_TYPE_BF16, s->x, nullptr, T, D, m->hp.norm_eps, L.norm_a, s->h_a, moe ? L.norm_b : nullptr, moe ? s->h_b : nullptr, s->d_ld, 1, st));
    if (moe) PI_TRY(pi_k_gemm_bf16_ol_two(L.w_z, L.z_rows, s->h_a, s->z, L.router, d.n_expert, s->h_b, s->rl, s->d_ld, T, st));
    else     PI_TRY(pi_k_gemm_bf16_ol(L.w_z, L.z_rows, s->d_ld, s->h_a, T, PI_EPI_NONE, nullptr, nullptr, s->z, nullptr, st));
    const pi_latent_prep p = prep_args(m, L, in);
    PI_TRY(pi_k_latent_step(&p, L.uk_t, s->rl, d.n_expert, d.n_top, d.n_group, d.n_group_keep, L.bias, moe ? s->ids : nullptr, s->wts, st));
    const pi_latent_attn a = attn_args(m, L, src, in);
    PI_TRY(pi_k_latent_attn_parts(&a, st));
    PI_TRY(pi_k_value_up_step(&a, L.uv, d.vdim, s->att, L.hv_ld, L.up, d.n_expert, d.expert_ff, s->d_ld, s->h_b, moe ? s->ids : nullptr, s->wts, d.n_top, s->act, L.ff_ld, st));
    pi_layer_out o{};
    o.x = s->x; o.wo = L.wo; o.att = s->att; o.rows = D; o.ld_att = L.hv_ld; o.T = T; o.out = s->x2; o.keep = keep;
    if (moe) { o.down = L.down; o.act = s->act; o.ids = s->ids; o.ld_act = L.ff_ld; o.top = d.n_top; o.n_expert = d.n_expert; }
    return pi_k_layer_out_step(&o, st);
}

int pass_layers(pi_model * m, const Step & in) {
    LayerState * s = m->lay;
    const int type = s->opts.compute, T = in.T, D = m->hp.n_embd;
    hipStream_t st = m->stream;
    if (s->family != kTwoNorms) PI_TRY(pi_k_embed_bigram(s->embed, D, in.tokens, in.prev, T, s->opts.embed_scale, s->bigram, s->opts.bigram_buckets, s->opts.bigram_mul_prev, s->opts.bigram_mul_cur,
                                              in.carry, s->x, s->opts.loop_times > 0 ? s->x0 : nullptr, st));
    else PI_TRY(pi_k_embed_norm(s->embed, D, in.tokens, T, s->embd_norm, m->hp.norm_eps, s->x, st));
    if (s->family == kPostNorm) {                      // the first product's operand
        pi_res_norm n{};
        n.x = n.out = s->x; n.T = T; n.cols = D; n.h = s->h_a; n.ld = s->d_ld; n.ol = bf16_mode(s) && pi_k_layer_step_supported(T, 0, 0);
        PI_TRY(pi_k_res_norm(type, &n, st));
    }
    for (size_t k = 0; k < s->rots.size(); ++k) {
        const Rotation & r = s->rots[k];
        PI_TRY(r.scaling ? pi_k_rope_angles_table(in.pos, T, r.dims, r.freq, r.length(), s->cs[k], st) : pi_k_rope_angles(in.pos, T, r.dims, r.base, s->cs[k], st));
    }
    for (size_t k = 0; k < s->order.size(); ++k) {
        Layer & L = s->layers[s->order[k].layer];
        const bool moe = L.moe();
        float * keep = s->streams_T ? s->streams + k * (size_t)s->streams_T * D : nullptr;
        if (s->family == kBothNorms) {
            PI_TRY(both_norms_layer(m, L, s->order[k], in, keep));
            continue;
        }
        if (s->family == kPostNorm) {
            PI_TRY(post_norm_layer(m, L, s->order[k], in, keep));
            continue;
        }
        if (s->family == kOneNorm) {
            PI_TRY(one_norm_layer(m, L, s->order[k], in, keep));
            std::swap(s->x, s->x2);
            continue;
        }
        if (bf16_mode(s) && pi_k_layer_step_supported(T, moe ? L.d.n_expert : 0, moe ? L.d.n_top : 0)) {
            PI_TRY(step_layer(m, L, in, keep));
            std::swap(s->x, s->x2);
            continue;
        }
        PI_TRY(pi_k_norm_pair(type, s->x, nullptr, T, D, m->hp.norm_eps, L.norm_a, s->h_a, moe ? L.norm_b : nullptr, moe ? s->h_b : nullptr, s->d_ld, 0, st));
        PI_TRY(mix_latent(m, L, in));
        if (moe) PI_TRY(ffn_moe(m, L, in));
        PI_TRY(pi_k_moe_combine(type, s->x, s->mix, s->y_exp, s->inv, moe ? s->wts : nullptr, moe ? L.d.n_top : 0, T, D, s->x2, keep, st));
        std::swap(s->x, s->x2);
    }
    return PI_OK;
}

// logits of `n` rows of the residual stream (rows: device indices, null: the first n) into s->logits
int pass_head(pi_model * m, const int32_t * rows, int n) {
    LayerState * s = m->lay;
    const int D = m->hp.n_embd;
    const bool ol = bf16_mode(s) && n <= 16;
    if (s->family == kBothNorms) {
        pi_sum_norm h{};
        h.x = s->x; h.w_next = s->out_norm; h.rows = rows; h.T = n; h.cols = D; h.groups = s->opts.norm_groups; h.eps = m->hp.norm_eps; h.h = s->h_head; h.ld = s->d_ld; h.ol = ol;
        PI_TRY(pi_k_sum_norm(s->opts.compute, &h, m->stream));
    } else if (s->family == kOneNorm) PI_TRY(pi_k_layer_norm(s->opts.compute, s->x, rows, n, D, m->hp.norm_eps, s->out_norm, nullptr, nullptr, s->h_head, s->d_ld, ol, m->stream));
    else PI_TRY(pi_k_norm_pair(s->opts.compute, s->x, rows, n, D, m->hp.norm_eps, s->out_norm, s->h_head, nullptr, nullptr, s->d_ld, ol, m->stream));
    if (ol) return pi_k_gemm_bf16_ol(s->head, m->hp.n_vocab, s->d_ld, s->h_head, n, PI_EPI_NONE, nullptr, nullptr, s->logits, nullptr, m->stream);
    return dense(m, s->head, m->hp.n_vocab, s->d_ld, s->h_head, n, s->logits);
}

int head_buffers(pi_model * m) {
    LayerState * s = m->lay;
    if (s->logits) return PI_OK;
    s->h_head = m->alloc<unsigned char>((size_t)kHeadRows * s->d_ld * s->es);
    s->d_next = m->alloc<int32_t>(kHeadRows);
    s->logits = m->alloc<float>((size_t)kHeadRows * m->hp.n_vocab);
    if (!s->h_head || !s->d_next || !s->logits) return PI_E_HIP;
    return pi_memset(s->h_head, 0, (size_t)kHeadRows * s->d_ld * s->es);
}

// Tokens fall into runs (consecutive, of one sequence, with ascending cells).  A long run pays for expanding its cells' keys and values:
// per (token, cell) pair and head the latent form multiplies kd + rank_ld numbers, the expanded one dim + rot_dim + vdim, and an
// expansion costs rank_ld * (dim + vdim) per cell and head.
bool worth_expanding(const HeadKind & h, int T, int n_cells) {
    const long long latent = (long long)h.kd + h.rank_ld, expanded = (long long)h.dim + h.rot_dim + h.vdim;
    return pi_k_latent_expanded_supported(h.dim, h.rot_dim, h.vdim) && T >= 64 && T * (latent - expanded) > (long long)h.rank_ld * (h.dim + h.vdim) &&
           (long long)n_cells * h.n_head * (h.dim + h.vdim) <= kExpandedValues;
}

// work items {first token, first row, rows, sequence} of the tokens that attend in latent space, appended to `out`; long runs to `runs`
void work_items(const int32_t * seq, const int32_t * n_vis, int n, const HeadKind & h, std::vector<int32_t> & out, std::vector<Step::Run> * runs) {
    for (int t0 = 0; t0 < n;) {
        int t1 = t0 + 1;
        while (t1 < n && seq[t1] == seq[t0] && n_vis[t1] >= n_vis[t1 - 1]) ++t1;
        const int rows = (t1 - t0) * h.n_head;
        if (runs && worth_expanding(h, t1 - t0, n_vis[t1 - 1])) runs->push_back({t0, t1 - t0, seq[t0], n_vis[t1 - 1]});
        else for (int r = 0; r < rows; r += kItemRows) { out.push_back(t0); out.push_back(r); out.push_back(std::min(kItemRows, rows - r)); out.push_back(seq[t0]); }
        t0 = t1;
    }
}

// the same for grouped-query attention: runs of at least kWideRows rows as wide items (where the caller takes them)
void gqa_items(const int32_t * seq, const int32_t * n_vis, int n, int per, std::vector<int32_t> & narrow, std::vector<int32_t> * wide) {
    for (int t0 = 0; t0 < n;) {
        int t1 = t0 + 1;
        while (t1 < n && seq[t1] == seq[t0] && n_vis[t1] >= n_vis[t1 - 1]) ++t1;
        const int rows = (t1 - t0) * per;
        const bool w = wide && rows >= kWideRows;
        const int step = pi_k_gqa_rows(w);
        for (int r = 0; r < rows; r += step) { const int32_t item[4] = {t0, r, std::min(step, rows - r), seq[t0]}; (w ? *wide : narrow).insert((w ? *wide : narrow).end(), item, item + 4); }
        t0 = t1;
    }
}

// the tokens of the runs that gqa_items takes as wide ones, as items of pi_k_gqa_talk, and all others
void talk_items(const int32_t * seq, const int32_t * n_vis, int n, const HeadKind & h, std::vector<int32_t> & items, std::vector<int32_t> & others) {
    for (int t0 = 0; t0 < n;) {
        int t1 = t0 + 1;
        while (t1 < n && seq[t1] == seq[t0] && n_vis[t1] >= n_vis[t1 - 1]) ++t1;
        if ((t1 - t0) * h.n_head >= kWideRows)
            for (int t = t0; t < t1; t += h.talk_tokens) { const int32_t item[4] = {t, std::min(h.talk_tokens, t1 - t), seq[t0], 0}; items.insert(items.end(), item, item + 4); }
        else
            for (int t = t0; t < t1; ++t) others.push_back(t);
        t0 = t1;
    }
}

// Items {first token, tokens, sequence, 0} of pi_k_gqa_talk from place `at` on, in up to max_parts parts each, so that none has much more than a compute unit's
// share of the cells; by falling cells from the end, where the device begins.  Returns the most parts of an item.
int split_talk_items(std::vector<int32_t> & items, size_t at, const int32_t * n_vis, int max_parts) {
    struct Item { int32_t v[4]; long long cells; };
    std::vector<Item> all;
    long long total = 0;
    for (size_t k = at; k < items.size(); k += 4) total += n_vis[items[k] + items[k + 1] - 1];
    const long long share = std::max<long long>(kTalkCells, total / std::max(pi::compute_units(), 1) + 1);
    int most = 1;
    for (size_t k = at; k < items.size(); k += 4) {
        const long long n = n_vis[items[k] + items[k + 1] - 1];
        const int parts = (int)std::max<long long>(1, std::min<long long>((n + share - 1) / share, max_parts));
        most = std::max(most, parts);
        for (int j = 0; j < parts; ++j) all.push_back({{items[k], items[k + 1], items[k + 2], parts > 1 ? parts << 16 | j : 0}, n / parts});
    }
    std::stable_sort(all.begin(), all.end(), [](const Item & a, const Item & b) { return a.cells < b.cells; });
    items.resize(at);
    for (const Item & i : all) items.insert(items.end(), i.v, i.v + 4);
    return most;
}

// span: the most cells a work item sees
int gqa_span(const HeadKind & h, int n_vis_max, bool wide) { return h.window > 0 ? std::min(n_vis_max, h.window + pi_k_gqa_rows(wide)) : n_vis_max; }
int gqa_parts(int n_groups, int n_vis_max, int cells) { return n_groups <= 0 ? 1 : std::max(1, std::min({kAttnItems / n_groups, (n_vis_max + cells - 1) / cells, 64})); }

// how many workgroups share one work item's cells
int choose_parts(LayerState * s, int n_work, int n_vis_max) {
    if (!bf16_mode(s) || n_work <= 0) return 1;
    const int tiles = (n_vis_max + 31) / 32;
    return std::max(1, std::min({kAttnItems / n_work, tiles, 64}));
}

// ---- cells -----------------------------------------------------------------------------------------------------------------------
// the host's list of a sequence's cells, rebuilt after an edit; `app` receives what the device has to learn
void refresh_list(LayerState * s, int q, std::vector<int32_t> & app) {
    if (!(s->kv.edited >> q & 1u)) return;
    s->kv.edited &= ~(1u << q);
    std::vector<std::pair<int32_t, int32_t>> v;
    for (int i = 0; i < s->kv.n; ++i) if (s->kv.pos[i] >= 0 && (s->kv.seq[i] >> q & 1u)) v.push_back({s->kv.pos[i], i});
    std::sort(v.begin(), v.end());
    s->list_cells[q].clear(); s->list_pos[q].clear();
    for (size_t k = 0; k < v.size(); ++k) {
        s->list_pos[q].push_back(v[k].first); s->list_cells[q].push_back(v[k].second);
        app.push_back(q); app.push_back((int32_t)k); app.push_back(v[k].second);
    }
}

int live_cells(LayerState * s, int q) {
    int n = 0;
    for (int i = 0; i < s->kv.n; ++i) n += s->kv.pos[i] >= 0 && (s->kv.seq[i] >> q & 1u) ? 1 : 0;
    return n;
}

// takes the cell for sequences `mask` at position p; false: some sequence's list has to be rebuilt (the position is not behind its last)
void take_cell(LayerState * s, int cell, int32_t p, uint32_t mask, int32_t tok, std::vector<int32_t> & app) {
    s->kv.take(cell, p, mask);
    s->cell_tok[cell] = tok;
    for (uint32_t b = mask; b; b &= b - 1) {
        const int q = __builtin_ctz(b);
        if (s->kv.edited >> q & 1u) continue;                      // rebuilt as a whole later
        if (!s->list_pos[q].empty() && s->list_pos[q].back() >= p) { s->kv.edited |= 1u << q; continue; }
        app.push_back(q); app.push_back((int32_t)s->list_pos[q].size()); app.push_back(cell);
        s->list_pos[q].push_back(p); s->list_cells[q].push_back(cell);
    }
}

int apply_shift(pi_model * m) {
    LayerState * s = m->lay;
    if (!s->kv.has_shift) return PI_OK;
    PI_HIP_TRY(hipStreamSynchronize(m->stream));
    PI_TRY(pi_memcpy_h2d(s->d_delta, s->kv.delta.data(), sizeof(int32_t) * s->kv.n));
    for (Layer & L : s->layers) {
        if (L.d.mixer == PI_MIXER_GROUPED)
            for (void * c : L.cache)
                PI_TRY(L.d.rot_scaling ? pi_k_gqa_shift_table(s->opts.compute, c, s->kv.n, L.d.n_kv_head, L.hd, L.d.rot_dim, s->rots[L.rot].freq, L.d.rot_pairs, s->d_delta, m->stream)
                                       : pi_k_gqa_shift(s->opts.compute, c, s->kv.n, L.d.n_kv_head, L.hd, L.d.rot_dim, L.d.rot_base, L.d.rot_pairs, s->d_delta, m->stream));
        else if (L.cell_values()) PI_TRY(pi_k_latent_shift(s->opts.compute, L.cache[0], s->kv.n, L.kd, L.rank_ld, L.d.rot_dim, L.d.rot_base, s->d_delta, m->stream));
    }
    PI_HIP_TRY(hipStreamSynchronize(m->stream));
    s->kv.shift_done();
    return PI_OK;
}

// ---- slots of recurrent states ----------------------------------------------------------------------------------------------------
int resize_slots(pi_model * m, int n) {
    LayerState * s = m->lay;
    PI_HIP_TRY(hipStreamSynchronize(m->stream));
    drop_graph(s);
    for (Layer & L : s->layers)
        for (float *& st : L.state) {
            const size_t one = L.state_floats();
            float * p = m->alloc<float>(n * one);
            if (!p) return PI_E_HIP;
            PI_TRY(pi_memset(p, 0, n * one * 4));
            if (st) PI_TRY(pi_memcpy_d2d(p, st, s->n_slots * one * 4));
            PI_TRY(pi_sync());
            for (auto & o : m->owned) if (st && o == st) { pi_free(o); o = nullptr; }
            st = p;
        }
    s->n_slots = n;
    return PI_OK;
}

// the sequence's slot; one of a sequence without cells (other than those of `keep`) is taken, or there will be more of them
int take_slot(pi_model * m, int q, uint32_t keep) {
    LayerState * s = m->lay;
    if (s->slot_of[q] >= 0) return PI_OK;
    std::vector<char> used(s->n_slots, 0);
    for (int o = 0; o < 32; ++o) {
        if (s->slot_of[o] < 0) continue;
        if (!(keep >> o & 1u) && live_cells(s, o) == 0) s->slot_of[o] = -1;
        else used[s->slot_of[o]] = 1;
    }
    int k = 0;
    while (k < s->n_slots && used[k]) ++k;
    if (k == s->n_slots) PI_TRY(resize_slots(m, std::max(4, 2 * s->n_slots)));
    s->slot_of[q] = k;
    return PI_OK;
}

// a recurrent state holds all of a sequence's tokens: true if the edit leaves every sequence whole or empty
template <typename F> bool keeps_whole(LayerState * s, F && edit) {
    KvCells trial = s->kv;
    edit(trial);
    uint32_t lost = 0, left = 0;                                  // sequences that lose a cell, and that keep one
    for (int i = 0; i < s->kv.n; ++i) {
        const uint32_t before = s->kv.pos[i] >= 0 ? s->kv.seq[i] : 0u, after = trial.pos[i] >= 0 ? trial.seq[i] : 0u;
        lost |= before & ~after;
        left |= after;
    }
    return (lost & left) == 0;
}

int upload_appends(pi_model * m, const std::vector<int32_t> & app) {
    if (app.empty()) return PI_OK;
    LayerState * s = m->lay;
    PI_TRY(ensure_inputs(m, app.size()));
    PI_HIP_TRY(hipStreamSynchronize(m->stream));                   // the staging buffer's last copy is done
    memcpy(s->h_in, app.data(), app.size() * 4);
    PI_HIP_TRY(hipMemcpyAsync(s->d_in, s->h_in, app.size() * 4, hipMemcpyHostToDevice, m->stream));
    const int n = (int)(app.size() / 3);
    hipLaunchKernelGGL(cells_append_kernel, dim3((n + 255) / 256), dim3(256), 0, m->stream, s->d_in, n, s->lists, (size_t)s->kv.n);
    return pi::check_launch("cells_append");
}

}  // namespace

namespace pi {

KvCells * layers_cells(pi_model * m) { return m->lay->kv.n ? &m->lay->kv : nullptr; }

// caches and lists for n_cells cells; what earlier cells hold is kept
static int resize_pool(pi_model * m, int n_cells) {
    LayerState * s = m->lay;
    PI_HIP_TRY(hipStreamSynchronize(m->stream));
    drop_graph(s);
    auto give_back = [&](void * p) { for (auto & o : m->owned) if (p && o == p) { pi_free(o); o = nullptr; } };
    for (Layer & L : s->layers) {
        const size_t row = L.cell_values() * s->es;
        if (!row) continue;
        for (void *& old : L.cache) {
            unsigned char * c = m->alloc<unsigned char>(n_cells * row);
            if (!c) return PI_E_HIP;
            PI_TRY(pi_memset(c, 0, n_cells * row));
            if (old) PI_TRY(pi_memcpy_d2d(c, old, s->kv.n * row));
            PI_TRY(pi_sync());
            give_back(old);
            old = c;
        }
    }
    s->cell_tok.resize(n_cells, -1);
    give_back(s->lists); give_back(s->d_delta);
    s->lists = m->alloc<int32_t>((size_t)32 * n_cells);
    s->d_delta = m->alloc<int32_t>(n_cells);
    if (!s->lists || !s->d_delta) return PI_E_HIP;
    PI_TRY(pi_memset(s->lists, 0, sizeof(int32_t) * 32 * (size_t)n_cells));
    PI_TRY(pi_sync());
    if (s->kv.n) s->kv.grow(n_cells); else s->kv.init(n_cells);
    return PI_OK;
}

int layers_cells_init(pi_model * m, int n_cells) {
    if (!m->finalized) return fail(PI_E_STATE, "pi_model_kv_cells_init: model not finalized");
    if (m->lay->kv.n) return fail(PI_E_STATE, "pi_model_kv_cells_init: already initialised");
    if (n_cells < 1) return fail(PI_E_ARG, "pi_model_kv_cells_init: at least one cell");
    return resize_pool(m, n_cells);
}

int layers_finalize(pi_model * m) {
    LayerState * s = m->lay;
    const int D = m->hp.n_embd;
    PI_HIP_TRY(hipEventCreate(&m->ev0));
    PI_HIP_TRY(hipEventCreate(&m->ev1));
    s->es = bf16_mode(s) ? 2 : 4;
    s->d_ld = up_to(D, 256);
    PI_TRY(want_tensor(m->glob[PI_T_TOK_EMBD], PI_TYPE_BF16, D, m->hp.n_vocab, "tok_embd"));
    PI_TRY(want_tensor(m->glob[PI_T_OUTPUT], PI_TYPE_BF16, D, m->hp.n_vocab, "output"));
    PI_TRY(want_tensor(m->glob[PI_T_OUTPUT_NORM], PI_TYPE_F32, D, 1, "output_norm"));
    s->embed = m->glob[PI_T_TOK_EMBD].dev;
    PI_TRY(padded(m, m->glob[PI_T_OUTPUT], s->d_ld, &s->head));
    if (s->family == kTwoNorms) {
        PI_TRY(want_tensor(m->embd_norm, PI_TYPE_F32, D, 1, "embd_norm"));
        PI_TRY(norm_weights(m, m->embd_norm, s->opts.norm_offset, 1.0f, &s->embd_norm));
    }
    if (s->opts.bigram_buckets > 0) {
        PI_TRY(want_tensor(m->bigram, PI_TYPE_BF16, D, (int64_t)s->opts.bigram_buckets + 1, "bigram"));
        s->bigram = m->bigram.dev;
    }
    if (s->opts.loop_times > 0) {
        PI_TRY(want_tensor(m->loop_step, PI_TYPE_F32, D, s->opts.loop_times, "loop_step"));
        s->loop_step = (const float *)m->loop_step.dev;
    }
    PI_TRY(norm_weights(m, m->glob[PI_T_OUTPUT_NORM], s->opts.norm_offset, s->opts.logit_scale, &s->out_norm));
    size_t scratch = 0;
    for (size_t il = 0; il < s->layers.size(); ++il) {
        Layer & L = s->layers[il];
        const pi_layer_desc & d = L.d;
        const auto rotation = [&]() -> int {
            size_t r = 0;
            while (r < s->rots.size() && !s->rots[r].same(d)) ++r;
            L.rot = (int)r;
            if (r < s->rots.size()) return PI_OK;
            Rotation n{d.rot_dim, d.rot_base, d.rot_scaling, d.rot_factor, d.rot_original, d.rot_low, d.rot_high, nullptr};
            if (n.scaling) {
                const std::vector<double> f = n.frequencies();
                double * p = m->alloc<double>(f.size());
                if (!p) return PI_E_HIP;
                PI_TRY(pi_memcpy_h2d(p, f.data(), sizeof(double) * f.size()));
                n.freq = p;
            }
            s->rots.push_back(n);
            return PI_OK;
        };
        const auto kind = [&](const HeadKind & hk) {
            size_t h = 0;
            while (h < s->kinds.size() && memcmp(&s->kinds[h], &hk, sizeof hk)) ++h;
            if (h == s->kinds.size()) s->kinds.push_back(hk);
            L.hc = (int)h;
        };
        if (s->family != kTwoNorms) {
            if (s->family == kOneNorm) one_norm_sizes(L); else if (s->family == kBothNorms) both_norms_sizes(L); else post_norm_sizes(L, D);
            if (d.mixer == PI_MIXER_GROUPED) {
                L.hd = pi_k_gqa_head_ld(s->opts.compute, d.dim, d.vdim);
                if (!L.hd) return fail(PI_E_UNSUPPORTED, "pi_model_finalize: head sizes outside the attention kernels (up to 256)");
                if (d.rot_dim > 0) PI_TRY(rotation()); else L.rot = -1;
                kind(HeadKind{d.mixer, d.n_head / d.n_kv_head, d.n_kv_head * (L.heads_apart() ? d.n_kv_head : 1), 0, 0, 0, 0, L.hd, d.window,
                              L.heads_apart() && bf16_mode(s) ? pi_k_gqa_talk_tokens(d.n_head, d.n_kv_head, d.dim, d.vdim) : 0});
                scratch = std::max(scratch, pi_k_gqa_scratch_floats(kAttnItems, 1, 1, L.hd, 2) / 2);      // items x groups x parts <= kAttnItems
            }
            if (L.rec.on() && !pi_k_linear_supported(L.rec.dim, L.rec.vdim)) return fail(PI_E_UNSUPPORTED, "pi_model_finalize: head sizes outside the linear attention's kernels (up to 256)");
            if (d.weights_of) continue;
            PI_TRY(s->family == kOneNorm ? one_norm_weights(m, (int)il) : s->family == kBothNorms ? both_norms_weights(m, (int)il) : post_norm_weights(m, (int)il));
            continue;
        }
        L.own_kv = d.kv_from < 0;
        L.nq = d.n_head * (d.dim + d.rot_dim);
        L.z_rows = L.nq + (L.own_kv ? d.kv_rank + d.rot_dim : 0);
        L.dim_ld = up_to(d.dim, 64); L.rank_ld = up_to(d.kv_rank, 64); L.kd = L.rank_ld + up_to(d.rot_dim, 32);
        L.hv_ld = up_to(d.n_head * d.vdim, 128); L.ff_ld = d.ffn == PI_FFN_MOE ? up_to(d.expert_ff, 64) : 0;
        if (!pi_k_latent_attn_supported(s->opts.compute, L.rank_ld, L.kd)) return fail(PI_E_UNSUPPORTED, "pi_model_finalize: latent sizes outside the attention kernels (rank up to 1024)");
        PI_TRY(rotation());
        kind(HeadKind{d.mixer, d.n_head, 1, d.dim, d.rot_dim, d.vdim, L.rank_ld, L.kd, 0, 0});
        scratch = std::max(scratch, pi_k_latent_attn_scratch_floats(kItemRows * kAttnItems / 2, L.rank_ld, 2));      // items x parts <= kAttnItems
        PI_TRY(layer_weights(m, (int)il));
    }
    for (Layer & L : s->layers) {                      // another layer's weights, caches and states of its own
        if (!L.d.weights_of) continue;
        Layer own = s->layers[L.d.weights_of - 1];
        own.cache = L.cache; own.state = L.state;
        L = own;
    }
    if (bf16_mode(s)) {
        s->scratch = m->alloc<float>(scratch);
        if (!s->scratch) return PI_E_HIP;
    }
    PI_TRY(head_buffers(m));
    if (s->recurrent) PI_TRY(resize_slots(m, s->opts.n_slots > 0 ? s->opts.n_slots : 4));
    s->g_lin = m->alloc<int32_t>(4 * kMaxLockstep);
    s->g_conv = m->alloc<int32_t>(8 * kMaxLockstep);
    if (!s->g_lin || !s->g_conv) return PI_E_HIP;
    for (int32_t ** p : {&s->g_tok, &s->g_pos, &s->g_cell, &s->g_vis, &s->g_seq, &s->g_step, &s->g_prev}) {
        *p = m->alloc<int32_t>(kMaxLockstep);
        if (!*p) return PI_E_HIP;
    }
    size_t items = 0;
    for (const HeadKind & h : s->kinds) items += (size_t)kMaxLockstep * ((h.n_head + 15) / 16);      // (16: the smaller of the two kinds of items)
    s->g_work = m->alloc<int32_t>(4 * items);
    s->g_out = m->alloc<int32_t>((size_t)s->max_steps * kMaxLockstep);
    if (!s->g_work || !s->g_out) return PI_E_HIP;
    PI_HIP_TRY(hipDeviceSynchronize());
    m->finalized = true;
    return PI_OK;
}

void layers_destroy(pi_model * m) {
    LayerState * s = m->lay;
    drop_graph(s);
    if (s->arena) pi_free(s->arena);
    if (s->h_in) (void)hipHostFree(s->h_in);
    if (s->d_in) pi_free(s->d_in);
    if (s->streams) pi_free(s->streams);
    if (s->expanded) pi_free(s->expanded);
    delete s;
    m->lay = nullptr;
}

// One step: cells for every token (or PI_E_STATE with nothing changed), then passes of at most max_batch tokens.
int layers_step(pi_model * m, const int32_t * tokens, const int32_t * positions, const uint32_t * seq_masks, int n_tokens, const int32_t * want, int n_want,
                int32_t * next_tokens, float * logits_out) {
    LayerState * s = m->lay;
    if (!m->finalized || !s->kv.n) return fail(PI_E_STATE, "pi_model_kv_cells_step: pi_model_kv_cells_init first");
    if (!tokens || !positions || !seq_masks || n_tokens < 1 || n_want < 0 || (n_want && !want)) return fail(PI_E_ARG, "pi_model_kv_cells_step: bad arguments");
    for (int w = 0; w < n_want; ++w) if (want[w] < 0 || want[w] >= n_tokens) return fail(PI_E_ARG, "pi_model_kv_cells_step: a wanted place is outside the step");
    for (int t = 0; t < n_tokens; ++t)
        if (tokens[t] < 0 || tokens[t] >= m->hp.n_vocab || positions[t] < 0 || seq_masks[t] == 0) return fail(PI_E_ARG, "pi_model_kv_cells_step: a token needs an id, a position and a sequence");
    std::vector<int32_t> cells(n_tokens), app;
    if (!s->kv.find_free(n_tokens, cells.data())) return fail(PI_E_STATE, "pi_model_kv_cells_step: not enough free cells");
    const int batch = s->opts.max_batch > 0 ? s->opts.max_batch : 2048;
    PI_TRY(ensure_capacity(m, std::min(n_tokens, batch)));
    PI_TRY(apply_shift(m));
    for (int t = 0; t < n_tokens; ++t) for (uint32_t b = seq_masks[t]; b; b &= b - 1) refresh_list(s, __builtin_ctz(b), app);
    uint32_t fresh = 0;                                          // recurrent models: sequences whose state starts at zero
    if (s->recurrent) {
        uint32_t met = 0;
        const char * why = nullptr;
        for (int t = 0; t < n_tokens && !why; ++t) {
            const int q = __builtin_ctz(seq_masks[t]);
            if (seq_masks[t] & (seq_masks[t] - 1)) why = "pi_model_kv_cells_step: a token of several sequences in a model with recurrent states";
            else if (t && seq_masks[t] == seq_masks[t - 1]) { if (positions[t] <= positions[t - 1]) why = "pi_model_kv_cells_step: a recurrent state takes its tokens in order"; }
            else if (met >> q & 1u) why = "pi_model_kv_cells_step: a sequence's tokens follow one another in a step";
            else if (!s->list_pos[q].empty() && s->list_pos[q].back() >= positions[t]) why = "pi_model_kv_cells_step: a recurrent state takes its tokens in order";
            else { met |= 1u << q; if (s->list_pos[q].empty()) fresh |= 1u << q; }
        }
        if (why) { PI_TRY(upload_appends(m, app)); return fail(PI_E_UNSUPPORTED, why); }
        for (uint32_t b = met; b; b &= b - 1) PI_TRY(take_slot(m, __builtin_ctz(b), met));
    }
    for (int t = 0; t < n_tokens; ++t) take_cell(s, cells[t], positions[t], seq_masks[t], tokens[t], app);
    s->kv.move_head(cells[n_tokens - 1] + 1);
    for (int t = 0; t < n_tokens; ++t) for (uint32_t b = seq_masks[t]; b; b &= b - 1) refresh_list(s, __builtin_ctz(b), app);
    PI_TRY(upload_appends(m, app));
    std::vector<int32_t> vis(n_tokens), seq(n_tokens), prev(n_tokens, -1);
    for (int t = 0; t < n_tokens; ++t) {
        seq[t] = __builtin_ctz(seq_masks[t]);                    // a token attends the cells of its first sequence
        const auto & lp = s->list_pos[seq[t]];
        vis[t] = (int32_t)(std::upper_bound(lp.begin(), lp.end(), positions[t]) - lp.begin());
        if (vis[t] >= 2) prev[t] = s->cell_tok[s->list_cells[seq[t]][vis[t] - 2]];
    }
    std::vector<int32_t> rows, place, items, wide, lin;
    for (int t0 = 0; t0 < n_tokens; t0 += batch) {
        const int T = std::min(batch, n_tokens - t0);
        rows.clear(); place.clear(); items.clear();
        for (int w = 0; w < n_want; ++w) if (want[w] >= t0 && want[w] < t0 + T) { rows.push_back(want[w] - t0); place.push_back(w); }
        Step in;
        in.T = T;
        const int vmax = *std::max_element(vis.begin() + t0, vis.begin() + t0 + T);
        std::vector<size_t> begin, begin_wide;
        wide.clear(); lin.clear();
        for (const HeadKind & h : s->kinds) {
            begin.push_back(items.size());
            begin_wide.push_back(wide.size());
            in.runs.emplace_back();
            if (h.mixer == PI_MIXER_GROUPED) { if (bf16_mode(s)) gqa_items(seq.data() + t0, vis.data() + t0, T, h.n_head, items, T > 16 ? &wide : nullptr); }
            else if (bf16_mode(s)) work_items(seq.data() + t0, vis.data() + t0, T, h, items, T > 16 ? &in.runs.back() : nullptr);
        }
        begin.push_back(items.size());
        begin_wide.push_back(wide.size());
        items.insert(items.end(), wide.begin(), wide.end());
        std::vector<size_t> at_talk, at_apart;
        std::vector<int> n_talk, n_apart, talk_parts;
        std::vector<int32_t> others;
        for (const HeadKind & h : s->kinds) {
            at_talk.push_back(items.size()); at_apart.push_back(others.size());
            if (h.talk_tokens > 0 && T > 16) talk_items(seq.data() + t0, vis.data() + t0, T, h, items, others);
            n_talk.push_back((int)(items.size() - at_talk.back()) / 4);
            if (n_talk.back() < kTalkItems) { items.resize(at_talk.back()); others.resize(at_apart.back()); n_talk.back() = 0; }
            talk_parts.push_back(n_talk.back() > 0 ? split_talk_items(items, at_talk.back(), vis.data() + t0, h.value_groups()) : 1);
            n_talk.back() = (int)(items.size() - at_talk.back()) / 4;
            n_apart.push_back((int)(others.size() - at_apart.back()));
        }
        const size_t at_conv = items.size();
        if (s->opts.conv_taps > 0) {
            const int back = s->opts.conv_taps - 1, per = pi_k_conv_tokens(T, s->opts.conv_taps);
            for (int a = 0; a < T;) {
                int b = a + 1;
                while (b < T && seq[t0 + b] == seq[t0 + a]) ++b;
                const int q = seq[t0 + a];
                for (int c = a; c < b;) {
                    const int n = std::min(c == a ? std::max(per, back) : per, b - c);
                    const int32_t item[8] = {c, n, c - a, b - a, std::max(s->slot_of[q], 0), (int32_t)(fresh >> q & 1u), 0, 0};
                    items.insert(items.end(), item, item + 8);
                    c += n;
                }
                a = b;
            }
            in.n_conv = (int)(items.size() - at_conv) / 8;
        }
        const size_t at_lin = items.size();
        if (s->recurrent) {                                       // runs walked token by token, long runs, their first chunks, the chunks
            std::vector<int32_t> lng, first, chunks;
            const int C = pi_k_linear_chunk();
            for (int a = 0; a < T;) {
                int b = a + 1;
                while (b < T && seq[t0 + b] == seq[t0 + a]) ++b;
                // A sequence's first results are few products (q . k) v, of which a norm over the head leaves the direction: the less of q . k is
                // rounded the better.  They are walked with unrounded projections, and the chunks begin behind them.
                if (s->family == kPostNorm && bf16_mode(s) && (fresh >> seq[t0 + a] & 1u) && b - a >= kLinearChunked + kFreshSteps) b = a + kFreshSteps;
                const int q = seq[t0 + a], new_state = fresh >> q & 1u;
                const int32_t run[4] = {a, b - a, s->slot_of[q], new_state};
                fresh &= ~(1u << q);                              // a later pass of this step goes on
                const bool chunked = bf16_mode(s) && b - a >= kLinearChunked;
                (chunked ? lng : lin).insert((chunked ? lng : lin).end(), run, run + 4);
                if (chunked) {
                    first.push_back((int32_t)(chunks.size() / 3));
                    for (int c = a; c < b; c += C) { const int32_t ch[3] = {c, std::min(C, b - c), new_state && c == a}; chunks.insert(chunks.end(), ch, ch + 3); }
                }
                a = b;
            }
            in.n_lin = (int)lin.size() / 4; in.n_lin_long = (int)lng.size() / 4; in.n_lin_chunks = (int)chunks.size() / 3;
            items.insert(items.end(), lin.begin(), lin.end());
            items.insert(items.end(), lng.begin(), lng.end());
            items.insert(items.end(), first.begin(), first.end());
            items.insert(items.end(), chunks.begin(), chunks.end());
        }
        std::vector<long long> at_first;                          // kinds with a window over positions that are not 0, 1, 2 ..: first cells by position
        for (const HeadKind & h : s->kinds) {
            bool gaps = false;
            for (int t = 0; t < T && h.window > 0; ++t) gaps = gaps || s->list_pos[seq[t0 + t]][vis[t0 + t] - 1] != vis[t0 + t] - 1;
            at_first.push_back(gaps ? (long long)items.size() : -1);
            for (int t = 0; t < T && gaps; ++t) {
                const auto & lp = s->list_pos[seq[t0 + t]];
                items.push_back((int32_t)(std::upper_bound(lp.begin(), lp.end(), positions[t0 + t] - h.window) - lp.begin()));
            }
        }
        const size_t at_others = items.size();
        items.insert(items.end(), others.begin(), others.end());
        const size_t n_in = (size_t)8 * T + items.size() + rows.size();
        PI_TRY(ensure_inputs(m, n_in));
        PI_HIP_TRY(hipStreamSynchronize(m->stream));
        int32_t * h = s->h_in;
        memcpy(h, tokens + t0, 4 * (size_t)T); memcpy(h + T, positions + t0, 4 * (size_t)T); memcpy(h + 2 * T, cells.data() + t0, 4 * (size_t)T);
        memcpy(h + 3 * T, vis.data() + t0, 4 * (size_t)T); memcpy(h + 4 * T, seq.data() + t0, 4 * (size_t)T);
        memcpy(h + 5 * T, prev.data() + t0, 4 * (size_t)T);      // (the items behind start on a multiple of 16 bytes)
        if (!items.empty()) memcpy(h + 8 * T, items.data(), 4 * items.size());
        if (!rows.empty()) memcpy(h + 8 * T + items.size(), rows.data(), 4 * rows.size());
        PI_HIP_TRY(hipMemcpyAsync(s->d_in, h, 4 * n_in, hipMemcpyHostToDevice, m->stream));
        in.tokens = s->d_in; in.pos = s->d_in + T; in.cell = s->d_in + 2 * T; in.n_vis = s->d_in + 3 * T; in.seq = s->d_in + 4 * T; in.prev = s->d_in + 5 * T;
        in.conv = s->d_in + 8 * T + at_conv;
        in.lin = s->d_in + 8 * T + at_lin; in.lin_long = in.lin + 4 * in.n_lin; in.lin_first = in.lin_long + 4 * in.n_lin_long; in.lin_chunks = in.lin_first + in.n_lin_long;
        for (size_t k = 0; k < s->kinds.size(); ++k) {
            Step::Work w;
            w.items = s->d_in + 8 * T + begin[k];
            w.n = bf16_mode(s) ? (int)(begin[k + 1] - begin[k]) / 4 : T;
            const HeadKind & hk = s->kinds[k];
            w.parts = hk.mixer == PI_MIXER_GROUPED ? (bf16_mode(s) ? gqa_parts(w.n * hk.n_kv, gqa_span(hk, vmax, false), 128) : 1) : choose_parts(s, w.n, vmax);
            in.work.push_back(w);
            Step::Work wd;
            wd.items = s->d_in + 8 * T + begin.back() + begin_wide[k];
            wd.n = (int)(begin_wide[k + 1] - begin_wide[k]) / 4;
            wd.parts = gqa_parts(wd.n * hk.n_kv, gqa_span(hk, vmax, true), 512);
            in.wide.push_back(wd);
            Step::Work talk, apart;
            talk.items = s->d_in + 8 * T + at_talk[k]; talk.n = n_talk[k]; talk.parts = talk_parts[k];
            apart.items = s->d_in + 8 * T + at_others + at_apart[k]; apart.n = n_apart[k];
            in.talk.push_back(talk); in.apart.push_back(apart);
            in.first.push_back(at_first[k] < 0 ? nullptr : s->d_in + 8 * T + at_first[k]);
        }
        s->streams_T = 0;
        if (m->capture) {
            const size_t need = s->order.size() * (size_t)T * m->hp.n_embd;
            if (need > s->streams_cap) {
                if (s->streams) pi_free(s->streams);
                s->streams_cap = 0;
                s->streams = (float *)pi_malloc(need * 4);
                if (!s->streams) return PI_E_HIP;
                s->streams_cap = need;
            }
            s->streams_T = T;
        }
        PI_TRY(ensure_expanded(m, in));
        PI_TRY(pass_layers(m, in));
        const int32_t * d_rows = s->d_in + 8 * T + items.size();
        for (int r0 = 0; r0 < (int)rows.size(); r0 += kHeadRows) {
            const int n = std::min(kHeadRows, (int)rows.size() - r0);
            const size_t V = m->hp.n_vocab;
            PI_TRY(pass_head(m, d_rows + r0, n));
            if (next_tokens) for (int k = 0; k < n; k += 16) PI_TRY(pi_k_argmax_batch(s->logits + k * V, (int)V, std::min(16, n - k), s->d_next + k, nullptr, nullptr, nullptr, 0, m->stream));
            PI_HIP_TRY(hipStreamSynchronize(m->stream));
            std::vector<int32_t> nx(next_tokens ? n : 0);
            if (next_tokens) PI_TRY(pi_memcpy_d2h(nx.data(), s->d_next, 4 * (size_t)n));
            for (int k = 0; k < n; ) {                              // runs of places that follow one another leave in one copy
                int e = k + 1;
                while (e < n && place[r0 + e] == place[r0 + k] + (e - k)) ++e;
                if (logits_out) PI_TRY(pi_memcpy_d2h(logits_out + (size_t)place[r0 + k] * V, s->logits + (size_t)k * V, sizeof(float) * V * (e - k)));
                if (next_tokens) for (int j = k; j < e; ++j) next_tokens[place[r0 + j]] = nx[j];
                k = e;
            }
        }
    }
    PI_HIP_TRY(hipStreamSynchronize(m->stream));
    return PI_OK;
}

static int ensure_pool(pi_model * m, int64_t n) {
    LayerState * s = m->lay;
    if (s->kv.n && (!s->auto_pool || s->kv.n >= n)) return PI_OK;      // a pool the caller has sized stays as it is
    if (n > INT32_MAX / 2) return fail(PI_E_ARG, "the cache pool is too large");
    s->auto_pool = true;
    return resize_pool(m, (int)n);
}

// tokens at n_past .. of sequence q, behind exactly n_past cells (what lies at n_past and beyond is dropped first)
static int continue_at(pi_model * m, int q, int n_past) {
    LayerState * s = m->lay;
    std::vector<int32_t> app;
    refresh_list(s, q, app);
    PI_TRY(upload_appends(m, app));
    const auto & lp = s->list_pos[q];
    const int before = (int)(std::lower_bound(lp.begin(), lp.end(), n_past) - lp.begin());
    if (before != n_past || (n_past && (lp[0] != 0 || lp[n_past - 1] != n_past - 1))) return fail(PI_E_STATE, "the sequence's cells do not hold the positions 0 .. n_past - 1");
    if ((int)lp.size() == before) return PI_OK;
    if (s->recurrent && before > 0) return fail(PI_E_UNSUPPORTED, "a model with recurrent states cannot go back to an earlier position");
    s->kv.seq_rm(q, n_past, -1);
    app.clear();
    refresh_list(s, q, app);
    return upload_appends(m, app);
}

int layers_decode(pi_model * m, const int32_t * tokens, int n_tokens, int n_past, float * logits_out) {
    LayerState * s = m->lay;
    if (!tokens || n_tokens <= 0 || n_past < 0 || n_past + n_tokens > m->hp.n_ctx) return fail(PI_E_ARG, "pi_model_decode: token range exceeds the context");
    PI_TRY(ensure_pool(m, m->hp.n_ctx));
    PI_TRY(continue_at(m, kOwnSeq, n_past));
    std::vector<int32_t> pos(n_tokens);
    for (int i = 0; i < n_tokens; ++i) pos[i] = n_past + i;
    const std::vector<uint32_t> mask(n_tokens, 1u << kOwnSeq);
    const int32_t last = n_tokens - 1;
    int32_t next = -1;
    PI_TRY(layers_step(m, tokens, pos.data(), mask.data(), n_tokens, &last, 1, &next, logits_out));
    s->last_tok[kOwnSeq] = next; s->last_pos[kOwnSeq] = n_past + n_tokens;
    return next;
}

int layers_batch_init(pi_model * m, int n_seq) {
    LayerState * s = m->lay;
    if (s->n_seq) return fail(PI_E_STATE, "pi_model_batch_init: already initialised");
    PI_TRY(ensure_pool(m, (int64_t)m->hp.n_ctx * (n_seq + 1)));
    PI_TRY(ensure_capacity(m, n_seq));
    s->n_seq = n_seq;
    for (int q = 0; q < n_seq; ++q) { s->last_tok[q] = 0; s->last_pos[q] = 0; }
    return PI_OK;
}

int layers_batch_decode(pi_model * m, const int32_t * tokens, const int32_t * positions, int32_t * next_tokens, float * logits_out) {
    LayerState * s = m->lay;
    if (!s->n_seq) return fail(PI_E_STATE, "pi_model_batch_decode: pi_model_batch_init first");
    if (!tokens || !positions) return fail(PI_E_ARG, "pi_model_batch_decode: null pointer");
    uint32_t mask[kMaxLockstep]; int32_t want[kMaxLockstep], next[kMaxLockstep];
    for (int q = 0; q < s->n_seq; ++q) {
        if (positions[q] < 0 || positions[q] >= m->hp.n_ctx) return fail(PI_E_ARG, "pi_model_batch_decode: position outside the context");
        if (!s->list_pos[q].empty() && s->list_pos[q].back() >= positions[q]) PI_TRY(continue_at(m, q, positions[q]));
        mask[q] = 1u << q; want[q] = q;
    }
    PI_TRY(layers_step(m, tokens, positions, mask, s->n_seq, want, s->n_seq, next, logits_out));
    for (int q = 0; q < s->n_seq; ++q) {
        s->last_tok[q] = next[q]; s->last_pos[q] = positions[q] + 1;
        if (next_tokens) next_tokens[q] = next[q];
    }
    return PI_OK;
}

// the greedy loop of the model's own sequence (own) or of the lockstep sequences: one captured step, replayed
int layers_generate(pi_model * m, int own, int n_steps, int32_t * out_tokens, float * ms_out) {
    LayerState * s = m->lay;
    const int T = own ? 1 : s->n_seq, q0 = own ? kOwnSeq : 0;
    if (!T || !s->kv.n) return fail(PI_E_STATE, "pi_model_generate: decode a prompt first");
    if (n_steps <= 0 || n_steps > s->max_steps || !out_tokens) return fail(PI_E_ARG, "pi_model_generate: bad step count");
    std::vector<int32_t> tok(T), pos(T), vis(T), seq(T), cell(T), prev(T), lin(4 * T), cells((size_t)n_steps * T), app;
    PI_TRY(apply_shift(m));
    for (int t = 0; t < T; ++t) {
        seq[t] = q0 + t; tok[t] = s->last_tok[q0 + t]; pos[t] = s->last_pos[q0 + t];
        refresh_list(s, q0 + t, app);
        if (pos[t] + n_steps > m->hp.n_ctx) return fail(PI_E_ARG, "pi_model_generate: would run past the context");
        if ((int)s->list_pos[q0 + t].size() != pos[t]) return fail(PI_E_STATE, "pi_model_generate: a sequence's cells do not end at its next position");
        prev[t] = pos[t] ? s->cell_tok[s->list_cells[q0 + t].back()] : -1;
        if (s->recurrent) {
            PI_TRY(take_slot(m, q0 + t, ((1u << T) - 1) << q0));
            if (pos[t] == 0)
                for (Layer & L : s->layers) for (float * st : L.state) PI_TRY(pi_memset(st + s->slot_of[q0 + t] * L.state_floats(), 0, L.state_floats() * 4));
        }
    }
    if (!s->kv.find_free(n_steps * T, cells.data())) return fail(PI_E_STATE, "pi_model_generate: not enough free cells");
    for (int k = 0; k < n_steps; ++k)
        for (int t = 0; t < T; ++t) take_cell(s, cells[(size_t)k * T + t], pos[t] + k, 1u << (q0 + t), k ? -1 : tok[t], app);
    s->kv.move_head(cells.back() + 1);
    PI_TRY(upload_appends(m, app));
    PI_TRY(ensure_capacity(m, T));
    for (int t = 0; t < T; ++t) { vis[t] = pos[t] + 1; cell[t] = cells[t]; }
    std::vector<int32_t> items;
    Step in;
    in.T = T; in.tokens = s->g_tok; in.pos = s->g_pos; in.cell = s->g_cell; in.n_vis = s->g_vis; in.seq = s->g_seq;
    std::vector<int> parts;
    for (const HeadKind & h : s->kinds) {
        Step::Work w;
        const size_t at = items.size();
        const int vmax = *std::max_element(pos.begin(), pos.end()) + n_steps;
        if (bf16_mode(s)) { if (h.mixer == PI_MIXER_GROUPED) gqa_items(seq.data(), vis.data(), T, h.n_head, items, nullptr); else work_items(seq.data(), vis.data(), T, h, items, nullptr); }
        w.items = s->g_work + at;
        w.n = bf16_mode(s) ? (int)(items.size() - at) / 4 : T;
        w.parts = h.mixer == PI_MIXER_GROUPED ? (bf16_mode(s) ? gqa_parts(w.n * h.n_kv, gqa_span(h, vmax, false), 128) : 1) : choose_parts(s, w.n, vmax);
        in.work.push_back(w);
        in.wide.emplace_back(); in.talk.emplace_back(); in.apart.emplace_back();
        in.first.push_back(nullptr);                           // (the positions are 0, 1, 2 ..)
        parts.push_back(w.parts);
    }
    PI_HIP_TRY(hipStreamSynchronize(m->stream));
    if (s->recurrent) {
        for (int t = 0; t < T; ++t) { lin[4 * t] = t; lin[4 * t + 1] = 1; lin[4 * t + 2] = s->slot_of[q0 + t]; lin[4 * t + 3] = 0; }
        in.lin = s->g_lin; in.n_lin = T;
        PI_TRY(pi_memcpy_h2d(s->g_lin, lin.data(), 16 * T));
    }
    if (s->opts.conv_taps > 0) {
        std::vector<int32_t> conv;
        for (int t = 0; t < T; ++t) { const int32_t item[8] = {t, 1, 0, 1, std::max(s->slot_of[q0 + t], 0), 0, 0, 0}; conv.insert(conv.end(), item, item + 8); }
        in.conv = s->g_conv; in.n_conv = T;
        PI_TRY(pi_memcpy_h2d(s->g_conv, conv.data(), 4 * conv.size()));
    }
    in.prev = s->g_prev; in.carry = true;
    PI_TRY(pi_memcpy_h2d(s->g_prev, prev.data(), 4 * T));
    const int32_t zero = 0;
    PI_TRY(pi_memcpy_h2d(s->g_tok, tok.data(), 4 * T)); PI_TRY(pi_memcpy_h2d(s->g_pos, pos.data(), 4 * T)); PI_TRY(pi_memcpy_h2d(s->g_vis, vis.data(), 4 * T));
    PI_TRY(pi_memcpy_h2d(s->g_seq, seq.data(), 4 * T)); PI_TRY(pi_memcpy_h2d(s->g_cell, cell.data(), 4 * T)); PI_TRY(pi_memcpy_h2d(s->g_step, &zero, 4));
    if (!items.empty()) PI_TRY(pi_memcpy_h2d(s->g_work, items.data(), 4 * items.size()));
    s->streams_T = 0;
    float * const x0 = s->x, * const x20 = s->x2;
    auto step = [&]() -> int {
        s->x = x0; s->x2 = x20;                                    // every step starts on the same buffers, whatever the layer count
        PI_TRY(pass_layers(m, in));
        PI_TRY(pass_head(m, nullptr, T));
        PI_TRY(pi_k_argmax_batch(s->logits, m->hp.n_vocab, T, s->g_tok, s->g_pos, s->g_step, s->g_out, s->max_steps, m->stream));
        return pi_k_cells_advance(T, s->g_seq, s->lists, s->kv.n, s->g_vis, s->g_cell, s->g_step, m->stream);
    };
    const char * no_graph = getenv("PI_NO_GRAPH");
    const bool use_graph = !(no_graph && no_graph[0] == '1');
    if (use_graph && s->exec && (s->graph_T != T || s->graph_seq0 != q0 || s->graph_parts != parts)) drop_graph(s);
    if (use_graph && !s->exec) {
        PI_HIP_TRY(hipStreamBeginCapture(m->stream, hipStreamCaptureModeThreadLocal));
        const int rc = step();
        hipGraph_t g = nullptr;
        const hipError_t e = hipStreamEndCapture(m->stream, &g);
        if (rc != PI_OK) { if (g) (void)hipGraphDestroy(g); return rc; }
        if (e != hipSuccess) return hip_fail(e, "hipStreamEndCapture");
        s->graph = g;
        PI_HIP_TRY(hipGraphInstantiate(&s->exec, g, nullptr, nullptr, 0));
        s->graph_T = T; s->graph_seq0 = q0; s->graph_parts = parts;
    }
    PI_HIP_TRY(hipEventRecord(m->ev0, m->stream));
    for (int k = 0; k < n_steps; ++k) {
        if (use_graph) PI_HIP_TRY(hipGraphLaunch(s->exec, m->stream));
        else PI_TRY(step());
    }
    PI_HIP_TRY(hipEventRecord(m->ev1, m->stream));
    PI_HIP_TRY(hipStreamSynchronize(m->stream));
    if (ms_out) PI_HIP_TRY(hipEventElapsedTime(ms_out, m->ev0, m->ev1));
    PI_TRY(pi_memcpy_d2h(out_tokens, s->g_out, sizeof(int32_t) * (size_t)n_steps * T));
    for (int k = 1; k < n_steps; ++k) for (int t = 0; t < T; ++t) s->cell_tok[cells[(size_t)k * T + t]] = out_tokens[(size_t)(k - 1) * T + t];
    for (int t = 0; t < T; ++t) { s->last_tok[q0 + t] = out_tokens[(size_t)(n_steps - 1) * T + t]; s->last_pos[q0 + t] = pos[t] + n_steps; }
    return PI_OK;
}

// a recurrent state cannot lose or move some of its tokens: edits that leave a sequence neither whole nor empty are refused (edit empty: any)
int layers_edit_allowed(pi_model * m, const std::function<void(KvCells &)> & edit) {
    LayerState * s = m->lay;
    if (!s->recurrent || (edit && keeps_whole(s, edit))) return PI_OK;
    return fail(PI_E_UNSUPPORTED, "KV edit: a model with recurrent states cannot drop or move part of a sequence");
}

// before the cells of src in [p0, p1) become dst's as well: its states do, if that is all of src and dst is empty
int layers_copy_state(pi_model * m, int src, int dst, int p0, int p1) {
    LayerState * s = m->lay;
    if (!s->recurrent || src == dst) return PI_OK;
    int all = 0, taken = 0;
    for (int i = 0; i < s->kv.n; ++i) {
        if (s->kv.pos[i] < 0 || !(s->kv.seq[i] >> src & 1u)) continue;
        ++all;
        taken += s->kv.pos[i] >= std::max(p0, 0) && (p1 < 0 || s->kv.pos[i] < p1);
    }
    if (taken == 0) return PI_OK;
    if (taken != all || live_cells(s, dst) != 0 || s->slot_of[src] < 0) return fail(PI_E_UNSUPPORTED, "KV edit: a model with recurrent states copies whole sequences into empty ones");
    PI_TRY(take_slot(m, dst, 1u << dst));
    PI_HIP_TRY(hipStreamSynchronize(m->stream));
    for (Layer & L : s->layers)
        for (float * st : L.state) PI_TRY(pi_memcpy_d2d(st + s->slot_of[dst] * L.state_floats(), st + s->slot_of[src] * L.state_floats(), L.state_floats() * 4));
    return pi_sync();
}

int layers_seq_edit(pi_model * m, int seq, int p0, int p1, int delta, bool shift) {
    LayerState * s = m->lay;
    if (seq < -1 || seq >= s->n_seq || !s->kv.n) return fail(PI_E_ARG, "KV edit: bad sequence");
    const int q = seq < 0 ? kOwnSeq : seq;
    PI_TRY(shift ? layers_edit_allowed(m, nullptr) : layers_edit_allowed(m, [&](KvCells & kv) { kv.seq_rm(q, p0, p1); }));
    if (shift) s->kv.seq_shift(q, p0, p1, delta); else s->kv.seq_rm(q, p0, p1);
    const int n = live_cells(s, q);
    s->last_pos[q] = n;
    return n;
}

int layers_seq_cp(pi_model * m, int src, int dst, int p0, int p1) {
    LayerState * s = m->lay;
    if (src < 0 || dst < 0 || src >= s->n_seq || dst >= s->n_seq || src == dst) return fail(PI_E_ARG, "pi_model_batch_kv_seq_cp: bad sequences");
    if (live_cells(s, dst) != std::max(p0, 0)) return fail(PI_E_UNSUPPORTED, "pi_model_batch_kv_seq_cp: the destination must hold exactly p0 cells");
    PI_TRY(layers_copy_state(m, src, dst, p0, p1));
    s->kv.seq_cp(src, dst, p0, p1);                                // shared, not copied
    s->last_pos[dst] = live_cells(s, dst);
    return s->last_pos[dst];
}

}  // namespace pi

extern "C" {

pi_model * pi_model_create_layers(const pi_hparams * hp, const pi_layers_opts * opts, const pi_layer_desc * layers, int n_layer) {
    const auto bad = [](const char * why) -> pi_model * { pi::set_error(why); return nullptr; };
    if (!hp || !opts || !layers || n_layer <= 0 || hp->n_embd <= 0 || hp->n_vocab <= 0 || hp->n_ctx <= 0 || (hp->arch != PI_ARCH_LERASUN && hp->arch != PI_ARCH_PIBALORN && hp->arch != PI_ARCH_FIKEVIK && hp->arch != PI_ARCH_PUFIVIK) ||
        (opts->compute != PI_TYPE_BF16 && opts->compute != PI_TYPE_F32) || opts->max_batch < 0)
        return bad("pi_model_create_layers: inconsistent hyper-parameters");
    const Family family = opts->both_norms ? kBothNorms : opts->post_norm ? kPostNorm : layers[0].mixer != PI_MIXER_LATENT ? kOneNorm : kTwoNorms;
    if (opts->both_norms && (opts->post_norm || opts->norm_groups <= 0 || hp->n_embd % opts->norm_groups || opts->norm_groups > 1024 || opts->conv_taps < 0 || opts->conv_taps > 64))
        return bad("pi_model_create_layers: norm_groups parts of n_embd (up to 1024) and up to 64 conv_taps");
    if (!opts->both_norms && opts->conv_taps) return bad("pi_model_create_layers: conv_taps needs both_norms");
    const pi_layer_desc * first_values = nullptr;      // the first layer with value_mix
    for (int il = 0; il < n_layer; ++il) {
        const pi_layer_desc & d = layers[il];
        if (family != kBothNorms && (d.softcap != 0.0f || d.head_sinks || d.head_mix || d.head_gate || d.value_mix || d.rot_scaling || d.route_scores || d.weigh_input))
            return bad("pi_model_create_layers: soft caps, mixed heads and values, scaled rotations and scores of experts need both_norms");
        if (family == kBothNorms) {
            if (d.mixer != PI_MIXER_GROUPED || (d.ffn != PI_FFN_NONE && (d.ffn != PI_FFN_GLU_MOE || d.glu_ff || !d.route_scores))) return bad("pi_model_create_layers: a layer's mixer or feed-forward");
            if (!(d.softcap >= 0.0f) || (d.head_mix && d.n_head > 128)) return bad("pi_model_create_layers: a layer's soft cap or its heads (up to 128 are mixed)");
            if (d.rot_scaling < PI_ROT_PLAIN || d.rot_scaling > PI_ROT_RAMP || (d.rot_scaling && (!(d.rot_factor > 0.0) || !(d.rot_original > 0.0) || !(d.rot_low > 0.0) || !(d.rot_high > 0.0) ||
                (d.rot_scaling == PI_ROT_RAMP && !(d.rot_base > 1.0)))))
                return bad("pi_model_create_layers: a layer's rotation");
            if (d.value_mix && !first_values) first_values = &d;
            if (d.value_mix && (d.values_are_keys || d.n_kv_head * d.vdim != first_values->n_kv_head * first_values->vdim)) return bad("pi_model_create_layers: layers that mix values need as many of them");
        }
        if ((d.mixer == PI_MIXER_LATENT) != (family == kTwoNorms)) return bad("pi_model_create_layers: layers of several families in one model");
        if (family != kPostNorm && (d.weights_of || d.gated_residual || d.mem_heads)) return bad("pi_model_create_layers: shared weights, gated residuals and memories need post_norm");
        if (family != kTwoNorms) {
            if ((d.mixer != PI_MIXER_GROUPED && d.mixer != (family == kPostNorm ? PI_MIXER_KEYED : PI_MIXER_LINEAR)) || d.n_head <= 0 || d.dim <= 0 || d.vdim <= 0)
                return bad("pi_model_create_layers: a layer's mixer");
            if (d.mixer == PI_MIXER_GROUPED && (d.n_kv_head <= 0 || d.n_head % d.n_kv_head || d.rot_dim < 0 || d.rot_dim % 2 || d.rot_dim > d.dim || (d.rot_dim && !(d.rot_base > 0.0)) ||
                                                (d.values_are_keys && d.vdim != d.dim) || d.window < 0 || (d.qk_norm && d.unit_qk)))
                return bad("pi_model_create_layers: a layer's grouped-query attention");
            if (d.mixer == PI_MIXER_KEYED && (d.decay_rank <= 0 || d.decay_rank > 512 || !(d.decay_tau > 0.0f))) return bad("pi_model_create_layers: a layer's key decays (rank up to 512)");
            if (d.mem_heads < 0 || (d.mem_heads > 0 && (d.mixer != PI_MIXER_GROUPED || d.mem_dim <= 0 || d.mem_vdim <= 0 || !(d.mem_cap > 0.0f)))) return bad("pi_model_create_layers: a layer's memory");
            if (d.weights_of) {
                pi_layer_desc same = d;
                same.weights_of = 0;
                if (d.weights_of < 0 || d.weights_of > n_layer || memcmp(&same, &layers[d.weights_of - 1], sizeof same))
                    return bad("pi_model_create_layers: weights_of must name a layer with weights of its own and the same description");
            }
            if (family == kPostNorm && d.ffn == PI_FFN_GLU_MOE) return bad("pi_model_create_layers: a layer's feed-forward");
            if (d.ffn != PI_FFN_NONE && d.ffn != PI_FFN_GLU && d.ffn != PI_FFN_GLU_MOE) return bad("pi_model_create_layers: a layer's feed-forward");
            if (d.glu_ff < 0 || (d.ffn == PI_FFN_GLU) > (d.glu_ff > 0) || (d.ffn == PI_FFN_NONE && d.glu_ff) ||
                (d.ffn == PI_FFN_GLU_MOE && (d.n_expert <= 0 || d.n_expert > 4096 || d.n_top <= 0 || d.n_top > d.n_expert || d.expert_ff <= 0)))
                return bad("pi_model_create_layers: a layer's experts");
            continue;
        }
        if (d.n_head <= 0 || d.dim <= 0 || d.rot_dim <= 0 || d.rot_dim % 2 || d.vdim <= 0 || d.kv_rank <= 0 || !(d.rot_base > 0.0))
            return bad("pi_model_create_layers: a layer's mixer");
        if (d.kv_from >= 0) {
            if (d.kv_from >= il) return bad("pi_model_create_layers: kv_from must name an earlier layer");
            const pi_layer_desc & o = layers[d.kv_from];
            if (o.kv_from >= 0 || o.kv_rank != d.kv_rank || o.rot_dim != d.rot_dim || o.rot_base != d.rot_base)
                return bad("pi_model_create_layers: kv_from must name a layer with cells of its own and the same latent and rotation");
        }
        if (d.ffn != PI_FFN_NONE && (d.ffn != PI_FFN_MOE || d.n_expert <= 0 || d.n_group <= 0 || d.n_expert % d.n_group || d.n_group_keep <= 0 || d.n_group_keep > d.n_group ||
                                     d.n_top <= 0 || d.n_top > d.n_group_keep * (d.n_expert / d.n_group) || d.expert_ff <= 0))
            return bad("pi_model_create_layers: a layer's experts");
    }
    if (opts->loop_times < 0 || (opts->loop_times > 0 && (family != kOneNorm || opts->loop_start < 0 || opts->loop_start >= opts->loop_stop || opts->loop_stop > n_layer)) || opts->bigram_buckets < 0 ||
        (opts->bigram_buckets && (family == kTwoNorms || opts->bigram_mul_prev < 0 || opts->bigram_mul_cur < 0)))
        return bad("pi_model_create_layers: the loop or the bigram table");
    if (pi_init(0) != PI_OK) return nullptr;
    pi_model * m = new pi_model();
    m->hp = *hp;
    m->hp.n_layer = n_layer;
    m->layers.resize((size_t)n_layer * PI_T_COUNT);
    m->lay = new LayerState();
    m->lay->opts = *opts;
    LayerState * s = m->lay;
    s->family = family;
    std::fill(s->slot_of, s->slot_of + 32, -1);
    const int lo = opts->loop_times > 0 ? opts->loop_start : n_layer, hi = opts->loop_times > 0 ? opts->loop_stop : n_layer;
    for (int il = 0; il < n_layer; ++il) {
        Layer L;
        L.d = layers[il];
        const int passes = il >= lo && il < hi ? opts->loop_times : 1;
        L.rec = recurrent_part(L.d);
        if (opts->conv_taps > 1) L.conv_floats = (size_t)(opts->conv_taps - 1) * hp->n_embd;
        L.first_values = &layers[il] == first_values;
        if (L.state_floats()) { L.state.resize(passes, nullptr); s->recurrent = true; }
        if (L.d.mixer == PI_MIXER_GROUPED || (L.d.mixer == PI_MIXER_LATENT && L.d.kv_from < 0)) L.cache.resize(passes, nullptr);
        s->layers.push_back(L);
    }
    for (int il = 0; il < lo; ++il) s->order.push_back({il, 0, false});
    for (int t = 0; t < opts->loop_times; ++t) for (int il = lo; il < hi; ++il) s->order.push_back({il, t, il == lo});
    for (int il = hi; il < n_layer; ++il) s->order.push_back({il, 0, false});
    return m;
}

int pi_model_get_streams(pi_model * m, float * out) {
    if (!m || !m->finalized || !m->lay || !m->capture || !m->lay->streams_T) return pi::fail(PI_E_STATE, "pi_model_get_streams: run a step with capture enabled first");
    LayerState * s = m->lay;
    PI_HIP_TRY(hipStreamSynchronize(m->stream));
    if (out) PI_TRY(pi_memcpy_d2h(out, s->streams, sizeof(float) * s->order.size() * (size_t)s->streams_T * m->hp.n_embd));
    return s->streams_T;
}

}  // extern "C"
