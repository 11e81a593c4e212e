// Layered decoders: stacks whose layers are described one by one (fa_layered_config).  Weights, the paged latent caches and
// the recurrent states live here; sequences, sampling, recorded steps and the entry points are decoder.cpp's.
// One launch sequence serves decode steps, prompt passes and mixed batches: a pass is a list of rows, each with its
// sequence, position, cache row and state slot (k::RaggedRows), and every kernel takes any number of rows per sequence.
#include <algorithm>
#include <cmath>
#include <cstring>
#include <functional>
#include <new>
#include <string>
#include <vector>

#include "decoder.hpp"
#include "validate.hpp"

namespace fa {

int g_layered_rows = 0;      // rows per internal pass of a prompt (tuning; below 64: the built-in figure)

namespace {

uint32_t pad_to(uint32_t v, uint32_t to) { return (v + to - 1) / to * to; }

struct Tensor {
    std::string name;
    uint64_t rows, cols;                              // cols 0: a vector
    bool set = false;
    // places the tensor, already on the device as bf16 bits or f32, where the kernels read it
    std::function<void(const void *src, int src_f32, hipStream_t s)> place;
};

// What mixes the tokens of a layer.  Its projections of the layer's input are columns of the layer's `in`: those that stay in the
// activations' type start at column lo_at of Arena::y, f32 ones at hi_at of Arena::y32.  Its output is columns o_at .. of Arena::o.
struct Mixer {
    fa_layer_config cfg;
    std::string prefix;                               // of its tensors
    uint32_t lo = 0, lo_at = 0, hi = 0, hi_at = 0, o_at = 0;
    float out_scale = 1.0f;
    uint32_t out_width() const { return cfg.heads * cfg.vdim; }
    // attention; q_norm below
    k::AttentionShape at{};
    uint32_t gate_at = 0;                             // column of its `lo` part where the gate starts
    float *k_norm = nullptr, *sink = nullptr, *slope = nullptr, *score_bias = nullptr;
    uint32_t head_gate_at = 0;                        // column of its `hi` part where the gates per head start
    void *k_pool = nullptr, *v_pool = nullptr;
    // latent attention
    k::LatentShape la{};
    k::LinearWeight uq, uk, uv, ukv;                  // ukv: keys and values of all heads from the latent (expanded form)
    uint32_t window_index = 0;
    float *q_norm = nullptr, *kv_norm = nullptr;
    void *pool = nullptr;
    uint32_t rotation = 0;                            // index of its cos / sin table
    // delta, lightning
    k::DeltaShape de{};
    float *conv = nullptr, *a_log = nullptr, *dt_bias = nullptr, *head_norm = nullptr, *state = nullptr, *decay = nullptr;
    void *ring = nullptr;
    // minimal gated recurrence: biases of z and u; state above
    float *z_bias = nullptr, *u_bias = nullptr;
    // low-rank gates and decays: their inner values start at column rank_at of the `lo` part (decay first, gate from its padded
    // rank on); one weight with zeros in the other's place makes both
    k::LinearWeight low_rank;
    uint32_t rank_at = 0;
};

// States that are matrices per head (DeltaShape)
bool recurrent(const fa_layer_config &c) { return c.mixer == FA_MIXER_DELTA || c.mixer == FA_MIXER_LIGHTNING; }

struct Layer {
    fa_layer_config cfg;
    std::vector<Mixer> mixers;                        // one, or two side by side
    uint32_t lo = 0, hi = 0, o_width = 0;             // columns of in (lo a multiple of eight) and inputs of out, all mixers
    float *norm1 = nullptr, *norm2 = nullptr, *post1 = nullptr, *post2 = nullptr;     // post: layer scale, or norm of the output
    float *in_bias = nullptr;                         // attention alone in its layer
    k::LinearWeight in, out, gate_up, down;           // with experts: gate_up and down hold one batch entry each
    k::LinearWeight router;
    float *correction = nullptr;                      // of the experts' scores
    float *act = nullptr;                             // xIELU: the two factors, and the two numbers they come from
    uint32_t lists() const { return cfg.experts - cfg.identity; }        // experts with tensors
};

// A rotation's frequencies follow from these
struct Rotation {
    uint32_t dims;
    double base, factor, low, high, original;
    bool operator==(const Rotation &o) const {
        return dims == o.dims && base == o.base && factor == o.factor && low == o.low && high == o.high && original == o.original;
    }
};
Rotation rotation_of(const fa_layer_config &c) {
    if (!(c.rot_factor > 0.0)) return Rotation{c.rot_dim, c.rot_base, 0.0, 0.0, 0.0, 0.0};
    return Rotation{c.rot_dim, c.rot_base, c.rot_factor, c.rot_low, c.rot_high, c.rot_original};
}
std::vector<double> frequencies(const Rotation &r) {
    std::vector<double> f(r.dims / 2);
    for (uint32_t i = 0; i < f.size(); ++i) {
        f[i] = std::pow(r.base, -2.0 * (double)i / (double)r.dims);
        if (r.factor > 0.0) {
            const double turns = r.original * f[i] / (2.0 * 3.14159265358979323846);
            const double ramp = turns < r.low ? 0.0 : turns > r.high ? 1.0 : (turns - r.low) / (r.high - r.low);
            f[i] = (1.0 - ramp) * f[i] / r.factor + ramp * f[i];
        }
    }
    return f;
}

// Activations of a pass of up to `rows` rows, one allocation.  Every section keeps its place and element type for the
// arena's life and starts as zeros: what lies behind a row's own width is always finite.
struct Arena {
    void *base = nullptr;
    uint64_t bytes = 0, cls = 0;
    uint32_t rows = 0;
    float *x = nullptr, *y32 = nullptr, *head_x = nullptr, *delta_scratch = nullptr, *raw = nullptr, *decay = nullptr, *gate = nullptr, *identity_gate = nullptr;
    uint32_t *expert_count = nullptr, *expert_list = nullptr;       // counts are zero between feed-forwards
    void *hn = nullptr, *y = nullptr, *cq = nullptr, *q = nullptr, *qa = nullptr, *olat = nullptr, *o = nullptr, *act = nullptr, *low_gate = nullptr;
    uint32_t *row_seq = nullptr, *kv_slot = nullptr, *row_start = nullptr;
    int32_t *pos = nullptr, *tokens = nullptr, *want = nullptr;
    std::vector<float *> cos_sin;
    // expanded latent attention: latents, rotated parts, keys and values of up to `expand_rows` cached tokens
    uint32_t expand_rows = 0;
    void *ec = nullptr, *er = nullptr, *ekv = nullptr;
    uint32_t *expand_meta = nullptr;                 // per distinct window: start [batch + 1], first [batch]
};

// Which cached tokens a pass expands, per distinct window; rows 0: the absorbed form is cheaper
struct ExpandPlan {
    std::vector<uint32_t> rows, meta;
};

}  // namespace

struct LayeredState {
    fa_layered_config cfg{};
    std::vector<Layer> layers;
    std::vector<Tensor> tensors;
    std::vector<fa_buffer *> owned;
    std::vector<Rotation> rotations;                         // distinct ones
    std::vector<double *> rotation_freq;
    std::vector<uint32_t> windows;                           // distinct windows
    void *embed = nullptr;
    double *position_freq = nullptr;                         // additive positions: of every pair of entries
    float *final_norm = nullptr;
    k::LinearWeight head;
    fa_buffer *state_slots = nullptr, *unit_starts = nullptr, *last_rows = nullptr;
    Arena step, pass;
    bool has_state = false, slots_set = false;
    // test aid: the next pass copies the residual after every layer here ([layers, rows, d_model])
    float *trace = nullptr;
    uint64_t trace_rows = 0;
    int is_f32 = 0;
    uint64_t esz = 2;
};

namespace {

// widest of every activation over the layers
struct Widths {
    uint64_t hn = 0, y32 = 0, y = 0, cq = 0, q = 0, qa = 0, olat = 0, o = 0, act = 0, top = 0, experts = 0, raw = 0, decay = 0, low_gate = 0;
};

Widths widths(const LayeredState &L) {
    Widths w;
    w.hn = pad_to(L.cfg.d_model, 64);
    for (const Layer &l : L.layers) {
        w.y = std::max<uint64_t>(w.y, l.lo);
        w.y32 = std::max<uint64_t>(w.y32, pad_to(l.hi, 4));
        w.o = std::max<uint64_t>(w.o, pad_to(l.o_width, 64));
        for (const Mixer &m : l.mixers) {
            if (recurrent(m.cfg)) {
                w.raw = std::max<uint64_t>(w.raw, m.out_width());
                if (m.low_rank.w) {
                    w.decay = std::max<uint64_t>(w.decay, pad_to(m.de.heads * m.de.dim, 4));
                    w.low_gate = std::max<uint64_t>(w.low_gate, pad_to(m.out_width(), 8));
                }
            } else if (m.cfg.mixer == FA_MIXER_ATTENTION) {
                w.q = std::max<uint64_t>(w.q, (uint64_t)m.at.heads * m.at.dim_p);
            } else if (m.cfg.mixer == FA_MIXER_LATENT_ATTENTION) {
                w.cq = std::max<uint64_t>(w.cq, pad_to(m.la.q_rank, 64));
                w.q = std::max<uint64_t>(w.q, (uint64_t)m.la.heads * (m.la.dim_p + m.la.rot_p));
                w.qa = std::max<uint64_t>(w.qa, (uint64_t)m.la.heads * (m.la.rank_p + m.la.rot_p));
                w.olat = std::max<uint64_t>(w.olat, (uint64_t)m.la.heads * m.la.rank_p);
            }
        }
        const uint64_t parts = l.cfg.experts ? l.cfg.top : 1;
        if (l.cfg.d_ffn) w.act = std::max<uint64_t>(w.act, parts * pad_to(l.cfg.d_ffn, 64));
        if (L.cfg.norm != FA_NORM_INPUT && (L.cfg.norm != FA_NORM_INPUT_RMS || l.cfg.experts)) w.y32 = std::max<uint64_t>(w.y32, parts * L.cfg.d_model);
        w.top = std::max<uint64_t>(w.top, l.cfg.experts ? l.cfg.top : 0);
        w.experts = std::max<uint64_t>(w.experts, l.cfg.experts);
    }
    return w;
}

fa_status arena_reserve(fa_context *ctx, LayeredState &L, Arena &a, uint32_t rows, uint32_t expand_rows = 0) {
    if (a.rows >= rows && a.expand_rows >= expand_rows) return FA_OK;
    rows = std::max(rows, a.rows);
    expand_rows = std::max(expand_rows, a.expand_rows);
    if (ctx->capturing) return fail(FA_ERR_CAPTURE_IN_PROGRESS, "layered decoder: activations must be sized before a capture");
    if (a.base) pool_free(ctx, a.base, a.bytes, a.cls);
    a = Arena();
    const Widths w = widths(L);
    const uint64_t R = rows, B = L.cfg.max_batch, E = L.esz;
    uint64_t total = 0;
    std::vector<std::pair<void **, uint64_t>> parts;
    auto add = [&](void **p, uint64_t bytes) {
        parts.emplace_back(p, total);
        total += round_up(bytes + 512, 256);          // slack: operand reads may run past a row's own width
    };
    a.cos_sin.resize(L.rotations.size());
    add((void **)&a.x, R * L.cfg.d_model * 4);
    add((void **)&a.head_x, std::max(R, B) * L.cfg.d_model * 4);
    add(&a.hn, std::max(R, B) * w.hn * E);
    add((void **)&a.y32, R * w.y32 * 4);
    add(&a.y, R * w.y * E);
    add((void **)&a.raw, R * w.raw * 4);
    add((void **)&a.decay, R * w.decay * 4);
    add(&a.low_gate, R * w.low_gate * E);
    add(&a.cq, R * w.cq * E);
    add(&a.q, R * w.q * E);
    add(&a.qa, R * w.qa * E);
    add(&a.olat, R * w.olat * E);
    add(&a.o, R * w.o * E);
    add(&a.act, R * w.act * E);
    add((void **)&a.gate, R * w.top * 4);
    add((void **)&a.identity_gate, w.top ? R * 4 : 0);
    add((void **)&a.expert_count, w.experts * 4);
    add((void **)&a.expert_list, w.experts * R * 4);
    add((void **)&a.row_seq, R * 4);
    add((void **)&a.kv_slot, R * 4);
    add((void **)&a.pos, R * 4);
    add((void **)&a.tokens, R * 4);
    add((void **)&a.want, std::max(R, B) * 4);
    add((void **)&a.row_start, (B + 1) * 4);
    for (size_t i = 0; i < L.rotations.size(); ++i) add((void **)&a.cos_sin[i], R * L.rotations[i].dims * 4);
    uint64_t scratch = 0;
    for (const Layer &l : L.layers)
        for (const Mixer &m : l.mixers)
            if (recurrent(m.cfg)) scratch = std::max(scratch, k::delta_scratch_bytes(m.de, rows, (uint32_t)B));
    add((void **)&a.delta_scratch, scratch);
    uint64_t ec = 0, er = 0, ekv = 0;
    for (const Layer &l : L.layers)
        for (const Mixer &m : l.mixers)
            if (m.cfg.mixer == FA_MIXER_LATENT_ATTENTION) {
                ec = std::max<uint64_t>(ec, pad_to(m.la.rank_p, 64));
                er = std::max<uint64_t>(er, m.la.rot_p);
                ekv = std::max<uint64_t>(ekv, (uint64_t)m.la.heads * (m.la.dim_p + m.la.v_p));
            }
    if (L.is_f32) expand_rows = 0;
    add(&a.ec, expand_rows * ec * E);
    add(&a.er, expand_rows * er * E);
    add(&a.ekv, expand_rows * ekv * E);
    add((void **)&a.expand_meta, L.windows.size() * (2 * B + 1) * 4);
    if (fa_status s = pool_alloc(ctx, total, &a.base, &a.cls)) {
        a = Arena();
        return s;
    }
    a.bytes = total;
    a.rows = rows;
    a.expand_rows = expand_rows;
    for (auto &p : parts) *p.first = (uint8_t *)a.base + p.second;
    k::fill_u32((uint32_t *)a.base, 0, total / 4, ctx->stream);
    return after_launch(ctx, "layered decoder activations");
}

void linear(fa_context *ctx, const LayeredState &L, const void *a, uint64_t lda, uint64_t a_batch, uint64_t m, const k::LinearWeight &w,
            k::LinearEpilogue ep) {
    if (L.is_f32) k::linear_f32((const float *)a, lda, a_batch, m, w, ep, ctx->stream);
    else k::linear_bf16((const uint16_t *)a, lda, a_batch, m, w, ep, ctx->props.multiProcessorCount, ctx->stream);
}

k::LinearEpilogue store_to(void *out, uint64_t ld, int out_f32) {
    k::LinearEpilogue e;
    e.out = out;
    e.ld_out = (uint32_t)ld;
    e.out_f32 = out_f32;
    return e;
}

void linear_grouped(fa_context *ctx, const LayeredState &L, const void *a, uint64_t lda, const k::LinearWeight &w, const k::RowGroups &rg,
                    const k::LinearEpilogue &ep) {
    if (L.is_f32) k::linear_grouped_f32((const float *)a, lda, w, rg, ep, ctx->stream);
    else k::linear_grouped_bf16((const uint16_t *)a, lda, w, rg, ep, ctx->props.multiProcessorCount, ctx->stream);
}

// The new tokens of a pass's sequences, none not counted
struct Portions {
    uint32_t min_new, max_new;
};

// Element `at` of an activation section in the activations' type
void *element(const LayeredState &L, void *base, uint64_t at) { return (uint8_t *)base + at * L.esz; }

// The layer's input a.hn -> what its mixers read, a.y and a.y32.
void enqueue_in(fa_context *ctx, LayeredState &L, Arena &a, const Layer &l, uint32_t rows, uint32_t ld_hn) {
    k::LinearEpilogue e = l.lo ? store_to(a.y, l.lo, L.is_f32) : store_to(a.y32, pad_to(l.hi, 4), 1);
    if (l.lo) {
        e.n_lo = l.lo;
        e.out_hi = a.y32;
        e.ld_hi = pad_to(l.hi, 4);
    }
    e.bias = l.in_bias;
    linear(ctx, L, a.hn, ld_hn, 0, rows, l.in, e);
}

// The mixers: from a.y and a.y32 to their columns of a.o (pitch ld_o).
void enqueue_recurrence(fa_context *ctx, LayeredState &L, Arena &a, const Layer &l, const Mixer &m, const k::RaggedRows &rr, uint32_t max_new, uint32_t ld_o) {
    const k::DeltaShape &sh = m.de;
    const uint32_t ld_hi = pad_to(l.hi, 4), ow = m.out_width();
    k::DeltaIo io{};
    io.y = element(L, a.y, m.lo_at);
    io.ld_y = l.lo;
    io.gate = element(L, a.y, m.lo_at + m.gate_at);
    io.ld_gate = l.lo;
    io.beta = a.y32 + m.hi_at;
    io.ld_beta = ld_hi;
    if (m.low_rank.w) {
        k::LinearEpilogue e = store_to(a.low_gate, pad_to(ow, 8), L.is_f32);
        e.n_lo = pad_to(ow, 8);
        e.out_hi = a.decay;
        e.ld_hi = pad_to(sh.heads * sh.dim, 4);
        linear(ctx, L, element(L, a.y, m.lo_at + m.rank_at), l.lo, 0, rr.rows, m.low_rank, e);
        io.gate = a.low_gate;
        io.ld_gate = e.ld_out;
        io.decay = a.decay;
        io.ld_decay = e.ld_hi;
    } else {
        io.decay = sh.kind == k::Recurrence::kLightning ? m.decay : io.beta + sh.heads;
        io.ld_decay = ld_hi;
    }
    io.conv = m.conv;
    io.a_log = m.a_log;
    io.dt_bias = m.dt_bias;
    io.norm = m.head_norm;
    io.state = m.state;
    io.ring = m.ring;
    io.out = element(L, a.o, m.o_at);
    io.ld_out = ld_o;
    io.out_scale = m.out_scale;
    io.scratch = a.delta_scratch;
    io.raw = a.raw;
    k::delta_mixer(sh, io, L.is_f32, rr, max_new, ctx->stream);
}

void enqueue_latent(fa_context *ctx, const fa_decoder *d, Arena &a, const Layer &l, const Mixer &m, const k::RaggedRows &rr, uint32_t max_new,
                    uint32_t ld_o, const ExpandPlan *expand) {
    LayeredState &L = *d->layered;
    hipStream_t s = ctx->stream;
    const int f32 = L.is_f32;
    const uint32_t M = rr.rows;
    const k::LatentShape &sh = m.la;
    const uint32_t ld_y = pad_to(l.hi, 4), ld_cq = pad_to(sh.q_rank, 64), qw = sh.dim_p + sh.rot_p, kw = sh.rank_p + sh.rot_p;
    const bool own = m.cfg.kv_from < 0;
    const float *cs = a.cos_sin[m.rotation], *y = a.y32 + m.hi_at;
    void *pool = own ? m.pool : L.layers[m.cfg.kv_from].mixers[0].pool, *o = element(L, a.o, m.o_at);
    k::latent_prepare(y, ld_y, m.q_norm, m.kv_norm, cs, a.cq, ld_cq, own ? pool : nullptr, f32, sh, rr, s);
    linear(ctx, L, a.cq, ld_cq, 0, M, m.uq, store_to(a.q, (uint64_t)sh.heads * qw, f32));
    const float *gate = m.cfg.ungated ? nullptr : y + sh.q_rank + (own ? sh.kv_rank + sh.rot : 0);
    if (expand && expand->rows[m.window_index]) {
        const uint32_t *meta = a.expand_meta + (uint64_t)m.window_index * (2 * d->cfg.max_batch + 1);
        const k::LatentExpand ex{meta, meta + d->cfg.max_batch + 1, expand->rows[m.window_index]};
        const uint32_t ld_c = pad_to(sh.rank_p, 64);
        k::latent_rotate_query(a.q, cs, a.q, qw, sh.dim_p, f32, sh, M, s);
        k::latent_gather(pool, a.ec, ld_c, a.er, sh, rr, ex, s);
        linear(ctx, L, a.ec, ld_c, 0, ex.rows, m.ukv, store_to(a.ekv, m.ukv.n, f32));
        k::latent_attention_expanded(a.q, a.ekv, a.er, gate, ld_y, m.out_scale, o, ld_o, sh, rr, ex, s);
    } else {
        k::LinearEpilogue e = store_to(a.qa, (uint64_t)sh.heads * kw, f32);
        e.out_batch = kw;
        linear(ctx, L, a.q, (uint64_t)sh.heads * qw, qw, M, m.uk, e);
        k::latent_rotate_query(a.q, cs, a.qa, kw, sh.rank_p, f32, sh, M, s);
        k::latent_attention(a.qa, pool, a.olat, f32, sh, rr, max_new, ctx->workspace, ctx->props.multiProcessorCount, s);
        e = store_to(o, ld_o, f32);
        if (gate) e.mode = k::LinearEpilogue::kHeadGate;
        e.factor = m.out_scale;
        e.out_batch = sh.vdim;
        e.gate = gate;
        e.ld_gate = ld_y;
        linear(ctx, L, a.olat, (uint64_t)sh.heads * sh.rank_p, sh.rank_p, M, m.uv, e);
    }
}

void enqueue_gated(fa_context *ctx, LayeredState &L, Arena &a, const Layer &l, const Mixer &m, const k::RaggedRows &rr, uint32_t max_new, uint32_t ld_o) {
    k::GatedIo io{};
    io.zu = a.y32 + m.hi_at;
    io.ld_zu = pad_to(l.hi, 4);
    io.z_bias = m.z_bias;
    io.u_bias = m.u_bias;
    io.gate = element(L, a.y, m.lo_at);
    io.ld_gate = l.lo;
    io.state = m.state;
    io.out = element(L, a.o, m.o_at);
    io.ld_out = ld_o;
    io.out_scale = m.out_scale;
    k::gated_mixer(m.cfg.vdim, io, L.is_f32, rr, max_new, ctx->props.multiProcessorCount, ctx->stream);
}

// What an attention mixer does to its scores and to their result; y: its f32 columns
k::AttentionOutput attention_output(const LayeredState &L, const Arena &a, const Layer &l, const Mixer &m) {
    k::AttentionOutput ao;
    ao.slope = m.slope;
    ao.bias = m.score_bias;
    ao.sigmoid = m.cfg.attention & FA_ATTENTION_SIGMOID;
    ao.sink = m.sink;
    if (m.cfg.attention & FA_ATTENTION_GATE) {
        ao.gate = element(L, a.y, m.lo_at + m.gate_at);
        ao.ld_gate = l.lo;
    }
    if (m.cfg.attention & FA_ATTENTION_HEAD_GATE) {
        ao.head_gate = a.y32 + m.hi_at + m.head_gate_at;
        ao.ld_head_gate = pad_to(l.hi, 4);
    }
    ao.scale = m.out_scale;
    return ao;
}

void enqueue_attention(fa_context *ctx, LayeredState &L, Arena &a, const Layer &l, const Mixer &m, const k::RaggedRows &rr, Portions n, uint32_t ld_o) {
    const k::AttentionShape &sh = m.at;
    const uint32_t ld_y = pad_to(l.hi, 4), flags = m.cfg.attention;
    const bool own = m.cfg.kv_from < 0;
    const Mixer &kv = own ? m : L.layers[m.cfg.kv_from].mixers[0];
    const float *y = a.y32 + m.hi_at;
    const bool norms = flags & (FA_ATTENTION_HEAD_NORM | FA_ATTENTION_HEAD_UNIT), key_values = flags & FA_ATTENTION_KEY_VALUES;
    if (norms || key_values || sh.rot || sh.q_temp != 0.0f)
        k::attention_prepare_heads(y, ld_y, norms, m.q_norm, m.k_norm, sh.rot ? a.cos_sin[m.rotation] : nullptr, key_values, a.q, m.k_pool, m.v_pool, L.is_f32,
                                   sh, rr, ctx->stream);
    else
        k::attention_prepare(y, ld_y, m.q_norm, m.k_norm, a.q, m.k_pool, m.v_pool, L.is_f32, sh, rr, ctx->stream);
    k::attention(a.q, kv.k_pool, kv.v_pool, element(L, a.o, m.o_at), ld_o, attention_output(L, a, l, m), L.is_f32, sh, rr, n.min_new, n.max_new, ctx->workspace,
                 ctx->props.multiProcessorCount, ctx->stream);
}

void enqueue_mixers(fa_context *ctx, fa_decoder *d, Arena &a, const Layer &l, const k::RaggedRows &rr, Portions n, uint32_t ld_hn, uint32_t ld_o,
                    const ExpandPlan *expand) {
    LayeredState &L = *d->layered;
    enqueue_in(ctx, L, a, l, rr.rows, ld_hn);
    for (const Mixer &m : l.mixers) {
        if (recurrent(m.cfg)) enqueue_recurrence(ctx, L, a, l, m, rr, n.max_new, ld_o);
        else if (m.cfg.mixer == FA_MIXER_MINGRU) enqueue_gated(ctx, L, a, l, m, rr, n.max_new, ld_o);
        else if (m.cfg.mixer == FA_MIXER_LATENT_ATTENTION) enqueue_latent(ctx, d, a, l, m, rr, n.max_new, ld_o, expand);
        else enqueue_attention(ctx, L, a, l, m, rr, n, ld_o);
    }
}

// Dense feed-forward: from a.hn to what `out` does with the down projection.
void enqueue_dense(fa_context *ctx, LayeredState &L, Arena &a, const Layer &l, uint32_t M, uint32_t ld_hn, const k::LinearEpilogue &out) {
    const uint32_t ld_act = pad_to(l.cfg.d_ffn, 64);
    k::LinearEpilogue g = store_to(a.act, ld_act, L.is_f32);
    g.mode = l.cfg.glu == FA_GLU_SILU ? k::LinearEpilogue::kSiluGlu : l.cfg.glu == FA_FFN_XIELU ? k::LinearEpilogue::kXielu : k::LinearEpilogue::kGlu;
    g.act = l.act;
    g.limit = l.cfg.ffn_limit;
    g.alpha = l.cfg.ffn_alpha;
    linear(ctx, L, a.hn, ld_hn, 0, M, l.gate_up, g);
    linear(ctx, L, a.act, ld_act, 0, M, l.down, out);
}

k::RouteIo route_io(const Arena &a, const Layer &l) {
    k::RouteIo io{l.router.w, l.cfg.experts, l.cfg.top, a.expert_count, a.expert_list, a.rows, a.gate};
    io.scored = l.cfg.route == FA_ROUTE_SCORED;
    io.correction = l.correction;
    io.identity = l.cfg.identity;
    io.groups = l.cfg.groups ? l.cfg.groups : 1;
    io.keep = l.cfg.groups ? l.cfg.groups_kept : 1;
    io.scale = l.cfg.route_scale;
    io.identity_gate = l.cfg.identity ? a.identity_gate : nullptr;
    return io;
}

// Sparse feed-forward: from a.hn to the rows' experts' outputs in a.y32.  The choice of experts is there (route_rows).
void enqueue_experts(fa_context *ctx, LayeredState &L, Arena &a, const Layer &l, uint32_t M, uint32_t ld_hn) {
    const uint32_t D = L.cfg.d_model, ld_act = pad_to(l.cfg.d_ffn, 64), top = l.cfg.top;
    k::RowGroups rg{a.expert_count, a.expert_list, l.lists(), a.rows, top, M * top};
    rg.most = M;
    rg.likely = (uint32_t)((uint64_t)M * top * l.lists() / l.cfg.experts);
    k::LinearEpilogue up = store_to(a.act, ld_act, L.is_f32);
    up.mode = l.cfg.glu == FA_GLU_SILU ? k::LinearEpilogue::kSiluGlu : k::LinearEpilogue::kSquaredRelu;
    linear_grouped(ctx, L, a.hn, ld_hn, l.gate_up, rg, up);
    rg.a_div = 1;
    linear_grouped(ctx, L, a.act, ld_act, l.down, rg, store_to(a.y32, D, 1));
}

// The residual update after the experts
void add_experts(k::ResidualNorm &rn, const Arena &a, const Layer &l) {
    rn.y = a.y32;
    rn.gate = a.gate;
    rn.identity_gate = l.cfg.identity ? a.identity_gate : nullptr;
    rn.parts = l.cfg.top;
    rn.clear = a.expert_count;
    rn.n_clear = l.lists();
}

// All layers over the rows of a pass whose embeddings are in a.x (and, with norms at the output, in a.hn).
fa_status enqueue_layers(fa_context *ctx, fa_decoder *d, Arena &a, const k::RaggedRows &rr, Portions n, uint64_t trace_row0,
                         const ExpandPlan *expand = nullptr) {
    LayeredState &L = *d->layered;
    hipStream_t s = ctx->stream;
    const uint32_t M = rr.rows, D = L.cfg.d_model, ld_hn = pad_to(D, 64);
    const float eps = L.cfg.norm_eps;
    const int f32 = L.is_f32;
    for (size_t i = 0; i < L.rotations.size(); ++i) k::rotation_table(rr.pos, a.cos_sin[i], M, L.rotations[i].dims, L.rotation_freq[i], s);
    if (L.cfg.norm == FA_NORM_BOTH) k::layernorm_rows(a.x, L.layers[0].norm1, a.hn, f32, M, D, ld_hn, eps, s);
    if (L.cfg.norm == FA_NORM_INPUT_RMS) {
        k::ResidualNorm rn;
        rn.kind = k::ResidualNorm::kInput;
        rn.next = L.layers[0].norm1;
        rn.eps = eps;
        k::residual_norm(rn, a.x, a.hn, f32, M, D, ld_hn, nullptr, s);
    }
    for (size_t li = 0; li < L.layers.size(); ++li) {
        const Layer &l = L.layers[li];
        if (L.cfg.norm == FA_NORM_INPUT) k::layernorm_rows(a.x, l.norm1, a.hn, f32, M, D, ld_hn, eps, s);
        const uint32_t ld_o = pad_to(l.o_width, 64);
        enqueue_mixers(ctx, d, a, l, rr, n, ld_hn, ld_o, expand);
        k::ResidualNorm rn;
        rn.y = a.y32;
        rn.eps = eps;
        if (L.cfg.norm == FA_NORM_OUTPUT) {
            linear(ctx, L, a.o, ld_o, 0, M, l.out, store_to(a.y32, D, 1));
            rn.w = l.norm1;
            const k::RouteIo route = route_io(a, l);
            const bool fused = l.cfg.experts && k::residual_norm_routes(f32, M);
            k::residual_norm(rn, a.x, a.hn, f32, M, D, ld_hn, fused ? &route : nullptr, s);
            if (l.cfg.d_ffn) {
                if (l.cfg.experts) {
                    if (!fused) k::route_rows(a.hn, M, ld_hn, route, s);
                    enqueue_experts(ctx, L, a, l, M, ld_hn);
                    add_experts(rn, a, l);
                } else {
                    enqueue_dense(ctx, L, a, l, M, ld_hn, store_to(a.y32, D, 1));
                }
                rn.w = l.norm2;
                k::residual_norm(rn, a.x, a.hn, f32, M, D, ld_hn, nullptr, s);
            }
        } else if (L.cfg.norm == FA_NORM_BOTH) {
            // a residual update norms the new stream for the sublayer that comes next; the head norms its own rows
            const float *next_layer = li + 1 < L.layers.size() ? L.layers[li + 1].norm1 : nullptr;
            linear(ctx, L, a.o, ld_o, 0, M, l.out, store_to(a.y32, D, 1));
            rn.kind = k::ResidualNorm::kBoth;
            rn.w = l.post1;
            rn.next = l.cfg.d_ffn ? l.norm2 : next_layer;
            k::residual_norm(rn, a.x, a.hn, f32, M, D, ld_hn, nullptr, s);
            if (l.cfg.d_ffn) {
                enqueue_dense(ctx, L, a, l, M, ld_hn, store_to(a.y32, D, 1));
                rn.w = l.post2;
                rn.next = next_layer;
                k::residual_norm(rn, a.x, a.hn, f32, M, D, ld_hn, nullptr, s);
            }
        } else if (L.cfg.norm == FA_NORM_INPUT_RMS) {
            // outputs are added where they are made, a sparse feed-forward's with the norm for the sublayer that comes next
            const float *next_layer = li + 1 < L.layers.size() ? L.layers[li + 1].norm1 : nullptr;
            k::LinearEpilogue r = store_to(a.x, D, 1);
            r.mode = k::LinearEpilogue::kResidual;
            linear(ctx, L, a.o, ld_o, 0, M, l.out, r);
            rn.kind = k::ResidualNorm::kInput;
            rn.y = nullptr;
            rn.next = l.cfg.d_ffn ? l.norm2 : next_layer;
            if (l.cfg.experts) {
                const k::RouteIo route = route_io(a, l);
                const bool fused = k::residual_norm_routes(f32, M);
                k::residual_norm(rn, a.x, a.hn, f32, M, D, ld_hn, fused ? &route : nullptr, s);
                if (!fused) k::route_rows(a.hn, M, ld_hn, route, s);
                enqueue_experts(ctx, L, a, l, M, ld_hn);
                add_experts(rn, a, l);
                rn.next = next_layer;
                k::residual_norm(rn, a.x, a.hn, f32, M, D, ld_hn, nullptr, s);
            } else {
                if (rn.next) k::residual_norm(rn, a.x, a.hn, f32, M, D, ld_hn, nullptr, s);
                if (l.cfg.d_ffn) {
                    enqueue_dense(ctx, L, a, l, M, ld_hn, r);
                    rn.next = next_layer;
                    if (rn.next) k::residual_norm(rn, a.x, a.hn, f32, M, D, ld_hn, nullptr, s);
                }
            }
        } else {
            k::LinearEpilogue r = store_to(a.x, D, 1);
            r.mode = k::LinearEpilogue::kResidual;
            r.scale = l.post1;
            linear(ctx, L, a.o, ld_o, 0, M, l.out, r);
            if (l.cfg.d_ffn) {
                k::layernorm_rows(a.x, l.norm2, a.hn, f32, M, D, ld_hn, eps, s);
                r.scale = l.post2;
                enqueue_dense(ctx, L, a, l, M, ld_hn, r);
            }
        }
        if (L.trace) {
            hipError_t e = hipMemcpyAsync(L.trace + (li * L.trace_rows + trace_row0) * D, a.x, (uint64_t)M * D * 4, hipMemcpyDeviceToHost, s);
            if (e == hipSuccess) e = hipStreamSynchronize(s);
            if (e != hipSuccess) return hip_fail(ctx, e, "residual download", FA_ERR_TRANSFER_FAILED);
        }
    }
    return FA_OK;
}

// Embeddings of the pass's tokens.
void enqueue_embed(fa_context *ctx, const LayeredState &L, Arena &a, const int32_t *tokens, const k::RaggedRows &rr) {
    if (L.cfg.norm == FA_NORM_OUTPUT || L.cfg.norm == FA_NORM_INPUT_RMS)
        k::embed_rows(L.embed, L.is_f32, L.cfg.vocab, L.cfg.d_model, tokens, rr.pos, L.position_freq, L.cfg.embed_scale, a.x,
                      L.cfg.norm == FA_NORM_OUTPUT ? a.hn : nullptr, pad_to(L.cfg.d_model, 64), rr.rows, ctx->stream);
    else
        k::gather_rows_any(L.embed, L.is_f32, L.cfg.vocab, L.cfg.d_model, tokens, a.x, rr.rows, ctx->stream);
}

// Final norm and head over rows of f32 residuals.
void enqueue_head(fa_context *ctx, LayeredState &L, Arena &a, const float *x, uint32_t rows, float *logits) {
    const uint32_t ld_hn = pad_to(L.cfg.d_model, 64);
    if (L.cfg.norm == FA_NORM_OUTPUT || L.cfg.norm == FA_NORM_INPUT_RMS) k::rmsnorm_rows(x, L.final_norm, a.hn, L.is_f32, rows, L.cfg.d_model, ld_hn, L.cfg.norm_eps, ctx->stream);
    else k::layernorm_rows(x, L.final_norm, a.hn, L.is_f32, rows, L.cfg.d_model, ld_hn, L.cfg.norm_eps, ctx->stream);
    k::LinearEpilogue e = store_to(logits, L.cfg.vocab, 1);
    e.mode = k::LinearEpilogue::kSoftcap;
    e.factor = L.cfg.logit_scale;
    e.cap = L.cfg.logit_softcap;
    linear(ctx, L, a.hn, ld_hn, 0, rows, L.head, e);
}

k::RaggedRows ragged(const fa_decoder *d, const Arena &a, const uint32_t *row_start, uint32_t rows) {
    const fa_decoder_config &c = d->cfg;
    return k::RaggedRows{row_start, a.row_seq, a.pos, a.kv_slot, (const uint32_t *)d->layered->state_slots->ptr, (const uint32_t *)d->tables->ptr,
                         rows, d->batch, c.block_size, c.max_blocks_per_seq, c.num_blocks};
}

void prepare_rows(fa_context *ctx, fa_decoder *d, Arena &a, const uint32_t *row_start, uint32_t rows) {
    const fa_decoder_config &c = d->cfg;
    k::ragged_prepare(row_start, (const uint32_t *)d->tables->ptr, (const uint32_t *)d->seq_lens->ptr, a.row_seq, a.pos, a.kv_slot,
                      (int32_t *)d->layered->last_rows->ptr, d->batch, rows, c.block_size, c.max_blocks_per_seq, c.num_blocks, ctx->stream);
    k::ragged_advance(row_start, (uint32_t *)d->seq_lens->ptr, d->batch, ctx->stream);
}

fa_status attention_workspace(fa_context *ctx, const LayeredState &L, const Arena &a, uint32_t rows, uint32_t batch, Portions n) {
    uint64_t need = 0;
    const int cus = ctx->props.multiProcessorCount;
    for (const Layer &l : L.layers)
        for (const Mixer &m : l.mixers) {
            if (m.cfg.mixer == FA_MIXER_LATENT_ATTENTION)
                need = std::max(need, k::latent_attention_workspace_bytes(m.la, L.is_f32, rows, batch, n.max_new, cus));
            else if (m.cfg.mixer == FA_MIXER_ATTENTION)
                need = std::max(need, k::attention_workspace_bytes(m.at, attention_output(L, a, l, m), L.is_f32, batch, n.min_new, n.max_new, L.cfg.max_blocks_per_seq * L.cfg.block_size, cus));
        }
    return need ? ensure_workspace(ctx, need) : FA_OK;
}

// The expanded form of a pass, per distinct window: sequence b (lens[b] cached tokens, n[b] new ones) needs the keys its
// first new token sees onwards.  It is taken where forming keys and values per head costs less than attending over
// latents, counted in multiply-adds per head.
ExpandPlan plan_expand(const LayeredState &L, const std::vector<uint32_t> &lens, const std::vector<uint32_t> &n, uint32_t max_batch) {
    constexpr uint64_t kMaxRows = 1u << 17;
    ExpandPlan p;
    p.rows.assign(L.windows.size(), 0);
    p.meta.assign(L.windows.size() * (2 * (size_t)max_batch + 1), 0);
    if (L.is_f32) return p;
    for (size_t w = 0; w < L.windows.size(); ++w) {
        const Mixer *l = nullptr;
        bool ok = true;
        for (const Layer &c : L.layers)
            for (const Mixer &m : c.mixers)
                if (m.cfg.mixer == FA_MIXER_LATENT_ATTENTION && m.window_index == w) {
                    ok = ok && k::latent_expand_applies(m.la);
                    l = &m;
                }
        if (!l || !ok) continue;
        const uint64_t W = L.windows[w];
        uint64_t rows = 0, fresh = 0;
        double pairs = 0;
        uint32_t *start = p.meta.data() + w * (2 * (size_t)max_batch + 1), *first = start + max_batch + 1;
        for (size_t b = 0; b < n.size(); ++b) {
            start[b] = (uint32_t)rows;
            first[b] = lens[b] + 1 > W ? (uint32_t)(lens[b] + 1 - W) : 0;
            if (n[b] == 0) continue;
            rows += (uint64_t)lens[b] + n[b] - first[b];
            fresh += n[b];
            pairs += (double)n[b] * (double)std::min<uint64_t>(W, lens[b] + (n[b] + 1) / 2);
        }
        for (size_t b = n.size(); b <= max_batch; ++b) start[b] = (uint32_t)rows;
        const double up = (double)l->la.kv_rank * (l->la.dim + l->la.vdim);
        const double expanded = rows * up + pairs * (l->la.dim + l->la.rot + l->la.vdim);
        const double absorbed = fresh * up + pairs * (2.0 * l->la.kv_rank + l->la.rot);
        if (rows <= kMaxRows && (k::latent_expand_always() || (expanded < absorbed && fresh >= 128))) p.rows[w] = (uint32_t)rows;
    }
    return p;
}

uint64_t pass_rows() { return g_layered_rows >= 64 ? (uint64_t)g_layered_rows : 8192; }

fa_status upload(fa_context *ctx, void *dst, const void *src, uint64_t bytes) {
    hipError_t e = hipMemcpyAsync(dst, src, bytes, hipMemcpyHostToDevice, ctx->stream);
    if (e == hipSuccess) e = hipStreamSynchronize(ctx->stream);
    return e == hipSuccess ? FA_OK : hip_fail(ctx, e, "upload of a pass", FA_ERR_TRANSFER_FAILED);
}

}  // namespace

void layered_free(fa_context *ctx, fa_decoder *d) {
    LayeredState *L = d->layered;
    for (Arena *a : {&L->step, &L->pass})
        if (a->base) pool_free(ctx, a->base, a->bytes, a->cls);
    for (fa_buffer *b : L->owned) fa_buffer_free(ctx, b);
    delete L;
    d->layered = nullptr;
}

fa_status layered_ready(const fa_decoder *d, const char *what) {
    for (const Tensor &t : d->layered->tensors)
        if (!t.set) return fail(FA_ERR_INVALID_ARGUMENT, std::string(what) + ": tensor " + t.name + " missing");
    if (d->layered->has_state && !d->layered->slots_set) return fail(FA_ERR_INVALID_ARGUMENT, std::string(what) + ": state slots missing");
    return FA_OK;
}

bool layered_has_state(const fa_decoder *d) { return d->layered->has_state; }

fa_status layered_sequences_set(fa_context *ctx, fa_decoder *d) {
    LayeredState &L = *d->layered;
    L.slots_set = d->batch <= L.cfg.state_slots;
    if (!L.slots_set) return FA_OK;
    std::vector<uint32_t> iota(d->batch);
    for (uint32_t b = 0; b < d->batch; ++b) iota[b] = b;
    return fa_upload_into(ctx, iota.data(), d->batch, L.state_slots, 0);
}

fa_status layered_prepare_step(fa_context *ctx, fa_decoder *d) {
    LayeredState &L = *d->layered;
    if (fa_status s = arena_reserve(ctx, L, L.step, L.cfg.max_batch)) return s;
    return attention_workspace(ctx, L, L.step, d->batch, d->batch, Portions{1, 1});
}

fa_status layered_enqueue_step(fa_context *ctx, fa_decoder *d) {
    LayeredState &L = *d->layered;
    Arena &a = L.step;
    const uint32_t B = d->batch;
    const uint32_t *starts = (const uint32_t *)L.unit_starts->ptr;
    prepare_rows(ctx, d, a, starts, B);
    const k::RaggedRows rr = ragged(d, a, starts, B);
    enqueue_embed(ctx, L, a, (const int32_t *)d->tokens->ptr, rr);
    if (fa_status s = enqueue_layers(ctx, d, a, rr, Portions{1, 1}, 0)) return s;
    enqueue_head(ctx, L, a, a.x, B, (float *)d->logits->ptr);
    enqueue_pick(d, ctx->stream);
    return after_launch(ctx, "layered decoder step");
}

fa_status layered_forward(fa_context *ctx, fa_decoder *d, const uint32_t *counts, const int32_t *tokens, uint64_t n_want,
                          const uint32_t *want, float *logits, int32_t *picked) {
    LayeredState &L = *d->layered;
    const fa_decoder_config &c = d->cfg;
    const uint32_t B = d->batch;
    if (fa_status s = layered_ready(d, "decoder pass")) return s;
    uint64_t total = 0;
    for (uint32_t b = 0; b < B; ++b) {
        const uint64_t end = (uint64_t)d->host_lens[b] + counts[b];
        if (end > (uint64_t)c.max_blocks_per_seq * c.block_size)
            return fail(FA_ERR_INVALID_ARGUMENT, "paged_kv: row " + std::to_string(b) + " has no room for the prompt");
        for (uint64_t i = 0; i < (end + c.block_size - 1) / c.block_size; ++i)
            if (d->host_tables[(uint64_t)b * c.max_blocks_per_seq + i] >= c.num_blocks)
                return fail(FA_ERR_INVALID_ARGUMENT, "paged_kv: row " + std::to_string(b) + " entry " + std::to_string(i) + " is not a valid block id");
        total += counts[b];
    }
    if (total == 0 || total > INT32_MAX) return fail(FA_ERR_INVALID_ARGUMENT, "decoder pass: no tokens");
    for (uint64_t i = 0; i < total; ++i)
        if (tokens[i] < 0 || (uint32_t)tokens[i] >= c.vocab) return fail(FA_ERR_INVALID_ARGUMENT, "decoder pass: token id outside the vocabulary");
    const bool last_only = want == nullptr && picked == nullptr && logits == nullptr;
    for (uint64_t i = 0; i < n_want; ++i)
        if (want[i] >= total || (i && want[i] <= want[i - 1]))
            return fail(FA_ERR_INVALID_ARGUMENT, "decoder pass: wanted places must be ascending and below the number of tokens");
    if (last_only)
        for (uint32_t b = 0; b < B; ++b)
            if (counts[b] == 0) return fail(FA_ERR_INVALID_ARGUMENT, "decoder pass: row " + std::to_string(b) + " brings no tokens");

    // the arena grows in powers of two up to a full pass
    const uint64_t budget = pass_rows();
    uint32_t cap = 64;
    while (cap < std::min<uint64_t>(total, budget)) cap *= 2;
    if (fa_status s = arena_reserve(ctx, L, L.pass, cap)) return s;
    Arena &a = L.pass;
    // logits of wanted rows: at most kHeadRows at a time
    constexpr uint32_t kHeadRows = 1024;
    fa_buffer *lbuf = nullptr, *pbuf = nullptr;
    if (n_want) {
        const uint64_t rows = std::min<uint64_t>({n_want, kHeadRows, a.rows});
        if (fa_status s = make_buffer(ctx, FA_F32, rows * c.vocab, false, &lbuf)) return s;
        if (picked)
            if (fa_status s = make_buffer(ctx, FA_I32, rows, false, &pbuf)) {
                fa_buffer_free(ctx, lbuf);
                return s;
            }
    }
    auto run = [&]() -> fa_status {
        std::vector<uint32_t> done(B, 0), starts(B + 1), first(B), fresh(B);
        std::vector<int32_t> stage, pick_rows;
        uint64_t w_at = 0, placed = 0, tok0 = 0;
        for (uint32_t b = 0; b < B; ++b) {
            first[b] = (uint32_t)tok0;
            tok0 += counts[b];
        }
        while (placed < total) {
            // sequences in order, each as much as the pass has room for
            uint32_t rows = 0;
            Portions portions{0xffffffffu, 0};
            stage.clear();
            pick_rows.clear();
            std::vector<int32_t> last(B, -1);
            const uint64_t w_lo = w_at;
            for (uint32_t b = 0; b < B; ++b) {
                starts[b] = rows;
                const uint32_t n = (uint32_t)std::min<uint64_t>(counts[b] - done[b], budget - rows);
                if (n == 0) continue;
                const uint32_t g0 = first[b] + done[b];
                for (uint32_t i = 0; i < n; ++i) stage.push_back(tokens[g0 + i]);
                while (w_at < n_want && want[w_at] < g0 + n) pick_rows.push_back((int32_t)(rows + want[w_at++] - g0));
                done[b] += n;
                rows += n;
                portions.min_new = std::min(portions.min_new, n);
                portions.max_new = std::max(portions.max_new, n);
                if (done[b] == counts[b]) last[b] = (int32_t)rows - 1;
            }
            starts[B] = rows;
            for (uint32_t b = 0; b < B; ++b) fresh[b] = starts[b + 1] - starts[b];
            const ExpandPlan expand = plan_expand(L, d->host_lens, fresh, c.max_batch);
            uint32_t e_rows = 0;
            for (uint32_t r : expand.rows) e_rows = std::max(e_rows, r);
            if (e_rows) {
                uint32_t e_cap = 256;
                while (e_cap < e_rows) e_cap *= 2;
                if (fa_status s = arena_reserve(ctx, L, a, a.rows, e_cap)) return s;
                if (fa_status s = upload(ctx, a.expand_meta, expand.meta.data(), expand.meta.size() * 4)) return s;
            }
            if (fa_status s = attention_workspace(ctx, L, a, rows, B, portions)) return s;
            if (fa_status s = upload(ctx, a.row_start, starts.data(), (B + 1) * 4)) return s;
            if (fa_status s = upload(ctx, a.tokens, stage.data(), (uint64_t)rows * 4)) return s;
            prepare_rows(ctx, d, a, a.row_start, rows);
            const k::RaggedRows rr = ragged(d, a, a.row_start, rows);
            enqueue_embed(ctx, L, a, a.tokens, rr);
            if (fa_status s = enqueue_layers(ctx, d, a, rr, portions, placed, &expand)) return s;
            for (uint32_t b = 0; b < B; ++b) d->host_lens[b] += starts[b + 1] - starts[b];
            placed += rows;
            if (last_only) {
                // the last rows of the sequences that end in this pass wait in the decoder's own residual rows
                for (uint32_t b = 0; b < B; ++b)
                    if (last[b] >= 0) {
                        hipError_t e = hipMemcpyAsync((float *)d->h->ptr + (uint64_t)b * c.d_model, a.x + (uint64_t)last[b] * c.d_model,
                                                      (uint64_t)c.d_model * 4, hipMemcpyDeviceToDevice, ctx->stream);
                        if (e != hipSuccess) return hip_fail(ctx, e, "last rows", FA_ERR_TRANSFER_FAILED);
                    }
            }
            for (uint64_t i = 0; i < pick_rows.size(); i += kHeadRows) {
                const uint32_t n = (uint32_t)std::min<uint64_t>(pick_rows.size() - i, kHeadRows);
                if (fa_status s = upload(ctx, a.want, pick_rows.data() + i, (uint64_t)n * 4)) return s;
                k::gather_rows_f32(a.x, rows, c.d_model, a.want, a.head_x, n, ctx->stream);
                enqueue_head(ctx, L, a, a.head_x, n, (float *)lbuf->ptr);
                hipError_t e = hipSuccess;
                if (logits) e = hipMemcpyAsync(logits + (w_lo + i) * c.vocab, lbuf->ptr, (uint64_t)n * c.vocab * 4, hipMemcpyDeviceToHost, ctx->stream);
                if (picked && e == hipSuccess) {
                    k::argmax_rows_f32((const float *)lbuf->ptr, (int32_t *)pbuf->ptr, n, c.vocab, ctx->stream);
                    e = hipMemcpyAsync(picked + w_lo + i, pbuf->ptr, (uint64_t)n * 4, hipMemcpyDeviceToHost, ctx->stream);
                }
                if (e == hipSuccess) e = hipStreamSynchronize(ctx->stream);
                if (e != hipSuccess) return hip_fail(ctx, e, "logits download", FA_ERR_TRANSFER_FAILED);
            }
        }
        if (last_only) {
            enqueue_head(ctx, L, a, (const float *)d->h->ptr, B, (float *)d->logits->ptr);
            enqueue_pick(d, ctx->stream);
        }
        return after_launch(ctx, "layered decoder pass");
    };
    fa_status st;
    try {
        st = run();
    } catch (const std::exception &) {
        st = fail(FA_ERR_ALLOCATION_FAILED, "decoder pass: out of host memory");
    }
    L.trace = nullptr;
    if (lbuf) fa_buffer_free(ctx, lbuf);
    if (pbuf) fa_buffer_free(ctx, pbuf);
    return st;
}

}  // namespace fa

using namespace fa;

namespace {

fa_status check_layered(const fa_decoder *d, const char *what) {
    if (!d || d->magic != kDecMagic) return fail(FA_ERR_INVALID_ARGUMENT, "decoder: not a decoder");
    if (!d->layered) return fail(FA_ERR_UNSUPPORTED, std::string(what) + ": layered decoders only");
    return FA_OK;
}

// One mixer; alone: it is the only one of its layer.
fa_status check_mixer(const fa_layered_config &c, const fa_layer_config &l, uint32_t i, bool alone) {
    auto bad = [&](const char *why) { return fail(FA_ERR_INVALID_ARGUMENT, "layer " + std::to_string(i) + ": " + why); };
    if (l.mixer == FA_MIXER_MINGRU) {
        if (l.heads != 1 || l.vdim == 0 || l.vdim > 65536) return bad("a minimal gated recurrence has one head of a width up to 65536");
        if (c.state_slots == 0) return bad("a recurrent layer needs state slots");
        return FA_OK;
    }
    if (l.heads == 0 || l.dim == 0 || l.vdim == 0 || l.heads > 1024 || l.dim > 4096 || l.vdim > 4096) return bad("heads, dim and vdim must be positive");
    if (l.mixer == FA_MIXER_DELTA || l.mixer == FA_MIXER_LIGHTNING) {
        if (l.dim > k::kDeltaMaxDim || l.vdim > k::kDeltaMaxVdim) return fail(FA_ERR_UNSUPPORTED, "delta layer: dim above 256 or vdim above 1024");
        if (c.state_slots == 0) return bad("a recurrent layer needs state slots");
        if (l.mixer == FA_MIXER_LIGHTNING) {
            if (!l.decay) return bad("lightning attention needs its decays");
            for (uint32_t h = 0; h < l.heads; ++h)
                if (!(l.decay[h] >= 0.0f && l.decay[h] <= 1.0f)) return bad("decays must be between 0 and 1");
            return FA_OK;
        }
        if (l.kv_heads == 0 || l.heads % l.kv_heads != 0) return bad("heads must be a multiple of kv_heads");
        if (l.conv == 0 || l.conv > 16) return bad("the convolution takes 1 to 16 taps");
        if ((l.decay_rank == 0) != (l.gate_rank == 0)) return bad("low-rank decays and gates go together");
        if (l.decay_rank > 65536 || l.gate_rank > 65536) return bad("bad ranks");
        return FA_OK;
    }
    if (!std::isfinite(l.scale)) return bad("bad scale");
    if (l.mixer == FA_MIXER_LATENT_ATTENTION) {
        if (l.q_rank == 0 || l.kv_rank == 0) return bad("q_rank and kv_rank must be positive");
        if (l.rot_dim == 0 || l.rot_dim % 2 != 0) return bad("rot_dim must be positive and even");
        if (l.kv_rank > 2048 || l.rot_dim > 1024) return fail(FA_ERR_UNSUPPORTED, "latent attention: kv_rank above 2048 or rot_dim above 1024");
    } else if (l.mixer == FA_MIXER_ATTENTION) {
        if (l.kv_heads == 0 || l.heads % l.kv_heads != 0) return bad("heads must be a multiple of kv_heads");
        const uint32_t per_head = FA_ATTENTION_HEAD_NORM | FA_ATTENTION_HEAD_UNIT, all = FA_ATTENTION_BIAS | FA_ATTENTION_QK_NORM | per_head |
                                                                                        FA_ATTENTION_KEY_VALUES | FA_ATTENTION_GATE | FA_ATTENTION_SINK | FA_ATTENTION_SIGMOID |
                                                                                        FA_ATTENTION_HEAD_GATE;
        if (l.attention & ~all) return bad("unknown attention flags");
        if ((l.attention & per_head) == per_head) return bad("one kind of norm per head");
        if ((l.attention & FA_ATTENTION_SIGMOID) && (l.attention & FA_ATTENTION_SINK)) return bad("a sink needs a softmax");
        if (!std::isfinite(l.distance) || !std::isfinite(l.q_temp) || (l.q_temp != 0.0f && l.q_temp_every == 0)) return bad("bad distance or query temperature");
        const bool heads_form = (l.attention & (per_head | FA_ATTENTION_KEY_VALUES)) || l.rot_dim || l.q_temp != 0.0f;
        if (heads_form && (l.attention & FA_ATTENTION_QK_NORM)) return fail(FA_ERR_UNSUPPORTED, "attention: norms over all heads beside norms per head, keys as values, rotation or query temperature");
        if ((l.attention & FA_ATTENTION_BIAS) && (!alone || (l.attention & (FA_ATTENTION_GATE | FA_ATTENTION_HEAD_GATE)))) return fail(FA_ERR_UNSUPPORTED, "attention: biases beside a gate or a second mixer");
        if ((l.attention & FA_ATTENTION_KEY_VALUES) && l.vdim != l.dim) return bad("keys as values need vdim = dim");
        if (l.rot_dim % 2 != 0 || l.rot_dim > l.dim) return bad("rot_dim must be even and at most dim");
        if (heads_form && l.kv_from >= 0) return fail(FA_ERR_UNSUPPORTED, "attention: an earlier layer's cache beside norms per head, keys as values or rotation");
    } else {
        return bad("unknown mixer");
    }
    if (l.rot_dim && !(l.rot_base > 0.0)) return bad("bad rotation base");
    if (l.rot_dim && l.rot_factor > 0.0 && !(std::isfinite(l.rot_factor) && l.rot_high > l.rot_low && l.rot_original > 0.0)) return bad("bad rotation scaling");
    if (l.kv_from < 0) return FA_OK;
    if (!alone) return fail(FA_ERR_UNSUPPORTED, "two mixers side by side: caches of their own only");
    if ((uint32_t)l.kv_from >= i) return bad("kv_from must name an earlier layer");
    const fa_layer_config &j = c.layers[l.kv_from];
    if (j.right) return fail(FA_ERR_UNSUPPORTED, "kv_from names a layer of two mixers");
    if (j.mixer != l.mixer || j.kv_from >= 0) return bad("kv_from must name an attention layer of the same kind with a cache of its own");
    if (l.mixer == FA_MIXER_LATENT_ATTENTION) {
        if (j.kv_rank != l.kv_rank || j.rot_interleaved != l.rot_interleaved || !(rotation_of(j) == rotation_of(l)))
            return bad("kv_from: the two layers' latents or rotations differ");
    } else {
        if (j.kv_heads != l.kv_heads || j.dim != l.dim || j.vdim != l.vdim) return bad("kv_from: the two layers' key and value sizes differ");
        if (j.rot_dim || (j.attention & (FA_ATTENTION_HEAD_NORM | FA_ATTENTION_HEAD_UNIT | FA_ATTENTION_KEY_VALUES)))
            return fail(FA_ERR_UNSUPPORTED, "kv_from names a layer with norms per head, keys as values or rotation");
    }
    return FA_OK;
}

fa_status check_layer(const fa_layered_config &c, uint32_t i) {
    const fa_layer_config &l = c.layers[i];
    auto bad = [&](const char *why) { return fail(FA_ERR_INVALID_ARGUMENT, "layer " + std::to_string(i) + ": " + why); };
    if (fa_status s = check_mixer(c, l, i, !l.right)) return s;
    if (l.right) {
        if (fa_status s = check_mixer(c, *l.right, i, false)) return s;
        if (!std::isfinite(l.left_scale) || !std::isfinite(l.right_scale)) return bad("bad scale of a mixer");
    }
    if (l.experts) {
        if (l.experts > k::kMaxExperts || l.identity >= l.experts || l.top > k::kMaxTop)
            return fail(FA_ERR_UNSUPPORTED, "sparse experts: none or more than 256 of them, or more than 64 per token");
        if (l.top == 0 || l.top > l.experts || l.d_ffn == 0) return bad("top must be between 1 and experts, d_ffn positive");
        if (c.norm != FA_NORM_OUTPUT && c.norm != FA_NORM_INPUT_RMS) return fail(FA_ERR_UNSUPPORTED, "sparse experts: with RMS norms only");
        if (l.glu != FA_GLU_CLAMPED && l.glu != FA_GLU_SILU) return bad("experts: unknown feed-forward");
        if (l.route != FA_ROUTE_CHOSEN && l.route != FA_ROUTE_SCORED) return bad("unknown choice of experts");
        if (l.route == FA_ROUTE_SCORED) {
            if (!std::isfinite(l.route_scale)) return bad("bad scale of the experts' weights");
            if (l.groups && (l.experts % l.groups != 0 || l.groups_kept == 0 || l.groups_kept > l.groups || l.top > l.experts / l.groups * l.groups_kept))
                return bad("groups must be equal, and those kept hold at least `top` experts");
        } else if (l.groups) {
            return fail(FA_ERR_UNSUPPORTED, "groups of experts need scores");
        }
        return FA_OK;
    }
    if (l.glu != FA_GLU_CLAMPED && l.glu != FA_GLU_SILU && l.glu != FA_FFN_XIELU) return bad("unknown feed-forward");
    if (l.d_ffn && l.glu == FA_GLU_CLAMPED && !(l.ffn_limit >= 0.0f && std::isfinite(l.ffn_alpha))) return bad("bad feed-forward constants");
    return FA_OK;
}

}  // namespace

extern "C" {

fa_status fa_decoder_create_layered(fa_context *ctx, const fa_layered_config *cfg, fa_decoder **out) {
    if (fa_status s = check_ctx(ctx)) return s;
    if (!cfg || !out || !cfg->layers) return fail(FA_ERR_INVALID_ARGUMENT, "decoder_create_layered: null argument");
    if (ctx->capturing) return fail(FA_ERR_CAPTURE_IN_PROGRESS, "decoder_create_layered during graph capture");
    const fa_layered_config &c = *cfg;
    if (c.n_layers == 0 || c.d_model == 0 || c.vocab == 0 || c.max_batch == 0) return fail(FA_ERR_INVALID_ARGUMENT, "decoder_create_layered: zero dimension");
    if (c.max_batch > 256) return fail(FA_ERR_UNSUPPORTED, "decoder_create_layered: at most 256 sequences per step");
    if (c.d_model > 16384) return fail(FA_ERR_UNSUPPORTED, "decoder_create_layered: d_model above 16384");
    if (c.dtype != FA_BF16 && c.dtype != FA_F32) return fail(FA_ERR_INVALID_ARGUMENT, "decoder_create_layered: dtype must be bf16 or f32");
    if (!std::isfinite(c.norm_eps) || c.norm_eps < 0.0f || !std::isfinite(c.logit_softcap)) return fail(FA_ERR_INVALID_ARGUMENT, "decoder_create_layered: bad constants");
    if (c.norm < FA_NORM_INPUT || c.norm > FA_NORM_INPUT_RMS || !std::isfinite(c.embed_scale) || !std::isfinite(c.position_base) || c.position_base < 0.0 ||
        !std::isfinite(c.logit_scale))
        return fail(FA_ERR_INVALID_ARGUMENT, "decoder_create_layered: bad norm, embed_scale, position_base or logit_scale");
    if (c.norm != FA_NORM_OUTPUT && c.norm != FA_NORM_INPUT_RMS && (c.position_base > 0.0 || (c.embed_scale != 0.0f && c.embed_scale != 1.0f)))
        return fail(FA_ERR_UNSUPPORTED, "decoder_create_layered: scaled or positioned embeddings need RMS norms");
    if (c.block_size == 0 || (c.block_size & (c.block_size - 1)) != 0 || c.block_size > 256 || c.num_blocks == 0)
        return fail(FA_ERR_INVALID_ARGUMENT, "decoder_create_layered: block_size must be a power of two up to 256, num_blocks positive");
    if (c.max_blocks_per_seq == 0 || (uint64_t)c.max_blocks_per_seq * c.block_size > (uint64_t)INT32_MAX)
        return fail(FA_ERR_INVALID_ARGUMENT, "decoder_create_layered: bad max_blocks_per_seq");
    for (uint32_t i = 0; i < c.n_layers; ++i)
        if (fa_status s = check_layer(c, i)) return s;

    fa_decoder *d = new (std::nothrow) fa_decoder();
    LayeredState *L = new (std::nothrow) LayeredState();
    if (!d || !L) {
        delete d;
        delete L;
        return fail(FA_ERR_ALLOCATION_FAILED, "decoder_create_layered: host allocation failed");
    }
    d->magic = kDecMagic;
    d->ctx = ctx;
    d->layered = L;
    d->cfg = fa_decoder_config{};
    d->cfg.n_layers = c.n_layers;
    d->cfg.d_model = c.d_model;
    d->cfg.vocab = c.vocab;
    d->cfg.block_size = c.block_size;
    d->cfg.max_blocks_per_seq = c.max_blocks_per_seq;
    d->cfg.num_blocks = c.num_blocks;
    d->cfg.max_batch = c.max_batch;
    fa_status st = FA_OK;
    try {
        L->cfg = c;
        L->cfg.layers = nullptr;                             // the caller's; every layer keeps its own
        if (L->cfg.logit_scale == 0.0f) L->cfg.logit_scale = 1.0f;
        if (L->cfg.embed_scale == 0.0f) L->cfg.embed_scale = 1.0f;
        L->is_f32 = c.dtype == FA_F32;
        L->esz = L->is_f32 ? 4 : 2;
        const int f32 = L->is_f32;
        auto mk = [&](fa_dtype t, uint64_t n, fa_buffer **b) {
            if (st == FA_OK) st = make_buffer(ctx, t, n, true, b);
        };
        auto own = [&](fa_dtype t, uint64_t n) -> void * {
            fa_buffer *b = nullptr;
            mk(t, n, &b);
            if (b) L->owned.push_back(b);
            return b ? b->ptr : nullptr;
        };
        auto add = [&](const std::string &name, uint64_t rows, uint64_t cols, std::function<void(const void *, int, hipStream_t)> place) {
            L->tensors.push_back(Tensor{name, rows, cols, false, std::move(place)});
        };
        // f32 vector (or small matrix) in row-major order
        auto vec = [&](const std::string &name, uint64_t rows, uint64_t cols, float *dst) {
            const uint64_t n = rows * (cols ? cols : 1);
            add(name, rows, cols, [=](const void *src, int src_f32, hipStream_t s) {
                if (src_f32) (void)hipMemcpyAsync(dst, src, n * 4, hipMemcpyDeviceToDevice, s);
                else k::convert_bf16_to_f32((const uint16_t *)src, dst, n, s);
            });
        };
        auto weight = [&](uint32_t n_store, uint32_t n_cols, uint32_t kk, uint32_t batches = 1) {
            k::LinearWeight w;
            w.n = n_store;
            w.n_tiles = (n_cols + 15) / 16;
            w.k_tiles = pad_to(kk, 64) / 32;
            w.batches = batches;
            w.w = own(f32 ? FA_F32 : FA_BF16, (uint64_t)batches * w.n_tiles * 16 * w.k_tiles * 32);
            return w;
        };
        // whole linear [rows, cols] into output columns n0 ..
        auto lin = [&](const std::string &name, uint32_t rows, uint32_t cols, const k::LinearWeight &w, uint32_t n0, uint32_t group = 0, uint32_t pitch = 0,
                       uint32_t k0 = 0) {
            add(name, rows, cols, [=](const void *src, int src_f32, hipStream_t s) {
                k::pack_linear(src, src_f32, cols, 1, rows, cols, (void *)w.w, f32, w.k_tiles, n0, group ? group : 0x40000000u, pitch, s, k0);
            });
        };
        auto row_ptr = [](const void *src, int src_f32, uint64_t elem) { return (const void *)((const uint8_t *)src + elem * (src_f32 ? 4 : 2)); };

        const uint32_t D = c.d_model;
        L->embed = own(f32 ? FA_F32 : FA_BF16, (uint64_t)c.vocab * D);
        {
            void *dst = L->embed;
            const uint64_t n = (uint64_t)c.vocab * D;
            add("embed", c.vocab, D, [=](const void *src, int src_f32, hipStream_t s) {
                if (src_f32 == f32) (void)hipMemcpyAsync(dst, src, n * (f32 ? 4 : 2), hipMemcpyDeviceToDevice, s);
                else if (f32) k::convert_bf16_to_f32((const uint16_t *)src, (float *)dst, n, s);
                else k::convert_f32_to_bf16((const float *)src, (uint16_t *)dst, n, s);
            });
        }
        if (c.position_base > 0.0) {
            std::vector<double> freq((D + 1) / 2);
            for (uint32_t i = 0; i < freq.size(); ++i) freq[i] = std::pow(c.position_base, -2.0 * (double)i / (double)D);
            L->position_freq = (double *)own(FA_F32, 2 * freq.size());
            if (st == FA_OK) st = fa_upload_into(ctx, freq.data(), 2 * freq.size(), L->owned.back(), 0);
        }
        // what sublayer outputs pass on their way to the residual: a layer scale or a second norm
        const char *post[4][2] = {{"ls1", "ls2"}, {nullptr, nullptr}, {"norm1b", "norm2b"}, {nullptr, nullptr}};
        const uint32_t max_ctx = (uint32_t)std::min<uint64_t>((uint64_t)c.max_blocks_per_seq * c.block_size, k::kWholeContext);
        auto rotation = [&](Mixer &m) {
            const Rotation r = rotation_of(m.cfg);
            m.rotation = (uint32_t)(std::find(L->rotations.begin(), L->rotations.end(), r) - L->rotations.begin());
            if (m.rotation < L->rotations.size()) return;
            L->rotations.push_back(r);
            const std::vector<double> f = frequencies(r);
            L->rotation_freq.push_back((double *)own(FA_F32, 2 * f.size()));
            if (st == FA_OK) st = fa_upload_into(ctx, f.data(), 2 * f.size(), L->owned.back(), 0);
        };
        // How many columns of `in` a mixer takes, in its own order: first those kept in the activations' type, then the f32 ones.
        auto measure = [&](Mixer &m) {
            const fa_layer_config &g = m.cfg;
            const uint32_t ow = m.out_width();
            if (recurrent(g)) {
                const bool lightning = g.mixer == FA_MIXER_LIGHTNING, low_rank = g.decay_rank && !lightning;
                const k::Recurrence kind = lightning ? k::Recurrence::kLightning : low_rank ? k::Recurrence::kChannelDelta : k::Recurrence::kDelta;
                m.de = k::DeltaShape{kind, g.heads, lightning ? g.heads : g.kv_heads, g.dim, g.vdim, lightning ? 0 : g.conv, lightning, lightning || low_rank, c.norm_eps};
                m.gate_at = m.de.qkv();
                m.rank_at = pad_to(m.de.qkv(), 8);
                m.lo = low_rank ? m.rank_at + pad_to(g.decay_rank, 8) + g.gate_rank : m.gate_at + ow;
                m.hi = lightning ? 0 : low_rank ? g.heads : 2 * g.heads;
            } else if (g.mixer == FA_MIXER_MINGRU) {
                m.lo = ow;
                m.hi = 2 * ow;
            } else if (g.mixer == FA_MIXER_ATTENTION) {
                const bool own_kv = g.kv_from < 0;
                m.hi = g.heads * g.dim + (own_kv ? g.kv_heads * g.dim + (g.attention & FA_ATTENTION_KEY_VALUES ? 0 : g.kv_heads * g.vdim) : 0);
                m.head_gate_at = m.hi;
                if (g.attention & FA_ATTENTION_HEAD_GATE) m.hi += g.heads;
                m.lo = g.attention & FA_ATTENTION_GATE ? ow : 0;
            } else {
                m.hi = g.q_rank + (g.kv_from < 0 ? g.kv_rank + g.rot_dim : 0) + (g.ungated ? 0 : g.heads);
            }
        };
        auto set_recurrence = [&](Mixer &m, const Layer &l) {
            const fa_layer_config &g = m.cfg;
            const uint32_t H = g.heads, ow = m.out_width(), nq = m.de.kv_heads * g.dim, ch = m.de.qkv(), lo = m.lo_at, hi = l.lo + m.hi_at;
            L->has_state = true;
            lin(m.prefix + "q", nq, D, l.in, lo);
            lin(m.prefix + "k", nq, D, l.in, lo + nq);
            lin(m.prefix + "v", ow, D, l.in, lo + 2 * nq);
            const uint32_t n_norm = m.de.norm_all ? ow : g.vdim;
            m.head_norm = (float *)own(FA_F32, n_norm);
            vec(m.prefix + "norm", n_norm, 0, m.head_norm);
            m.state = (float *)own(FA_F32, (uint64_t)c.state_slots * H * g.dim * m.de.vdim_p());
            if (m.de.kind == k::Recurrence::kLightning) {
                lin(m.prefix + "g", ow, D, l.in, lo + m.gate_at);
                m.decay = (float *)own(FA_F32, H);
                if (st == FA_OK) st = fa_upload_into(ctx, g.decay, H, L->owned.back(), 0);
                return;
            }
            lin(m.prefix + "b", H, D, l.in, hi);
            m.conv = (float *)own(FA_F32, (uint64_t)ch * g.conv);
            vec(m.prefix + "q.conv", nq, g.conv, m.conv);
            vec(m.prefix + "k.conv", nq, g.conv, m.conv + (uint64_t)nq * g.conv);
            vec(m.prefix + "v.conv", ow, g.conv, m.conv + 2ull * nq * g.conv);
            m.ring = own(f32 ? FA_F32 : FA_BF16, (uint64_t)c.state_slots * g.conv * ch);
            const uint32_t n_decay = g.decay_rank ? H * g.dim : H;
            m.a_log = (float *)own(FA_F32, H);
            m.dt_bias = (float *)own(FA_F32, n_decay);
            vec(m.prefix + "A_log", H, 0, m.a_log);
            vec(m.prefix + "dt_bias", n_decay, 0, m.dt_bias);
            if (g.decay_rank) {
                const uint32_t gate_k = pad_to(g.decay_rank, 8), decay_n = pad_to(ow, 8);
                m.low_rank = weight(decay_n + n_decay, decay_n + n_decay, gate_k + g.gate_rank);
                lin(m.prefix + "a1", g.decay_rank, D, l.in, lo + m.rank_at);
                lin(m.prefix + "g1", g.gate_rank, D, l.in, lo + m.rank_at + gate_k);
                lin(m.prefix + "a2", n_decay, g.decay_rank, m.low_rank, decay_n);
                lin(m.prefix + "g2", ow, g.gate_rank, m.low_rank, 0, 0, 0, gate_k);
            } else {
                lin(m.prefix + "g", ow, D, l.in, lo + m.gate_at);
                lin(m.prefix + "a", H, D, l.in, hi + H);
            }
        };
        auto set_gated = [&](Mixer &m, const Layer &l) {
            const uint32_t ow = m.out_width(), hi = l.lo + m.hi_at;
            L->has_state = true;
            m.z_bias = (float *)own(FA_F32, k::gated_pitch(ow));
            m.u_bias = (float *)own(FA_F32, k::gated_pitch(ow));
            lin(m.prefix + "z", ow, D, l.in, hi);
            lin(m.prefix + "x", ow, D, l.in, hi + ow);
            lin(m.prefix + "g", ow, D, l.in, m.lo_at);
            vec(m.prefix + "z.b", ow, 0, m.z_bias);
            vec(m.prefix + "x.b", ow, 0, m.u_bias);
            m.state = (float *)own(FA_F32, (uint64_t)c.state_slots * k::gated_pitch(ow));
        };
        auto set_attention = [&](Mixer &m, Layer &l) {
            const fa_layer_config &g = m.cfg;
            const uint32_t H = g.heads, hi = l.lo + m.hi_at;
            k::AttentionShape &a = m.at;
            a = k::AttentionShape{H, g.kv_heads, g.dim, g.vdim, 0, 0, g.scale, c.norm_eps, (uint64_t)c.num_blocks * c.block_size,
                                  g.window ? std::min(g.window, k::kWholeContext) : k::kWholeContext, g.rot_dim, g.rot_interleaved ? 1u : 0u, g.q_temp, g.q_temp_every};
            k::attention_pad(a);
            const bool own_kv = g.kv_from < 0, bias = g.attention & FA_ATTENTION_BIAS, norms = g.attention & FA_ATTENTION_QK_NORM;
            const uint32_t nq = H * g.dim, nk = own_kv ? g.kv_heads * g.dim : 0, nv = m.head_gate_at - nq - nk;
            if (bias) l.in_bias = (float *)own(FA_F32, pad_to(nq + nk + nv, 4));
            const std::pair<const char *, std::pair<uint32_t, uint32_t>> parts[3] = {{"q", {0, nq}}, {"k", {nq, nk}}, {"v", {nq + nk, nv}}};
            for (const auto &[name, at] : parts) {
                if (at.second == 0) continue;
                lin(m.prefix + name, at.second, D, l.in, hi + at.first);
                if (bias) vec(m.prefix + name + ".b", at.second, 0, l.in_bias + at.first);
            }
            auto norm = [&](const char *name, uint32_t n) {
                float *p = (float *)own(FA_F32, n);
                vec(m.prefix + name, n, 0, p);
                return p;
            };
            if (norms) m.q_norm = norm("q.norm", nq);
            if (norms && own_kv) m.k_norm = norm("k.norm", nk);
            if (g.attention & FA_ATTENTION_HEAD_NORM) {
                m.q_norm = norm("q.norm", g.dim);
                m.k_norm = norm("k.norm", g.dim);
            }
            if (g.attention & FA_ATTENTION_SINK) m.sink = norm("sink", H);
            if (g.attention & FA_ATTENTION_SIGMOID) m.score_bias = norm("pb", H);
            if (g.attention & FA_ATTENTION_HEAD_GATE) lin(m.prefix + "g", H, D, l.in, hi + m.head_gate_at);
            if (g.distance != 0.0f) {
                std::vector<float> slopes(H);
                for (uint32_t h = 0; h < H; ++h) slopes[h] = (float)std::exp2(-(double)g.distance * (h + 1.0) / H);
                m.slope = (float *)own(FA_F32, H);
                if (st == FA_OK) st = fa_upload_into(ctx, slopes.data(), H, L->owned.back(), 0);
            }
            if (g.attention & FA_ATTENTION_GATE) lin(m.prefix + "g", m.out_width(), D, l.in, m.lo_at + m.gate_at);
            if (g.rot_dim) rotation(m);
            if (own_kv) {
                m.k_pool = own(f32 ? FA_F32 : FA_BF16, a.pool_rows * g.kv_heads * a.dim_p);
                m.v_pool = own(f32 ? FA_F32 : FA_BF16, a.pool_rows * g.kv_heads * a.v_p);
            }
        };
        auto set_latent = [&](Mixer &m, const Layer &l) {
            const fa_layer_config &g = m.cfg;
            const uint32_t H = g.heads, hi = l.lo + m.hi_at;
            k::LatentShape &a = m.la;
            a.heads = H;
            a.dim = g.dim;
            a.rot = g.rot_dim;
            a.vdim = g.vdim;
            a.q_rank = g.q_rank;
            a.kv_rank = g.kv_rank;
            k::latent_pad(a);
            a.window = g.window ? std::min(g.window, max_ctx) : max_ctx;
            a.interleaved = g.rot_interleaved ? 1 : 0;
            a.scale = g.scale;
            a.eps = c.norm_eps;
            a.pool_rows = (uint64_t)c.num_blocks * c.block_size;
            const bool own_kv = g.kv_from < 0;
            const uint32_t kvn = own_kv ? g.kv_rank + g.rot_dim : 0;
            lin(m.prefix + "dq", g.q_rank, D, l.in, hi);
            m.q_norm = (float *)own(FA_F32, g.q_rank);
            vec(m.prefix + "dq.norm", g.q_rank, 0, m.q_norm);
            if (own_kv) {
                lin(m.prefix + "dkv", kvn, D, l.in, hi + g.q_rank);
                m.kv_norm = (float *)own(FA_F32, g.kv_rank);
                vec(m.prefix + "dkv.norm", g.kv_rank, 0, m.kv_norm);
                m.pool = own(f32 ? FA_F32 : FA_BF16, a.pool_rows * (a.rank_p + a.rot_p));
            }
            if (!g.ungated) lin(m.prefix + "g", H, D, l.in, hi + g.q_rank + kvn);
            // queries: per head [dim padded][rot padded]
            const uint32_t qw = a.dim_p + a.rot_p, hd = g.dim + g.rot_dim, qr = g.q_rank, dim = g.dim, rot = g.rot_dim, dim_p = a.dim_p;
            m.uq = weight(H * qw, H * qw, qr);
            {
                const k::LinearWeight w = m.uq;
                add(m.prefix + "uq", (uint64_t)H * hd, qr, [=](const void *src, int sf, hipStream_t s) {
                    for (uint32_t h = 0; h < H; ++h) {
                        k::pack_linear(row_ptr(src, sf, (uint64_t)h * hd * qr), sf, qr, 1, dim, qr, (void *)w.w, f32, w.k_tiles, h * qw, 0x40000000u, 0, s);
                        k::pack_linear(row_ptr(src, sf, ((uint64_t)h * hd + dim) * qr), sf, qr, 1, rot, qr, (void *)w.w, f32, w.k_tiles, h * qw + dim_p, 0x40000000u, 0, s);
                    }
                });
            }
            // per head, latent = W_uk^T q: the key projection transposed
            const uint32_t kr = g.kv_rank, vd = g.vdim;
            const uint32_t hw = dim_p + a.v_p;
            if (!f32) m.ukv = weight(H * hw, H * hw, kr);
            const k::LinearWeight both = m.ukv;
            m.uk = weight(a.rank_p, a.rank_p, dim, H);
            {
                const k::LinearWeight w = m.uk;
                const uint64_t one = (uint64_t)w.n_tiles * 16 * w.k_tiles * 32 * L->esz;
                add(m.prefix + "uk", (uint64_t)H * dim, kr, [=](const void *src, int sf, hipStream_t s) {
                    for (uint32_t h = 0; h < H; ++h)
                        k::pack_linear(row_ptr(src, sf, (uint64_t)h * dim * kr), sf, 1, kr, kr, dim, (uint8_t *)w.w + h * one, f32, w.k_tiles, 0, 0x40000000u, 0, s);
                    if (both.w) k::pack_linear(src, sf, kr, 1, H * dim, kr, (void *)both.w, f32, both.k_tiles, 0, dim, hw, s);
                });
            }
            m.uv = weight(vd, vd, kr, H);
            {
                const k::LinearWeight w = m.uv;
                const uint64_t one = (uint64_t)w.n_tiles * 16 * w.k_tiles * 32 * L->esz;
                add(m.prefix + "uv", (uint64_t)H * vd, kr, [=](const void *src, int sf, hipStream_t s) {
                    for (uint32_t h = 0; h < H; ++h)
                        k::pack_linear(row_ptr(src, sf, (uint64_t)h * vd * kr), sf, kr, 1, vd, kr, (uint8_t *)w.w + h * one, f32, w.k_tiles, 0, 0x40000000u, 0, s);
                    if (both.w) k::pack_linear(src, sf, kr, 1, H * vd, kr, (void *)both.w, f32, both.k_tiles, dim_p, vd, hw, s);
                });
            }
            m.window_index = (uint32_t)(std::find(L->windows.begin(), L->windows.end(), a.window) - L->windows.begin());
            if (m.window_index == L->windows.size()) L->windows.push_back(a.window);
            rotation(m);
        };
        L->layers.resize(c.n_layers);
        for (uint32_t i = 0; i < c.n_layers; ++i) {
            Layer &l = L->layers[i];
            l.cfg = c.layers[i];
            const std::string p = "l" + std::to_string(i) + ".", f = p + "mlp.";
            const fa_layer_config g = l.cfg;
            l.norm1 = (float *)own(FA_F32, D);
            vec(p + "norm1", D, 0, l.norm1);
            if (post[c.norm][0]) {
                l.post1 = (float *)own(FA_F32, D);
                vec(p + post[c.norm][0], D, 0, l.post1);
            }
            l.mixers.resize(g.right ? 2 : 1);
            l.mixers[0].cfg = g;
            l.mixers[0].prefix = p + (g.right ? "mix.left." : "mix.");
            if (g.right) {
                l.mixers[0].out_scale = g.left_scale;
                l.mixers[1].out_scale = g.right_scale;
                l.mixers[1].cfg = *g.right;
                l.mixers[1].prefix = p + "mix.right.";
            }
            for (Mixer &m : l.mixers) {
                measure(m);
                m.lo_at = l.lo;
                m.hi_at = l.hi;
                m.o_at = l.o_width = pad_to(l.o_width, 8);
                l.lo = pad_to(l.lo + m.lo, 8);
                l.hi = pad_to(l.hi + m.hi, &m == &l.mixers.back() ? 1 : 4);
                l.o_width += m.out_width();
            }
            l.in = weight(l.lo + l.hi, l.lo + l.hi, D);
            l.out = weight(D, D, l.o_width);
            for (Mixer &m : l.mixers) {
                if (recurrent(m.cfg)) set_recurrence(m, l);
                else if (m.cfg.mixer == FA_MIXER_MINGRU) set_gated(m, l);
                else if (m.cfg.mixer == FA_MIXER_ATTENTION) set_attention(m, l);
                else set_latent(m, l);
                lin(m.prefix + "o", D, m.out_width(), l.out, 0, 0, 0, m.o_at);
                m.cfg.right = nullptr;                       // the caller's
                m.cfg.decay = nullptr;
            }
            l.cfg.right = nullptr;
            l.cfg.decay = nullptr;
            if (g.d_ffn) {
                l.norm2 = (float *)own(FA_F32, D);
                vec(p + "norm2", D, 0, l.norm2);
                if (post[c.norm][1]) {
                    l.post2 = (float *)own(FA_F32, D);
                    vec(p + post[c.norm][1], D, 0, l.post2);
                }
            }
            if (g.experts) {
                l.router = weight(g.experts, g.experts, D);
                lin(f + "router", g.experts, D, l.router, 0);
                if (g.route == FA_ROUTE_SCORED) {
                    l.correction = (float *)own(FA_F32, g.experts);
                    vec(f + "correction", g.experts, 0, l.correction);
                }
                const bool glu = g.glu == FA_GLU_SILU;
                l.gate_up = weight(g.d_ffn, glu ? 2 * pad_to(g.d_ffn, 16) : g.d_ffn, D, l.lists());
                l.down = weight(D, D, g.d_ffn, l.lists());
                const auto one = [&](const k::LinearWeight &w, uint32_t e) {
                    k::LinearWeight t = w;
                    t.batches = 1;
                    t.w = (uint8_t *)w.w + (uint64_t)e * w.n_tiles * 16 * w.k_tiles * 32 * L->esz;
                    return t;
                };
                for (uint32_t e = 0; e < l.lists(); ++e) {
                    const std::string x = f + "e" + std::to_string(e) + ".";
                    if (glu) lin(x + "gate", g.d_ffn, D, one(l.gate_up, e), 0, 16, 32);
                    if (glu) lin(x + "up", g.d_ffn, D, one(l.gate_up, e), 16, 16, 32);
                    else lin(x + "up", g.d_ffn, D, one(l.gate_up, e), 0);
                    lin(x + "down", D, g.d_ffn, one(l.down, e), 0);
                }
            } else if (g.d_ffn && g.glu == FA_FFN_XIELU) {
                l.gate_up = weight(g.d_ffn, g.d_ffn, D);
                lin(f + "up", g.d_ffn, D, l.gate_up, 0);
                l.down = weight(D, D, g.d_ffn);
                lin(f + "down", D, g.d_ffn, l.down, 0);
                l.act = (float *)own(FA_F32, 4);
                float *act = l.act;
                add(f + "act", 2, 0, [=](const void *src, int src_f32, hipStream_t s) {
                    if (src_f32) (void)hipMemcpyAsync(act + 2, src, 8, hipMemcpyDeviceToDevice, s);
                    else k::convert_bf16_to_f32((const uint16_t *)src, act + 2, 2, s);
                    k::xielu_constants(act + 2, act, s);
                });
            } else if (g.d_ffn) {
                // gate and up alternate in tiles of 16 columns
                l.gate_up = weight(g.d_ffn, 2 * pad_to(g.d_ffn, 16), D);
                lin(f + "gate", g.d_ffn, D, l.gate_up, 0, 16, 32);
                lin(f + "up", g.d_ffn, D, l.gate_up, 16, 16, 32);
                l.down = weight(D, D, g.d_ffn);
                lin(f + "down", D, g.d_ffn, l.down, 0);
            }
        }
        L->final_norm = (float *)own(FA_F32, D);
        vec("final.norm", D, 0, L->final_norm);
        L->head = weight(c.vocab, c.vocab, D);
        lin("head", c.vocab, D, L->head, 0);

        const uint64_t B = c.max_batch;
        mk(FA_I32, B, &d->tokens);
        mk(FA_U32, B * c.max_blocks_per_seq, &d->tables);
        mk(FA_U32, B, &d->seq_lens);
        mk(FA_F32, B * D, &d->h);
        mk(FA_F32, B * c.vocab, &d->logits);
        mk(FA_U32, 2, &d->rng);
        mk(FA_U32, 6 * B, &d->policy);
        for (fa_buffer **b : {&L->state_slots, &L->unit_starts, &L->last_rows}) {
            mk(FA_U32, B + 1, b);
            if (*b) L->owned.push_back(*b);
        }
        if (st == FA_OK) {
            std::vector<uint32_t> iota(B + 1);
            for (uint64_t b = 0; b <= B; ++b) iota[b] = (uint32_t)b;
            st = fa_upload_into(ctx, iota.data(), B + 1, L->unit_starts, 0);
        }
    } catch (const std::exception &) {
        st = fail(FA_ERR_ALLOCATION_FAILED, "decoder_create_layered: out of host memory");
    }
    if (st != FA_OK) {
        fa_decoder_destroy(ctx, d);
        return st;
    }
    *out = d;
    return FA_OK;
}

fa_status fa_decoder_tensor_count(const fa_decoder *d, uint32_t *count) {
    if (fa_status s = check_layered(d, "decoder_tensor_count")) return s;
    if (!count) return fail(FA_ERR_INVALID_ARGUMENT, "decoder_tensor_count: null output");
    *count = (uint32_t)d->layered->tensors.size();
    return FA_OK;
}

fa_status fa_decoder_tensor_info(const fa_decoder *d, uint32_t index, const char **name, uint64_t *rows, uint64_t *cols) {
    if (fa_status s = check_layered(d, "decoder_tensor_info")) return s;
    if (!name || !rows || !cols || index >= d->layered->tensors.size()) return fail(FA_ERR_INVALID_ARGUMENT, "decoder_tensor_info: bad argument");
    const Tensor &t = d->layered->tensors[index];
    *name = t.name.c_str();
    *rows = t.rows;
    *cols = t.cols;
    return FA_OK;
}

fa_status fa_decoder_set_tensor(fa_context *ctx, fa_decoder *d, const char *name, fa_dtype dtype, const void *data, uint64_t rows, uint64_t cols) {
    if (fa_status s = check_ctx(ctx)) return s;
    if (fa_status s = check_layered(d, "decoder_set_tensor")) return s;
    if (d->ctx != ctx) return fail(FA_ERR_DEVICE_MISMATCH, "decoder_set_tensor: decoder belongs to another context");
    if (ctx->capturing) return fail(FA_ERR_CAPTURE_IN_PROGRESS, "decoder_set_tensor during graph capture");
    if (!name || !data) return fail(FA_ERR_INVALID_ARGUMENT, "decoder_set_tensor: null argument");
    if (dtype != FA_BF16 && dtype != FA_F32) return fail(FA_ERR_INVALID_ARGUMENT, std::string("decoder_set_tensor: ") + name + ": must be bf16 or f32");
    auto &ts = d->layered->tensors;
    auto it = std::find_if(ts.begin(), ts.end(), [&](const Tensor &t) { return t.name == name; });
    if (it == ts.end()) return fail(FA_ERR_INVALID_ARGUMENT, std::string("decoder_set_tensor: no tensor ") + name);
    if (it->rows != rows || it->cols != cols)
        return fail(FA_ERR_SHAPE_MISMATCH, std::string("decoder_set_tensor: ") + name + ": expected [" + std::to_string(it->rows) + ", " + std::to_string(it->cols) +
                                               "], got [" + std::to_string(rows) + ", " + std::to_string(cols) + "]");
    fa_buffer *tmp = nullptr;
    if (fa_status s = fa_upload(ctx, dtype, data, rows * (cols ? cols : 1), &tmp)) return s;
    it->place(tmp->ptr, dtype == FA_F32, ctx->stream);
    fa_status s = after_launch(ctx, "decoder_set_tensor");
    fa_buffer_free(ctx, tmp);                            // the stream is in order: a later user is queued behind the copy
    if (s == FA_OK) it->set = true;
    return s;
}

fa_status fa_decoder_set_state_slots(fa_context *ctx, fa_decoder *d, const uint32_t *slots) {
    if (fa_status s = check_ctx(ctx)) return s;
    if (fa_status s = check_layered(d, "decoder_set_state_slots")) return s;
    if (d->ctx != ctx) return fail(FA_ERR_DEVICE_MISMATCH, "decoder_set_state_slots: decoder belongs to another context");
    if (d->batch == 0 || !slots) return fail(FA_ERR_INVALID_ARGUMENT, "decoder_set_state_slots: no sequences or null slots");
    for (uint32_t b = 0; b < d->batch; ++b) {
        if (slots[b] >= d->layered->cfg.state_slots) return fail(FA_ERR_INVALID_ARGUMENT, "decoder_set_state_slots: row " + std::to_string(b) + " has no such slot");
        for (uint32_t o = 0; o < b; ++o)
            if (slots[o] == slots[b]) return fail(FA_ERR_INVALID_ARGUMENT, "decoder_set_state_slots: two rows share a slot");
    }
    if (fa_status s = fa_upload_into(ctx, slots, d->batch, d->layered->state_slots, 0)) return s;
    d->layered->slots_set = true;
    return FA_OK;
}

fa_status fa_decoder_forward(fa_context *ctx, fa_decoder *d, const uint32_t *counts, const int32_t *tokens, uint64_t n_want, const uint32_t *want, float *logits) {
    if (fa_status s = check_ctx(ctx)) return s;
    if (fa_status s = check_layered(d, "decoder_forward")) return s;
    if (d->ctx != ctx) return fail(FA_ERR_DEVICE_MISMATCH, "decoder_forward: decoder belongs to another context");
    if (ctx->capturing) return fail(FA_ERR_CAPTURE_IN_PROGRESS, "decoder_forward during graph capture");
    if (d->batch == 0) return fail(FA_ERR_INVALID_ARGUMENT, "decoder_forward: no sequences installed");
    if (!counts || !tokens || (n_want && (!want || !logits))) return fail(FA_ERR_INVALID_ARGUMENT, "decoder_forward: null argument");
    static const uint32_t none = 0;
    return layered_forward(ctx, d, counts, tokens, n_want, want ? want : &none, logits, nullptr);
}

fa_status fa_decoder_debug_residuals(fa_decoder *d, float *residuals, uint64_t rows) {
    if (fa_status s = check_layered(d, "decoder_debug_residuals")) return s;
    d->layered->trace = residuals;
    d->layered->trace_rows = rows;
    return FA_OK;
}

}  // extern "C"
