// The resident decoder behind fa_decoder_*: what its two kinds (the W8A8 Llama-style stack of decoder.cpp and the
// layered stacks of layered_decoder.cpp) share: installed sequences, next tokens, sampling, recorded steps.
#pragma once

#include <map>
#include <vector>

#include "kernels.hpp"
#include "runtime.hpp"

namespace fa {
struct LayeredState;
}

struct fa_decoder {
    uint32_t magic;
    fa_context *ctx;
    fa_decoder_config cfg;
    struct Layer {
        const fa_buffer *attn_norm = nullptr, *ffn_norm = nullptr;
        const fa_qweight *wqkv = nullptr, *wo = nullptr, *wgu = nullptr, *wdown = nullptr;
        fa_buffer *k_pool = nullptr, *v_pool = nullptr;
    };
    std::vector<Layer> layers;
    // The large activation buffers of a prompt pass stay with the decoder from one pass to the next (grow only, until the
    // decoder goes): the context's pool keeps at most 128 MiB of idle blocks, so buffers of hundreds of megabytes went
    // back to the driver after every pass and were allocated again for the next (1024 prompt tokens: 12.9 -> 12.3 ms,
    // 4 x 2048: 71.4 -> 69.1 ms without those calls).  At most kRows rows of them: about 1.8 GB at the benchmark's width.
    struct KeptBlock {
        void *ptr = nullptr;
        uint64_t bytes = 0, cls = 0;
    };
    static constexpr int kKept = 8;
    KeptBlock kept[kKept];
    const fa_buffer *embed = nullptr, *final_norm = nullptr;
    const fa_qweight *lm_head = nullptr;
    uint32_t batch = 0;
    // resident state and activations
    fa_buffer *tokens = nullptr, *tables = nullptr, *seq_lens = nullptr, *pos = nullptr, *slots = nullptr;
    fa_buffer *cos_sin = nullptr, *h = nullptr, *xq = nullptr, *sx = nullptr, *q_bf = nullptr;
    fa_buffer *attn = nullptr, *act = nullptr, *pmax = nullptr, *logits = nullptr;
    // captured steps, one per batch size seen (a scheduler changes the batch as requests come and go)
    std::map<uint32_t, fa_graph *> graphs;
    int graph_waves = 0;
    // how the step and the prompt pass pick the next token; rng holds the generator state on the device
    fa_sampling strategy = FA_SAMPLE_GREEDY;
    float temperature = 1.0f;
    uint32_t top_k = 0;
    fa_buffer *rng = nullptr;
    // per-row sampling table (k::RowPolicy per row) and whether the pick uses it
    fa_buffer *policy = nullptr;
    bool per_row = false;
    // host mirror of the installed block tables and of the sequence lengths (advanced with every step and
    // prompt chunk), used to validate that a prompt fits before anything is queued
    std::vector<uint32_t> host_tables, host_lens;
    // layered decoders only: configuration, weights, caches and states (cfg then holds the sizes the two kinds share)
    fa::LayeredState *layered = nullptr;
};

namespace fa {

constexpr uint32_t kDecMagic = 0xFA0DEC01u;

inline uint64_t round_up(uint64_t v, uint64_t to) { return (v + to - 1) / to * to; }

// logits [batch, vocab] -> next tokens, by the decoder's sampling strategy
void enqueue_pick(fa_decoder *d, hipStream_t s);

// layered_decoder.cpp: what the entry points of decoder.cpp do for a layered decoder
void layered_free(fa_context *ctx, fa_decoder *d);
fa_status layered_ready(const fa_decoder *d, const char *what);
// recurrent state in any layer: sequences cannot be cut back
bool layered_has_state(const fa_decoder *d);
// after fa_decoder_set_sequences: state slot b for row b until the caller names others
fa_status layered_sequences_set(fa_context *ctx, fa_decoder *d);
fa_status layered_prepare_step(fa_context *ctx, fa_decoder *d);
fa_status layered_enqueue_step(fa_context *ctx, fa_decoder *d);
// counts [batch] new tokens per installed sequence, tokens concatenated.  want (row indices in the concatenated order)
// selects the logits rows copied to the host; want null: the last row of every sequence, left in d->logits with the
// next tokens picked.
fa_status layered_forward(fa_context *ctx, fa_decoder *d, const uint32_t *counts, const int32_t *tokens, uint64_t n_want,
                          const uint32_t *want, float *logits, int32_t *picked);

}  // namespace fa
