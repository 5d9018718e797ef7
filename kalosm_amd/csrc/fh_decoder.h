// What every decoder of the library shares: the position and token history of its sequence, the forward pass in portions
// with context trimming, and the device-side greedy and sampled decode loops with their captured step.  A decoder family
// (fh_llama.hip, fh_hybrid.hip) supplies its layers, its output head and its caches.
#pragma once
#include "fh_internal.h"

#include <string>
#include <vector>

struct fh_decoder {
    fh_device *dev = nullptr;
    int vocab = 0, d_model = 0, ctx = 0, n_layers = 0;
    bool use_graph = true;
    bool finalized = false;
    int pos = 0;
    // the token ids whose state the caches hold (KvCache::tokens of the reference, raw/cache.rs): what a forward pass
    // re-runs the tail of when the context is full
    std::vector<uint32_t> history;
    uint32_t *ids = nullptr;   // token ids of the current portion (owned by the family's step buffers)
    float *logits = nullptr;   // [logit_rows, vocab]
    int logit_rows = 0;
    // greedy decode state
    uint32_t *tok_dev = nullptr, *out_tok_dev = nullptr;
    int *step_dev = nullptr;
    hipGraphExec_t graph_exec = nullptr;
    hipGraph_t graph = nullptr;
    int64_t captured_capacity = -1;
    uint64_t captured_gen = 0, samp_gen = 0; // dev->scratch_gen at the captures
    uint64_t captured_opt = 0, samp_opt = 0; // dev->opt_gen at the captures (options pick the kernels of a step)
    // sampled decode state: [0..63] previous ids, [64] their count, [65] next slot, [66] Mirostat mu (f32),
    // [68..69] status and token of the last step, [128..] one random number per step
    uint32_t *samp_dev = nullptr;
    hipGraphExec_t samp_exec = nullptr;
    hipGraph_t samp_graph = nullptr;
    int64_t samp_capacity = -1;
    uint32_t samp_range = 0;
    fh_sampler_params samp_params = {};

    virtual ~fh_decoder();
    // Device buffers for portions of s tokens (ids among them).
    virtual fh_status ensure_steps(int s) = 0;
    // The most tokens one call of layers() takes.
    virtual int max_portion() const { return 65535; }
    // All layers over the s tokens in `ids`, at position `pos`, or at *len_dev() when dev_pos (s is 1 then): appends to
    // the caches, leaves the residual stream behind for head().
    virtual fh_status layers(int s, bool dev_pos) = 0;
    // Final norm and output matrix on row `row` of the last portion: out [vocab]; hidden() is the normed row.
    virtual fh_status head(int row, float *out) = 0;
    virtual const float *hidden() const = 0;
    // Cache storage for `positions` positions of the sequence; capacity() changes when a captured step no longer fits it.
    virtual fh_status reserve(int positions) = 0;
    virtual int64_t capacity() const = 0;
    // The sequence has `len` positions; without `device` the device-side length is already right (a decode loop).
    virtual fh_status set_len(int len, bool device) = 0;
    virtual int *len_dev() = 0;
    virtual uint64_t weight_bytes() const = 0;
    virtual fh_status load_tensor(const char *name, uint32_t ggml_type, int64_t n, int64_t k, const void *bytes, size_t len) = 0;
    virtual fh_status finalize() = 0;
    virtual fh_status layer_output(int, float *, int64_t) { FH_FAIL(FH_ERR_UNSUPPORTED, "this decoder keeps no layer outputs"); }
    virtual fh_status keep_layers(bool) { FH_FAIL(FH_ERR_UNSUPPORTED, "this decoder keeps no layer outputs"); }
    // Around a forward pass of the host (traces).
    virtual fh_status forward_begin() { return FH_OK; }
    virtual fh_status forward_end(int) { return FH_OK; }

    fh_status create_loop_buffers(); // after the sizes are known
    void drop_captures() { captured_capacity = samp_capacity = -1; }
    fh_status reset();
    fh_status forward(const uint32_t *tokens, int count, const int32_t *want, int n_want, float *logits_host, float *hidden_host);
    fh_status decode_greedy(uint32_t first_token, int steps, uint32_t *out_tokens, float *elapsed_ms);
    fh_status decode_sampled(uint32_t first_token, int steps, const fh_sampler_params *params, const float *randoms,
                             const uint32_t *previous, uint32_t n_previous, uint32_t repetition_range, float *mu,
                             uint32_t *out_tokens, float *elapsed_ms);

  private:
    fh_status ensure_logits(int rows);
    fh_status greedy_step();
    fh_status sampled_step();
};

// The layer-list decoder (fh_hybrid.hip) for a configuration text; dtype FH_F32 or FH_DECODER_BF16.
fh_status fh_hybrid_create(fh_device *dev, const char *config_json, int dtype, int ctx, fh_decoder **out);
bool fh_hybrid_knows(const char *architecture);
