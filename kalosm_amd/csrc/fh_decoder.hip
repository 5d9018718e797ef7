// The part all decoders share (fh_decoder.h): forward passes in portions, the device-side decode loops, and the entry
// points of the handle.
// Reference: models/kalosm-llama/src/raw/mod.rs:769-865 (Model::forward and its context trimming),
// model/inference.rs:11-396 (decode loop).
#include "fh_decoder.h"
#include "fh_json.h"
#include "fh_safetensors.h"

#include <algorithm>
#include <cstring>

fh_decoder::~fh_decoder() {
    if (!dev) return;
    (void)hipStreamSynchronize(dev->stream);
    if (graph_exec) (void)hipGraphExecDestroy(graph_exec);
    if (graph) (void)hipGraphDestroy(graph);
    if (samp_exec) (void)hipGraphExecDestroy(samp_exec);
    if (samp_graph) (void)hipGraphDestroy(samp_graph);
    for (void *p : {(void *)logits, (void *)tok_dev, (void *)out_tok_dev, (void *)step_dev, (void *)samp_dev})
        if (p) (void)hipFree(p);
}

fh_status fh_decoder::create_loop_buffers() {
    FH_TRY(ensure_logits(1));
    FH_TRY(fh_malloc(dev, 256, (void **)&tok_dev));
    FH_TRY(fh_malloc(dev, (size_t)ctx * 4 + 256, (void **)&out_tok_dev));
    FH_TRY(fh_malloc(dev, 256, (void **)&step_dev));
    return fh_malloc(dev, (size_t)(128 + ctx) * 4, (void **)&samp_dev);
}

fh_status fh_decoder::ensure_logits(int rows) {
    if (rows <= logit_rows) return FH_OK;
    (void)hipStreamSynchronize(dev->stream);
    if (logits) (void)hipFree(logits);
    logits = nullptr;
    logit_rows = 0;
    drop_captures(); // a captured decode step holds the pointer
    FH_TRY(fh_malloc(dev, (size_t)rows * vocab * 4, (void **)&logits));
    logit_rows = rows;
    return FH_OK;
}

fh_status fh_decoder::reset() {
    FH_REQUIRE(finalized, "decoder not finalized");
    pos = 0;
    history.clear();
    return set_len(0, true);
}

fh_status fh_decoder::forward(const uint32_t *tokens, int count, const int32_t *want, int n_want, float *logits_host,
                              float *hidden_host) {
    FH_REQUIRE(finalized && tokens, "decoder not finalized or NULL tokens");
    FH_REQUIRE(count > 0 && count <= 65535, "count %d out of range", count);
    for (int i = 0; i < count; i++)
        FH_REQUIRE(tokens[i] < (uint32_t)vocab, "token id %u at %d outside the vocabulary of %d", tokens[i], i, vocab);
    const int32_t last = count - 1;
    if (!want) want = &last, n_want = 1;
    for (int i = 0; i < n_want; i++)
        FH_REQUIRE(want[i] >= 0 && want[i] < count, "wanted place %d outside the %d tokens", want[i], count);
    // Model::forward, raw/mod.rs:769-801: when the new tokens do not fit the context, the cache is cleared and the last
    // context_length - 32 (at least 8) of all tokens, cached and new, are run again from position 0.
    std::vector<uint32_t> trimmed;
    int skip = 0; // tokens ahead of the caller's first one
    if (pos + count > ctx) {
        const int cutoff = std::max(ctx - 32, 8);
        FH_REQUIRE(cutoff <= ctx && cutoff <= 65535, "context of %d positions is too short to trim to %d", ctx, cutoff);
        FH_REQUIRE((int)history.size() == pos, "the cache holds %d positions but %zu token ids are on record", pos, history.size());
        trimmed = history;
        trimmed.insert(trimmed.end(), tokens, tokens + count);
        skip = cutoff - count;
        for (int i = 0; i < n_want; i++) FH_REQUIRE(want[i] + skip >= 0, "wanted place %d was trimmed away", want[i]);
        trimmed.erase(trimmed.begin(), trimmed.end() - cutoff);
        FH_TRY(reset());
        tokens = trimmed.data();
        count = cutoff;
    }
    FH_TRY(ensure_logits(std::max(n_want, 1)));
    FH_TRY(forward_begin());
    const int portion = std::min(count, max_portion());
    FH_TRY(ensure_steps(portion));
    FH_TRY(reserve(pos + count));
    for (int at = 0; at < count; at += portion) {
        const int n = std::min(portion, count - at);
        FH_TRY(fh_upload(dev, ids, tokens + at, (size_t)n * 4));
        FH_TRY(layers(n, false));
        for (int i = 0; i < n_want; i++) {
            const int row = want[i] + skip - at;
            if (row >= 0 && row < n) FH_TRY(head(row, logits + (size_t)i * vocab));
        }
        // all layers appended: advance the caches
        history.insert(history.end(), tokens + at, tokens + at + n);
        pos += n;
        FH_TRY(set_len(pos, true));
    }
    if (hidden_host) FH_TRY(fh_download(dev, hidden_host, hidden(), (size_t)d_model * 4));
    if (logits_host && n_want) FH_TRY(fh_download(dev, logits_host, logits, (size_t)n_want * vocab * 4));
    FH_TRY(fh_device_sync(dev));
    return forward_end(count);
}

__global__ void k_set_u32(uint32_t *p, uint32_t v) { *p = v; }

fh_status fh_decoder::greedy_step() {
    FH_TRY(layers(1, true));
    FH_TRY(head(0, logits));
    // the last stage of the pick also stores the token, feeds it to the next step and advances the cache length
    return fh_argmax_step(dev, logits, vocab, tok_dev,
                          FhStepTail{ids, out_tok_dev, step_dev, len_dev()});
}

fh_status fh_decoder::decode_greedy(uint32_t first_token, int steps, uint32_t *out_tokens_host, float *elapsed_ms) {
    FH_REQUIRE(finalized && out_tokens_host, "decoder not finalized or NULL output");
    FH_REQUIRE(steps > 0 && pos + steps <= ctx,
               "context overflow: %d + %d > %d (the device-side loops stop at the context length; a forward pass trims)", pos,
               steps, ctx);
    FH_REQUIRE(first_token < (uint32_t)vocab, "token id %u outside the vocabulary", first_token);
    hipStream_t s = dev->stream;
    // capacity is fixed for the whole run so that no reallocation happens between steps
    FH_TRY(ensure_steps(1));
    FH_TRY(reserve(pos + steps));
    k_set_u32<<<1, 1, 0, s>>>(ids, first_token);
    k_set_u32<<<1, 1, 0, s>>>((uint32_t *)step_dev, 0u);
    FH_HIP(hipGetLastError());
    int done = 0;
    if (use_graph && !dev->opt_step_eager) {
        // One eager step sizes every scratch buffer and sets kernel attributes; the capture then
        // records launches only.  The graph depends on the cache capacity (strides), so it is
        // rebuilt when the capacity changed since the last capture.
        if (!graph_exec || captured_capacity != capacity() || captured_gen != dev->scratch_gen ||
            captured_opt != dev->opt_gen) {
            FH_TRY(fh_timer_start(dev));
            FH_TRY(greedy_step());
            done = 1;
            FH_HIP(hipStreamSynchronize(s));
            if (graph_exec) { (void)hipGraphExecDestroy(graph_exec); graph_exec = nullptr; }
            if (graph) { (void)hipGraphDestroy(graph); graph = nullptr; }
            FH_HIP(hipStreamBeginCapture(s, hipStreamCaptureModeThreadLocal));
            fh_status st = greedy_step();
            hipError_t e = hipStreamEndCapture(s, &graph);
            if (st != FH_OK) return st;
            FH_HIP(e);
            FH_HIP(hipGraphInstantiate(&graph_exec, graph, nullptr, nullptr, 0));
            captured_capacity = capacity();
            captured_gen = dev->scratch_gen;
            captured_opt = dev->opt_gen;
        } else {
            FH_TRY(fh_timer_start(dev));
        }
        for (; done < steps; done++) FH_HIP(hipGraphLaunch(graph_exec, s));
    } else {
        FH_TRY(fh_timer_start(dev));
        for (; done < steps; done++) FH_TRY(greedy_step());
    }
    float ms = 0.f;
    FH_TRY(fh_timer_stop(dev, &ms));
    if (elapsed_ms) *elapsed_ms = ms;
    pos += steps;
    FH_TRY(set_len(pos, false));
    FH_TRY(fh_download(dev, out_tokens_host, out_tok_dev, (size_t)steps * 4));
    history.push_back(first_token); // the cache now holds the step inputs: the first token and all outputs but the last
    history.insert(history.end(), out_tokens_host, out_tokens_host + steps - 1);
    return FH_OK;
}

// Sampled decode (models/kalosm-llama/src/model/inference.rs:38-173, forward.rs:346-404): the sampled id stays in
// device memory and feeds the next step; it also joins the window of previous ids that the repetition penalty
// looks at (membership only, so the window is a ring).
__global__ void k_store_sampled(const uint32_t *result, uint32_t *ids, uint32_t *out, int *step, uint32_t *prev,
                                uint32_t range, int *kv_len) {
    *kv_len = *kv_len + 1;
    const uint32_t t = result[0] == FH_SAMPLE_STATUS_SAMPLED ? result[1] : 0xFFFFFFFFu;
    const uint32_t next = t == 0xFFFFFFFFu ? 0u : t;
    ids[0] = next;
    out[*step] = t;
    *step = *step + 1;
    if (range) {
        const uint32_t slot = prev[65];
        prev[slot] = next;
        prev[65] = slot + 1 == range ? 0u : slot + 1;
        if (prev[64] < range) prev[64] = prev[64] + 1;
    }
}

fh_status fh_decoder::sampled_step() {
    FH_TRY(layers(1, true));
    FH_TRY(head(0, logits));
    uint32_t *sd = samp_dev;
    FH_TRY(fh_sample_token_dev(dev, logits, vocab, &samp_params, sd, sd + 64, 0, (const float *)(sd + 128),
                               step_dev, (float *)(sd + 66), sd + 68, nullptr, nullptr));
    k_store_sampled<<<1, 1, 0, dev->stream>>>(sd + 68, ids, out_tok_dev, step_dev, sd, samp_range,
                                                len_dev());
    FH_HIP(hipGetLastError());
    return FH_OK;
}

fh_status fh_decoder::decode_sampled(uint32_t first_token, int steps, const fh_sampler_params *params, const float *randoms_host,
                                     const uint32_t *previous_host, uint32_t n_previous, uint32_t repetition_range, float *mu,
                                     uint32_t *out_tokens_host, float *elapsed_ms) {
    FH_REQUIRE(finalized && out_tokens_host && params && randoms_host, "decoder not finalized or NULL argument");
    FH_REQUIRE(steps > 0 && pos + steps <= ctx,
               "context overflow: %d + %d > %d (the device-side loops stop at the context length; a forward pass trims)", pos,
               steps, ctx);
    FH_REQUIRE(first_token < (uint32_t)vocab, "token id %u outside the vocabulary", first_token);
    FH_REQUIRE(n_previous == 0 || previous_host, "previous tokens missing");
    FH_REQUIRE(params->kind != FH_SAMPLER_MIROSTAT2 || mu, "Mirostat 2 needs its state");
    hipStream_t s = dev->stream;
    const uint32_t range = repetition_range < FH_SAMPLER_PREVIOUS_TOKENS ? repetition_range : FH_SAMPLER_PREVIOUS_TOKENS;
    // window = the last `range` ids of (history, first_token)
    uint32_t head[128] = {0};
    uint32_t len = 0;
    if (range) {
        const uint32_t keep = n_previous < range - 1 ? n_previous : range - 1;
        for (uint32_t i = 0; i < keep; i++) head[len++] = previous_host[n_previous - keep + i];
        head[len++] = first_token;
    }
    head[64] = len;
    head[65] = range ? len % range : 0u;
    const float mu0 = mu ? *mu : 0.f;
    memcpy(&head[66], &mu0, 4);
    FH_TRY(fh_upload(dev, samp_dev, head, sizeof(head)));
    FH_TRY(fh_upload(dev, samp_dev + 128, randoms_host, (size_t)steps * 4));
    FH_TRY(ensure_steps(1));
    FH_TRY(reserve(pos + steps));
    k_set_u32<<<1, 1, 0, s>>>(ids, first_token);
    k_set_u32<<<1, 1, 0, s>>>((uint32_t *)step_dev, 0u);
    FH_HIP(hipGetLastError());
    int done = 0;
    if (use_graph && !dev->opt_step_eager) {
        // the captured step holds the sampler's parameters and the window size as kernel arguments
        fh_sampler_params want = *params;
        want.random = 0.f; // every step takes its number from randoms_host
        const bool same = samp_exec && samp_capacity == capacity() && samp_range == range &&
                          samp_gen == dev->scratch_gen && samp_opt == dev->opt_gen &&
                          memcmp(&samp_params, &want, sizeof(want)) == 0;
        samp_params = want;
        samp_range = range;
        if (!same) {
            FH_TRY(fh_timer_start(dev));
            FH_TRY(sampled_step());
            done = 1;
            FH_HIP(hipStreamSynchronize(s));
            if (samp_exec) { (void)hipGraphExecDestroy(samp_exec); samp_exec = nullptr; }
            if (samp_graph) { (void)hipGraphDestroy(samp_graph); samp_graph = nullptr; }
            samp_capacity = -1;
            FH_HIP(hipStreamBeginCapture(s, hipStreamCaptureModeThreadLocal));
            fh_status st = sampled_step();
            hipError_t e = hipStreamEndCapture(s, &samp_graph);
            if (st != FH_OK) return st;
            FH_HIP(e);
            FH_HIP(hipGraphInstantiate(&samp_exec, samp_graph, nullptr, nullptr, 0));
            samp_capacity = capacity();
            samp_gen = dev->scratch_gen;
            samp_opt = dev->opt_gen;
        } else {
            FH_TRY(fh_timer_start(dev));
        }
        for (; done < steps; done++) FH_HIP(hipGraphLaunch(samp_exec, s));
    } else {
        samp_params = *params;
        samp_range = range;
        FH_TRY(fh_timer_start(dev));
        for (; done < steps; done++) FH_TRY(sampled_step());
    }
    float ms = 0.f;
    FH_TRY(fh_timer_stop(dev, &ms));
    if (elapsed_ms) *elapsed_ms = ms;
    pos += steps;
    FH_TRY(set_len(pos, false));
    FH_TRY(fh_download(dev, out_tokens_host, out_tok_dev, (size_t)steps * 4));
    if (mu) FH_TRY(fh_download(dev, mu, samp_dev + 66, 4));
    history.push_back(first_token);
    history.insert(history.end(), out_tokens_host, out_tokens_host + steps - 1);
    return FH_OK;
}

// ------------------------------------------------------------------------------ entry points
// Architectures by the "architecture" of a configuration; Llama models come in GGUF files (fh_llama_config_from_gguf).
extern "C" fh_status fh_decoder_create(fh_device *dev, const char *config_json, int32_t dtype, int32_t ctx, fh_decoder **out) {
    FH_REQUIRE(dev && config_json && out, "NULL argument");
    *out = nullptr;
    FH_REQUIRE(dtype == FH_F32 || dtype == FH_DECODER_BF16, "decoder dtype must be FH_F32 or FH_DECODER_BF16");
    FH_REQUIRE(ctx > 0, "context of %d positions", ctx);
    FhJson j;
    std::string err;
    if (!FhJson::parse(config_json, strlen(config_json), j, err)) FH_FAIL(FH_ERR_INVALID, "configuration: %s", err.c_str());
    const FhJson *a = j.find("architecture");
    FH_REQUIRE(a && a->is_string(), "the configuration names no architecture");
    if (fh_hybrid_knows(a->str.c_str())) return fh_hybrid_create(dev, config_json, dtype, ctx, out);
    FH_FAIL(FH_ERR_UNSUPPORTED, "unknown architecture '%s'", a->str.c_str());
}

extern "C" fh_status fh_decoder_open(fh_device *dev, const char *dir, int32_t dtype, int32_t ctx, fh_decoder **out) {
    FH_REQUIRE(dev && dir && out, "NULL argument");
    *out = nullptr;
    const std::string base = std::string(dir) + "/";
    std::string text;
    FH_TRY(fh_read_file((base + "config.json").c_str(), text));
    fh_decoder *m = nullptr;
    FH_TRY(fh_decoder_create(dev, text.c_str(), dtype, ctx, &m));
    fh_status st = fh_decoder_load_safetensors(m, (base + "model.safetensors").c_str());
    if (st == FH_OK) st = m->finalize();
    if (st != FH_OK) {
        delete m;
        return st;
    }
    *out = m;
    return FH_OK;
}

fh_status fh_decoder_load_safetensors(fh_decoder *m, const char *path) {
    FhSafetensors f;
    FH_TRY(f.open(path));
    for (const FhSafetensors::Entry &e : f.entries) {
        FH_REQUIRE(e.ggml_type >= 0, "%s: tensors of type %s are not supported", e.name.c_str(), e.dtype.c_str());
        FH_REQUIRE(e.shape.size() == 1 || e.shape.size() == 2, "%s: rank %zu (1 or 2 expected)", e.name.c_str(), e.shape.size());
        FH_TRY(m->load_tensor(e.name.c_str(), (uint32_t)e.ggml_type, e.shape[0], e.shape.size() == 2 ? e.shape[1] : 0, e.data, e.bytes));
    }
    return FH_OK;
}

extern "C" fh_status fh_decoder_load_tensor(fh_decoder *m, const char *name, uint32_t ggml_type, int64_t n, int64_t k,
                                            const void *bytes, size_t len) {
    FH_REQUIRE(m && name && bytes, "NULL argument");
    return m->load_tensor(name, ggml_type, n, k, bytes, len);
}
extern "C" fh_status fh_decoder_finalize(fh_decoder *m) {
    FH_REQUIRE(m, "NULL argument");
    return m->finalize();
}
extern "C" fh_status fh_decoder_destroy(fh_decoder *m) {
    delete m;
    return FH_OK;
}
extern "C" fh_status fh_decoder_info(const fh_decoder *m, int32_t *vocab, int32_t *d_model, int32_t *n_layers, int32_t *ctx,
                                     int32_t *position) {
    FH_REQUIRE(m, "NULL argument");
    if (vocab) *vocab = m->vocab;
    if (d_model) *d_model = m->d_model;
    if (n_layers) *n_layers = m->n_layers;
    if (ctx) *ctx = m->ctx;
    if (position) *position = m->pos;
    return FH_OK;
}
extern "C" fh_status fh_decoder_reset(fh_decoder *m) {
    FH_REQUIRE(m, "NULL argument");
    return m->reset();
}
extern "C" fh_status fh_decoder_forward(fh_decoder *m, const uint32_t *tokens_host, int32_t count, const int32_t *want_host,
                                        int32_t n_want, float *logits_host, float *hidden_host) {
    FH_REQUIRE(m && n_want >= 0, "NULL decoder or negative count");
    return m->forward(tokens_host, count, want_host, n_want, logits_host, hidden_host);
}
extern "C" fh_status fh_decoder_decode_greedy(fh_decoder *m, uint32_t first_token, int32_t steps, uint32_t *out_tokens_host,
                                              float *elapsed_ms) {
    FH_REQUIRE(m, "NULL decoder");
    return m->decode_greedy(first_token, steps, out_tokens_host, elapsed_ms);
}
extern "C" fh_status fh_decoder_decode_sampled(fh_decoder *m, uint32_t first_token, int32_t steps, const fh_sampler_params *params,
                                               const float *randoms_host, const uint32_t *previous_host, uint32_t n_previous,
                                               uint32_t repetition_range, float *mu, uint32_t *out_tokens_host,
                                               float *elapsed_ms) {
    FH_REQUIRE(m, "NULL decoder");
    return m->decode_sampled(first_token, steps, params, randoms_host, previous_host, n_previous, repetition_range, mu,
                             out_tokens_host, elapsed_ms);
}
extern "C" fh_status fh_decoder_weight_bytes(const fh_decoder *m, uint64_t *bytes) {
    FH_REQUIRE(m && bytes, "NULL argument");
    *bytes = m->weight_bytes();
    return FH_OK;
}
extern "C" fh_status fh_decoder_keep_layers(fh_decoder *m, int32_t on) {
    FH_REQUIRE(m, "NULL decoder");
    return m->keep_layers(on != 0);
}
extern "C" fh_status fh_decoder_layer_output(fh_decoder *m, int32_t layer, float *out_host, int64_t count) {
    FH_REQUIRE(m && out_host, "NULL argument");
    return m->layer_output(layer, out_host, count);
}
