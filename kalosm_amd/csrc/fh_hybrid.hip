// Decoders whose configuration lists their layers one by one: each layer has a mixer (latent attention, gated delta rule,
// state space, retention, or grouped-query attention beside time mixing with channel decays, with sizes of its own) and,
// optionally, a feed-forward (mixture of experts, or dense).  Registered designs:
//   Fidasun   parallel residual (one norm feeds mixer and feed-forward), norm weights as distances from one, sinks
//   Zovovik   sublayers read the residual stream and are normed at their end, learned positions, sinks
// Weights are dense bf16 (safetensors).  Prefill portions run on the matrix cores (fh_dense.hip), one token through the
// fused step kernels (fh_step.hip); both use the same caches.
#include "fh_decoder.h"
#include "fh_json.h"
#include "fh_step.h"

#include <algorithm>
#include <cmath>
#include <cstring>
#include <functional>
#include <map>
#include <memory>

namespace {

// What a design fixes for all of its models.
struct Design {
    const char *name;
    bool norm_one_plus; // layer and final norm weights are distances from one
    bool sink;          // attention heads have a learned sink
    bool output_norm;   // x <- x + norm(sublayer(x)), mixer and feed-forward one after the other; otherwise parallel residual
    bool positions;     // a learned vector per position joins the embedding
};
const Design DESIGNS[] = {{"Fidasun", true, true, false, false}, {"Zovovik", false, true, true, true}};
const Design *find_design(const char *name) {
    for (const Design &d : DESIGNS)
        if (!strcmp(d.name, name)) return &d;
    return nullptr;
}

enum { MIX_PAIR = 2 }; // beside FH_MIX_*: attention and a recurrence on the same input
struct Layer {
    int kind = FH_MIX_LATENT;
    FhLatent lat;
    FhGqa gqa;
    FhRecurrent rec;
    FhRecState rec_state;
    FhMoe moe;
    fh_kvcache *cache = nullptr;
    int np = 0;              // columns of a projection row: the mixer's inputs, then the router
    int inner = 0, kpo = 0;  // input length of the output projection, padded
    int nl = 0, kpl = 0;     // pair: columns of the attention's projections, its part of kpo
    int ff = 0, ffp = 0;     // dense feed-forward, padded
    float *norm = nullptr, *norm2 = nullptr;
    const float *mu[5] = {}; // token shift of r, k, v, gate, decay
    fh_qmatrix *rkvg = nullptr, *w1 = nullptr, *w2 = nullptr, *up = nullptr;
    fh_qmatrix *in = nullptr, *wo = nullptr, *uk = nullptr, *uv = nullptr, *gate_up = nullptr, *down = nullptr,
               *s_gate_up = nullptr, *s_down = nullptr;
};

// A tensor the model file must hold.
struct Slot {
    int64_t n, k; // k 0: a vector; -1: the file's
    std::function<fh_status(const void *bytes, uint32_t type, int64_t n, int64_t k)> put;
    bool done = false, optional = false;
};

struct Hybrid : fh_decoder {
    const Design *design = nullptr;
    int dtype = FH_F32;
    float eps = 0.f;
    int kpd = 0; // width, padded
    std::vector<Layer> layer;
    std::map<std::string, Slot> slots;
    std::vector<void *> owned;           // device vectors and states, freed with the decoder
    std::vector<fh_qmatrix *> matrices;
    std::map<std::string, std::pair<float *, float *>> ropes;
    fh_qmatrix *embd = nullptr, *out = nullptr, *pos_table = nullptr;
    float *out_norm = nullptr;
    int *pos_dev = nullptr;
    // step buffers for portions of cap_s tokens over cap_keys visible positions
    int cap_s = 0, cap_keys = 0;
    std::vector<void *> steps, key_steps;
    float *x = nullptr, *proj = nullptr, *mix = nullptr, *hn = nullptr, *qa = nullptr, *part = nullptr, *o = nullptr, *s_gu = nullptr,
          *act1 = nullptr;
    void *h = nullptr, *oact = nullptr;
    // sublayers normed at their end: the other residual row of a decode step; token shifts (operand rows, and f32 rows of the
    // decay's), their products, the decay's low-rank row and argument, feed-forward activations
    float *x2 = nullptr, *shift_w = nullptr, *rkvg = nullptr, *low = nullptr, *z = nullptr;
    void *shift = nullptr, *fact = nullptr;
    FhTile *group_rows = nullptr;
    int *n_group_rows = nullptr;
    const float *cur = nullptr, *pend = nullptr; // decode: residual row so far; norm weight of the sublayer output in `mix` to add
    FhGqaWork gw{};
    FhRecWork rw{};
    FhMoeWork mw{};
    FhLatentWork lw{};
    float *normed = nullptr; // final-norm hidden state of the last head() row
    bool keep = false;
    float *kept = nullptr;
    int kept_s = 0, kept_cap = 0;

    ~Hybrid() override;
    fh_status init(const FhJson &j);
    fh_status init_layer(int i, const FhJson &j);
    fh_status init_mlp(int i, const FhJson &j);
    fh_status init_dense(int i, const FhJson &j);
    fh_status init_attention(Layer &l, const std::string &base, const FhJson &c);
    fh_status init_time_mixing(Layer &l, const std::string &base, const FhJson &c);
    fh_status rope(const FhJson &rot, int most, const float **cos_t, const float **sin_t, int *pairs);
    fh_status ensure_steps(int s) override;
    fh_status ensure_keys(int keys);
    int max_portion() const override { return 2048; }
    fh_status layers(int s, bool dev_pos) override;
    fh_status prefill_layer(Layer &l, int s);
    fh_status prefill_apart(Layer &l, int s);
    fh_status step_apart(Layer &l);
    FhMvAdd take();
    fh_status step_layer(Layer &l);
    fh_status head(int row, float *dst) override;
    const float *hidden() const override { return normed; }
    fh_status reserve(int positions) override;
    int64_t capacity() const override {
        int64_t c = 0; // every cache only grows
        for (auto &l : layer) c += l.cache ? l.cache->capacity : 0;
        return c;
    }
    fh_status set_len(int len, bool device) override;
    int *len_dev() override { return pos_dev; }
    uint64_t weight_bytes() const override;
    fh_status load_tensor(const char *name, uint32_t type, int64_t n, int64_t k, const void *bytes, size_t len) override;
    fh_status finalize() override;
    fh_status keep_layers(bool on) override {
        keep = on;
        return FH_OK;
    }
    fh_status layer_output(int li, float *dst, int64_t count) override;

    // ---- construction helpers
    fh_status dev_floats(float **p, size_t n) {
        FH_TRY(fh_malloc(dev, n * 4, (void **)p));
        owned.push_back(*p);
        return FH_OK;
    }
    fh_status matrix(int64_t n, int64_t k, fh_qmatrix **q) {
        FH_TRY(fh_qmatrix_alloc_bf16(dev, n, k, q));
        matrices.push_back(*q);
        return FH_OK;
    }
    // rows [row0, row0 + n) of a matrix; group 16: row r goes to row0 + 32 (r / 16) + r % 16 (gate and up interleaved)
    void slot_rows(const std::string &name, fh_qmatrix *q, int64_t row0, int64_t n, int64_t k, bool interleave = false) {
        slots[name] = Slot{n, k, [=](const void *b, uint32_t type, int64_t, int64_t) -> fh_status {
            if (type != FH_BF16) FH_FAIL(FH_ERR_UNSUPPORTED, "%s: matrices are bf16", name.c_str());
            return fh_qmatrix_put_bf16(q, row0, n, k, b, interleave);
        }};
    }
    // columns [col0, col0 + k) of a matrix
    void slot_cols(const std::string &name, fh_qmatrix *q, int64_t col0, int64_t n, int64_t k) {
        slots[name] = Slot{n, k, [=](const void *b, uint32_t type, int64_t, int64_t) -> fh_status {
            if (type != FH_BF16) FH_FAIL(FH_ERR_UNSUPPORTED, "%s: matrices are bf16", name.c_str());
            return fh_qmatrix_put_bf16(q, 0, n, k, b, false, col0);
        }};
    }
    // a matrix one side of which only the file knows
    void slot_matrix(const std::string &name, fh_qmatrix **q, int64_t n, int64_t k) {
        slots[name] = Slot{n, k, [=](const void *b, uint32_t type, int64_t rows, int64_t cols) -> fh_status {
            if (type != FH_BF16) FH_FAIL(FH_ERR_UNSUPPORTED, "%s: matrices are bf16", name.c_str());
            FH_REQUIRE(!*q || ((*q)->n == rows && (*q)->k == cols), "%s: loaded twice with different shapes", name.c_str());
            if (!*q) FH_TRY(matrix(rows, cols, q));
            return fh_qmatrix_put_bf16(*q, 0, rows, cols, b, false);
        }};
    }
    // a head's rows are padded from `per` to `padded`
    void slot_heads(const std::string &name, fh_qmatrix *q, int heads, int per, int padded, int64_t k) {
        slots[name] = Slot{(int64_t)heads * per, k, [=](const void *b, uint32_t type, int64_t, int64_t) -> fh_status {
            if (type != FH_BF16) FH_FAIL(FH_ERR_UNSUPPORTED, "%s: matrices are bf16", name.c_str());
            for (int i = 0; i < heads; i++)
                FH_TRY(fh_qmatrix_put_bf16(q, (int64_t)i * padded, per, k, (const uint8_t *)b + (size_t)i * per * k * 2, false));
            return FH_OK;
        }};
    }
    fh_status slot_vector(const std::string &name, float **p, int64_t n, int64_t k = 0, float add = 0.f) {
        const int64_t count = n * (k ? k : 1);
        FH_TRY(dev_floats(p, (size_t)count));
        float *dst = *p;
        slots[name] = Slot{n, k, [=](const void *b, uint32_t type, int64_t, int64_t) -> fh_status {
            std::vector<float> v((size_t)count);
            for (int64_t i = 0; i < count; i++) {
                uint16_t u;
                if (type == FH_BF16) {
                    memcpy(&u, (const uint8_t *)b + 2 * i, 2);
                    const uint32_t w = (uint32_t)u << 16;
                    memcpy(&v[i], &w, 4);
                } else if (type == FH_W_F16) {
                    memcpy(&u, (const uint8_t *)b + 2 * i, 2);
                    _Float16 f;
                    memcpy(&f, &u, 2);
                    v[i] = (float)f;
                } else if (type == FH_W_F32) memcpy(&v[i], (const uint8_t *)b + 4 * i, 4);
                else FH_FAIL(FH_ERR_UNSUPPORTED, "%s: unsupported type %u", name.c_str(), type);
                v[i] += add;
            }
            return fh_upload(dev, dst, v.data(), (size_t)count * 4);
        }};
        return FH_OK;
    }
};

// ---- configuration values
fh_status get_int(const FhJson &j, const char *name, int lo, int *out) {
    const FhJson *v = j.find(name);
    FH_REQUIRE(v && v->is_number(), "configuration: '%s' is missing", name);
    FH_REQUIRE(v->num == std::floor(v->num) && v->num >= lo && v->num <= 1 << 30, "configuration: '%s' = %g is out of range", name, v->num);
    *out = (int)v->num;
    return FH_OK;
}
fh_status get_double(const FhJson &j, const char *name, double *out) {
    const FhJson *v = j.find(name);
    FH_REQUIRE(v && v->is_number(), "configuration: '%s' is missing", name);
    *out = v->num;
    return FH_OK;
}
fh_status get_object(const FhJson &j, const char *name, const FhJson **out) {
    const FhJson *v = j.find(name);
    FH_REQUIRE(v && v->is_object(), "configuration: '%s' is missing", name);
    *out = v;
    return FH_OK;
}

fh_status Hybrid::init(const FhJson &j) {
    FH_TRY(get_int(j, "width", 1, &d_model));
    FH_TRY(get_int(j, "vocab", 1, &vocab));
    const FhJson *norm, *ls = j.find("layers");
    FH_TRY(get_object(j, "norm", &norm));
    double e;
    FH_TRY(get_double(*norm, "eps", &e));
    eps = (float)e;
    FH_REQUIRE(ls && ls->is_array() && !ls->items.empty(), "configuration: 'layers' is missing");
    n_layers = (int)ls->items.size();
    kpd = (int)fh_pad64(d_model);
    layer.resize(n_layers);
    const float one = design->norm_one_plus ? 1.f : 0.f;
    FH_TRY(matrix(vocab, d_model, &embd));
    FH_TRY(matrix(vocab, d_model, &out));
    slot_rows("embed", embd, 0, vocab, d_model);
    slot_rows("head", out, 0, vocab, d_model);
    FH_TRY(slot_vector("final.norm", &out_norm, d_model, 0, one));
    if (design->positions) {
        int most;
        FH_TRY(get_int(j, "max_positions", 1, &most));
        ctx = std::min(ctx, most);
        FH_TRY(matrix(most, d_model, &pos_table));
        slot_rows("pos", pos_table, 0, most, d_model);
    }
    FH_TRY(fh_malloc(dev, 256, (void **)&pos_dev));
    owned.push_back(pos_dev);
    for (int i = 0; i < n_layers; i++) {
        FH_REQUIRE(ls->items[i].is_object(), "configuration: layer %d is not an object", i);
        FH_TRY(init_layer(i, ls->items[i]));
    }
    return FH_OK;
}

// Tables of a rotation (shared by layers with the same one) over at most `most` dimensions of a head.
fh_status Hybrid::rope(const FhJson &rot, int most, const float **cos_t, const float **sin_t, int *pairs) {
    int dims;
    double rbase;
    FH_TRY(get_int(rot, "dims", 2, &dims));
    FH_TRY(get_double(rot, "base", &rbase));
    FH_REQUIRE(dims % 2 == 0 && dims <= most, "rotation of %d of %d dimensions", dims, most);
    *pairs = dims / 2;
    fh_yarn_scaling y{};
    const FhJson *sc = rot.find("scaling");
    if (sc) {
        double v;
        FH_TRY(get_double(*sc, "factor", &v)); y.factor = (float)v;
        FH_TRY(get_double(*sc, "original", &v)); y.original = (float)v;
        FH_TRY(get_double(*sc, "fast", &v)); y.fast = (float)v;
        FH_TRY(get_double(*sc, "slow", &v)); y.slow = (float)v;
    }
    char key[160];
    snprintf(key, sizeof key, "%d %.17g %.9g %.9g %.9g %.9g", dims, rbase, y.factor, y.original, y.fast, y.slow);
    auto &t = ropes[key];
    if (!t.first) {
        FH_TRY(dev_floats(&t.first, (size_t)ctx * *pairs));
        FH_TRY(dev_floats(&t.second, (size_t)ctx * *pairs));
        FH_TRY(fh_rope_tables_yarn(dev, dims, ctx, rbase, sc ? &y : nullptr, t.first, t.second));
    }
    *cos_t = t.first, *sin_t = t.second;
    return FH_OK;
}

// Grouped-query attention: its projections are the first columns of the layer's row.
fh_status Hybrid::init_attention(Layer &l, const std::string &base, const FhJson &c) {
    FhGqa &a = l.gqa;
    FH_TRY(get_int(c, "heads", 1, &a.heads));
    FH_TRY(get_int(c, "kv_heads", 1, &a.kv_heads));
    FH_TRY(get_int(c, "dim", 1, &a.dim));
    FH_TRY(get_int(c, "vdim", 1, &a.vdim));
    FH_REQUIRE(a.heads % a.kv_heads == 0, "%d heads do not share %d key heads evenly", a.heads, a.kv_heads);
    FH_REQUIRE(a.dim <= 256 && a.vdim <= 256, "attention heads of %d and %d dimensions (at most 256)", a.dim, a.vdim);
    double scale;
    FH_TRY(get_double(c, "scale", &scale));
    a.scale = (float)scale, a.eps = eps;
    if (const FhJson *m = c.find("mask")) {
        FH_TRY(get_int(*m, "size", 1, &a.window));
        if (m->find("keep_first")) FH_TRY(get_int(*m, "keep_first", 0, &a.keep));
    }
    a.dnp = (a.dim + 7) / 8 * 8, a.dvp = (a.vdim + 7) / 8 * 8;
    const FhJson *rot;
    FH_TRY(get_object(c, "rot", &rot));
    FH_TRY(rope(*rot, a.dim, &a.cos_t, &a.sin_t, &a.pairs));
    const int nq = a.heads * a.dim, nk = a.kv_heads * a.dim, nv = a.kv_heads * a.vdim;
    a.col_q = 0, a.col_k = nq, a.col_v = nq + nk;
    l.nl = nq + nk + nv;
    FH_TRY(matrix(l.nl, d_model, &l.in));
    slot_rows(base + "q", l.in, a.col_q, nq, d_model);
    slot_rows(base + "k", l.in, a.col_k, nk, d_model);
    slot_rows(base + "v", l.in, a.col_v, nv, d_model);
    float *p;
    FH_TRY(slot_vector(base + "q.norm", &p, a.dim)); a.q_norm = p;
    FH_TRY(slot_vector(base + "k.norm", &p, a.dim)); a.k_norm = p;
    if (design->sink) {
        FH_TRY(slot_vector(base + "sink", &p, a.heads));
        a.sink = p;
    }
    const bool wraps = a.window && (int64_t)a.window + a.keep < ctx;
    return fh_kvcache_create_ring(dev, fh_gqa_row(a), wraps ? a.window + a.keep : ctx, dtype, &l.cache);
}

// Time mixing with channel decays: its products are the columns behind the attention's.
fh_status Hybrid::init_time_mixing(Layer &l, const std::string &base, const FhJson &c) {
    FhRecurrent &r = l.rec;
    r.kind = FH_REC_CHANNEL, r.eps = eps;
    FH_TRY(get_int(c, "heads", 1, &r.heads));
    FH_TRY(get_int(c, "dim", 1, &r.dim));
    FH_REQUIRE(r.dim <= 256, "recurrent state of %d rows (at most 256)", r.dim);
    r.kv_heads = r.heads, r.vdim = r.dim;
    const int inner = r.heads * r.dim;
    r.col_q = l.nl, r.col_k = l.nl + inner, r.col_v = l.nl + 2 * inner, r.col_g = l.nl + 3 * inner, r.col_a = l.nl + 4 * inner;
    FH_TRY(matrix((int64_t)4 * inner, d_model, &l.rkvg));
    const char *names[5] = {"r", "k", "v", "g", "w"};
    float *p;
    for (int i = 0; i < 5; i++) {
        if (i < 4) slot_rows(base + names[i], l.rkvg, (int64_t)i * inner, inner, d_model);
        FH_TRY(slot_vector(base + "mu." + names[i], &p, d_model));
        l.mu[i] = p;
    }
    slot_matrix(base + "w1", &l.w1, -1, d_model);
    slot_matrix(base + "w2", &l.w2, inner, -1);
    FH_TRY(slot_vector(base + "w0", &p, inner)); r.w0 = p;
    FH_TRY(slot_vector(base + "u", &p, r.heads, r.dim)); r.bonus = p;
    FH_TRY(slot_vector(base + "norm", &p, inner)); r.norm = p;
    r.norm_len = inner, r.norm_groups = r.heads;
    FH_TRY(dev_floats(&l.rec_state.s, (size_t)inner * r.dim));
    return dev_floats(&l.rec_state.conv, (size_t)2 * d_model);
}

fh_status Hybrid::init_dense(int i, const FhJson &j) {
    Layer &l = layer[i];
    const std::string base = "l" + std::to_string(i) + ".mlp.";
    const FhJson *kind = j.find("kind");
    if (!kind || !kind->is_string() || kind->str != "dense")
        FH_FAIL(FH_ERR_UNSUPPORTED, "configuration: layer %d has an unknown feed-forward", i);
    FH_TRY(get_int(j, "ff", 1, &l.ff));
    l.ffp = (int)fh_pad64(l.ff);
    FH_TRY(matrix(l.ffp, d_model, &l.up));
    FH_TRY(matrix(d_model, l.ff, &l.down));
    slot_rows(base + "up", l.up, 0, l.ff, d_model);
    slot_rows(base + "down", l.down, 0, d_model, l.ff);
    return FH_OK;
}

fh_status Hybrid::init_layer(int i, const FhJson &j) {
    Layer &l = layer[i];
    const std::string base = "l" + std::to_string(i) + ".", mix_ = base + "mix.";
    const FhJson *type = j.find("type"), *c;
    FH_REQUIRE(type && type->is_string(), "configuration: layer %d has no type", i);
    FH_TRY(get_object(j, "mixer", &c));
    FH_TRY(slot_vector(base + "norm1", &l.norm, d_model, 0, design->norm_one_plus ? 1.f : 0.f));
    // the routed experts' logits are the last columns of the projection row
    int experts = 0;
    const FhJson *mlp = j.find("mlp");
    if (design->output_norm) {
        FH_TRY(slot_vector(base + "norm2", &l.norm2, d_model, 0, design->norm_one_plus ? 1.f : 0.f));
        slots[base + "norm2"].optional = !mlp; // nothing uses it without a feed-forward
    } else if (mlp) {
        const FhJson *router;
        FH_TRY(get_object(*mlp, "router", &router));
        FH_TRY(get_int(*router, "experts", 1, &experts));
    }
    auto inputs = [&](int cols) -> fh_status {
        l.np = cols + experts;
        l.moe.col_z = cols;
        return matrix(l.np, d_model, &l.in);
    };
    const bool apart = type->str == "retention" || type->str == "parallel";
    if (apart != design->output_norm)
        FH_FAIL(FH_ERR_UNSUPPORTED, "configuration: layer %d: %s has no mixer '%s'", i, design->name, type->str.c_str());
    if (type->str == "parallel") {
        const FhJson *left, *right;
        double ls, rs;
        l.kind = MIX_PAIR;
        FH_TRY(get_object(*c, "left", &left));
        FH_TRY(get_object(*c, "right", &right));
        FH_TRY(get_double(*c, "left_scale", &ls));
        FH_TRY(get_double(*c, "right_scale", &rs));
        FH_TRY(init_attention(l, mix_ + "left.", *left));
        FH_TRY(init_time_mixing(l, mix_ + "right.", *right));
        l.gqa.out_scale = (float)ls, l.rec.out_scale = (float)rs;
        // one output matrix over both, their inputs side by side
        const int nl = l.gqa.heads * l.gqa.vdim, nr = l.rec.heads * l.rec.vdim;
        l.kpl = (int)fh_pad64(nl), l.inner = l.kpl + nr, l.kpo = (int)fh_pad64(l.inner);
        FH_TRY(matrix(d_model, l.inner, &l.wo));
        slot_cols(mix_ + "left.o", l.wo, 0, d_model, nl);
        slot_cols(mix_ + "right.o", l.wo, l.kpl, d_model, nr);
        return mlp ? init_dense(i, *mlp) : FH_OK;
    }
    if (type->str == "retention") {
        FhRecurrent &r = l.rec;
        l.kind = FH_MIX_RECURRENT;
        r.kind = FH_REC_RETENTION, r.eps = eps, r.halves = 1;
        FH_TRY(get_int(*c, "heads", 1, &r.heads));
        FH_TRY(get_int(*c, "dim", 1, &r.dim));
        FH_TRY(get_int(*c, "vdim", 1, &r.vdim));
        FH_REQUIRE(r.dim <= 256, "recurrent state of %d rows (at most 256)", r.dim);
        r.kv_heads = r.heads;
        r.k_scale = (float)(1.0 / std::sqrt((double)r.dim));
        const FhJson *rot, *decay = c->find("decay");
        FH_TRY(get_object(*c, "rot", &rot));
        FH_TRY(rope(*rot, r.dim, &r.cos_t, &r.sin_t, &r.pairs));
        FH_REQUIRE(decay && decay->is_array() && (int)decay->items.size() == r.heads, "configuration: layer %d needs one decay per head", i);
        std::vector<float> ld;
        for (const FhJson &d : decay->items) {
            FH_REQUIRE(d.is_number() && d.num >= 0.0 && d.num <= 1.0, "configuration: layer %d: a decay lies between 0 and 1", i);
            ld.push_back((float)std::max(std::log(d.num), -1e4)); // e^-10000 is zero
        }
        float *p;
        FH_TRY(dev_floats(&p, ld.size()));
        FH_TRY(fh_upload(dev, p, ld.data(), ld.size() * 4));
        r.log_decay = p;
        const int nq = r.heads * r.dim, inner = r.heads * r.vdim;
        r.col_q = 0, r.col_k = nq, r.col_v = 2 * nq, r.col_g = 2 * nq + inner;
        FH_TRY(inputs(r.col_g + inner));
        slot_rows(mix_ + "q", l.in, r.col_q, nq, d_model);
        slot_rows(mix_ + "k", l.in, r.col_k, nq, d_model);
        slot_rows(mix_ + "v", l.in, r.col_v, inner, d_model);
        slot_rows(mix_ + "g", l.in, r.col_g, inner, d_model);
        r.norm_len = r.vdim, r.norm_groups = r.heads;
        l.inner = inner;
        FH_TRY(dev_floats(&l.rec_state.s, (size_t)inner * r.dim));
    } else if (type->str == "latent_attention") {
        FhLatent &a = l.lat;
        l.kind = FH_MIX_LATENT;
        FH_TRY(get_int(*c, "heads", 1, &a.heads));
        FH_TRY(get_int(*c, "dim", 1, &a.dn));
        FH_TRY(get_int(*c, "rot_dim", 1, &a.dr));
        FH_TRY(get_int(*c, "vdim", 1, &a.dv));
        FH_TRY(get_int(*c, "kv_rank", 1, &a.rank));
        double scale;
        FH_TRY(get_double(*c, "scale", &scale));
        a.scale = (float)scale;
        a.eps = eps;
        if (const FhJson *m = c->find("mask")) FH_TRY(get_int(*m, "size", 1, &a.window));
        a.dnp = (a.dn + 7) / 8 * 8, a.drp = (a.dr + 7) / 8 * 8, a.r8 = (a.rank + 7) / 8 * 8, a.rp = (int)fh_pad64(a.rank);
        FH_REQUIRE(fh_latent_dq(a), "attention over %d + %d query dimensions (at most 256)", a.dn, a.dr);
        const FhJson *rot;
        FH_TRY(get_object(*c, "rot", &rot));
        FH_TRY(rope(*rot, a.dr, &a.cos_t, &a.sin_t, &a.pairs));
        const int nq = a.heads * (a.dn + a.dr);
        a.col_q = 0, a.col_kv = nq;
        FH_TRY(inputs(nq + a.rank + a.dr));
        slot_rows(mix_ + "q", l.in, 0, nq, d_model);
        slot_rows(mix_ + "dkv", l.in, nq, a.rank + a.dr, d_model);
        float *p;
        FH_TRY(slot_vector(mix_ + "dkv.norm", &p, a.rank));
        a.c_norm = p;
        FH_TRY(matrix((int64_t)a.heads * a.dnp, a.rank, &l.uk));
        FH_TRY(matrix((int64_t)a.heads * a.dv, a.rank, &l.uv));
        slot_heads(mix_ + "uk", l.uk, a.heads, a.dn, a.dnp, a.rank);
        slot_rows(mix_ + "uv", l.uv, 0, (int64_t)a.heads * a.dv, a.rank);
        a.uk = (const uint16_t *)l.uk->data, a.uv = (const uint16_t *)l.uv->data;
        if (design->sink) {
            FH_TRY(slot_vector(mix_ + "sink", &p, a.heads));
            a.sink = p;
        }
        l.inner = a.heads * a.dv;
        FH_TRY(fh_kvcache_create_ring(dev, fh_latent_row(a), a.window && a.window < ctx ? a.window : ctx, dtype, &l.cache));
    } else if (type->str == "delta" || type->str == "mamba2") {
        FhRecurrent &r = l.rec;
        l.kind = FH_MIX_RECURRENT;
        r.kind = type->str == "delta" ? FH_REC_DELTA : FH_REC_SPACE;
        r.eps = eps;
        FH_TRY(get_int(*c, "heads", 1, &r.heads));
        FH_TRY(get_int(*c, "vdim", 1, &r.vdim));
        FH_TRY(get_int(*c, "conv", 1, &r.taps));
        FH_TRY(get_int(*c, r.delta() ? "kv_heads" : "groups", 1, &r.kv_heads));
        FH_TRY(get_int(*c, r.delta() ? "dim" : "state", 1, &r.dim));
        FH_REQUIRE(r.heads % r.kv_heads == 0, "%d heads do not share %d key heads evenly", r.heads, r.kv_heads);
        FH_REQUIRE(r.dim <= 256, "recurrent state of %d rows (at most 256)", r.dim);
        const int nq = r.kv_heads * r.dim, inner = r.heads * r.vdim;
        l.inner = inner;
        float *p;
        if (r.delta()) {
            r.q_scale = (float)(1.0 / std::sqrt((double)r.dim));
            r.col_q = 0, r.col_k = nq, r.col_v = 2 * nq, r.col_b = r.col_v + inner, r.col_a = r.col_b + r.heads, r.col_g = r.col_a + r.heads;
            FH_TRY(inputs(r.col_g + inner));
            slot_rows(mix_ + "q", l.in, r.col_q, nq, d_model);
            slot_rows(mix_ + "k", l.in, r.col_k, nq, d_model);
            slot_rows(mix_ + "v", l.in, r.col_v, inner, d_model);
            slot_rows(mix_ + "b", l.in, r.col_b, r.heads, d_model);
            slot_rows(mix_ + "a", l.in, r.col_a, r.heads, d_model);
            slot_rows(mix_ + "g", l.in, r.col_g, inner, d_model);
            FH_TRY(slot_vector(mix_ + "q.conv", &p, nq, r.taps)); r.conv_q = p;
            FH_TRY(slot_vector(mix_ + "k.conv", &p, nq, r.taps)); r.conv_k = p;
            FH_TRY(slot_vector(mix_ + "v.conv", &p, inner, r.taps)); r.conv_v = p;
            r.norm_len = r.vdim, r.norm_groups = r.heads;
        } else {
            // rows of the input matrix: gate | x | B | C | step size
            r.col_g = 0, r.col_v = inner, r.col_k = 2 * inner, r.col_q = 2 * inner + nq, r.col_a = 2 * inner + 2 * nq, r.col_b = r.col_a;
            FH_TRY(inputs(r.col_a + r.heads));
            slot_rows(mix_ + "in", l.in, 0, r.col_a + r.heads, d_model);
            FH_TRY(slot_vector(mix_ + "conv", &p, inner + 2 * nq, r.taps));
            r.conv_v = p, r.conv_k = p + (size_t)inner * r.taps, r.conv_q = p + (size_t)(inner + nq) * r.taps;
            FH_TRY(slot_vector(mix_ + "conv.b", &p, inner + 2 * nq));
            r.bias_v = p, r.bias_k = p + inner, r.bias_q = p + inner + nq;
            FH_TRY(slot_vector(mix_ + "D", &p, r.heads)); r.d_skip = p;
            FH_TRY(get_int(*c, "norm_groups", 1, &r.norm_groups));
            FH_REQUIRE(inner % r.norm_groups == 0, "%d channels do not split into %d norm groups", inner, r.norm_groups);
            r.norm_len = inner, r.gate_first = 1;
        }
        FH_TRY(slot_vector(mix_ + "A_log", &p, r.heads)); r.a_log = p;
        FH_TRY(slot_vector(mix_ + "dt_bias", &p, r.heads)); r.dt_bias = p;
        FH_TRY(slot_vector(mix_ + "norm", &p, r.norm_len)); r.norm = p;
        FH_TRY(dev_floats(&l.rec_state.s, (size_t)inner * r.dim));
        FH_TRY(dev_floats(&l.rec_state.conv, (size_t)r.taps * fh_rec_channels(r)));
    } else FH_FAIL(FH_ERR_UNSUPPORTED, "configuration: layer %d has an unknown mixer '%s'", i, type->str.c_str());
    l.kpo = (int)fh_pad64(l.inner);
    FH_TRY(matrix(d_model, l.inner, &l.wo));
    slot_rows(mix_ + "o", l.wo, 0, d_model, l.inner);
    return !mlp ? FH_OK : design->output_norm ? init_dense(i, *mlp) : init_mlp(i, *mlp);
}

fh_status Hybrid::init_mlp(int i, const FhJson &j) {
    Layer &l = layer[i];
    FhMoe &m = l.moe;
    const std::string base = "l" + std::to_string(i) + ".mlp.";
    const FhJson *kind = j.find("kind"), *router, *ex;
    if (kind && kind->is_string() && kind->str != "moe")
        FH_FAIL(FH_ERR_UNSUPPORTED, "configuration: layer %d has an unknown feed-forward '%s'", i, kind->str.c_str());
    FH_TRY(get_object(j, "router", &router));
    FH_TRY(get_object(j, "expert", &ex));
    double scale;
    FH_TRY(get_int(*router, "experts", 1, &m.experts));
    FH_TRY(get_int(*router, "top", 1, &m.top));
    FH_TRY(get_double(*router, "scale", &scale));
    FH_TRY(get_int(*ex, "ff", 1, &m.ff));
    m.scale = (float)scale;
    FH_REQUIRE(m.top <= m.experts && m.experts <= FH_MOE_MAX_EXPERTS, "%d of %d experts (at most %d)", m.top, m.experts,
               FH_MOE_MAX_EXPERTS);
    m.ffp = (int)fh_pad64(m.ff);
    const int dp = (d_model + 15) / 16 * 16;
    m.gu_stride = (int64_t)2 * m.ffp * kpd, m.down_stride = (int64_t)dp * m.ffp;
    FH_TRY(matrix((int64_t)m.experts * 2 * m.ffp, d_model, &l.gate_up));
    FH_TRY(matrix((int64_t)m.experts * dp, m.ff, &l.down));
    m.gate_up = (const uint16_t *)l.gate_up->data, m.down = (const uint16_t *)l.down->data;
    for (int e = 0; e < m.experts; e++) {
        const std::string n = base + "e" + std::to_string(e);
        slot_rows(n + ".gate", l.gate_up, (int64_t)e * 2 * m.ffp, m.ff, d_model, true);
        slot_rows(n + ".up", l.gate_up, (int64_t)e * 2 * m.ffp + 16, m.ff, d_model, true);
        slot_rows(n + ".down", l.down, (int64_t)e * dp, d_model, m.ff);
    }
    slot_rows(base + "router", l.in, m.col_z, m.experts, d_model);
    if (const FhJson *s = j.find("shared")) {
        FH_TRY(get_int(*s, "ff", 1, &m.sff));
        m.sffp = (int)fh_pad64(m.sff);
        FH_TRY(matrix(2 * m.sffp, d_model, &l.s_gate_up));
        FH_TRY(matrix(d_model, m.sff, &l.s_down));
        m.s_gate_up = (const uint16_t *)l.s_gate_up->data, m.s_down = (const uint16_t *)l.s_down->data;
        slot_rows(base + "shared.gate", l.s_gate_up, 0, m.sff, d_model, true);
        slot_rows(base + "shared.up", l.s_gate_up, 16, m.sff, d_model, true);
        slot_rows(base + "shared.down", l.s_down, 0, d_model, m.sff);
    }
    return FH_OK;
}

void free_all(std::vector<void *> &v) {
    for (void *p : v) (void)hipFree(p);
    v.clear();
}

Hybrid::~Hybrid() {
    (void)hipStreamSynchronize(dev->stream);
    for (fh_qmatrix *q : matrices) fh_qmatrix_free(q);
    for (Layer &l : layer) fh_kvcache_destroy(l.cache);
    free_all(owned);
    free_all(steps);
    free_all(key_steps);
    if (kept) (void)hipFree(kept);
}

fh_status Hybrid::load_tensor(const char *name, uint32_t type, int64_t n, int64_t k, const void *bytes, size_t len) {
    FH_REQUIRE(!finalized, "decoder already finalized");
    auto it = slots.find(name);
    if (it == slots.end()) FH_FAIL(FH_ERR_INVALID, "unknown tensor name '%s'", name);
    Slot &s = it->second;
    FH_REQUIRE((n == s.n || (s.n < 0 && n > 0)) && (k == s.k || (s.k < 0 && k > 0)), "%s: expected [%lld, %lld], got [%lld, %lld]", name, (long long)s.n, (long long)s.k, (long long)n,
               (long long)k);
    FH_REQUIRE(len == (size_t)n * (size_t)(k ? k : 1) * (type == FH_W_F32 ? 4u : 2u), "%s: %zu bytes do not fit its shape", name, len);
    FH_TRY(s.put(bytes, type, n, k));
    s.done = true;
    return FH_OK;
}

fh_status Hybrid::finalize() {
    FH_REQUIRE(!finalized, "decoder already finalized");
    for (auto &s : slots) FH_REQUIRE(s.second.done || s.second.optional, "tensor '%s' is missing", s.first.c_str());
    for (int i = 0; i < n_layers; i++) {
        Layer &l = layer[i];
        if (l.kind != MIX_PAIR) continue;
        FH_REQUIRE(l.w1->n == l.w2->k, "layer %d: the decay's low rank is %lld and %lld", i, (long long)l.w1->n, (long long)l.w2->k);
        l.rec.rank = (int)l.w1->n, l.rec.rp = (int)fh_pad64(l.rec.rank), l.rec.w2 = (const uint16_t *)l.w2->data;
        l.np = l.rec.col_a + l.rec.rank;
    }
    FH_TRY(create_loop_buffers());
    FH_TRY(ensure_steps(1));
    finalized = true;
    return set_len(0, true);
}

fh_status Hybrid::ensure_steps(int s) {
    if (s <= cap_s) return FH_OK;
    (void)hipStreamSynchronize(dev->stream);
    free_all(steps);
    drop_captures(); // a captured decode step holds these pointers
    cap_s = 0;
    int np = 1, kpo = 64, nq = 1, inner = 1, heads = 1, top = 0, ffp = 0, sffp = 0, row = 1, part_ = 1, tiles = 1;
    size_t ql = 1, chunk = 0, gq = 0, four = 0, rp = 0, dff = 0, group_tiles = 0;
    for (const Layer &l : layer) {
        dff = std::max(dff, (size_t)l.ffp);
        if (l.kind == MIX_PAIR) {
            part_ = std::max(part_, (int)fh_gqa_part_floats(l.gqa));
            gq = std::max(gq, (size_t)l.gqa.heads * fh_window_dq(l.gqa.dnp));
            four = std::max(four, (size_t)4 * l.rec.heads * l.rec.dim), rp = std::max(rp, (size_t)l.rec.rp);
            group_tiles = std::max(group_tiles, (size_t)4 * ((s + 63) / 64));
        }
        np = std::max(np, l.np), kpo = std::max(kpo, l.kpo), inner = std::max(inner, l.inner);
        top = std::max(top, l.moe.experts ? l.moe.top : 0), ffp = std::max(ffp, l.moe.ffp), sffp = std::max(sffp, l.moe.sffp);
        if (l.moe.experts) tiles = std::max(tiles, fh_moe_max_tiles(l.moe, s, 64));
        if (l.kind != FH_MIX_LATENT) {
            nq = std::max(nq, l.rec.kv_heads * fh_rec_dp(l.rec)), heads = std::max(heads, l.rec.heads);
            chunk = std::max(chunk, fh_rec_chunk_floats(l.rec, s));
        } else {
            row = std::max(row, l.lat.heads * fh_latent_row(l.lat));
            part_ = std::max(part_, (int)fh_latent_part_floats(l.lat));
            ql = std::max(ql, (size_t)l.lat.heads * fh_latent_dq(l.lat));
        }
    }
    const size_t S = (size_t)s, D = (size_t)d_model, as = fh_act_size(dtype);
    auto get = [&](auto **p, size_t bytes) -> fh_status {
        FH_TRY(fh_malloc(dev, bytes + 256, (void **)p));
        steps.push_back(*p);
        return FH_OK;
    };
    FH_TRY(get(&ids, S * 4));
    FH_TRY(get(&x, S * D * 4));
    FH_TRY(get(&proj, S * np * 4));
    FH_TRY(get(&mix, S * D * 4));
    FH_TRY(get(&h, S * kpd * as));
    FH_TRY(get(&oact, S * kpo * as));
    FH_TRY(get(&hn, (size_t)kpd * 4));
    FH_TRY(get(&normed, (size_t)kpd * 4));
    FH_TRY(get(&qa, (size_t)std::max(row, kpo) * 4)); // a latent row per head, or the input of an output projection
    FH_TRY(get(&part, (size_t)part_ * 4));
    FH_TRY(get(&o, (size_t)kpo * 4));
    FH_TRY(get(&s_gu, (size_t)2 * sffp * 4));
    FH_TRY(get(&act1, std::max((size_t)top * ffp, dff) * 4));
    if (design->output_norm) {
        FH_TRY(get(&x2, D * 4));
        FH_TRY(get(&fact, S * dff * as));
        FH_TRY(get(&shift, four ? S * 4 * kpd * as : 0));
        FH_TRY(get(&shift_w, four ? S * kpd * 4 : 0));
        FH_TRY(get(&rkvg, S * four * 4));
        FH_TRY(get(&low, S * rp * 4));
        FH_TRY(get(&z, S * four));
        FH_TRY(get(&gw.q, S * gq * as));
        FH_TRY(get(&group_rows, group_tiles * sizeof(FhTile)));
        FH_TRY(get(&n_group_rows, 4));
    }
    FH_TRY(get(&rw.q, S * nq * 4));
    FH_TRY(get(&rw.k, S * nq * 4));
    FH_TRY(get(&rw.v, S * inner * 4));
    FH_TRY(get(&rw.beta, S * heads * 4));
    FH_TRY(get(&rw.la, S * heads * 4));
    FH_TRY(get(&rw.o, S * inner * 4));
    rw.chunk = nullptr;
    if (chunk) FH_TRY(get(&rw.chunk, chunk * 4));
    FH_TRY(get(&lw.q, S * ql * as));
    FH_TRY(get(&mw.ids, S * top * 4));
    FH_TRY(get(&mw.wts, S * top * 4));
    FH_TRY(get(&mw.src, S * top * 4));
    FH_TRY(get(&mw.inv, S * top * 4));
    FH_TRY(get(&mw.tiles, (size_t)tiles * sizeof(FhTile)));
    FH_TRY(get(&mw.n_tiles, 4));
    FH_TRY(get(&mw.act, S * top * ffp * as));
    FH_TRY(get(&mw.y, S * top * D * 4));
    FH_TRY(get(&mw.s_act, S * sffp * as));
    FH_TRY(get(&mw.s_y, S * D * 4));
    cap_s = s;
    return FH_OK;
}

// Buffers of a portion's expanded keys and values.
fh_status Hybrid::ensure_keys(int keys) {
    if (keys <= cap_keys) return FH_OK;
    (void)hipStreamSynchronize(dev->stream);
    free_all(key_steps);
    cap_keys = 0;
    const int cap = (keys + 255) / 256 * 256;
    size_t rp = 1, drp = 1, kn = 1, vt = 1, gk = 0, gv = 0;
    for (const Layer &l : layer)
        if (l.kind == MIX_PAIR)
            gk = std::max(gk, (size_t)l.gqa.kv_heads * l.gqa.dnp), gv = std::max(gv, (size_t)l.gqa.kv_heads * l.gqa.dvp);
    for (const Layer &l : layer)
        if (l.kind == FH_MIX_LATENT) {
            rp = std::max(rp, (size_t)l.lat.rp), drp = std::max(drp, (size_t)l.lat.drp);
            kn = std::max(kn, (size_t)l.lat.heads * l.lat.dnp), vt = std::max(vt, (size_t)l.lat.heads * l.lat.dv);
        }
    const size_t as = fh_act_size(dtype);
    auto get = [&](void **p, size_t per) -> fh_status {
        FH_TRY(fh_malloc(dev, per * cap * as + 256, p));
        key_steps.push_back(*p);
        return FH_OK;
    };
    FH_TRY(get(&lw.lat, rp));
    FH_TRY(get(&lw.kr, drp));
    FH_TRY(get(&lw.kn, kn));
    FH_TRY(get(&lw.vt, vt));
    FH_TRY(get(&gw.kn, gk));
    FH_TRY(get(&gw.vr, gv));
    FH_TRY(get(&gw.vt, gv));
    cap_keys = cap;
    return FH_OK;
}

fh_status Hybrid::reserve(int positions) {
    for (Layer &l : layer)
        if (l.cache) FH_TRY(fh_kvcache_reserve(l.cache, positions));
    return FH_OK;
}

__global__ void k_set_position(int *p, int v) { *p = v; }

fh_status Hybrid::set_len(int len, bool device) {
    for (Layer &l : layer)
        if (l.cache) l.cache->len = len;
    if (!device) return FH_OK;
    k_set_position<<<1, 1, 0, dev->stream>>>(pos_dev, len);
    FH_HIP(hipGetLastError());
    return FH_OK;
}

fh_status Hybrid::prefill_layer(Layer &l, int s) {
    FH_TRY(fh_rows_to_act(dev, dtype, x, d_model, s, d_model, l.norm, eps, h, kpd));
    FhGemm g;
    g.w = (const uint16_t *)l.in->data, g.x = h, g.y = proj, g.ldy = l.np, g.n = l.np, g.kp = kpd, g.m = s;
    FH_TRY(fh_gemm(dev, dtype, FH_GEMM_F32, g));
    if (l.kind == FH_MIX_LATENT) {
        const int keys = fh_latent_old(l.lat, pos) + s;
        FH_TRY(ensure_keys(keys));
        lw.ldt = fh_pad64(keys);
        FH_TRY(fh_latent_prefill(dev, dtype, l.lat, l.cache, proj, l.np, s, pos, lw, oact, l.kpo));
    } else FH_TRY(fh_recurrent_prefill(dev, dtype, l.rec, l.rec_state, proj, l.np, s, pos, rw, oact, l.kpo));
    g = FhGemm();
    g.w = (const uint16_t *)l.wo->data, g.x = oact, g.y = mix, g.ldy = d_model, g.n = d_model, g.kp = l.kpo, g.m = s;
    FH_TRY(fh_gemm(dev, dtype, FH_GEMM_F32, g));
    return fh_moe_prefill(dev, dtype, l.moe, h, kpd, proj, l.np, s, d_model, mw, mix, x);
}

fh_status Hybrid::step_layer(Layer &l) {
    const FhMvSeg segs[2] = {{(const uint16_t *)l.in->data, proj, l.np}, {l.moe.s_gate_up, s_gu, 2 * l.moe.sffp}};
    FH_TRY(fh_matvec_norm(dev, x, d_model, l.norm, eps, segs, l.moe.sff ? 2 : 1, hn));
    FhStep st;
    st.kind = l.kind;
    st.rec = l.rec, st.rec_state = l.rec_state, st.lat = l.lat;
    st.proj = proj, st.hn = hn, st.kp = kpd, st.pos_dev = pos_dev;
    st.qa = qa, st.o = o;
    st.moe = l.moe, st.act = act1, st.ids = mw.ids, st.wts = mw.wts, st.s_gu = s_gu;
    st.wo = (const uint16_t *)l.wo->data, st.kpo = l.kpo, st.width = d_model, st.x = x;
    FH_TRY(fh_step_middle(dev, dtype, st, l.cache));
    if (l.kind == FH_MIX_LATENT) FH_TRY(fh_latent_decode(dev, dtype, l.lat, l.cache, pos_dev, qa, part, o));
    return fh_step_out(dev, st);
}

// One portion through a layer whose sublayers are normed at their end: x and its operand rows h in, both out.
fh_status Hybrid::prefill_apart(Layer &l, int s) {
    auto product = [&](int dt, int epi, const fh_qmatrix *w, int64_t n, const void *in, int kp, void *out, int64_t ld) {
        FhGemm g;
        g.w = (const uint16_t *)w->data, g.x = in, g.y = out, g.ldy = ld, g.n = (int)n, g.kp = kp, g.m = s;
        return fh_gemm(dev, dt, epi, g);
    };
    if (l.kind == MIX_PAIR) {
        const int inner = l.rec.heads * l.rec.dim, rp = l.rec.rp;
        FH_TRY(product(dtype, FH_GEMM_F32, l.in, l.nl, h, kpd, proj, l.nl));
        FhShift m;
        m.n = 5;
        const size_t plane = (size_t)s * kpd * fh_act_size(dtype);
        for (int i = 0; i < 5; i++) m.mu[i] = l.mu[i], m.y[i] = i < 4 ? (void *)((char *)shift + i * plane) : (void *)shift_w;
        m.f32[4] = 1;
        FH_TRY(fh_token_shift(dev, dtype, m, x, s, d_model, pos, l.rec_state.conv, kpd));
        FhGemm g; // the four inputs are the row groups of one product
        g.w = (const uint16_t *)l.rkvg->data, g.w_group = (int64_t)inner * kpd, g.x = shift, g.y = rkvg, g.ldy = inner, g.n = inner, g.kp = kpd;
        g.tile_rows = fh_group_tile_rows(dev, dtype, 4, s, inner);
        g.max_tiles = 4 * ((s + g.tile_rows - 1) / g.tile_rows), g.tiles = group_rows, g.n_tiles = n_group_rows;
        FH_TRY(fh_group_tiles(dev, 4, s, g.tile_rows, group_rows, n_group_rows));
        FH_TRY(fh_gemm(dev, dtype, FH_GEMM_F32, g));
        // the decay's argument is worked out in 32 bits whatever the activation type
        FH_TRY(fh_low_rank_tanh(dev, shift_w, kpd, s, (const uint16_t *)l.w1->data, l.rec.rank, low, rp));
        FH_TRY(product(FH_F32, FH_GEMM_F32, l.w2, inner, low, rp, z, inner));
        const int keys = fh_gqa_keys(l.gqa, s, pos);
        FH_TRY(ensure_keys(keys));
        gw.ldt = fh_pad64(keys);
        FH_TRY(fh_gqa_prefill(dev, dtype, l.gqa, l.cache, proj, l.nl, s, pos, gw, oact, l.kpo, l.kpl));
        const size_t rows = (size_t)s * inner;
        const FhRecRows in{rkvg, rkvg + rows, rkvg + 2 * rows, rkvg + 3 * rows, z};
        FH_TRY(fh_recurrent_channel(dev, dtype, l.rec, l.rec_state, in, s, pos, rw, (char *)oact + l.kpl * fh_act_size(dtype), l.kpo,
                                    l.kpo - l.kpl));
    } else {
        FH_TRY(product(dtype, FH_GEMM_F32, l.in, l.np, h, kpd, proj, l.np));
        FH_TRY(fh_recurrent_prefill(dev, dtype, l.rec, l.rec_state, proj, l.np, s, pos, rw, oact, l.kpo));
    }
    FH_TRY(product(dtype, FH_GEMM_F32, l.wo, d_model, oact, l.kpo, mix, d_model));
    FH_TRY(fh_add_normed(dev, dtype, x, mix, s, d_model, l.norm, eps, x, h, kpd));
    if (!l.ff) return FH_OK;
    FH_TRY(product(dtype, FH_GEMM_RELU2, l.up, l.ffp, h, kpd, fact, l.ffp));
    FH_TRY(product(dtype, FH_GEMM_F32, l.down, d_model, fact, l.ffp, mix, d_model));
    return fh_add_normed(dev, dtype, x, mix, s, d_model, l.norm2, eps, x, h, kpd);
}

// Decode: the residual row for the next sublayer, with the output of the one before still to be normed and added.
FhMvAdd Hybrid::take() {
    FhMvAdd in;
    in.x = cur, in.eps = eps;
    if (pend) {
        float *to = cur == x ? x2 : x;
        in.y = mix, in.w = pend, in.x_out = to;
        cur = to, pend = nullptr;
    }
    return in;
}

fh_status Hybrid::step_apart(Layer &l) {
    FhMixStep st;
    st.rec = 1, st.r = l.rec, st.state = l.rec_state, st.proj = proj, st.pos_dev = pos_dev, st.o = o, st.act = qa, st.part = part;
    FhMvAdd in = take();
    const uint16_t *w = (const uint16_t *)l.in->data;
    if (l.kind == MIX_PAIR) {
        st.attn = 1, st.gqa = l.gqa, st.kpl = l.kpl;
        in.state = l.rec_state.conv, in.pos_dev = pos_dev;
        const int inner = l.rec.heads * l.rec.dim;
        FhMvMix segs[6] = {{w, nullptr, proj, l.nl, FH_MV_ACT_NONE}};
        for (int i = 0; i < 4; i++)
            segs[1 + i] = FhMvMix{(const uint16_t *)l.rkvg->data + (int64_t)i * inner * kpd, l.mu[i], proj + l.nl + i * inner, inner, FH_MV_ACT_NONE};
        segs[5] = FhMvMix{(const uint16_t *)l.w1->data, l.mu[4], proj + l.rec.col_a, l.rec.rank, FH_MV_ACT_TANH};
        FH_TRY(fh_matvec_mix(dev, in, d_model, segs, 6));
    } else {
        const FhMvMix seg{w, nullptr, proj, l.np, FH_MV_ACT_NONE};
        FH_TRY(fh_matvec_mix(dev, in, d_model, &seg, 1));
    }
    FH_TRY(fh_step_mixers(dev, dtype, st, l.cache));
    auto plain = [&](const float *v, int k, const fh_qmatrix *q) {
        FhMvAdd a;
        a.x = v;
        const FhMvMix seg{(const uint16_t *)q->data, nullptr, mix, d_model, FH_MV_ACT_NONE};
        return fh_matvec_mix(dev, a, k, &seg, 1);
    };
    if (l.kind == MIX_PAIR) {
        FH_TRY(fh_step_mix_out(dev, st, l.cache));
        FH_TRY(plain(qa, l.inner, l.wo));
    } else { // norm and gate on the way into the output projection
        FhMvAdd a;
        a.x = o, a.eps = eps, a.gate = proj + l.rec.col_g, a.groups = l.rec.norm_groups, a.w = l.rec.norm, a.w_len = l.rec.norm_len;
        a.scale = l.rec.out_scale;
        const FhMvMix seg{(const uint16_t *)l.wo->data, nullptr, mix, d_model, FH_MV_ACT_NONE};
        FH_TRY(fh_matvec_mix(dev, a, l.inner, &seg, 1));
    }
    pend = l.norm;
    if (!l.ff) return FH_OK;
    const FhMvMix up{(const uint16_t *)l.up->data, nullptr, act1, l.ff, FH_MV_ACT_RELU2};
    FH_TRY(fh_matvec_mix(dev, take(), d_model, &up, 1));
    FH_TRY(plain(act1, l.ff, l.down));
    pend = l.norm2;
    return FH_OK;
}

fh_status Hybrid::layers(int s, bool dev_pos) {
    if (keep && !dev_pos) {
        if (s > kept_cap) {
            (void)hipStreamSynchronize(dev->stream);
            if (kept) (void)hipFree(kept);
            kept = nullptr, kept_cap = 0;
            FH_TRY(fh_malloc(dev, (size_t)n_layers * s * d_model * 4, (void **)&kept));
            kept_cap = s;
        }
        kept_s = s;
    }
    if (design->output_norm) {
        FH_TRY(fh_embed_at(dev, dtype, embd, pos_table, ids, s, pos, dev_pos ? pos_dev : nullptr, x, s > 1 ? h : nullptr, kpd));
        cur = x, pend = nullptr;
        for (int i = 0; i < n_layers; i++) {
            FH_TRY(s == 1 ? step_apart(layer[i]) : prefill_apart(layer[i], s));
            if (!keep || dev_pos) continue;
            float *to = kept + (size_t)i * s * d_model;
            if (s == 1) FH_TRY(fh_add_normed(dev, dtype, cur, mix, 1, d_model, pend, eps, to, nullptr, kpd));
            else FH_TRY(fh_copy(dev, to, x, (size_t)s * d_model * 4));
        }
        return s == 1 ? fh_add_normed(dev, dtype, cur, mix, 1, d_model, pend, eps, x, nullptr, kpd) : FH_OK;
    }
    FH_TRY(fh_embed_rows(embd, ids, nullptr, s, x));
    for (int i = 0; i < n_layers; i++) {
        FH_TRY(s == 1 ? step_layer(layer[i]) : prefill_layer(layer[i], s));
        if (keep && !dev_pos) FH_TRY(fh_copy(dev, kept + (size_t)i * s * d_model, x, (size_t)s * d_model * 4));
    }
    return FH_OK;
}

fh_status Hybrid::head(int row, float *dst) {
    const FhMvSeg seg{(const uint16_t *)out->data, dst, vocab};
    return fh_matvec_norm(dev, x + (size_t)row * d_model, d_model, out_norm, eps, &seg, 1, normed);
}

fh_status Hybrid::layer_output(int li, float *dst, int64_t count) {
    FH_REQUIRE(keep && kept, "layer outputs are not kept (fh_decoder_keep_layers)");
    FH_REQUIRE(li >= 0 && li < n_layers && count == (int64_t)kept_s * d_model, "layer %d of %d, %lld values of the last portion's %d x %d",
               li, n_layers, (long long)count, kept_s, d_model);
    return fh_download(dev, dst, kept + (size_t)li * count, (size_t)count * 4);
}

uint64_t Hybrid::weight_bytes() const {
    auto b = [](const fh_qmatrix *q) { return q ? (uint64_t)q->n * q->k * 2 : 0; };
    uint64_t t = b(out);
    for (const Layer &l : layer) {
        t += b(l.in) + b(l.wo) + b(l.uk) + b(l.uv) + b(l.s_down) + (uint64_t)2 * l.moe.sff * d_model * 2;
        t += b(l.rkvg) + b(l.w1) + b(l.w2);
        if (l.ff) t += (uint64_t)2 * l.ff * d_model * 2;
        if (l.moe.experts) t += (uint64_t)l.moe.top * 3 * l.moe.ff * d_model * 2;
    }
    return t;
}

} // namespace

bool fh_hybrid_knows(const char *architecture) { return find_design(architecture) != nullptr; }

fh_status fh_hybrid_create(fh_device *dev, const char *config_json, int dtype, int ctx, fh_decoder **out) {
    FhJson j;
    std::string err;
    if (!FhJson::parse(config_json, strlen(config_json), j, err)) FH_FAIL(FH_ERR_INVALID, "configuration: %s", err.c_str());
    const FhJson *a = j.find("architecture");
    FH_REQUIRE(a && a->is_string(), "the configuration names no architecture");
    std::unique_ptr<Hybrid> m(new Hybrid());
    m->dev = dev;
    m->dtype = dtype;
    m->ctx = ctx;
    m->design = find_design(a->str.c_str());
    FH_REQUIRE(m->design, "unknown architecture '%s'", a->str.c_str());
    FH_TRY(m->init(j));
    *out = m.release();
    return FH_OK;
}
