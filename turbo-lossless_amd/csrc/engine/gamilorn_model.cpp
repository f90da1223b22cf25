// Configuration, loading and saving of Gamilorn models (gamilorn.h).
// Directory forms: part_store.h.
#include "gamilorn.h"

#include <cmath>
#include <cstdio>
#include <cstdlib>
#include <cstring>

#include "family.h"
#include "json.h"
#include "part_store.h"

using namespace model_store;
using part_store::Parts;
using part_store::ends_with;
using part_store::is_checkpoint;
using part_store::layer_name;
using part_store::values;

namespace gamilorn {

Data* data_of(const Model* m) { return (Data*)m->family_data; }

namespace {

const char* const kArchitecture = "Gamilorn";

// Everything config.json says.  The rank of the decay projection and the position table's length are sizes of tensors.
void parse_config(const std::string& text, Config& c)
{
    const Json j = Json::parse(text);
    if (j.str("architecture") != kArchitecture) throw JsonError("the architecture is not Gamilorn");
    const int64_t top = 1 << 24;
    c.text = text;
    c.vocab = (int)j.integer("vocab", 1, top);
    c.width = (int)j.integer("width", 1, 1 << 20);
    c.max_positions = j.has("max_positions") ? (int)j.integer("max_positions", 1, top) : 0;
    c.eps = (float)j.at("norm").real("eps");
    c.softcap = j.has("logit_softcap") && !j.at("logit_softcap").is_null() ? (float)j.real("logit_softcap") : 0.0f;
    if (!(c.eps >= 0.0f) || !(c.softcap >= 0.0f)) throw JsonError("norm.eps or logit_softcap is negative");
    c.layers.clear();
    const Json& ls = j.at("layers");
    if (ls.kind != Json::ARR || ls.items.empty()) throw JsonError("\"layers\" is not a list of layers");
    for (const Json& l : ls.items) {
        LayerConfig k = {};
        if (l.str("type") != "parallel") throw JsonError("a layer has the unknown type \"" + l.str("type") + "\"");
        const Json &m = l.at("mixer"), &a = m.at("left"), &b = m.at("right"), &mask = a.at("mask");
        k.heads = (int)a.integer("heads", 1, 65536);
        k.kv_heads = (int)a.integer("kv_heads", 1, 65536);
        k.dim = (int)a.integer("dim", 1, 4096);
        k.vdim = (int)a.integer("vdim", 1, 4096);
        k.scale = (float)a.real("scale");
        k.window = (int)mask.integer("size", 1, 1 << 30);
        k.keep_first = mask.has("keep_first") && !mask.at("keep_first").is_null() ? (int)mask.integer("keep_first", 0, 1 << 30) : 0;
        k.d_heads = (int)b.integer("heads", 1, 65536);
        k.d_dim = (int)b.integer("dim", 1, 512);
        k.left_scale = (float)m.real("left_scale");
        k.right_scale = (float)m.real("right_scale");
        if (k.heads % k.kv_heads) throw JsonError("heads is not a multiple of kv_heads");
        if (l.has("mlp") && !l.at("mlp").is_null()) {
            const Json& f = l.at("mlp");
            if (f.str("kind") != "dense") throw JsonError("a feed-forward has the unknown kind \"" + f.str("kind") + "\"");
            k.ff = (int)f.integer("ff", 1, top);
        }
        c.layers.push_back(k);
    }
}

// ---- the parts a model is stored and held as
void walk(const Config& c, Model* m, Data* d, const Parts& p)
{
    p.table("embed", m->token_embd, (size_t)c.vocab * c.width);
    p.table("pos", d->pos_table, (size_t)c.max_positions * c.width);
    for (size_t i = 0; i < d->layers.size(); i++) {
        Layer& L = d->layers[i];
        const LayerConfig& k = L.c;
        p.vector(layer_name(i, "norm1"), L.norm1, c.width);
        p.weight(layer_name(i, "mix.in"), L.w_in, k.in_rows(), c.width);
        p.vector(layer_name(i, "mix.in.b"), L.in_bias, k.in_rows());
        p.vector(layer_name(i, "mix.head_bias"), L.head_bias, k.heads);
        p.vector(layer_name(i, "mix.w2t"), L.w2t, (size_t)k.rank * k.del());
        p.vector(layer_name(i, "mix.w0"), L.w0, k.del());
        p.vector(layer_name(i, "mix.norm"), L.o_norm, k.del());
        p.weight(layer_name(i, "mix.out"), L.w_out, c.width, k.out_cols());
        if (!k.ff) continue;
        p.vector(layer_name(i, "norm2"), L.norm2, c.width);
        p.weight(layer_name(i, "mlp.up"), L.up, k.ff, c.width);
        p.weight(layer_name(i, "mlp.down"), L.down, c.width, k.ff);
        p.vector(layer_name(i, "mlp.act"), L.act, 2);
    }
    p.vector("final.norm", m->output_norm, c.width);
    p.weight("head", m->output_proj, c.vocab, c.width);
}

void empty_layers(const Config& c, Data& d)
{
    d.layers.clear();
    for (const LayerConfig& k : c.layers) {
        Layer L;
        L.c = k;
        L.norm1 = L.norm2 = L.in_bias = L.head_bias = L.w2t = L.w0 = L.o_norm = L.act = nullptr;
        for (CompressedWeight* w : {&L.w_in, &L.w_out, &L.up, &L.down}) clear_weight(*w);
        L.xielu = {T12_ACT_XIELU, 0.0f, 0.0f};
        d.layers.push_back(L);
    }
}

// ---- checkpoint ------------------------------------------------------------------------------------------------
struct Piece {
    const char* name;                    // below the layer
    int rows, cols;                      // cols 0: a vector
};
std::vector<Piece> layer_tensors(const LayerConfig& k, int width)
{
    std::vector<Piece> t = {
        {"norm1", width, 0},
        {"mix.left.q", k.heads * k.dim, width}, {"mix.left.q.b", k.heads * k.dim, 0},
        {"mix.left.k", k.kv_heads * k.dim, width}, {"mix.left.k.b", k.kv_heads * k.dim, 0},
        {"mix.left.v", k.kv_heads * k.vdim, width}, {"mix.left.v.b", k.kv_heads * k.vdim, 0},
        {"mix.left.pb", k.heads, 0}, {"mix.left.o", width, k.att()},
        {"mix.right.r", k.del(), width}, {"mix.right.k", k.del(), width}, {"mix.right.v", k.del(), width},
        {"mix.right.g", k.del(), width}, {"mix.right.a", k.del(), width}, {"mix.right.a.b", k.del(), 0},
        {"mix.right.w1", k.rank, width}, {"mix.right.w2", k.del(), k.rank}, {"mix.right.w0", k.del(), 0},
        {"mix.right.norm", k.del(), 0}, {"mix.right.o", width, k.del()}};
    if (k.ff) {
        t.push_back({"norm2", width, 0});
        t.push_back({"mlp.up", k.ff, width});
        t.push_back({"mlp.down", width, k.ff});
        t.push_back({"mlp.act", 2, 0});
    }
    return t;
}

// Opens the checkpoint, takes the sizes only tensors know, and checks that every tensor is there with its shape.
bool open_checkpoint(const std::string& dir, Config& c, Checkpoint& ck, std::string& err)
{
    if (!ck.open(dir + "/model.safetensors", err)) return false;
    const Checkpoint::Entry* pos = ck.find("pos");
    if (!pos || pos->shape.size() != 2 || pos->shape[0] < 1) return fail(err, "tensor pos is missing or not a table");
    const int rows = (int)pos->shape[0];
    c.max_positions = rows;
    for (size_t i = 0; i < c.layers.size(); i++) {
        const std::string n = layer_name(i, "mix.right.w1");
        const Checkpoint::Entry* w1 = ck.find(n);
        if (!w1 || w1->shape.size() != 2 || w1->shape[0] < 1 || w1->shape[0] > 512) return fail(err, "tensor " + n + " is missing or not a matrix");
        c.layers[i].rank = (int)w1->shape[0];
    }
    auto have = [&](const std::string& name, int64_t r, int64_t k) {
        return ck.bf16(name, k ? std::vector<int64_t>{r, k} : std::vector<int64_t>{r}, err) != nullptr;
    };
    if (!have("embed", c.vocab, c.width) || !have("pos", c.max_positions, c.width) || !have("final.norm", c.width, 0) ||
        !have("head", c.vocab, c.width))
        return false;
    for (size_t i = 0; i < c.layers.size(); i++)
        for (const Piece& p : layer_tensors(c.layers[i], c.width))
            if (!have(layer_name(i, p.name), p.rows, p.cols)) return false;
    return true;
}

void load_checkpoint(const Checkpoint& ck, const Config& c, Model* m, Data* d)
{
    Parts p;
    p.table = [&](const std::string& name, int16_t*& dst, size_t n) { dst = upload<int16_t>(ck.data(*ck.find(name)), n); };
    p.vector = [&](const std::string& name, float*& dst, size_t n) {
        const std::string base = name.substr(0, name.find('.') + 1);
        std::vector<float> v;
        if (ends_with(name, "norm1") || ends_with(name, "norm2") || name == "final.norm") v = values(ck, name, 1.0f);   // stored around zero
        else if (ends_with(name, "mix.in.b")) {
            v.assign(n, 0.0f);
            const LayerConfig& k = d->layers[std::stoul(name.substr(1))].c;
            auto put = [&](const char* t, int off) {
                const std::vector<float> b = values(ck, base + t);
                std::copy(b.begin(), b.end(), v.begin() + off);
            };
            put("mix.left.q.b", k.q_off());
            put("mix.left.k.b", k.k_off());
            put("mix.left.v.b", k.v_off());
            put("mix.right.a.b", k.a_off());
        } else if (ends_with(name, "mix.head_bias")) v = values(ck, base + "mix.left.pb");
        else if (ends_with(name, "mix.w2t")) {
            const std::vector<float> w = values(ck, base + "mix.right.w2");
            const LayerConfig& k = d->layers[std::stoul(name.substr(1))].c;
            v.resize(n);
            for (int r = 0; r < k.rank; r++)
                for (int i = 0; i < k.del(); i++) v[(size_t)r * k.del() + i] = w[(size_t)i * k.rank + r];
        } else if (ends_with(name, "mix.w0")) v = values(ck, base + "mix.right.w0");
        else if (ends_with(name, "mix.norm")) v = values(ck, base + "mix.right.norm");
        else v = values(ck, name);
        dst = upload<float>(v.data(), n);
    };
    p.weight = [&](const std::string& name, CompressedWeight& w, int M, int K) {
        const std::string b = name.substr(0, name.find('.') + 1);
        if (ends_with(name, "mix.in"))
            part_store::pack(name, part_store::below(ck, {b + "mix.left.q", b + "mix.left.k", b + "mix.left.v", b + "mix.right.r", b + "mix.right.k",
                                                          b + "mix.right.v", b + "mix.right.a", b + "mix.right.g", b + "mix.right.w1"}), M, K, w);
        else if (ends_with(name, "mix.out")) part_store::pack(name, part_store::beside(ck, {b + "mix.left.o", b + "mix.right.o"}, M), M, K, w);
        else part_store::pack(name, part_store::below(ck, {name}), M, K, w);
    };
    walk(c, m, d, p);
}

// ---- the packed directory ----------------------------------------------------------------------------------------
bool check_packed(const std::string& dir, Config& c, std::string& err)
{
    const long long pos = file_size(part_store::table_file(dir, "pos"));
    if (pos <= 0 || pos % (2LL * c.width)) return fail(err, "neither model.safetensors nor a usable pos.bf16.bin in " + dir);
    c.max_positions = (int)(pos / (2LL * c.width));
    for (size_t i = 0; i < c.layers.size(); i++) {
        const long long b = file_size(part_store::vector_file(dir, layer_name(i, "mix.w2t"))), per = 4LL * c.layers[i].del();
        if (b <= 0 || b % per || b / per > 512) return fail(err, layer_name(i, "mix.w2t") + " is missing or has the wrong size");
        c.layers[i].rank = (int)(b / per);
    }
    Model m;
    Data d;
    empty_layers(c, d);
    return part_store::check_packed(dir, [&](const Parts& p) { walk(c, &m, &d, p); }, err);
}

// ---- family entries ------------------------------------------------------------------------------------------------
bool owns(const std::string& dir) { return part_store::has_architecture(dir, kArchitecture); }

bool read_config(const std::string& dir, Config& c, std::string& err)
{
    std::string text;
    if (!part_store::read_config_text(dir, text)) return fail(err, "no config.json in " + dir);
    try {
        parse_config(text, c);
    } catch (const JsonError& e) {
        return fail(err, dir + "/config.json: " + e.what());
    }
    return true;
}

bool check(const std::string& dir, std::string& err)
{
    Config c;
    if (!read_config(dir, c, err)) return false;
    if (!is_checkpoint(dir)) return check_packed(dir, c, err);
    Checkpoint ck;
    return open_checkpoint(dir, c, ck, err);
}

void release(Model* m)
{
    Data* d = data_of(m);
    part_store::release([&](const Parts& p) { walk(d->config, m, d, p); });
    delete d;
    delete m;
}

double softplus(double x) { return x > 30.0 ? x : log1p(exp(x)); }

// A model object with nothing on the device yet.
Model* new_model(const Config& c)
{
    Model* m = new Model();
    Data* d = new Data();
    m->family = &kGamilornFamily;
    m->family_data = d;
    d->config = c;
    empty_layers(c, *d);
    m->token_embd = nullptr;
    m->output_norm = nullptr;
    clear_weight(m->output_proj);
    m->kv_cache_k = m->kv_cache_v = nullptr;
    m->kv_scale_k = m->kv_scale_v = nullptr;
    ModelConfig& mc = m->config;
    mc = ModelConfig();
    mc.n_vocab = c.vocab;
    mc.n_embd = c.width;
    mc.n_layer = (int)c.layers.size();
    mc.n_head = c.layers[0].heads;
    mc.n_head_kv = c.layers[0].kv_heads;
    for (const LayerConfig& k : c.layers) mc.n_ff = std::max(mc.n_ff, k.ff);
    mc.n_ctx = c.max_positions;
    mc.rms_norm_eps = c.eps;
    const char* ctx = getenv("TURBO_CTX");
    m->max_seq_len = ctx && atoi(ctx) > 0 ? std::min(atoi(ctx), c.max_positions) : c.max_positions;
    return m;
}

// What is computed once from the loaded tensors.
void derive(Model* m)
{
    for (Layer& L : data_of(m)->layers) {
        if (!L.c.ff) continue;
        float pq[2] = {0.0f, 0.0f};
        if (!gpu_ok(hipMemcpy(pq, L.act, sizeof pq, hipMemcpyDeviceToHost), "activation constants")) engine_fail("reading mlp.act failed");
        L.xielu = {T12_ACT_XIELU, (float)softplus(pq[0]), (float)(0.5 + softplus(pq[1]))};
    }
}

Model* load(const std::string& dir)
{
    Config c;
    std::string err;
    Checkpoint ck;
    const bool raw = is_checkpoint(dir);
    if (!read_config(dir, c, err) || !(raw ? open_checkpoint(dir, c, ck, err) : check_packed(dir, c, err))) {
        fprintf(stderr, "%s\n", err.c_str());
        return nullptr;
    }
    printf("  Config: vocab=%d width=%d layers=%zu positions=%d\n", c.vocab, c.width, c.layers.size(), c.max_positions);
    Model* m = new_model(c);
    try {
        if (raw) load_checkpoint(ck, c, m, data_of(m));
        else if (!part_store::load_packed(dir, [&](const Parts& p) { walk(c, m, data_of(m), p); })) {
            release(m);
            return nullptr;
        }
        derive(m);
    } catch (...) {
        release(m);
        throw;
    }
    printf("  Context length: %d\n  Model loaded.\n", m->max_seq_len);
    return m;
}

bool save(const Model* cm, const std::string& dir)
{
    Model* m = const_cast<Model*>(cm);                     // the walk hands out references; nothing is changed
    Data* d = data_of(m);
    return part_store::save_packed(dir, d->config.text, [&](const Parts& p) { walk(d->config, m, d, p); });
}

}  // namespace
}  // namespace gamilorn

ModelFamily kGamilornFamily = {
    "gamilorn", gamilorn::owns, gamilorn::check, gamilorn::load, gamilorn::save, gamilorn::release, &kGamilornRun,
};

// Matrices and tables N(0, 0.02) with the outliers of create_synthetic_model; norms 1; a small head bias and decay bias so
// that the mixers neither saturate nor vanish.
Model* create_synthetic_gamilorn(const std::string& config_json, int rank, uint64_t seed, float p_outlier)
{
    using namespace gamilorn;
    Config c;
    try {
        parse_config(config_json, c);
    } catch (const JsonError& e) {
        fprintf(stderr, "ERROR: %s\n", e.what());
        return nullptr;
    }
    if (rank < 1 || rank > 512 || c.max_positions < 1) {
        fprintf(stderr, "ERROR: a synthetic model needs max_positions and a rank of 1..512\n");
        return nullptr;
    }
    for (LayerConfig& k : c.layers) k.rank = rank;
    Model* m = new_model(c);
    try {
        part_store::synthesize([&](const Parts& p) { walk(c, m, data_of(m), p); }, seed, p_outlier, [](const std::string& n) {
            if (n.find("head_bias") != std::string::npos) return -3.0f;
            if (n.find("w2t") != std::string::npos) return 0.01f;
            if (n.find("w0") != std::string::npos) return -2.0f;
            if (n.find("mlp.act") != std::string::npos) return 0.5f;
            return n.find("norm") != std::string::npos ? 1.0f : 0.0f;
        });
        derive(m);
    } catch (...) {
        release(m);
        throw;
    }
    return m;
}
