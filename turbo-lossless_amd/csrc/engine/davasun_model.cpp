// Configuration, loading and saving of Davasun models (davasun.h).  Directory forms: part_store.h.
#include "davasun.h"

#include <cmath>
#include <cstdio>
#include <cstdlib>

#include "family.h"
#include "json.h"
#include "part_store.h"

using namespace model_store;
using part_store::Parts;
using part_store::ends_with;
using part_store::is_checkpoint;
using part_store::layer_name;
using part_store::values;

namespace davasun {

Data* data_of(const Model* m) { return (Data*)m->family_data; }

std::vector<int> Config::runs() const
{
    std::vector<int> order;
    const int n = (int)layers.size();
    for (int i = 0; i < loop_start; i++) order.push_back(i);
    for (int t = 0; t < loop_times; t++)
        for (int i = loop_start; i < loop_stop; i++) order.push_back(i);
    for (int i = loop_stop; i < n; i++) order.push_back(i);
    return order;
}

namespace {

const char* const kArchitecture = "Davasun";
constexpr int kContext = 32768;          // positions of a state unless the caller or TURBO_CTX says; the design has no limit

// Everything config.json says.
void parse_config(const std::string& text, Config& c)
{
    const Json j = Json::parse(text);
    if (j.str("architecture") != kArchitecture) throw JsonError("the architecture is not Davasun");
    const int64_t top = 1 << 24;
    c.text = text;
    c.vocab = (int)j.integer("vocab", 1, top);
    c.width = (int)j.integer("width", 1, 1 << 20);
    c.eps = (float)j.at("norm").real("eps");
    c.logit_scale = (float)j.real("logit_scale");
    if (!(c.eps >= 0.0f)) throw JsonError("norm.eps is negative");
    c.layers.clear();
    const Json& ls = j.at("layers");
    if (ls.kind != Json::ARR || ls.items.empty()) throw JsonError("\"layers\" is not a list of layers");
    for (const Json& l : ls.items) {
        LayerConfig k = {};
        const Json& m = l.at("mixer");
        k.heads = (int)m.integer("heads", 1, 65536);
        k.vdim = (int)m.integer("vdim", 1, 65536);
        if (l.str("type") == "mlstm") {
            k.kind = MLSTM;
            k.dim = (int)m.integer("dim", 1, 512);
            k.gate_cap = (float)m.real("gate_cap");
            if (!(k.gate_cap > 0.0f)) throw JsonError("gate_cap is not positive");
        } else if (l.str("type") == "latent_attention") {
            k.kind = LATENT;
            k.dim = (int)m.integer("dim", 1, 8192);
            k.rank = (int)m.integer("kv_rank", 1, 8192);
            k.rot_dim = (int)m.integer("rot_dim", 2, 8192);
            k.rot_base = (float)m.at("rot").real("base");
            k.scale = (float)m.real("scale");
            if (k.rot_dim % 2) throw JsonError("rot_dim is odd");
            if (m.at("rot").has("dims") && m.at("rot").integer("dims", 2, 8192) != k.rot_dim) throw JsonError("rot.dims is not rot_dim");
            if (!(k.rot_base > 0.0f)) throw JsonError("rot.base is not positive");
        } else {
            throw JsonError("a layer has the unknown type \"" + l.str("type") + "\"");
        }
        if ((int64_t)k.heads * (2 * (int64_t)k.dim + 2 * (int64_t)k.vdim + 2 * (int64_t)k.rot_dim + 2) + k.rank > (1 << 26) ||
            (int64_t)k.heads * k.rank > (1 << 26))
            throw JsonError("heads times their sizes is too large");
        if (l.has("mlp") && !l.at("mlp").is_null()) {
            const Json& f = l.at("mlp");
            if (f.str("kind") != "dense") throw JsonError("a feed-forward has the unknown kind \"" + f.str("kind") + "\"");
            k.ff = (int)f.integer("ff", 1, top);
            k.limit = (float)f.real("limit");
            if (!(k.limit >= 0.0f)) throw JsonError("limit is negative");
        }
        c.layers.push_back(k);
    }
    c.loop_start = c.loop_stop = 0;
    c.loop_times = 1;
    if (j.has("loop") && !j.at("loop").is_null()) {
        const Json& o = j.at("loop");
        c.loop_start = (int)o.integer("start", 0, (int64_t)ls.items.size());
        c.loop_stop = (int)o.integer("stop", c.loop_start, (int64_t)ls.items.size());
        c.loop_times = (int)o.integer("times", 1, 4096);
    }
}

// ---- the parts a model is stored and held as
void walk(const Config& c, Model* m, Data* d, const Parts& p)
{
    p.table("embed", m->token_embd, (size_t)c.vocab * c.width);
    p.vector("embed.norm", d->embed_norm, c.width);
    for (size_t i = 0; i < d->layers.size(); i++) {
        Layer& L = d->layers[i];
        const LayerConfig& k = L.c;
        p.vector(layer_name(i, "norm1"), L.norm1, c.width);
        p.vector(layer_name(i, "norm1b"), L.norm1b, c.width);
        p.weight(layer_name(i, "mix.in"), L.w_in, k.in_rows(), c.width);
        p.weight(layer_name(i, "mix.out"), L.w_out, c.width, k.out_cols());
        if (k.kind == MLSTM) {
            p.vector(layer_name(i, "mix.in.b"), L.in_bias, k.in_ld());
            p.vector(layer_name(i, "mix.norm"), L.o_norm, k.out_cols());
        } else {
            p.vector(layer_name(i, "mix.c.norm"), L.o_norm, k.rank);
            p.weight(layer_name(i, "mix.k_up"), L.k_up, k.heads * k.rank, k.dim);
            p.weight(layer_name(i, "mix.v_up"), L.v_up, k.heads * k.vdim, k.rank);
            p.vector(layer_name(i, "mix.freqs"), L.freqs, k.rot_dim / 2);
        }
        if (!k.ff) continue;
        p.vector(layer_name(i, "norm2"), L.norm2, c.width);
        p.vector(layer_name(i, "norm2b"), L.norm2b, c.width);
        p.weight(layer_name(i, "mlp.gate"), L.gate, k.ff, c.width);
        p.weight(layer_name(i, "mlp.up"), L.up, k.ff, c.width);
        p.weight(layer_name(i, "mlp.down"), L.down, c.width, k.ff);
    }
    p.vector("final.norm", m->output_norm, c.width);                       // times the logit scale
    p.weight("head", m->output_proj, c.vocab, c.width);
}

void empty_layers(const Config& c, Data& d)
{
    d.layers.clear();
    for (const LayerConfig& k : c.layers) {
        Layer L;
        L.c = k;
        L.gain1 = L.gain1b = L.gain2 = L.gain2b = 1.0f;
        L.norm1 = L.norm1b = L.norm2 = L.norm2b = L.in_bias = L.o_norm = L.freqs = nullptr;
        for (CompressedWeight* w : {&L.w_in, &L.w_out, &L.k_up, &L.v_up, &L.gate, &L.up, &L.down}) clear_weight(*w);
        d.layers.push_back(L);
    }
}

std::vector<float> rotation_frequencies(const LayerConfig& k)
{
    std::vector<float> f(k.rot_dim / 2);
    for (size_t i = 0; i < f.size(); i++) f[i] = (float)pow((double)k.rot_base, -2.0 * (double)i / k.rot_dim);
    return f;
}

// ---- checkpoint ------------------------------------------------------------------------------------------------
struct Piece {
    const char* name;                    // below the layer
    std::vector<int64_t> shape;
};
std::vector<Piece> layer_tensors(const LayerConfig& k, int64_t width)
{
    const int64_t H = k.heads, hv = H * k.vdim;
    std::vector<Piece> t = {{"norm1", {}}, {"norm1b", {}}, {"mix.o", {width, hv}}};
    auto add = [&](std::initializer_list<Piece> more) { t.insert(t.end(), more); };
    if (k.kind == MLSTM)
        add({{"mix.q", {H * k.dim, width}}, {"mix.k", {H * k.dim, width}}, {"mix.v", {hv, width}}, {"mix.g", {hv, width}}, {"mix.norm", {hv}},
             {"mix.i", {H, width}}, {"mix.i.b", {H}}, {"mix.f", {H, width}}, {"mix.f.b", {H}}});
    else
        add({{"mix.q", {H * (k.dim + k.rot_dim), width}}, {"mix.dkv", {k.rank + k.rot_dim, width}}, {"mix.dkv.norm", {k.rank}},
             {"mix.uk", {H * k.dim, k.rank}}, {"mix.uv", {hv, k.rank}}, {"mix.g", {H, width}}});
    if (k.ff)
        add({{"norm2", {}}, {"norm2b", {}}, {"mlp.gate", {k.ff, width}}, {"mlp.up", {k.ff, width}}, {"mlp.down", {width, k.ff}}});
    return t;
}

// Opens the checkpoint and checks that every tensor is there with its shape.
bool open_checkpoint(const std::string& dir, const Config& c, Checkpoint& ck, std::string& err)
{
    if (!ck.open(dir + "/model.safetensors", err)) return false;
    if (!ck.bf16("embed", {c.vocab, c.width}, err) || !ck.bf16("embed.norm", {}, err) || !ck.bf16("final.norm", {}, err) ||
        !ck.bf16("head", {c.vocab, c.width}, err))
        return false;
    for (size_t i = 0; i < c.layers.size(); i++)
        for (const Piece& p : layer_tensors(c.layers[i], c.width))
            if (!ck.bf16(layer_name(i, p.name), p.shape, err)) return false;
    return true;
}

void load_checkpoint(const Checkpoint& ck, const Config& c, Model* m, Data* d)
{
    Parts p;
    auto layer = [&](const std::string& name) -> const LayerConfig& { return d->layers[std::stoul(name.substr(1))].c; };
    p.table = [&](const std::string& name, int16_t*& dst, size_t n) { dst = upload<int16_t>(ck.data(*ck.find(name)), n); };
    p.vector = [&](const std::string& name, float*& dst, size_t n) {
        const std::string base = name.substr(0, name.find('.') + 1);
        std::vector<float> v;
        if (ends_with(name, "mix.in.b")) {
            v.assign(n, 0.0f);
            const std::vector<float> i = values(ck, base + "mix.i.b"), f = values(ck, base + "mix.f.b");
            std::copy(i.begin(), i.end(), v.begin() + layer(name).i_off());
            std::copy(f.begin(), f.end(), v.begin() + layer(name).f_off());
        } else if (ends_with(name, "mix.norm")) v = values(ck, name);
        else if (ends_with(name, "mix.c.norm")) v = values(ck, base + "mix.dkv.norm");
        else if (ends_with(name, "mix.freqs")) v = rotation_frequencies(layer(name));
        else v.assign(n, values(ck, name)[0] * (name == "final.norm" ? c.logit_scale : 1.0f));      // one gain
        dst = upload<float>(v.data(), n);
    };
    p.weight = [&](const std::string& name, CompressedWeight& w, int M, int K) {
        const std::string b = name.substr(0, name.find('.') + 1) + "mix.";
        std::vector<uint8_t> bits;
        if (ends_with(name, "mix.in")) {
            bits = layer(name).kind == MLSTM ? part_store::below(ck, {b + "q", b + "k", b + "v", b + "g", b + "i", b + "f"})
                                             : part_store::below(ck, {b + "q", b + "dkv", b + "g"});
        } else if (ends_with(name, "mix.out")) bits = part_store::below(ck, {b + "o"});
        else if (ends_with(name, "mix.v_up")) bits = part_store::below(ck, {b + "uv"});
        else if (ends_with(name, "mix.k_up")) {
            const LayerConfig& k = layer(name);
            const uint8_t* from = ck.data(*ck.find(b + "uk"));             // [heads][dim][rank] -> [heads][rank][dim]
            bits.resize((size_t)M * K * 2);
            for (int h = 0; h < k.heads; h++)
                for (int e = 0; e < k.dim; e++)
                    for (int r = 0; r < k.rank; r++) {
                        const size_t src = ((size_t)h * k.dim + e) * k.rank + r, dst = ((size_t)h * k.rank + r) * k.dim + e;
                        bits[2 * dst] = from[2 * src];
                        bits[2 * dst + 1] = from[2 * src + 1];
                    }
        } else bits = part_store::below(ck, {name});
        part_store::pack(name, bits, M, K, w);
    };
    walk(c, m, d, p);
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

bool check_packed(const std::string& dir, const Config& c, std::string& err)
{
    if (file_size(part_store::table_file(dir, "embed")) < 0) return fail(err, "neither model.safetensors nor embed.bf16.bin in " + dir);
    Model m;
    Data d;
    empty_layers(c, d);
    return part_store::check_packed(dir, [&](const Parts& p) { walk(c, &m, &d, p); }, err);
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

// A model object with nothing on the device yet.
Model* new_model(const Config& c)
{
    Model* m = new Model();
    Data* d = new Data();
    m->family = &kDavasunFamily;
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
    mc.n_head = mc.n_head_kv = c.layers[0].heads;
    for (const LayerConfig& k : c.layers) mc.n_ff = std::max(mc.n_ff, k.ff);
    mc.rms_norm_eps = c.eps;
    const char* ctx = getenv("TURBO_CTX");
    mc.n_ctx = m->max_seq_len = ctx && atoi(ctx) > 0 ? atoi(ctx) : kContext;
    return m;
}

// What is read back once from the loaded tensors.
void derive(Model* m)
{
    auto first = [](const float* v) {
        float g = 1.0f;
        if (v && !gpu_ok(hipMemcpy(&g, v, sizeof g, hipMemcpyDeviceToHost), "norm gain")) engine_fail("reading a norm's gain failed");
        return g;
    };
    Data* d = data_of(m);
    d->final_gain = first(m->output_norm);
    for (Layer& L : d->layers) {
        L.gain1 = first(L.norm1);
        L.gain1b = first(L.norm1b);
        L.gain2 = first(L.norm2);
        L.gain2b = first(L.norm2b);
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
    printf("  Config: vocab=%d width=%d layers=%zu (%zu runs)\n", c.vocab, c.width, c.layers.size(), c.runs().size());
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
}  // namespace davasun

ModelFamily kDavasunFamily = {
    "davasun", davasun::owns, davasun::check, davasun::load, davasun::save, davasun::release, &kDavasunRun,
};

// Matrices and tables N(0, 0.02) with the outliers of create_synthetic_model; gains 1; forget gates open, input gates low.
Model* create_synthetic_davasun(const std::string& config_json, uint64_t seed, float p_outlier)
{
    using namespace davasun;
    Config c;
    try {
        parse_config(config_json, c);
    } catch (const JsonError& e) {
        fprintf(stderr, "ERROR: %s\n", e.what());
        return nullptr;
    }
    Model* m = new_model(c);
    try {
        part_store::synthesize([&](const Parts& p) { walk(c, m, data_of(m), p); }, seed, p_outlier,
                               [](const std::string& n) { return n.find("norm") != std::string::npos ? 1.0f : 0.0f; });
        for (Layer& L : data_of(m)->layers) {
            std::vector<float> v;
            float* dst = L.freqs;
            if (L.c.kind == LATENT) v = rotation_frequencies(L.c);
            else {
                dst = L.in_bias;
                v.assign(L.c.in_ld(), 0.0f);
                for (int h = 0; h < L.c.heads; h++) {
                    v[L.c.i_off() + h] = -3.0f;
                    v[L.c.f_off() + h] = 4.0f;
                }
            }
            if (!gpu_ok(hipMemcpy(dst, v.data(), v.size() * sizeof(float), hipMemcpyHostToDevice), "synthetic constants"))
                engine_fail("synthetic constants failed");
        }
        derive(m);
    } catch (...) {
        release(m);
        throw;
    }
    return m;
}
