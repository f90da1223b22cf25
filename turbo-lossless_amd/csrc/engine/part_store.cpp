// Models as lists of named parts (part_store.h).
#include "part_store.h"

#include <cstring>

#include "json.h"
#include "t12_abi.h"

extern "C" int t12_synth_normal_bf16(void*, size_t, uint64_t, float, float, float, void*);
extern "C" int t12_fill_f32(void*, size_t, float, void*);

using namespace model_store;

namespace part_store {

std::string layer_name(size_t i, const char* what) { return "l" + std::to_string(i) + "." + what; }

bool ends_with(const std::string& s, const char* end)
{
    const size_t n = strlen(end);
    return s.size() >= n && s.compare(s.size() - n, n, end) == 0;
}

// ---- directories -------------------------------------------------------------------------------------------------
bool read_config_text(const std::string& dir, std::string& text)
{
    std::vector<uint8_t> b;
    if (!read_file(dir + "/config.json", b, true)) return false;
    text.assign((const char*)b.data(), b.size());
    return true;
}

bool has_architecture(const std::string& dir, const char* name)
{
    std::string text;
    if (!read_config_text(dir, text)) return false;
    try {
        const Json j = Json::parse(text);
        return j.has("architecture") && j.at("architecture").kind == Json::STR && j.at("architecture").text == name;
    } catch (const JsonError&) {
        return false;
    }
}

bool is_checkpoint(const std::string& dir) { return file_size(dir + "/model.safetensors") >= 0; }
std::string vector_file(const std::string& dir, const std::string& n) { return dir + "/" + n + ".f32.bin"; }
std::string table_file(const std::string& dir, const std::string& n) { return dir + "/" + n + ".bf16.bin"; }

// ---- the packed form ---------------------------------------------------------------------------------------------
bool check_packed(const std::string& dir, const Walk& walk, std::string& err)
{
    bool ok = true;
    Parts p;
    p.weight = [&](const std::string& n, CompressedWeight&, int M, int K) { ok = ok && check_tensor(dir, n, M, K, err); };
    p.vector = [&](const std::string& n, float*&, size_t k) {
        if (ok && file_size(vector_file(dir, n)) != (long long)k * 4) ok = fail(err, n + ".f32.bin missing or not the right size");
    };
    p.table = [&](const std::string& n, int16_t*&, size_t k) {
        if (ok && file_size(table_file(dir, n)) != (long long)k * 2) ok = fail(err, n + ".bf16.bin missing or not the right size");
    };
    walk(p);
    return ok;
}

bool load_packed(const std::string& dir, const Walk& walk)
{
    bool ok = true;
    Parts p;
    p.weight = [&](const std::string& n, CompressedWeight& w, int, int) { ok = ok && load_compressed(dir, n, w); };
    auto bytes = [&](const std::string& path, size_t want) {
        std::vector<uint8_t> b;
        if (!read_file(path, b) || b.size() != want) ok = false;
        return b;
    };
    p.vector = [&](const std::string& n, float*& v, size_t k) {
        const std::vector<uint8_t> b = bytes(vector_file(dir, n), k * 4);
        if (ok) v = upload<float>(b.data(), k);
    };
    p.table = [&](const std::string& n, int16_t*& v, size_t k) {
        const std::vector<uint8_t> b = bytes(table_file(dir, n), k * 2);
        if (ok) v = upload<int16_t>(b.data(), k);
    };
    walk(p);
    return ok;
}

bool save_packed(const std::string& dir, const std::string& config_text, const Walk& walk)
{
    {
        std::ofstream f(dir + "/config.json", std::ios::binary);
        f.write(config_text.data(), (std::streamsize)config_text.size());
        if (!f) {
            fprintf(stderr, "Cannot write: %s/config.json (the directory must exist)\n", dir.c_str());
            return false;
        }
    }
    bool ok = true;
    Parts p;
    p.weight = [&](const std::string& n, CompressedWeight& w, int, int) { ok = ok && save_weight(dir, n, w); };
    p.vector = [&](const std::string& n, float*& v, size_t k) { ok = ok && dump<float>(vector_file(dir, n), v, k); };
    p.table = [&](const std::string& n, int16_t*& v, size_t k) { ok = ok && dump<int16_t>(table_file(dir, n), v, k); };
    walk(p);
    return ok;
}

// ---- checkpoints -------------------------------------------------------------------------------------------------
float bf16_value(const uint8_t* p)
{
    uint16_t b;
    memcpy(&b, p, 2);
    const uint32_t u = (uint32_t)b << 16;
    float f;
    memcpy(&f, &u, 4);
    return f;
}

std::vector<float> values(const Checkpoint& ck, const std::string& name, float add)
{
    const Checkpoint::Entry& e = *ck.find(name);
    std::vector<float> v((size_t)e.count());
    const uint8_t* b = ck.data(e);
    for (size_t i = 0; i < v.size(); i++) v[i] = bf16_value(b + 2 * i) + add;
    return v;
}

std::vector<uint8_t> below(const Checkpoint& ck, const std::vector<std::string>& names)
{
    std::vector<uint8_t> out;
    for (const std::string& n : names) {
        const Checkpoint::Entry& e = *ck.find(n);
        out.insert(out.end(), ck.data(e), ck.data(e) + (size_t)e.count() * 2);
    }
    return out;
}

std::vector<uint8_t> beside(const Checkpoint& ck, const std::vector<std::string>& names, int M)
{
    std::vector<uint8_t> out;
    for (int r = 0; r < M; r++)
        for (const std::string& n : names) {
            const Checkpoint::Entry& e = *ck.find(n);
            const size_t row = (size_t)e.count() / M * 2;
            const uint8_t* b = ck.data(e) + row * r;
            out.insert(out.end(), b, b + row);
        }
    return out;
}

void pack(const std::string& name, const std::vector<uint8_t>& bits, int M, int K, CompressedWeight& w)
{
    uint16_t* dev = upload<uint16_t>(bits.data(), (size_t)M * K);
    const bool ok = pack_on_gpu(dev, M, K, w);
    (void)hipFree(dev);
    if (!ok) engine_fail("packing %s (%d x %d) failed: %s", name.c_str(), M, K, t12_last_error());
}

// ---- on the device -----------------------------------------------------------------------------------------------
void release(const Walk& walk)
{
    Parts p;
    p.weight = [](const std::string&, CompressedWeight& w, int, int) { free_weight(w); };
    p.vector = [](const std::string&, float*& v, size_t) { if (v) (void)hipFree(v); v = nullptr; };
    p.table = [](const std::string&, int16_t*& v, size_t) { if (v) (void)hipFree(v); v = nullptr; };
    walk(p);
}

void synthesize(const Walk& walk, uint64_t seed, float p_outlier, const std::function<float(const std::string&)>& fill)
{
    uint64_t s = seed;
    Parts p;
    p.weight = [&](const std::string& n, CompressedWeight& w, int M, int K) {
        uint16_t* stage = device_alloc<uint16_t>((size_t)M * K);
        const bool ok = t12_synth_normal_bf16(stage, (size_t)M * K, ++s, 0.02f, p_outlier, 8.0f, nullptr) == T12_OK && pack_on_gpu(stage, M, K, w);
        (void)hipFree(stage);
        if (!ok) engine_fail("synthetic tensor %s failed", n.c_str());
    };
    p.vector = [&](const std::string& n, float*& v, size_t k) {
        v = device_alloc<float>(k);
        if (t12_fill_f32(v, k, fill(n), nullptr) != T12_OK) engine_fail("synthetic vector %s failed", n.c_str());
    };
    p.table = [&](const std::string& n, int16_t*& v, size_t k) {
        v = device_alloc<int16_t>(k);
        if (t12_synth_normal_bf16(v, k, ++s, 0.02f, 0.0f, 0.0f, nullptr) != T12_OK) engine_fail("synthetic table %s failed", n.c_str());
    };
    walk(p);
    if (!gpu_ok(hipDeviceSynchronize(), "synthetic model")) engine_fail("synthetic model failed");
}

}  // namespace part_store
