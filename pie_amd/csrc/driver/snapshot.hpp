// Hugging Face snapshot reader: `config.json` -> ModelConfig, `*.safetensors` -> named tensors
// (memory-mapped, zero copies on the host).  Pure host C++.
//
// Takes the place of the reference's loaders for this path: the portable driver's safetensors
// archive + HF config reader (driver/portable/src/safetensors.cpp, driver/portable/src/
// hf_config.cpp; tensor names bound in driver/portable/src/model.cpp:1476-1479 via
// build_dense_) and the storage-program loader of the CUDA driver (driver/weight_loader).
// File format: 8-byte little-endian header length, a JSON header
// {name: {dtype, shape, data_offsets: [begin, end]}, "__metadata__": {...}}, then the data.
#pragma once

#include <dirent.h>
#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <algorithm>
#include <cstdint>
#include <cstring>
#include <fstream>
#include <map>
#include <memory>
#include <sstream>
#include <stdexcept>
#include <string>
#include <vector>

#include "config.hpp"

namespace pie_hip_driver {

// ---- a small JSON reader (objects, arrays, strings, numbers, true / false / null) ------------
struct Json {
    enum Kind { Null, Bool, Number, String, Array, Object } kind = Null;
    bool b = false;
    double num = 0.0;
    std::string str;
    std::vector<Json> arr;
    std::vector<std::pair<std::string, Json>> obj;

    const Json* get(const std::string& key) const {
        if (kind != Object) return nullptr;
        for (const auto& kv : obj)
            if (kv.first == key) return &kv.second;
        return nullptr;
    }
    double number_or(const std::string& key, double dflt) const {
        const Json* j = get(key);
        return j && j->kind == Number ? j->num : dflt;
    }
    std::string string_or(const std::string& key, const std::string& dflt) const {
        const Json* j = get(key);
        return j && j->kind == String ? j->str : dflt;
    }
    bool bool_or(const std::string& key, bool dflt) const {
        const Json* j = get(key);
        return j && j->kind == Bool ? j->b : dflt;
    }
};

class JsonParser {
  public:
    JsonParser(const char* p, size_t n) : p_(p), end_(p + n) {}
    Json parse() {
        Json v = value();
        ws();
        if (p_ != end_) fail("trailing characters");
        return v;
    }

  private:
    [[noreturn]] void fail(const char* what) const { throw std::runtime_error(std::string("json: ") + what); }
    void ws() {
        while (p_ < end_ && (*p_ == ' ' || *p_ == '\t' || *p_ == '\n' || *p_ == '\r')) ++p_;
    }
    bool eat(char c) {
        ws();
        if (p_ < end_ && *p_ == c) {
            ++p_;
            return true;
        }
        return false;
    }
    Json value() {
        ws();
        if (p_ >= end_) fail("unexpected end");
        Json v;
        const char c = *p_;
        if (c == '{') {
            ++p_;
            v.kind = Json::Object;
            if (eat('}')) return v;
            do {
                ws();
                std::string key = string();
                if (!eat(':')) fail("expected ':'");
                v.obj.emplace_back(std::move(key), value());
            } while (eat(','));
            if (!eat('}')) fail("expected '}'");
        } else if (c == '[') {
            ++p_;
            v.kind = Json::Array;
            if (eat(']')) return v;
            do v.arr.push_back(value());
            while (eat(','));
            if (!eat(']')) fail("expected ']'");
        } else if (c == '"') {
            v.kind = Json::String;
            v.str = string();
        } else if (literal("true")) {
            v.kind = Json::Bool;
            v.b = true;
        } else if (literal("false")) {
            v.kind = Json::Bool;
        } else if (literal("null")) {
        } else {
            char* e = nullptr;
            const std::string tmp(p_, std::min<size_t>(end_ - p_, 64));
            v.num = std::strtod(tmp.c_str(), &e);
            if (e == tmp.c_str()) fail("bad value");
            p_ += e - tmp.c_str();
            v.kind = Json::Number;
        }
        return v;
    }
    bool literal(const char* s) {
        const size_t n = std::strlen(s);
        if (static_cast<size_t>(end_ - p_) >= n && std::memcmp(p_, s, n) == 0) {
            p_ += n;
            return true;
        }
        return false;
    }
    std::string string() {
        if (p_ >= end_ || *p_ != '"') fail("expected string");
        ++p_;
        std::string out;
        while (p_ < end_ && *p_ != '"') {
            if (*p_ == '\\') {
                if (++p_ >= end_) fail("bad escape");
                switch (*p_) {
                    case 'n': out.push_back('\n'); break;
                    case 't': out.push_back('\t'); break;
                    case 'r': out.push_back('\r'); break;
                    case 'b': out.push_back('\b'); break;
                    case 'f': out.push_back('\f'); break;
                    case 'u':   // names here are ASCII; keep the low byte of the code unit
                        if (end_ - p_ < 5) fail("bad \\u escape");
                        out.push_back(static_cast<char>(std::strtol(std::string(p_ + 1, 4).c_str(), nullptr, 16)));
                        p_ += 4;
                        break;
                    default: out.push_back(*p_); break;
                }
                ++p_;
            } else {
                out.push_back(*p_++);
            }
        }
        if (p_ >= end_) fail("unterminated string");
        ++p_;
        return out;
    }
    const char* p_;
    const char* end_;
};

inline Json parse_json_file(const std::string& path) {
    std::ifstream f(path, std::ios::binary);
    if (!f) throw std::runtime_error("snapshot: cannot open '" + path + "'");
    std::stringstream ss;
    ss << f.rdbuf();
    const std::string text = ss.str();
    return JsonParser(text.data(), text.size()).parse();
}

// ---- safetensors --------------------------------------------------------------------------
// Bytes per element of a safetensors dtype name (0: not a dtype of that format).
inline size_t st_dtype_size(const std::string& dt) {
    if (dt == "F64" || dt == "I64" || dt == "U64") return 8;
    if (dt == "F32" || dt == "I32" || dt == "U32") return 4;
    if (dt == "BF16" || dt == "F16" || dt == "I16" || dt == "U16") return 2;
    if (dt == "I8" || dt == "U8" || dt == "BOOL" || dt == "F8_E4M3" || dt == "F8_E5M2") return 1;
    return 0;
}

struct StTensor {
    std::string dtype;            // "BF16", "F16", "F32", "I32", "U8", "I8", "F8_E4M3", ...
    std::vector<int64_t> shape;
    const uint8_t* data = nullptr;
    size_t bytes = 0;
    int64_t elems() const {
        int64_t n = 1;
        for (int64_t s : shape) n *= s;
        return n;
    }
};

class Snapshot {
  public:
    explicit Snapshot(const std::string& dir) : dir_(dir) {
        std::vector<std::string> files;
        if (DIR* d = opendir(dir.c_str())) {
            while (const dirent* e = readdir(d)) {
                const std::string n = e->d_name;
                if (n.size() > 12 && n.compare(n.size() - 12, 12, ".safetensors") == 0) files.push_back(n);
            }
            closedir(d);
        } else {
            throw std::runtime_error("snapshot: cannot list '" + dir + "'");
        }
        std::sort(files.begin(), files.end());
        if (files.empty()) throw std::runtime_error("snapshot: no .safetensors file in '" + dir + "'");
        for (const std::string& f : files) map_file(dir + "/" + f);
    }
    ~Snapshot() {
        for (const auto& m : maps_) munmap(m.first, m.second);
    }
    Snapshot(const Snapshot&) = delete;
    Snapshot& operator=(const Snapshot&) = delete;

    const StTensor* find(const std::string& name) const {
        const auto it = tensors_.find(name);
        return it == tensors_.end() ? nullptr : &it->second;
    }
    const StTensor& at(const std::string& name) const {
        const StTensor* t = find(name);
        if (!t) throw std::runtime_error("snapshot: tensor '" + name + "' not found in " + dir_);
        return *t;
    }
    const std::map<std::string, StTensor>& tensors() const { return tensors_; }

  private:
    void map_file(const std::string& path) {
        const int fd = open(path.c_str(), O_RDONLY);
        if (fd < 0) throw std::runtime_error("snapshot: cannot open '" + path + "'");
        struct stat st {};
        if (fstat(fd, &st) != 0 || st.st_size < 8) {
            close(fd);
            throw std::runtime_error("snapshot: '" + path + "' is too short");
        }
        void* base = mmap(nullptr, static_cast<size_t>(st.st_size), PROT_READ, MAP_PRIVATE, fd, 0);
        close(fd);
        if (base == MAP_FAILED) throw std::runtime_error("snapshot: mmap failed for '" + path + "'");
        maps_.emplace_back(base, static_cast<size_t>(st.st_size));
        const auto* bytes = static_cast<const uint8_t*>(base);
        uint64_t hlen = 0;
        std::memcpy(&hlen, bytes, 8);
        if (hlen > static_cast<uint64_t>(st.st_size) - 8 || hlen > (128ull << 20))
            throw std::runtime_error("snapshot: bad header length in '" + path + "'");
        const Json header = JsonParser(reinterpret_cast<const char*>(bytes + 8), hlen).parse();
        if (header.kind != Json::Object) throw std::runtime_error("snapshot: header of '" + path + "' is not an object");
        const uint8_t* data0 = bytes + 8 + hlen;
        const uint64_t data_bytes = static_cast<uint64_t>(st.st_size) - 8 - hlen;
        for (const auto& kv : header.obj) {
            if (kv.first == "__metadata__") continue;
            const Json* dt = kv.second.get("dtype");
            const Json* sh = kv.second.get("shape");
            const Json* off = kv.second.get("data_offsets");
            if (!dt || !sh || !off || off->arr.size() != 2)
                throw std::runtime_error("snapshot: malformed entry '" + kv.first + "'");
            // Nothing in the header is trusted: kinds, dtype names, dimensions (whole, >= 0, no
            // overflow of the element count), offsets inside the file, and a byte count that is
            // exactly elements * element size — later copies size themselves from these.
            if (dt->kind != Json::String || sh->kind != Json::Array || off->kind != Json::Array ||
                off->arr[0].kind != Json::Number || off->arr[1].kind != Json::Number)
                throw std::runtime_error("snapshot: malformed entry '" + kv.first + "'");
            StTensor t;
            t.dtype = dt->str;
            const size_t esize = st_dtype_size(t.dtype);
            if (esize == 0) throw std::runtime_error("snapshot: unknown dtype '" + t.dtype + "' in '" + kv.first + "'");
            uint64_t elems = 1;
            for (const Json& s : sh->arr) {
                if (s.kind != Json::Number || !(s.num >= 0.0) || s.num > 9.0e15 ||
                    s.num != static_cast<double>(static_cast<int64_t>(s.num)))
                    throw std::runtime_error("snapshot: bad dimension in '" + kv.first + "'");
                const uint64_t dim = static_cast<uint64_t>(s.num);
                if (dim != 0 && elems > (uint64_t(1) << 62) / dim)
                    throw std::runtime_error("snapshot: element count of '" + kv.first + "' overflows");
                elems *= dim;
                t.shape.push_back(static_cast<int64_t>(dim));
            }
            auto whole = [](double v) { return v >= 0.0 && v <= 9.0e15 && v == static_cast<double>(static_cast<uint64_t>(v)); };
            if (!whole(off->arr[0].num) || !whole(off->arr[1].num))
                throw std::runtime_error("snapshot: offsets of '" + kv.first + "' out of range");
            const uint64_t b = static_cast<uint64_t>(off->arr[0].num), e = static_cast<uint64_t>(off->arr[1].num);
            if (b > e || e > data_bytes) throw std::runtime_error("snapshot: offsets of '" + kv.first + "' out of range");
            if (e - b != elems * esize)
                throw std::runtime_error("snapshot: '" + kv.first + "' holds " + std::to_string(e - b) +
                                         " bytes, its shape and dtype need " + std::to_string(elems * esize));
            t.data = data0 + b;
            t.bytes = e - b;
            tensors_[kv.first] = std::move(t);
        }
    }
    std::string dir_;
    std::vector<std::pair<void*, size_t>> maps_;
    std::map<std::string, StTensor> tensors_;
};

// ---- checkpoint tensors as weights -----------------------------------------------------------
// Widens / narrows a checkpoint tensor to bf16 bits on the host when it is not bf16 already.
inline const uint16_t* as_bf16(const StTensor& t, std::vector<uint16_t>& staging) {
    const size_t n = static_cast<size_t>(t.elems());
    if (t.dtype == "BF16") {
        if (t.bytes != n * 2) throw std::runtime_error("snapshot: BF16 tensor with a wrong byte count");
        return reinterpret_cast<const uint16_t*>(t.data);
    }
    staging.resize(n);
    auto rne = [](float f) {
        uint32_t u;
        std::memcpy(&u, &f, 4);
        if ((u & 0x7FFFFFFFu) > 0x7F800000u) return static_cast<uint16_t>((u >> 16) | 0x40u);
        return static_cast<uint16_t>((u + 0x7FFFu + ((u >> 16) & 1u)) >> 16);
    };
    if (t.dtype == "F32") {
        if (t.bytes != n * 4) throw std::runtime_error("snapshot: F32 tensor with a wrong byte count");
        for (size_t i = 0; i < n; ++i) {
            float f;
            std::memcpy(&f, t.data + 4 * i, 4);
            staging[i] = rne(f);
        }
    } else if (t.dtype == "F16") {
        if (t.bytes != n * 2) throw std::runtime_error("snapshot: F16 tensor with a wrong byte count");
        for (size_t i = 0; i < n; ++i) {
            uint16_t h;
            std::memcpy(&h, t.data + 2 * i, 2);
            const uint32_t sign = (h & 0x8000u) << 16, exp = (h >> 10) & 0x1Fu, man = h & 0x3FFu;
            uint32_t u;
            if (exp == 0) {
                if (man == 0) u = sign;
                else {   // subnormal half: normalise
                    int e = -1;
                    uint32_t m2 = man;
                    do { ++e; m2 <<= 1; } while (!(m2 & 0x400u));
                    u = sign | ((127 - 15 - e) << 23) | ((m2 & 0x3FFu) << 13);
                }
            } else if (exp == 31) u = sign | 0x7F800000u | (man << 13);
            else u = sign | ((exp + 112) << 23) | (man << 13);
            float f;
            std::memcpy(&f, &u, 4);
            staging[i] = rne(f);
        }
    } else {
        throw std::runtime_error("snapshot: dtype " + t.dtype + " is not a floating weight");
    }
    return staging.data();
}

inline void expect_shape(const StTensor& t, const std::string& name, int64_t rows, int64_t cols) {
    const bool ok = cols < 0 ? (t.shape.size() == 1 && t.shape[0] == rows)
                             : (t.shape.size() == 2 && t.shape[0] == rows && t.shape[1] == cols);
    if (!ok) throw std::runtime_error("snapshot: tensor '" + name + "' has an unexpected shape");
}

// ---- config.json -> ModelConfig: layer stacks ---------------------------------------------------
inline int json_size(const Json& j, const std::string& key, const std::string& at) {
    const Json* v = j.get(key);
    if (!v || v->kind != Json::Number || v->num != static_cast<double>(static_cast<int>(v->num)))
        throw std::runtime_error("snapshot: " + at + " needs an integer '" + key + "'");
    return static_cast<int>(v->num);
}
inline std::uint64_t json_count(const Json& j, const std::string& key, const std::string& at) {
    const Json* v = j.get(key);
    if (!v || v->kind != Json::Number || !(v->num >= 0.0) || v->num > 9.0e15 || v->num != static_cast<double>(static_cast<std::uint64_t>(v->num)))
        throw std::runtime_error("snapshot: " + at + " needs a whole number '" + key + "' that is not negative");
    return static_cast<std::uint64_t>(v->num);
}
inline double json_number(const Json& j, const std::string& key, const std::string& at) {
    const Json* v = j.get(key);
    if (!v || v->kind != Json::Number) throw std::runtime_error("snapshot: " + at + " needs a number '" + key + "'");
    return v->num;
}

inline RotarySpec parse_rotary(const Json& j, const std::string& at) {
    RotarySpec r;
    r.dims = json_size(j, "dims", at);
    r.base = json_number(j, "base", at);
    if (const Json* s = j.get("scaling"); s && s->kind == Json::Object) {
        r.yarn = true;
        r.factor = json_number(*s, "factor", at);
        r.original = json_number(*s, "original", at);
        r.fast = json_number(*s, "fast", at);
        r.slow = json_number(*s, "slow", at);
    }
    return r;
}

// A mixer's sub-object (or the error that it is missing).
inline const Json& json_object(const Json& j, const std::string& key, const std::string& at) {
    const Json* v = j.get(key);
    if (!v || v->kind != Json::Object) throw std::runtime_error("snapshot: " + at + " needs '" + key + "'");
    return *v;
}

inline GroupAttentionSpec parse_group_attention(const Json& j, const std::string& at) {
    GroupAttentionSpec a;
    a.heads = json_size(j, "heads", at);
    a.kv_heads = json_size(j, "kv_heads", at);
    a.dim = json_size(j, "dim", at);
    a.vdim = json_size(j, "vdim", at);
    a.scale = json_number(j, "scale", at);
    a.sink = 1.f;   // a sink of score 0
    if (const Json* m = j.get("mask"); m && m->kind == Json::Object) {
        a.window = json_size(*m, "size", at + " mask");
        if (a.window <= 0) throw std::runtime_error("snapshot: " + at + ": mask.size must be positive");
    }
    if (const Json* r = j.get("rot"); r && r->kind == Json::Object) a.rot = parse_rotary(*r, at + " rot");
    return a;
}

// Attention as a mixer of its own: interleaved rotation, no biases, no sink.
inline void read_attention(LayerSpec& l, const Json& j, const std::string& at, QueryKeyNorm norm, bool own_values, bool gate) {
    l.mixer = MixerKind::Attention;
    l.attn = parse_group_attention(j, at);
    l.attn.sink = 0.f;
    l.attn.half_split = l.attn.biases = false;
    l.attn.norm = norm;
    l.attn.own_values = own_values;
    l.attn.gate = gate;
}

inline DecayMemorySpec parse_retention(const Json& j, const std::string& at) {
    DecayMemorySpec d;
    d.kind = DecayKind::Retention;
    d.heads = d.kv_heads = json_size(j, "heads", at);
    d.dim = json_size(j, "dim", at);
    d.vdim = json_size(j, "vdim", at);
    const Json* list = j.get("decay");
    if (!list || list->kind != Json::Array) throw std::runtime_error("snapshot: " + at + " needs a list 'decay'");
    for (const Json& v : list->arr) {
        if (v.kind != Json::Number) throw std::runtime_error("snapshot: " + at + ": decay must hold numbers");
        d.decay.push_back(v.num);
    }
    return d;
}

inline MixtureSpec parse_mixture(const Json& j, const std::string& at, RouterKind kind, ExpertKind form) {
    MixtureSpec e;
    e.router = kind;
    e.expert = form;
    const Json &expert = json_object(j, "expert", at), &router = json_object(j, "router", at);
    e.ff = json_size(expert, "ff", at + " expert");
    if (kind == RouterKind::CorrectedScores) {
        e.experts = json_size(router, "experts", at + " router");
        e.top = json_size(router, "top", at + " router");
        if (const Json* shared = j.get("shared"); shared && shared->kind == Json::Object) {
            e.shared_ff = json_size(*shared, "ff", at + " shared");
            if (e.shared_ff <= 0) throw std::runtime_error("snapshot: " + at + ": shared.ff must be positive");
        }
        if (e.experts <= 0) throw std::runtime_error("snapshot: " + at + ": router.experts must be positive");
        return e;
    }
    e.limit = static_cast<float>(json_number(expert, "limit", at + " expert"));
    e.alpha = 1.702f;
    e.shift = 1.f;
    e.experts = json_size(router, "experts", at + " router");
    e.top = json_size(router, "top", at + " router");
    e.scale = static_cast<float>(router.number_or("scale", 1.0));
    if (const Json* g = router.get("groups"); g && g->kind == Json::Object) {
        e.groups = json_size(*g, "count", at + " groups");
        e.keep = json_size(*g, "keep", at + " groups");
    }
    if (e.experts <= 0) throw std::runtime_error("snapshot: " + at + ": router.experts must be positive");
    return e;
}

// One entry per mixer kind: config name -> reader of its sizes.
struct MixerReader {
    const char* type;
    void (*read)(LayerSpec& l, const Json& mixer, const std::string& at);
};
inline const std::vector<MixerReader>& mixer_registry() {
    static const std::vector<MixerReader> table = {
        {"latent_attention",
         [](LayerSpec& l, const Json& j, const std::string& at) {
             l.mixer = MixerKind::LatentAttention;
             auto& a = l.latent;
             a.heads = json_size(j, "heads", at);
             a.dim = json_size(j, "dim", at);
             if (j.get("rot_dim")) a.rot_dim = json_size(j, "rot_dim", at);   // (left out: no rotated part)
             a.vdim = json_size(j, "vdim", at);
             a.q_rank = json_size(j, "q_rank", at);
             a.kv_rank = json_size(j, "kv_rank", at);
             a.scale = json_number(j, "scale", at);
             const Json* rot = j.get("rot");
             if (rot && rot->kind == Json::Object) a.rot = parse_rotary(*rot, at + " rot");
             if (const Json* from = j.get("kv_from"); from && from->kind == Json::Number) {
                 a.kv_from = json_size(j, "kv_from", at);
                 if (a.kv_from < 0) throw std::runtime_error("snapshot: " + at + ": kv_from must not be negative");
             }
         }},
        {"attention",
         [](LayerSpec& l, const Json& j, const std::string& at) {
             read_attention(l, j, at, QueryKeyNorm::WholeProjection, true, false);
         }},
        {"attention_2",
         [](LayerSpec& l, const Json& j, const std::string& at) { read_attention(l, j, at, QueryKeyNorm::None, false, true); }},
        {"channel_delta",
         [](LayerSpec& l, const Json& j, const std::string& at) {
             l.mixer = MixerKind::ChannelDelta;
             auto& d = l.delta;
             d.heads = json_size(j, "heads", at);
             d.kv_heads = json_size(j, "kv_heads", at);
             d.dim = json_size(j, "dim", at);
             d.vdim = json_size(j, "vdim", at);
             d.taps = json_size(j, "conv", at);
         }},
        {"parallel",
         [](LayerSpec& l, const Json& j, const std::string& at) {
             l.mixer = MixerKind::Parallel;
             l.attn = parse_group_attention(json_object(j, "left", at), at + " left");
             l.memory = parse_retention(json_object(j, "right", at), at + " right");
             l.attention_scale = static_cast<float>(json_number(j, "left_scale", at));
             l.memory_scale = static_cast<float>(json_number(j, "right_scale", at));
         }},
        {"mlstm",
         [](LayerSpec& l, const Json& j, const std::string& at) {
             l.mixer = MixerKind::DecayMemory;
             auto& d = l.memory;
             d.kind = DecayKind::MatrixLstm;
             d.heads = d.kv_heads = json_size(j, "heads", at);
             d.dim = json_size(j, "dim", at);
             d.vdim = json_size(j, "vdim", at);
             d.gate_cap = json_number(j, "gate_cap", at);
         }},
        {"mamba2",
         [](LayerSpec& l, const Json& j, const std::string& at) {
             l.mixer = MixerKind::DecayMemory;
             auto& d = l.memory;
             d.kind = DecayKind::StateSpace;
             d.heads = json_size(j, "heads", at);
             d.kv_heads = json_size(j, "groups", at);
             d.dim = json_size(j, "state", at);
             d.vdim = json_size(j, "vdim", at);
             d.taps = json_size(j, "conv", at);
             d.norm_parts = json_size(j, "norm_groups", at);
         }},
    };
    return table;
}

// What sets one layer-stack architecture apart from another besides the mixers its layers name.
struct StackArchitecture {
    const char* name;   // config.json's "architecture"
    const char* arch;
    bool sandwich_norms;
    FeedForwardAct ff_act;
    bool shared_norm = false;
    bool half_split_latents = false;   // rotation of latent attention
    OutputGate latent_gate = OutputGate::None;
    bool latent_sinks = false;
    bool ff_biases = false;
    bool gated_sublayers = false;
    RouterKind router = RouterKind::GroupSoftmax;
    ExpertKind expert = ExpertKind::ClampedPair;
};
inline const std::vector<StackArchitecture>& stack_registry() {
    static const std::vector<StackArchitecture> table = {
        {"Varasun", "varasun", false, FeedForwardAct::SquaredRelu},
        {"Lofudra", "lofudra", true, FeedForwardAct::Gelu},
        {"Fobanex", "fobanex", false, FeedForwardAct::GatedSilu, true, true, OutputGate::PerValue, false, true},
        {"Minodra", "minodra", false, FeedForwardAct::GatedSilu, false, false, OutputGate::PerHead, true, false, true, RouterKind::CorrectedScores,
         ExpertKind::SquaredRelu},
    };
    return table;
}

// {"architecture", "width", "vocab", "norm": {"eps"}, "logit_scale", "logit_softcap",
//  "loop": {"start", "stop", "times"}, "embedding": {"scale", "bigram": {"buckets", "mul_prev", "mul_cur"}},
//  "canon": {"taps"},
//  "layers": [{"type", "mixer": {...}, "mlp": {"kind": "dense", "ff"} | {"kind": "moe", "expert": {"ff", "limit"},
//              "router": {"experts", "top", "scale", "groups": {"count", "keep"}}, "shared": {"ff"}} | null}, ...]}
inline void apply_stack_config(ModelConfig& m, const Json& c, const StackArchitecture& a) {
    m.arch = a.arch;
    m.sandwich_norms = a.sandwich_norms;
    m.ff_act = a.ff_act;
    m.shared_norm = a.shared_norm;
    m.ff_biases = a.ff_biases;
    m.gated_sublayers = a.gated_sublayers;
    m.canon_taps = a.gated_sublayers ? json_size(json_object(c, "canon", "config.json"), "taps", "canon") : 0;
    m.embed_scale = 1.f;
    m.bigram = BigramSpec{};
    if (const Json* e = c.get("embedding"); (a.shared_norm || a.gated_sublayers) && e && e->kind == Json::Object) {
        m.embed_scale = static_cast<float>(e->number_or("scale", 1.0));
        if (const Json* b = e->get("bigram"); a.gated_sublayers && b && b->kind == Json::Object) {
            m.bigram.buckets = json_count(*b, "buckets", "embedding.bigram");
            m.bigram.mul_prev = json_count(*b, "mul_prev", "embedding.bigram");
            m.bigram.mul_cur = json_count(*b, "mul_cur", "embedding.bigram");
            if (m.bigram.buckets == 0) throw std::runtime_error("snapshot: embedding.bigram.buckets must be positive");
        }
    }
    m.hidden = json_size(c, "width", "config.json");
    m.vocab = json_size(c, "vocab", "config.json");
    const Json* norm = c.get("norm");
    if (!norm) throw std::runtime_error("snapshot: config.json needs 'norm'");
    m.rms_eps = static_cast<float>(json_number(*norm, "eps", "norm"));
    m.logit_scale = static_cast<float>(c.number_or("logit_scale", 1.0));
    m.logit_softcap = static_cast<float>(c.number_or("logit_softcap", 0.0));
    m.loop = LayerLoop{};
    if (const Json* loop = c.get("loop"); loop && loop->kind == Json::Object) {
        m.loop.start = json_size(*loop, "start", "loop");
        m.loop.stop = json_size(*loop, "stop", "loop");
        m.loop.times = json_size(*loop, "times", "loop");
    }
    const Json* layers = c.get("layers");
    if (!layers || layers->kind != Json::Array || layers->arr.empty())
        throw std::runtime_error("snapshot: config.json needs a list 'layers'");
    m.stack.clear();
    for (const Json& j : layers->arr) {
        const std::string at = "layer " + std::to_string(m.stack.size());
        LayerSpec l;
        const std::string type = j.string_or("type", "");
        const Json* mixer = j.get("mixer");
        if (!mixer || mixer->kind != Json::Object) throw std::runtime_error("snapshot: " + at + " needs 'mixer'");
        bool known = false;
        for (const MixerReader& r : mixer_registry())
            if (type == r.type) {
                r.read(l, *mixer, at);
                known = true;
            }
        if (!known) throw std::runtime_error("snapshot: " + at + ": unknown mixer '" + type + "'");
        l.latent.half_split = a.half_split_latents;
        l.latent.gate = a.latent_gate;
        l.latent.sinks = a.latent_sinks;
        if (const Json* mlp = j.get("mlp"); mlp && mlp->kind == Json::Object) {
            const std::string kind = mlp->string_or("kind", "");
            if (kind == "dense") {
                l.ff = json_size(*mlp, "ff", at + " mlp");
                if (l.ff <= 0) throw std::runtime_error("snapshot: " + at + ": mlp.ff must be positive");
            } else if (kind == "moe" && (a.shared_norm || a.gated_sublayers)) {
                l.moe = parse_mixture(*mlp, at + " mlp", a.router, a.expert);
            } else {
                throw std::runtime_error("snapshot: " + at + ": unknown mlp kind '" + kind + "'");
            }
        }
        m.stack.push_back(l);
    }
}

// ---- config.json -> ModelConfig ----------------------------------------------------------------
// Field names as transformers writes them (llama / qwen3 / qwen3_moe); the reference reads the
// same keys in driver/portable/src/hf_config.cpp.  Checkpoints use the half-split RoPE pairing
// (the CUDA driver's default, driver/cuda/src/kernels/rope.cu:10-21) unless the TOML says otherwise.
inline void apply_hf_fields(ModelConfig& m, const Json& c, const std::string& type) {
    if (type == "llama" || type == "mistral") m.arch = "llama3";
    else if (type == "qwen3") m.arch = "qwen3";
    else if (type == "qwen3_moe") m.arch = "qwen3_moe";
    else throw std::runtime_error("snapshot: unsupported model_type '" + type + "'");
    m.hidden = static_cast<int>(c.number_or("hidden_size", 0));
    // (Mistral-type checkpoints: "sliding_window": N or null; Qwen3 writes one next to
    // "use_sliding_window": false, which switches it off)
    if (m.sliding_window <= 0 && c.bool_or("use_sliding_window", true))
        m.sliding_window = static_cast<int>(c.number_or("sliding_window", 0));
    m.layers = static_cast<int>(c.number_or("num_hidden_layers", 0));
    m.q_heads = static_cast<int>(c.number_or("num_attention_heads", 0));
    m.kv_heads = static_cast<int>(c.number_or("num_key_value_heads", m.q_heads));
    m.head_dim = static_cast<int>(c.number_or("head_dim", m.q_heads ? m.hidden / m.q_heads : 0));
    m.intermediate = static_cast<int>(c.number_or("intermediate_size", 0));
    m.vocab = static_cast<int>(c.number_or("vocab_size", 0));
    m.rms_eps = static_cast<float>(c.number_or("rms_norm_eps", 1e-5));
    m.rope_theta = static_cast<float>(c.number_or("rope_theta", 10000.0));
    m.tie_embeddings = c.bool_or("tie_word_embeddings", false);
    m.rope_factor = 0.f;
    if (const Json* rs = c.get("rope_scaling"); rs && rs->kind == Json::Object) {
        const std::string rt = rs->string_or("rope_type", rs->string_or("type", ""));
        if (rt == "llama3") {
            m.rope_factor = static_cast<float>(rs->number_or("factor", 8.0));
            m.rope_low_freq_factor = static_cast<float>(rs->number_or("low_freq_factor", 1.0));
            m.rope_high_freq_factor = static_cast<float>(rs->number_or("high_freq_factor", 4.0));
            m.rope_original_max_pos = static_cast<int>(rs->number_or("original_max_position_embeddings", 8192));
        } else if (rt == "yarn") {
            m.rope_scaling = "yarn";
            m.rope_factor = static_cast<float>(rs->number_or("factor", 1.0));
            m.rope_beta_fast = static_cast<float>(rs->number_or("beta_fast", 32.0));
            m.rope_beta_slow = static_cast<float>(rs->number_or("beta_slow", 1.0));
            m.rope_attention_factor = static_cast<float>(rs->number_or("attention_factor", 0.0));
            m.rope_original_max_pos = static_cast<int>(rs->number_or(
                "original_max_position_embeddings", c.number_or("max_position_embeddings", 8192)));
        } else if (!rt.empty() && rt != "default") {
            throw std::runtime_error("snapshot: unsupported rope_scaling type '" + rt + "'");
        }
    }
    if (m.arch == "qwen3_moe") {
        m.num_experts = static_cast<int>(c.number_or("num_experts", 0));
        m.top_k = static_cast<int>(c.number_or("num_experts_per_tok", 0));
        m.expert_intermediate = static_cast<int>(c.number_or("moe_intermediate_size", 0));
        m.norm_topk = c.bool_or("norm_topk_prob", true);
    }
    if (m.rope_interleaved < 0) m.rope_interleaved = 0;
}

// The registry of architectures: config.json's "model_type" (Hugging Face checkpoints) or
// "architecture" (layer stacks) picks the reader.
inline void apply_hf_config(ModelConfig& m, const std::string& dir) {
    const Json c = parse_json_file(dir + "/config.json");
    const std::string arch = c.string_or("architecture", "");
    for (const StackArchitecture& a : stack_registry())
        if (arch == a.name) return apply_stack_config(m, c, a);
    const std::string type = c.string_or("model_type", "");
    if (type.empty() && !arch.empty()) throw std::runtime_error("snapshot: unsupported architecture '" + arch + "'");
    apply_hf_fields(m, c, type);
}

}  // namespace pie_hip_driver
