// loader.h — safetensors -> device, without the reference's fp32 host expansion and host transposes
// (SURVEY §8 f-2).  Host-only C++; included at the end of nvllm.hip.
//
// Replaces tensor.LoadModelFromDirectory / LoadModel / LoadShardedModel (purego/tensor/generic_loader.go:184-265,
// 1016-1163) and LoadModelConfig (:808-972).  The checkpoint is mmap'ed; every 2-D weight goes to nvl_upload_tensor
// in the checkpoint's own dtype (F32 / F16 / BF16, :645-663) and PyTorch [out, in] layout — the dtype conversion,
// the [in, out] view the reference builds with Transpose (:398-403, :533-552) and the tiling into the kernels'
// operand layout all happen on the device.  Only the fused projections go through a host fp32 copy (GPT-2 c_attn,
// Falcon query_key_value: split rules of :674-748), because their split is defined on the fp32 [in, out] matrix.
// Differences from the reference, on purpose: sharded checkpoints may hold MoE layers (the reference's shard path has
// none, :1270-1273); a tensor is looked up under its name and under "transformer." + name in every file (:622-629).
#pragma once

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cstdlib>
#include <map>
#include <memory>
#include <string>
#include <vector>

namespace nvl_loader {

// ---------------------------------------------------------------------------------------------
// JSON (just what config.json / safetensors headers need)
// ---------------------------------------------------------------------------------------------
struct JVal {
    enum Kind { NUL, BOOL, NUM, STR, ARR, OBJ } kind = NUL;
    bool b = false;
    double num = 0;
    std::string str;
    std::vector<JVal> arr;
    std::vector<std::pair<std::string, JVal>> obj;
    const JVal* get(const std::string& k) const {
        if (kind != OBJ) return nullptr;
        for (auto& kv : obj) if (kv.first == k) return &kv.second;
        return nullptr;
    }
};

struct JParser {
    const char* p; const char* end;
    int depth = 0;                         // nesting is capped: a hostile header must not recurse the stack away
    static constexpr int MAX_DEPTH = 64;
    JParser(const char* s, size_t n) : p(s), end(s + n) {}
    [[noreturn]] void bad(const char* what) { throw std::runtime_error(std::string("json: ") + what); }
    void ws() { while (p < end && (*p == ' ' || *p == '\n' || *p == '\t' || *p == '\r')) p++; }
    JVal parse() { ws(); JVal v = value(); ws(); return v; }
    struct Depth { int& d; explicit Depth(int& d_) : d(d_) { ++d; } ~Depth() { --d; } };
    JVal value() {
        if (p >= end) bad("unexpected end");
        Depth guard(depth);
        if (depth > MAX_DEPTH) bad("nesting deeper than 64 levels");
        JVal v;
        switch (*p) {
            case '{': {
                v.kind = JVal::OBJ; p++; ws();
                if (p < end && *p == '}') { p++; return v; }
                for (;;) {
                    ws();
                    if (p >= end || *p != '"') bad("expected a key");
                    std::string k = string();
                    ws();
                    if (p >= end || *p != ':') bad("expected ':'");
                    p++; ws();
                    v.obj.emplace_back(std::move(k), value());
                    ws();
                    if (p < end && *p == ',') { p++; continue; }
                    if (p < end && *p == '}') { p++; return v; }
                    bad("expected ',' or '}'");
                }
            }
            case '[': {
                v.kind = JVal::ARR; p++; ws();
                if (p < end && *p == ']') { p++; return v; }
                for (;;) {
                    ws();
                    v.arr.push_back(value());
                    ws();
                    if (p < end && *p == ',') { p++; continue; }
                    if (p < end && *p == ']') { p++; return v; }
                    bad("expected ',' or ']'");
                }
            }
            case '"': v.kind = JVal::STR; v.str = string(); return v;
            case 't': lit("true"); v.kind = JVal::BOOL; v.b = true; return v;
            case 'f': lit("false"); v.kind = JVal::BOOL; v.b = false; return v;
            case 'n': lit("null"); return v;
            default: {
                char* e = nullptr;
                v.num = std::strtod(p, &e);          // (headers are NUL-terminated copies: strtod cannot run off the end)
                if (e == p) bad("unexpected character");
                v.kind = JVal::NUM; p = e; return v;
            }
        }
    }
    void lit(const char* s) { const size_t n = strlen(s); if ((size_t)(end - p) < n || strncmp(p, s, n) != 0) bad("bad literal"); p += n; }
    std::string string() {
        std::string out; p++;
        while (p < end && *p != '"') {
            if (*p == '\\') {
                if (++p >= end) bad("bad escape");
                switch (*p) {
                    case 'n': out += '\n'; break; case 't': out += '\t'; break; case 'r': out += '\r'; break;
                    case 'b': out += '\b'; break; case 'f': out += '\f'; break;
                    case 'u': {     // keep BMP code points as UTF-8; names in checkpoints are ASCII anyway
                        if (end - p < 5) bad("bad \\u escape");
                        const unsigned cp = (unsigned)std::strtoul(std::string(p + 1, 4).c_str(), nullptr, 16);
                        if (cp < 0x80) out += (char)cp;
                        else if (cp < 0x800) { out += (char)(0xC0 | (cp >> 6)); out += (char)(0x80 | (cp & 63)); }
                        else { out += (char)(0xE0 | (cp >> 12)); out += (char)(0x80 | ((cp >> 6) & 63)); out += (char)(0x80 | (cp & 63)); }
                        p += 4; break;
                    }
                    default: out += *p;
                }
                p++;
            } else out += *p++;
        }
        if (p >= end) bad("unterminated string");
        p++;
        return out;
    }
};

inline std::string read_text(const std::string& path) {
    FILE* f = fopen(path.c_str(), "rb");
    if (!f) throw std::runtime_error("cannot open " + path);
    std::string s; char buf[1 << 16]; size_t n;
    while ((n = fread(buf, 1, sizeof buf, f)) > 0) s.append(buf, n);
    fclose(f);
    return s;
}
inline bool exists(const std::string& path, bool* is_dir = nullptr) {
    struct stat st;
    if (stat(path.c_str(), &st) != 0) return false;
    if (is_dir) *is_dir = S_ISDIR(st.st_mode);
    return true;
}

// ---------------------------------------------------------------------------------------------
// safetensors: 8-byte LE header length, JSON header {name: {dtype, shape, data_offsets}}, raw little-endian data
// (generic_loader.go:184-199, loader.go:13-17)
// ---------------------------------------------------------------------------------------------
struct StTensor { const uint8_t* data = nullptr; int dtype = 0; std::vector<int64_t> shape; size_t bytes = 0; int64_t numel = 1; };

struct StFile {
    int fd = -1; void* map = MAP_FAILED; size_t size = 0;
    ~StFile() { if (map != MAP_FAILED) munmap(map, size); if (fd >= 0) close(fd); }
};

struct StSet {
    std::vector<std::unique_ptr<StFile>> files;
    std::map<std::string, StTensor> tensors;

    void add_file(const std::string& path) {
        std::unique_ptr<StFile> f(new StFile);
        f->fd = open(path.c_str(), O_RDONLY);
        if (f->fd < 0) throw std::runtime_error("cannot open " + path);
        struct stat st; fstat(f->fd, &st); f->size = (size_t)st.st_size;
        if (f->size < 8) throw std::runtime_error(path + ": not a safetensors file");
        f->map = mmap(nullptr, f->size, PROT_READ, MAP_PRIVATE, f->fd, 0);
        if (f->map == MAP_FAILED) throw std::runtime_error("mmap failed for " + path);
        const uint8_t* base = (const uint8_t*)f->map;
        uint64_t hlen = 0; memcpy(&hlen, base, 8);
        if (hlen > f->size - 8) throw std::runtime_error(path + ": header length exceeds the file");
        const std::string header((const char*)base + 8, (size_t)hlen);
        const JVal root = JParser(header.c_str(), header.size()).parse();
        if (root.kind != JVal::OBJ) throw std::runtime_error(path + ": header is not a JSON object");
        const uint8_t* data = base + 8 + hlen;
        const size_t data_len = f->size - 8 - (size_t)hlen;
        for (auto& kv : root.obj) {
            if (kv.first == "__metadata__") continue;
            const JVal *dt = kv.second.get("dtype"), *sh = kv.second.get("shape"), *off = kv.second.get("data_offsets");
            if (!dt || !sh || !off || off->arr.size() != 2) throw std::runtime_error(path + ": malformed entry " + kv.first);
            StTensor t;
            if (dt->str == "F32") t.dtype = NVL_DTYPE_F32; else if (dt->str == "BF16") t.dtype = NVL_DTYPE_BF16;
            else if (dt->str == "F16") t.dtype = NVL_DTYPE_F16; else t.dtype = -1;      // refused only if the model needs it (:660-662)
            for (auto& d : sh->arr) {      // dimensions: non-negative integers whose product stays far inside int64
                if (d.kind != JVal::NUM || !(d.num >= 0) || d.num > 4.0e12 || d.num != (double)(int64_t)d.num)
                    throw std::runtime_error(path + ": bad dimension in the shape of " + kv.first);
                const int64_t dim = (int64_t)d.num;
                if (dim != 0 && t.numel > ((int64_t)1 << 46) / dim)
                    throw std::runtime_error(path + ": shape of " + kv.first + " overflows");
                t.shape.push_back(dim); t.numel *= dim;
            }
            if (off->arr[0].kind != JVal::NUM || off->arr[1].kind != JVal::NUM || !(off->arr[0].num >= 0) || !(off->arr[1].num >= 0) ||
                off->arr[0].num > 9.0e15 || off->arr[1].num > 9.0e15)
                throw std::runtime_error(path + ": bad data_offsets of " + kv.first);
            const size_t b = (size_t)off->arr[0].num, e = (size_t)off->arr[1].num;
            if (e < b || e > data_len) throw std::runtime_error(path + ": data_offsets of " + kv.first + " outside the file");
            t.data = data + b; t.bytes = e - b;
            if (t.dtype >= 0 && t.bytes != (size_t)t.numel * (t.dtype == NVL_DTYPE_F32 ? 4 : 2))
                throw std::runtime_error(path + ": byte size of " + kv.first + " does not match its shape");
            tensors[kv.first] = std::move(t);
        }
        files.push_back(std::move(f));
    }
    // a file, or a directory with model.safetensors or model.safetensors.index.json + shards (:1016-1040, :1042-1075)
    void open_path(const std::string& path) {
        bool dir = false;
        if (!exists(path, &dir)) throw std::runtime_error("no such file or directory: " + path);
        if (!dir) { add_file(path); return; }
        const std::string idx = path + "/model.safetensors.index.json";
        if (exists(idx)) {
            const std::string txt = read_text(idx);
            const JVal root = JParser(txt.c_str(), txt.size()).parse();
            const JVal* wm = root.get("weight_map");
            if (!wm || wm->kind != JVal::OBJ) throw std::runtime_error(idx + ": no weight_map");
            std::vector<std::string> shards;
            for (auto& kv : wm->obj) {
                const std::string& sn = kv.second.str;      // a shard is a plain file name inside the model directory
                if (kv.second.kind != JVal::STR || sn.empty() || sn.find('/') != std::string::npos || sn.find('\\') != std::string::npos ||
                    sn == "." || sn.find("..") != std::string::npos)
                    throw std::runtime_error(idx + ": weight_map names a shard outside the model directory: '" + sn + "'");
                if (std::find(shards.begin(), shards.end(), sn) == shards.end()) shards.push_back(sn);
            }
            for (auto& s : shards) add_file(path + "/" + s);
            return;
        }
        add_file(path + "/model.safetensors");
    }
    const StTensor* find(const std::string& name) const {           // :619-632
        auto it = tensors.find(name);
        if (it == tensors.end()) it = tensors.find("transformer." + name);
        return it == tensors.end() ? nullptr : &it->second;
    }
    const StTensor& need(const std::string& name) const {
        const StTensor* t = find(name);
        if (!t) throw std::runtime_error("required tensor '" + name + "' not found (also tried: transformer." + name + ")");
        if (t->dtype < 0) throw std::runtime_error("unsupported dtype for tensor '" + name + "'");
        return *t;
    }
};

inline float f32_of(const StTensor& t, int64_t i) {                  // :769-805
    if (t.dtype == NVL_DTYPE_F32) { float f; memcpy(&f, t.data + i * 4, 4); return f; }
    uint16_t h; memcpy(&h, t.data + i * 2, 2);
    uint32_t u;
    if (t.dtype == NVL_DTYPE_BF16) u = (uint32_t)h << 16;
    else {
        const uint32_t s = (h >> 15) & 1u, e = (h >> 10) & 31u, m = h & 1023u;
        if (e == 0) {
            if (m == 0) u = s << 31;
            else { int k = 0; uint32_t mm = m; while (!(mm & 1024u)) { mm <<= 1; k++; } u = (s << 31) | ((uint32_t)(113 - k) << 23) | ((mm & 1023u) << 13); }
        } else if (e == 31) u = (s << 31) | 0x7F800000u | (m << 13);
        else u = (s << 31) | ((e + 112u) << 23) | (m << 13);
    }
    float f; memcpy(&f, &u, 4); return f;
}

}  // namespace nvl_loader

// ---------------------------------------------------------------------------------------------
// C ABI
// ---------------------------------------------------------------------------------------------
namespace {
using nvl_loader::StSet; using nvl_loader::StTensor; using nvl_loader::JVal;

void up2d(nvl_model* m, int kind, int layer, const StTensor& t, int layout) {
    if (t.shape.size() != 2) throw std::runtime_error("loader: a 2-D tensor was expected");
    const int rc = nvl_upload_tensor(m, kind, layer, t.data, t.dtype, t.shape[0], t.shape[1], layout);
    if (rc) throw std::runtime_error(std::string("loader: ") + nvl_last_error(m));
}
void up1d(nvl_model* m, int kind, int layer, const StTensor& t) {
    const int rc = nvl_upload_tensor(m, kind, layer, t.data, t.dtype, t.numel, 1, NVL_LAYOUT_IN_OUT);
    if (rc) throw std::runtime_error(std::string("loader: ") + nvl_last_error(m));
}
// loadNorm (:595-604): weight required, bias (".weight" -> ".bias") optional
void load_norm(nvl_model* m, const StSet& st, const std::string& key, int kind_w, int kind_b, int layer) {
    up1d(m, kind_w, layer, st.need(key));
    std::string bk = key;
    const size_t p = bk.find(".weight");
    if (p != std::string::npos) bk.replace(p, 7, ".bias");
    if (const StTensor* b = st.find(bk)) if (b->dtype >= 0) up1d(m, kind_b, layer, *b);
}
std::vector<float> to_f32(const StTensor& t) {
    std::vector<float> v((size_t)t.numel);
    for (int64_t i = 0; i < t.numel; i++) v[(size_t)i] = nvl_loader::f32_of(t, i);
    return v;
}

// ---- models described by a list of layers ----
struct LayeredArch { const char* name; int block_style, activation; float norm_offset; int norm_type, position_type; };
const LayeredArch LAYERED_ARCHS[] = {{"Potuzen", NVL_BLOCK_SANDWICH, NVL_ACT_GEGLU, 0.f, NVL_NORM_RMS, NVL_POS_NONE},
                                     {"Lufazen", NVL_BLOCK_POST, NVL_ACT_CLAMPED_GLU, 1.f, NVL_NORM_RMS, NVL_POS_NONE},
                                     {"Bolinex", NVL_BLOCK_PARALLEL, NVL_ACT_RELU2, 0.f, NVL_NORM_LAYER, NVL_POS_LEARNED},
                                     {"Medulorn", NVL_BLOCK_SUM_NORM, NVL_ACT_REGLU, 0.f, NVL_NORM_RMS_SCALAR, NVL_POS_NONE}};
const LayeredArch* layered_arch(const std::string& name) {
    for (const LayeredArch& a : LAYERED_ARCHS) if (name == a.name) return &a;
    return nullptr;
}
double need_num(const JVal* o, const char* key, const std::string& where) {
    const JVal* v = o ? o->get(key) : nullptr;
    if (!v || v->kind != JVal::NUM) throw std::runtime_error(where + "number '" + key + "' expected");
    return v->num;
}
int need_int(const JVal* o, const char* key, const std::string& where) {
    const double v = need_num(o, key, where);
    if (v != std::floor(v) || v < -2147483648.0 || v > 2147483647.0) throw std::runtime_error(where + "'" + key + "' is not an integer");
    return (int)v;
}
// the rotation of a latent attention layer: {dims, base, scaling: null | {factor, original, fast, slow}}
void parse_rotation(const JVal* mx, nvl_layer_config& c, const std::string& at) {
    c.rot_dim = need_int(mx, "rot_dim", at);
    const JVal* rot = mx->get("rot");
    if (need_int(rot, "dims", at) != c.rot_dim) throw std::runtime_error(at + "rot.dims differs from rot_dim");
    c.rot_base = need_num(rot, "base", at);
    const JVal* sc = rot->get("scaling");
    if (sc && sc->kind == JVal::OBJ) {
        c.rot_factor = need_num(sc, "factor", at); c.rot_original = need_num(sc, "original", at);
        c.rot_fast = need_num(sc, "fast", at); c.rot_slow = need_num(sc, "slow", at);
    }
}
// grouped-query attention: kv_heads, softcap (a number or null), v_mix (true / false)
void parse_attention(const JVal* mx, nvl_layer_config& c, const std::string& at) {
    c.mixer = NVL_MIXER_ATTENTION;
    c.dim = need_int(mx, "dim", at); c.kv_heads = need_int(mx, "kv_heads", at); c.scale = (float)need_num(mx, "scale", at);
    const JVal *cap = mx->get("softcap"), *mix = mx->get("v_mix");
    if (cap && cap->kind != JVal::NUL) {
        c.softcap = (float)need_num(mx, "softcap", at);
        if (!(c.softcap > 0.f)) throw std::runtime_error(at + "softcap is not positive");
    }
    c.v_mix = mix && ((mix->kind == JVal::BOOL && mix->b) || (mix->kind == JVal::NUM && mix->num != 0));
}
// a mixture of experts: {expert: {ff}, router: {experts, top, groups: null | {count, keep}}, shared: null | {ff}}
void parse_experts(const JVal* mlp, nvl_layer_config& c, const std::string& at) {
    const JVal *ex = mlp->get("expert"), *ro = mlp->get("router"), *sh = mlp->get("shared");
    c.expert_dim = need_int(ex, "ff", at); c.experts = need_int(ro, "experts", at); c.top_k = need_int(ro, "top", at);
    c.expert_groups = c.groups_kept = 1;
    const JVal* gr = ro->get("groups");
    if (gr && gr->kind == JVal::OBJ) { c.expert_groups = need_int(gr, "count", at); c.groups_kept = need_int(gr, "keep", at); }
    c.ffn_act = NVL_ACT_SWIGLU;
    if (sh && sh->kind == JVal::OBJ) c.ffn_dim = need_int(sh, "ff", at);
    if (c.experts <= 0 || c.expert_dim <= 0 || c.ffn_dim < 0) throw std::runtime_error(at + "an expert size is not positive");
}
// a key mask {size, keep_first} (null: none); returns the size
int parse_mask(const JVal* mx, int* keep_first, const std::string& at) {
    const JVal* mask = mx->get("mask");
    if (!mask || mask->kind != JVal::OBJ) return 0;
    const int size = need_int(mask, "size", at);
    if (size <= 0) throw std::runtime_error(at + "the mask's size is not positive");
    const JVal* kept = mask->get("keep_first");
    if (keep_first && kept && kept->kind != JVal::NUL) *keep_first = need_int(mask, "keep_first", at);
    return size;
}
// what the two attentions of the design with norms of sums share: sizes, scale, rotation {dims, base, scaling: null | {factor, original, low, high}}
void parse_plain_attention(const JVal* mx, nvl_layer_config& c, const std::string& at) {
    c.mixer = NVL_MIXER_ATTENTION;
    c.heads = need_int(mx, "heads", at); c.kv_heads = need_int(mx, "kv_heads", at); c.dim = need_int(mx, "dim", at); c.vdim = need_int(mx, "vdim", at);
    c.scale = (float)need_num(mx, "scale", at);
    c.ungated = 1;
    const JVal* rot = mx->get("rot");
    if (!rot || rot->kind != JVal::OBJ) return;
    c.rot_dim = need_int(rot, "dims", at); c.rot_base = need_num(rot, "base", at);
    const JVal* sc = rot->get("scaling");
    if (sc && sc->kind == JVal::OBJ) {
        c.rot_factor = need_num(sc, "factor", at); c.rot_original = need_num(sc, "original", at);
        c.rot_low = need_num(sc, "low", at); c.rot_high = need_num(sc, "high", at);
    }
}
// a layer of that design
nvl_layer_config parse_sum_norm_layer(const std::string& type, const JVal* mx, const JVal* mlp, const std::string& at) {
    nvl_layer_config c;
    memset(&c, 0, sizeof c);
    c.kv_from = c.weights_of = -1;
    if (type == "attention") {
        parse_plain_attention(mx, c, at);
        c.qk_norm = NVL_QK_NORM_HEAD; c.sink = NVL_SINK_ZERO; c.qkv_bias = 1;
        c.chunk = parse_mask(mx, nullptr, at);
    } else if (type == "parallel") {
        const JVal *left = mx->get("left"), *right = mx->get("right");
        if (!left || left->kind != JVal::OBJ || !right || right->kind != JVal::OBJ) throw std::runtime_error(at + "'left' and 'right' expected");
        parse_plain_attention(left, c, at);
        c.qk_norm = NVL_QK_NORM_ROW; c.sink = NVL_SINK_LEARNED;
        c.window = parse_mask(left, &c.keep_first, at);
        c.out_scale = (float)need_num(mx, "left_scale", at); c.out_scale2 = (float)need_num(mx, "right_scale", at);
        c.mixer2 = NVL_MIXER_LIGHTNING;
        c.heads2 = need_int(right, "heads", at); c.dim2 = need_int(right, "dim", at); c.vdim2 = need_int(right, "vdim", at);
        const JVal* decay = right->get("decay");
        if (!decay || decay->kind != JVal::ARR || c.heads2 <= 0 || decay->arr.size() != (size_t)c.heads2) throw std::runtime_error(at + "as many decays as heads expected");
        if (c.heads2 > NVL_MAX_DECAYS) throw std::runtime_error(at + "too many heads of lightning attention");
        for (size_t h = 0; h < decay->arr.size(); h++) {
            if (decay->arr[h].kind != JVal::NUM) throw std::runtime_error(at + "a decay is not a number");
            c.decay[h] = decay->arr[h].num;
        }
    } else throw std::runtime_error(at + "unknown mixer '" + type + "'");
    if (!mlp || mlp->kind != JVal::OBJ) return c;
    const JVal* kind = mlp->get("kind");
    const std::string k = kind && kind->kind == JVal::STR ? kind->str : kind ? "?" : "dense";
    if (k == "moe") {
        parse_experts(mlp, c, at);
        c.expert_limit = (float)need_num(mlp->get("expert"), "limit", at);
        c.route_softmax = 1;
        c.ffn_act = 0;
        if (c.ffn_dim) { c.ffn_act = NVL_ACT_CLAMPED_GLU; c.ffn_limit = (float)need_num(mlp->get("shared"), "limit", at); }
    } else if (k == "dense") {
        c.ffn_dim = need_int(mlp, "ff", at);
        if (c.ffn_dim <= 0) throw std::runtime_error(at + "the feed-forward size is not positive");
    } else throw std::runtime_error(at + "unknown feed-forward kind");
    return c;
}
std::vector<nvl_layer_config> parse_layers(const JVal& raw, const LayeredArch& arch) {
    const bool post = arch.block_style == NVL_BLOCK_POST, par = arch.block_style == NVL_BLOCK_PARALLEL;
    const JVal* ls = raw.get("layers");
    if (!ls || ls->kind != JVal::ARR || ls->arr.empty()) throw std::runtime_error("config: list 'layers' expected");
    std::vector<nvl_layer_config> out;
    for (size_t i = 0; i < ls->arr.size(); i++) {
        const JVal& e = ls->arr[i];
        const std::string at = "config: layer " + std::to_string(i) + ": ";
        nvl_layer_config c;
        memset(&c, 0, sizeof c);
        c.kv_from = -1;
        const JVal *ty = e.get("type"), *mx = e.get("mixer"), *mlp = e.get("mlp"), *wo = e.get("weights_of");
        if (!ty || ty->kind != JVal::STR || !mx || mx->kind != JVal::OBJ) throw std::runtime_error(at + "'type' and 'mixer' expected");
        if (arch.block_style == NVL_BLOCK_SUM_NORM) { out.push_back(parse_sum_norm_layer(ty->str, mx, mlp, at)); continue; }
        c.weights_of = wo && wo->kind == JVal::NUM ? need_int(&e, "weights_of", at) : -1;
        c.heads = need_int(mx, "heads", at); c.vdim = need_int(mx, "vdim", at);
        if (ty->str == "attention" && par) parse_attention(mx, c, at);
        else if (ty->str == "latent_attention" && !par) {
            c.mixer = NVL_MIXER_LATENT_ATTENTION;
            c.dim = need_int(mx, "dim", at); c.q_rank = need_int(mx, "q_rank", at); c.kv_rank = need_int(mx, "kv_rank", at);
            c.scale = (float)need_num(mx, "scale", at);
            if (post) {
                parse_rotation(mx, c, at);
                c.gate_per_head = 1;
                const JVal* kf = mx->get("kv_from");
                if (kf && kf->kind == JVal::NUM) c.kv_from = need_int(mx, "kv_from", at);
            }
        } else if (ty->str == "channel_delta" && post) {
            c.mixer = NVL_MIXER_CHANNEL_DELTA;
            c.dim = need_int(mx, "dim", at); c.kv_heads = need_int(mx, "kv_heads", at); c.conv_taps = need_int(mx, "conv", at);
        } else if (ty->str == "mamba2" && !post && !par) {
            c.mixer = NVL_MIXER_MAMBA2;
            c.state = need_int(mx, "state", at); c.groups = need_int(mx, "groups", at); c.norm_groups = need_int(mx, "norm_groups", at);
            c.conv_taps = need_int(mx, "conv", at);
        } else if (ty->str == "gla" && !post && !par) {
            c.mixer = NVL_MIXER_GLA;
            c.dim = need_int(mx, "dim", at); c.tau = (float)need_num(mx, "tau", at);
        } else throw std::runtime_error(at + "unknown mixer '" + ty->str + "'");
        const JVal* mask = mx->get("mask");
        if (mask && mask->kind == JVal::OBJ && (c.mixer == NVL_MIXER_LATENT_ATTENTION || c.mixer == NVL_MIXER_ATTENTION)) {
            c.window = need_int(mask, "size", at);
            if (c.window <= 0) throw std::runtime_error(at + "the window is not positive");
        }
        if (mlp && mlp->kind == JVal::OBJ) {
            const JVal* kind = mlp->get("kind");
            if (par && kind && kind->kind == JVal::STR && kind->str == "moe") { parse_experts(mlp, c, at); out.push_back(c); continue; }
            if (kind && !(kind->kind == JVal::STR && kind->str == "dense")) throw std::runtime_error(at + "unknown feed-forward kind");
            c.ffn_dim = need_int(mlp, "ff", at);
            if (c.ffn_dim <= 0) throw std::runtime_error(at + "the feed-forward size is not positive");
            if (arch.activation == NVL_ACT_CLAMPED_GLU) c.ffn_limit = (float)need_num(mlp, "limit", at);
        }
        out.push_back(c);
    }
    return out;
}
void load_layered(nvl_model* m, const StSet& st) {
    const int OI = NVL_LAYOUT_OUT_IN;
    auto mat = [&](int kind, int layer, const std::string& name) { up2d(m, kind, layer, st.need(name), OI); };
    auto vec = [&](int kind, int layer, const std::string& name) { up1d(m, kind, layer, st.need(name)); };
    auto cat = [&](int kind, int layer, const std::vector<std::string>& names) {      // tensors one after the other (along their rows)
        const StTensor& a = st.need(names[0]);
        std::vector<uint8_t> all;
        int64_t rows = 0;
        for (const std::string& n : names) {
            const StTensor& t = st.need(n);
            if (t.dtype != a.dtype || t.shape.size() != 2 || a.shape.size() != 2 || t.shape[1] != a.shape[1]) throw std::runtime_error("loader: " + names[0] + " and " + n + " do not match");
            all.insert(all.end(), (const uint8_t*)t.data, (const uint8_t*)t.data + t.bytes);
            rows += t.shape[0];
        }
        if (nvl_upload_tensor(m, kind, layer, all.data(), a.dtype, rows, a.shape[1], OI)) throw std::runtime_error(nvl_last_error(m));
    };
    const bool post = m->cfg.block_style == NVL_BLOCK_POST, par = m->cfg.block_style == NVL_BLOCK_PARALLEL, sum = m->cfg.block_style == NVL_BLOCK_SUM_NORM;
    if (m->cfg.norm_type == NVL_NORM_LAYER) vec(NVL_T_FINAL_NORM_B, 0, "final.norm.b");
    if (m->cfg.position_type == NVL_POS_LEARNED) mat(NVL_T_POS_EMB, 0, "pos");
    if (m->cfg.side_dim) mat(NVL_T_SIDE_EMB, 0, "side.embed");
    mat(NVL_T_TOK_EMB, 0, "embed");
    mat(NVL_T_LM_HEAD, 0, "head");
    vec(NVL_T_FINAL_NORM_W, 0, "final.norm");
    for (int i = 0; i < m->L; i++) {
        const LayerRun& r = m->runs[(size_t)i];
        if (r.owner != i) continue;
        const std::string l = "l" + std::to_string(i) + ".", x = l + "mix.";
        if (par) {
            vec(NVL_T_ATTN_NORM_W, i, l + "norm1");
            if (m->cfg.norm_type == NVL_NORM_LAYER) vec(NVL_T_ATTN_NORM_B, i, l + "norm1.b");
            if (m->cfg.side_dim) { mat(NVL_T_SIDE_GATE, i, l + "side.gate"); mat(NVL_T_SIDE_PROJ, i, l + "side.proj"); vec(NVL_T_SIDE_NORM, i, l + "side.norm"); }
        } else if (sum) {
            vec(NVL_T_MIX_POST_NORM, i, l + "norm1");
            if (r.c.ffn_dim || r.c.experts) vec(NVL_T_FFN_POST_NORM, i, l + "norm2");
        } else if (post) {
            vec(NVL_T_MIX_POST_NORM, i, l + "norm1"); vec(NVL_T_MIX_SCALE, i, l + "ls1");
            if (r.c.ffn_dim) { vec(NVL_T_FFN_POST_NORM, i, l + "norm2"); vec(NVL_T_FFN_SCALE, i, l + "ls2"); }
        } else {
            vec(NVL_T_ATTN_NORM_W, i, l + "norm1"); vec(NVL_T_MIX_POST_NORM, i, l + "norm1b");
            if (r.c.ffn_dim) { vec(NVL_T_FFN_NORM_W, i, l + "norm2"); vec(NVL_T_FFN_POST_NORM, i, l + "norm2b"); }
        }
        if (m->cfg.token_shift) vec(NVL_T_SHIFT, i, l + "shift");
        if (r.c.ffn_dim) {
            const std::string f = l + (r.c.experts ? "mlp.shared." : "mlp.");
            if (r.act == NVL_ACT_RELU2) mat(NVL_T_W1, i, f + "up"); else cat(NVL_T_W1, i, {f + "gate", f + "up"});
            mat(NVL_T_W2, i, f + "down");
        }
        if (r.c.experts) {
            std::vector<std::string> up, down;
            for (int e = 0; e < r.c.experts; e++) {
                const std::string x = l + "mlp.e" + std::to_string(e) + ".";
                up.push_back(x + "gate"); up.push_back(x + "up"); down.push_back(x + "down");
            }
            cat(NVL_T_MOE_IN, i, up); cat(NVL_T_MOE_OUT, i, down);
            mat(NVL_T_ROUTER, i, l + "mlp.router"); vec(NVL_T_ROUTER_BIAS, i, l + (r.c.route_softmax ? "mlp.router.b" : "mlp.correction"));
        }
        switch (r.c.mixer) {
            case NVL_MIXER_LATENT_ATTENTION:
                mat(NVL_T_LAT_DQ, i, x + "dq"); vec(NVL_T_LAT_DQ_NORM, i, x + "dq.norm"); mat(NVL_T_LAT_UQ, i, x + "uq");
                if (r.c.kv_from < 0) { mat(NVL_T_LAT_DKV, i, x + "dkv"); vec(NVL_T_LAT_DKV_NORM, i, x + "dkv.norm"); }
                mat(NVL_T_LAT_UK, i, x + "uk"); mat(NVL_T_LAT_UV, i, x + "uv");
                mat(NVL_T_MIX_GATE, i, x + "g"); mat(NVL_T_WO, i, x + "o");
                break;
            case NVL_MIXER_ATTENTION: {
                const std::string a = r.c.mixer2 ? x + "left." : x, b = x + "right.";
                mat(NVL_T_WQ, i, a + "q"); mat(NVL_T_WK, i, a + "k"); mat(NVL_T_WV, i, a + "v"); mat(NVL_T_WO, i, a + "o");
                if (r.c.qkv_bias) { vec(NVL_T_BQ, i, a + "q.b"); vec(NVL_T_BK, i, a + "k.b"); vec(NVL_T_BV, i, a + "v.b"); }
                if (r.c.qk_norm) { vec(NVL_T_Q_NORM, i, a + "q.norm"); vec(NVL_T_K_NORM, i, a + "k.norm"); }
                if (r.c.sink == NVL_SINK_LEARNED) vec(NVL_T_SINK, i, a + "sink");
                if (par) { mat(NVL_T_MIX_GATE, i, a + "g"); vec(NVL_T_BIAS_R1, i, a + "r1"); vec(NVL_T_BIAS_R2, i, a + "r2"); }
                if (r.c.v_mix) vec(NVL_T_V_MIX, i, a + "vmix");
                if (r.c.mixer2) {
                    mat(NVL_T_LIN_Q, i, b + "q"); mat(NVL_T_LIN_K, i, b + "k"); mat(NVL_T_LIN_V, i, b + "v"); mat(NVL_T_LIN_GATE, i, b + "g");
                    vec(NVL_T_LIN_NORM, i, b + "norm"); mat(NVL_T_LIN_O, i, b + "o");
                }
                break;
            }
            case NVL_MIXER_MAMBA2:
                mat(NVL_T_MAMBA_IN_PROJ, i, x + "in"); vec(NVL_T_MAMBA_CONV_W, i, x + "conv"); vec(NVL_T_MAMBA_CONV_B, i, x + "conv.b");
                vec(NVL_T_MAMBA_DT_BIAS, i, x + "dt_bias"); vec(NVL_T_MAMBA_A_LOG, i, x + "A_log"); vec(NVL_T_MAMBA_D, i, x + "D");
                vec(NVL_T_MAMBA_NORM, i, x + "norm"); mat(NVL_T_MAMBA_OUT_PROJ, i, x + "o");
                break;
            case NVL_MIXER_CHANNEL_DELTA:
                mat(NVL_T_WQ, i, x + "q"); mat(NVL_T_WK, i, x + "k"); mat(NVL_T_WV, i, x + "v"); mat(NVL_T_WO, i, x + "o");
                cat(NVL_T_DELTA_CONV, i, {x + "q.conv", x + "k.conv", x + "v.conv"}); mat(NVL_T_DELTA_BETA, i, x + "b");
                vec(NVL_T_MAMBA_A_LOG, i, x + "A_log"); vec(NVL_T_GLA_NORM, i, x + "norm");
                mat(NVL_T_GLA_A1, i, x + "a1"); mat(NVL_T_GLA_A2, i, x + "a2"); vec(NVL_T_GLA_A2_B, i, x + "dt_bias");
                mat(NVL_T_DELTA_G1, i, x + "g1"); mat(NVL_T_DELTA_G2, i, x + "g2");
                break;
            default:
                mat(NVL_T_WQ, i, x + "q"); mat(NVL_T_WK, i, x + "k"); mat(NVL_T_WV, i, x + "v"); mat(NVL_T_MIX_GATE, i, x + "g"); mat(NVL_T_WO, i, x + "o");
                vec(NVL_T_GLA_NORM, i, x + "norm"); mat(NVL_T_GLA_A1, i, x + "a1"); mat(NVL_T_GLA_A2, i, x + "a2"); vec(NVL_T_GLA_A2_B, i, x + "a2.b");
        }
    }
}
}  // namespace

extern "C" int nvl_load_layers_json(const char* path, nvl_layer_config* layers, int cap) {
    if (!path || (cap > 0 && !layers)) return NVL_ERR_INVALID;
    try {
        const std::string txt = nvl_loader::read_text(path);
        const JVal raw = nvl_loader::JParser(txt.c_str(), txt.size()).parse();
        const JVal* a = raw.get("architecture");
        const LayeredArch* arch = a && a->kind == JVal::STR ? layered_arch(a->str) : nullptr;
        if (!arch) return 0;
        const auto ls = parse_layers(raw, *arch);
        for (size_t i = 0; i < ls.size() && (int)i < cap; i++) layers[i] = ls[i];
        return (int)ls.size();
    } catch (const std::exception& e) {
        g_create_err = std::string("nvl_load_layers_json: ") + e.what();
        return NVL_ERR_INVALID;
    }
}

extern "C" int nvl_load_safetensors(nvl_model* m, const char* path) {
    if (!m || !path) return NVL_ERR_INVALID;
    if (m->finalized) return fail(m, NVL_ERR_STATE, "nvl_load_safetensors: model already finalized");
    NVL_TRY(m)
    StSet st;
    st.open_path(path);
    const nvl_model_config& c = m->cfg;
    if (m->layered) {
        load_layered(m, st);
        NVL_HIP(hipStreamSynchronize(m->stream));
        return NVL_OK;
    }
    // which WeightMapping (:60-181) — told from the checkpoint's own names
    const bool gpt2 = st.find("wte.weight") != nullptr;
    const bool falcon = st.find("transformer.word_embeddings.weight") != nullptr || st.find("word_embeddings.weight") != nullptr;
    const bool llama = st.find("model.embed_tokens.weight") != nullptr;       // Llama and Granite-MoE share the naming
    if (gpt2 + falcon + llama != 1) throw std::runtime_error("nvl_load_safetensors: cannot tell the architecture from the tensor names");
    const int OI = NVL_LAYOUT_OUT_IN, IO = NVL_LAYOUT_IN_OUT;

    if (gpt2) {                                                                // GetGPT2Mapping (:60-78): weights already [in, out]
        up2d(m, NVL_T_TOK_EMB, 0, st.need("wte.weight"), IO);
        if (const StTensor* pe = st.find("wpe.weight")) up2d(m, NVL_T_POS_EMB, 0, *pe, IO);
        for (int l = 0; l < c.num_layers; l++) {
            const std::string p = "h." + std::to_string(l);
            const std::vector<float> w = to_f32(st.need(p + ".attn.c_attn.weight"));     // splitGPT2QKV (:674-702)
            std::vector<float> b;
            if (const StTensor* bt = st.find(p + ".attn.c_attn.bias")) b = to_f32(*bt);
            if (nvl_upload_gpt2_qkv(m, l, w.data(), b.empty() ? nullptr : b.data())) throw std::runtime_error(nvl_last_error(m));
            up2d(m, NVL_T_WO, l, st.need(p + ".attn.c_proj.weight"), IO);
            if (const StTensor* bo = st.find(p + ".attn.c_proj.bias")) up1d(m, NVL_T_BO, l, *bo);
            up2d(m, NVL_T_W1, l, st.need(p + ".mlp.c_fc.weight"), IO);
            up2d(m, NVL_T_W2, l, st.need(p + ".mlp.c_proj.weight"), IO);
            // (the FFN biases are looked up as "...c_fc.weight.bias" by the reference and never found: :559-560 — not loaded)
            load_norm(m, st, p + ".ln_1.weight", NVL_T_ATTN_NORM_W, NVL_T_ATTN_NORM_B, l);
            load_norm(m, st, p + ".ln_2.weight", NVL_T_FFN_NORM_W, NVL_T_FFN_NORM_B, l);
        }
        load_norm(m, st, "ln_f.weight", NVL_T_FINAL_NORM_W, NVL_T_FINAL_NORM_B, 0);
    } else if (falcon) {                                                       // GetFalconMapping (:81-98): PyTorch [out, in]
        up2d(m, NVL_T_TOK_EMB, 0, st.need("transformer.word_embeddings.weight"), IO);
        for (int l = 0; l < c.num_layers; l++) {
            const std::string p = "transformer.h." + std::to_string(l);
            const StTensor& qkv = st.need(p + ".self_attention.query_key_value.weight");   // [(nH+2)*hd, H]
            if (qkv.shape.size() != 2) throw std::runtime_error("query_key_value: 2-D expected");
            const int64_t R = qkv.shape[0], K = qkv.shape[1];
            std::vector<float> t((size_t)(R * K));                             // Transpose BEFORE splitting (:366-369)
            for (int64_t r = 0; r < R; r++)
                for (int64_t k = 0; k < K; k++) t[(size_t)(k * R + r)] = nvl_loader::f32_of(qkv, r * K + k);
            if (nvl_upload_falcon_qkv(m, l, t.data())) throw std::runtime_error(nvl_last_error(m));
            up2d(m, NVL_T_WO, l, st.need(p + ".self_attention.dense.weight"), OI);
            up2d(m, NVL_T_W1, l, st.need(p + ".mlp.dense_h_to_4h.weight"), OI);
            up2d(m, NVL_T_W2, l, st.need(p + ".mlp.dense_4h_to_h.weight"), OI);
            load_norm(m, st, p + ".input_layernorm.weight", NVL_T_ATTN_NORM_W, NVL_T_ATTN_NORM_B, l);   // parallel block: InputLN
        }
        load_norm(m, st, "transformer.ln_f.weight", NVL_T_FINAL_NORM_W, NVL_T_FINAL_NORM_B, 0);
        if (!c.tied_embedding) if (const StTensor* lm = st.find("lm_head.weight")) up2d(m, NVL_T_LM_HEAD, 0, *lm, OI);
    } else {                                                                   // GetLlamaMapping / GetGraniteMoEMapping (:101-141)
        up2d(m, NVL_T_TOK_EMB, 0, st.need("model.embed_tokens.weight"), IO);
        for (int l = 0; l < c.num_layers; l++) {
            const std::string p = "model.layers." + std::to_string(l);
            const bool is_mamba = l < 128 && ((c.mamba_layer_mask[l >> 6] >> (l & 63)) & 1);
            const bool hybrid = (c.mamba_layer_mask[0] | c.mamba_layer_mask[1]) != 0;
            if (hybrid) {
                // GetGraniteMapping (:145-181) + loadMamba2 (:461-512): Mamba2 tensors keep the checkpoint's layouts; every block
                // of the hybrid has the shared MLP (shared_mlp.input_linear = gate | up already fused, output_linear)
                if (is_mamba) {
                    up2d(m, NVL_T_MAMBA_IN_PROJ, l, st.need(p + ".mamba.in_proj.weight"), OI);
                    up2d(m, NVL_T_MAMBA_OUT_PROJ, l, st.need(p + ".mamba.out_proj.weight"), OI);
                    up1d(m, NVL_T_MAMBA_CONV_W, l, st.need(p + ".mamba.conv1d.weight"));          // [conv_dim, 1, K]
                    if (const StTensor* t = st.find(p + ".mamba.conv1d.bias")) up1d(m, NVL_T_MAMBA_CONV_B, l, *t);
                    up1d(m, NVL_T_MAMBA_A_LOG, l, st.need(p + ".mamba.A_log"));
                    up1d(m, NVL_T_MAMBA_D, l, st.need(p + ".mamba.D"));
                    up1d(m, NVL_T_MAMBA_DT_BIAS, l, st.need(p + ".mamba.dt_bias"));
                    up1d(m, NVL_T_MAMBA_NORM, l, st.need(p + ".mamba.norm.weight"));
                } else {
                    up2d(m, NVL_T_WQ, l, st.need(p + ".self_attn.q_proj.weight"), OI);
                    up2d(m, NVL_T_WK, l, st.need(p + ".self_attn.k_proj.weight"), OI);
                    up2d(m, NVL_T_WV, l, st.need(p + ".self_attn.v_proj.weight"), OI);
                    up2d(m, NVL_T_WO, l, st.need(p + ".self_attn.o_proj.weight"), OI);
                }
                up2d(m, NVL_T_W1, l, st.need(p + ".shared_mlp.input_linear.weight"), OI);
                up2d(m, NVL_T_W2, l, st.need(p + ".shared_mlp.output_linear.weight"), OI);
                load_norm(m, st, p + ".input_layernorm.weight", NVL_T_ATTN_NORM_W, NVL_T_ATTN_NORM_B, l);
                load_norm(m, st, p + ".post_attention_layernorm.weight", NVL_T_FFN_NORM_W, NVL_T_FFN_NORM_B, l);
                continue;
            }
            up2d(m, NVL_T_WQ, l, st.need(p + ".self_attn.q_proj.weight"), OI);
            up2d(m, NVL_T_WK, l, st.need(p + ".self_attn.k_proj.weight"), OI);
            up2d(m, NVL_T_WV, l, st.need(p + ".self_attn.v_proj.weight"), OI);
            up2d(m, NVL_T_WO, l, st.need(p + ".self_attn.o_proj.weight"), OI);
            if (c.use_moe) {                                                   // loadMoE (:566-592)
                up2d(m, NVL_T_ROUTER, l, st.need(p + ".block_sparse_moe.router.layer.weight"), OI);   // [E, H]: "always transpose"
                for (int which = 0; which < 2; which++) {
                    const StTensor& e = st.need(p + (which ? ".block_sparse_moe.output_linear.weight" : ".block_sparse_moe.input_linear.weight"));
                    if (e.shape.size() != 3) throw std::runtime_error("expert weights: 3-D [E, out, in] expected");
                    const int rc = nvl_upload_tensor(m, which ? NVL_T_MOE_OUT : NVL_T_MOE_IN, l, e.data, e.dtype,
                                                     e.shape[0] * e.shape[1], e.shape[2], IO);
                    if (rc) throw std::runtime_error(nvl_last_error(m));
                }
            } else {                                                           // loadFFN (:513-563): gate | up -> W1
                const StTensor& g = st.need(p + ".mlp.gate_proj.weight");
                const StTensor* u = st.find(p + ".mlp.up_proj.weight");
                if (u) {
                    if (u->dtype != g.dtype || u->shape != g.shape || g.shape.size() != 2) throw std::runtime_error("gate_proj / up_proj mismatch");
                    std::vector<uint8_t> cat(g.bytes + u->bytes);              // [2F, H] in the checkpoint's dtype == ([H, F] | [H, F])^T
                    memcpy(cat.data(), g.data, g.bytes);
                    memcpy(cat.data() + g.bytes, u->data, u->bytes);
                    const int rc = nvl_upload_tensor(m, NVL_T_W1, l, cat.data(), g.dtype, 2 * g.shape[0], g.shape[1], OI);
                    if (rc) throw std::runtime_error(nvl_last_error(m));
                } else {
                    up2d(m, NVL_T_W1, l, g, OI);                               // a checkpoint with the pair already fused
                }
                up2d(m, NVL_T_W2, l, st.need(p + ".mlp.down_proj.weight"), OI);
            }
            load_norm(m, st, p + ".input_layernorm.weight", NVL_T_ATTN_NORM_W, NVL_T_ATTN_NORM_B, l);
            load_norm(m, st, p + ".post_attention_layernorm.weight", NVL_T_FFN_NORM_W, NVL_T_FFN_NORM_B, l);
        }
        load_norm(m, st, "model.norm.weight", NVL_T_FINAL_NORM_W, NVL_T_FINAL_NORM_B, 0);
        // LM head (:245-258): own matrix unless tied; a missing one falls back to the transposed embedding
        if (!c.tied_embedding) if (const StTensor* lm = st.find("lm_head.weight")) up2d(m, NVL_T_LM_HEAD, 0, *lm, OI);
    }
    NVL_HIP(hipStreamSynchronize(m->stream));   // the mmaps go away when `st` does
    return NVL_OK;
    NVL_CATCH(m)
}

// LoadModelConfig (generic_loader.go:808-972) on top of the New*Config templates (config.go:125-376)
extern "C" int nvl_load_config_json(const char* path, nvl_model_config* out) {
    if (!path || !out) return NVL_ERR_INVALID;
    try {
        const std::string txt = nvl_loader::read_text(path);
        const JVal raw = nvl_loader::JParser(txt.c_str(), txt.size()).parse();
        if (raw.kind != JVal::OBJ) throw std::runtime_error("config is not a JSON object");
        auto str = [&](const char* k) { const JVal* v = raw.get(k); return v && v->kind == JVal::STR ? v->str : std::string(); };
        auto num = [&](const char* k, double& dst) { const JVal* v = raw.get(k); if (v && v->kind == JVal::NUM) { dst = v->num; return true; } return false; };
        nvl_model_config c;
        memset(&c, 0, sizeof c);
        // ---- templates (config.go:125-376); `architecture` first, then model_type (:822-836, :975-1007), default GPT-2
        std::string arch = str("architecture");
        if (const LayeredArch* la = layered_arch(arch)) {       // sizes and constants come from the file
            c.vocab_size = need_int(&raw, "vocab", "config: "); c.hidden = need_int(&raw, "width", "config: ");
            c.num_layers = (int)parse_layers(raw, *la).size();
            c.norm_eps = (float)need_num(raw.get("norm"), "eps", "config: norm: ");
            c.max_seq_len = raw.get("max_positions") ? need_int(&raw, "max_positions", "config: ") : 4096;
            if (la->position_type == NVL_POS_LEARNED && !raw.get("max_positions")) throw std::runtime_error("config: number 'max_positions' expected");
            c.attention_type = NVL_ATTN_GQA; c.norm_type = la->norm_type; c.position_type = la->position_type;
            if (const JVal* ts = raw.get("token_side")) if (ts->kind == JVal::OBJ && la->block_style == NVL_BLOCK_PARALLEL) c.side_dim = need_int(ts, "dim", "config: token_side: ");
            c.activation_type = la->activation; c.block_style = la->block_style; c.norm_weight_offset = la->norm_offset;
            double cap;
            if (num("logit_softcap", cap)) c.logit_softcap = (float)cap;
            if (la->block_style == NVL_BLOCK_SUM_NORM) {
                c.stream_scale = (float)need_num(&raw, "postln_alpha", "config: "); c.token_shift = 1;
                c.embedding_multiplier = (float)need_num(raw.get("embedding"), "scale", "config: embedding: ");
            }
            *out = c;
            return NVL_OK;
        }
        const std::string mt = str("model_type");
        if (arch != "gpt2" && arch != "falcon" && arch != "llama") {
            if (mt == "gpt2") arch = "gpt2";
            else if (mt == "falcon" || mt == "RefinedWeb" || mt == "RefinedWebModel") arch = "falcon";
            else if (mt == "llama" || mt == "LlamaForCausalLM") arch = "llama";
            else if (mt == "granitemoe") arch = "granitemoe";
            else if (mt == "granitemoehybrid") arch = "granitehybrid";
            else arch = "gpt2";
        }
        c.rope_base = 10000.0; c.norm_eps = 1e-5f;
        if (arch == "gpt2") {            // NewGPT2Config (config.go:125-148)
            c.vocab_size = 50257; c.hidden = 768; c.num_layers = 12; c.num_heads = 12; c.num_kv_heads = 12; c.head_dim = 64; c.ffn_dim = 3072;
            c.max_seq_len = 1024; c.attention_type = NVL_ATTN_MHA; c.norm_type = NVL_NORM_LAYER; c.position_type = NVL_POS_LEARNED;
            c.activation_type = NVL_ACT_GELU; c.block_style = NVL_BLOCK_SEQUENTIAL; c.tied_embedding = 1;
        } else if (arch == "falcon") {   // NewFalconConfig("7b") (config.go:151-194)
            c.vocab_size = 65024; c.hidden = 4544; c.num_layers = 32; c.num_heads = 71; c.num_kv_heads = 1; c.head_dim = 64; c.ffn_dim = 18176;
            c.max_seq_len = 2048; c.attention_type = NVL_ATTN_MQA; c.norm_type = NVL_NORM_LAYER; c.position_type = NVL_POS_ROPE;
            c.activation_type = NVL_ACT_GELU; c.block_style = NVL_BLOCK_PARALLEL; c.tied_embedding = 0;
        } else if (arch == "llama") {    // NewLlamaConfig("7b") (config.go:197-242)
            c.vocab_size = 32000; c.hidden = 4096; c.num_layers = 32; c.num_heads = 32; c.num_kv_heads = 8; c.head_dim = 128; c.ffn_dim = 11008;
            c.max_seq_len = 4096; c.attention_type = NVL_ATTN_GQA; c.norm_type = NVL_NORM_RMS; c.position_type = NVL_POS_ROPE;
            c.activation_type = NVL_ACT_SWIGLU; c.block_style = NVL_BLOCK_SEQUENTIAL; c.tied_embedding = 0; c.norm_eps = 1e-6f;
        } else if (arch == "granitehybrid") {   // NewGraniteConfig (config.go:241-330): "350m" when hidden_size <= 800, else "1b" (:993-1001)
            double hs = 768;
            num("hidden_size", hs);
            const bool small = hs <= 800;
            c.vocab_size = 49152; c.hidden = small ? 768 : 1536; c.num_layers = small ? 32 : 40; c.num_heads = 12; c.num_kv_heads = 4;
            c.head_dim = small ? 64 : 128; c.ffn_dim = small ? 2048 : 4096; c.max_seq_len = small ? 32768 : 128000;
            c.attention_type = NVL_ATTN_GQA; c.norm_type = NVL_NORM_RMS; c.position_type = NVL_POS_NONE; c.activation_type = NVL_ACT_SWIGLU;
            c.block_style = NVL_BLOCK_SEQUENTIAL; c.tied_embedding = 1; c.norm_eps = 1e-5f;
            c.mamba_expand = 2; c.mamba_state_size = 128; c.mamba_conv_kernel = 4; c.mamba_num_heads = 48; c.mamba_head_dim = small ? 32 : 0;
            c.mamba_n_groups = small ? 1 : 8;
            const int nl = c.num_layers;
            for (int i = 0; i < nl; i++) c.mamba_layer_mask[i >> 6] |= 1ull << (i & 63);
            if (small) for (int a : {10, 13, 17, 27}) c.mamba_layer_mask[0] &= ~(1ull << a);      // template pattern, layer_types overrides
        } else {                         // NewGraniteMoEConfig("350m") (config.go:333-376); use_moe comes from num_local_experts
            c.vocab_size = 49155; c.hidden = 1024; c.num_layers = 24; c.num_heads = 16; c.num_kv_heads = 8; c.head_dim = 64; c.ffn_dim = 512;
            c.max_seq_len = 4096; c.attention_type = NVL_ATTN_GQA; c.norm_type = NVL_NORM_RMS; c.position_type = NVL_POS_ROPE;
            c.activation_type = NVL_ACT_SWIGLU; c.block_style = NVL_BLOCK_SEQUENTIAL; c.tied_embedding = 1; c.norm_eps = 1e-6f;
            c.use_moe = 0; c.num_experts = 32; c.num_experts_per_tok = 8;
        }
        // ---- overrides, in the reference's order (:838-968)
        double v;
        if (num("vocab_size", v)) c.vocab_size = (int)v;
        if (num("n_embd", v)) c.hidden = (int)v;
        if (num("hidden_size", v)) c.hidden = (int)v;
        if (num("n_layer", v)) c.num_layers = (int)v;
        if (num("num_hidden_layers", v)) c.num_layers = (int)v;
        if (num("num_layers", v)) c.num_layers = (int)v;
        if (num("n_head", v)) c.num_heads = (int)v;
        if (num("num_attention_heads", v)) c.num_heads = (int)v;
        if (num("num_heads", v)) c.num_heads = (int)v;
        if (num("num_key_value_heads", v)) c.num_kv_heads = (int)v;
        if (num("num_kv_heads", v)) c.num_kv_heads = (int)v;
        if (const JVal* mq = raw.get("multi_query")) if (mq->kind == JVal::BOOL && mq->b) c.num_kv_heads = 1;
        if (num("head_dim", v)) c.head_dim = (int)v;
        if (c.head_dim == 0 && c.hidden > 0 && c.num_heads > 0) c.head_dim = c.hidden / c.num_heads;   // (:884-886)
        if (num("rope_theta", v)) c.rope_base = v;
        if (num("rms_norm_eps", v)) c.norm_eps = (float)v;
        if (num("layer_norm_epsilon", v)) c.norm_eps = (float)v;
        if (num("n_inner", v)) c.ffn_dim = (int)v;
        if (num("intermediate_size", v)) c.ffn_dim = (int)v;
        if (c.ffn_dim == 0 && c.hidden > 0) c.ffn_dim = 4 * c.hidden;
        if (const JVal* t = raw.get("tie_word_embeddings")) if (t->kind == JVal::BOOL) c.tied_embedding = t->b ? 1 : 0;
        if (num("embedding_multiplier", v)) c.embedding_multiplier = (float)v;
        if (num("attention_multiplier", v)) c.attention_multiplier = (float)v;
        if (num("residual_multiplier", v)) c.residual_multiplier = (float)v;
        if (num("logits_scaling", v)) c.logits_scaling = (float)v;
        // Granite hybrid fields (:917-946)
        if (const JVal* lt = raw.get("layer_types")) if (lt->kind == JVal::ARR) {
            c.mamba_layer_mask[0] = c.mamba_layer_mask[1] = 0;
            for (size_t i = 0; i < lt->arr.size() && i < 128; i++)
                if (lt->arr[i].kind == JVal::STR && (lt->arr[i].str == "mamba" || lt->arr[i].str == "mamba2"))
                    c.mamba_layer_mask[i >> 6] |= 1ull << (i & 63);
        }
        if (num("mamba_expand", v)) c.mamba_expand = (int)v;
        if (num("mamba_d_state", v)) c.mamba_state_size = (int)v;
        if (num("mamba_n_heads", v)) c.mamba_num_heads = (int)v;
        if (num("mamba_d_head", v)) c.mamba_head_dim = (int)v;
        if (num("mamba_n_groups", v)) c.mamba_n_groups = (int)v;
        if (num("mamba_d_conv", v)) c.mamba_conv_kernel = (int)v;
        // (the reference sets UseMoE for ANY num_local_experts, 0 included; a hybrid checkpoint says 0 and its blocks
        // run the dense shared MLP: 0 experts is treated as "no MoE" here)
        if (num("num_local_experts", v)) { c.num_experts = (int)v; c.use_moe = v > 0 ? 1 : 0; }
        if (num("num_experts_per_tok", v)) c.num_experts_per_tok = (int)v;
        *out = c;
        return NVL_OK;
    } catch (const std::exception& e) {
        g_create_err = std::string("nvl_load_config_json: ") + e.what();
        return NVL_ERR_INVALID;
    }
}
