// Readers and registry of model_registry.h.
#include "model_registry.h"

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cctype>
#include <cstdio>
#include <cstdlib>
#include <cstring>
#include <fstream>
#include <sstream>

#include "host_util.h"

namespace xfthost {

namespace {

[[noreturn]] void broken(const std::string &what) {
    printf("Could not load the model: %s\n", what.c_str());
    exit(-1);
}

struct Parser {
    const char *p, *end;
    std::string error;
    int depth = 0;

    bool fail(const char *what) {
        if (error.empty()) error = what;
        return false;
    }
    void space() {
        while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) ++p;
    }
    bool word(const char *w) {
        const size_t n = strlen(w);
        if ((size_t)(end - p) < n || strncmp(p, w, n) != 0) return fail("unknown word");
        p += n;
        return true;
    }
    static void utf8(std::string &s, unsigned c) {
        if (c < 0x80) s += (char)c;
        else if (c < 0x800) s += (char)(0xC0 | (c >> 6)), s += (char)(0x80 | (c & 63));
        else if (c < 0x10000) s += (char)(0xE0 | (c >> 12)), s += (char)(0x80 | ((c >> 6) & 63)), s += (char)(0x80 | (c & 63));
        else s += (char)(0xF0 | (c >> 18)), s += (char)(0x80 | ((c >> 12) & 63)), s += (char)(0x80 | ((c >> 6) & 63)), s += (char)(0x80 | (c & 63));
    }
    bool hex4(unsigned &c) {
        c = 0;
        for (int i = 0; i < 4; ++i) {
            if (p >= end || !isxdigit((unsigned char)*p)) return fail("bad \\u escape");
            const char d = *p++;
            c = c * 16 + (unsigned)(d <= '9' ? d - '0' : (d | 32) - 'a' + 10);
        }
        return true;
    }
    bool str(std::string &out) {
        ++p; // the quote
        while (p < end && *p != '"') {
            if (*p != '\\') {
                out += *p++;
                continue;
            }
            if (++p >= end) break;
            const char e = *p++;
            switch (e) {
                case 'n': out += '\n'; break;
                case 't': out += '\t'; break;
                case 'r': out += '\r'; break;
                case 'b': out += '\b'; break;
                case 'f': out += '\f'; break;
                case 'u': {
                    unsigned c;
                    if (!hex4(c)) return false;
                    if (c >= 0xD800 && c < 0xDC00 && end - p >= 6 && p[0] == '\\' && p[1] == 'u') {
                        unsigned lo;
                        p += 2;
                        if (!hex4(lo)) return false;
                        c = 0x10000 + ((c - 0xD800) << 10) + (lo - 0xDC00);
                    }
                    utf8(out, c);
                    break;
                }
                default: out += e;
            }
        }
        if (p >= end) return fail("unterminated string");
        ++p;
        return true;
    }
    bool value(Json &v) {
        space();
        if (p >= end) return fail("unexpected end");
        if (++depth > 64) return fail("nested too deeply");
        bool ok = true;
        switch (*p) {
            case '{':
                v.kind = Json::Object;
                ++p, space();
                if (p < end && *p == '}') {
                    ++p;
                    break;
                }
                for (;;) {
                    space();
                    if (p >= end || *p != '"') return fail("a key is missing");
                    std::string key;
                    if (!str(key)) return false;
                    space();
                    if (p >= end || *p != ':') return fail("a colon is missing");
                    ++p;
                    if (!value(v.fields[key])) return false;
                    space();
                    if (p < end && *p == ',') {
                        ++p;
                        continue;
                    }
                    if (p < end && *p == '}') {
                        ++p;
                        break;
                    }
                    return fail("an object does not end");
                }
                break;
            case '[':
                v.kind = Json::Array;
                ++p, space();
                if (p < end && *p == ']') {
                    ++p;
                    break;
                }
                for (;;) {
                    v.items.emplace_back();
                    if (!value(v.items.back())) return false;
                    space();
                    if (p < end && *p == ',') {
                        ++p;
                        continue;
                    }
                    if (p < end && *p == ']') {
                        ++p;
                        break;
                    }
                    return fail("an array does not end");
                }
                break;
            case '"': v.kind = Json::String, ok = str(v.text); break;
            case 't': v.kind = Json::Bool, v.flag = true, ok = word("true"); break;
            case 'f': v.kind = Json::Bool, ok = word("false"); break;
            case 'n': ok = word("null"); break;
            default: {
                const std::string rest(p, end - p < 64 ? end : p + 64);
                char *stop = nullptr;
                v.kind = Json::Number;
                v.number = strtod(rest.c_str(), &stop);
                if (stop == rest.c_str()) return fail("not a value");
                p += stop - rest.c_str();
            }
        }
        --depth;
        return ok;
    }
};

std::string read_file(const std::string &path, bool &ok) {
    std::ifstream f(path, std::ios::binary);
    ok = (bool)f;
    std::stringstream s;
    if (ok) s << f.rdbuf();
    return s.str();
}

} // namespace

bool Json::parse(const std::string &src, Json &out, std::string &error) {
    Parser ps {src.data(), src.data() + src.size(), "", 0};
    out = Json();
    bool ok = ps.value(out);
    ps.space();
    if (ok && ps.p != ps.end) ok = ps.fail("text behind the value");
    error = ps.error;
    return ok;
}

bool Json::has(const std::string &key) const {
    auto it = fields.find(key);
    return it != fields.end() && it->second.kind != Null;
}
const Json &Json::at(const std::string &key) const {
    auto it = fields.find(key);
    if (it == fields.end()) broken("config.json lacks '" + key + "'");
    return it->second;
}
long Json::integer(const std::string &key) const {
    const double v = real(key);
    if (v != (double)(long)v) broken("'" + key + "' of config.json is not a whole number");
    return (long)v;
}
double Json::real(const std::string &key) const {
    const Json &v = at(key);
    if (v.kind != Number) broken("'" + key + "' of config.json is not a number");
    return v.number;
}
const std::string &Json::string(const std::string &key) const {
    const Json &v = at(key);
    if (v.kind != String) broken("'" + key + "' of config.json is not a string");
    return v.text;
}

long TensorRef::count() const {
    long n = 1;
    for (long d : shape) n *= d;
    return n;
}

SafeTensors::~SafeTensors() {
    if (base) munmap(base, length);
}

bool SafeTensors::open(const std::string &path, std::string &error) {
    const int fd = ::open(path.c_str(), O_RDONLY);
    struct stat st;
    if (fd < 0 || fstat(fd, &st) != 0 || st.st_size < 8) {
        if (fd >= 0) close(fd);
        error = "cannot read " + path;
        return false;
    }
    length = (size_t)st.st_size;
    base = mmap(nullptr, length, PROT_READ, MAP_PRIVATE, fd, 0);
    close(fd);
    if (base == MAP_FAILED) {
        base = nullptr;
        error = "cannot map " + path;
        return false;
    }
    const unsigned char *b = (const unsigned char *)base;
    uint64_t header = 0;
    for (int i = 7; i >= 0; --i) header = header << 8 | b[i];
    if (header > length - 8) {
        error = path + " is shorter than its header says";
        return false;
    }
    Json j;
    if (!Json::parse(std::string((const char *)b + 8, (size_t)header), j, error) || j.kind != Json::Object) {
        error = "header of " + path + ": " + error;
        return false;
    }
    const size_t room = length - 8 - (size_t)header;
    for (auto &kv : j.fields) {
        if (kv.first == "__metadata__") continue;
        TensorRef t;
        t.dtype = kv.second.string("dtype");
        long n = 1;
        for (const Json &d : kv.second.at("shape").items) t.shape.push_back((long)d.number), n *= (long)d.number;
        const Json &off = kv.second.at("data_offsets");
        const size_t width = t.dtype == "BF16" || t.dtype == "F16" || t.dtype == "I16" ? 2 : t.dtype == "F32" || t.dtype == "I32" ? 4 : t.dtype == "F64" || t.dtype == "I64" ? 8 : 1;
        if (off.items.size() != 2 || off.items[0].number < 0 || off.items[1].number < off.items[0].number || off.items[1].number > (double)room
                || n < 0 || (double)n * width != off.items[1].number - off.items[0].number) {
            error = "tensor " + kv.first + " of " + path + " does not fit the file";
            return false;
        }
        t.data = b + 8 + header + (size_t)off.items[0].number;
        t.bytes = (size_t)(off.items[1].number - off.items[0].number);
        tensors[kv.first] = t;
    }
    return true;
}

const TensorRef *SafeTensors::find(const std::string &name) const {
    auto it = tensors.find(name);
    return it == tensors.end() ? nullptr : &it->second;
}

namespace {

long first_dim(const SafeTensors &w, const std::string &name) {
    const TensorRef *t = w.find(name);
    if (!t || t->shape.empty()) broken("model.safetensors lacks " + name);
    return t->shape[0];
}

// ---- Pinepel: latent attention (windowed with interleaved rotation, or over everything with a sink and half rotation) and a
// channel-wise gated delta rule, clamped gated feed-forwards, a norm on both sides of every sublayer, layers run in a loop ----
PlanSpec pinepel(const Json &c, const SafeTensors &w) {
    PlanSpec s;
    s.cfg.hidden = (int)c.integer("width");
    s.cfg.vocab = (int)c.integer("vocab");
    s.cfg.eps = (float)c.at("norm").real("eps");
    s.cfg.logit_scale = (float)c.real("logit_scale");
    s.cfg.loop_times = 1;
    if (c.has("loop")) {
        const Json &l = c.at("loop");
        s.cfg.loop_start = (int)l.integer("start"), s.cfg.loop_stop = (int)l.integer("stop"), s.cfg.loop_times = (int)l.integer("times");
    }
    const Json &layers = c.at("layers");
    for (size_t i = 0; i < layers.items.size(); ++i) {
        const Json &e = layers.items[i], &m = e.at("mixer");
        const std::string &type = e.string("type"), mix = "l" + std::to_string(i) + ".mix.";
        xfthip_plan_layer L {};
        L.heads = (int)m.integer("heads"), L.dim = (int)m.integer("dim"), L.vdim = (int)m.integer("vdim");
        if (type == "latent_attention" || type == "latent_attention_2") {
            const bool windowed = type == "latent_attention";
            L.mixer = XFTHIP_MIXER_LATENT;
            L.kv_rank = (int)m.integer("kv_rank"), L.q_rank = (int)m.integer("q_rank"), L.rot_dim = (int)m.integer("rot_dim");
            L.scale = (float)m.real("scale");
            L.rot_base = m.at("rot").real("base");
            if (m.at("rot").integer("dims") != L.rot_dim) broken("layer " + std::to_string(i) + ": rot.dims differs from rot_dim");
            L.rot_interleaved = windowed ? 1 : 0;
            L.window = windowed ? (int)m.at("mask").integer("size") : 0;
            if (windowed && L.window < 1) broken("layer " + std::to_string(i) + ": an empty window");
            L.has_sink = windowed ? 0 : 1;
        } else if (type == "channel_delta") {
            L.mixer = XFTHIP_MIXER_DELTA;
            L.kv_heads = (int)m.integer("kv_heads"), L.taps = (int)m.integer("conv");
            L.decay_rank = (int)first_dim(w, mix + "a1"), L.gate_rank = (int)first_dim(w, mix + "g1");
        } else {
            broken("layer type '" + type + "' of config.json is not known");
        }
        if (e.has("mlp")) {
            const Json &f = e.at("mlp");
            if (f.string("kind") != "dense") broken("feed-forward '" + f.string("kind") + "' of config.json is not known");
            L.inter = (int)f.integer("ff");
            L.glu_limit = (float)f.real("limit");
            L.glu_alpha = 1.702f;
        }
        s.layers.push_back(L);
    }
    s.cfg.layers = (int)s.layers.size();
    return s;
}

// ---- Veterax: grouped attention with normed heads, a sink and values mixed with an earlier layer's, beside routed experts (some of
// them the identity) and a shared one, both reading the residual through a tanh in the place of a norm; a second embedding of
// the token joins behind every layer ----
PlanSpec veterax(const Json &c, const SafeTensors &) {
    PlanSpec s;
    s.cfg.hidden = (int)c.integer("width");
    s.cfg.vocab = (int)c.integer("vocab");
    s.cfg.eps = (float)c.at("norm").real("eps");
    s.cfg.logit_scale = 1.0f;
    s.cfg.loop_times = 1;
    s.cfg.block = XFTHIP_BLOCK_PARALLEL, s.cfg.norm = XFTHIP_NORM_DYNAMIC_TANH, s.cfg.tied_head = 1;
    if (c.has("token_side")) s.cfg.side_dim = (int)c.at("token_side").integer("dim");
    const Json &layers = c.at("layers");
    for (size_t i = 0; i < layers.items.size(); ++i) {
        const std::string at = "layer " + std::to_string(i) + ": ";
        const Json &e = layers.items[i], &m = e.at("mixer");
        if (e.string("type") != "attention") broken("layer type '" + e.string("type") + "' of config.json is not known");
        xfthip_plan_layer L {};
        L.mixer = XFTHIP_MIXER_GROUPED;
        L.heads = (int)m.integer("heads"), L.kv_heads = (int)m.integer("kv_heads"), L.dim = (int)m.integer("dim"), L.vdim = (int)m.integer("vdim");
        L.scale = (float)m.real("scale");
        L.has_sink = 1, L.qk_norm = 1;
        L.v_mix = m.has("v_mix") && m.at("v_mix").flag ? 1 : 0;
        const Json &rot = m.at("rot");
        L.rot_dim = (int)rot.integer("dims"), L.rot_base = rot.real("base"), L.rot_interleaved = 1;
        if (rot.has("scaling")) {
            const Json &x = rot.at("scaling");
            L.rot_factor = x.real("factor"), L.rot_original = x.real("original"), L.rot_fast = x.real("fast"), L.rot_slow = x.real("slow");
            if (!(L.rot_factor > 0.0)) broken(at + "a rotation scaled by nothing");
        }
        if (e.has("mlp")) {
            const Json &f = e.at("mlp");
            if (f.string("kind") != "moe") broken("feed-forward '" + f.string("kind") + "' of config.json is not known");
            const Json &r = f.at("router"), &x = f.at("expert");
            L.experts = (int)r.integer("experts"), L.top = (int)r.integer("top");
            L.identity = r.has("identity") ? (int)r.integer("identity") : 0;
            if (L.experts < 1) broken(at + "a router without experts");
            L.expert_inter = (int)x.integer("ff"), L.expert_limit = (float)x.real("limit");
            L.glu_alpha = 1.702f;
            if (f.has("shared")) L.inter = (int)f.at("shared").integer("ff"), L.glu_limit = (float)f.at("shared").real("limit");
        }
        s.layers.push_back(L);
    }
    s.cfg.layers = (int)s.layers.size();
    return s;
}

// ---- Duvadra: pre-norm layers whose mixer is chunked attention with capped scores and a cost of distance (its keys and values
// perhaps an earlier layer's), or a windowed attention beside a recurrence: with a sink beside a gated delta rule, or with keys that
// serve as values beside a gated linear recurrence; dense or routed feed-forwards, embeddings of token pairs ----
PlanSpec duvadra(const Json &c, const SafeTensors &) {
    PlanSpec s;
    s.cfg.hidden = (int)c.integer("width");
    s.cfg.vocab = (int)c.integer("vocab");
    s.cfg.eps = (float)c.at("norm").real("eps");
    s.cfg.logit_scale = 1.0f;
    s.cfg.loop_times = 1;
    s.cfg.block = XFTHIP_BLOCK_SERIAL, s.cfg.norm = XFTHIP_NORM_RMS;
    s.cfg.residual_mult = (float)c.real("residual_mult");
    if (c.has("logit_softcap")) s.cfg.logit_softcap = (float)c.real("logit_softcap");
    const Json &emb = c.at("embedding");
    s.cfg.embed_scale = (float)emb.real("scale");
    if (emb.has("bigram")) {
        const Json &b = emb.at("bigram");
        s.cfg.bigram_buckets = b.integer("buckets"), s.cfg.bigram_mul_prev = b.integer("mul_prev"), s.cfg.bigram_mul_cur = b.integer("mul_cur");
    }
    auto sizes = [](const Json &m) {
        xfthip_plan_layer L {};
        L.heads = (int)m.integer("heads"), L.kv_heads = (int)m.integer("kv_heads"), L.dim = (int)m.integer("dim"), L.vdim = (int)m.integer("vdim");
        return L;
    };
    const Json &layers = c.at("layers");
    for (size_t i = 0; i < layers.items.size(); ++i) {
        const std::string at = "layer " + std::to_string(i) + ": ";
        const Json &e = layers.items[i], &m = e.at("mixer");
        const std::string &type = e.string("type");
        const bool one = type == "attention", first = type == "parallel";
        if (!one && !first && type != "parallel_2") broken("layer type '" + type + "' of config.json is not known");
        const Json &a = one ? m : m.at("left");
        xfthip_plan_layer L = sizes(a), R {};
        L.mixer = XFTHIP_MIXER_GROUPED;
        L.scale = (float)a.real("scale");
        const int span = (int)a.at("mask").integer("size");
        if (span < 1) broken(at + "an empty window or chunk");
        (one ? L.chunk : L.window) = span;
        if (one) {
            L.softcap = (float)a.real("softcap");
            L.distance_bias = 1, L.out_gate = XFTHIP_GATE_HEAD;
            if (a.has("kv_from")) {
                const long j = a.integer("kv_from");
                if (j < 0 || j >= (long)i) broken(at + "keys and values of a layer that is not before it");
                L.kv_from = s.record[(size_t)j] + 1;
            }
        } else {
            const Json &r = m.at("right");
            L.out_gate = XFTHIP_GATE_ELEMENT;
            L.scaled = 1, L.mix_scale = (float)m.real("left_scale");
            if (first) {
                L.qkv_bias = 1, L.has_sink = 1;
                R = sizes(r);
                R.mixer = XFTHIP_MIXER_DELTA;
            } else {
                L.key_values = 1, L.qk_norm = XFTHIP_QK_NORM_ALL;
                L.rot_dim = (int)a.at("rot").integer("dims"), L.rot_base = a.at("rot").real("base"), L.rot_interleaved = 1;
                R.mixer = XFTHIP_MIXER_UNIT;
                const long width = r.integer("width");
                R.heads = (int)r.integer("blocks");
                if (R.heads < 1 || width % R.heads) broken(at + "a recurrence that does not divide into its blocks");
                R.dim = R.vdim = (int)(width / R.heads);
            }
            R.taps = (int)r.integer("conv");
            R.beside = 1, R.scaled = 1, R.mix_scale = (float)m.real("right_scale");
        }
        if (e.has("mlp")) {
            const Json &f = e.at("mlp");
            const std::string &kind = f.string("kind");
            if (kind == "dense") {
                L.inter = (int)f.integer("ff"), L.glu_limit = (float)f.real("limit"), L.glu_alpha = 1.702f;
            } else if (kind == "moe") {
                const Json &r = f.at("router"), &g = r.at("groups");
                L.experts = (int)r.integer("experts"), L.top = (int)r.integer("top"), L.expert_inter = (int)f.at("expert").integer("ff");
                if (L.experts < 1) broken(at + "a router without experts");
                L.router = XFTHIP_ROUTE_SIGMOID_GROUPS;
                L.route_groups = (int)g.integer("count"), L.route_keep = (int)g.integer("keep"), L.route_scale = (float)r.real("scale");
            } else {
                broken("feed-forward '" + kind + "' of config.json is not known");
            }
        }
        s.record.push_back((int)s.layers.size());
        s.layers.push_back(L);
        if (!one) s.layers.push_back(R);
    }
    s.cfg.layers = (int)s.layers.size();
    return s;
}

// ---- Balenex: norms in groups on both sides of every sublayer; a windowed attention with unit heads that sees older tokens as means of blocks, or
// an attention with filters, turned values and a window beside the first tokens next to gated linear attention, their normed results
// added; dense feed-forwards, biases nearly everywhere ----
PlanSpec balenex(const Json &c, const SafeTensors &w) {
    PlanSpec s;
    s.cfg.hidden = (int)c.integer("width");
    s.cfg.vocab = (int)c.integer("vocab");
    s.cfg.eps = (float)c.at("norm").real("eps");
    s.cfg.norm_groups = (int)c.at("norm").integer("groups");
    if (s.cfg.norm_groups < 1) broken("norms without groups");
    s.cfg.logit_scale = 1.0f;
    s.cfg.loop_times = 1;
    s.cfg.block = XFTHIP_BLOCK_SANDWICH, s.cfg.norm = XFTHIP_NORM_RMS;
    const Json &layers = c.at("layers");
    for (size_t i = 0; i < layers.items.size(); ++i) {
        const std::string at = "layer " + std::to_string(i) + ": ";
        const Json &e = layers.items[i], &m = e.at("mixer");
        const std::string &type = e.string("type");
        const bool one = type == "attention";
        if (!one && type != "parallel") broken("layer type '" + type + "' of config.json is not known");
        const Json &a = one ? m : m.at("left");
        xfthip_plan_layer L {}, R {};
        L.mixer = XFTHIP_MIXER_GROUPED;
        L.heads = (int)a.integer("heads"), L.kv_heads = (int)a.integer("kv_heads"), L.dim = (int)a.integer("dim"), L.vdim = (int)a.integer("vdim");
        L.scale = (float)a.real("scale");
        L.qkv_bias = 1;
        L.window = (int)a.at("mask").integer("size");
        if (L.window < 1) broken(at + "an empty window");
        if (one) {
            L.o_bias = 1, L.qk_norm = XFTHIP_QK_NORM_UNIT;
            L.pool = (int)a.at("mask").integer("pool");
            if (L.pool < 1) broken(at + "empty blocks");
        } else {
            L.qk_norm = XFTHIP_QK_NORM_HEAD;
            L.keep_first = (int)a.at("mask").integer("keep_first");
            L.taps = (int)a.integer("conv");
            L.rot_dim = (int)a.at("rot").integer("dims"), L.rot_base = a.at("rot").real("base");
            L.v_rot = 1;
            const Json &r = m.at("right");
            R.mixer = XFTHIP_MIXER_LINEAR;
            R.heads = (int)r.integer("heads"), R.dim = (int)r.integer("dim"), R.vdim = (int)r.integer("vdim");
            R.tau = (float)r.real("tau");
            R.decay_rank = (int)first_dim(w, "l" + std::to_string(i) + ".mix.right.a1");
            R.beside = 1;
            L.result_norm = R.result_norm = 1, L.scaled = R.scaled = 1, L.mix_scale = R.mix_scale = 0.5f;
        }
        if (e.has("mlp")) {
            const Json &f = e.at("mlp");
            if (f.string("kind") != "dense") broken("feed-forward '" + f.string("kind") + "' of config.json is not known");
            L.inter = (int)f.integer("ff"), L.mlp_bias = 1;
        }
        s.record.push_back((int)s.layers.size());
        s.layers.push_back(L);
        if (!one) s.layers.push_back(R);
    }
    s.cfg.layers = (int)s.layers.size();
    return s;
}

struct Architecture {
    const char *name;
    PlanSpec (*describe)(const Json &config, const SafeTensors &weights);
};
const Architecture kArchitectures[] = {{"Pinepel", pinepel}, {"Veterax", veterax}, {"Duvadra", duvadra}, {"Balenex", balenex}};

const Architecture *find_architecture(const Json &c) {
    if (c.kind != Json::Object || !c.has("architecture") || c.at("architecture").kind != Json::String) return nullptr;
    for (const Architecture &a : kArchitectures)
        if (c.at("architecture").text == a.name) return &a;
    return nullptr;
}

} // namespace

bool plan_architecture(const std::string &dir, std::string &name) {
    bool ok = false;
    const std::string src = read_file(dir + "/config.json", ok);
    Json c;
    std::string error;
    if (!ok || !Json::parse(src, c, error)) return false;
    const Architecture *a = find_architecture(c);
    if (a) name = a->name;
    return a != nullptr;
}

xfthip_plan_t load_plan(const std::string &dir, PlanSpec &spec) {
    bool ok = false;
    const std::string src = read_file(dir + "/config.json", ok);
    Json c;
    std::string error;
    if (!ok) broken("cannot read " + dir + "/config.json");
    if (!Json::parse(src, c, error)) broken("config.json: " + error);
    const Architecture *a = find_architecture(c);
    if (!a) broken("the architecture of config.json is not known");
    SafeTensors w;
    if (!w.open(dir + "/model.safetensors", error)) broken(error);
    spec = a->describe(c, w);
    xfthip_plan_t plan = nullptr;
    CK(xfthip_plan_create(&spec.cfg, spec.layers.data(), &plan));
    std::vector<uint16_t> widened;
    for (auto &kv : w.all()) {
        // 'l<i>.<name>' belongs to layer i, everything else to the model
        int layer = -1;
        std::string name = kv.first;
        if (name.size() > 2 && name[0] == 'l' && isdigit((unsigned char)name[1])) {
            char *end = nullptr;
            const long i = strtol(name.c_str() + 1, &end, 10);
            const long layers = spec.record.empty() ? spec.cfg.layers : (long)spec.record.size();
            if (*end == '.' && i < layers) {
                layer = spec.record.empty() ? (int)i : spec.record[(size_t)i], name = std::string(end + 1);
                // mixers side by side: 'mix.left.' is the layer's record, 'mix.right.' the one behind it
                if (name.compare(0, 9, "mix.left.") == 0) name.erase(4, 5);
                else if (name.compare(0, 10, "mix.right.") == 0) name.erase(4, 6), ++layer;
            }
        }
        const TensorRef &t = kv.second;
        const long rows = t.shape.empty() ? 1 : t.shape[0], n = t.count();
        if (rows <= 0 || n <= 0) continue;
        const uint16_t *data = (const uint16_t *)t.data;
        if (t.dtype == "F32") {
            widened.resize((size_t)n);
            for (long i = 0; i < n; ++i) {
                float f;
                memcpy(&f, t.data + 4 * i, 4);
                widened[(size_t)i] = to_bf16(f);
            }
            data = widened.data();
        } else if (t.dtype != "BF16") {
            continue; // integer tables: none of the known plans has any
        } else if ((uintptr_t)t.data & 1) {
            widened.resize((size_t)n);
            memcpy(widened.data(), t.data, (size_t)n * 2);
            data = widened.data();
        }
        CK(xfthip_plan_set_tensor(plan, layer, name.c_str(), data, (int)rows, (int)(n / rows)));
    }
    CK(xfthip_plan_finish(plan));
    return plan;
}

} // namespace xfthost
