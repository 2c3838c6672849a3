// Folders with config.json and model.safetensors: the readers of both, the registry of architectures and the builder that
// turns a configuration and its tensors into a mixer program (model.h).
//
// A safetensors file is an 8-byte little-endian length, that many bytes of JSON (name -> dtype, shape, data_offsets) and
// the data; it is mapped read-only. Matrices go to the device as they are and are packed there (vx_linear_pack); vectors and
// small tables become float32 on the host.
#include <errno.h>
#include <fcntl.h>
#include <math.h>
#include <stdio.h>
#include <stdlib.h>
#include <string.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <functional>
#include <utility>

#include "model.h"

namespace vh {
namespace {

// ---------------------------------------------------------------- JSON
struct Json {
    enum Type { NIL, BOOL, NUM, STR, ARR, OBJ } type = NIL;
    bool b = false;
    double num = 0;
    std::string str;
    std::vector<Json> arr;
    std::vector<std::pair<std::string, Json>> obj;
    const Json *get(const char *key) const {
        for (const auto &kv : obj)
            if (kv.first == key) return &kv.second;
        return nullptr;
    }
    bool absent() const { return type == NIL; }
};

struct JsonReader {
    const char *p, *end;
    int depth = 0;
    void space() {
        while (p < end && (*p == ' ' || *p == '\t' || *p == '\n' || *p == '\r')) p++;
    }
    bool word(const char *w) {
        const size_t n = strlen(w);
        if ((size_t)(end - p) < n || memcmp(p, w, n)) return false;
        p += n;
        return true;
    }
    bool hex4(unsigned *u) {
        if (end - p < 4) return false;
        *u = 0;
        for (int i = 0; i < 4; i++, p++) {
            const char c = *p;
            const int v = c >= '0' && c <= '9' ? c - '0' : c >= 'a' && c <= 'f' ? c - 'a' + 10 : c >= 'A' && c <= 'F' ? c - 'A' + 10 : -1;
            if (v < 0) return false;
            *u = *u * 16 + v;
        }
        return true;
    }
    bool string(std::string *out) {
        if (p >= end || *p != '"') return false;
        for (p++; p < end && *p != '"';) {
            if (*p != '\\') {
                out->push_back(*p++);
                continue;
            }
            if (++p >= end) return false;
            const char c = *p++;
            switch (c) {
                case 'n': out->push_back('\n'); break;
                case 't': out->push_back('\t'); break;
                case 'r': out->push_back('\r'); break;
                case 'b': out->push_back('\b'); break;
                case 'f': out->push_back('\f'); break;
                case 'u': {  // as UTF-8; a surrogate pair makes one character
                    unsigned u, lo;
                    if (!hex4(&u)) return false;
                    if (u >= 0xD800 && u < 0xDC00) {
                        if (!word("\\u") || !hex4(&lo) || lo < 0xDC00 || lo > 0xDFFF) return false;
                        u = 0x10000 + ((u - 0xD800) << 10) + (lo - 0xDC00);
                    }
                    if (u < 0x80) {
                        out->push_back((char)u);
                    } else {
                        const int more = u < 0x800 ? 1 : u < 0x10000 ? 2 : 3;
                        out->push_back((char)((more == 1 ? 0xC0 : more == 2 ? 0xE0 : 0xF0) | (u >> (6 * more))));
                        for (int i = more - 1; i >= 0; i--) out->push_back((char)(0x80 | ((u >> (6 * i)) & 0x3F)));
                    }
                    break;
                }
                default: out->push_back(c);  // quote, backslash, slash
            }
        }
        if (p >= end) return false;
        p++;
        return true;
    }
    bool value(Json *v) {
        space();
        if (p >= end || depth > 64) return false;
        if (*p == '{' || *p == '[') {
            const bool is_obj = *p++ == '{';
            const char close = is_obj ? '}' : ']';
            v->type = is_obj ? Json::OBJ : Json::ARR;
            depth++;
            space();
            if (p < end && *p == close) {
                p++, depth--;
                return true;
            }
            for (;;) {
                std::string key;
                if (is_obj) {
                    space();
                    if (!string(&key)) return false;
                    space();
                    if (p >= end || *p++ != ':') return false;
                }
                Json e;
                if (!value(&e)) return false;
                if (is_obj)
                    v->obj.emplace_back(std::move(key), std::move(e));
                else
                    v->arr.push_back(std::move(e));
                space();
                if (p >= end) return false;
                const char c = *p++;
                if (c == close) break;
                if (c != ',') return false;
            }
            depth--;
            return true;
        }
        if (*p == '"') {
            v->type = Json::STR;
            return string(&v->str);
        }
        if (word("null")) return true;
        if (word("true") || word("false")) {
            v->type = Json::BOOL;
            v->b = p[-1] == 'e' && p[-2] == 'u';
            return true;
        }
        std::string n;
        while (p < end && (strchr("+-.eE", *p) || (*p >= '0' && *p <= '9'))) n.push_back(*p++);
        char *stop = nullptr;
        v->type = Json::NUM;
        v->num = n.empty() ? 0 : strtod(n.c_str(), &stop);
        return !n.empty() && stop && *stop == 0;
    }
};

bool parse_json(const char *text, size_t n, Json *out) {
    JsonReader r{text, text + n};
    if (!r.value(out)) return false;
    r.space();
    return r.p == r.end;
}

// ---------------------------------------------------------------- safetensors
struct Mapped {
    const uint8_t *base = nullptr;
    size_t size = 0;
    ~Mapped() {
        if (base) munmap((void *)base, size);
    }
    int open(const std::string &path) {
        const int fd = ::open(path.c_str(), O_RDONLY | O_CLOEXEC);
        if (fd < 0) return fail("%s: %s", path.c_str(), strerror(errno));
        struct stat st;
        void *p = MAP_FAILED;
        if (fstat(fd, &st) == 0 && st.st_size > 0) p = mmap(nullptr, (size_t)st.st_size, PROT_READ, MAP_PRIVATE, fd, 0);
        ::close(fd);
        if (p == MAP_FAILED) return fail("%s: cannot be mapped", path.c_str());
        base = (const uint8_t *)p, size = (size_t)st.st_size;
        return VH_OK;
    }
};

struct TensorView {
    std::string dtype;
    std::vector<int64_t> shape;
    const uint8_t *data = nullptr;
};

struct SafeTensors {
    Mapped file;
    std::unordered_map<std::string, TensorView> tensors;
    int open(const std::string &path) {
        VHC(file.open(path));
        uint64_t n = 0;
        if (file.size < 8) return fail("%s: too short", path.c_str());
        for (int i = 0; i < 8; i++) n |= (uint64_t)file.base[i] << (8 * i);
        Json head;
        if (n > file.size - 8 || !parse_json((const char *)file.base + 8, (size_t)n, &head) || head.type != Json::OBJ)
            return fail("%s: no safetensors header", path.c_str());
        const uint8_t *data = file.base + 8 + n;
        const uint64_t room = file.size - 8 - n;
        for (const auto &kv : head.obj) {
            if (kv.first == "__metadata__") continue;
            const Json *dt = kv.second.get("dtype"), *sh = kv.second.get("shape"), *off = kv.second.get("data_offsets");
            if (!dt || dt->type != Json::STR || !sh || sh->type != Json::ARR || !off || off->type != Json::ARR || off->arr.size() != 2)
                return fail("%s: %s: incomplete entry", path.c_str(), kv.first.c_str());
            TensorView t;
            t.dtype = dt->str;
            uint64_t elems = 1;
            for (const Json &d : sh->arr) {
                if (d.type != Json::NUM || d.num < 0 || d.num > 1e12) return fail("%s: %s: bad shape", path.c_str(), kv.first.c_str());
                t.shape.push_back((int64_t)d.num);
                elems *= (uint64_t)d.num;
            }
            const int es = t.dtype == "BF16" || t.dtype == "F16" || t.dtype == "I16" ? 2 : t.dtype == "F32" || t.dtype == "I32" ? 4 : t.dtype == "I64" || t.dtype == "F64" ? 8 : 1;
            const double lo = off->arr[0].num, hi = off->arr[1].num;
            if (lo < 0 || hi < lo || hi > (double)room || (uint64_t)(hi - lo) != elems * es)
                return fail("%s: %s: its bytes do not fit its shape or the file", path.c_str(), kv.first.c_str());
            t.data = data + (uint64_t)lo;
            tensors[kv.first] = std::move(t);
        }
        return VH_OK;
    }
};

float bf16_to_f32(const uint8_t *p) {
    const uint32_t u = ((uint32_t)p[0] | (uint32_t)p[1] << 8) << 16;
    float f;
    memcpy(&f, &u, 4);
    return f;
}

// ---------------------------------------------------------------- configuration
// Reads numbers out of nested objects; the first thing missing or out of range is kept as the error.
struct Fields {
    std::string where;
    const Json *o;
    int *rc;
    Fields(const std::string &w, const Json *obj, int *r) : where(w), o(obj), rc(r) {
        if ((!o || o->type != Json::OBJ) && *rc == VH_OK) *rc = fail("config.json: %s is not an object", where.c_str());
    }
    const Json *need(const char *key, Json::Type t) const {
        const Json *v = o && o->type == Json::OBJ ? o->get(key) : nullptr;
        if (v && v->type == t) return v;
        if (*rc == VH_OK) *rc = fail("config.json: %s.%s is missing or of another type", where.c_str(), key);
        return nullptr;
    }
    double num(const char *key) const {
        const Json *v = need(key, Json::NUM);
        return v ? v->num : 0;
    }
    int count(const char *key, int lo = 1, int hi = 1 << 24) const {
        const double d = num(key);
        if (*rc == VH_OK && (d != floor(d) || d < lo || d > hi)) *rc = fail("config.json: %s.%s = %g is not a whole number in %d..%d", where.c_str(), key, d, lo, hi);
        return *rc == VH_OK ? (int)d : lo;
    }
    Fields sub(const char *key) const { return Fields(where + "." + key, o && o->type == Json::OBJ ? o->get(key) : nullptr, rc); }
    bool has(const char *key) const {
        const Json *v = o && o->type == Json::OBJ ? o->get(key) : nullptr;
        return v && !v->absent();
    }
};

// What a Lozedra config.json says, layer by layer.
struct LozedraLayer {
    int heads = 1, kv_heads = 1, dim = 1, vdim = 1, bias_max = 1, temp_every = 0;
    float scale = 1.f, temp_coef = 0.f, left_scale = 1.f, right_scale = 1.f;
    int inner = 1, state = 1, dt_rank = 1, conv = 1;
    int ff = 0;  // 0: no feed-forward
};
struct LozedraConfig {
    std::vector<LozedraLayer> layers;
    int loop_start = 0, loop_stop = 0, loop_times = 1;
    float eps = 1e-5f, mult = 1.f;
    int vocab = 1, width = 1;
};

int parse_lozedra(const Json &j, LozedraConfig *c) {
    int rc = VH_OK;
    const Fields root("config", &j, &rc);
    c->vocab = root.count("vocab");
    c->width = root.count("width", 1, 1 << 20);
    c->mult = (float)root.num("residual_mult");
    c->eps = (float)root.sub("norm").num("eps");
    const Json *layers = root.need("layers", Json::ARR);
    if (rc != VH_OK) return rc;
    if (layers->arr.empty()) return fail("config.json: no layers");
    for (size_t i = 0; i < layers->arr.size(); i++) {
        const Fields l("layers[" + std::to_string(i) + "]", &layers->arr[i], &rc);
        const Json *type = l.need("type", Json::STR);
        if (rc != VH_OK) return rc;
        if (type->str != "parallel") return fail("config.json: layer %zu has the unknown mixer type '%s'", i, type->str.c_str());
        LozedraLayer o;
        const Fields mx = l.sub("mixer"), left = mx.sub("left"), right = mx.sub("right");
        o.left_scale = (float)mx.num("left_scale"), o.right_scale = (float)mx.num("right_scale");
        o.heads = left.count("heads", 1, 4096), o.kv_heads = left.count("kv_heads", 1, 4096);
        o.dim = left.count("dim", 1, 2048), o.vdim = left.count("vdim", 1, 2048);
        o.scale = (float)left.num("scale");
        o.bias_max = left.count("bias_max");
        if (left.has("q_temp")) {
            const Fields q = left.sub("q_temp");
            o.temp_coef = (float)q.num("coef"), o.temp_every = q.count("every");
        }
        o.inner = right.count("inner", 1, 1 << 20), o.state = right.count("state", 1, 256);
        o.dt_rank = right.count("dt_rank", 1, 1 << 16), o.conv = right.count("conv", 1, 64);
        if (l.has("mlp")) {
            const Fields mlp = l.sub("mlp");
            const Json *kind = mlp.need("kind", Json::STR);
            if (rc == VH_OK && kind->str != "dense") return fail("config.json: layer %zu has the unknown feed-forward '%s'", i, kind->str.c_str());
            o.ff = mlp.count("ff", 1, 1 << 20);
        }
        if (rc != VH_OK) return rc;
        if (o.heads % o.kv_heads) return fail("config.json: layer %zu: %d heads are no multiple of %d", i, o.heads, o.kv_heads);
        c->layers.push_back(o);
    }
    if (root.has("loop")) {
        const Fields lp = root.sub("loop");
        const int n = (int)c->layers.size();
        c->loop_start = lp.count("start", 0, n), c->loop_stop = lp.count("stop", 0, n), c->loop_times = lp.count("times", 1, 4096);
        if (rc == VH_OK && c->loop_stop < c->loop_start) return fail("config.json: loop of layers %d .. %d", c->loop_start, c->loop_stop);
    }
    return rc;
}

// ---------------------------------------------------------------- weights
struct Builder {
    vx_backend *be;
    const SafeTensors *st;
    vh_model *m;
    int block_size;
    void *stage = nullptr;       // device copy of the matrix being packed
    size_t stage_bytes = 0;
    int pad(int n, int to) const { return (n + to - 1) / to * to; }

    ~Builder() {
        if (stage) vx_free(be, stage);
    }
    int view(const std::string &name, std::vector<int64_t> shape, const TensorView **out) const {
        const auto it = st->tensors.find(name);
        if (it == st->tensors.end()) return fail("tensor %s is missing", name.c_str());
        if (it->second.shape != shape) {
            std::string want, have;
            for (int64_t d : shape) want += " " + std::to_string(d);
            for (int64_t d : it->second.shape) have += " " + std::to_string(d);
            return fail("tensor %s: shape [%s ], the configuration needs [%s ]", name.c_str(), have.c_str(), want.c_str());
        }
        if (it->second.dtype != "BF16") return fail("tensor %s: type %s, not BF16", name.c_str(), it->second.dtype.c_str());
        *out = &it->second;
        return VH_OK;
    }
    int floats(const std::string &name, std::vector<int64_t> shape, std::vector<float> *out) const {
        const TensorView *t;
        VHC(view(name, shape, &t));
        size_t n = 1;
        for (int64_t d : shape) n *= (size_t)d;
        out->resize(n);
        for (size_t i = 0; i < n; i++) (*out)[i] = bf16_to_f32(t->data + 2 * i);
        return VH_OK;
    }
    int upload(const std::vector<float> &v, const float **out) {
        void *p = vx_alloc_permanent(be, (v.size() * 4 + 15) / 16 * 16 + 16);
        if (!p) return fail("device memory: %s", vx_last_error());
        m->adopted.push_back(p);
        VXC(vx_to_device(be, p, v.data(), v.size() * 4));
        *out = (const float *)p;
        return VH_OK;
    }
    int vec(const std::string &name, int n, const float **out) {
        std::vector<float> v;
        VHC(floats(name, {n}, &v));
        return upload(v, out);
    }
    int packed(Linear *w, int n, int k) {
        w->n = pad(n, 16), w->k = pad(k, 64);
        w->w = vx_alloc_permanent(be, vx_linear_bytes(w->n, w->k));
        if (!w->w) return fail("device memory: %s", vx_last_error());
        m->adopted.push_back(w->w);
        VXC(vx_fill_zero(be, w->w, vx_linear_bytes(w->n, w->k)));
        return VH_OK;
    }
    // rows first .. first + n - 1 of the matrix [total, k] -> rows row0 .. (tile step `step`), columns col0 ..
    int pack(const std::string &name, int total, int k, int first, int n, const Linear &w, int row0, int step, int col0) {
        const TensorView *t;
        VHC(view(name, {total, k}, &t));
        const size_t bytes = (size_t)n * k * 2;
        if (bytes > stage_bytes) {
            if (stage) vx_free(be, stage);
            stage = vx_alloc_permanent(be, bytes);
            stage_bytes = stage ? bytes : 0;
            if (!stage) return fail("device memory: %s", vx_last_error());
        }
        VXC(vx_to_device(be, stage, t->data + (size_t)first * k * 2, bytes));
        VXC(vx_linear_pack(be, stage, n, k, w.w, w.n, w.k, row0 / 16, step, col0));
        return VH_OK;
    }
    int pack_host(const std::vector<uint16_t> &h, int n, int k, const Linear &w, int row0) {
        const size_t bytes = h.size() * 2;
        if (bytes > stage_bytes) {
            if (stage) vx_free(be, stage);
            stage = vx_alloc_permanent(be, bytes);
            stage_bytes = stage ? bytes : 0;
            if (!stage) return fail("device memory: %s", vx_last_error());
        }
        VXC(vx_to_device(be, stage, h.data(), bytes));
        VXC(vx_linear_pack(be, stage, n, k, w.w, w.n, w.k, row0 / 16, 1, 0));
        return VH_OK;
    }
    // A matrix [n, k] put together on the host from the elements of that tensor [total, from]: place(row, col) says which element
    // (row * from + col) goes there, -1 none.
    template <class Place>
    int pack_placed(const std::string &name, int total, int from, int n, int k, const Linear &w, int row0, Place &&place) {
        const TensorView *t;
        VHC(view(name, {total, from}, &t));
        std::vector<uint16_t> h((size_t)n * k, 0);
        for (int r = 0; r < n; r++)
            for (int c = 0; c < k; c++) {
                const int64_t e = place(r, c);
                if (e >= 0) memcpy(&h[(size_t)r * k + c], t->data + 2 * e, 2);
            }
        return pack_host(h, n, k, w, row0);
    }
    // The same in whole rows: row r is row src(r) of the tensor, -1 none.
    template <class Row>
    int pack_rows(const std::string &name, int total, int k, int n, const Linear &w, int row0, Row &&src) {
        const TensorView *t;
        VHC(view(name, {total, k}, &t));
        std::vector<uint16_t> h((size_t)n * k, 0);
        for (int r = 0; r < n; r++)
            if (const int s = src(r); s >= 0) memcpy(&h[(size_t)r * k], t->data + (size_t)s * k * 2, (size_t)k * 2);
        return pack_host(h, n, k, w, row0);
    }
};

int distance_bucket(int n, int rows, int bias_max) {
    const int half = rows / 2;
    if (rows < 2 || bias_max <= half || n < 0) return -1;
    if (n < half) return n;
    if (n >= bias_max) return rows - 1;
    // a distance at which the logarithm reaches a whole number has reached it, whatever the last bit of the quotient says
    const double v = log((double)n / half) / log((double)bias_max / half) * (rows - half), near = round(v);
    const int b = half + (int)(fabs(v - near) < 1e-9 ? near : floor(v));
    return b < rows - 1 ? b : rows - 1;
}

int build_lozedra(Builder &b, const Json &config, MixModel *x, vh_config *cfg) {
    LozedraConfig c;
    VHC(parse_lozedra(config, &c));
    cfg->hidden = c.width, cfg->vocab = c.vocab, cfg->eps = c.eps;
    x->eps = c.eps, x->mult = c.mult, x->recurrent = true;
    for (size_t i = 0; i < c.layers.size(); i++) {
        const LozedraLayer &s = c.layers[i];
        const std::string l = "l" + std::to_string(i) + ".", left = l + "mix.left.", right = l + "mix.right.", mlp = l + "mlp.";
        const int W = c.width, qd = s.heads * s.dim, kd = s.kv_heads * s.dim, vd = s.kv_heads * s.vdim, od = s.heads * s.vdim;
        MixLayer o;
        VHC(b.vec(l + "norm1", W, &o.norm1));
        VHC(b.vec(l + "norm1b", W, &o.norm1b));
        // one input projection for both mixers, its parts at whole tiles
        AttnMixer &a = o.attn;
        ScanMixer &n = o.scan;
        o.has_attn = o.has_scan = true;
        a.heads = s.heads, a.kv_heads = s.kv_heads, a.k_dim = s.dim, a.v_dim = s.vdim;
        a.scale = s.scale, a.temp_coef = s.temp_coef, a.temp_every = s.temp_every, a.gate = true, a.out_scale = s.left_scale;
        n.channels = s.inner, n.states = s.state, n.pad = vx_scan_state_pad(s.state), n.taps = s.conv, n.dt_rank = s.dt_rank;
        n.dt_pad = b.pad(s.dt_rank, 64), n.out_scale = s.right_scale;
        a.q_col = 0;
        a.k_col = b.pad(qd, 16);
        a.v_col = a.k_col + b.pad(kd, 16);
        a.g_col = a.v_col + b.pad(vd, 16);
        n.x_col = a.g_col + b.pad(od, 16);
        n.z_col = n.x_col + b.pad(s.inner, 16);
        VHC(b.packed(&o.in, n.z_col + s.inner, W));
        VHC(b.pack(left + "q", qd, W, 0, qd, o.in, a.q_col, 1, 0));
        VHC(b.pack(left + "k", kd, W, 0, kd, o.in, a.k_col, 1, 0));
        VHC(b.pack(left + "v", vd, W, 0, vd, o.in, a.v_col, 1, 0));
        VHC(b.pack(left + "g", od, W, 0, od, o.in, a.g_col, 1, 0));
        VHC(b.pack(right + "in", 2 * s.inner, W, 0, s.inner, o.in, n.x_col, 1, 0));
        VHC(b.pack(right + "in", 2 * s.inner, W, s.inner, s.inner, o.in, n.z_col, 1, 0));
        // one output projection: its inputs are the heads, then the channels
        VHC(b.packed(&o.out, W, od + s.inner));
        VHC(b.pack(left + "o", W, od, 0, W, o.out, 0, 1, 0));
        VHC(b.pack(right + "o", W, s.inner, 0, W, o.out, 0, 1, od));
        // the distance bias, spread out to one value per distance
        std::vector<float> rel;
        const auto it = b.st->tensors.find(left + "rel");
        if (it == b.st->tensors.end() || it->second.shape.size() != 2) return fail("tensor %srel is missing or no table", left.c_str());
        const int rows = (int)it->second.shape[0];
        VHC(b.floats(left + "rel", {rows, s.heads}, &rel));
        if (distance_bucket(0, rows, s.bias_max) < 0)
            return fail("layer %zu: a bias table of %d rows with bias_max %d", i, rows, s.bias_max);
        a.bias_len = s.bias_max + 1;
        std::vector<float> bias((size_t)s.heads * a.bias_len);
        for (int h = 0; h < s.heads; h++)
            for (int d = 0; d < a.bias_len; d++)
                bias[(size_t)h * a.bias_len + d] = rel[(size_t)distance_bucket(d, rows, s.bias_max) * s.heads + h];
        VHC(b.upload(bias, &a.bias));
        // the scan's own weights
        std::vector<float> cw, t, tr;
        VHC(b.floats(right + "conv", {s.inner, s.conv}, &cw));
        tr.resize(cw.size());
        for (int ch = 0; ch < s.inner; ch++)
            for (int k = 0; k < s.conv; k++) tr[(size_t)k * s.inner + ch] = cw[(size_t)ch * s.conv + k];
        VHC(b.upload(tr, &n.conv_w));
        VHC(b.vec(right + "conv.b", s.inner, &n.conv_b));
        VHC(b.packed(&n.x, n.dt_pad + 2 * n.pad, s.inner));
        const int xr = s.dt_rank + 2 * s.state;
        VHC(b.pack(right + "x", xr, s.inner, 0, s.dt_rank, n.x, 0, 1, 0));
        VHC(b.pack(right + "x", xr, s.inner, s.dt_rank, s.state, n.x, n.dt_pad, 1, 0));
        VHC(b.pack(right + "x", xr, s.inner, s.dt_rank + s.state, s.state, n.x, n.dt_pad + n.pad, 1, 0));
        VHC(b.packed(&n.dt, s.inner, s.dt_rank));
        VHC(b.pack(right + "dt", s.inner, s.dt_rank, 0, s.inner, n.dt, 0, 1, 0));
        VHC(b.vec(right + "dt.b", s.inner, &n.dt_bias));
        VHC(b.floats(right + "A_log", {s.inner, s.state}, &t));
        std::vector<float> a2((size_t)s.inner * n.pad, 0.f);
        for (int ch = 0; ch < s.inner; ch++)
            for (int k = 0; k < s.state; k++)
                a2[(size_t)ch * n.pad + k] = (float)(-exp((double)t[(size_t)ch * s.state + k]) * 1.4426950408889634);
        VHC(b.upload(a2, &n.a2));
        VHC(b.vec(right + "D", s.inner, &n.d));
        if (s.ff > 0) {
            o.has_mlp = true;
            o.ff_pad = b.pad(s.ff, 64);
            VHC(b.vec(l + "norm2", W, &o.norm2));
            VHC(b.vec(l + "norm2b", W, &o.norm2b));
            VHC(b.packed(&o.gate_up, 2 * o.ff_pad, W));
            VHC(b.pack(mlp + "gate", s.ff, W, 0, s.ff, o.gate_up, 0, 2, 0));
            VHC(b.pack(mlp + "up", s.ff, W, 0, s.ff, o.gate_up, 16, 2, 0));
            VHC(b.packed(&o.down, W, s.ff));
            VHC(b.pack(mlp + "down", W, s.ff, 0, W, o.down, 0, 1, 0));
        }
        x->layers.push_back(o);
    }
    auto run = [&](int layer, bool again) {
        LayerRun r;
        r.layer = layer, r.add_embedding = again;
        x->runs.push_back(r);
    };
    const int n = (int)c.layers.size();
    for (int i = 0; i < c.loop_start; i++) run(i, false);
    for (int pass = 0; pass < c.loop_times; pass++)
        for (int i = c.loop_start; i < c.loop_stop; i++) run(i, pass > 0 && i == c.loop_start);
    for (int i = c.loop_stop; i < n; i++) run(i, false);
    std::vector<float> emb;
    VHC(b.floats("embed", {c.vocab, c.width}, &emb));
    VHC(b.upload(emb, &b.m->embedding));
    VHC(b.vec("final.norm", c.width, &b.m->final_norm));
    VHC(b.packed(&x->head, c.vocab, c.width));
    return b.pack("head", c.vocab, c.width, 0, c.vocab, x->head, 0, 1, 0);
}

int check_lozedra(const Json &config) {
    LozedraConfig c;
    return parse_lozedra(config, &c);
}

// ---------------------------------------------------------------- Tulipel
struct TulipelLayer {
    int heads = 1, dim = 1, rot_dim = 2, vdim = 1, rank = 1, q_rank = 0;  // q_rank 0: queries straight from the stream
    float scale = 1.f;
    bool halves = false;          // rotated pairs are (i, i + n / 2) in the tensors; packed as neighbours
    double base = 1.0;
    bool yarn = false;
    double factor = 1.0, original = 1.0, fast = 1.0, slow = 1.0;
    int kv_from = -1, ff = 0;     // ff 0: no feed-forward
    bool same_rotation(const TulipelLayer &o) const {
        return rot_dim == o.rot_dim && halves == o.halves && base == o.base && yarn == o.yarn &&
               (!yarn || (factor == o.factor && original == o.original && fast == o.fast && slow == o.slow));
    }
};
struct TulipelConfig {
    std::vector<TulipelLayer> layers;
    float eps = 1e-5f, alpha = 1.f, softcap = 0.f;
    int vocab = 1, width = 1;
};

int parse_tulipel(const Json &j, TulipelConfig *c) {
    int rc = VH_OK;
    const Fields root("config", &j, &rc);
    c->vocab = root.count("vocab");
    c->width = root.count("width", 1, 1 << 20);
    c->alpha = (float)root.num("postln_alpha");
    c->eps = (float)root.sub("norm").num("eps");
    if (root.has("logit_softcap")) {
        c->softcap = (float)root.num("logit_softcap");
        if (rc == VH_OK && !(c->softcap > 0.f)) return fail("config.json: logit_softcap is not above 0");
    }
    const Json *layers = root.need("layers", Json::ARR);
    if (rc != VH_OK) return rc;
    if (layers->arr.empty()) return fail("config.json: no layers");
    for (size_t i = 0; i < layers->arr.size(); i++) {
        const Fields l("layers[" + std::to_string(i) + "]", &layers->arr[i], &rc);
        const Json *type = l.need("type", Json::STR);
        if (rc != VH_OK) return rc;
        TulipelLayer o;
        const Fields mx = l.sub("mixer"), rot = mx.sub("rot");
        if (type->str == "latent_attention")
            o.q_rank = mx.count("q_rank", 1, 1 << 16);
        else if (type->str == "latent_attention_2")
            o.halves = true;
        else
            return fail("config.json: layer %zu has the unknown mixer type '%s'", i, type->str.c_str());
        o.heads = mx.count("heads", 1, 4096), o.dim = mx.count("dim", 1, 2048), o.vdim = mx.count("vdim", 1, 2048);
        o.rank = mx.count("kv_rank", 1, 2048), o.rot_dim = mx.count("rot_dim", 2, 1024);
        o.scale = (float)mx.num("scale");
        o.base = rot.num("base");
        const int dims = rot.count("dims", 2, 1024);
        if (rot.has("scaling")) {
            const Fields y = rot.sub("scaling");
            o.yarn = true;
            o.factor = y.num("factor"), o.original = y.num("original"), o.fast = y.num("fast"), o.slow = y.num("slow");
            if (rc == VH_OK && !(o.factor > 0 && o.original > 0 && o.fast > 0 && o.slow > 0)) return fail("config.json: layer %zu: rot.scaling is not above 0", i);
        }
        if (mx.has("kv_from")) o.kv_from = mx.count("kv_from", 0, 1 << 16);
        if (l.has("mlp")) {
            const Fields mlp = l.sub("mlp");
            const Json *kind = mlp.need("kind", Json::STR);
            if (rc == VH_OK && kind->str != "dense") return fail("config.json: layer %zu has the unknown feed-forward '%s'", i, kind->str.c_str());
            o.ff = mlp.count("ff", 1, 1 << 20);
        }
        if (rc != VH_OK) return rc;
        if (o.rot_dim % 2 || dims != o.rot_dim) return fail("config.json: layer %zu turns %d of %d dimensions", i, dims, o.rot_dim);
        if (!(o.base > 1.0)) return fail("config.json: layer %zu: rot.base is not above 1", i);
        if (o.kv_from >= 0) {
            if (o.kv_from >= (int)i || c->layers[o.kv_from].kv_from >= 0)
                return fail("config.json: layer %zu: layer %d holds no latents for it", i, o.kv_from);
            const TulipelLayer &f = c->layers[o.kv_from];
            if (f.rank != o.rank || !f.same_rotation(o)) return fail("config.json: layer %zu: the latents of layer %d are of another kind", i, o.kv_from);
        }
        c->layers.push_back(o);
    }
    return rc;
}

// Radians per position of every pair, and the factor of cosine and sine.
void rotary_frequencies(int dims, double base, bool yarn, double factor, double original, double fast, double slow, std::vector<double> *f, double *both) {
    f->resize(dims / 2);
    for (int i = 0; i < dims / 2; i++) (*f)[i] = pow(base, -2.0 * i / dims);
    *both = 1.0;
    if (!yarn) return;
    // the (fractional) dimension whose pair makes that many turns over the original length
    const auto dim_of = [&](double turns) { return dims * log(original / (2 * M_PI * turns)) / (2 * log(base)); };
    const double lo = fmax(floor(dim_of(fast)), 0.0), hi = fmin(ceil(dim_of(slow)), dims - 1.0);
    for (int i = 0; i < dims / 2; i++) {
        const double ramp = fmin(fmax((i - lo) / fmax(hi - lo, 0.001), 0.0), 1.0);
        (*f)[i] = (*f)[i] / factor * ramp + (*f)[i] * (1.0 - ramp);
    }
    *both = 0.1 * log(factor) + 1.0;
}

// From how many rows of a sequence on it pays to spell its keys and values out: per (row, key, head) that takes 2 rank - dim - vdim
// products less, and rank (dim + vdim) per (key, head) once. Half as many rows again, since the keys before the sequence's
// new rows count in full and the spelled-out ones have to be written and read.
int spell_out_rows(int rank, int dim, int vdim) {
    const int64_t less = 2 * (int64_t)rank - dim - vdim;
    if (less <= 0) return 0;
    const int64_t rows = (3 * (int64_t)rank * (dim + vdim) / 2 + less - 1) / less;
    return rows < (1 << 20) ? (int)(rows < 2 ? 2 : rows) : 0;
}

int build_tulipel(Builder &b, const Json &config, MixModel *x, vh_config *cfg) {
    TulipelConfig c;
    VHC(parse_tulipel(config, &c));
    cfg->hidden = c.width, cfg->vocab = c.vocab, cfg->eps = c.eps;
    x->eps = c.eps, x->post_norm = true, x->alpha = c.alpha, x->softcap = c.softcap;
    const int W = c.width;
    std::vector<int> rotation_layer;  // a layer that has rotation 0, 1, ..
    const auto around_zero = [&](const std::string &name, const float **out) -> int {
        std::vector<float> v;
        VHC(b.floats(name, {W}, &v));
        for (float &f : v) f += 1.0f;
        return b.upload(v, out);
    };
    for (size_t i = 0; i < c.layers.size(); i++) {
        const TulipelLayer &s = c.layers[i];
        const std::string l = "l" + std::to_string(i) + ".", mix = l + "mix.", mlp = l + "mlp.";
        MixLayer o;
        o.has_latent = true;
        LatentMixer &t = o.latent;
        VHC(around_zero(l + "norm1", &o.norm1));
        t.heads = s.heads, t.rank = s.rank, t.rot_dim = s.rot_dim, t.q_rank = s.q_rank, t.scale = s.scale, t.kv_from = s.kv_from;
        t.dim_pad = b.pad(s.dim, 64), t.head_cols = t.dim_pad + b.pad(s.rot_dim, 16), t.v_pad = b.pad(s.vdim, 16);
        t.rank_pad = vx_latent_pad(s.rank), t.row = vx_latent_row(s.rank, s.rot_dim);
        for (size_t k = 0; k < rotation_layer.size(); k++)
            if (s.same_rotation(c.layers[rotation_layer[k]])) t.rotation = (int)k;
        if (t.rotation < 0) {
            t.rotation = (int)rotation_layer.size();
            rotation_layer.push_back((int)i);
            Rotation r;
            double both;
            rotary_frequencies(s.rot_dim, s.base, s.yarn, s.factor, s.original, s.fast, s.slow, &r.freqs, &both);
            r.factor = (float)both;
            x->rotations.push_back(r);
        }
        // columns: heads, each its plain part, then its rotated part with the pairs as neighbours
        const int half = s.rot_dim / 2, q_cols = s.heads * t.head_cols, qd = s.heads * (s.dim + s.rot_dim);
        const auto pair_place = [&](int d) { return s.halves ? d / 2 + d % 2 * half : d; };  // packed rotated column -> stored one
        const auto q_row = [&](int r) {
            const int h = r / t.head_cols, d = r % t.head_cols, rd = d - t.dim_pad;
            if (rd >= 0) return rd < s.rot_dim ? h * (s.dim + s.rot_dim) + s.dim + pair_place(rd) : -1;
            return d < s.dim ? h * (s.dim + s.rot_dim) + d : -1;
        };
        const bool own = s.kv_from < 0;
        const int first = s.q_rank > 0 ? b.pad(s.q_rank, 16) : q_cols;
        const int kv_cols = own ? b.pad(s.rank, 16) + b.pad(s.rot_dim, 16) : 0;
        t.c_col = s.q_rank > 0 ? first : 0, t.kr_col = t.c_col + b.pad(s.rank, 16), t.kv_cols = kv_cols;
        VHC(b.packed(&o.in, first + kv_cols, W));
        if (s.q_rank > 0) {
            VHC(b.pack(mix + "dq", s.q_rank, W, 0, s.q_rank, o.in, 0, 1, 0));
            VHC(b.vec(mix + "dq.norm", s.q_rank, &t.norm_q));
            VHC(b.packed(&t.q_up, q_cols, s.q_rank));
            VHC(b.pack_rows(mix + "uq", qd, s.q_rank, q_cols, t.q_up, 0, q_row));
        } else {
            VHC(b.pack_rows(mix + "q", qd, W, q_cols, o.in, 0, q_row));
        }
        if (own) {
            VHC(b.pack(mix + "dkv", s.rank + s.rot_dim, W, 0, s.rank, o.in, first, 1, 0));
            VHC(b.pack_rows(mix + "dkv", s.rank + s.rot_dim, W, s.rot_dim, o.in, first + b.pad(s.rank, 16), [&](int r) { return s.rank + pair_place(r); }));
            VHC(b.vec(mix + "dkv.norm", s.rank, &t.norm_c));
        }
        VHC(b.vec(mix + "sink", s.heads, &t.sink));
        // out of the latents: keys of all heads, then values; into them: per head, the keys' matrix transposed
        const int k_cols = s.heads * t.dim_pad;
        VHC(b.packed(&t.expand, k_cols + s.heads * t.v_pad, t.rank_pad));
        VHC(b.pack_rows(mix + "uk", s.heads * s.dim, s.rank, k_cols, t.expand, 0, [&](int r) {
            const int h = r / t.dim_pad, d = r % t.dim_pad;
            return d < s.dim ? h * s.dim + d : -1;
        }));
        VHC(b.pack_rows(mix + "uv", s.heads * s.vdim, s.rank, s.heads * t.v_pad, t.expand, k_cols, [&](int r) {
            const int h = r / t.v_pad, d = r % t.v_pad;
            return d < s.vdim ? h * s.vdim + d : -1;
        }));
        VHC(b.packed(&t.absorb, s.heads * t.rank_pad, t.dim_pad));
        VHC(b.pack_placed(mix + "uk", s.heads * s.dim, s.rank, s.heads * t.rank_pad, s.dim, t.absorb, 0, [&](int r, int d) -> int64_t {
            const int h = r / t.rank_pad, e = r % t.rank_pad;
            return e < s.rank ? ((int64_t)h * s.dim + d) * s.rank + e : -1;
        }));
        VHC(b.packed(&o.out, W, s.heads * t.v_pad));
        VHC(b.pack_placed(mix + "o", W, s.heads * s.vdim, W, s.heads * t.v_pad, o.out, 0, [&](int r, int k) -> int64_t {
            const int h = k / t.v_pad, d = k % t.v_pad;
            return d < s.vdim ? (int64_t)r * s.heads * s.vdim + h * s.vdim + d : -1;
        }));
        if (x->act == VX_ACT_BF16 && vx_attn_latent_fast(x->act, b.block_size, s.rank, s.rot_dim) &&
            vx_attn_ragged_fast(x->act, b.block_size, s.heads, s.heads, t.head_cols, t.v_pad)) {
            t.expand_rows = spell_out_rows(s.rank, s.dim, s.vdim);
            if (t.expand_rows > 0 && (x->expand_rows == 0 || t.expand_rows < x->expand_rows)) x->expand_rows = t.expand_rows;
        }
        if (s.ff > 0) {
            o.has_mlp = true;
            o.ff = s.ff, o.ff_pad = b.pad(s.ff, 64);
            VHC(around_zero(l + "norm2", &o.norm2));
            VHC(b.packed(&o.gate_up, o.ff_pad, W));
            VHC(b.pack(mlp + "up", s.ff, W, 0, s.ff, o.gate_up, 0, 1, 0));
            VHC(b.packed(&o.down, W, s.ff));
            VHC(b.pack(mlp + "down", W, s.ff, 0, W, o.down, 0, 1, 0));
            VHC(b.vec(mlp + "act", 4, &o.poly));
        }
        VHC(b.vec(l + "dwa", (int)i + 2, &o.depth_avg));
        x->layers.push_back(o);
        LayerRun r;
        r.layer = (int)i;
        x->runs.push_back(r);
    }
    std::vector<float> emb;
    VHC(b.floats("embed", {c.vocab, W}, &emb));
    VHC(b.upload(emb, &b.m->embedding));
    VHC(around_zero("final.norm", &b.m->final_norm));
    VHC(b.packed(&x->head, c.vocab, W));
    return b.pack("head", c.vocab, W, 0, c.vocab, x->head, 0, 1, 0);
}

int check_tulipel(const Json &config) {
    TulipelConfig c;
    return parse_tulipel(config, &c);
}

// ---------------------------------------------------------------- Kitodra
struct KitodraLayer {
    enum Kind { DIFFERENTIAL, KEY_VALUE, LIGHTNING } kind = LIGHTNING;
    int weights_of = -1;          // >= 0: a layer whose tensors this one uses; the rest of its entry says the same
    int heads = 1, kv_heads = 1, dim = 1, vdim = 1, mask = 0, rot_dims = 0;
    double rot_base = 1.0;
    float scale = 1.f, softcap = 0.f, diff = 0.f;
    std::vector<double> decay;
    bool experts = false, shared = false;
    int n_experts = 1, top = 1, groups = 1, keep = 1, ff = 1, shared_ff = 1;
    float limit = 0.f, shared_limit = 0.f;
};
struct KitodraConfig {
    std::vector<KitodraLayer> layers;
    std::vector<int> own;         // the layer whose tensors layer i uses
    float eps = 1e-5f;
    int vocab = 1, width = 1, buckets = 0;
    int64_t mul_prev = 0, mul_cur = 0;
};

int parse_kitodra(const Json &j, KitodraConfig *c) {
    int rc = VH_OK;
    const Fields root("config", &j, &rc);
    c->vocab = root.count("vocab");
    c->width = root.count("width", 1, 1 << 20);
    c->eps = (float)root.sub("norm").num("eps");
    if (root.has("embedding") && root.sub("embedding").has("bigram")) {
        const Fields p = root.sub("embedding").sub("bigram");
        c->buckets = p.count("buckets", 1, 1 << 30);
        c->mul_prev = p.count("mul_prev", 0, 0x7fffffff), c->mul_cur = p.count("mul_cur", 0, 0x7fffffff);
    }
    const Json *layers = root.need("layers", Json::ARR);
    if (rc != VH_OK) return rc;
    if (layers->arr.empty()) return fail("config.json: no layers");
    for (size_t i = 0; i < layers->arr.size(); i++) {
        const Fields l("layers[" + std::to_string(i) + "]", &layers->arr[i], &rc);
        const Json *type = l.need("type", Json::STR);
        if (rc != VH_OK) return rc;
        KitodraLayer o;
        if (type->str == "attention")
            o.kind = KitodraLayer::DIFFERENTIAL;
        else if (type->str == "attention_2")
            o.kind = KitodraLayer::KEY_VALUE;
        else if (type->str != "lightning")
            return fail("config.json: layer %zu has the unknown mixer type '%s'", i, type->str.c_str());
        if (l.has("weights_of")) o.weights_of = l.count("weights_of", 0, (int)layers->arr.size() - 1);
        const Fields mx = l.sub("mixer");
        const bool light = o.kind == KitodraLayer::LIGHTNING;
        o.heads = mx.count("heads", 1, 4096);
        o.dim = mx.count("dim", 1, light ? 512 : 2048), o.vdim = mx.count("vdim", 1, light ? 512 : 2048);
        if (light) {
            const Json *decay = mx.need("decay", Json::ARR);
            if (rc != VH_OK) return rc;
            for (const Json &d : decay->arr) {
                if (d.type != Json::NUM || !(d.num >= 0.0 && d.num <= 1.0)) return fail("config.json: layer %zu: mixer.decay is not between 0 and 1", i);
                o.decay.push_back(d.num);
            }
            if ((int)o.decay.size() != o.heads) return fail("config.json: layer %zu: mixer.decay holds %zu numbers for %d heads", i, o.decay.size(), o.heads);
        } else {
            o.kv_heads = mx.count("kv_heads", 1, 4096);
            o.scale = (float)mx.num("scale");
            if (mx.has("mask")) o.mask = mx.sub("mask").count("size", 1, 1 << 30);
            if (mx.has("softcap")) {
                o.softcap = (float)mx.num("softcap");
                if (rc == VH_OK && !(o.softcap > 0.f)) return fail("config.json: layer %zu: mixer.softcap is not above 0", i);
            }
            if (o.kind == KitodraLayer::DIFFERENTIAL) o.diff = (float)mx.num("diff");
            if (o.kind == KitodraLayer::KEY_VALUE && mx.has("rot")) {
                const Fields rot = mx.sub("rot");
                o.rot_dims = rot.count("dims", 0, 2048), o.rot_base = rot.num("base");
            }
        }
        if (l.has("mlp")) {
            const Fields mlp = l.sub("mlp"), router = mlp.sub("router"), expert = mlp.sub("expert");
            const Json *kind = mlp.need("kind", Json::STR);
            if (rc == VH_OK && kind->str != "moe") return fail("config.json: layer %zu has the unknown feed-forward '%s'", i, kind->str.c_str());
            o.experts = true;
            o.n_experts = router.count("experts", 1, 1024), o.top = router.count("top", 1, 1024);
            if (router.has("groups")) {
                const Fields g = router.sub("groups");
                o.groups = g.count("count", 1, 1024), o.keep = g.count("keep", 1, 1024);
            }
            const auto cut = [&](const Fields &f) {
                const float v = f.has("limit") ? (float)f.num("limit") : 0.f;
                if (rc == VH_OK && f.has("limit") && !(v > 0.f)) rc = fail("config.json: %s.limit is not above 0", f.where.c_str());
                return v;
            };
            o.ff = expert.count("ff", 1, 1 << 20), o.limit = cut(expert);
            if (mlp.has("shared")) {
                o.shared = true;
                o.shared_ff = mlp.sub("shared").count("ff", 1, 1 << 20), o.shared_limit = cut(mlp.sub("shared"));
            }
        }
        if (rc != VH_OK) return rc;
        if (o.heads % o.kv_heads) return fail("config.json: layer %zu: %d heads are no multiple of %d", i, o.heads, o.kv_heads);
        if (o.kind == KitodraLayer::KEY_VALUE && o.vdim != o.dim) return fail("config.json: layer %zu: keys of %d are values of %d", i, o.dim, o.vdim);
        if (o.rot_dims % 2 || o.rot_dims > o.dim) return fail("config.json: layer %zu turns %d of %d dimensions", i, o.rot_dims, o.dim);
        if (o.rot_dims > 0 && !(o.rot_base > 0.0)) return fail("config.json: layer %zu: rot.base is not above 0", i);
        if (o.n_experts % o.groups || o.keep > o.groups) return fail("config.json: layer %zu: %d of %d groups of %d experts", i, o.keep, o.groups, o.n_experts);
        if (o.top > (o.groups > 1 ? o.keep * (o.n_experts / o.groups) : o.n_experts))
            return fail("config.json: layer %zu: %d of %d experts in %d groups", i, o.top, o.n_experts, o.keep);
        c->layers.push_back(o);
    }
    for (size_t i = 0; i < c->layers.size(); i++) {
        int at = (int)i;
        for (size_t n = 0; c->layers[at].weights_of >= 0; n++) {
            if (n == c->layers.size()) return fail("config.json: layer %zu: weights_of leads in a circle", i);
            at = c->layers[at].weights_of;
        }
        const KitodraLayer &a = c->layers[i], &b = c->layers[at];
        if (a.kind != b.kind || a.heads != b.heads || a.kv_heads != b.kv_heads || a.dim != b.dim || a.vdim != b.vdim || a.experts != b.experts)
            return fail("config.json: layer %zu is of another kind than layer %d, whose weights it uses", i, at);
        c->own.push_back(at);
    }
    return rc;
}

// A float32 logarithm of a decay that a kernel may multiply with any count of tokens: 0 becomes a decay that nothing outlives.
float decay_log2(double d) { return d > 0.0 ? (float)fmax(log2(d), -1e4) : -1e4f; }

int build_kitodra_attention(Builder &b, const KitodraLayer &s, const std::string &l, int W, int router_cols, MixModel *x, MixLayer *o, int *router_col) {
    const std::string mix = l + "mix.";
    const bool diff = s.kind == KitodraLayer::DIFFERENTIAL;
    AttnMixer &a = o->attn;
    o->has_attn = true;
    a.by_heads = a.norm = true;
    a.heads = s.heads, a.kv_heads = s.kv_heads, a.k_dim = s.dim, a.v_dim = s.vdim, a.scale = s.scale, a.softcap = s.softcap, a.maps = diff ? 2 : 1;
    const int qd = s.heads * a.maps * s.dim, kd = s.kv_heads * a.maps * s.dim, vd = s.kv_heads * s.vdim, od = s.heads * s.vdim;
    a.k_col = b.pad(qd, 16), a.v_col = diff ? a.k_col + b.pad(kd, 16) : -1;
    *router_col = diff ? a.v_col + b.pad(vd, 16) : a.k_col + b.pad(kd, 16);
    VHC(b.packed(&o->in, *router_col + router_cols, W));
    std::vector<float> bias(o->in.n, 0.f), v;
    const auto part = [&](const char *name, int n, int col) -> int {
        VHC(b.pack(mix + name, n, W, 0, n, o->in, col, 1, 0));
        VHC(b.floats(mix + name + ".b", {n}, &v));
        std::copy(v.begin(), v.end(), bias.begin() + col);
        return VH_OK;
    };
    VHC(part("q", qd, a.q_col));
    VHC(part("k", kd, a.k_col));
    if (diff) VHC(part("v", vd, a.v_col));
    VHC(b.upload(bias, &a.in_bias));
    VHC(b.packed(&o->out, W, od));
    VHC(b.pack(mix + "o", W, od, 0, W, o->out, 0, 1, 0));
    VHC(b.vec(mix + "o.b", W, &o->out_bias));
    if (diff) {
        a.chunk = s.mask;
        VHC(b.vec(mix + "q.norm", s.dim, &a.norm_q));
        VHC(b.vec(mix + "k.norm", s.dim, &a.norm_k));
        double sum[2] = {0, 0};
        for (int n = 0; n < 2; n++) {
            std::vector<float> q, k;
            VHC(b.floats(mix + (n ? "lq2" : "lq1"), {s.dim}, &q));
            VHC(b.floats(mix + (n ? "lk2" : "lk1"), {s.dim}, &k));
            for (int d = 0; d < s.dim; d++) sum[n] += (double)q[d] * k[d];
        }
        a.diff_lambda = (float)(exp(sum[0]) - exp(sum[1]) + s.diff), a.diff_scale = 1.f - s.diff;
    } else {
        a.window = s.mask;
        VHC(b.upload(std::vector<float>(s.heads, 0.f), &a.sink));
        if (s.rot_dims > 0) {
            Rotation r;
            double both;
            rotary_frequencies(s.rot_dims, s.rot_base, false, 0, 0, 0, 0, &r.freqs, &both);
            for (size_t k = 0; k < x->rotations.size(); k++)
                if (x->rotations[k].freqs == r.freqs) a.rotation = (int)k;
            if (a.rotation < 0) {
                a.rotation = (int)x->rotations.size();
                x->rotations.push_back(r);
            }
        }
    }
    return VH_OK;
}

int build_kitodra_lightning(Builder &b, const KitodraLayer &s, const std::string &l, int W, int router_cols, MixLayer *o, int *router_col) {
    const std::string mix = l + "mix.";
    DecayMixer &t = o->decay;
    o->has_decay = true;
    t.heads = s.heads, t.vdim = s.vdim, t.dim_pad = b.pad(s.dim, 32), t.v_pad = b.pad(s.vdim, 16);
    const int qs = s.heads * t.dim_pad, vs = s.heads * t.v_pad, vd = s.heads * s.vdim;
    t.split = 2 * qs + vs, t.g_col = 0;
    *router_col = vs;
    VHC(b.packed(&o->in, t.split + vs + router_cols, W));
    // heads of `dim` rows spread to heads of `to`
    const auto spread = [&](const char *name, int dim, int to, int row0) {
        return b.pack_rows(mix + name, s.heads * dim, W, s.heads * to, o->in, row0, [&](int r) { return r % to < dim ? r / to * dim + r % to : -1; });
    };
    VHC(spread("q", s.dim, t.dim_pad, 0));
    VHC(spread("k", s.dim, t.dim_pad, qs));
    VHC(spread("v", s.vdim, t.v_pad, 2 * qs));
    VHC(spread("g", s.vdim, t.v_pad, t.split));
    std::vector<float> w, wp(vs, 0.f), decay;
    VHC(b.floats(mix + "norm", {vd}, &w));
    for (int i = 0; i < vd; i++) wp[i / s.vdim * t.v_pad + i % s.vdim] = w[i];
    VHC(b.upload(wp, &t.norm));
    for (double d : s.decay) {
        decay.push_back((float)(d - 1.0));
        decay.push_back(decay_log2(d));
    }
    VHC(b.upload(decay, &t.decay));
    VHC(b.packed(&o->out, W, vs));
    return b.pack_placed(mix + "o", W, vd, W, vs, o->out, 0, [&](int r, int k) -> int64_t {
        return k % t.v_pad < s.vdim ? (int64_t)r * vd + k / t.v_pad * s.vdim + k % t.v_pad : -1;
    });
}

int build_kitodra_experts(Builder &b, const KitodraLayer &s, const std::string &mlp, int W, MixLayer *o) {
    ExpertMlp &e = o->moe;
    o->has_experts = true;
    e.experts = s.n_experts, e.top = s.top, e.groups = s.groups, e.keep = s.keep, e.shared = s.shared;
    e.limit = s.limit, e.shared_limit = s.shared_limit, e.alpha = 1.702f, e.add = 1.f;
    VHC(b.vec(mlp + "correction", s.n_experts, &e.correction));
    // n maps of that feed-forward size, one behind the other
    const auto maps = [&](int n, int ff, const std::function<std::string(int)> &name, Linear *gate_up, Linear *down, int *ff_pad) -> int {
        const int fp = *ff_pad = b.pad(ff, 64), wp = b.pad(W, 32);
        VHC(b.packed(gate_up, n * 2 * fp, W));
        VHC(b.packed(down, n * wp, ff));
        for (int i = 0; i < n; i++) {
            const std::string p = mlp + name(i);
            VHC(b.pack(p + ".gate", ff, W, 0, ff, *gate_up, i * 2 * fp, 2, 0));
            VHC(b.pack(p + ".up", ff, W, 0, ff, *gate_up, i * 2 * fp + 16, 2, 0));
            VHC(b.pack(p + ".down", W, ff, 0, W, *down, i * wp, 1, 0));
        }
        gate_up->n /= n, down->n /= n;
        return VH_OK;
    };
    VHC(maps(s.n_experts, s.ff, [](int i) { return "e" + std::to_string(i); }, &e.gate_up, &e.down, &e.ff_pad));
    if (s.shared) VHC(maps(1, s.shared_ff, [](int) { return std::string("shared"); }, &e.shared_gate_up, &e.shared_down, &e.shared_pad));
    return VH_OK;
}

int build_kitodra(Builder &b, const Json &config, MixModel *x, vh_config *cfg) {
    KitodraConfig c;
    VHC(parse_kitodra(config, &c));
    cfg->hidden = c.width, cfg->vocab = c.vocab, cfg->eps = c.eps;
    x->eps = c.eps;
    const int W = c.width;
    std::vector<int> place(c.layers.size(), -1);  // of a layer with tensors of its own, in the program
    for (size_t i = 0; i < c.layers.size(); i++) {
        if (c.own[i] != (int)i) continue;
        const KitodraLayer &s = c.layers[i];
        const std::string l = "l" + std::to_string(i) + ".";
        MixLayer o;
        VHC(b.vec(l + "norm1", W, &o.norm1));
        int router_col = 0;
        const int router_cols = s.experts ? s.n_experts : 0;
        if (s.kind == KitodraLayer::LIGHTNING) {
            VHC(build_kitodra_lightning(b, s, l, W, router_cols, &o, &router_col));
            x->recurrent = true;
        } else {
            VHC(build_kitodra_attention(b, s, l, W, router_cols, x, &o, &router_col));
        }
        if (s.experts) {
            VHC(b.pack(l + "mlp.router", s.n_experts, W, 0, s.n_experts, o.in, (o.has_decay ? o.decay.split : 0) + router_col, 1, 0));
            VHC(build_kitodra_experts(b, s, l + "mlp.", W, &o));
            o.moe.router_col = router_col;
        }
        place[i] = (int)x->layers.size();
        x->layers.push_back(o);
    }
    for (size_t i = 0; i < c.layers.size(); i++) {
        LayerRun r;
        r.layer = place[c.own[i]];
        x->runs.push_back(r);
    }
    std::vector<float> emb;
    VHC(b.floats("embed", {c.vocab, W}, &emb));
    VHC(b.upload(emb, &b.m->embedding));
    if (c.buckets > 0) {
        VHC(b.floats("bigram", {c.buckets + 1, W}, &emb));
        VHC(b.upload(emb, &x->pairs));
        x->buckets = c.buckets, x->mul_prev = c.mul_prev, x->mul_cur = c.mul_cur;
    }
    VHC(b.vec("final.norm", W, &b.m->final_norm));
    VHC(b.packed(&x->head, c.vocab, W));
    return b.pack("embed", c.vocab, W, 0, c.vocab, x->head, 0, 1, 0);
}

int check_kitodra(const Json &config) {
    KitodraConfig c;
    return parse_kitodra(config, &c);
}

// ---------------------------------------------------------------- Fitevik
struct FitevikLayer {
    bool states = false;          // hgrn2, else attention
    int heads = 1, kv_heads = 1, dim = 1, vdim = 1, window = 0, kv_from = -1;
    float scale = 1.f;
    enum Ff { NONE, DENSE, EXPERTS } mlp = NONE;
    int ff = 1, experts = 1, top = 1;
};
struct FitevikConfig {
    std::vector<FitevikLayer> layers;
    float eps = 1e-5f, logit_scale = 1.f;
    int vocab = 1, width = 1, max_positions = 1;
};

int parse_fitevik(const Json &j, FitevikConfig *c) {
    int rc = VH_OK;
    const Fields root("config", &j, &rc);
    c->vocab = root.count("vocab");
    c->width = root.count("width", 1, 15360);
    c->max_positions = root.count("max_positions");
    c->logit_scale = (float)root.num("logit_scale");
    c->eps = (float)root.sub("norm").num("eps");
    const Json *layers = root.need("layers", Json::ARR);
    if (rc != VH_OK) return rc;
    if (layers->arr.empty()) return fail("config.json: no layers");
    for (size_t i = 0; i < layers->arr.size(); i++) {
        const Fields l("layers[" + std::to_string(i) + "]", &layers->arr[i], &rc);
        const Json *type = l.need("type", Json::STR);
        if (rc != VH_OK) return rc;
        FitevikLayer o;
        o.states = type->str == "hgrn2";
        if (!o.states && type->str != "attention") return fail("config.json: layer %zu has the unknown mixer type '%s'", i, type->str.c_str());
        const Fields mx = l.sub("mixer");
        o.heads = mx.count("heads", 1, 4096);
        o.dim = mx.count("dim", 1, o.states ? 512 : 2048), o.vdim = mx.count("vdim", 1, o.states ? 512 : 2048);
        if (!o.states) {
            o.kv_heads = mx.count("kv_heads", 1, 4096);
            o.scale = (float)mx.num("scale");
            if (mx.has("mask")) o.window = mx.sub("mask").count("size", 1, 1 << 30);
            if (mx.has("kv_from")) o.kv_from = mx.count("kv_from", 0, 1 << 16);
        }
        if (l.has("mlp")) {
            const Fields mlp = l.sub("mlp");
            const Json *kind = mlp.need("kind", Json::STR);
            if (rc != VH_OK) return rc;
            if (kind->str == "dense") {
                o.mlp = FitevikLayer::DENSE;
                o.ff = mlp.count("ff", 1, 1 << 20);
            } else if (kind->str == "moe") {
                o.mlp = FitevikLayer::EXPERTS;
                o.experts = mlp.sub("router").count("experts", 1, 1024), o.top = mlp.sub("router").count("top", 1, 1024);
                o.ff = mlp.sub("expert").count("ff", 1, 1 << 20);
            } else {
                return fail("config.json: layer %zu has the unknown feed-forward '%s'", i, kind->str.c_str());
            }
        }
        if (rc != VH_OK) return rc;
        if (o.heads % o.kv_heads) return fail("config.json: layer %zu: %d heads are no multiple of %d", i, o.heads, o.kv_heads);
        if (!o.states && (int64_t)o.kv_heads * o.dim > 15360) return fail("config.json: layer %zu: %d key heads of %d", i, o.kv_heads, o.dim);
        if (o.top > o.experts) return fail("config.json: layer %zu: %d of %d experts", i, o.top, o.experts);
        if (o.kv_from >= 0) {
            if (o.kv_from >= (int)i || c->layers[o.kv_from].states || c->layers[o.kv_from].kv_from >= 0)
                return fail("config.json: layer %zu: layer %d holds no keys for it", i, o.kv_from);
            const FitevikLayer &f = c->layers[o.kv_from];
            if (f.kv_heads != o.kv_heads || f.dim != o.dim || f.vdim != o.vdim)
                return fail("config.json: layer %zu: the keys of layer %d are of another kind", i, o.kv_from);
        }
        c->layers.push_back(o);
    }
    return rc;
}

int build_fitevik_attention(Builder &b, const FitevikLayer &s, const std::string &mix, int W, MixLayer *o) {
    AttnMixer &a = o->attn;
    o->has_attn = true;
    a.by_heads = a.row_norm = true;
    a.heads = s.heads, a.kv_heads = s.kv_heads, a.k_dim = s.dim, a.v_dim = s.vdim, a.scale = s.scale, a.window = s.window, a.kv_from = s.kv_from;
    const int qd = s.heads * s.dim, kd = s.kv_heads * s.dim, vd = s.kv_heads * s.vdim, od = s.heads * s.vdim;
    a.k_col = b.pad(qd, 16), a.v_col = a.k_col + b.pad(kd, 16);
    VHC(b.packed(&o->in, s.kv_from < 0 ? a.v_col + vd : qd, W));
    VHC(b.pack(mix + "q", qd, W, 0, qd, o->in, a.q_col, 1, 0));
    VHC(b.vec(mix + "q.norm", qd, &a.norm_q));
    if (s.kv_from < 0) {
        VHC(b.pack(mix + "k", kd, W, 0, kd, o->in, a.k_col, 1, 0));
        VHC(b.pack(mix + "v", vd, W, 0, vd, o->in, a.v_col, 1, 0));
        VHC(b.vec(mix + "k.norm", kd, &a.norm_k));
    } else {
        a.k_col = a.v_col = 0;
    }
    VHC(b.packed(&o->out, W, od));
    VHC(b.pack(mix + "o", W, od, 0, W, o->out, 0, 1, 0));
    VHC(b.vec(mix + "sink", s.heads, &a.sink));
    // the matrix that mixes scores, and every head's slope as the mixing leaves it
    const TensorView *t;
    VHC(b.view(mix + "talk", {s.heads, s.heads}, &t));
    const size_t bytes = (size_t)s.heads * s.heads * 2;
    void *p = vx_alloc_permanent(b.be, (bytes + 15) / 16 * 16 + 16);
    if (!p) return fail("device memory: %s", vx_last_error());
    b.m->adopted.push_back(p);
    VXC(vx_to_device(b.be, p, t->data, bytes));
    a.talk = p;
    std::vector<float> talk, slopes;
    VHC(b.floats(mix + "talk", {s.heads, s.heads}, &talk));
    for (int h = 0; h < s.heads; h++) {
        double sum = 0.0;
        for (int g = 0; g < s.heads; g++) sum += (double)talk[(size_t)h * s.heads + g] * exp2(-8.0 * (g + 1) / s.heads);
        slopes.push_back((float)sum);
    }
    return b.upload(slopes, &a.slopes);
}

int build_fitevik_states(Builder &b, const FitevikLayer &s, const std::string &mix, int W, MixLayer *o) {
    ForgetMixer &t = o->forget;
    o->has_forget = true;
    t.heads = s.heads, t.vdim = s.vdim, t.dim_pad = b.pad(s.dim, 32), t.v_pad = b.pad(s.vdim, 16);
    const int qs = s.heads * t.dim_pad, vs = s.heads * t.v_pad, vd = s.heads * s.vdim, fd = s.heads * s.dim;
    VHC(b.packed(&o->in, 2 * qs + vs, W));
    const auto spread = [&](const char *name, int dim, int to, int row0) {  // heads of `dim` rows to heads of `to`
        return b.pack_rows(mix + name, s.heads * dim, W, s.heads * to, o->in, row0, [&](int r) { return r % to < dim ? r / to * dim + r % to : -1; });
    };
    VHC(spread("q", s.dim, t.dim_pad, 0));
    VHC(spread("v", s.vdim, t.v_pad, qs));
    VHC(spread("f", s.dim, t.dim_pad, qs + vs));
    std::vector<float> fb, lower, bias(qs, 0.f), keep(qs, 0.f), w;  // (channels that pad a head write nothing)
    VHC(b.floats(mix + "f.b", {fd}, &fb));
    VHC(b.floats(mix + "lower", {fd}, &lower));
    for (int i = 0; i < fd; i++) {
        const int at = i / s.dim * t.dim_pad + i % s.dim;
        bias[at] = fb[i], keep[at] = (float)(1.0 - (double)lower[i]);
    }
    VHC(b.upload(bias, &t.bias));
    VHC(b.upload(keep, &t.keep));
    VHC(b.floats(mix + "norm", {s.vdim}, &w));
    w.resize(t.v_pad, 0.f);
    VHC(b.upload(w, &t.norm));
    VHC(b.packed(&o->out, W, vs));
    return b.pack_placed(mix + "o", W, vd, W, vs, o->out, 0, [&](int r, int k) -> int64_t {
        return k % t.v_pad < s.vdim ? (int64_t)r * vd + k / t.v_pad * s.vdim + k % t.v_pad : -1;
    });
}

int build_fitevik_mlp(Builder &b, const FitevikLayer &s, const std::string &mlp, int W, MixLayer *o) {
    if (s.mlp == FitevikLayer::DENSE) {
        o->has_mlp = o->relu2 = true;
        o->ff = s.ff, o->ff_pad = b.pad(s.ff, 64);
        VHC(b.packed(&o->gate_up, o->ff_pad, W));
        VHC(b.pack(mlp + "up", s.ff, W, 0, s.ff, o->gate_up, 0, 1, 0));
        VHC(b.packed(&o->down, W, s.ff));
        VHC(b.pack(mlp + "down", W, s.ff, 0, W, o->down, 0, 1, 0));
        std::vector<float> up;
        VHC(b.floats(mlp + "up.b", {s.ff}, &up));
        up.resize(o->ff_pad, 0.f);
        VHC(b.upload(up, &o->up_bias));
        return b.vec(mlp + "down.b", W, &o->down_bias);
    }
    ExpertMlp &e = o->moe;
    o->has_experts = true;
    e.experts = s.experts, e.top = s.top, e.relu2 = e.softmax = true;
    VHC(b.packed(&e.router, s.experts, W));
    VHC(b.pack(mlp + "router", s.experts, W, 0, s.experts, e.router, 0, 1, 0));
    VHC(b.vec(mlp + "router.b", s.experts, &e.router_bias));
    const int fp = e.ff_pad = b.pad(s.ff, 64), wp = b.pad(W, 32);
    VHC(b.packed(&e.gate_up, s.experts * fp, W));
    VHC(b.packed(&e.down, s.experts * wp, s.ff));
    for (int i = 0; i < s.experts; i++) {
        const std::string p = mlp + "e" + std::to_string(i);
        VHC(b.pack(p + ".up", s.ff, W, 0, s.ff, e.gate_up, i * fp, 1, 0));
        VHC(b.pack(p + ".down", W, s.ff, 0, W, e.down, i * wp, 1, 0));
    }
    e.gate_up.n = fp, e.down.n = wp;
    return VH_OK;
}

int build_fitevik(Builder &b, const Json &config, MixModel *x, vh_config *cfg) {
    FitevikConfig c;
    VHC(parse_fitevik(config, &c));
    cfg->hidden = c.width, cfg->vocab = c.vocab, cfg->eps = c.eps;
    x->eps = c.eps, x->branch_norm = true, x->logit_mult = c.logit_scale, x->max_positions = c.max_positions;
    const int W = c.width;
    for (size_t i = 0; i < c.layers.size(); i++) {
        const FitevikLayer &s = c.layers[i];
        const std::string l = "l" + std::to_string(i) + ".";
        MixLayer o;
        VHC(b.vec(l + "norm1", W, &o.norm1));
        VHC(b.vec(l + "norm1.b", W, &o.norm1b));
        VHC(s.states ? build_fitevik_states(b, s, l + "mix.", W, &o) : build_fitevik_attention(b, s, l + "mix.", W, &o));
        x->recurrent = x->recurrent || s.states;
        if (s.mlp != FitevikLayer::NONE) {
            VHC(b.vec(l + "norm2", W, &o.norm2));
            VHC(b.vec(l + "norm2.b", W, &o.norm2b));
            VHC(build_fitevik_mlp(b, s, l + "mlp.", W, &o));
        }
        x->layers.push_back(o);
        LayerRun r;
        r.layer = (int)i;
        x->runs.push_back(r);
    }
    std::vector<float> emb;
    VHC(b.floats("embed", {c.vocab, W}, &emb));
    VHC(b.upload(emb, &b.m->embedding));
    VHC(b.floats("pos", {c.max_positions, W}, &emb));
    VHC(b.upload(emb, &x->positions));
    VHC(b.vec("embed.norm", W, &x->emb_norm));
    VHC(b.vec("embed.norm.b", W, &x->emb_norm_b));
    VHC(b.vec("final.norm", W, &b.m->final_norm));
    VHC(b.vec("final.norm.b", W, &x->final_norm_b));
    VHC(b.packed(&x->head, c.vocab, W));
    return b.pack("head", c.vocab, W, 0, c.vocab, x->head, 0, 1, 0);
}

int check_fitevik(const Json &config) {
    FitevikConfig c;
    return parse_fitevik(config, &c);
}

// ---------------------------------------------------------------- registry
struct Architecture {
    const char *name;                                                    // config.json "architecture"
    int (*check)(const Json &);
    int (*build)(Builder &, const Json &, MixModel *, vh_config *);      // fills program, weights, and width / vocab / eps
};
const Architecture kArchitectures[] = {
    {"Lozedra", check_lozedra, build_lozedra},
    {"Tulipel", check_tulipel, build_tulipel},
    {"Kitodra", check_kitodra, build_kitodra},
    {"Fitevik", check_fitevik, build_fitevik},
};

const Architecture *find_architecture(const Json &config) {
    const Json *name = config.type == Json::OBJ ? config.get("architecture") : nullptr;
    if (!name || name->type != Json::STR) {
        fail("config.json names no architecture");
        return nullptr;
    }
    for (const Architecture &a : kArchitectures)
        if (name->str == a.name) return &a;
    std::string known;
    for (const Architecture &a : kArchitectures) known += std::string(known.empty() ? "" : ", ") + a.name;
    fail("config.json: unknown architecture '%s' (known: %s)", name->str.c_str(), known.c_str());
    return nullptr;
}

}  // namespace
}  // namespace vh

using namespace vh;

extern "C" {

const char *vh_architecture_name(int i) {
    return i >= 0 && i < (int)(sizeof kArchitectures / sizeof kArchitectures[0]) ? kArchitectures[i].name : nullptr;
}

int vh_distance_bucket(int distance, int rows, int bias_max) { return distance_bucket(distance, rows, bias_max); }

int vh_rotary_frequencies(int dims, double base, double factor, double original, double fast, double slow, double *freqs, double *both) {
    if (dims < 2 || dims % 2 || !(base > 1.0) || !freqs || !both) return fail("vh_rotary_frequencies: bad arguments");
    std::vector<double> f;
    rotary_frequencies(dims, base, factor > 0, factor, original, fast, slow, &f, both);
    memcpy(freqs, f.data(), f.size() * sizeof(double));
    return VH_OK;
}

int vh_spell_out_rows(int rank, int dim, int vdim) { return rank > 0 && dim > 0 && vdim > 0 ? spell_out_rows(rank, dim, vdim) : 0; }

int vh_check_config(const char *json_text) {
    Json config;
    if (!json_text || !parse_json(json_text, strlen(json_text), &config)) return fail("config.json is not JSON");
    const Architecture *arch = find_architecture(config);
    return arch ? arch->check(config) : (int)VH_ERR;
}

int vh_model_load(vx_backend *be, const char *path, const vh_load_options *opt, vh_model **out) {
    if (!be || !path || !opt || !out) return fail("vh_model_load: null argument");
    *out = nullptr;
    struct stat sb;
    if (stat(path, &sb) != 0) return fail("%s: %s", path, strerror(errno));
    if (!S_ISDIR(sb.st_mode)) return vh_model_load_gguf(be, path, opt, out);
    const std::string dir = path;
    Json config;
    {
        Mapped text;
        VHC(text.open(dir + "/config.json"));
        if (!parse_json((const char *)text.base, text.size, &config)) return fail("%s/config.json is not JSON", path);
    }
    const Architecture *arch = find_architecture(config);
    if (!arch) return VH_ERR;
    VHC(arch->check(config));
    SafeTensors st;
    VHC(st.open(dir + "/model.safetensors"));
    vh_config c;
    memset(&c, 0, sizeof c);
    c.block_size = opt->block_size > 0 ? opt->block_size : 16;
    c.pool_blocks = opt->pool_blocks, c.max_seqs = opt->max_seqs, c.max_blocks_per_seq = opt->max_blocks_per_seq, c.max_batch = opt->max_batch;
    if (c.block_size % 8 || c.pool_blocks <= 0 || c.max_seqs <= 0 || c.max_blocks_per_seq <= 0 || c.max_batch <= 0 || c.max_batch > 1024)
        return fail("bad pool or batch sizes");
    if (opt->dtype < VH_DTYPE_DEFAULT || opt->dtype > VH_DTYPE_F32) return fail("unknown dtype %d", opt->dtype);
    vh_model *m = new vh_model();
    m->be = be;
    m->mix.reset(new MixModel());
    m->mix->act = opt->dtype == VH_DTYPE_F32 ? VX_ACT_F32 : VX_ACT_BF16;
    int rc;
    {
        Builder b{be, &st, m, c.block_size};
        rc = arch->build(b, config, m->mix.get(), &c);
    }
    c.num_layers = (int)m->mix->runs.size();  // (the layers that hold a cache: every pass has its own)
    m->cfg = c;
    if (rc == VH_OK) rc = mix_finish(m);
    if (rc != VH_OK) {
        const std::string keep = vh_last_error();
        vh_model_destroy(m);
        vh_set_error(keep.c_str());
        return VH_ERR;
    }
    *out = m;
    return VH_OK;
}

}  // extern "C"
