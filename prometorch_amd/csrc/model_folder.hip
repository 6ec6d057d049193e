// Model folders: a safetensors reader, the registry of architectures config.json may name, and their loaders.
//
// safetensors: u64 length n (little endian) | n bytes of JSON: name -> {dtype, shape, data_offsets [begin, end)} | data.
// A loader turns config.json and the tensors into a ptm_block_config: bfloat16 matrices are uploaded with rows padded to
// multiples of 64 values, projections of one input stacked, heads padded to multiples of 8 rows or columns; vectors become fp32.
#include "dense.h"
#include "json.h"
#include "model.h"

#include <fcntl.h>
#include <sys/mman.h>
#include <sys/stat.h>
#include <unistd.h>

#include <cmath>
#include <new>

using namespace ptm;

struct ptm_safetensors {
    const uint8_t* map = nullptr;
    size_t size = 0;
    struct Entry { std::string name, dtype; std::vector<int64_t> dims; int64_t begin, end; };
    std::vector<Entry> entries;
    const uint8_t* data = nullptr;
};

namespace {

int64_t dtype_bytes(const std::string& t) {
    if (t == "BF16" || t == "F16" || t == "I16" || t == "U16") return 2;
    if (t == "F32" || t == "I32" || t == "U32") return 4;
    if (t == "F64" || t == "I64" || t == "U64") return 8;
    if (t == "I8" || t == "U8" || t == "BOOL") return 1;
    return 0;
}

// a JSON number that is an integer in [0, 2^53)
bool as_int(const Json* j, int64_t* out) {
    if (!j || j->kind != Json::Number || !(j->num >= 0.0) || j->num >= 9007199254740992.0 || j->num != std::floor(j->num)) return false;
    *out = (int64_t)j->num;
    return true;
}

int st_parse(ptm_safetensors* f) {
    if (f->size < 8) return PTM_E_FORMAT;
    uint64_t n;
    memcpy(&n, f->map, 8);
    if (n > f->size - 8) return PTM_E_FORMAT;
    Json root;
    if (!JsonParser(reinterpret_cast<const char*>(f->map) + 8, (size_t)n).parse(&root) || root.kind != Json::Object) return PTM_E_FORMAT;
    f->data = f->map + 8 + n;
    const int64_t room = (int64_t)(f->size - 8 - (size_t)n);
    for (const auto& m : root.members) {
        if (m.first == "__metadata__") continue;
        const Json *dt = m.second.find("dtype"), *sh = m.second.find("shape"), *of = m.second.find("data_offsets");
        if (!dt || dt->kind != Json::String || !sh || sh->kind != Json::Array || sh->items.size() > 8 || !of || of->kind != Json::Array || of->items.size() != 2) return PTM_E_FORMAT;
        ptm_safetensors::Entry e;
        e.name = m.first;
        e.dtype = dt->str;
        int64_t count = 1;
        for (const Json& d : sh->items) {
            int64_t v;
            if (!as_int(&d, &v) || (v > 0 && count > (int64_t)1 << 46) || (v > 0 && count * v / v != count)) return PTM_E_FORMAT;
            e.dims.push_back(v);
            count *= v;
        }
        if (!as_int(&of->items[0], &e.begin) || !as_int(&of->items[1], &e.end) || e.begin > e.end || e.end > room) return PTM_E_FORMAT;
        const int64_t b = dtype_bytes(e.dtype);
        if (b && count * b != e.end - e.begin) return PTM_E_FORMAT;
        f->entries.push_back(std::move(e));
    }
    return PTM_OK;
}

}  // namespace

extern "C" {

void ptm_safetensors_close(ptm_safetensors* f) {
    if (!f) return;
    if (f->map) munmap(const_cast<uint8_t*>(f->map), f->size);
    delete f;
}

int ptm_safetensors_open(const char* path, ptm_safetensors** out) {
    if (!path || !out) return PTM_E_NULL;
    *out = nullptr;
    const int fd = open(path, O_RDONLY | O_CLOEXEC);
    if (fd < 0) return PTM_E_IO;
    struct stat st;
    if (fstat(fd, &st) != 0 || st.st_size <= 0) { close(fd); return PTM_E_IO; }
    void* p = mmap(nullptr, (size_t)st.st_size, PROT_READ, MAP_PRIVATE, fd, 0);
    close(fd);
    if (p == MAP_FAILED) return PTM_E_IO;
    ptm_safetensors* f = new (std::nothrow) ptm_safetensors();
    if (!f) { munmap(p, (size_t)st.st_size); return PTM_E_STATE; }
    f->map = static_cast<const uint8_t*>(p);
    f->size = (size_t)st.st_size;
    const int rc = st_parse(f);
    if (rc != PTM_OK) { ptm_safetensors_close(f); return rc; }
    *out = f;
    return PTM_OK;
}

int64_t ptm_safetensors_n_tensors(const ptm_safetensors* f) { return f ? (int64_t)f->entries.size() : 0; }

int ptm_safetensors_tensor_at(const ptm_safetensors* f, int64_t i, ptm_st_tensor* out) {
    if (!f || !out) return PTM_E_NULL;
    if (i < 0 || i >= (int64_t)f->entries.size()) return PTM_E_RANGE;
    const auto& e = f->entries[(size_t)i];
    *out = ptm_st_tensor{};
    out->name = e.name.c_str();
    out->dtype = e.dtype.c_str();
    out->n_dims = (int32_t)e.dims.size();
    for (size_t d = 0; d < e.dims.size(); ++d) out->dims[d] = e.dims[d];
    out->nbytes = e.end - e.begin;
    out->data = f->data + e.begin;
    return PTM_OK;
}

int ptm_safetensors_find(const ptm_safetensors* f, const char* name, ptm_st_tensor* out) {
    if (!f || !name || !out) return PTM_E_NULL;
    for (size_t i = 0; i < f->entries.size(); ++i)
        if (f->entries[i].name == name) return ptm_safetensors_tensor_at(f, (int64_t)i, out);
    return PTM_E_NOT_FOUND;
}

}  // extern "C"

namespace {

int read_file(const std::string& path, std::string* out) {
    FILE* f = fopen(path.c_str(), "rb");
    if (!f) return PTM_E_IO;
    char buf[65536];
    size_t n;
    while ((n = fread(buf, 1, sizeof buf, f)) > 0) out->append(buf, n);
    const bool bad = ferror(f) != 0;
    fclose(f);
    return bad ? PTM_E_IO : PTM_OK;
}

// Reads sizes and constants; the first missing or unusable one leaves PTM_E_FORMAT in rc.
struct ConfigReader {
    int rc = PTM_OK;
    int32_t size(const Json* o, const char* key, int32_t def = -1) {  // def < 0: required
        const Json* j = o ? o->find(key) : nullptr;
        if (!j || j->is_null()) {
            if (def < 0) rc = PTM_E_FORMAT;
            return def < 0 ? 0 : def;
        }
        int64_t v;
        if (!as_int(j, &v) || v > 0x3fffffff) { rc = PTM_E_FORMAT; return 0; }
        return (int32_t)v;
    }
    double real(const Json* o, const char* key, double def = NAN) {  // def NaN: required
        const Json* j = o ? o->find(key) : nullptr;
        if (!j || j->is_null()) {
            if (std::isnan(def)) rc = PTM_E_FORMAT;
            return std::isnan(def) ? 0.0 : def;
        }
        if (j->kind != Json::Number || !std::isfinite(j->num)) { rc = PTM_E_FORMAT; return 0.0; }
        return j->num;
    }
    std::string text(const Json* o, const char* key) {
        const Json* j = o ? o->find(key) : nullptr;
        if (!j || j->kind != Json::String) { rc = PTM_E_FORMAT; return {}; }
        return j->str;
    }
    ptm_rotation rotation(const Json* o) {
        ptm_rotation r{};
        r.base = 1.0;
        if (!o || o->is_null()) return r;
        r.dims = size(o, "dims");
        r.base = real(o, "base");
        const Json* s = o->find("scaling");
        if (s && !s->is_null()) {
            r.factor = real(s, "factor");
            r.original = real(s, "original");
            r.fast = real(s, "fast");
            r.slow = real(s, "slow");
            if (!(r.factor > 0.0 && r.original > 0.0 && r.fast > 0.0 && r.slow > 0.0)) rc = PTM_E_FORMAT;
        }
        return r;
    }
};

// A padded bfloat16 matrix put together on the host from tensors of the file.
struct HostMatrix {
    int rows, cols, ld;
    std::vector<uint16_t> v;
    HostMatrix(int r, int c) : rows(r), cols(c), ld(up64(c)), v((size_t)r * (size_t)up64(c), 0) {}
};

struct FolderLoader {
    ptm_model* m;
    const ptm_safetensors* f;

    // tensor of exactly these dimensions (one, if cols is 0)
    int tensor(const std::string& name, int64_t rows, int64_t cols, ptm_st_tensor* t) const {
        const int rc = ptm_safetensors_find(f, name.c_str(), t);
        if (rc != PTM_OK) return rc;
        if (t->n_dims != (cols ? 2 : 1) || t->dims[0] != rows || (cols && t->dims[1] != cols)) return PTM_E_SHAPE;
        return PTM_OK;
    }
    // rows of a tensor: source row g * group + r goes to dst row at + g * padded + r; likewise columns
    int place(HostMatrix& h, const std::string& name, int rows, int cols, int at, int group = 0, int padded = 0, int col_group = 0,
              int col_padded = 0) const {
        ptm_st_tensor t;
        const int rc = tensor(name, rows, cols, &t);
        if (rc != PTM_OK) return rc;
        if (strcmp(t.dtype, "BF16") != 0) return PTM_E_UNSUPPORTED;
        if (!group) group = padded = rows;
        if (!col_group) col_group = col_padded = cols;
        const uint8_t* src = static_cast<const uint8_t*>(t.data);
        for (int r = 0; r < rows; ++r) {
            uint16_t* dst = h.v.data() + (size_t)(at + r / group * padded + r % group) * h.ld;
            for (int c = 0; c < cols; c += col_group)
                memcpy(dst + c / col_group * col_padded, src + 2 * ((size_t)r * cols + c), 2 * (size_t)col_group);
        }
        return PTM_OK;
    }
    // a tensor's columns at dst column `at` on, all rows
    int place_columns(HostMatrix& h, const std::string& name, int rows, int cols, int at) const {
        ptm_st_tensor t;
        const int rc = tensor(name, rows, cols, &t);
        if (rc != PTM_OK) return rc;
        if (strcmp(t.dtype, "BF16") != 0) return PTM_E_UNSUPPORTED;
        for (int r = 0; r < rows; ++r)
            memcpy(h.v.data() + (size_t)r * h.ld + at, static_cast<const uint8_t*>(t.data) + 2 * (size_t)r * cols, 2 * (size_t)cols);
        return PTM_OK;
    }
    int upload(const HostMatrix& h, ptm_qweight* w) const {
        void* d = nullptr;
        const int rc = model_upload(m, h.v.data(), h.v.size() * 2, &d);
        if (rc != PTM_OK) return rc;
        w->data = d;
        w->ggml_type = PTM_TYPE_BF16;
        w->rows = h.rows;
        w->cols = h.cols;
        w->row_stride_bytes = 2 * (int64_t)h.ld;
        return PTM_OK;
    }
    int matrix(const std::string& name, int rows, int cols, ptm_qweight* w) const {
        HostMatrix h(rows, cols);
        const int rc = place(h, name, rows, cols, 0);
        return rc != PTM_OK ? rc : upload(h, w);
    }
    // a tensor's values as fp32, row by row
    int values(const std::string& name, int rows, int cols, bool is_2d, std::vector<float>* out) const {
        ptm_st_tensor t;
        const int rc = is_2d ? tensor(name, rows, cols, &t) : tensor(name, cols, 0, &t);
        if (rc != PTM_OK) return rc;
        const bool bf = strcmp(t.dtype, "BF16") == 0;
        if (!bf && strcmp(t.dtype, "F32") != 0) return PTM_E_UNSUPPORTED;
        out->resize((size_t)rows * (size_t)cols);
        for (size_t i = 0; i < out->size(); ++i) {
            uint32_t u = 0;
            if (bf) {
                uint16_t b;
                memcpy(&b, static_cast<const uint8_t*>(t.data) + 2 * i, 2);
                u = (uint32_t)b << 16;
            } else {
                memcpy(&u, static_cast<const uint8_t*>(t.data) + 4 * i, 4);
            }
            memcpy(&(*out)[i], &u, 4);
        }
        return PTM_OK;
    }
    int upload_floats(const std::vector<float>& v, const float** out) const {
        void* d = nullptr;
        const int rc = model_upload(m, v.data(), v.size() * 4, &d);
        if (rc == PTM_OK) *out = static_cast<const float*>(d);
        return rc;
    }
    // fp32 rows of `cols` values, padded
    int vectors(const std::string& name, int rows, int cols, bool is_2d, const float** out) const {
        std::vector<float> v, padded((size_t)rows * (size_t)up64(cols), 0.0f);
        const int rc = values(name, rows, cols, is_2d, &v);
        if (rc != PTM_OK) return rc;
        for (int r = 0; r < rows; ++r) memcpy(&padded[(size_t)r * up64(cols)], &v[(size_t)r * cols], 4 * (size_t)cols);
        return upload_floats(padded, out);
    }
    // host copy, owned by the model
    int host(const std::string& name, int rows, int cols, bool is_2d, const float** out) const {
        m->host_vectors.emplace_back();
        const int rc = values(name, rows, cols, is_2d, &m->host_vectors.back());
        if (rc == PTM_OK) *out = m->host_vectors.back().data();
        return rc;
    }
    int vector(const std::string& name, int n, const float** out) const { return vectors(name, 1, n, false, out); }
};

#define PTM_L(x) do { const int rc_ = (x); if (rc_ != PTM_OK) return rc_; } while (0)

// "Tovasun": layers of `attention` and `latent_attention` mixers, norms before and after each branch, squared-relu
// feed-forward, optional loop and per-layer token input.
int load_tovasun(FolderLoader& F, const Json& cfg, ptm_block_config* c) {
    ConfigReader R;
    c->vocab = R.size(&cfg, "vocab");
    c->hidden = R.size(&cfg, "width");
    c->eps = (float)R.real(cfg.find("norm"), "eps");
    const Json *layers = cfg.find("layers"), *loop = cfg.find("loop"), *side = cfg.find("token_side");
    if (R.rc != PTM_OK || !layers || layers->kind != Json::Array || layers->items.empty() || layers->items.size() > 4096 || c->vocab <= 0 || c->hidden <= 0) return PTM_E_FORMAT;
    const int n = (int)layers->items.size(), W = c->hidden;
    c->n_blocks = n;
    if (loop && !loop->is_null()) {
        c->loop_start = R.size(loop, "start");
        c->loop_stop = R.size(loop, "stop");
        c->loop_times = R.size(loop, "times");
        if (R.rc != PTM_OK || c->loop_times <= 0 || c->loop_times > 65536 || c->loop_start >= c->loop_stop || c->loop_stop > n) return PTM_E_FORMAT;
        PTM_L(F.vectors("loop.step", c->loop_times, W, true, &c->loop_step));
    }
    if (side && !side->is_null()) {
        c->side_dim = R.size(side, "dim");
        if (R.rc != PTM_OK || c->side_dim <= 0 || (int64_t)c->side_dim * n > 0x3fffffff) return PTM_E_FORMAT;
        PTM_L(F.matrix("side.embed", c->vocab, n * c->side_dim, &c->side_table));
    }
    PTM_L(F.matrix("embed", c->vocab, W, &c->embedding));
    PTM_L(F.matrix("head", c->vocab, W, &c->lm_head));
    PTM_L(F.vector("final.norm", W, &c->out_norm));
    F.m->blocks.resize((size_t)n);
    for (int i = 0; i < n; ++i) {
        const Json& layer = layers->items[(size_t)i];
        ptm_block& L = F.m->blocks[(size_t)i];
        const std::string p = "l" + std::to_string(i) + ".", x = p + "mix.";
        const std::string type = R.text(&layer, "type");
        const Json *mix = layer.find("mixer"), *mask = mix ? mix->find("mask") : nullptr, *mlp = layer.find("mlp");
        L.heads = R.size(mix, "heads");
        L.dim = R.size(mix, "dim");
        L.vdim = R.size(mix, "vdim");
        L.scale = (float)R.real(mix, "scale");
        L.softcap = (float)R.real(mix, "softcap", 0.0);
        L.rot = R.rotation(mix ? mix->find("rot") : nullptr);
        if (mask && !mask->is_null()) {
            L.window = R.size(mask, "size", 0);
            L.keep_first = R.size(mask, "keep_first", 0);
        }
        if (R.rc != PTM_OK) return R.rc;
        if ((int64_t)L.heads * up8(L.dim) > 0x3fffff || (int64_t)L.heads * up8(L.vdim) > 0x3fffff) return PTM_E_UNSUPPORTED;
        const int vcols = L.heads * L.vdim;
        if (type == "attention") {
            L.mixer = PTM_MIX_ATTENTION;
            L.kv_heads = R.size(mix, "kv_heads");
            if (R.rc != PTM_OK || L.heads <= 0 || L.kv_heads <= 0 || L.dim <= 0 || L.vdim <= 0) return PTM_E_FORMAT;
            const int q = L.heads * L.dim, k = L.kv_heads * L.dim, v = L.kv_heads * L.vdim;
            HostMatrix h(q + k + v, W);
            PTM_L(F.place(h, x + "q", q, W, 0));
            PTM_L(F.place(h, x + "k", k, W, q));
            PTM_L(F.place(h, x + "v", v, W, q + k));
            PTM_L(F.upload(h, &L.in));
            PTM_L(F.vector(x + "q.norm", q, &L.q_norm));
            PTM_L(F.vector(x + "k.norm", k, &L.k_norm));
        } else if (type == "latent_attention") {
            L.mixer = PTM_MIX_LATENT;
            L.rot_dim = R.size(mix, "rot_dim");
            L.kv_rank = R.size(mix, "kv_rank");
            if (R.rc != PTM_OK || L.heads <= 0 || L.dim <= 0 || L.vdim <= 0 || L.rot_dim <= 0 || L.kv_rank <= 0) return PTM_E_FORMAT;
            const int q = L.heads * (L.dim + L.rot_dim), kd = L.kv_rank + L.rot_dim;
            HostMatrix h(q + kd, W);
            PTM_L(F.place(h, x + "q", q, W, 0));
            PTM_L(F.place(h, x + "dkv", kd, W, q));
            PTM_L(F.upload(h, &L.in));
            PTM_L(F.vector(x + "dkv.norm", L.kv_rank, &L.k_norm));
            HostMatrix e(L.heads * (up8(L.dim) + up8(L.vdim)), L.kv_rank);
            PTM_L(F.place(e, x + "uk", L.heads * L.dim, L.kv_rank, 0, L.dim, up8(L.dim)));
            PTM_L(F.place(e, x + "uv", vcols, L.kv_rank, L.heads * up8(L.dim), L.vdim, up8(L.vdim)));
            PTM_L(F.upload(e, &L.expand));
        } else {
            return PTM_E_UNSUPPORTED;
        }
        HostMatrix o(W, L.heads * up8(L.vdim));
        PTM_L(F.place(o, x + "o", W, vcols, 0, 0, 0, L.vdim, up8(L.vdim)));
        PTM_L(F.upload(o, &L.out));
        PTM_L(F.vector(p + "norm1", W, &L.norm1));
        PTM_L(F.vector(p + "norm1b", W, &L.norm1b));
        if (mlp && !mlp->is_null()) {
            if (R.text(mlp, "kind") != "dense") return R.rc != PTM_OK ? R.rc : PTM_E_UNSUPPORTED;
            L.ff = R.size(mlp, "ff");
            if (R.rc != PTM_OK || L.ff <= 0) return PTM_E_FORMAT;
            PTM_L(F.matrix(p + "mlp.up", L.ff, W, &L.up));
            PTM_L(F.matrix(p + "mlp.down", W, L.ff, &L.down));
            PTM_L(F.vector(p + "norm2", W, &L.norm2));
            PTM_L(F.vector(p + "norm2b", W, &L.norm2b));
        }
        if (c->side_dim > 0) {
            PTM_L(F.matrix(p + "side.gate", c->side_dim, W, &L.side_gate));
            PTM_L(F.matrix(p + "side.proj", W, c->side_dim, &L.side_proj));
            PTM_L(F.vector(p + "side.norm", W, &L.side_norm));
            L.side_offset = i * c->side_dim;
        }
    }
    c->blocks = F.m->blocks.data();
    return PTM_OK;
}

// Grouped-query attention over one projected input, read from `o`: sizes, sink and gate.  Returns the rows of its part of `in`.
int nadozen_attention_sizes(ConfigReader& R, const Json* o, ptm_block& L) {
    const Json* mask = o ? o->find("mask") : nullptr;
    L.heads = R.size(o, "heads");
    L.kv_heads = R.size(o, "kv_heads");
    L.dim = R.size(o, "dim");
    L.vdim = R.size(o, "vdim", L.dim);
    L.scale = (float)R.real(o, "scale");
    if (mask && !mask->is_null()) {
        L.window = R.size(mask, "size");
        if (L.window <= 0) R.rc = PTM_E_FORMAT;
    }
    if (R.rc != PTM_OK || L.heads <= 0 || L.kv_heads <= 0 || L.heads % L.kv_heads || L.dim <= 0 || L.vdim != L.dim) return PTM_E_FORMAT;
    if ((int64_t)L.heads * up8(L.dim) > 0x3fffff) return PTM_E_UNSUPPORTED;
    L.mixer = PTM_MIX_ATTENTION;
    L.rot.base = 1.0;
    L.head_norm = L.values_are_keys = L.out_gate = 1;
    return PTM_OK;
}

// Attention (the projected keys are the values, normed per head for the scores only; a sink; an output gate) and a state-space
// mixer side by side: one matrix in front of both and one behind.
int nadozen_parallel(FolderLoader& F, ConfigReader& R, const Json* mix, const std::string& x, int W, ptm_block& L) {
    const Json *left = mix ? mix->find("left") : nullptr, *right = mix ? mix->find("right") : nullptr;
    PTM_L(nadozen_attention_sizes(R, left, L));
    ptm_ssm& m = L.ssm;
    m.heads = R.size(right, "heads");
    m.vdim = R.size(right, "vdim");
    m.state = R.size(right, "state");
    m.groups = R.size(right, "groups");
    m.taps = R.size(right, "conv");
    m.norm_groups = R.size(right, "norm_groups");
    L.out_scale = (float)R.real(mix, "left_scale");
    m.scale = (float)R.real(mix, "right_scale");
    if (R.rc != PTM_OK || m.heads <= 0 || m.vdim <= 0 || m.state <= 0 || m.groups <= 0 || m.taps <= 0 || m.norm_groups <= 0) return PTM_E_FORMAT;
    if (L.out_scale == 0.0f || m.scale == 0.0f) return PTM_E_UNSUPPORTED;  // a branch that is not there
    if ((int64_t)m.heads * m.vdim > 0xfffff || (int64_t)m.groups * m.state > 0xfffff) return PTM_E_UNSUPPORTED;
    const std::string l = x + "left.", r = x + "right.";
    const int q = L.heads * L.dim, k = L.kv_heads * L.dim, inner = m.heads * m.vdim, channels = inner + 2 * m.groups * m.state,
              rows = inner + channels + m.heads;
    HostMatrix in(q + k + q + rows, W);
    PTM_L(F.place(in, l + "q", q, W, 0));
    PTM_L(F.place(in, l + "k", k, W, q));
    PTM_L(F.place(in, l + "g", q, W, q + k));
    PTM_L(F.place(in, r + "in", rows, W, q + k + q));
    PTM_L(F.upload(in, &L.in));
    auto per_head = [&](const std::string& name, int heads, const float** out) {  // weights shared by the heads
        std::vector<float> v, all;
        PTM_L(F.values(name, 1, L.dim, false, &v));
        for (int h = 0; h < heads; ++h) all.insert(all.end(), v.begin(), v.end());
        return F.upload_floats(all, out);
    };
    PTM_L(per_head(l + "q.norm", L.heads, &L.q_norm));
    PTM_L(per_head(l + "k.norm", L.kv_heads, &L.k_norm));
    PTM_L(F.vector(l + "sink", L.heads, &L.sink));
    std::vector<float> v;
    PTM_L(F.values(r + "conv", channels, m.taps, true, &v));
    PTM_L(F.upload_floats(v, &m.conv));
    PTM_L(F.vector(r + "conv.b", channels, &m.conv_b));
    PTM_L(F.vector(r + "dt_bias", m.heads, &m.dt_bias));
    PTM_L(F.vector(r + "D", m.heads, &m.D));
    PTM_L(F.vector(r + "norm", inner, &m.norm));
    PTM_L(F.values(r + "A_log", 1, m.heads, false, &v));
    for (float& a : v) a = (float)-std::exp((double)a);
    PTM_L(F.upload_floats(v, &m.neg_a));
    HostMatrix out(W, L.heads * up8(L.dim) + inner);
    PTM_L(F.place(out, l + "o", W, q, 0, 0, 0, L.dim, up8(L.dim)));
    PTM_L(F.place_columns(out, r + "o", W, inner, L.heads * up8(L.dim)));
    return F.upload(out, &L.out);
}

int nadozen_wkv(FolderLoader& F, ConfigReader& R, const Json* mix, const std::string& x, int W, ptm_block& L) {
    L.mixer = PTM_MIX_WKV;
    ptm_wkv& m = L.wkv;
    m.heads = R.size(mix, "heads");
    m.dim = R.size(mix, "dim");
    if (R.rc != PTM_OK || m.heads <= 0 || m.dim <= 0) return PTM_E_FORMAT;
    if ((int64_t)m.heads * m.dim > 0xfffff) return PTM_E_UNSUPPORTED;
    ptm_st_tensor t;
    PTM_L(ptm_safetensors_find(F.f, (x + "w1").c_str(), &t));  // its rows are the decay's rank
    if (t.n_dims != 2 || t.dims[0] <= 0 || t.dims[0] > 0xfffff) return PTM_E_SHAPE;
    m.rank = (int)t.dims[0];
    const int hd = m.heads * m.dim;
    HostMatrix in(4 * hd + m.rank, W);
    const char* const parts[5] = {"r", "k", "v", "g", "w"};
    std::vector<float> mu((size_t)5 * up64(W), 0.0f), v;
    for (int i = 0; i < 5; ++i) {
        if (i < 4) PTM_L(F.place(in, x + parts[i], hd, W, i * hd));
        PTM_L(F.values(x + "mu." + parts[i], 1, W, false, &v));
        memcpy(&mu[(size_t)i * up64(W)], v.data(), 4 * (size_t)W);
    }
    PTM_L(F.place(in, x + "w1", m.rank, W, 4 * hd));
    PTM_L(F.upload(in, &L.in));
    PTM_L(F.upload_floats(mu, &m.mu));
    PTM_L(F.matrix(x + "w2", hd, m.rank, &m.w2));
    PTM_L(F.vector(x + "w0", hd, &m.w0));
    PTM_L(F.values(x + "u", m.heads, m.dim, true, &v));
    PTM_L(F.upload_floats(v, &m.u));
    PTM_L(F.vector(x + "norm", hd, &m.norm));
    return F.matrix(x + "o", W, hd, &L.out);
}

// "Nadozen": layers of `wkv` and `parallel` mixers behind layer norms, hyper-connections, a gated-silu feed-forward in some layers,
// layers that use another one's weights, a position sinusoid on the embedding.
int load_nadozen(FolderLoader& F, const Json& cfg, ptm_block_config* c) {
    ConfigReader R;
    c->vocab = R.size(&cfg, "vocab");
    c->hidden = R.size(&cfg, "width");
    c->eps = (float)R.real(cfg.find("norm"), "eps");
    c->streams = R.size(&cfg, "streams");
    c->logit_scale = (float)R.real(&cfg, "logit_scale");
    c->position_base = 10000.0;
    const Json* layers = cfg.find("layers");
    if (R.rc != PTM_OK || !layers || layers->kind != Json::Array || layers->items.empty() || layers->items.size() > 4096 || c->vocab <= 0 || c->hidden <= 0 ||
        c->streams <= 0 || c->logit_scale == 0.0f)
        return PTM_E_FORMAT;
    const int n = (int)layers->items.size(), W = c->hidden, S = c->streams;
    c->n_blocks = n;
    PTM_L(F.matrix("embed", c->vocab, W, &c->embedding));
    PTM_L(F.matrix("head", c->vocab, W, &c->lm_head));
    PTM_L(F.vector("final.norm", W, &c->out_norm));
    PTM_L(F.vector("final.norm.b", W, &c->out_norm_bias));
    F.m->blocks.resize((size_t)n);
    std::vector<int> owner((size_t)n);  // the layer whose tensors layer i uses
    for (int i = 0; i < n; ++i) {
        owner[(size_t)i] = i;
        const Json* of = layers->items[(size_t)i].find("weights_of");
        if (!of || of->is_null()) continue;
        const int j = R.size(&layers->items[(size_t)i], "weights_of");
        if (R.rc != PTM_OK || j >= n) return PTM_E_FORMAT;
        owner[(size_t)i] = j;
    }
    for (int i = 0; i < n; ++i)
        for (int steps = 0; owner[(size_t)owner[(size_t)i]] != owner[(size_t)i]; ++steps) {
            if (steps > n) return PTM_E_FORMAT;  // layers that name each other
            owner[(size_t)i] = owner[(size_t)owner[(size_t)i]];
        }
    for (int i = 0; i < n; ++i) {
        if (owner[(size_t)i] != i) continue;
        const Json& layer = layers->items[(size_t)i];
        ptm_block& L = F.m->blocks[(size_t)i];
        const std::string p = "l" + std::to_string(i) + ".", type = R.text(&layer, "type");
        const Json *mix = layer.find("mixer"), *mlp = layer.find("mlp");
        if (R.rc != PTM_OK) return R.rc;
        if (type == "wkv") PTM_L(nadozen_wkv(F, R, mix, p + "mix.", W, L));
        else if (type == "parallel") PTM_L(nadozen_parallel(F, R, mix, p + "mix.", W, L));
        else return PTM_E_UNSUPPORTED;
        PTM_L(F.vector(p + "norm1", W, &L.norm1));
        PTM_L(F.vector(p + "norm1.b", W, &L.norm1_bias));
        if (mlp && !mlp->is_null()) {
            if (R.text(mlp, "kind") != "dense") return R.rc != PTM_OK ? R.rc : PTM_E_UNSUPPORTED;
            L.ff = R.size(mlp, "ff");
            if (R.rc != PTM_OK || L.ff <= 0 || L.ff > 0xfffff) return PTM_E_FORMAT;
            L.ff_kind = PTM_FF_SWIGLU;
            HostMatrix up(2 * L.ff, W);
            PTM_L(F.place(up, p + "mlp.gate", L.ff, W, 0));
            PTM_L(F.place(up, p + "mlp.up", L.ff, W, L.ff));
            PTM_L(F.upload(up, &L.up));
            PTM_L(F.matrix(p + "mlp.down", W, L.ff, &L.down));
            PTM_L(F.vector(p + "norm2", W, &L.norm2));
            PTM_L(F.vector(p + "norm2.b", W, &L.norm2_bias));
        }
        for (int q = 0; q < (L.ff > 0 ? 2 : 1); ++q) {
            const std::string h = p + "hc" + std::to_string(q + 1) + ".";
            PTM_L(F.host(h + "in", 1, S, false, &L.hc_in[q]));
            PTM_L(F.host(h + "out", 1, S, false, &L.hc_out[q]));
            PTM_L(F.host(h + "mix", S, S, true, &L.hc_mix[q]));
        }
    }
    for (int i = 0; i < n; ++i)
        if (owner[(size_t)i] != i) F.m->blocks[(size_t)i] = F.m->blocks[(size_t)owner[(size_t)i]];
    c->blocks = F.m->blocks.data();
    return PTM_OK;
}
#undef PTM_L

struct Architecture {
    const char* name;
    int (*load)(FolderLoader&, const Json&, ptm_block_config*);
};
const Architecture ARCHITECTURES[] = {{"Tovasun", load_tovasun}, {"Nadozen", load_nadozen}};

int load_folder(const std::string& dir, int max_seq, int precision, int use_graph, ptm_model** out) {
    std::string text;
    int rc = read_file(dir + "/config.json", &text);
    if (rc != PTM_OK) return rc;
    Json cfg;
    if (!JsonParser(text.data(), text.size()).parse(&cfg)) return PTM_E_FORMAT;
    const Json* name = cfg.find("architecture");
    if (!name || name->kind != Json::String) return PTM_E_FORMAT;
    const Architecture* arch = nullptr;
    for (const Architecture& a : ARCHITECTURES)
        if (name->str == a.name) arch = &a;
    if (!arch) return PTM_E_UNSUPPORTED;
    ptm_safetensors* f = nullptr;
    if ((rc = ptm_safetensors_open((dir + "/model.safetensors").c_str(), &f)) != PTM_OK) return rc;
    ptm_model* m = new (std::nothrow) ptm_model();
    if (!m) { ptm_safetensors_close(f); return PTM_E_STATE; }
    FolderLoader F{m, f};
    ptm_block_config c{};
    rc = arch->load(F, cfg, &c);
    ptm_safetensors_close(f);
    if (rc == PTM_OK) {
        c.max_seq = max_seq;
        c.precision = precision;
        c.use_graph = use_graph ? 1 : 0;
        rc = ptm_decode_create_blocks(&c, &m->dec);
    }
    if (rc != PTM_OK) { ptm_model_free(m); return rc; }
    m->cfg.vocab = c.vocab;
    m->cfg.hidden = c.hidden;
    m->cfg.n_layers = ptm_decode_layer_runs(m->dec);
    m->cfg.max_seq = max_seq;
    m->cfg.rms_eps = c.eps;
    m->cfg.use_graph = c.use_graph;
    m->cfg.out_norm = c.out_norm;
    m->cfg.lm_head = c.lm_head;
    *out = m;
    return PTM_OK;
}

}  // namespace

extern "C" int ptm_model_load(const char* path, int max_seq, int precision, int use_graph, ptm_model** out) {
    if (!path || !out) return PTM_E_NULL;
    *out = nullptr;
    if (max_seq <= 0) return PTM_E_SHAPE;
    if (precision != PTM_PRECISION_16 && precision != PTM_PRECISION_32) return PTM_E_UNSUPPORTED;
    struct stat st;
    if (stat(path, &st) != 0) return PTM_E_IO;
    if (S_ISDIR(st.st_mode)) return load_folder(path, max_seq, precision, use_graph, out);
    return ptm_model_load_gguf(path, max_seq, precision == PTM_PRECISION_16, use_graph, out);
}
