// Model registry: config.json -> the description of a decoder.  The table at the end maps an architecture name to the
// function that reads its keys; a new design adds a row and, if it needs one, a new kind of mixer or feed-forward.
// Host code only.
#include <algorithm>
#include <cmath>
#include <cstdarg>
#include <cstdio>
#include <mutex>

#include "json.h"
#include "model_spec.h"

namespace mynn {

double RotarySpec::frequency(int i) const {
    const double f = std::pow(base, -2.0 * i / dims);
    if (!scaled) return f;
    const double turns = original * f / (2.0 * M_PI);  // original context over the wavelength
    if (turns < low) return f / factor;
    if (turns > high) return f;
    const double s = (turns - low) / (high - low);
    return (1.0 - s) * f / factor + s * f;
}

// The checkpoint beside a config, opened when a reader asks for a tensor's shape.
struct Checkpoint {
    std::string dir;
    mynn_weights *weights = nullptr;
    bool opened = false;
    bool rows(const std::string &name, int64_t *out) {
        if (!opened) weights = mynn_weights_open(dir.c_str());
        opened = true;
        int64_t shape[8] = {};
        int nd = 0;
        if (!weights || mynn_weights_find(weights, name.c_str(), nullptr, shape, &nd, nullptr, nullptr) || nd < 1) return false;
        *out = shape[0];
        return true;
    }
    ~Checkpoint() { mynn_weights_close(weights); }
};

// ---- typed access to a config object: a missing or mistyped key is an error that names it -----------------------
struct Reader {
    const Json &obj;
    std::string where;
    bool *ok;
    Checkpoint *checkpoint;
    const Json *need(const char *key, Json::Kind kind) const {
        const Json *v = obj.get(key);
        if (!v || v->kind != kind) {
            if (*ok) fail(MYNN_ERR_INVALID, "config: %s has no %s '%s'", where.c_str(), kind == Json::NUM ? "number" : kind == Json::STR ? "string" : kind == Json::ARR ? "list" : "object", key);
            *ok = false;
            return nullptr;
        }
        return v;
    }
    bool has(const char *key) const {
        const Json *v = obj.get(key);
        return v && v->kind != Json::NUL;
    }
    double num(const char *key) const {
        const Json *v = need(key, Json::NUM);
        return v ? v->num : 0.0;
    }
    double num_or(const char *key, double dflt) const { return has(key) ? num(key) : dflt; }
    int64_t integer(const char *key, int64_t lo, int64_t hi) const {
        const double d = num(key);
        if (*ok && !(d >= (double)lo && d <= (double)hi && d == std::floor(d))) {
            fail(MYNN_ERR_INVALID, "config: %s: %s = %g is not an integer in [%lld, %lld]", where.c_str(), key, d, (long long)lo, (long long)hi);
            *ok = false;
        }
        return *ok ? (int64_t)d : 0;
    }
    int size(const char *key) const { return (int)integer(key, 1, 1 << 28); }
    int size_or(const char *key, int dflt) const { return has(key) ? size(key) : dflt; }
    Reader sub(const char *key) const {
        static const Json empty;
        const Json *v = need(key, Json::OBJ);
        return Reader{v ? *v : empty, where + "." + key, ok, checkpoint};
    }
    std::string str(const char *key) const {
        const Json *v = need(key, Json::STR);
        return v ? v->str : std::string();
    }
    // rows of a matrix whose size the config leaves to the checkpoint
    int tensor_rows(const std::string &name) const {
        if (!*ok) return 0;
        int64_t rows = 0;
        if (!checkpoint->rows(name, &rows) || rows < 1 || rows > 1 << 28) {
            fail(MYNN_ERR_INVALID, "config: %s: the checkpoint beside the config gives no rows of %s", where.c_str(), name.c_str());
            *ok = false;
        }
        return (int)rows;
    }
};

// ---- Llama / Qwen2 (model_type "llama", "qwen2"; crates/llm/src/decoder.rs:570-660) -------------------------------
static void read_llama(const Reader &r, ModelSpec &s) {
    s.family = ModelSpec::LLAMA;
    mynn_model_config &c = s.llama;
    c.hidden = s.width = r.size("hidden_size");
    c.n_layers = r.size("num_hidden_layers");
    c.n_heads = r.size("num_attention_heads");
    c.n_kv_heads = r.size_or("num_key_value_heads", c.n_heads);
    c.head_dim = r.size_or("head_dim", c.n_heads ? c.hidden / c.n_heads : 0);
    c.ffn = r.size("intermediate_size");
    c.vocab = s.vocab = r.size("vocab_size");
    c.eps = s.eps = (float)r.num_or("rms_norm_eps", 1e-6);
    c.rope_theta = (float)r.num_or("rope_theta", 10000.0);
    c.qkv_bias = s.architecture == "Qwen2ForCausalLM";
}

// ---- designs described layer by layer -------------------------------------------------------------------------------
static void read_latent_attention(const Reader &m, MixerSpec &x) {
    x.kind = MixerSpec::LATENT_ATTENTION;
    x.heads = m.size("heads");
    x.dim = m.size("dim");
    x.rot_dim = m.size("rot_dim");
    x.vdim = m.size("vdim");
    x.kv_rank = m.size("kv_rank");
    x.scale = (float)m.num("scale");
    const Reader rot = m.sub("rot");
    x.rot.base = rot.num("base");
    x.rot.dims = rot.size("dims");
    if (*m.ok && (x.rot.dims > x.rot_dim || x.rot.dims % 2 || !(x.rot.base > 0.0))) {
        fail(MYNN_ERR_INVALID, "config: %s.rot: %d rotated dimensions of %d, base %g", m.where.c_str(), x.rot.dims, x.rot_dim, x.rot.base);
        *m.ok = false;
    }
}

static void add_tensor(ModelSpec &s, const std::string &name, std::vector<int64_t> shape) {
    s.tensor_at.emplace(name, (int)s.tensors.size());
    s.tensors.push_back({name, std::move(shape)});
}
static bool refuse(const Reader &r, int code, const char *fmt, ...) __attribute__((format(printf, 3, 4)));
static bool refuse(const Reader &r, int code, const char *fmt, ...) {
    char text[256];
    va_list ap;
    va_start(ap, fmt);
    vsnprintf(text, sizeof text, fmt, ap);
    va_end(ap);
    fail(code, "config: %s", text);
    *r.ok = false;
    return false;
}

static void list_latent_attention_tensors(ModelSpec &s, const std::string &p, const MixerSpec &m) {
    const int64_t W = s.width, H = m.heads;
    add_tensor(s, p + "q", {H * (m.dim + m.rot_dim), W});
    add_tensor(s, p + "dkv", {m.kv_rank + m.rot_dim, W});
    add_tensor(s, p + "dkv.norm", {m.kv_rank});
    add_tensor(s, p + "uk", {H * m.dim, m.kv_rank});
    add_tensor(s, p + "uv", {H * m.vdim, m.kv_rank});
    add_tensor(s, p + "g", {H, W});
    add_tensor(s, p + "o", {W, H * m.vdim});
}

// Session state of a layered model: the token caches of the runs that have one, the token history, then the sequence
// states of the runs that have one.
static void plan_states(ModelSpec &s) {
    auto add = [&](StateSpec st) {
        s.states.push_back(st);
        return (int)s.states.size() - 1;
    };
    for (LayerRun &r : s.runs) {
        const MixerSpec &m = s.layers[r.layer].mixer;
        if (m.kind == MixerSpec::LATENT_ATTENTION) r.cache = add({(size_t)latent_dims(m).lw(), 0, 0});
        if (m.kind == MixerSpec::PARALLEL) r.cache = add({(size_t)parallel_dims(m).row(), 0, 0});
    }
    s.history = add({0, sizeof(int32_t), 0});
    for (LayerRun &r : s.runs) {
        const MixerSpec &m = s.layers[r.layer].mixer;
        if (m.kind == MixerSpec::PARALLEL) r.memory = add({0, 0, (size_t)parallel_dims(m).state()});
        if (m.kind == MixerSpec::CHANNEL_DELTA) r.memory = add({0, 0, (size_t)delta_dims(m.delta).state()});
    }
}

// "Dudilix": sandwich-normed layers of latent attention with a gate per head and tanh-gelu gated feed-forwards, a bigram
// embedding, and a range of layers run several times over [x; embedding]
static void read_dudilix(const Reader &r, ModelSpec &s) {
    s.family = ModelSpec::LAYERED;
    s.vocab = r.size("vocab");
    s.width = r.size("width");
    s.eps = (float)r.sub("norm").num("eps");
    s.logit_scale = (float)r.num_or("logit_scale", 1.0);
    if (r.has("embedding")) {
        const Reader e = r.sub("embedding");
        if (e.has("bigram")) {
            const Reader b = e.sub("bigram");
            s.bigram.buckets = b.integer("buckets", 1, 1 << 28);
            s.bigram.mul_prev = b.integer("mul_prev", 0, (int64_t)1 << 32);
            s.bigram.mul_cur = b.integer("mul_cur", 0, (int64_t)1 << 32);
        }
    }
    const Json *layers = r.need("layers", Json::ARR);
    if (!layers) return;
    for (size_t i = 0; i < layers->arr.size() && *r.ok; i++) {
        const Reader l{layers->arr[i], "layers[" + std::to_string(i) + "]", r.ok, r.checkpoint};
        LayerSpec ls;
        const std::string type = l.str("type");
        if (!*r.ok) return;
        if (type == "latent_attention") read_latent_attention(l.sub("mixer"), ls.mixer);
        else {
            fail(MYNN_ERR_UNSUPPORTED, "config: layers[%zu] has the mixer '%s', which %s does not have", i, type.c_str(), s.architecture.c_str());
            *r.ok = false;
            return;
        }
        if (l.has("mlp")) {
            const Reader m = l.sub("mlp");
            const std::string kind = m.str("kind");
            if (*r.ok && kind != "dense") {
                fail(MYNN_ERR_UNSUPPORTED, "config: layers[%zu] has the feed-forward '%s', which %s does not have", i, kind.c_str(), s.architecture.c_str());
                *r.ok = false;
                return;
            }
            ls.mlp.kind = MlpSpec::GATED_DENSE;
            ls.mlp.ff = m.size("ff");
        }
        s.layers.push_back(ls);
    }
    if (!*r.ok) return;
    const int n = (int)s.layers.size();
    if (r.has("loop")) {
        const Reader l = r.sub("loop");
        s.loop.start = (int)l.integer("start", 0, n);
        s.loop.stop = (int)l.integer("stop", 0, n);
        s.loop.times = (int)l.integer("times", 1, 1 << 16);
        if (*r.ok && s.loop.start >= s.loop.stop) {
            fail(MYNN_ERR_INVALID, "config: loop over layers %d .. %d", s.loop.start, s.loop.stop);
            *r.ok = false;
        }
    }
    if (*r.ok && n == 0) {
        fail(MYNN_ERR_INVALID, "config: no layers");
        *r.ok = false;
    }
    if (!*r.ok) return;

    for (int i = 0; i < (s.loop.times ? s.loop.start : n); i++) s.runs.push_back({i, false});
    for (int t = 0; t < s.loop.times; t++)
        for (int i = s.loop.start; i < s.loop.stop; i++) s.runs.push_back({i, i == s.loop.start});
    for (int i = s.loop.times ? s.loop.stop : n; i < n; i++) s.runs.push_back({i, false});

    plan_states(s);
    const int64_t W = s.width;
    add_tensor(s, "embed", {s.vocab, W});
    if (s.bigram.buckets) add_tensor(s, "bigram", {s.bigram.buckets + 1, W});
    if (s.loop.times) add_tensor(s, "loop.in", {W, 2 * W});
    for (int i = 0; i < n; i++) {
        const LayerSpec &l = s.layers[i];
        const std::string p = "l" + std::to_string(i) + ".";
        add_tensor(s, p + "norm1", {W});
        add_tensor(s, p + "norm1b", {W});
        list_latent_attention_tensors(s, p + "mix.", l.mixer);
        if (l.mlp.kind == MlpSpec::NONE) continue;
        add_tensor(s, p + "norm2", {W});
        add_tensor(s, p + "norm2b", {W});
        add_tensor(s, p + "mlp.gate", {l.mlp.ff, W});
        add_tensor(s, p + "mlp.up", {l.mlp.ff, W});
        add_tensor(s, p + "mlp.down", {W, l.mlp.ff});
    }
    add_tensor(s, "final.norm", {W});
    add_tensor(s, "head", {s.vocab, W});
}

// ---- "Kulanex": norms behind the sublayers only; a gated delta rule with channel decays, or a windowed attention beside a
// matrix memory; sparse feed-forwards
static void read_rotary(const Reader &rot, int dim, RotarySpec &x) {
    x.base = rot.num("base");
    x.dims = rot.size("dims");
    if (rot.has("scaling")) {
        const Reader sc = rot.sub("scaling");
        x.scaled = true;
        x.factor = sc.num("factor");
        x.low = sc.num("low");
        x.high = sc.num("high");
        x.original = sc.num("original");
        if (*rot.ok && !(x.factor > 0.0 && x.high > x.low && x.low > 0.0 && x.original > 0.0))
            refuse(rot, MYNN_ERR_INVALID, "%s.scaling: factor %g, low %g, high %g, original %g", rot.where.c_str(), x.factor, x.low, x.high, x.original);
    }
    if (*rot.ok && (x.dims > dim || x.dims % 2 || !(x.base > 0.0)))
        refuse(rot, MYNN_ERR_INVALID, "%s: %d rotated dimensions of %d, base %g", rot.where.c_str(), x.dims, dim, x.base);
}
static void check_groups(const Reader &m, int heads, int kv_heads) {
    if (*m.ok && heads % kv_heads) refuse(m, MYNN_ERR_INVALID, "%s: %d heads over %d key/value heads", m.where.c_str(), heads, kv_heads);
}
static void read_window_attention(const Reader &m, WindowAttentionSpec &x) {
    x.heads = m.size("heads");
    x.kv_heads = m.size("kv_heads");
    x.dim = m.size("dim");
    x.taps = m.size("conv");
    x.scale = (float)m.num("scale");
    check_groups(m, x.heads, x.kv_heads);
    if (*m.ok && m.size("vdim") != x.dim) refuse(m, MYNN_ERR_INVALID, "%s: values are the keys, but vdim is not dim", m.where.c_str());
    if (*m.ok) read_rotary(m.sub("rot"), x.dim, x.rot);
    if (*m.ok && m.has("mask")) {
        const Reader k = m.sub("mask");
        x.window = k.size("size");
        x.keep_first = k.has("keep_first") ? (int)k.integer("keep_first", 0, 1 << 28) : 0;
    }
}
static void read_matrix_memory(const Reader &m, MatrixMemorySpec &x) {
    x.heads = m.size("heads");
    x.dim = m.size("dim");
    x.vdim = m.size("vdim");
    x.gate_cap = (float)m.num("gate_cap");
    if (*m.ok && !(x.gate_cap > 0.f)) refuse(m, MYNN_ERR_INVALID, "%s: gate_cap %g", m.where.c_str(), x.gate_cap);
}
static void read_channel_delta(const Reader &m, ChannelDeltaSpec &x) {
    x.heads = m.size("heads");
    x.kv_heads = m.size("kv_heads");
    x.dim = m.size("dim");
    x.vdim = m.size("vdim");
    x.taps = m.size("conv");
    check_groups(m, x.heads, x.kv_heads);
}

static void list_parallel_tensors(ModelSpec &s, const std::string &p, const MixerSpec &m) {
    const int64_t W = s.width;
    {
        const WindowAttentionSpec &a = m.window;
        const int64_t q = (int64_t)a.heads * a.dim, k = (int64_t)a.kv_heads * a.dim;
        const std::string l = p + "left.";
        add_tensor(s, l + "q", {q, W});
        add_tensor(s, l + "k", {k, W});
        add_tensor(s, l + "q.norm", {q});
        add_tensor(s, l + "k.norm", {k});
        add_tensor(s, l + "q.conv", {q, a.taps});
        add_tensor(s, l + "k.conv", {k, a.taps});
        add_tensor(s, l + "o", {W, q});
    }
    const MatrixMemorySpec &r = m.memory;
    const int64_t H = r.heads, d = H * r.dim, v = H * r.vdim;
    const std::string l = p + "right.";
    add_tensor(s, l + "q", {d, W});
    add_tensor(s, l + "k", {d, W});
    add_tensor(s, l + "v", {v, W});
    add_tensor(s, l + "g", {v, W});
    add_tensor(s, l + "o", {W, v});
    add_tensor(s, l + "norm", {v});
    add_tensor(s, l + "i", {H, W});
    add_tensor(s, l + "i.b", {H});
    add_tensor(s, l + "f", {H, W});
    add_tensor(s, l + "f.b", {H});
}
static void list_channel_delta_tensors(ModelSpec &s, const std::string &p, const ChannelDeltaSpec &m) {
    const int64_t W = s.width, H = m.heads, k = (int64_t)m.kv_heads * m.dim, v = H * m.vdim;
    add_tensor(s, p + "q", {k, W});
    add_tensor(s, p + "q.conv", {k, m.taps});
    add_tensor(s, p + "k", {k, W});
    add_tensor(s, p + "k.conv", {k, m.taps});
    add_tensor(s, p + "v", {v, W});
    add_tensor(s, p + "v.conv", {v, m.taps});
    add_tensor(s, p + "b", {H, W});
    add_tensor(s, p + "A_log", {H});
    add_tensor(s, p + "norm", {m.vdim});
    add_tensor(s, p + "a1", {m.decay_rank, W});
    add_tensor(s, p + "a2", {H * m.dim, m.decay_rank});
    add_tensor(s, p + "dt_bias", {H * m.dim});
    add_tensor(s, p + "g1", {m.gate_rank, W});
    add_tensor(s, p + "g2", {v, m.gate_rank});
    add_tensor(s, p + "o", {W, v});
}
static void list_expert_tensors(ModelSpec &s, const std::string &p, const MlpSpec &m) {
    const int64_t W = s.width;
    for (int e = 0; e < m.experts; e++) {
        const std::string x = p + "e" + std::to_string(e) + ".";
        add_tensor(s, x + "gate", {m.ff, W});
        add_tensor(s, x + "up", {m.ff, W});
        add_tensor(s, x + "down", {W, m.ff});
    }
    add_tensor(s, p + "router", {m.experts, W});
}

static void read_kulanex(const Reader &r, ModelSpec &s) {
    s.family = ModelSpec::LAYERED;
    s.vocab = r.size("vocab");
    s.width = r.size("width");
    s.eps = (float)r.sub("norm").num("eps");
    s.pre_norm = false;
    s.norm_offset = 1.f;
    s.residual_mult = (float)r.num("residual_mult");
    const Json *layers = r.need("layers", Json::ARR);
    if (!layers) return;
    if (layers->arr.empty()) refuse(r, MYNN_ERR_INVALID, "no layers");
    for (size_t i = 0; i < layers->arr.size() && *r.ok; i++) {
        const Reader l{layers->arr[i], "layers[" + std::to_string(i) + "]", r.ok, r.checkpoint};
        const std::string p = "l" + std::to_string(i) + ".";
        LayerSpec ls;
        const std::string type = l.str("type");
        if (!*r.ok) return;
        const Reader m = l.sub("mixer");
        if (type == "parallel") {
            ls.mixer.kind = MixerSpec::PARALLEL;
            read_window_attention(m.sub("left"), ls.mixer.window);
            read_matrix_memory(m.sub("right"), ls.mixer.memory);
            ls.mixer.left_scale = (float)m.num("left_scale");
            ls.mixer.right_scale = (float)m.num("right_scale");
        } else if (type == "channel_delta") {
            ls.mixer.kind = MixerSpec::CHANNEL_DELTA;
            read_channel_delta(m, ls.mixer.delta);
            // (the ranks of the low-rank maps are the tensors')
            ls.mixer.delta.decay_rank = m.tensor_rows(p + "mix.a1");
            ls.mixer.delta.gate_rank = m.tensor_rows(p + "mix.g1");
        } else {
            refuse(l, MYNN_ERR_UNSUPPORTED, "layers[%zu] has the mixer '%s', which %s does not have", i, type.c_str(), s.architecture.c_str());
            return;
        }
        if (l.has("mlp")) {
            const Reader f = l.sub("mlp");
            const std::string kind = f.str("kind");
            if (*r.ok && kind != "moe") {
                refuse(l, MYNN_ERR_UNSUPPORTED, "layers[%zu] has the feed-forward '%s', which %s does not have", i, kind.c_str(), s.architecture.c_str());
                return;
            }
            ls.mlp.kind = MlpSpec::EXPERTS;
            ls.mlp.ff = f.sub("expert").size("ff");
            ls.mlp.experts = f.sub("router").size("experts");
            ls.mlp.top = f.sub("router").size("top");
            if (*r.ok && ls.mlp.top > ls.mlp.experts) refuse(l, MYNN_ERR_INVALID, "layers[%zu]: top %d of %d experts", i, ls.mlp.top, ls.mlp.experts);
        }
        s.layers.push_back(ls);
        s.runs.push_back({(int)i, false});
    }
    if (!*r.ok) return;
    plan_states(s);
    const int64_t W = s.width;
    add_tensor(s, "embed", {s.vocab, W});
    for (size_t i = 0; i < s.layers.size(); i++) {
        const LayerSpec &l = s.layers[i];
        const std::string p = "l" + std::to_string(i) + ".";
        add_tensor(s, p + "norm1", {W});
        if (l.mixer.kind == MixerSpec::PARALLEL) list_parallel_tensors(s, p + "mix.", l.mixer);
        else list_channel_delta_tensors(s, p + "mix.", l.mixer.delta);
        if (l.mlp.kind == MlpSpec::NONE) continue;
        add_tensor(s, p + "norm2", {W});
        list_expert_tensors(s, p + "mlp.", l.mlp);
    }
    add_tensor(s, "final.norm", {W});
    add_tensor(s, "head", {s.vocab, W});
}

struct RegistryRow {
    const char *architecture;
    void (*read)(const Reader &, ModelSpec &);
};
static const RegistryRow kRegistry[] = {
    {"LlamaForCausalLM", read_llama},
    {"Qwen2ForCausalLM", read_llama},
    {"Dudilix", read_dudilix},
    {"Kulanex", read_kulanex},
};

static std::mutex g_arch_mu;
static std::vector<std::shared_ptr<const ModelSpec>> &arch_table() {
    static std::vector<std::shared_ptr<const ModelSpec>> t;
    return t;
}
std::shared_ptr<const ModelSpec> arch_spec(int arch) {
    std::lock_guard<std::mutex> lk(g_arch_mu);
    auto &t = arch_table();
    return arch >= 1 && arch <= (int)t.size() ? t[arch - 1] : nullptr;
}

static int arch_open_impl(const char *path) {
    MYNN_REQUIRE(path, MYNN_ERR_INVALID, "arch_open: null path");
    std::string file = path;
    if (file.size() < 5 || file.compare(file.size() - 5, 5, ".json")) file += "/config.json";
    FILE *f = fopen(file.c_str(), "rb");
    MYNN_REQUIRE(f, MYNN_ERR_INVALID, "config: cannot open %s", file.c_str());
    std::string text;
    char buf[65536];
    size_t n;
    while ((n = fread(buf, 1, sizeof buf, f)) > 0) text.append(buf, n);
    fclose(f);
    Json j;
    MYNN_REQUIRE(parse_json(text.data(), text.size(), j) && j.kind == Json::OBJ, MYNN_ERR_INVALID, "config: %s is not a JSON object", file.c_str());
    auto spec = std::make_shared<ModelSpec>();
    // "architecture": one name; "architectures": a list whose first entry counts
    const Json *a = j.get("architecture"), *as = j.get("architectures");
    if (a && a->kind == Json::STR) spec->architecture = a->str;
    else if (as && as->kind == Json::ARR && !as->arr.empty() && as->arr[0].kind == Json::STR) spec->architecture = as->arr[0].str;
    for (const RegistryRow &row : kRegistry)
        if (spec->architecture == row.architecture) {
            bool ok = true;
            Checkpoint beside{file.find('/') == std::string::npos ? "." : file.substr(0, file.rfind('/'))};
            row.read(Reader{j, "the config", &ok, &beside}, *spec);
            if (!ok) return MYNN_ERR_INVALID;
            std::lock_guard<std::mutex> lk(g_arch_mu);
            arch_table().push_back(std::move(spec));
            return (int)arch_table().size();
        }
    return fail(MYNN_ERR_UNSUPPORTED, "config: %s: no model of architecture '%s'", file.c_str(), spec->architecture.c_str());
}

}  // namespace mynn

using namespace mynn;

extern "C" int mynn_arch_open(const char *path) {
    try {
        return arch_open_impl(path);
    } catch (const std::exception &e) {
        return fail(MYNN_ERR_INVALID, "config: %s", e.what());
    }
}

extern "C" const char *mynn_arch_name(int arch) {
    auto s = arch_spec(arch);
    return s ? s->architecture.c_str() : nullptr;  // (the table keeps the description for the life of the process)
}

extern "C" int mynn_arch_config(int arch, int dtype, int max_seq, int seq_q, int batch, mynn_model_config *cfg) {
    auto s = arch_spec(arch);
    MYNN_REQUIRE(s && cfg, MYNN_ERR_INVALID, "arch_config: no architecture %d", arch);
    mynn_model_config c = s->llama;
    if (s->family == ModelSpec::LAYERED) {
        c = mynn_model_config{};
        c.arch = arch;
        c.n_layers = (int)s->runs.size();
        c.hidden = s->width;
        c.vocab = s->vocab;
        c.eps = s->eps;
        c.n_kv_heads = 1;
        c.rope_theta = (float)s->layers[0].mixer.rot.base;
        for (const LayerSpec &l : s->layers) {
            const MixerSpec &m = l.mixer;
            const int heads = std::max({m.heads, m.window.heads, m.memory.heads, m.delta.heads});
            c.n_heads = std::max(c.n_heads, heads);
            c.head_dim = std::max({c.head_dim, m.dim + m.rot_dim, m.window.dim, m.memory.dim, m.delta.dim});
            c.ffn = std::max(c.ffn, l.mlp.ff);
        }
    }
    c.dtype = dtype;
    c.max_seq = max_seq;
    c.seq_q = seq_q;
    c.batch = batch;
    *cfg = c;
    return 0;
}

extern "C" int mynn_arch_tensor_count(int arch) {
    auto s = arch_spec(arch);
    return s ? (int)s->tensors.size() : MYNN_ERR_INVALID;
}
extern "C" const char *mynn_arch_tensor(int arch, int i, int64_t *shape, int *ndim) {
    auto s = arch_spec(arch);
    if (!s || i < 0 || i >= (int)s->tensors.size()) {
        fail(MYNN_ERR_INVALID, "arch_tensor: no tensor %d of architecture %d", i, arch);
        return nullptr;
    }
    const TensorSpec &t = s->tensors[i];
    if (ndim) *ndim = (int)t.shape.size();
    if (shape)
        for (size_t d = 0; d < t.shape.size(); d++) shape[d] = t.shape[d];
    return t.name.c_str();
}

// Layered models: what plan_states lists.  Llama: K and V of every layer.
extern "C" int mynn_arch_state_count(int arch) {
    auto s = arch_spec(arch);
    MYNN_REQUIRE(s, MYNN_ERR_INVALID, "arch_state_count: no architecture %d", arch);
    return s->family == ModelSpec::LLAMA ? 2 * s->llama.n_layers : (int)s->states.size();
}
extern "C" size_t mynn_arch_state_row_bytes(int arch, int i, int dtype) {
    auto s = arch_spec(arch);
    if (!s || i < 0 || i >= mynn_arch_state_count(arch)) return 0;
    if (s->family == ModelSpec::LLAMA) return (size_t)s->llama.n_kv_heads * s->llama.head_dim * dtype_size(dtype);
    return s->states[i].row_elems * dtype_size(dtype) + s->states[i].row_bytes;
}
extern "C" size_t mynn_arch_state_seq_bytes(int arch, int i) {
    auto s = arch_spec(arch);
    if (!s || s->family == ModelSpec::LLAMA || i < 0 || i >= (int)s->states.size()) return 0;
    return s->states[i].seq_floats * sizeof(float);
}
