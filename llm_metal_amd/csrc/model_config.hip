// config.json: which model a checkpoint holds, and the layer list of models that are described layer by layer.
// Host code only.
#include "stack.h"
#include "json.h"

#include <fstream>
#include <math.h>
#include <sstream>
#include <string.h>
#include <sys/stat.h>

using namespace lmhip;

namespace lmhip {

std::string config_path_of(const char *model_path)
{
    std::string path = model_path ? model_path : "";
    struct stat st;
    if (stat(path.c_str(), &st) == 0 && S_ISDIR(st.st_mode)) return path + "/config.json";
    const size_t sl = path.rfind('/');
    return sl == std::string::npos ? "config.json" : path.substr(0, sl) + "/config.json";
}

namespace {

struct Reader {
    std::string &why;
    std::string at;
    bool ok = true;
    void fail(const std::string &m) { if (ok) why = at + m; ok = false; }
    int count(const JsonValue &v, const char *key, int lo = 1)
    {
        const JsonValue &n = v[key];
        if (!n.is_number() || n.num != floor(n.num) || n.num < lo || n.num > 1e9) { fail(std::string("'") + key + "' is missing or not a whole number from " + std::to_string(lo)); return lo; }
        return (int)n.num;
    }
    double real(const JsonValue &v, const char *key)
    {
        const JsonValue &n = v[key];
        if (!n.is_number() || !(fabs(n.num) < 1e30)) { fail(std::string("'") + key + "' is missing or not a number"); return 0.0; }
        return n.num;
    }
};

// rotation of the first `dims` entries of a head part of `most`
Rotation read_rotation(Reader &r, const JsonValue &v, int most, const char *most_name)
{
    Rotation t;
    t.dims = r.count(v, "dims"); t.base = r.real(v, "base");
    if (r.ok && (t.dims > most || (t.dims & 1))) r.fail(std::string("'rot.dims' is odd or above '") + most_name + "'");
    if (r.ok && !(t.base > 0.0)) r.fail("'rot.base' is not positive");
    const JsonValue &s = v["scaling"];
    if (s.kind == JsonValue::OBJECT) {
        t.factor = r.real(s, "factor"); t.low = r.real(s, "low"); t.high = r.real(s, "high"); t.original = r.real(s, "original");
        if (r.ok && !(t.factor > 0.0 && t.low > 0.0 && t.high >= t.low && t.original > 0.0)) r.fail("'rot.scaling' has values that make no scale");
    }
    return t;
}

}  // namespace

std::vector<double> Rotation::frequencies() const
{
    std::vector<double> out;
    for (int i = 0; i < dims / 2; i++) {
        const double f = pow(base, -2.0 * i / dims);
        if (factor <= 0.0) { out.push_back(f); continue; }
        const double turns = original * f / 6.283185307179586476925;     // within the original context
        const double keep = turns < low ? 0.0 : turns > high ? 1.0 : high > low ? (turns - low) / (high - low) : 1.0;
        out.push_back(keep * f + (1.0 - keep) * f / factor);
    }
    return out;
}

bool read_stack_config(const std::string &text, ModelType type, StackConfig &out, std::string &why)
{
    JsonValue root;
    if (!JsonValue::parse_text(text, root)) { why = "not valid JSON"; return false; }
    Reader r{why, ""};
    out = StackConfig();
    const bool around = type == MODEL_PAPOSUN;
    out.vocab = r.count(root, "vocab");
    out.width = r.count(root, "width");
    out.eps = (float)r.real(root["norm"], "eps");
    if (around) {
        out.norms = NORMS_AROUND; out.tied = true;
        out.residual_mult = (float)r.real(root, "residual_mult");
        out.logit_scale = (float)r.real(root, "logit_scale");
    } else out.emb_scale = (float)r.real(root["embedding"], "scale");
    if (root["layers"].items.empty()) r.fail("'layers' is missing or empty");
    for (size_t i = 0; i < root["layers"].items.size() && r.ok; i++) {
        const JsonValue &L = root["layers"].items[i], &mx = L["mixer"], &mlp = L["mlp"];
        r.at = "layer " + std::to_string(i) + ": ";
        LayerConfig c;
        const std::string &type = L["type"].str;
        c.heads = r.count(mx, "heads"); c.dim = r.count(mx, "dim"); c.vdim = r.count(mx, "vdim");
        if (around && type == "attention") {
            c.mixer = MIX_GROUPED;
            c.kv_heads = r.count(mx, "kv_heads"); c.chunk = r.count(mx["mask"], "size");
            c.rot = read_rotation(r, mx["rot"], c.dim, "dim");
            c.scale = (float)r.real(mx, "scale");
            if (r.ok && c.heads % c.kv_heads) r.fail("'heads' is not a multiple of 'kv_heads'");
            if (c.dim > 1024 || c.vdim > 1024) r.fail("head dimension above 1024");
            if (!mx["kv_from"].is_null()) {
                c.kv_from = r.count(mx, "kv_from", 0);
                const LayerConfig *s = r.ok && c.kv_from < (int)i ? &out.layers[c.kv_from] : nullptr;
                if (r.ok && (!s || s->mixer != MIX_GROUPED || s->kv_from >= 0)) r.fail("'kv_from' is not an earlier attention layer with keys of its own");
                else if (r.ok && (s->heads != c.heads || s->kv_heads != c.kv_heads || s->dim != c.dim || s->vdim != c.vdim || !(s->rot == c.rot)))
                    r.fail("'kv_from' has other heads or another rotation");
            }
        } else if (around && type == "mlstm") {
            c.mixer = MIX_MLSTM;
            c.gate_cap = (float)r.real(mx, "gate_cap");
            if (r.ok && !(c.gate_cap > 0.f)) r.fail("'gate_cap' is not positive");
            if (c.dim > 2048) r.fail("key dimension above 2048");
        } else if (around) r.fail("unknown mixer '" + type + "'");
        else if (type == "delta" || type == "channel_delta") {
            c.mixer = type == "delta" ? MIX_DELTA : MIX_CHANNEL_DELTA;
            c.kv_heads = r.count(mx, "kv_heads"); c.taps = r.count(mx, "conv");
            if (r.ok && c.heads % c.kv_heads) r.fail("'heads' is not a multiple of 'kv_heads'");
            if (c.dim > 256) r.fail("key dimension above 256");
            if (c.taps > 16) r.fail("more than 16 convolution taps");
        } else if (type == "latent_attention") {
            c.mixer = MIX_LATENT;
            c.rot_dim = r.count(mx, "rot_dim"); c.kv_rank = r.count(mx, "kv_rank");
            c.window = r.count(mx["mask"], "size");
            c.rot = read_rotation(r, mx["rot"], c.rot_dim, "rot_dim");
            c.scale = (float)r.real(mx, "scale");
            if (c.kv_rank > 1024 || c.rot_dim > 1024 || c.dim > 1024) r.fail("latent size or head dimension above 1024");
        } else r.fail("unknown mixer '" + type + "'");
        if (around && mlp.kind == JsonValue::OBJECT) {
            if (mlp["kind"].str != "dense") r.fail("unknown feed-forward '" + mlp["kind"].str + "'");
            c.dense_ff = r.count(mlp, "ff");
        } else if (mlp.kind == JsonValue::OBJECT) {
            if (mlp["kind"].str != "moe") r.fail("unknown feed-forward '" + mlp["kind"].str + "'");
            c.experts = r.count(mlp["router"], "experts"); c.top = r.count(mlp["router"], "top"); c.ff = r.count(mlp["expert"], "ff");
            if (mlp["shared"].kind == JsonValue::OBJECT) c.shared_ff = r.count(mlp["shared"], "ff");
            if (r.ok && (c.top > c.experts || c.top > 32 || c.experts > 1024)) r.fail("'top' above 'experts' or above 32, or more than 1024 experts");
        }
        out.layers.push_back(c);
    }
    return r.ok;
}

}  // namespace lmhip

extern "C" {

// main.c:286-324 for the reference's two models: "gemma3" / "gemma2" in the config.json next to (or inside) the model
// path, else Qwen3.  A design that lists its layers is told by its "architecture".
ModelType model_type_detect(const char *path)
{
    std::ifstream f(config_path_of(path));
    if (!f) return MODEL_QWEN3;
    std::stringstream ss;
    ss << f.rdbuf();
    const std::string text = ss.str();
    JsonValue root;
    if (JsonValue::parse_text(text, root)) {
        if (root["architecture"].str == "Nevurax") return MODEL_NEVURAX;
        if (root["architecture"].str == "Paposun") return MODEL_PAPOSUN;
    }
    const std::string head = text.substr(0, 4095);
    if (head.find("\"gemma3") != std::string::npos || head.find("\"gemma2") != std::string::npos) return MODEL_GEMMA3;
    return MODEL_QWEN3;
}

int model_type_layered(ModelType t) { return t == MODEL_NEVURAX || t == MODEL_PAPOSUN; }

const char *model_type_name(ModelType t)
{
    return t == MODEL_GEMMA3 ? "Gemma3" : t == MODEL_NEVURAX ? "Nevurax" : t == MODEL_PAPOSUN ? "Paposun" : "Qwen3";
}

}  // extern "C"
