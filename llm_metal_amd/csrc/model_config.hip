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

}  // namespace

bool read_stack_config(const std::string &text, StackConfig &out, std::string &why)
{
    JsonValue root;
    if (!JsonValue::parse_text(text, root)) { why = "not valid JSON"; return false; }
    Reader r{why, ""};
    out = StackConfig();
    out.vocab = r.count(root, "vocab");
    out.width = r.count(root, "width");
    out.emb_scale = (float)r.real(root["embedding"], "scale");
    out.eps = (float)r.real(root["norm"], "eps");
    if (root["layers"].items.empty()) r.fail("'layers' is missing or empty");
    for (size_t i = 0; i < root["layers"].items.size() && r.ok; i++) {
        const JsonValue &L = root["layers"].items[i], &mx = L["mixer"], &mlp = L["mlp"];
        r.at = "layer " + std::to_string(i) + ": ";
        LayerConfig c;
        const std::string &type = L["type"].str;
        c.heads = r.count(mx, "heads"); c.dim = r.count(mx, "dim"); c.vdim = r.count(mx, "vdim");
        if (type == "delta" || type == "channel_delta") {
            c.mixer = type == "delta" ? MIX_DELTA : MIX_CHANNEL_DELTA;
            c.kv_heads = r.count(mx, "kv_heads"); c.taps = r.count(mx, "conv");
            if (r.ok && c.heads % c.kv_heads) r.fail("'heads' is not a multiple of 'kv_heads'");
            if (c.dim > 256) r.fail("key dimension above 256");
            if (c.taps > 16) r.fail("more than 16 convolution taps");
        } else if (type == "latent_attention") {
            c.mixer = MIX_LATENT;
            c.rot_dim = r.count(mx, "rot_dim"); c.kv_rank = r.count(mx, "kv_rank");
            c.window = r.count(mx["mask"], "size");
            c.rot_dims = r.count(mx["rot"], "dims"); c.rot_base = r.real(mx["rot"], "base");
            c.scale = (float)r.real(mx, "scale");
            if (r.ok && (c.rot_dims > c.rot_dim || (c.rot_dims & 1))) r.fail("'rot.dims' is odd or above 'rot_dim'");
            if (r.ok && !(c.rot_base > 0.0)) r.fail("'rot.base' is not positive");
            if (c.kv_rank > 1024 || c.rot_dim > 1024 || c.dim > 1024) r.fail("latent size or head dimension above 1024");
        } else r.fail("unknown mixer '" + type + "'");
        if (mlp.kind == JsonValue::OBJECT) {
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
    if (JsonValue::parse_text(text, root) && root["architecture"].str == "Nevurax") return MODEL_NEVURAX;
    const std::string head = text.substr(0, 4095);
    if (head.find("\"gemma3") != std::string::npos || head.find("\"gemma2") != std::string::npos) return MODEL_GEMMA3;
    return MODEL_QWEN3;
}

const char *model_type_name(ModelType t)
{
    return t == MODEL_GEMMA3 ? "Gemma3" : t == MODEL_NEVURAX ? "Nevurax" : "Qwen3";
}

}  // extern "C"
