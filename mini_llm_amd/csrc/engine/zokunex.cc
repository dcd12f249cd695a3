// Zokunex: a decoder whose configuration lists its layers one by one. The sub-layers read the residual stream itself and a
// layer norm (weight, no bias) stands behind each of them. The mixer is a matrix memory with exponential gates ("mlstm") or
// latent attention without a query latent, with half-split rotary pairs, a gate per head and no window
// ("latent_attention"). The feed-forward squares the rectified hidden values, or is a mixture of small ungated experts
// (exact GELU), some of which hand on their input, chosen by softmax score plus a correction and weighed by the score. The
// logits are scaled; the head is a matrix of its own behind a final layer norm. This file reads the configuration, names the
// tensors and chooses the parts; the mechanisms are the parts' own.
//
// config.json: {"architecture": "Zokunex", "vocab", "width", "norm": {"eps"}, "logit_scale",
//   "layers": [{"type": "mlstm", "mixer": {"heads", "dim", "vdim", "gate_cap"}, "mlp": ...},
//              {"type": "latent_attention", "mixer": {"heads", "dim", "rot_dim", "vdim", "kv_rank", "scale", "rot": {"base", "dims"}}, "mlp": ...}]}
//   mlp: {"kind": "dense", "ff"} | {"kind": "moe", "router": {"experts", "top", "identity"}, "expert": {"ff"}} | null
// Tensors: embed, head, final.norm, l<i>.norm1[/norm2], l<i>.mix.{q, k, v, g, o, norm, i, i.b, f, f.b} or l<i>.mix.{q, dkv,
// dkv.norm, uk, uv, g, o}, l<i>.mlp.{up, down} or l<i>.mlp.{router, correction, e<k>.{up, down}}; linear weights are stored
// [out, in].
#include <cmath>

#include "arch.h"

namespace minillm {

namespace {

int64_t need_int(const Json& c, const char* key, const std::string& where, int64_t least = 1) {
    const Json* v = c.find(key);
    if (v == nullptr || !v->is_integer()) throw ConfigError("config.json: " + where + "integer key '" + key + "' is missing");
    if (v->integer() < least) throw ConfigError("config.json: " + where + "'" + key + "' must be at least " + std::to_string(least));
    return v->integer();
}
double need_num(const Json& c, const char* key, const std::string& where) {
    const Json* v = c.find(key);
    if (v == nullptr || !v->is_number()) throw ConfigError("config.json: " + where + "number key '" + key + "' is missing");
    return v->number();
}
const Json& need_object(const Json& c, const char* key, const std::string& where) {
    const Json* v = c.find(key);
    if (v == nullptr || !v->is_object()) throw ConfigError("config.json: " + where + "object '" + key + "' is missing");
    return *v;
}
// absent and null are the same
bool present(const Json& c, const char* key) {
    const Json* v = c.find(key);
    return v != nullptr && !v->is_null();
}

struct LayerConfig {
    enum Kind { Memory, Latent } kind = Memory;
    int64_t heads = 0, dim = 0, vdim = 0, kv_rank = 0, rot_dim = 0, rot_dims = 0;
    double gate_cap = 0.0, scale = 1.0, rot_base = 10000.0;
    enum Mlp { None, Dense, Moe } mlp = None;
    int64_t ff = 0, experts = 0, top = 0, identity = 0;
};

struct ZokunexConfig {
    int64_t vocab = 0, width = 0;
    double eps = 1e-6, logit_scale = 1.0;
    std::vector<LayerConfig> layers;

    explicit ZokunexConfig(const Json& c) {
        vocab = need_int(c, "vocab", "");
        width = need_int(c, "width", "");
        eps = need_num(need_object(c, "norm", ""), "eps", "norm: ");
        if (!(eps > 0)) throw ConfigError("config.json: norm.eps must be positive");
        if (present(c, "logit_scale")) logit_scale = need_num(c, "logit_scale", "");
        const Json* ls = c.find("layers");
        if (ls == nullptr || !ls->is_array() || ls->array().empty()) throw ConfigError("config.json: 'layers' must be a list of layers");
        for (size_t i = 0; i < ls->array().size(); ++i) {
            const Json& l = ls->array()[i];
            const std::string where = "layer " + std::to_string(i) + ": ";
            if (!l.is_object()) throw ConfigError("config.json: " + where + "not an object");
            const Json* type = l.find("type");
            if (type == nullptr || !type->is_string()) throw ConfigError("config.json: " + where + "'type' is missing");
            const Json& m = need_object(l, "mixer", where);
            LayerConfig x;
            x.heads = need_int(m, "heads", where);
            x.dim = need_int(m, "dim", where);
            x.vdim = present(m, "vdim") ? need_int(m, "vdim", where) : x.dim;
            if (type->string() == "mlstm") {
                x.kind = LayerConfig::Memory;
                x.gate_cap = need_num(m, "gate_cap", where);
                if (!(x.gate_cap > 0)) throw ConfigError("config.json: " + where + "gate_cap must be positive");
            } else if (type->string() == "latent_attention") {
                x.kind = LayerConfig::Latent;
                x.kv_rank = need_int(m, "kv_rank", where);
                x.rot_dim = present(m, "rot_dim") ? need_int(m, "rot_dim", where, 0) : 0;
                x.scale = need_num(m, "scale", where);
                if (x.rot_dim > 0) {
                    const Json& rot = need_object(m, "rot", where);
                    x.rot_base = need_num(rot, "base", where + "rot: ");
                    x.rot_dims = need_int(rot, "dims", where + "rot: ", 0);
                    if (!(x.rot_base > 0) || x.rot_dims % 2 != 0 || x.rot_dim % 2 != 0 || x.rot_dims > x.rot_dim)
                        throw ConfigError("config.json: " + where + "rot.base must be positive, rot.dims and rot_dim even, rot.dims at most rot_dim");
                }
            } else {
                throw ConfigError("config.json: " + where + "unknown layer type '" + type->string() + "' (known: latent_attention, mlstm)");
            }
            if (present(l, "mlp")) {
                const Json& mlp = need_object(l, "mlp", where);
                std::string kind = "dense";
                if (const Json* k = mlp.find("kind")) {
                    if (!k->is_string()) throw ConfigError("config.json: " + where + "mlp.kind must be a string");
                    kind = k->string();
                }
                if (kind == "dense") {
                    x.mlp = LayerConfig::Dense;
                    x.ff = need_int(mlp, "ff", where + "mlp: ");
                } else if (kind == "moe") {
                    x.mlp = LayerConfig::Moe;
                    const Json& r = need_object(mlp, "router", where + "mlp: ");
                    x.experts = need_int(r, "experts", where + "mlp: router: ");
                    x.top = need_int(r, "top", where + "mlp: router: ");
                    x.identity = present(r, "identity") ? need_int(r, "identity", where + "mlp: router: ", 0) : 0;
                    if (x.top > x.experts + x.identity) throw ConfigError("config.json: " + where + "mlp: router.top exceeds the experts");
                    if (x.experts + x.identity > 256) throw ConfigError("config.json: " + where + "mlp: more than 256 experts are not supported");
                    x.ff = need_int(need_object(mlp, "expert", where + "mlp: "), "ff", where + "mlp: expert: ");
                } else {
                    throw ConfigError("config.json: " + where + "mlp.kind must be 'dense' or 'moe'");
                }
            }
            layers.push_back(x);
        }
    }
};

std::vector<ParamSpec> zokunex_specs(const Json& config) {
    const ZokunexConfig c(config);
    const int64_t D = c.width;
    std::vector<ParamSpec> s;
    auto matrix = [&](const std::string& n, int64_t r, int64_t k) { s.push_back({n, {r, k}, ParamSpec::Matrix, false, 0.0, 1.0 / std::sqrt(static_cast<double>(k))}); };
    auto vector = [&](const std::string& n, int64_t k, double mean, double std) { s.push_back({n, {k}, ParamSpec::Vector, false, mean, std}); };
    s.push_back({"embed", {c.vocab, D}, ParamSpec::Matrix, false, 0.0, 1.0});
    for (size_t i = 0; i < c.layers.size(); ++i) {
        const LayerConfig& x = c.layers[i];
        const std::string L = "l" + std::to_string(i) + ".", M = L + "mix.";
        vector(L + "norm1", D, 1.0, 0.1);
        if (x.mlp != LayerConfig::None) vector(L + "norm2", D, 1.0, 0.1);
        if (x.kind == LayerConfig::Memory) {
            matrix(M + "q", x.heads * x.dim, D);
            matrix(M + "k", x.heads * x.dim, D);
            matrix(M + "v", x.heads * x.vdim, D);
            matrix(M + "g", x.heads * x.vdim, D);
            matrix(M + "o", D, x.heads * x.vdim);
            vector(M + "norm", x.heads * x.vdim, 1.0, 0.1);
            matrix(M + "i", x.heads, D);
            vector(M + "i.b", x.heads, -1.0, 1.0);
            matrix(M + "f", x.heads, D);
            vector(M + "f.b", x.heads, 3.0, 1.5);
        } else {
            matrix(M + "q", x.heads * (x.dim + x.rot_dim), D);
            matrix(M + "dkv", x.kv_rank + x.rot_dim, D);
            vector(M + "dkv.norm", x.kv_rank, 1.0, 0.1);
            // (kept transposed, [kv_rank, heads * dim]: queries are multiplied by it, not the latent)
            s.push_back({M + "uk", {x.heads * x.dim, x.kv_rank}, ParamSpec::Matrix, true, 0.0, 1.0 / std::sqrt(static_cast<double>(x.kv_rank))});
            matrix(M + "uv", x.heads * x.vdim, x.kv_rank);
            matrix(M + "g", x.heads, D);
            matrix(M + "o", D, x.heads * x.vdim);
        }
        if (x.mlp == LayerConfig::Dense) {
            matrix(L + "mlp.up", x.ff, D);
            matrix(L + "mlp.down", D, x.ff);
        } else if (x.mlp == LayerConfig::Moe) {
            for (int64_t e = 0; e < x.experts; ++e) {
                const std::string E = L + "mlp.e" + std::to_string(e) + ".";
                matrix(E + "up", x.ff, D);
                matrix(E + "down", D, x.ff);
            }
            matrix(L + "mlp.router", x.experts + x.identity, D);
            vector(L + "mlp.correction", x.experts + x.identity, 0.0, 0.05);
        }
    }
    vector("final.norm", D, 1.0, 0.1);
    matrix("head", c.vocab, D);
    return s;
}

void zokunex_assemble(const Json& config, const std::map<std::string, Tensor2>& t, int dtype, LoadedModel& out) {
    const ZokunexConfig c(config);
    const int D = static_cast<int>(c.width);
    DecoderModel& m = out.model;
    {
        Params e, h;
        e.tensor["table"] = t.at("embed");
        m.embedding = build_embedding("token_table", e);
        h.tensor["weight"] = t.at("head");
        h.num["dtype"] = dtype;
        m.head = build_head("linear", h);
    }
    auto norm = [&](const Tensor2& weight) {
        Params p;
        p.num["size"] = D; p.num["eps"] = c.eps; p.num["dtype"] = dtype;
        p.tensor["gamma"] = weight;
        return build_norm("layernorm", p);
    };
    auto column = [](const Tensor2& v) { return Tensor2(v.data, v.dtype, v.rows * v.cols, 1); };
    for (size_t i = 0; i < c.layers.size(); ++i) {
        const LayerConfig& x = c.layers[i];
        const std::string L = "l" + std::to_string(i) + ".", M = L + "mix.";
        Params p;
        p.num["dtype"] = dtype; p.num["eps"] = c.eps;
        p.num["heads"] = static_cast<double>(x.heads); p.num["value_dim"] = static_cast<double>(x.vdim);
        p.tensor["out.weight"] = t.at(M + "o");
        std::unique_ptr<Mixer> mixer;
        if (x.kind == LayerConfig::Memory) {
            p.num["dim"] = static_cast<double>(x.dim); p.num["gate_cap"] = x.gate_cap;
            p.tensor["in.weight"] = out.store.join_rows({t.at(M + "q"), t.at(M + "k"), t.at(M + "v"), t.at(M + "g"), t.at(M + "i"), t.at(M + "f")});
            p.tensor["i.bias"] = t.at(M + "i.b"); p.tensor["f.bias"] = t.at(M + "f.b"); p.tensor["norm.weight"] = t.at(M + "norm");
            mixer = build_mixer("matrix_memory", p);
        } else {
            // In bfloat16 the latent, its rotated part and the heads' plain columns are widened with zeros to the sizes of the
            // matrix-core kernels: the scores and the result stay what they are, the pages hold a few more columns.
            int rank = static_cast<int>(x.kv_rank), rot = static_cast<int>(x.rot_dim), plain = static_cast<int>(x.dim);
            if (dtype == BF16 && latent_tile_shape(rank, rot)) plain = (plain + 31) / 32 * 32;
            else { rank = static_cast<int>(x.kv_rank); rot = static_cast<int>(x.rot_dim); }
            const Tensor2 q = out.store.pad_row_parts(t.at(M + "q"), {x.dim, x.rot_dim}, {plain, rot});
            const Tensor2 dkv = out.store.pad_row_parts(t.at(M + "dkv"), {x.kv_rank, x.rot_dim}, {rank, rot});
            p.num["plain_dim"] = plain; p.num["rot_dim"] = rot; p.num["kv_rank"] = rank; p.num["q_rank"] = 0;
            p.num["norm_cols"] = static_cast<double>(x.kv_rank);
            p.num["scale"] = x.scale; p.num["rot_base"] = x.rot_base; p.num["rot_dims"] = static_cast<double>(x.rot_dims); p.num["half_split"] = 1;
            p.num["gated"] = 1;
            p.tensor["in.weight"] = out.store.join_rows({q, dkv, t.at(M + "g")});
            p.tensor["dkv.norm"] = out.store.pad_row_blocks(column(t.at(M + "dkv.norm")), x.kv_rank, rank);
            p.tensor["uk.weight"] = out.store.pad_col_blocks(out.store.pad_row_blocks(t.at(M + "uk"), x.kv_rank, rank), x.dim, plain);
            p.tensor["uv.weight"] = out.store.pad_col_blocks(t.at(M + "uv"), x.kv_rank, rank);
            mixer = build_mixer("latent_attention", p);
        }
        std::unique_ptr<FeedForward> ff;
        std::vector<std::unique_ptr<Norm>> norms;
        norms.push_back(norm(t.at(L + "norm1")));
        if (x.mlp == LayerConfig::Dense) {
            Params f;
            f.num["dtype"] = dtype;
            f.str["activation"] = "relu2";
            f.tensor["up.weight"] = t.at(L + "mlp.up"); f.tensor["down.weight"] = t.at(L + "mlp.down");
            ff = build_feed_forward("dense_mlp", f);
        } else if (x.mlp == LayerConfig::Moe) {
            Params f;
            f.num["dtype"] = dtype; f.num["experts"] = static_cast<double>(x.experts); f.num["ff"] = static_cast<double>(x.ff);
            f.num["top"] = static_cast<double>(x.top); f.num["identity"] = static_cast<double>(x.identity);
            f.str["activation"] = "gelu_erf";
            std::vector<Tensor2> ups, downs;
            for (int64_t e = 0; e < x.experts; ++e) {
                const std::string E = L + "mlp.e" + std::to_string(e) + ".";
                ups.push_back(t.at(E + "up"));
                downs.push_back(t.at(E + "down"));
            }
            ups.push_back(t.at(L + "mlp.router"));
            // the experts' first products and behind them the router's, one matrix: steps of few rows run it as one product
            const Tensor2 joined = out.store.join_rows(ups);
            f.tensor["up_router.weight"] = joined;
            f.tensor["up.weight"] = joined.row_range(0, x.experts * x.ff);
            f.tensor["router"] = joined.row_range(x.experts * x.ff, x.experts + x.identity);
            f.tensor["down.weight"] = out.store.join_cols(downs);
            f.tensor["correction"] = t.at(L + "mlp.correction");
            ff = build_feed_forward("routed_experts", f);
        }
        if (ff) norms.push_back(norm(t.at(L + "norm2")));
        Params b;
        b.num["dtype"] = dtype; b.num["size"] = D;
        m.layers.push_back(build_block("post_norm", std::move(mixer), std::move(ff), std::move(norms), b));
        LayerCall call;
        call.layer = call.cache = static_cast<int>(i);
        m.order.push_back(call);
    }
    // (the logits' scale stands in the final norm's weight: the head is linear)
    m.final_norm = norm(out.store.scaled(t.at("final.norm"), static_cast<float>(c.logit_scale)));
    out.max_positions = 0;          // positions are not bounded by a table
    if (const Json* e = config.find("eos_token_id")) if (e->is_integer()) out.eos_token_id = static_cast<int>(e->integer());
}

}  // namespace

void register_zokunex() {
    Architecture a;
    a.name = "Zokunex";
    a.param_specs = zokunex_specs;
    a.assemble = zokunex_assemble;
    register_architecture(a, "zokunex");
}

}  // namespace minillm
