// Gisedra: a decoder whose configuration lists its layers one by one and may run a group of them several times. Every
// sub-layer stands between two dynamic tanh norms (no statistics); behind the sub-layers each layer adds an RMS-normed
// vector made from the stream and the token's own columns of a second table. A mixer is either latent attention
// ("latent_attention": queries straight from the input, a normed latent and one rotated key part per token, interleaved
// pairs, a sliding window) or two mixers on one input ("parallel"): grouped softmax attention with a short causal
// convolution over queries, keys and values, a partial half-split rotation with scaled frequencies, a window that keeps
// the sequence's first positions and a gate per output column, beside retention (one fixed decay per head, heads normed and
// gated); their results are added with fixed scales. The feed-forward is a mixture of gated experts (silu) weighed by a
// softmax over the chosen router logits. In front of every pass of the loop a vector of that pass, and from the second pass
// on the embedding's output, is added to the stream. The head is a matrix of its own behind a final norm. This file reads
// the configuration, names the tensors and chooses the parts; the mechanisms are the parts' own.
//
// config.json: {"architecture": "Gisedra", "vocab", "width", "norm": {"eps"}, "token_side": {"dim"} | null,
//   "loop": {"start", "stop", "times"} | null,
//   "layers": [{"type": "latent_attention", "mixer": {"heads", "dim", "rot_dim", "vdim", "kv_rank", "scale", "rot": {"base", "dims"},
//                                                    "mask": {"size"}}, "mlp": ...},
//              {"type": "parallel", "mixer": {"left": {"heads", "kv_heads", "dim", "vdim", "conv", "scale", "mask": {"size", "keep_first"},
//                 "rot": {"base", "dims", "scaling": {"factor", "low", "high", "original"}}}, "left_scale",
//                 "right": {"heads", "dim", "vdim", "decay": [...]}, "right_scale"}, "mlp": ...}]}
//   mlp: {"kind": "moe", "router": {"experts", "top"}, "expert": {"ff"}} | null
//   May be absent or null: token_side (no such input), loop, vdim (as wide as dim), kv_heads (as many as heads), conv (none), rot
//   (none; rot_dim then 0), rot.scaling (frequencies as they are), mask (plain causal), mask.keep_first (0), left_scale and
//   right_scale (1), mlp.kind (moe), mlp.
// Tensors: embed, head, side.embed, loop.step, final.norm[.alpha, .b], l<i>.{norm1, norm1b, norm2, norm2b}[.alpha, .b],
// l<i>.mix.{q, dkv, dkv.norm, uk, uv, o} or l<i>.mix.left.{q, k, v}[.conv], l<i>.mix.left.{g, o}, l<i>.mix.right.{q, k, v, g, o},
// l<i>.mlp.{router, router.b}, l<i>.mlp.e<k>.{gate, up, down}, l<i>.side.{gate, proj, norm}; linear weights are stored [out, in].
#include <algorithm>
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
bool present(const Json& c, const char* key) {
    const Json* v = c.find(key);
    return v != nullptr && !v->is_null();
}
int64_t int_or(const Json& c, const char* key, const std::string& where, int64_t fallback, int64_t least = 1) {
    return present(c, key) ? need_int(c, key, where, least) : fallback;
}
double num_or(const Json& c, const char* key, const std::string& where, double fallback) { return present(c, key) ? need_num(c, key, where) : fallback; }

struct Rotation {
    int64_t dims = 0;
    double base = 10000.0;
    bool scaled = false;
    double factor = 1.0, low = 1.0, high = 1.0, original = 1.0;
    // The angle per position of pair i. Scaled: wavelengths beyond original / low are stretched by `factor`, those below
    // original / high kept, and between them the frequency goes from one to the other linearly in original / wavelength.
    double frequency(int64_t i) const {
        const double f = std::pow(base, -2.0 * static_cast<double>(i) / static_cast<double>(dims));
        if (!scaled) return f;
        const double wavelength = 2.0 * M_PI / f;
        if (wavelength < original / high) return f;
        if (wavelength > original / low) return f / factor;
        const double s = (original / wavelength - low) / (high - low);
        return (1.0 - s) * f / factor + s * f;
    }
};
struct AttentionConfig {                  // the left mixer of a pair
    int64_t heads = 0, kv_heads = 0, dim = 0, vdim = 0, taps = 0, window = 0, keep_first = 0;
    double scale = 1.0;
    Rotation rot;
};
struct RetentionConfig {                  // the right one
    int64_t heads = 0, dim = 0, vdim = 0;
    std::vector<float> decay;
};
struct LatentConfig {
    int64_t heads = 0, dim = 0, rot_dim = 0, vdim = 0, kv_rank = 0, window = 0;
    double scale = 1.0;
    Rotation rot;
};
struct LayerConfig {
    bool pair = false;                    // two mixers side by side, or latent attention
    AttentionConfig left;
    RetentionConfig right;
    LatentConfig latent;
    double left_scale = 1.0, right_scale = 1.0;
    int64_t experts = 0, top = 0, ff = 0;         // experts 0: no feed-forward
};

Rotation read_rotation(const Json& m, int64_t columns, const std::string& where) {
    Rotation r;
    if (!present(m, "rot")) return r;
    const Json& rot = need_object(m, "rot", where);
    const std::string w = where + "rot: ";
    r.base = need_num(rot, "base", w);
    r.dims = need_int(rot, "dims", w, 0);
    if (!(r.base > 0) || r.dims % 2 != 0 || r.dims > columns)
        throw ConfigError("config.json: " + where + "rot.base must be positive, rot.dims even and at most " + std::to_string(columns));
    if (r.dims > 512) throw ConfigError("config.json: " + where + "more than 512 rotated dimensions are not supported");
    if (present(rot, "scaling")) {
        const Json& s = need_object(rot, "scaling", w);
        r.scaled = true;
        r.factor = need_num(s, "factor", w + "scaling: ");
        r.low = need_num(s, "low", w + "scaling: ");
        r.high = need_num(s, "high", w + "scaling: ");
        r.original = need_num(s, "original", w + "scaling: ");
        if (!(r.factor > 0) || !(r.low > 0) || !(r.high > r.low) || !(r.original > 0))
            throw ConfigError("config.json: " + where + "rot.scaling needs factor, low and original positive and high above low");
    }
    return r;
}
// a sliding window (0: none) and, where it may have them, kept first positions
void read_mask(const Json& m, int64_t& window, int64_t* keep_first, const std::string& where) {
    if (!present(m, "mask")) return;
    const Json& mask = need_object(m, "mask", where);
    window = need_int(mask, "size", where + "mask: ");
    if (present(mask, "keep_first")) {
        const int64_t keep = need_int(mask, "keep_first", where + "mask: ", 0);
        if (keep_first != nullptr) *keep_first = keep;
        else if (keep > 0) throw ConfigError("config.json: " + where + "mask.keep_first: this mixer's window keeps no first positions");
    }
}

struct GisedraConfig {
    int64_t vocab = 0, width = 0, side_dim = 0;          // side_dim 0: no input of the tokens' own
    double eps = 1e-5;
    bool has_loop = false;
    int64_t loop_start = 0, loop_stop = 0, loop_times = 1;
    std::vector<LayerConfig> layers;

    explicit GisedraConfig(const Json& c) {
        vocab = need_int(c, "vocab", "");
        width = need_int(c, "width", "");
        eps = need_num(need_object(c, "norm", ""), "eps", "norm: ");
        if (!(eps > 0)) throw ConfigError("config.json: norm.eps must be positive");
        if (present(c, "token_side")) side_dim = need_int(need_object(c, "token_side", ""), "dim", "token_side: ");
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
            if (type->string() == "latent_attention") {
                LatentConfig& a = x.latent;
                a.heads = need_int(m, "heads", where);
                a.dim = need_int(m, "dim", where);
                a.vdim = int_or(m, "vdim", where, a.dim);
                a.rot_dim = int_or(m, "rot_dim", where, 0, 0);
                a.kv_rank = need_int(m, "kv_rank", where);
                a.scale = need_num(m, "scale", where);
                a.rot = read_rotation(m, a.rot_dim, where);
                if (a.rot_dim % 2 != 0) throw ConfigError("config.json: " + where + "rot_dim must be even");
                if (a.rot.scaled) throw ConfigError("config.json: " + where + "rot.scaling: latent attention's frequencies are not scaled");
                read_mask(m, a.window, nullptr, where);
            } else if (type->string() == "parallel") {
                x.pair = true;
                const std::string wl = where + "left: ", wr = where + "right: ";
                const Json &left = need_object(m, "left", where), &right = need_object(m, "right", where);
                AttentionConfig& a = x.left;
                a.heads = need_int(left, "heads", wl);
                a.kv_heads = int_or(left, "kv_heads", wl, a.heads);
                if (a.heads % a.kv_heads != 0) throw ConfigError("config.json: " + wl + "heads is not a multiple of kv_heads");
                a.dim = need_int(left, "dim", wl);
                a.vdim = int_or(left, "vdim", wl, a.dim);
                a.scale = need_num(left, "scale", wl);
                a.taps = int_or(left, "conv", wl, 0, 0);
                if (a.taps > 16) throw ConfigError("config.json: " + wl + "a convolution of more than 16 taps is not supported");
                a.rot = read_rotation(left, a.dim, wl);
                read_mask(left, a.window, &a.keep_first, wl);
                RetentionConfig& r = x.right;
                r.heads = need_int(right, "heads", wr);
                r.dim = need_int(right, "dim", wr);
                r.vdim = int_or(right, "vdim", wr, r.dim);
                const Json* decay = right.find("decay");
                if (decay == nullptr || !decay->is_array() || static_cast<int64_t>(decay->array().size()) != r.heads)
                    throw ConfigError("config.json: " + wr + "'decay' must be a list of one number per head");
                for (const Json& d : decay->array()) {
                    if (!d.is_number() || !(d.number() > 0.0) || d.number() > 1.0) throw ConfigError("config.json: " + wr + "a decay must lie above 0 and be at most 1");
                    r.decay.push_back(static_cast<float>(d.number()));
                }
                x.left_scale = num_or(m, "left_scale", where, 1.0);
                x.right_scale = num_or(m, "right_scale", where, 1.0);
            } else {
                throw ConfigError("config.json: " + where + "unknown layer type '" + type->string() + "' (known: latent_attention, parallel)");
            }
            if (present(l, "mlp")) {
                const Json& mlp = need_object(l, "mlp", where);
                if (const Json* kind = mlp.find("kind"))
                    if (!kind->is_string() || kind->string() != "moe") throw ConfigError("config.json: " + where + "mlp.kind must be 'moe'");
                const Json& r = need_object(mlp, "router", where + "mlp: ");
                x.experts = need_int(r, "experts", where + "mlp: router: ");
                x.top = need_int(r, "top", where + "mlp: router: ");
                if (x.top > x.experts) throw ConfigError("config.json: " + where + "mlp: router.top exceeds router.experts");
                if (x.experts > 256) throw ConfigError("config.json: " + where + "mlp: more than 256 experts are not supported");
                x.ff = need_int(need_object(mlp, "expert", where + "mlp: "), "ff", where + "mlp: expert: ");
            }
            layers.push_back(x);
        }
        if (present(c, "loop")) {
            const Json& loop = need_object(c, "loop", "");
            has_loop = true;
            loop_start = need_int(loop, "start", "loop: ", 0);
            loop_stop = need_int(loop, "stop", "loop: ", 0);
            loop_times = need_int(loop, "times", "loop: ");
            if (loop_start >= loop_stop || loop_stop > static_cast<int64_t>(layers.size()))
                throw ConfigError("config.json: loop: start < stop <= the number of layers is needed");
        }
    }
};

std::vector<ParamSpec> gisedra_specs(const Json& config) {
    const GisedraConfig c(config);
    const int64_t D = c.width;
    std::vector<ParamSpec> s;
    auto matrix = [&](const std::string& n, int64_t r, int64_t k) { s.push_back({n, {r, k}, ParamSpec::Matrix, false, 0.0, 1.0 / std::sqrt(static_cast<double>(k))}); };
    auto vector = [&](const std::string& n, int64_t k, double mean, double std) { s.push_back({n, {k}, ParamSpec::Vector, false, mean, std}); };
    auto norm = [&](const std::string& n) {
        vector(n, D, 1.0, 0.1);
        vector(n + ".b", D, 0.0, 0.1);
        s.push_back({n + ".alpha", {}, ParamSpec::Vector, false, 0.5, 0.1});
    };
    auto taps = [&](const std::string& n, int64_t channels, int64_t k) {
        s.push_back({n, {channels, k}, ParamSpec::Vector, false, 0.0, 1.0 / std::sqrt(static_cast<double>(k))});
    };
    s.push_back({"embed", {c.vocab, D}, ParamSpec::Matrix, false, 0.0, 1.0});
    if (c.side_dim > 0) s.push_back({"side.embed", {c.vocab, static_cast<int64_t>(c.layers.size()) * c.side_dim}, ParamSpec::Matrix, false, 0.0, 1.0});
    if (c.has_loop) s.push_back({"loop.step", {c.loop_times, D}, ParamSpec::Vector, false, 0.0, 0.3});
    for (size_t i = 0; i < c.layers.size(); ++i) {
        const LayerConfig& l = c.layers[i];
        const std::string L = "l" + std::to_string(i) + ".", M = L + "mix.";
        norm(L + "norm1");
        norm(L + "norm1b");
        if (l.experts > 0) {
            norm(L + "norm2");
            norm(L + "norm2b");
        }
        if (l.pair) {
            const AttentionConfig& a = l.left;
            const RetentionConfig& r = l.right;
            const std::string A = M + "left.", R = M + "right.";
            matrix(A + "q", a.heads * a.dim, D);
            matrix(A + "k", a.kv_heads * a.dim, D);
            matrix(A + "v", a.kv_heads * a.vdim, D);
            if (a.taps > 0) {
                taps(A + "q.conv", a.heads * a.dim, a.taps);
                taps(A + "k.conv", a.kv_heads * a.dim, a.taps);
                taps(A + "v.conv", a.kv_heads * a.vdim, a.taps);
            }
            matrix(A + "g", a.heads * a.vdim, D);
            matrix(A + "o", D, a.heads * a.vdim);
            matrix(R + "q", r.heads * r.dim, D);
            matrix(R + "k", r.heads * r.dim, D);
            matrix(R + "v", r.heads * r.vdim, D);
            matrix(R + "g", r.heads * r.vdim, D);
            matrix(R + "o", D, r.heads * r.vdim);
        } else {
            const LatentConfig& a = l.latent;
            matrix(M + "q", a.heads * (a.dim + a.rot_dim), D);
            matrix(M + "dkv", a.kv_rank + a.rot_dim, D);
            vector(M + "dkv.norm", a.kv_rank, 1.0, 0.1);
            // (kept transposed, [kv_rank, heads * dim]: queries are multiplied by it, not the latent)
            s.push_back({M + "uk", {a.heads * a.dim, a.kv_rank}, ParamSpec::Matrix, true, 0.0, 1.0 / std::sqrt(static_cast<double>(a.kv_rank))});
            matrix(M + "uv", a.heads * a.vdim, a.kv_rank);
            matrix(M + "o", D, a.heads * a.vdim);
        }
        for (int64_t e = 0; e < l.experts; ++e) {
            const std::string E = L + "mlp.e" + std::to_string(e) + ".";
            matrix(E + "gate", l.ff, D);
            matrix(E + "up", l.ff, D);
            matrix(E + "down", D, l.ff);
        }
        if (l.experts > 0) {
            matrix(L + "mlp.router", l.experts, D);
            vector(L + "mlp.router.b", l.experts, 0.0, 0.3);
        }
        if (c.side_dim > 0) {
            matrix(L + "side.gate", c.side_dim, D);
            matrix(L + "side.proj", D, c.side_dim);
            vector(L + "side.norm", D, 0.5, 0.1);
        }
    }
    norm("final.norm");
    matrix("head", c.vocab, D);
    return s;
}

using Tensors = std::map<std::string, Tensor2>;

Tensor2 column(const Tensor2& v) { return Tensor2(v.data, v.dtype, v.rows * v.cols, 1); }

std::unique_ptr<Mixer> latent_mixer(const LatentConfig& a, const std::string& M, double eps, int dtype, const Tensors& t, DeviceTensors& store) {
    // In bfloat16 the latent, its rotated part and the heads' plain columns are widened with zeros to the sizes of the
    // matrix-core kernels: the scores and the result stay what they are, the pages hold a few more columns.
    int rank = static_cast<int>(a.kv_rank), rot = static_cast<int>(a.rot_dim), plain = static_cast<int>(a.dim);
    if (dtype == BF16 && latent_tile_shape(rank, rot)) plain = (plain + 31) / 32 * 32;
    else { rank = static_cast<int>(a.kv_rank); rot = static_cast<int>(a.rot_dim); }
    Params p;
    p.num["dtype"] = dtype; p.num["eps"] = eps;
    p.num["heads"] = static_cast<double>(a.heads); p.num["value_dim"] = static_cast<double>(a.vdim);
    p.num["plain_dim"] = plain; p.num["rot_dim"] = rot; p.num["kv_rank"] = rank; p.num["q_rank"] = 0;
    p.num["norm_cols"] = static_cast<double>(a.kv_rank);
    p.num["scale"] = a.scale; p.num["rot_base"] = a.rot.base; p.num["rot_dims"] = static_cast<double>(a.rot.dims);
    p.num["window"] = static_cast<double>(a.window);
    const Tensor2 q = store.pad_row_parts(t.at(M + "q"), {a.dim, a.rot_dim}, {plain, rot});
    const Tensor2 dkv = store.pad_row_parts(t.at(M + "dkv"), {a.kv_rank, a.rot_dim}, {rank, rot});
    p.tensor["in.weight"] = store.join_rows({q, dkv});
    p.tensor["dkv.norm"] = store.pad_row_blocks(column(t.at(M + "dkv.norm")), a.kv_rank, rank);
    p.tensor["uk.weight"] = store.pad_col_blocks(store.pad_row_blocks(t.at(M + "uk"), a.kv_rank, rank), a.dim, plain);
    p.tensor["uv.weight"] = store.pad_col_blocks(t.at(M + "uv"), a.kv_rank, rank);
    p.tensor["out.weight"] = t.at(M + "o");
    return build_mixer("latent_attention", p);
}

// How the left mixer's heads lie in the engine. The attention kernels that every model shares take keys and values of one
// width, and their matrix-core tiles widths of 32, 64 and 128. In bfloat16 a head's values are cut into `parts` of at most 128
// columns, each with the head's queries and keys once more, and both widths are filled up with zeros to the next of those sizes:
// a part's scores are the head's, and its result is the part of the head's. Within a key/value head the parts come one after the
// other, each with all of that head's queries. Otherwise (32-bit; keys wider than 128) the narrower of the two widths is filled
// up to the wider one.
struct HeadLayout {
    int64_t parts = 1, keys = 0, values = 0;          // columns of a head's keys and values as they are laid out
    std::vector<int64_t> query_rows, key_rows, value_rows, result_rows;      // which stored row (or -1) each laid-out one is
    HeadLayout(const AttentionConfig& a, int dtype) {
        keys = (a.vdim > a.dim && a.vdim % 16 == 0) ? a.vdim : a.dim;
        values = (a.vdim < a.dim && a.dim % 16 == 0) ? a.dim : a.vdim;
        int64_t width = a.vdim;                       // stored value columns of a part
        if (dtype == BF16 && a.dim <= 128) {
            int64_t n = (a.vdim + 127) / 128;
            while (n <= 8 && a.vdim % n != 0) ++n;
            if (n <= 8) {
                parts = n;
                width = a.vdim / n;
                const int64_t need = std::max(a.dim, width);
                keys = values = need <= 32 ? 32 : (need <= 64 ? 64 : 128);
            }
        }
        const int64_t group = a.heads / a.kv_heads;
        auto add = [](std::vector<int64_t>& to, int64_t first, int64_t n, int64_t padded) {
            for (int64_t i = 0; i < padded; ++i) to.push_back(i < n ? first + i : -1);
        };
        for (int64_t g = 0; g < a.kv_heads; ++g)
            for (int64_t p = 0; p < parts; ++p) {
                add(key_rows, g * a.dim, a.dim, keys);
                add(value_rows, g * a.vdim + p * width, width, values);
                for (int64_t r = 0; r < group; ++r) {
                    add(query_rows, (g * group + r) * a.dim, a.dim, keys);
                    add(result_rows, (g * group + r) * a.vdim + p * width, width, values);
                }
            }
    }
};

std::unique_ptr<Mixer> pair_mixer(const LayerConfig& l, const std::string& M, int width, double eps, int dtype, const Tensors& t, DeviceTensors& store) {
    const AttentionConfig& a = l.left;
    const RetentionConfig& r = l.right;
    const std::string A = M + "left.", R = M + "right.";
    const HeadLayout lay(a, dtype);
    Params p;
    p.num["heads"] = static_cast<double>(a.heads * lay.parts); p.num["kv_heads"] = static_cast<double>(a.kv_heads * lay.parts);
    p.num["dim"] = static_cast<double>(lay.keys); p.num["value_dim"] = static_cast<double>(lay.values);
    p.num["scale"] = a.scale; p.num["eps"] = eps; p.num["dtype"] = dtype; p.num["gated"] = 1;
    p.num["window"] = static_cast<double>(a.window); p.num["keep_first"] = static_cast<double>(a.window > 0 ? a.keep_first : 0);
    p.num["rot_dims"] = static_cast<double>(a.rot.dims); p.num["rot_base"] = a.rot.base;
    p.str["qk_norm"] = "none";
    if (a.rot.scaled && a.rot.dims > 0) {
        std::vector<float> freqs;          // two floats a pair: the frequency to double precision
        for (int64_t i = 0; i < a.rot.dims / 2; ++i) {
            const double f = a.rot.frequency(i);
            freqs.push_back(static_cast<float>(f));
            freqs.push_back(static_cast<float>(f - static_cast<double>(freqs.back())));
        }
        p.tensor["rot_freqs"] = store.upload(freqs, 1, a.rot.dims, F32);
    }
    // The scale of the left result stands in the values' taps (fp32; the mixer is linear in its values). Without a convolution
    // a scale other than 1 makes one of a single tap.
    if (a.taps > 0 || l.left_scale != 1.0) {
        const int64_t taps = std::max<int64_t>(a.taps, 1), nq = a.heads * a.dim, nk = a.kv_heads * a.dim, nv = a.kv_heads * a.vdim;
        Tensor2 tq, tk, tv;
        if (a.taps > 0) {
            tq = t.at(A + "q.conv"); tk = t.at(A + "k.conv"); tv = t.at(A + "v.conv");
        } else {
            tq = store.upload(std::vector<float>(static_cast<size_t>(nq), 1.f), nq, 1, F32);
            tk = store.upload(std::vector<float>(static_cast<size_t>(nk), 1.f), nk, 1, F32);
            tv = store.upload(std::vector<float>(static_cast<size_t>(nv), 1.f), nv, 1, F32);
        }
        const Tensor2 scaled(store.scaled(tv, static_cast<float>(l.left_scale)).data, F32, nv, taps);
        p.tensor["qkv_conv"] = store.join_rows({store.pick_rows(tq, lay.query_rows), store.pick_rows(tk, lay.key_rows), store.pick_rows(scaled, lay.value_rows)});
    }
    const Tensor2 left_in = store.join_rows({store.pick_rows(t.at(A + "q"), lay.query_rows), store.pick_rows(t.at(A + "k"), lay.key_rows),
                                             store.pick_rows(t.at(A + "v"), lay.value_rows), store.pick_rows(t.at(A + "g"), lay.result_rows)});
    const Tensor2 left_out = store.pick_cols(t.at(A + "o"), lay.result_rows);
    // One input product and one output product for both mixers.
    Params pair;
    pair.num["size"] = width; pair.num["eps"] = eps; pair.num["dtype"] = dtype;
    const Tensor2 in = store.join_rows({left_in, t.at(R + "q"), t.at(R + "k"), t.at(R + "v"), t.at(R + "g")});
    const Tensor2 out = store.join_cols({left_out, t.at(R + "o")});
    auto out_columns = [&](int64_t first, int64_t n) { return Tensor2(static_cast<char*>(out.data) + static_cast<size_t>(first) * out.esz(), out.dtype, out.rows, n, out.stride); };
    pair.tensor["in.weight"] = in; pair.tensor["out.weight"] = out;
    p.tensor["in.weight"] = in.row_range(0, left_in.rows);
    p.tensor["out.weight"] = out_columns(0, left_out.cols);
    Params q;
    q.num["heads"] = static_cast<double>(r.heads); q.num["dim"] = static_cast<double>(r.dim); q.num["value_dim"] = static_cast<double>(r.vdim);
    q.num["eps"] = eps; q.num["dtype"] = dtype;
    q.num["k_scale"] = 1.0 / std::sqrt(static_cast<double>(r.dim));
    q.tensor["head_decay"] = store.upload(r.decay, 1, r.heads, F32);
    // (the heads' norm has no weight: the scale of the right result takes its place)
    if (l.right_scale != 1.0)
        q.tensor["norm.weight"] = store.upload(std::vector<float>(static_cast<size_t>(r.heads * r.vdim), static_cast<float>(l.right_scale)), 1, r.heads * r.vdim, F32);
    q.tensor["in.weight"] = in.row_range(left_in.rows, in.rows - left_in.rows);
    q.tensor["out.weight"] = out_columns(left_out.cols, out.cols - left_out.cols);
    pair.mixers.push_back(std::shared_ptr<const Mixer>(build_mixer("scored_attention", p).release()));
    pair.mixers.push_back(std::shared_ptr<const Mixer>(build_mixer("linear_attention", q).release()));
    return build_mixer("parallel", pair);
}

std::unique_ptr<FeedForward> experts(const LayerConfig& l, const std::string& F, int dtype, const Tensors& t, DeviceTensors& store) {
    Params f;
    f.num["dtype"] = dtype; f.num["experts"] = static_cast<double>(l.experts); f.num["ff"] = static_cast<double>(l.ff); f.num["top"] = static_cast<double>(l.top);
    f.str["activation"] = "silu_glu"; f.str["router"] = "softmax_chosen";
    std::vector<Tensor2> ups, downs;
    for (int64_t e = 0; e < l.experts; ++e) {
        const std::string E = F + "e" + std::to_string(e) + ".";
        ups.push_back(t.at(E + "gate")); ups.push_back(t.at(E + "up"));
        downs.push_back(t.at(E + "down"));
    }
    ups.push_back(t.at(F + "router"));
    // the experts' first products and behind them the router's, one matrix: steps of few rows run it as one product
    const Tensor2 joined = store.join_rows(ups);
    const int64_t n = 2 * l.experts * l.ff;
    f.tensor["up_router.weight"] = joined;
    f.tensor["up_router.bias"] = store.join_rows({column(store.zeros(n)), column(t.at(F + "router.b"))});
    f.tensor["up.weight"] = joined.row_range(0, n);
    f.tensor["router"] = joined.row_range(n, l.experts);
    f.tensor["router.bias"] = t.at(F + "router.b");
    f.tensor["down.weight"] = store.join_cols(downs);
    return build_feed_forward("routed_experts", f);
}

void gisedra_assemble(const Json& config, const Tensors& t, int dtype, LoadedModel& out) {
    const GisedraConfig c(config);
    const int D = static_cast<int>(c.width), n = static_cast<int>(c.layers.size());
    DecoderModel& m = out.model;
    {
        Params e, h;
        e.tensor["table"] = t.at("embed");
        m.embedding = build_embedding("token_table", e);
        h.tensor["weight"] = t.at("head");
        h.num["dtype"] = dtype;
        m.head = build_head("linear", h);
    }
    auto norm = [&](const std::string& name) {
        Params p;
        p.num["size"] = D; p.num["dtype"] = dtype;
        p.tensor["alpha"] = t.at(name + ".alpha"); p.tensor["weight"] = t.at(name); p.tensor["bias"] = t.at(name + ".b");
        return build_norm("dynamic_tanh", p);
    };
    for (int i = 0; i < n; ++i) {
        const LayerConfig& l = c.layers[static_cast<size_t>(i)];
        const std::string L = "l" + std::to_string(i) + ".", M = L + "mix.";
        std::unique_ptr<Mixer> mixer = l.pair ? pair_mixer(l, M, D, c.eps, dtype, t, out.store) : latent_mixer(l.latent, M, c.eps, dtype, t, out.store);
        std::unique_ptr<FeedForward> ff;
        std::vector<std::unique_ptr<Norm>> norms;
        norms.push_back(norm(L + "norm1"));
        norms.push_back(norm(L + "norm1b"));
        if (l.experts > 0) {
            ff = experts(l, L + "mlp.", dtype, t, out.store);
            norms.push_back(norm(L + "norm2"));
            norms.push_back(norm(L + "norm2b"));
        }
        Params b;
        b.num["size"] = D;
        m.layers.push_back(build_block("sandwich_norm", std::move(mixer), std::move(ff), std::move(norms), b));
        if (c.side_dim > 0) {
            Params p;
            p.num["dtype"] = dtype; p.num["eps"] = c.eps; p.num["column"] = static_cast<double>(i * c.side_dim);
            p.tensor["table"] = t.at("side.embed");
            p.tensor["gate.weight"] = t.at(L + "side.gate"); p.tensor["proj.weight"] = t.at(L + "side.proj"); p.tensor["norm.weight"] = t.at(L + "side.norm");
            if (dtype == BF16 && token_side_fits(D, static_cast<int>(c.side_dim))) {
                const int64_t dim = token_side_padded(static_cast<int>(c.side_dim));
                p.tensor["gate.tiles"] = out.store.operand_tiles(t.at(L + "side.gate"), dim, D);
                p.tensor["proj.tiles"] = out.store.operand_tiles(t.at(L + "side.proj"), D, (dim + 31) / 32 * 32);
                p.tensor["proj.gram"] = out.store.gram_tiles(t.at(L + "side.proj"), dim);
            }
            m.stream_steps.push_back(build_stream_step("token_side", p));          // step i stands behind layer i
        }
    }
    if (c.has_loop) {
        Params p;
        p.num["dtype"] = dtype;
        p.tensor["steps"] = t.at("loop.step");
        m.stream_steps.push_back(build_stream_step("embedding_add", p));
    }
    // the order: the layers in front of the loop, the loop's layers once per pass (a cache of its own per run, the stream
    // step in front of each pass's first layer), the layers behind it
    int cache = 0;
    auto call = [&](int layer, int pass) {
        LayerCall lc;
        lc.layer = layer; lc.cache = cache++;
        if (pass >= 0) { lc.before = static_cast<int>(m.stream_steps.size()) - 1; lc.pass = pass; }
        if (c.side_dim > 0) lc.after = layer;
        m.order.push_back(lc);
    };
    const int start = c.has_loop ? static_cast<int>(c.loop_start) : n, stop = c.has_loop ? static_cast<int>(c.loop_stop) : n;
    for (int i = 0; i < start; ++i) call(i, -1);
    if (c.has_loop)
        for (int pass = 0; pass < c.loop_times; ++pass)
            for (int i = start; i < stop; ++i) call(i, i == start ? pass : -1);
    for (int i = stop; i < n; ++i) call(i, -1);
    m.final_norm = norm("final.norm");
    out.max_positions = 0;          // positions are not bounded by a table
    if (const Json* e = config.find("eos_token_id")) if (e->is_integer()) out.eos_token_id = static_cast<int>(e->integer());
}

}  // namespace

void register_gisedra() {
    Architecture a;
    a.name = "Gisedra";
    a.param_specs = gisedra_specs;
    a.assemble = gisedra_assemble;
    register_architecture(a, "gisedra");
}

}  // namespace minillm
