// The dynamic tanh norm, and what is added to the stream between layers: the embedding's output with a vector per pass of
// a loop, and a vector made from the stream and the token's own row of a second table.
#include "parts.h"

namespace minillm {

namespace {

const float* f32_vector(const Params& p, const char* key, int64_t n, const char* who) {
    const Tensor2& t = p.weights(key);
    if (t.dtype != F32 || t.rows * t.cols != n || !t.contiguous()) fail("%s: '%s' must be contiguous float32 [%lld]", who, key, (long long)n);
    return static_cast<const float*>(t.data);
}

// h = tanh(alpha x) * weight + bias, every column on its own (no mean, no variance), in fp32. Parameters: size, dtype;
// tensors alpha (one number), weight, bias.
class TanhNorm final : public Norm {
public:
    explicit TanhNorm(const Params& p) {
        size_ = p.integer("size");
        dtype = p.integer("dtype");
        n_.alpha = f32_vector(p, "alpha", 1, "dynamic_tanh");
        n_.weight = f32_vector(p, "weight", size_, "dynamic_tanh");
        n_.bias = f32_vector(p, "bias", size_, "dynamic_tanh");
    }
    Tensor2 forward(const Tensor2& x, const int* rows, int n, Arena& arena, hipStream_t s) const override {
        Tensor2 h = arena.tensor(dtype, n, size_);
        forward_into(x, rows, h, s);
        return h;
    }
    void forward_into(const Tensor2& x, const int* rows, const Tensor2& out, hipStream_t s) const override {
        if (x.cols != size_) fail("dynamic_tanh: rows of %lld, the norm is %d wide", (long long)x.cols, size_);
        tanh_norm(x, n_, out, rows, s);
    }
    void add_scaled(const Tensor2& y, const float* scale, float mult, const Tensor2& x, bool clear, hipStream_t s,
                    const Tensor2* copy) const override {
        if (scale != nullptr || mult != 1.f) fail("dynamic_tanh: a norm behind a sub-layer takes no scale or multiplier");
        StreamAdd add;
        add.norm = n_; add.x = x; add.y = y;
        if (copy != nullptr) add.copy = *copy;
        stream_add(add, nullptr, nullptr, dtype == F32, s);
        if (clear) fill_zero(y, s);
    }
    bool pointwise(MllmTanhNorm& n) const override { n = n_; return true; }
    size_t workspace_bytes(int rows) const override { return static_cast<size_t>(rows) * size_ * dtype_size(dtype) + 256; }
    void add_cost(StepCost& c) const override { c.weight_bytes += 8.0 * size_ + 4.0; }

private:
    int size_ = 0;
    MllmTanhNorm n_{};
};

// In front of every pass of a group of layers that runs several times: x += x0 (the embedding's output; not in front of
// pass 0), then x += steps[pass]. Parameter dtype; tensor steps ([passes, width] fp32).
class EmbeddingAdd final : public StreamStep {
public:
    explicit EmbeddingAdd(const Params& p) : dtype_(p.integer("dtype")), steps_(p.weights("steps")) {
        if (steps_.dtype != F32 || !steps_.contiguous() || steps_.rows < 1) fail("embedding_add: the steps must be contiguous float32 [passes, width]");
    }
    void forward(const Tensor2& x, const Tensor2& x0, int pass, const StepView& step, Arena&, hipStream_t s) const override {
        if (x.cols != steps_.cols) fail("embedding_add: steps of width %lld for a stream of %lld", (long long)steps_.cols, (long long)x.cols);
        if (pass < 0 || pass >= steps_.rows) fail("embedding_add: pass %d of %lld", pass, (long long)steps_.rows);
        if (pass > 0 && x0.data == nullptr) fail("embedding_add needs the embedding's output");
        StreamAdd add;
        add.x = x;
        if (step.leave.wanted) { add.copy = step.leave.into; add.next = step.leave.norm; }
        stream_add(add, pass > 0 ? &x0 : nullptr, static_cast<const float*>(steps_.data) + static_cast<size_t>(pass) * steps_.cols, dtype_ == F32, s);
    }
    size_t workspace_bytes(int) const override { return 0; }
    bool wants_embedding_output() const override { return steps_.rows > 1; }
    bool leaves_copy() const override { return true; }
    void add_cost(StepCost& c) const override { c.weight_bytes += 4.0 * steps_.cols; }

private:
    int dtype_ = BF16;
    Tensor2 steps_;
};

// Behind a layer: with e the `dim` columns from column `column` on of the token's row of a second table,
//   g = gelu_tanh(W_gate x) * e,  y = W_proj g,  x += y / sqrt(mean(y^2) + eps) * weight.
// Parameters: dtype, column, eps; tensors table [vocab, columns], gate.weight [dim, width], proj.weight [width, dim],
// norm.weight [width]; and, for one kernel that does it all, gate.tiles, proj.tiles and proj.gram (the two maps and the second
// one's square in operand order, see ops.h).
class TokenSide final : public StreamStep {
public:
    explicit TokenSide(const Params& p) : table_(p.weights("table")), gate_(p.weights("gate.weight"), nullptr), proj_(p.weights("proj.weight"), nullptr) {
        dtype_ = p.integer("dtype");
        column_ = p.integer("column");
        eps_ = static_cast<float>(p.number("eps"));
        dim_ = gate_.out_features();
        if (proj_.in_features() != dim_ || proj_.out_features() != gate_.in_features()) fail("token_side: the two maps' shapes do not fit");
        if (column_ < 0 || column_ + dim_ > table_.cols || table_.dtype != dtype_) fail("token_side: columns %d to %d of a table of %lld", column_, column_ + dim_, (long long)table_.cols);
        norm_ = f32_vector(p, "norm.weight", proj_.out_features(), "token_side");
        if (const Tensor2* g = p.weights_or_null("gate.tiles")) {
            gate_tiles_ = *g;
            proj_tiles_ = p.weights("proj.tiles");
            gram_tiles_ = p.weights("proj.gram");
            if (dtype_ != BF16 || !token_side_fits(proj_.out_features(), dim_)) fail("token_side: tiles for a width of %d and %d columns: no kernel takes them", proj_.out_features(), dim_);
        }
    }
    void forward(const Tensor2& x, const Tensor2&, int, const StepView& step, Arena& arena, hipStream_t s) const override {
        const int T = step.n_tokens, ldz = (dim_ + 3) / 4 * 4, ldg = (dim_ + 7) / 8 * 8;
        if (x.cols != proj_.out_features()) fail("token_side of width %d was handed a stream of %lld", proj_.out_features(), (long long)x.cols);
        if (gate_tiles_.data != nullptr) {
            StreamAdd add;
            add.x = x;
            if (step.leave.wanted) { add.copy = step.leave.into; add.next = step.leave.norm; }
            token_side(add, step.step_copy, gate_tiles_, proj_tiles_, gram_tiles_, norm_, eps_, step.token_ids, &step.fed, table_, column_, dim_, s);
            return;
        }
        Tensor2 h = x;
        if (dtype_ == BF16) { h = arena.tensor(BF16, T, x.cols); cast_stream(x, h, s); }
        const Tensor2 z(arena.take(static_cast<size_t>(T) * ldz * 4), F32, T, dim_, ldz);
        gate_(h, z, STORE_F32, nullptr, s);
        const Tensor2 g(arena.take(static_cast<size_t>(T) * ldg * dtype_size(dtype_)), dtype_, T, dim_, ldg);
        token_gate(z, step.token_ids, &step.fed, table_, column_, g, s);
        const Tensor2 y = arena.tensor(F32, T, x.cols);
        proj_(g, y, STORE_F32, nullptr, s);
        rmsnorm_add(y, norm_, nullptr, 1.f, eps_, x, false, s);
    }
    size_t workspace_bytes(int tokens) const override {
        return static_cast<size_t>(tokens) * (proj_.out_features() * 6 + (dim_ + 8) * 8) + 2048;
    }
    bool leaves_copy() const override { return gate_tiles_.data != nullptr; }
    bool wants_copy() const override { return gate_tiles_.data != nullptr; }
    void reserve(int, hipStream_t s) const override { reserve_linear_scratch(s); }
    void add_cost(StepCost& c) const override { gate_.add_cost(c); proj_.add_cost(c); c.weight_bytes += 4.0 * proj_.out_features(); }

private:
    Tensor2 table_, gate_tiles_, proj_tiles_, gram_tiles_;
    Linear gate_, proj_;
    const float* norm_ = nullptr;
    int dtype_ = BF16, column_ = 0, dim_ = 0;
    float eps_ = 1e-6f;
};

}  // namespace

void register_tanh_norm_parts() {
    register_norm("dynamic_tanh", [](const Params& p) { return std::unique_ptr<Norm>(new TanhNorm(p)); });
    register_stream_step("embedding_add", [](const Params& p) { return std::unique_ptr<StreamStep>(new EmbeddingAdd(p)); });
    register_stream_step("token_side", [](const Params& p) { return std::unique_ptr<StreamStep>(new TokenSide(p)); });
}

}  // namespace minillm
