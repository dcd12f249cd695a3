// The matrix-memory mixer: a memory per head that an exponential input gate writes and a sigmoid forget gate keeps.
#include <algorithm>
#include <cmath>

#include "parts.h"

namespace minillm {

namespace {

const float* f32_vector(const Params& p, const char* key, int64_t n) {
    const Tensor2& t = p.weights(key);
    if (t.dtype != F32 || t.rows * t.cols != n || !t.contiguous()) fail("matrix_memory: '%s' must be contiguous float32 [%lld]", key, (long long)n);
    return static_cast<const float*>(t.data);
}

// The mLSTM recurrence (equations in kernels/matrix_memory.hip): per head, with q = dim^(-1/2) W_q h, k = W_k h, v = W_v h and
// log gates i = cap tanh((W_i h + b_i) / cap), f = log sigmoid(cap tanh((W_f h + b_f) / cap)),
//   S <- exp(f) S + exp(i) k v^T,  n <- exp(f) n + exp(i) k,  o = S^T q / max(|n . q|, 1)
// kept in range by a running maximum that starts at 0. Every head's o is divided by its root mean square, multiplied by
// norm.weight and by sigmoid(W_g h), and W_o of the concatenated heads goes into the stream. One joined input projection with
// fp32 results, rows [q: heads * dim | k: heads * dim | v: heads * value_dim | g: heads * value_dim | i: heads | f: heads].
// State, gates, sums, norm and output gate are fp32 in both precisions; the two projections run in the compute dtype.
// Parameters: heads, dim, value_dim, gate_cap, eps, dtype; tensors in.weight, i.bias, f.bias, norm.weight, out.weight.
class MatrixMemory final : public Mixer {
public:
    explicit MatrixMemory(const Params& p) {
        sh_.heads = p.integer("heads"); sh_.dim = p.integer("dim"); sh_.value_dim = p.integer("value_dim");
        sh_.cap = static_cast<float>(p.number("gate_cap"));
        sh_.eps = static_cast<float>(p.number("eps"));
        dtype_ = p.integer("dtype");
        const int H = sh_.heads, d = sh_.dim, e = sh_.value_dim;
        if (H < 1 || d < 1 || e < 1 || !(sh_.cap > 0.f)) fail("matrix_memory: heads, sizes and gate_cap must be positive");
        sh_.q_scale = static_cast<float>(1.0 / std::sqrt(static_cast<double>(d)));
        sh_.k_col = H * d; sh_.v_col = 2 * H * d; sh_.g_col = sh_.v_col + H * e; sh_.i_col = sh_.g_col + H * e; sh_.f_col = sh_.i_col + H;
        in_ = Linear(p.weights("in.weight"), nullptr);
        out_ = Linear(p.weights("out.weight"), nullptr);
        if (in_.out_features() != sh_.f_col + H || out_.in_features() != H * e)
            fail("matrix_memory: the projections' shapes do not fit %d heads of %d / %d", H, d, e);
        sh_.i_bias = f32_vector(p, "i.bias", H);
        sh_.f_bias = f32_vector(p, "f.bias", H);
        sh_.norm = f32_vector(p, "norm.weight", static_cast<int64_t>(H) * e);
    }
    void forward(NormedInput& h, const StepView& step, const CacheView& cache, const Tensor2& x, bool write, Arena& arena,
                 hipStream_t s) const override {
        run(h, step, cache, x, write, arena, s, ADD_RESIDUAL);
    }
    void forward_set(NormedInput& h, const StepView& step, const CacheView& cache, const Tensor2& x, bool write, Arena& arena,
                     hipStream_t s) const override {
        run(h, step, cache, x, write, arena, s, STORE_F32);
    }
    void run(NormedInput& h, const StepView& step, const CacheView& cache, const Tensor2& x, bool write, Arena& arena, hipStream_t s,
             int out_epilogue) const {
        if (!cache.has_state() || cache.state_bytes < state_floats() * 4) fail("matrix_memory needs a state of %zu floats per request", state_floats());
        const int T = step.n_tokens, N = in_.out_features(), ld = (N + 3) / 4 * 4, inner = sh_.heads * sh_.value_dim;
        const Tensor2 proj(arena.take(static_cast<size_t>(T) * ld * 4), F32, T, N, ld);
        h.linear(in_, proj, STORE_F32, nullptr, arena, s);
        StageTimes::get().mark("in_proj", s);
        StateArgs st;
        st.token_seq = step.token_seq; st.cu_q = step.cu_q; st.state_slots = step.state_slots; st.n_seqs = step.n_seqs;
        st.max_q_len = step.max_q_len; st.n_single = step.n_single; st.state = static_cast<float*>(cache.state);
        st.slot_floats = cache.slot_bytes / 4; st.n_slots = cache.n_slots; st.write = write;
        const size_t ws_floats = matrix_memory_workspace_floats(T, step.n_seqs, sh_.heads, sh_.dim, sh_.value_dim);
        float* ws = static_cast<float*>(arena.take(ws_floats * 4));
        const Tensor2 o = arena.tensor(dtype_, T, inner), y = arena.tensor(F32, T, inner);
        matrix_memory(proj, sh_, st, o, y, ws, ws_floats, s);
        StageTimes::get().mark("memory", s);
        out_(o, x, out_epilogue, nullptr, s);
        StageTimes::get().mark("out_proj", s);
    }
    size_t workspace_bytes(int tokens) const override {
        return static_cast<size_t>(tokens) * ((in_.out_features() + 4) * 4 + sh_.heads * sh_.value_dim * (4 + dtype_size(dtype_)) + in_.in_features() * dtype_size(dtype_)) +
               // (every sequence of a step adds at most one chunk that is not full; a step holds at most as many
               // sequences as tokens)
               matrix_memory_workspace_floats(tokens, std::min(tokens, 256), sh_.heads, sh_.dim, sh_.value_dim) * 4 + 8192;
    }
    CacheNeed cache_need() const override {
        CacheNeed n;
        n.kind = 2;
        n.state_bytes = (state_floats() + 3) / 4 * 4 * 4;          // (whole 16-byte pieces: what lies behind in the slot stays aligned)
        return n;
    }
    void reserve(int, hipStream_t s) const override { reserve_linear_scratch(s); }
    void add_cost(StepCost& c) const override {
        in_.add_cost(c);
        out_.add_cost(c);
        c.weight_bytes += 4.0 * sh_.heads * (sh_.value_dim + 2);
        c.flops_per_token += 4.0 * sh_.heads * sh_.dim * (sh_.value_dim + 1);        // the memory's update and readout
    }

private:
    size_t state_floats() const { return matrix_memory_state_floats(sh_.heads, sh_.dim, sh_.value_dim); }
    MemoryShape sh_;
    int dtype_ = BF16;
    Linear in_, out_;
};

}  // namespace

void register_matrix_memory() {
    register_mixer("matrix_memory", [](const Params& p) { return std::unique_ptr<Mixer>(new MatrixMemory(p)); });
}

}  // namespace minillm
