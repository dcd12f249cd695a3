// The parts a model is put together from, natively: mixer, feed-forward, norm, block arrangement,
// and the model that runs them in the order its configuration gives.
//
// A part knows its own sizes and constants (parameters) and the tensors it owns; it does not know
// which model it is in. Parts are built by kind name through registries, from a bag of parameters
// (numbers, strings, device tensors), so that another kind of part is one class and one
// registration, and a configuration chooses layer by layer.
//
// Interfaces (`x` is the fp32 residual stream [T, hidden]; `h` a normalised activation in the
// compute dtype; `step` the batch's index arrays; `arena` memory for the step's temporaries):
//   Embedding::forward(step, position, x)     x[t,:] = the token's row (+ the position table's)
//   PositionEncoding::table() / in_mixer(qkv, heads, step)   a table for the embedding, or a turn of
//                                             queries and keys inside the mixer before keys are written
//   Norm::forward(x, rows, n) -> h            Norm::linear(x, lin, out, epilogue, rows)
//   Mixer::forward(h, step, cache, x, write)  adds the mixer's output into x
//   FeedForward::forward(h, step, x)          adds its output into x
//   Block::forward(x, step, cache, write)     runs one layer on the stream
//   Head::forward(x, final_norm, rows, logits)  fp32 logits of the wanted rows
// Every part also says what it asks of the cache (Mixer::cache_need), what scratch its kernels need
// (reserve), how much of the step's arena it takes (workspace_bytes) and what a step costs through it
// (add_cost: bytes of weights, flops).
//
// The reference's model has these pieces fixed in one class
// (/root/reference/src/model/gpt2_model.cu:275-363 block_prefill, :404-428 the head).
#pragma once

#include <functional>
#include <map>
#include <memory>
#include <string>
#include <vector>

#include "ops.h"

namespace minillm {

// Optional per-stage times of the native forward pass. With the environment variable MINI_LLM_STAGE_TIMES
// set, every step records an event behind each stage (embedding; per layer the QKV product with its norm,
// attention, output projection, first and second product of the feed-forward; final norm and head), waits
// for the step once at its end, and prints one line per stage to standard error in the reference's format
// `kind,batch_size,total_tokens,layer,stage,ms` (kind: prefill, decode or mixed)
// (/root/reference/include/profiling/stage_timer.cuh:13-101, which synchronises the device around every
// stage instead). Off: one branch per stage. A part of another kind marks its own stages with `mark`.
class StageTimes {
public:
    static StageTimes& get();
    bool enabled() const { return enabled_; }
    void begin_step(const char* kind, int batch, int tokens, hipStream_t s);
    void set_layer(int layer) { layer_ = layer; }
    void mark(const char* stage, hipStream_t s);        // the stage that ends here
    void end_step(hipStream_t s);                        // waits for the step and prints

private:
    StageTimes();
    hipEvent_t event(hipStream_t s);
    struct Mark { int layer; const char* stage; hipEvent_t at; };
    bool enabled_ = false, header_ = false;
    int layer_ = -1, batch_ = 0, tokens_ = 0;
    const char* kind_ = "";
    hipEvent_t start_ = nullptr;
    std::vector<Mark> marks_;
    std::vector<hipEvent_t> spare_;
};


// Memory for a step's temporaries: a bump allocator over one device buffer that the caller owns.
class Arena {
public:
    Arena(void* base, size_t bytes) : base_(static_cast<char*>(base)), capacity_(bytes) {}
    void* take(size_t bytes);
    Tensor2 tensor(int dtype, int64_t rows, int64_t cols) {
        return Tensor2(take(static_cast<size_t>(rows) * cols * dtype_size(dtype)), dtype, rows, cols);
    }
    size_t mark() const { return used_; }
    void release(size_t mark) { used_ = mark; }
    size_t peak() const { return peak_; }

private:
    char* base_;
    size_t capacity_, used_ = 0, peak_ = 0;
};

// The step's batch: sizes known to the host and device arrays (int32).
struct StepView {
    int n_tokens = 0, n_seqs = 0, n_logits = 0, max_q_len = 0, max_ctx_len = 0, n_single = 0;
    const int* token_ids = nullptr;    // [T]
    FedTokens fed;                     // tokens to take on the device from the step before (only if the model's embedding
                                       // says that it resolves them; otherwise token_ids holds every id already)
    const int* positions = nullptr;    // [T]
    const int* token_seq = nullptr;    // [T]
    const int* cu_q = nullptr;         // [B+1]
    const int* ctx_len = nullptr;      // [B]
    const int* starts = nullptr;       // [B]
    const int* state_slots = nullptr;  // [B]
    const int* logit_rows = nullptr;   // [n_logits]
    float* zeroed_rows = nullptr;      // fp32 [n_tokens, hidden], all zero, if a layer asked for it (Block::wants_zeroed_rows):
                                       // room for a sub-layer's result; whoever uses it leaves it zero again
    Tensor2 stream_copy;               // the stream in bfloat16 as a block is entered, if a block asked for it
                                       // (Block::wants_stream_copy): the stream itself, or the block's entry norm of it
    Tensor2 step_copy;                 // the stream in bfloat16 as a stream step is entered, if one asked for it
                                       // (StreamStep::wants_copy); another tensor than stream_copy
    // What the part that runs now is asked to leave for the part behind it (parts that can: leaves_copy): the stream's norm, or
    // the stream itself, in bfloat16, in `into` (stream_copy or step_copy).
    struct Leave {
        bool wanted = false;
        MllmTanhNorm norm{nullptr, nullptr, nullptr};      // weight null: the stream itself
        Tensor2 into;
        bool same(const Leave& o) const { return wanted == o.wanted && norm.weight == o.norm.weight && into.data == o.into.data; }
    } leave;
    int n_groups = 0;
    const int* const* block_tables = nullptr;   // per group [B, max_blocks[g]]
    const int* max_blocks = nullptr;            // per group
    const int* const* slots = nullptr;          // per group [T]
};

// What a call of the execution order sees of its cache.
struct CacheView {
    int kind = 0;                  // bits: 1 pages of keys and values, 2 fixed-size state slots (3: both)
    Tensor2 k_pages, v_pages;      // [n_pages * page_size, kv_dim]
    int group = 0, page_size = 0, window = 0;
    void* state = nullptr;         // this cache's state in slot 0; slot i lies i * slot_bytes further on
    size_t slot_bytes = 0;         // bytes between a slot and the next (the states of all caches lie side by side in a slot)
    size_t state_bytes = 0;        // bytes of a slot that are this cache's own
    int n_slots = 0;
    bool has_pages() const { return (kind & 1) != 0; }
    bool has_state() const { return (kind & 2) != 0; }
};

// What a cache of the execution order asks of the cache manager: said by the mixer that writes it.
struct CacheNeed {
    int kind = 0;                        // bits: 1 keys and values in pages, 2 fixed-size state (3: both), 0 none
    int n_kv_heads = 0, head_dim = 0, window = 0;
    int keep_first = 0;                  // with a window: the sequence's first keep_first positions are read for good
    int value_dim = -1;                  // width of a head's value rows; -1: as the keys; 0: the pages hold key rows only
    size_t state_bytes = 0;
};

// What one step costs, summed over the parts (the benchmark's roofline figures are made from these).
struct StepCost {
    double weight_bytes = 0;             // weights a step reads once, whatever its batch
    double flops_per_token = 0;          // matrix products of the layers, per token
    double attention_flops_per_key = 0;  // per (token, attended key), summed over the attention calls
    double flops_per_logits_row = 0;     // the head's product for one wanted row
};

class PositionEncoding;
class Mixer;

// A bag of parameters a part is built from.
struct Params {
    std::map<std::string, double> num;
    std::map<std::string, std::string> str;
    std::map<std::string, Tensor2> tensor;
    std::shared_ptr<const PositionEncoding> position;      // the model's position encoding, for mixers that take one
    std::vector<std::shared_ptr<const Mixer>> mixers;      // mixers that a mixer made of others runs side by side

    double number(const std::string& key) const;
    double number(const std::string& key, double fallback) const;
    int integer(const std::string& key) const { return static_cast<int>(number(key)); }
    const std::string& string(const std::string& key) const;
    const Tensor2& weights(const std::string& key) const;          // must be there
    const Tensor2* weights_or_null(const std::string& key) const;
};

class Linear {
public:
    Linear() = default;
    // weight [out, in] in the compute dtype (k contiguous: the layout the matrix kernels read), bias fp32 [out] or none
    Linear(const Tensor2& weight, const Tensor2* bias);
    void operator()(const Tensor2& a, const Tensor2& out, int epilogue, const KvScatter* kv, hipStream_t s) const {
        linear(a, weight, bias, out, epilogue, kv, s);
    }
    Tensor2 weight;
    const float* bias = nullptr;
    int in_features() const { return static_cast<int>(weight.cols); }
    int out_features() const { return static_cast<int>(weight.rows); }
    // The same with the result put where a sub-layer's belongs: into `x` by `epilogue`, or (add given) through it.
    void into(const Tensor2& a, const Tensor2& x, int epilogue, const StreamAdd* add, hipStream_t s) const {
        if (add != nullptr) linear_stream_add(a, weight, bias, *add, s);
        else linear(a, weight, bias, x, epilogue, nullptr, s);
    }
    void add_cost(StepCost& c) const {
        c.weight_bytes += static_cast<double>(weight.rows) * weight.cols * weight.esz() + (bias ? 4.0 * weight.rows : 0.0);
        c.flops_per_token += 2.0 * weight.rows * weight.cols;
    }
};

// How positions enter the model. Either a table whose row is added to the token's embedding (learned
// absolute positions: the embedding kernel adds it), or a turn of queries and keys inside the mixer,
// in place on the qkv rows, before the keys go to the pages (rotary schemes), or nothing.
class PositionEncoding {
public:
    virtual ~PositionEncoding() = default;
    virtual const Tensor2* table() const { return nullptr; }
    virtual bool applies_in_mixer() const { return false; }
    // qkv rows: n_heads query heads, then n_kv_heads key heads, then the values (left alone)
    virtual void in_mixer(const Tensor2& qkv, int n_heads, int n_kv_heads, int head_dim, const StepView& step,
                          hipStream_t s) const {
        (void)qkv; (void)n_heads; (void)n_kv_heads; (void)head_dim; (void)step; (void)s;
    }
    virtual int max_positions() const { return 0; }       // 0: unbounded
    virtual void add_cost(StepCost&) const {}
};

// Token ids to rows of the fp32 stream.
class Embedding {
public:
    virtual ~Embedding() = default;
    virtual int vocab_size() const = 0;
    virtual int hidden_size() const = 0;
    virtual void forward(const StepView& step, const PositionEncoding* position, const Tensor2& x, hipStream_t s) const = 0;
    // true: forward() takes `step.fed` into account itself (one kernel fewer in a decode step); false: the runner
    // writes the fed ids into token_ids with a kernel of its own before the step
    virtual bool resolves_fed_tokens() const { return false; }
    // true: forward() also writes step.stream_copy as step.leave asks; false: the model makes it behind it
    virtual bool writes_stream_copy() const { return false; }
    virtual void add_cost(StepCost&) const {}
};

class Norm {
public:
    virtual ~Norm() = default;
    // h[i,:] = norm(x[rows ? rows[i] : i, :]), n rows, from the arena
    virtual Tensor2 forward(const Tensor2& x, const int* rows, int n, Arena& arena, hipStream_t s) const = 0;
    // out[i,:] = norm(x[rows ? rows[i] : i, :]) into a tensor of the caller's (any activation dtype; out may be x
    // itself when rows is null and both are fp32). A norm without it refuses.
    virtual void forward_into(const Tensor2& x, const int* rows, const Tensor2& out, hipStream_t s) const;
    // For a step in which every sequence brings one token: out = h + conv(h) with h = norm(x), the convolution's
    // earlier inputs carried in the slots (StateArgs), in one kernel. False: this kind of norm has no such kernel,
    // and nothing was done.
    virtual bool conv_single(const Tensor2& x, const Tensor2& taps, const StateArgs& st, const Tensor2& out, hipStream_t s) const {
        (void)x; (void)taps; (void)st; (void)out; (void)s;
        return false;
    }
    // For the same kind of step and a norm BEHIND a sub-layer: x += norm(y) (y: the sub-layer's result, fp32) and
    // out = x + conv(x), the next sub-layer's input, in one kernel. False: no such kernel, nothing was done.
    virtual bool add_conv_single(const Tensor2& y, const Tensor2& x, const Tensor2& taps, const StateArgs& st, const Tensor2& out,
                                 hipStream_t s) const {
        (void)y; (void)x; (void)taps; (void)st; (void)out; (void)s;
        return false;
    }
    // out = epilogue(lin(norm(x[rows]))); a norm with a fused kernel overrides this
    // (kv: a key/value scatter of the linear map, passed through to it)
    virtual void linear(const Tensor2& x, const Linear& lin, const Tensor2& out, int epilogue, const int* rows,
                        const KvScatter* kv, Arena& arena, hipStream_t s) const;
    // x += mult * scale * norm(y), row by row (y and x fp32 [rows, size]; scale per column or null); with
    // `clear`, y is zero afterwards; `copy` (optional) receives the new x in bfloat16. For arrangements with a norm
    // behind a sub-layer; a norm without it refuses.
    virtual void add_scaled(const Tensor2& y, const float* scale, float mult, const Tensor2& x, bool clear,
                            hipStream_t s, const Tensor2* copy = nullptr) const;
    // True: the norm has no statistics (every value of a row on its own) and `n` is it: what makes or reads the row's
    // values can apply it in passing.
    virtual bool pointwise(MllmTanhNorm& n) const { (void)n; return false; }
    virtual size_t workspace_bytes(int rows) const = 0;
    virtual void add_cost(StepCost&) const {}
    int dtype = BF16;
};

// The input of a sub-layer as (stream, norm), not yet normalised: a part's first linear map may
// absorb the norm.
class NormedInput {
public:
    NormedInput(const Norm& norm, const Tensor2& x) : norm_(&norm), x_(x) {}
    explicit NormedInput(const Tensor2& h) : norm_(nullptr), x_(h), h_(h), have_(true) {}     // normalised already
    const Tensor2& tensor(Arena& arena, hipStream_t s);
    void linear(const Linear& lin, const Tensor2& out, int epilogue, const KvScatter* kv, Arena& arena, hipStream_t s);
    int64_t rows() const { return x_.rows; }

private:
    const Norm* norm_;
    Tensor2 x_, h_;
    bool have_ = false;
};

class Mixer {
public:
    virtual ~Mixer() = default;
    virtual void forward(NormedInput& h, const StepView& step, const CacheView& cache, const Tensor2& x, bool write,
                         Arena& arena, hipStream_t s) const = 0;
    // The same, but x is SET to the mixer's output (x need not hold anything before). A mixer whose last product can
    // store instead of add overrides this; otherwise x is cleared first.
    virtual void forward_set(NormedInput& h, const StepView& step, const CacheView& cache, const Tensor2& x, bool write,
                             Arena& arena, hipStream_t s) const {
        fill_zero(x, s);
        forward(h, step, cache, x, write, arena, s);
    }
    // The same with the output taken into the stream by `add` (a norm without statistics behind the mixer, the next
    // sub-layer's input): a mixer that ends in a product lets the product do it.
    virtual void forward_through(NormedInput& h, const StepView& step, const CacheView& cache, const StreamAdd& add, bool write,
                                 Arena& arena, hipStream_t s) const {
        forward_set(h, step, cache, add.y, write, arena, s);
        stream_add(add, nullptr, nullptr, add.copy.data == nullptr, s);
    }
    // A mixer between two products, for mixers side by side that share them: core() turns the input projection's fp32 rows
    // (`proj`, core_inputs() columns) into the rows in front of its output projection (`o`, core_outputs() columns, the
    // compute dtype). 0 inputs: the mixer has no such middle.
    virtual int core_inputs() const { return 0; }
    virtual int core_outputs() const { return 0; }
    virtual void core(const Tensor2& proj, const StepView& step, const CacheView& cache, const Tensor2& o, bool write, Arena& arena,
                      hipStream_t s) const {
        (void)proj; (void)step; (void)cache; (void)o; (void)write; (void)arena; (void)s;
        fail("this kind of mixer cannot share its products with another");
    }
    virtual size_t workspace_bytes(int tokens) const = 0;
    virtual CacheNeed cache_need() const = 0;
    // Scratch that the mixer's kernels need on stream `s` for steps of up to max_seqs sequences: taken
    // now, so that no step allocates.
    virtual void reserve(int max_seqs, hipStream_t s) const { (void)max_seqs; (void)s; }
    virtual void add_cost(StepCost&) const {}
};

class FeedForward {
public:
    virtual ~FeedForward() = default;
    virtual void forward(NormedInput& h, const StepView& step, const Tensor2& x, Arena& arena, hipStream_t s) const = 0;
    // The same, but x is SET to the result (x need not hold anything before). A feed-forward whose last product can
    // store instead of add overrides this; otherwise x is cleared first.
    virtual void forward_set(NormedInput& h, const StepView& step, const Tensor2& x, Arena& arena, hipStream_t s) const {
        fill_zero(x, s);
        forward(h, step, x, arena, s);
    }
    // The same with the result taken into the stream by `add`, as for mixers.
    virtual void forward_through(NormedInput& h, const StepView& step, const StreamAdd& add, Arena& arena, hipStream_t s) const {
        forward_set(h, step, add.y, arena, s);
        stream_add(add, nullptr, nullptr, add.copy.data == nullptr, s);
    }
    // The same in two halves, for an arrangement whose sub-layers read ONE stream: begin() does everything that reads
    // the input (the first products, with the norm inside them where the kernels allow) and leaves what it made in the
    // arena, in `pending`; finish() does the rest and adds into x, after somebody else may have changed x. What
    // begin() took from the arena must still be there when finish() runs. False from begin(): this kind has no halves,
    // and nothing was done.
    struct Pending { Tensor2 a, b, h; };
    virtual bool begin(NormedInput& h, const StepView& step, Arena& arena, hipStream_t s, Pending& pending) const {
        (void)h; (void)step; (void)arena; (void)s; (void)pending;
        return false;
    }
    virtual void finish(const Pending& pending, const StepView& step, const Tensor2& x, Arena& arena, hipStream_t s) const {
        (void)pending; (void)step; (void)x; (void)arena; (void)s;
    }
    virtual size_t workspace_bytes(int tokens) const = 0;
    virtual void reserve(int max_seqs, hipStream_t s) const { (void)max_seqs; (void)s; }
    virtual void add_cost(StepCost&) const {}
};

class Block {
public:
    virtual ~Block() = default;
    virtual void forward(const Tensor2& x, const StepView& step, const CacheView& cache, bool write, Arena& arena,
                         hipStream_t s) const = 0;
    virtual size_t workspace_bytes(int tokens) const = 0;
    virtual CacheNeed cache_need() const = 0;             // its mixer's
    // true: the model keeps one cleared fp32 buffer of the stream's shape for the step (StepView::zeroed_rows),
    // cleared once, instead of every layer clearing one of its own
    virtual bool wants_zeroed_rows() const { return false; }
    // true: the block's sub-layers read the stream itself, in bfloat16: the model keeps a copy of it for the step
    // (StepView::stream_copy), and the block leaves the copy equal to the stream it leaves
    virtual bool wants_stream_copy() const { return false; }
    // with wants_stream_copy: true and the norm if the copy is to be the block's first norm of the stream
    virtual bool entry_norm(MllmTanhNorm& n) const { (void)n; return false; }
    // true: the block leaves what StepView::leave asks for (the stream's norm, or the stream itself)
    virtual bool leaves_copy(bool normed) const { return wants_stream_copy() && !normed; }
    virtual void reserve(int max_seqs, hipStream_t s) const = 0;
    virtual void add_cost(StepCost&) const = 0;
};

// Something that happens to the whole stream between two layers (an entry of the execution order names it
// with `before` or `after`): x is the stream, x0 the embedding's output of the same step, `pass` the number the entry
// gives (a group of layers that runs several times counts its runs). A step that keeps streams of its own for the
// step (kept_streams() > 0) is handed x0 with that many more blocks of x's rows behind the embedding's output:
// room that is its own from one call to the next within a step.
class StreamStep {
public:
    virtual ~StreamStep() = default;
    virtual void forward(const Tensor2& x, const Tensor2& x0, int pass, const StepView& step, Arena& arena, hipStream_t s) const = 0;
    virtual size_t workspace_bytes(int tokens) const = 0;
    virtual bool wants_embedding_output() const { return false; }
    virtual int kept_streams() const { return 0; }         // > 0 goes with wants_embedding_output()
    virtual bool leaves_copy() const { return false; }     // true: it leaves what StepView::leave asks for
    virtual bool wants_copy() const { return false; }      // true: it reads the stream's bfloat16 copy, StepView::step_copy
    virtual void reserve(int max_seqs, hipStream_t s) const { (void)max_seqs; (void)s; }
    virtual void add_cost(StepCost&) const {}
};

// The stream's wanted rows to fp32 logits.
class Head {
public:
    virtual ~Head() = default;
    virtual int vocab_size() const = 0;
    // logits[i,:] = head(final_norm(x[rows[i],:]))
    virtual void forward(const Tensor2& x, const Norm& final_norm, const int* rows, const Tensor2& logits, Arena& arena,
                         hipStream_t s) const = 0;
    virtual size_t workspace_bytes(int rows) const = 0;
    virtual void add_cost(StepCost&) const {}
};

// -- registries: kind name -> factory ---------------------------------------------------------------
using PositionFactory = std::function<std::shared_ptr<const PositionEncoding>(const Params&)>;
using EmbeddingFactory = std::function<std::unique_ptr<Embedding>(const Params&)>;
using HeadFactory = std::function<std::unique_ptr<Head>(const Params&)>;
using NormFactory = std::function<std::unique_ptr<Norm>(const Params&)>;
using MixerFactory = std::function<std::unique_ptr<Mixer>(const Params&)>;
using FeedForwardFactory = std::function<std::unique_ptr<FeedForward>(const Params&)>;
using StreamStepFactory = std::function<std::unique_ptr<StreamStep>(const Params&)>;
// (the parameters are the arrangement's own: scales, multipliers; "pre_norm" has none)
using BlockFactory = std::function<std::unique_ptr<Block>(std::unique_ptr<Mixer>, std::unique_ptr<FeedForward>,
                                                         std::vector<std::unique_ptr<Norm>>, const Params&)>;
void register_position(const std::string& kind, PositionFactory f);
void register_embedding(const std::string& kind, EmbeddingFactory f);
void register_head(const std::string& kind, HeadFactory f);
void register_norm(const std::string& kind, NormFactory f);
void register_mixer(const std::string& kind, MixerFactory f);
void register_feed_forward(const std::string& kind, FeedForwardFactory f);
void register_block(const std::string& kind, BlockFactory f);
void register_stream_step(const std::string& kind, StreamStepFactory f);
// category: position | embedding | head | norm | mixer | feed_forward | block | stream_step
bool has_part(const std::string& category, const std::string& kind);
std::shared_ptr<const PositionEncoding> build_position(const std::string& kind, const Params& p);
std::unique_ptr<Embedding> build_embedding(const std::string& kind, const Params& p);
std::unique_ptr<Head> build_head(const std::string& kind, const Params& p);
std::unique_ptr<Norm> build_norm(const std::string& kind, const Params& p);
std::unique_ptr<Mixer> build_mixer(const std::string& kind, const Params& p);
std::unique_ptr<FeedForward> build_feed_forward(const std::string& kind, const Params& p);
std::unique_ptr<StreamStep> build_stream_step(const std::string& kind, const Params& p);
// (the feed-forward may be null: a layer without one; the norms are those of the sub-layers that exist)
std::unique_ptr<Block> build_block(const std::string& kind, std::unique_ptr<Mixer> m, std::unique_ptr<FeedForward> f,
                                   std::vector<std::unique_ptr<Norm>> norms, const Params& params = Params());
// Parts in files of their own, registered with the built-in ones: RMS norm, the arrangement with a norm on
// both sides of a sub-layer, the clamped gated feed-forward (parts_gated.cc); the Mamba-2 mixer (mamba2.cc);
// latent attention (latent_attention.cc).
void register_gated_parts();
void register_mamba2();
void register_latent_attention();
// Attention with shaped scores (scored_attention.cc); the gated linear recurrence, mixers side by side, the gated
// feed-forward with biases, the embedding with a norm, the stream step that mixes the embedding's output back in
// (recurrent_parts.cc).
void register_scored_attention();
void register_recurrent_parts();
// Linear attention with a decay, the feed-forward of routed experts, the stream step that hands on a weighted sum of
// all streams so far (linear_attention.cc); the arrangement with a norm behind each sub-layer only is registered with
// the gated parts.
void register_linear_attention_parts();
// The dynamic tanh norm, what is added to the stream between layers: the embedding's output with a vector per pass, a
// token's own gated input (tanh_norm.cc).
void register_tanh_norm_parts();
// The matrix memory with exponential gates (matrix_memory.cc).
void register_matrix_memory();

// One entry of the execution order: which layer runs, on which cache, and whether it writes it.
struct LayerCall {
    int layer = 0, cache = 0;
    bool write = true;
    int before = -1;               // >= 0: this stream step runs on the stream right before the layer
    int pass = 0;                  // handed to that stream step
    int after = -1;                // >= 0: this stream step runs on the stream right behind the layer
    int after_pass = 0;            // handed to that one
};

// A decoder-only model: the embedding (with the position encoding's table, if it has one), the calls
// of the execution order, and the final norm and the head on the wanted rows only.
class DecoderModel {
public:
    std::unique_ptr<Embedding> embedding;
    std::shared_ptr<const PositionEncoding> position;     // may be null: no position encoding
    std::vector<std::unique_ptr<Block>> layers;
    std::vector<std::unique_ptr<StreamStep>> stream_steps;
    std::vector<LayerCall> order;
    std::unique_ptr<Norm> final_norm;
    std::unique_ptr<Head> head;
    int dtype = BF16;

    int vocab_size() const { return head->vocab_size(); }
    int hidden_size() const { return embedding->hidden_size(); }
    // What each cache index of the execution order asks for: the need of the layer that writes it.
    std::vector<CacheNeed> cache_needs() const;
    // Every part takes the scratch its kernels need on `s` for steps of up to max_seqs sequences.
    void reserve(int max_seqs, hipStream_t s) const;
    StepCost cost() const;
    // Bytes of arena that a step of `tokens` tokens and `n_logits` wanted rows needs at most.
    size_t workspace_bytes(int tokens, int n_logits) const;
    // Runs the step; fp32 logits [n_logits, V] into `logits` (untouched if no logits are wanted).
    void forward(const StepView& step, const std::vector<CacheView>& caches, Arena& arena, const Tensor2& logits,
                 hipStream_t s) const;
};

}  // namespace minillm
