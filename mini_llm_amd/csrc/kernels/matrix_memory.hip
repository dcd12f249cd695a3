// A matrix memory per head with an exponential input gate and a sigmoid forget gate (the mLSTM recurrence), for gfx950.
// Per head with d key and e value columns, token by token, in logarithms:
//   i = cap tanh((i_raw + i_bias) / cap),   f = log sigmoid(cap tanh((f_raw + f_bias) / cap))
//   m' = max(f + m, i);  S <- exp(f + m - m') S + exp(i - m') k v^T;  n <- exp(f + m - m') n + exp(i - m') k;  m <- m'
//   o = S^T q / (max(|n . q|, exp(-m)) + 1e-6)
// from S = 0, n = 0, m = 0. Each head's o is then divided by its root mean square (eps inside), multiplied by a weight per
// column and by sigmoid of a raw gate, and stored in the compute dtype. Inputs are the fp32 rows of a joined input
// projection; gates, memories, sums, norm and output gate are fp32 in both precisions, and so are the products below
// (v_mfma_f32_16x16x4_f32).
//
// Single tokens: one workgroup per (sequence, head) (memory_single_kernel) does all of it; a head whose memory is large
// is shared by one workgroup per 64 value columns, and the norm is a kernel of its own then. For that the state holds
// one copy of n and m per workgroup that works on a head ("copies"), so that none reads what another writes.
//
// Portions: chunks of MM_CHUNK tokens side by side, in three launches. With F_t the sum of a chunk's f up to token t
// and u_t = i_t - F_t, everything inside a chunk is exp(u_s - r_t) with r_t = max(m, max_(s <= t) u_s), m the running
// maximum the chunk starts from (m_t = r_t + F_t):
//   memory_chunk_kernel    the chunk's own memory from zero, L = sum_t exp(u_t - U) k_t v_t^T, U = max_t u_t
//   memory_states_kernel   a sequence's chunks in order, S <- exp(m - M) S + exp(U - M) L with M = max(m, U), m <- M + F;
//                          leaves what every chunk starts from, and the last memory in the slot
//   memory_output_kernel   O_t = exp(m - r_t) S^T q_t + sum_(s <= t) exp(u_s - r_t) (q_t . k_s) v_s, the same for n, norm, gate
// F and u are double (64 log gates of up to `cap` each are summed, then subtracted from one another), rounded behind
// the subtraction.
//
// State of a request: S [H][d][e], then n [H][copies][d], then m [H][copies], fp32.
//
// The same kernels run retention (head_decay given): S <- decay_h S + k v^T, o = S^T q, no normaliser. With i = 0 and f = log
// decay_h every u_s = -F_s grows with s, so that r_t = -F_t, the weights inside a chunk are decay^(t - s), the carried memory's
// decay^(t + 1), and m stays 0; n and m are then neither kept nor read (the state is S alone) and nothing is divided.
#include "common.h"

#define MM_CHUNK 64
#define MM_STRIDE 68          // floats between rows of a 64-wide tile in LDS: conflict-free for the reads below

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));

struct MemoryArgs {
    const float* proj;                 // [T, ld]
    int ld, q_col, k_col, v_col, g_col, i_col, f_col;
    const float* i_bias;
    const float* f_bias;
    const float* norm_w;               // [H * e]
    float cap, q_scale, eps;
    const float* head_decay;           // [H]: retention with these decays; null: gates from the rows
    int silu;                          // the output gate is silu(raw) instead of sigmoid(raw)
    const int* cu_q;
    const int* state_slots;
    float* state;
    size_t slot_floats;
    int H, d, e, copies, write;
};

__device__ __forceinline__ float mm_sigmoid(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float mm_log_input(float raw, float bias, float cap) { return cap * tanhf((raw + bias) / cap); }
__device__ __forceinline__ float mm_log_forget(float raw, float bias, float cap) {
    const float z = cap * tanhf((raw + bias) / cap);
    return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}

__device__ __forceinline__ float mm_gate(const MemoryArgs& a, float z) { return (a.silu ? z : 1.f) * mm_sigmoid(z); }
__device__ __forceinline__ float mm_norm_weight(const MemoryArgs& a, int col) { return a.norm_w != nullptr ? a.norm_w[col] : 1.f; }

// Where a chunk's or a request's numbers lie.
__device__ __forceinline__ size_t state_n_at(const MemoryArgs& a, int h, int copy) {
    return static_cast<size_t>(a.H) * a.d * a.e + (static_cast<size_t>(h) * a.copies + copy) * a.d;
}
__device__ __forceinline__ size_t state_m_at(const MemoryArgs& a, int h, int copy) {
    return static_cast<size_t>(a.H) * a.d * a.e + static_cast<size_t>(a.H) * a.copies * a.d + static_cast<size_t>(h) * a.copies + copy;
}
// workspace per (chunk, head): the memory [d * e], n [d], then [log scale of the chunk's own memory, sum of its f, the
// request's m in front of the step (a sequence's first chunk only), the m this chunk starts from], and behind that, as
// doubles, u, its running maximum and F for the chunk's tokens
__host__ __device__ __forceinline__ size_t chunk_gates_at(int d, int e) { return (static_cast<size_t>(d) * e + d + 4 + 3) / 4 * 4; }
__host__ __device__ __forceinline__ size_t chunk_floats(int d, int e) { return chunk_gates_at(d, e) + 3 * 2 * MM_CHUNK; }
__device__ __forceinline__ size_t chunk_scalars_at(int d, int e) { return static_cast<size_t>(d) * e + d; }

// Which sequence (from first_seq on) and which of its chunks is number w, and the sequence's state slot: a wavefront looks
// at 64 sequences at a time. False: there are fewer chunks.
__device__ __forceinline__ bool find_chunk(const int* __restrict__ cu_q, const int* __restrict__ state_slots, int first_seq, int n_seqs, int w,
                                           int& slot, int& chunk, int& first, int& n) {
    const int lane = threadIdx.x % MLLM_WAVE;
    for (int b0 = first_seq; b0 < n_seqs; b0 += MLLM_WAVE) {
        const int mine = min(b0 + lane, n_seqs - 1);
        const int begin = cu_q[mine], len = cu_q[mine + 1] - begin, its_slot = state_slots[mine];
        const int nc = b0 + lane < n_seqs ? (len + MM_CHUNK - 1) / MM_CHUNK : 0;
        int upto = nc;
#pragma unroll
        for (int off = 1; off < MLLM_WAVE; off *= 2) {
            const int other = __shfl_up(upto, off, MLLM_WAVE);
            if (lane >= off) upto += other;
        }
        const unsigned long long here = __ballot(w < upto);
        if (here != 0) {
            const int l = __ffsll(here) - 1;
            slot = __builtin_amdgcn_readfirstlane(__shfl(its_slot, l, MLLM_WAVE));
            chunk = w - (__shfl(upto, l, MLLM_WAVE) - __shfl(nc, l, MLLM_WAVE));
            first = __shfl(begin, l, MLLM_WAVE) + chunk * MM_CHUNK;
            n = min(MM_CHUNK, __shfl(len, l, MLLM_WAVE) - chunk * MM_CHUNK);
            chunk = __builtin_amdgcn_readfirstlane(chunk);
            first = __builtin_amdgcn_readfirstlane(first);
            n = __builtin_amdgcn_readfirstlane(n);
            return true;
        }
        w -= __shfl(upto, MLLM_WAVE - 1, MLLM_WAVE);
    }
    return false;
}

// The gates of a chunk's tokens, token t in lane t: F_t and u_t = i_t - F_t (tokens beyond n: F stays, u = -inf).
__device__ __forceinline__ void chunk_gates(const MemoryArgs& a, int h, int first, int n, int lane, double& F, double& u) {
    if (a.head_decay != nullptr) {
        const int upto = min(lane + 1, n);
        F = upto * log(static_cast<double>(a.head_decay[h]));
        u = lane < n ? -F : -INFINITY;
        return;
    }
    const float* row = a.proj + static_cast<size_t>(first + min(lane, n - 1)) * a.ld;
    const float iz = row[a.i_col + h], fz = row[a.f_col + h];
    const float ig = mm_log_input(iz, a.i_bias[h], a.cap);
    F = lane < n ? static_cast<double>(mm_log_forget(fz, a.f_bias[h], a.cap)) : 0.0;
#pragma unroll
    for (int off = 1; off < MLLM_WAVE; off *= 2) {
        const double other = __shfl_up(F, off, MLLM_WAVE);
        if (lane >= off) F += other;
    }
    u = lane < n ? static_cast<double>(ig) - F : -INFINITY;
}
__device__ __forceinline__ double wave_prefix_max(double v, int lane) {
#pragma unroll
    for (int off = 1; off < MLLM_WAVE; off *= 2) {
        const double other = __shfl_up(v, off, MLLM_WAVE);
        if (lane >= off) v = fmax(v, other);
    }
    return v;
}

// A tile of 64 rows x 64 columns of which `rows` x `cols` exist (the rest reads as zero): 16 values a thread of 256, all
// loads without conditions, from clamped places. VEC: 16-byte loads (cols and every row's start are multiples of 4).
template <bool VEC>
__device__ __forceinline__ void tile_load(float (&v)[16], const float* __restrict__ src, size_t row_stride, int rows, int cols) {
    const int tid = threadIdx.x;
    if (VEC) {
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int idx = tid + 256 * u, r = min(idx / 16, rows - 1), c = min(4 * (idx % 16), cols - 4);
            const float4 x = *reinterpret_cast<const float4*>(src + r * row_stride + c);
            v[4 * u] = x.x; v[4 * u + 1] = x.y; v[4 * u + 2] = x.z; v[4 * u + 3] = x.w;
        }
    } else {
#pragma unroll
        for (int u = 0; u < 16; ++u) {
            const int idx = tid + 256 * u, r = min(idx / 64, rows - 1), c = min(idx % 64, cols - 1);
            v[u] = src[r * row_stride + c];
        }
    }
}
// The tile to LDS ([64][MM_STRIDE]), times `scale` and, with `by_row`, times by_row[row].
template <bool VEC>
__device__ __forceinline__ void tile_store(float* lds, const float (&v)[16], int rows, int cols, float scale, const float* by_row = nullptr) {
    const int tid = threadIdx.x;
    if (VEC) {
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int idx = tid + 256 * u, r = idx / 16, c = 4 * (idx % 16);
            const bool ok = r < rows && c < cols;
            const float s = by_row != nullptr ? scale * by_row[r] : scale;
            *reinterpret_cast<float4*>(lds + r * MM_STRIDE + c) =
                ok ? make_float4(v[4 * u] * s, v[4 * u + 1] * s, v[4 * u + 2] * s, v[4 * u + 3] * s) : make_float4(0.f, 0.f, 0.f, 0.f);
        }
    } else {
#pragma unroll
        for (int u = 0; u < 16; ++u) {
            const int idx = tid + 256 * u, r = idx / 64, c = idx % 64;
            const float s = by_row != nullptr ? scale * by_row[r] : scale;
            lds[r * MM_STRIDE + c] = (r < rows && c < cols) ? v[u] * s : 0.f;
        }
    }
}

// A lane's operand of a product over 64 key columns, straight from memory: columns 16 kk + 4 G .. + 3 of one row, kk < 4, of
// which the first `cols` exist (the rest becomes zero in query_finish). Loads without conditions.
template <bool VEC>
__device__ __forceinline__ void query_load(float4 (&q4)[4], const float* __restrict__ row, int cols, int G) {
#pragma unroll
    for (int kk = 0; kk < 4; ++kk) {
        const int col = 16 * kk + 4 * G;
        if (VEC) q4[kk] = *reinterpret_cast<const float4*>(row + min(col, cols - 4));
        else q4[kk] = make_float4(row[min(col, cols - 1)], row[min(col + 1, cols - 1)], row[min(col + 2, cols - 1)], row[min(col + 3, cols - 1)]);
    }
}
__device__ __forceinline__ void query_finish(float4 (&q4)[4], float scale, int cols, int G) {
#pragma unroll
    for (int kk = 0; kk < 4; ++kk) {
        const int col = 16 * kk + 4 * G;
        q4[kk].x = col < cols ? q4[kk].x * scale : 0.f;
        q4[kk].y = col + 1 < cols ? q4[kk].y * scale : 0.f;
        q4[kk].z = col + 2 < cols ? q4[kk].z * scale : 0.f;
        q4[kk].w = col + 3 < cols ? q4[kk].w * scale : 0.f;
    }
}

// A chunk's own memory, 64 x 64 of it a workgroup: grid (chunks, heads, key tiles * value tiles). Four wavefronts of 16
// key columns each; the products' inner dimension is the chunk's tokens.
template <bool VEC>
__global__ void __launch_bounds__(256)
memory_chunk_kernel(MemoryArgs a, int first_seq, int n_seqs, int value_tiles, float* __restrict__ ws) {
    __shared__ __attribute__((aligned(16))) float Ks[MM_CHUNK * MM_STRIDE];
    __shared__ __attribute__((aligned(16))) float Vs[MM_CHUNK * MM_STRIDE];
    __shared__ float weight[MM_CHUNK];
    int slot, chunk, first, n;
    if (!find_chunk(a.cu_q, a.state_slots, first_seq, n_seqs, blockIdx.x, slot, chunk, first, n) || slot < 0) return;
    const int h = blockIdx.y, kt = blockIdx.z / value_tiles, vt = blockIdx.z % value_tiles;
    const int tid = threadIdx.x, lane = tid % MLLM_WAVE, wave = __builtin_amdgcn_readfirstlane(tid / MLLM_WAVE);
    const int kc = min(64, a.d - 64 * kt), vc = min(64, a.e - 64 * vt);
    float kv[16], vv[16];
    tile_load<VEC>(kv, a.proj + static_cast<size_t>(first) * a.ld + a.k_col + h * a.d + 64 * kt, a.ld, n, kc);
    tile_load<VEC>(vv, a.proj + static_cast<size_t>(first) * a.ld + a.v_col + h * a.e + 64 * vt, a.ld, n, vc);
    float* W = ws + (static_cast<size_t>(blockIdx.x) * a.H + h) * chunk_floats(a.d, a.e);
    if (wave == 0) {
        double F, u;
        chunk_gates(a, h, first, n, lane, F, u);
        const double upto = wave_prefix_max(u, lane), U = __shfl(upto, MLLM_WAVE - 1, MLLM_WAVE);
        weight[lane] = expf(static_cast<float>(u - U));
        if (kt == 0 && vt == 0) {
            double* gates = reinterpret_cast<double*>(W + chunk_gates_at(a.d, a.e));
            gates[lane] = u;
            gates[MM_CHUNK + lane] = upto;
            gates[2 * MM_CHUNK + lane] = F;
            if (lane == MLLM_WAVE - 1) {
                float* sc = W + chunk_scalars_at(a.d, a.e);
                sc[0] = static_cast<float>(U + F);
                sc[1] = static_cast<float>(F);
                if (chunk == 0) sc[2] = a.head_decay != nullptr ? 0.f : a.state[static_cast<size_t>(slot) * a.slot_floats + state_m_at(a, h, 0)];
            }
        }
    }
    lds_barrier();
    tile_store<VEC>(Ks, kv, n, kc, 1.f, weight);
    tile_store<VEC>(Vs, vv, n, vc, 1.f);
    lds_barrier();
    const int G = lane / 16, c = lane % 16;
    f32x4 acc[4];
#pragma unroll
    for (int t = 0; t < 4; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    float key_sum = 0.f;                              // of key column 16 wave + c, over this lane group's tokens
#pragma unroll
    for (int j = 0; j < 16; ++j) {
        // (which of the 64 tokens a lane group's slot of step j stands for is free, as long as both operands agree;
        // groups four rows apart read conflict-free)
        const int t = (j / 4) * 16 + 4 * G + j % 4;
        const float av = Ks[t * MM_STRIDE + 16 * wave + c];
        key_sum += av;
#pragma unroll
        for (int ct = 0; ct < 4; ++ct) acc[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(av, Vs[t * MM_STRIDE + 16 * ct + c], acc[ct], 0, 0, 0);
    }
#pragma unroll
    for (int ct = 0; ct < 4; ++ct)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int i = 16 * wave + 4 * G + r, col = 16 * ct + c;
            if (i < kc && col < vc) W[static_cast<size_t>(64 * kt + i) * a.e + 64 * vt + col] = acc[ct][r];
        }
    key_sum = rows_sum(key_sum);
    if (vt == 0 && G == 0 && 16 * wave + c < kc) W[static_cast<size_t>(a.d) * a.e + 64 * kt + 16 * wave + c] = key_sum;
}

// One thread per cell of a head's memory and normaliser: grid (cells of all heads / 256, sequences). In the workspace a
// chunk's own memory is replaced by the one it starts from.
__global__ void __launch_bounds__(256)
memory_states_kernel(MemoryArgs a, int first_seq, float* __restrict__ ws) {
    const int b = first_seq + blockIdx.y, lane = threadIdx.x % MLLM_WAVE;
    const int slot = a.state_slots[b];
    if (slot < 0) return;
    int before = 0;                                   // chunks of the sequences in front of this one
    for (int bb = first_seq + lane; bb < b; bb += MLLM_WAVE) before += (a.cu_q[bb + 1] - a.cu_q[bb] + MM_CHUNK - 1) / MM_CHUNK;
#pragma unroll
    for (int off = 32; off > 0; off /= 2) before += __shfl_xor(before, off, MLLM_WAVE);
    const int nc = (a.cu_q[b + 1] - a.cu_q[b] + MM_CHUNK - 1) / MM_CHUNK;
    const long long per_head = static_cast<long long>(a.d) * a.e + (a.head_decay != nullptr ? 0 : a.d);
    const long long idx = static_cast<long long>(blockIdx.x) * 256 + threadIdx.x;
    if (idx >= per_head * a.H || nc == 0) return;
    const int h = static_cast<int>(idx / per_head);
    const long long r = idx % per_head;
    const bool is_n = r >= static_cast<long long>(a.d) * a.e;
    const int i = static_cast<int>(r - static_cast<long long>(a.d) * a.e);      // (of the normaliser)
    float* base = a.state + static_cast<size_t>(slot) * a.slot_floats;
    float* cell = is_n ? base + state_n_at(a, h, 0) + i : base + static_cast<size_t>(h) * a.d * a.e + r;
    const size_t per_chunk = static_cast<size_t>(a.H) * chunk_floats(a.d, a.e);
    float* W = ws + (static_cast<size_t>(before) * a.H + h) * chunk_floats(a.d, a.e);
    const size_t sc = chunk_scalars_at(a.d, a.e);
    float S = *cell, m = W[sc + 2];
    constexpr int AHEAD = 16;                          // chunks whose values are asked for together
    for (int c0 = 0; c0 < nc; c0 += AHEAD) {
        float L[AHEAD], scale[AHEAD], sum_f[AHEAD];
#pragma unroll
        for (int k = 0; k < AHEAD; ++k) {
            const float* w = W + static_cast<size_t>(min(c0 + k, nc - 1)) * per_chunk;
            L[k] = w[r];
            scale[k] = w[sc];
            sum_f[k] = w[sc + 1];
        }
#pragma unroll
        for (int k = 0; k < AHEAD; ++k) {
            if (c0 + k < nc) {
                float* w = W + static_cast<size_t>(c0 + k) * per_chunk;
                w[r] = S;
                if (r == 0) w[sc + 3] = m;
                const float kept = sum_f[k] + m, next = fmaxf(kept, scale[k]);
                S = expf(kept - next) * S + expf(scale[k] - next) * L[k];
                m = next;
            }
        }
    }
    if (!a.write) return;
    *cell = S;
    if (is_n) {
        for (int copy = 1; copy < a.copies; ++copy) base[state_n_at(a, h, copy) + i] = S;
        if (i == 0)
            for (int copy = 0; copy < a.copies; ++copy) base[state_m_at(a, h, copy)] = m;
    }
}

// Outputs of a chunk, one workgroup per (chunk, head, group of NT value tiles): four wavefronts of 16 tokens each.
// FUSED: the head's columns all lie in this workgroup, so norm and gate are done here and `out` is the compute dtype;
// otherwise o goes to y (fp32 [T, H * e]) and a norm kernel follows.
template <typename T, int NT, bool VEC, bool FUSED>
__global__ void __launch_bounds__(256)
memory_output_kernel(MemoryArgs a, int first_seq, int n_seqs, const float* __restrict__ ws, T* __restrict__ out, int ldo, float* __restrict__ y,
                     int ldy) {
    __shared__ __attribute__((aligned(16))) float Ks[MM_CHUNK * MM_STRIDE];       // keys; the weighted scores; the results
    __shared__ __attribute__((aligned(16))) float Bs[MM_CHUNK * MM_STRIDE];       // a tile of the starting memory, then of the values
    __shared__ double u_s[MM_CHUNK], r_s[MM_CHUNK];
    __shared__ float nq_s[MM_CHUNK], start_s[MM_CHUNK], floor_s[MM_CHUNK];
    __shared__ __attribute__((aligned(16))) float n_s[64];
    int slot, chunk, first, n;
    if (!find_chunk(a.cu_q, a.state_slots, first_seq, n_seqs, blockIdx.x, slot, chunk, first, n) || slot < 0) return;
    const int h = blockIdx.y, vt0 = blockIdx.z * NT;
    const int tid = threadIdx.x, lane = tid % MLLM_WAVE, wave = __builtin_amdgcn_readfirstlane(tid / MLLM_WAVE);
    const int G = lane / 16, c = lane % 16;
    const float* rows = a.proj + static_cast<size_t>(first) * a.ld;
    const float* W = ws + (static_cast<size_t>(blockIdx.x) * a.H + h) * chunk_floats(a.d, a.e);
    const int value_tiles = min(NT, (a.e + 63) / 64 - vt0);
    f32x4 p[4], o[NT][4];
#pragma unroll
    for (int t = 0; t < 4; ++t) p[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int ct = 0; ct < 4; ++ct) o[t][ct] = f32x4{0.f, 0.f, 0.f, 0.f};
    float nq = 0.f;                                  // this lane's share of q_t . n, t = 16 wave + c
    float vv[16];                                    // the first tile of values: asked for now, used behind the scores
    const int key_tiles = (a.d + 63) / 64;
    for (int kt = 0; kt < key_tiles; ++kt) {
        const int kc = min(64, a.d - 64 * kt);
        float kv[16], sv[16];
        float4 q4[4];                                // this lane's queries: token 16 wave + c, key columns 16 kk + 4 G ..
        query_load<VEC>(q4, rows + static_cast<size_t>(min(16 * wave + c, n - 1)) * a.ld + a.q_col + h * a.d + 64 * kt, kc, G);
        tile_load<VEC>(kv, rows + a.k_col + h * a.d + 64 * kt, a.ld, n, kc);
        tile_load<VEC>(sv, W + static_cast<size_t>(64 * kt) * a.e + 64 * vt0, a.e, kc, min(64, a.e - 64 * vt0));
        const float nv = W[static_cast<size_t>(a.d) * a.e + 64 * kt + min(tid, kc - 1)];
        if (kt == key_tiles - 1) tile_load<VEC>(vv, rows + a.v_col + h * a.e + 64 * vt0, a.ld, n, min(64, a.e - 64 * vt0));
        if (kt == 0 && wave == 0) {
            const double* gates = reinterpret_cast<const double*>(W + chunk_gates_at(a.d, a.e));
            const double u = gates[lane], upto = gates[MM_CHUNK + lane], F = gates[2 * MM_CHUNK + lane];
            const float m = W[chunk_scalars_at(a.d, a.e) + 3];
            const double r = fmax(upto, static_cast<double>(m));
            u_s[lane] = u;
            r_s[lane] = r;
            start_s[lane] = expf(static_cast<float>(static_cast<double>(m) - r));
            floor_s[lane] = expf(-static_cast<float>(r + F));
        }
        if (kt > 0) lds_barrier();                   // the tiles before are used up
        tile_store<VEC>(Ks, kv, n, kc, 1.f);
        tile_store<VEC>(Bs, sv, kc, min(64, a.e - 64 * vt0), 1.f);
        if (tid < 64) n_s[tid] = tid < kc ? nv : 0.f;
        query_finish(q4, 16 * wave + c < n ? a.q_scale : 0.f, kc, G);
        lds_barrier();
        // (a lane's float4 holds its operand for four steps: which key columns a step's slots stand for is free as long
        // as both operands agree)
#pragma unroll
        for (int kk = 0; kk < 4; ++kk) {
            const float4 q = q4[kk];
            const float4 n4 = *reinterpret_cast<const float4*>(n_s + 16 * kk + 4 * G);
            nq += (q.x * n4.x + q.y * n4.y) + (q.z * n4.z + q.w * n4.w);
#pragma unroll
            for (int ct = 0; ct < 4; ++ct) {
                const float4 k4 = *reinterpret_cast<const float4*>(Ks + (16 * ct + c) * MM_STRIDE + 16 * kk + 4 * G);
                p[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(q.x, k4.x, p[ct], 0, 0, 0);
                p[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(q.y, k4.y, p[ct], 0, 0, 0);
                p[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(q.z, k4.z, p[ct], 0, 0, 0);
                p[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(q.w, k4.w, p[ct], 0, 0, 0);
            }
        }
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            if (t > 0) {
                if (t >= value_tiles) break;
                tile_load<VEC>(sv, W + static_cast<size_t>(64 * kt) * a.e + 64 * (vt0 + t), a.e, kc, min(64, a.e - 64 * (vt0 + t)));
                lds_barrier();
                tile_store<VEC>(Bs, sv, kc, min(64, a.e - 64 * (vt0 + t)), 1.f);
                lds_barrier();
            }
#pragma unroll
            for (int kk = 0; kk < 4; ++kk) {
                const float qj[4] = {q4[kk].x, q4[kk].y, q4[kk].z, q4[kk].w};
#pragma unroll
                for (int j = 0; j < 4; ++j)
#pragma unroll
                    for (int ct = 0; ct < 4; ++ct)
                        o[t][ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(qj[j], Bs[(16 * kk + 4 * G + j) * MM_STRIDE + 16 * ct + c], o[t][ct], 0, 0, 0);
            }
        }
    }
    nq = rows_sum(nq);                               // the four lane groups' shares
    if (G == 0) nq_s[16 * wave + c] = nq;
    lds_barrier();                                   // keys and memory tiles are used up; nq_s is complete
    tile_store<VEC>(Bs, vv, n, min(64, a.e - 64 * vt0), 1.f);
    // p[ct][r] is q_t . k_s of t = 16 wave + 4 G + r, s = 16 ct + c: weighted, into this wavefront's rows of Ks
    float* Ps = Ks + 16 * wave * MM_STRIDE;
    float den[4], start[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int t = 16 * wave + 4 * G + r;
        const double rt = r_s[t];
        float sum = 0.f;
#pragma unroll
        for (int ct = 0; ct < 4; ++ct) {
            const int s = 16 * ct + c;
            const float wgt = (s <= t && s < n) ? expf(static_cast<float>(u_s[s] - rt)) : 0.f;
            const float x = wgt * p[ct][r];
            sum += x;
            Ps[(4 * G + r) * MM_STRIDE + s] = x;
        }
        start[r] = start_s[t];
        den[r] = a.head_decay != nullptr ? 1.f : 1.f / (fmaxf(fabsf(group_sum<16>(sum) + start[r] * nq_s[t]), floor_s[t]) + 1e-6f);
    }
    lds_barrier();
    float ss[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < NT; ++t) {
        if (t >= value_tiles) break;
        if (t > 0) {
            tile_load<VEC>(vv, rows + a.v_col + h * a.e + 64 * (vt0 + t), a.ld, n, min(64, a.e - 64 * (vt0 + t)));
            lds_barrier();
            tile_store<VEC>(Bs, vv, n, min(64, a.e - 64 * (vt0 + t)), 1.f);
            lds_barrier();
        }
#pragma unroll
        for (int ct = 0; ct < 4; ++ct)
#pragma unroll
            for (int r = 0; r < 4; ++r) o[t][ct][r] *= start[r];
#pragma unroll
        for (int kk = 0; kk < 4; ++kk) {
            const float4 p4 = *reinterpret_cast<const float4*>(Ps + c * MM_STRIDE + 16 * kk + 4 * G);
            const float pj[4] = {p4.x, p4.y, p4.z, p4.w};
#pragma unroll
            for (int j = 0; j < 4; ++j)
#pragma unroll
                for (int ct = 0; ct < 4; ++ct)
                    o[t][ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(pj[j], Bs[(16 * kk + 4 * G + j) * MM_STRIDE + 16 * ct + c], o[t][ct], 0, 0, 0);
        }
#pragma unroll
        for (int ct = 0; ct < 4; ++ct)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                o[t][ct][r] *= den[r];
                ss[r] += o[t][ct][r] * o[t][ct][r];      // (columns beyond the head's are zero)
            }
    }
    // (what the end reads from memory is asked for before the sums over the wavefront)
    float4 gate4[4], norm4;
    if (VEC && FUSED) {
        const int col = h * a.e + 64 * vt0 + min(4 * c, min(64, a.e - 64 * vt0) - 4);
        norm4 = a.norm_w != nullptr ? *reinterpret_cast<const float4*>(a.norm_w + col) : make_float4(1.f, 1.f, 1.f, 1.f);
#pragma unroll
        for (int u = 0; u < 4; ++u)
            gate4[u] = *reinterpret_cast<const float4*>(rows + static_cast<size_t>(min(16 * wave + 4 * u + G, n - 1)) * a.ld + a.g_col + col);
    }
    float inv[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) inv[r] = FUSED ? 1.f / sqrtf(group_sum<16>(ss[r]) / static_cast<float>(a.e) + a.eps) : 1.f;
    // the results pass through this wavefront's rows of Ks, so that a store covers whole rows
#pragma unroll
    for (int t = 0; t < NT; ++t) {
        if (t >= value_tiles) break;
        wave_lds_sync();
#pragma unroll
        for (int ct = 0; ct < 4; ++ct)
#pragma unroll
            for (int r = 0; r < 4; ++r) Ps[(4 * G + r) * MM_STRIDE + 16 * ct + c] = o[t][ct][r] * inv[r];
        wave_lds_sync();
        const int vc = min(64, a.e - 64 * (vt0 + t)), col0 = h * a.e + 64 * (vt0 + t);
        if (VEC) {
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const int tok = 16 * wave + 4 * u + G, col = 4 * c;
                if (tok >= n || col >= vc) continue;
                float4 x = *reinterpret_cast<const float4*>(Ps + (4 * u + G) * MM_STRIDE + col);
                if (!FUSED) {
                    *reinterpret_cast<float4*>(y + static_cast<size_t>(first + tok) * ldy + col0 + col) = x;
                    continue;
                }
                const float4 g = t == 0 ? gate4[u] : *reinterpret_cast<const float4*>(rows + static_cast<size_t>(tok) * a.ld + a.g_col + col0 + col);
                float4 w = norm4;
                if (t > 0 && a.norm_w != nullptr) w = *reinterpret_cast<const float4*>(a.norm_w + col0 + col);
                x.x *= w.x * mm_gate(a, g.x); x.y *= w.y * mm_gate(a, g.y); x.z *= w.z * mm_gate(a, g.z); x.w *= w.w * mm_gate(a, g.w);
                T* dst = out + static_cast<size_t>(first + tok) * ldo + col0 + col;
                if (sizeof(T) == 2) {
                    uint2 pk;
                    pk.x = pack_bf16x2(x.x, x.y);
                    pk.y = pack_bf16x2(x.z, x.w);
                    *reinterpret_cast<uint2*>(dst) = pk;
                } else {
                    *reinterpret_cast<float4*>(dst) = x;
                }
            }
        } else {
            for (int tt = 0; tt < 16; ++tt) {
                const int tok = 16 * wave + tt;
                if (tok >= n || lane >= vc) continue;
                const float x = Ps[tt * MM_STRIDE + lane];
                if (FUSED) {
                    const float g = rows[static_cast<size_t>(tok) * a.ld + a.g_col + col0 + lane];
                    out[static_cast<size_t>(first + tok) * ldo + col0 + lane] = from_float<T>(x * mm_norm_weight(a, col0 + lane) * mm_gate(a, g));
                } else {
                    y[static_cast<size_t>(first + tok) * ldy + col0 + lane] = x;
                }
            }
        }
    }
}

// Single tokens: workgroup (sequence, head, column tile) of 256 threads; `cols` columns a tile (FUSED: all of the head's).
// A thread owns CW neighbouring columns (VEC: 4) of every RG-th row of the memory, RG = 256 / (cols / CW).
// LDS: q [d] | k [d] | shares [RG * cols] | 8.
template <typename T, bool VEC, bool FUSED>
__global__ void __launch_bounds__(256)
memory_single_kernel(MemoryArgs a, int cols, T* __restrict__ out, int ldo, float* __restrict__ y, int ldy) {
    extern __shared__ __attribute__((aligned(16))) float mm_smem[];
    constexpr int CW = VEC ? 4 : 1, AHEAD = VEC ? 4 : 8;
    // (the sequences of single tokens stand in front: sequence b's token is row b)
    const int b = blockIdx.x, h = blockIdx.y, tile = blockIdx.z;
    const int slot = a.state_slots[b];
    if (slot < 0) return;
    const int tid = threadIdx.x, lane = tid % MLLM_WAVE, wave = __builtin_amdgcn_readfirstlane(tid / MLLM_WAVE);
    const int d = a.d, e = a.e, c0 = tile * cols, nc = min(cols, e - c0);
    const int groups = cols / CW, RG = 256 / groups;          // (cols is a multiple of CW, at most 256 CW)
    float* q_s = mm_smem;
    float* k_s = q_s + d;
    float* part = k_s + d;                                    // [RG][cols]
    float* red = part + RG * cols;                            // [4]: the wavefronts' shares of n . q
    const float* row = a.proj + static_cast<size_t>(b) * a.ld;
    float* base = a.state + static_cast<size_t>(slot) * a.slot_floats;
    float* S = base + static_cast<size_t>(h) * d * e + c0;
    float* N = base + state_n_at(a, h, tile);
    const bool fixed = a.head_decay != nullptr;               // (retention: a decay of the head's own, no normaliser)
    const float iz = fixed ? 0.f : row[a.i_col + h], fz = fixed ? 0.f : row[a.f_col + h], m_old = fixed ? 0.f : base[state_m_at(a, h, tile)];
    const int rg = tid / groups, col = (tid % groups) * CW;
    const bool active = rg < RG && col < nc;
    const int col_c = min(col, nc - CW);                      // a valid place in any case
    float v[CW];
#pragma unroll
    for (int k = 0; k < CW; ++k) v[k] = row[a.v_col + h * e + c0 + col_c + k];
    // the first rows of the memory, the normaliser and what the end needs are asked for before anything is waited for
    float s[AHEAD][CW];
    auto ask = [&](int i0) {
#pragma unroll
        for (int u = 0; u < AHEAD; ++u) {
            const float* p = S + static_cast<size_t>(min(i0 + u * RG + min(rg, RG - 1), d - 1)) * e + col_c;
            if (VEC) {
                const float4 x = *reinterpret_cast<const float4*>(p);
                s[u][0] = x.x; s[u][CW > 1 ? 1 : 0] = x.y; s[u][CW > 1 ? 2 : 0] = x.z; s[u][CW > 1 ? 3 : 0] = x.w;
            } else {
                s[u][0] = *p;
            }
        }
    };
    ask(0);
    const float n_first = fixed ? 0.f : N[min(tid, d - 1)];
    const float g_first = row[a.g_col + h * e + c0 + min(lane, nc - 1)], w_first = mm_norm_weight(a, h * e + c0 + min(lane, nc - 1));
    for (int i = tid; i < d; i += 256) {
        q_s[i] = row[a.q_col + h * d + i] * a.q_scale;
        k_s[i] = row[a.k_col + h * d + i];
    }
    float m = 0.f, keep, take = 1.f;
    if (fixed) {
        keep = a.head_decay[h];
    } else {
        const float ig = mm_log_input(iz, a.i_bias[h], a.cap), fg = mm_log_forget(fz, a.f_bias[h], a.cap);
        m = fmaxf(fg + m_old, ig);
        keep = expf(fg + m_old - m);
        take = expf(ig - m);
    }
    lds_barrier();
    // the normaliser (its new values are written behind the barrier below: m_old and N are this workgroup's own copy)
    float nq = 0.f;
    for (int i = fixed ? d : tid; i < d; i += 256) {
        const float x = keep * (i == tid ? n_first : N[i]) + take * k_s[i];
        if (a.write) N[i] = x;
        nq = fmaf(x, q_s[i], nq);
    }
    float acc[CW];
#pragma unroll
    for (int k = 0; k < CW; ++k) { acc[k] = 0.f; v[k] *= take; }
    for (int i0 = 0; i0 < d; i0 += RG * AHEAD) {
        if (i0 > 0) ask(i0);
#pragma unroll
        for (int u = 0; u < AHEAD; ++u) {
            const int i = i0 + u * RG + rg;
            if (active && i < d) {
                const float ki = k_s[i], qi = q_s[i];
#pragma unroll
                for (int k = 0; k < CW; ++k) {
                    s[u][k] = fmaf(keep, s[u][k], ki * v[k]);
                    acc[k] = fmaf(s[u][k], qi, acc[k]);
                }
                if (a.write) {
                    float* p = S + static_cast<size_t>(i) * e + col;
                    if (VEC) *reinterpret_cast<float4*>(p) = make_float4(s[u][0], s[u][CW > 1 ? 1 : 0], s[u][CW > 1 ? 2 : 0], s[u][CW > 1 ? 3 : 0]);
                    else *p = s[u][0];
                }
            }
        }
    }
    if (active) {
#pragma unroll
        for (int k = 0; k < CW; ++k) part[rg * cols + col + k] = acc[k];
    }
    nq = wave_sum(nq);
    if (lane == 0) red[wave] = nq;
    if (tid == 0 && a.write && !fixed) base[state_m_at(a, h, tile)] = m;        // (every wavefront has read m_old: it stands in front of the barrier above)
    lds_barrier();
    if (wave != 0) return;
    const float den = fixed ? 1.f : fmaxf(fabsf((red[0] + red[1]) + (red[2] + red[3])), expf(-m)) + 1e-6f;
    // one wavefront finishes: columns lane, lane + 64, ... (FUSED: two passes, the sums kept in LDS)
    float ss = 0.f;
    for (int j = lane; j < nc; j += MLLM_WAVE) {
        float x = 0.f;
        for (int r = 0; r < RG; ++r) x += part[r * cols + j];
        x /= den;
        if (FUSED) part[j] = x;                                       // (only this lane reads column j)
        else y[static_cast<size_t>(b) * ldy + h * e + c0 + j] = x;
        ss += x * x;
    }
    if (!FUSED) return;
    const float inv = 1.f / sqrtf(wave_sum(ss) / static_cast<float>(e) + a.eps);
    for (int j = lane; j < nc; j += MLLM_WAVE) {
        const float g = j == lane ? g_first : row[a.g_col + h * e + j], w = j == lane ? w_first : mm_norm_weight(a, h * e + j);
        out[static_cast<size_t>(b) * ldo + h * e + j] = from_float<T>(part[j] * inv * w * mm_gate(a, g));
    }
}

// Memories of up to this many floats a head are one workgroup's work in steps of single tokens.
constexpr int MM_ONE_WORKGROUP = 32768;

}  // namespace

extern "C" {

int mllm_matrix_memory_chunk() { return MM_CHUNK; }

// How many workgroups share a head's memory in steps of single tokens (and copies of n and m the state holds).
int mllm_matrix_memory_copies(int d, int e) {
    if (static_cast<long long>(d) * e <= MM_ONE_WORKGROUP && (e % 4 == 0 ? e <= 1024 : e <= 256)) return 1;
    return (e + 63) / 64;
}
size_t mllm_matrix_memory_state_floats(int H, int d, int e, int retention) {
    if (retention) return static_cast<size_t>(H) * d * e;
    const size_t copies = mllm_matrix_memory_copies(d, e);
    return static_cast<size_t>(H) * d * e + static_cast<size_t>(H) * copies * (static_cast<size_t>(d) + 1);
}
// Workspace of a step of T tokens in B sequences.
size_t mllm_matrix_memory_workspace_floats(int T, int B, int H, int d, int e) {
    return (static_cast<size_t>(T) / MM_CHUNK + B) * H * chunk_floats(d, e);
}

// proj [T, ld] fp32 holds, per token, raw queries (H * d from q_col; times q_scale), keys (H * d from k_col), values
// (H * e from v_col), raw output gates (H * e from g_col) and raw input and forget gates (H from i_col, f_col). The first
// n_single sequences bring one token each, the others any number; max_portion: the longest portion among those (0: there
// are none). out [T, H * e] in `dtype`: normed and gated, if *needs_norm comes back 0; otherwise y ([T, ldy] fp32) holds
// o of those rows that the caller must norm: *needs_norm bit 0 the single tokens' rows, bit 1 the portions' rows.
// A request's state starts at its slot. head_decay ([H], on the device; the i and f columns and biases and cap are then not used)
// makes it retention, norm_w may be null (no weight), silu: the output gate is silu. -1: sizes or pointers that do not fit; -2: a key width beyond the LDS.
int mllm_matrix_memory(const float* proj, int ld, int q_col, int k_col, int v_col, int g_col, int i_col, int f_col, const float* i_bias,
                       const float* f_bias, const float* norm_w, float cap, float q_scale, float eps, const int* cu_q, const int* state_slots,
                       float* state, size_t slot_floats, int T, int B, int n_single, int max_portion, int H, int d, int e, int write,
                       float* workspace, void* out, int ldo, float* y, int ldy, int dtype, int* needs_norm, hipStream_t stream,
                       const float* head_decay, int silu) {
    *needs_norm = 0;
    bool singles_in_chunks = false;
    if (T <= 0 || B <= 0) return 0;
    if (H < 1 || d < 1 || e < 1 || n_single < 0 || n_single > B || proj == nullptr) return -1;
    if (head_decay == nullptr && (!(cap > 0.f) || i_bias == nullptr || f_bias == nullptr)) return -1;
    const int copies = mllm_matrix_memory_copies(d, e);
    const MemoryArgs a{proj, ld, q_col, k_col, v_col, g_col, i_col, f_col, i_bias, f_bias, norm_w, cap, q_scale, eps, head_decay, silu, cu_q, state_slots,
                       state, slot_floats, H, d, e, copies, write};
    const auto a16 = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
    // (16-byte accesses: every row and head starts on a multiple of 4 floats; bfloat16 rows on 8 bytes)
    const bool vec = d % 4 == 0 && e % 4 == 0 && ld % 4 == 0 && q_col % 4 == 0 && k_col % 4 == 0 && v_col % 4 == 0 && g_col % 4 == 0 && ldo % 4 == 0 &&
                     ldy % 4 == 0 && slot_floats % 4 == 0 && a16(proj) && a16(state) && a16(workspace) && a16(out) && a16(y) && (norm_w == nullptr || a16(norm_w));
    if (n_single > 0) {
        const bool fused = copies == 1;
        const bool v4 = vec && (!fused || e <= 1024);
        const int cols = fused ? e : 64, cw = v4 ? 4 : 1;
        if (fused && !v4 && e > 256) {
            // (a wide head whose rows are not aligned: chunks of one token serve it)
            n_single = 0;
            singles_in_chunks = true;
            if (max_portion < 1) max_portion = 1;
        } else {
            const int rg = 256 / (cols / cw);
            const size_t lds = (static_cast<size_t>(2) * d + static_cast<size_t>(rg) * cols + 8) * sizeof(float);
            if (lds > 60 * 1024) return -2;
            const dim3 grid(n_single, H, fused ? 1 : (e + 63) / 64);
            if (!fused && y == nullptr) return -1;
#define MM_SINGLE(TYPE, VEC, FUSED) memory_single_kernel<TYPE, VEC, FUSED><<<grid, 256, lds, stream>>>(a, cols, static_cast<TYPE*>(out), ldo, y, ldy)
#define MM_SINGLE_T(TYPE) do { if (v4) { if (fused) MM_SINGLE(TYPE, true, true); else MM_SINGLE(TYPE, true, false); } \
                               else { if (fused) MM_SINGLE(TYPE, false, true); else MM_SINGLE(TYPE, false, false); } } while (0)
            if (dtype == MLLM_F32) MM_SINGLE_T(float); else MM_SINGLE_T(bf16_t);
#undef MM_SINGLE_T
#undef MM_SINGLE
            MLLM_LAUNCH_CHECK();
            if (!fused) *needs_norm |= 1;
        }
    }
    if (n_single == B || max_portion < 1) return 0;
    if (workspace == nullptr) return -1;
    const int kt = (d + 63) / 64, vt = (e + 63) / 64, seqs = B - n_single;
    const long long chunks = T / MM_CHUNK + seqs;           // an upper bound; surplus workgroups leave at once
    const long long cells = (static_cast<long long>(d) * e + d) * H;
    if (chunks >= (1ll << 31) || cells / 256 >= (1ll << 31) - 1 || seqs > 65535 || H > 65535 || static_cast<long long>(kt) * vt > 65535) return -1;
    const dim3 ga(static_cast<unsigned>(chunks), H, kt * vt);
    if (vec) memory_chunk_kernel<true><<<ga, 256, 0, stream>>>(a, n_single, B, vt, workspace);
    else memory_chunk_kernel<false><<<ga, 256, 0, stream>>>(a, n_single, B, vt, workspace);
    MLLM_LAUNCH_CHECK();
    memory_states_kernel<<<dim3(static_cast<unsigned>((cells + 255) / 256), seqs), 256, 0, stream>>>(a, n_single, workspace);
    MLLM_LAUNCH_CHECK();
    const bool fused = vt <= 8;
    if (!fused && y == nullptr) return -1;
#define MM_OUT(TYPE, NT, VEC, FUSED)                                                                                                        \
    memory_output_kernel<TYPE, NT, VEC, FUSED><<<dim3(static_cast<unsigned>(chunks), H, (vt + NT - 1) / NT), 256, 0, stream>>>(              \
        a, n_single, B, workspace, static_cast<TYPE*>(out), ldo, y, ldy)
#define MM_OUT_NT(TYPE, VEC)                                                                                                                \
    do {                                                                                                                                    \
        if (vt == 1) MM_OUT(TYPE, 1, VEC, true); else if (vt == 2) MM_OUT(TYPE, 2, VEC, true); else if (vt <= 4) MM_OUT(TYPE, 4, VEC, true); \
        else if (fused) MM_OUT(TYPE, 8, VEC, true); else MM_OUT(TYPE, 4, VEC, false);                                                       \
    } while (0)
    if (dtype == MLLM_F32) { if (vec) MM_OUT_NT(float, true); else MM_OUT_NT(float, false); }
    else { if (vec) MM_OUT_NT(bf16_t, true); else MM_OUT_NT(bf16_t, false); }
#undef MM_OUT_NT
#undef MM_OUT
    MLLM_LAUNCH_CHECK();
    if (!fused) *needs_norm |= singles_in_chunks ? 3 : 2;
    return 0;
}

}  // extern "C"
