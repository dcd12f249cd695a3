// A mixture of small feed-forward experts, for gfx950: the choice of experts and the activation between the experts'
// two products. Softmax and weights are fp32 whatever the activation dtype; the router's logits come from a product
// with fp32 results.
//
// The experts' first products are one joined product (rows [expert 0 | expert 1 | ... | shared expert]); the
// activation kernel applies the activation (squared rectified values, or the exact GELU) and multiplies every expert's
// block by the token's weight for that expert (zero for an expert that was not chosen, one for the shared expert), so that the experts' second products are
// one joined product as well: sum_e w_e W_down,e a_e = [W_down,0 | W_down,1 | ...] [w_0 a_0; w_1 a_1; ...].
// Experts that hand on their input (the identity, times the weight) have no rows; the kernel adds them up by itself.
// For many tokens and experts of which few are chosen the products are grouped instead (moe_route_kernel and what follows):
// every expert multiplies the tokens that chose it and no others.
// A second kernel serves experts that are gated and clamped, chosen by sigmoid or softmax scores, whose weight may
// stand on the expert's input, beside a shared expert that a sigmoid of the input scales.
#include "common.h"

#include <type_traits>

#define MOE_MAX_EXPERTS 256

namespace {

// The weights of a token's experts from its router logits z (in LDS, E of them): scores softmax(z) over all experts,
// the `top` largest chosen (the lower index wins a tie), wgt[e] = scale * score_e for them and 0 for the others.
// Thread e < E works out expert e's weight; the caller has a barrier before (z complete) and puts one behind.
// With `sigmoid` the scores are sigmoid(z), every expert's on its own (the order of the scores is the logits' either way).
__device__ __forceinline__ void expert_weight(const float* z, float* wgt, int E, int top, float scale, int e, bool sigmoid = false) {
    const float mine = z[e];
    float m = -INFINITY;
    for (int o = 0; o < E; ++o) m = fmaxf(m, z[o]);
    float sum = 0.f;
    int before = 0;
    for (int o = 0; o < E; ++o) {
        sum += expf(z[o] - m);
        before += (z[o] > mine || (z[o] == mine && o < e)) ? 1 : 0;
    }
    const float score = sigmoid ? 1.f / (1.f + expf(-mine)) : expf(mine - m) / sum;
    wgt[e] = before < top ? scale * score : 0.f;
}

// How scores become weights: a softmax over all experts' logits, every logit's sigmoid on its own, or a softmax over the
// chosen experts' logits alone.
enum RouterKind : int { ROUTER_SOFTMAX = 0, ROUTER_SIGMOID = 1, ROUTER_SOFTMAX_CHOSEN = 2 };

// Up to 64 experts: a wavefront works out a token's weights by itself, lane e expert e's (0 for lanes without an expert).
__device__ __forceinline__ float wave_expert_weight(float mine, int lane, int E, int top, float scale, int kind) {
    int before = 0;
    for (int o = 0; o < E; ++o) {
        const float other = row_lane(mine, o);
        before += (other > mine || (other == mine && o < lane)) ? 1 : 0;
    }
    const bool chosen = lane < E && before < top;
    if (kind == ROUTER_SIGMOID) return chosen ? scale / (1.f + expf(-mine)) : 0.f;
    const float m = wave_max(mine);                      // (the largest logit is always chosen)
    const bool counts = kind == ROUTER_SOFTMAX_CHOSEN ? chosen : lane < E;
    const float ex = counts ? expf(mine - m) : 0.f, sum = wave_sum(ex);
    return chosen ? scale * (ex / sum) : 0.f;
}

// The same for experts that are gated (and clamped): the joined first product's rows are [expert 0: gate | up] ...
// [expert E-1: gate | up] [shared: gate | up], and with g = min(w G, limit), u = clamp(w U, -limit, limit) (the weight
// on the expert's INPUT, which a linear map hands on to its result; `weight_on_input` 0: g and u unweighted and the
// weight on the result) out[t, e * ff + j] = g sigmoid(alpha g) (u + up_shift), zero for an expert that was not chosen
// (whose columns are not read). An infinite limit, alpha 1 and up_shift 0 make it silu(g) u. The
// shared expert's columns follow, unweighted, with its own limit, times sigmoid(logits[t, E]) if `shared_gate` (the
// router's product then has one more row). One workgroup per token. VEC: eight columns a thread at a time (16-byte
// loads of bfloat16, two of float; ff, shared_ff and the strides are then multiples of 8 and the rows aligned), all of
// one expert.
// AHEAD (few tokens): a thread's first columns are asked for before the weights are worked out, chosen expert or not.
template <typename TI, typename T, bool VEC, bool AHEAD>
__global__ void __launch_bounds__(256)
moe_glu_act_kernel(const TI* __restrict__ up, int ldu, const float* __restrict__ logits, int ldl, int E, int ff, int shared_ff, int top,
                   float scale, int router_kind, float limit, float shared_limit, float alpha, float up_shift, int weight_on_input,
                   int shared_gate, T* __restrict__ out, int ldo) {
    // weights: one copy a wavefront where up to 64 experts let every wavefront work them out by itself, without a barrier
    __shared__ float z[MOE_MAX_EXPERTS], weights[4][MOE_MAX_EXPERTS];
    const int t = blockIdx.x, tid = threadIdx.x, lane = tid % MLLM_WAVE;
    const int wave = __builtin_amdgcn_readfirstlane(tid / MLLM_WAVE);
    const float* lr = logits + static_cast<size_t>(t) * ldl;
    float g_first[8], u_first[8];
    if (VEC && AHEAD) {
        const int c = min(tid * 8, E * ff + shared_ff - 8), e = c / ff, j = c - e * ff;
        const TI* p = up + static_cast<size_t>(t) * ldu + (c < E * ff ? static_cast<size_t>(e) * 2 * ff + j : static_cast<size_t>(E) * ff * 2 + (c - E * ff));
        load8(p, g_first);
        load8(p + (c < E * ff ? ff : shared_ff), u_first);
        __builtin_amdgcn_sched_barrier(0);
    }
    const float sg = shared_gate ? 1.f / (1.f + expf(-lr[E])) : 1.f;
    float* wgt = weights[E <= MLLM_WAVE ? wave : 0];
    if (E <= MLLM_WAVE) {
        const float mine = lr[min(lane, E - 1)];
        wgt[lane] = wave_expert_weight(mine, lane, E, top, scale, router_kind);
        wave_lds_sync();
    } else {
        if (tid < E) z[tid] = lr[tid];
        __syncthreads();
        if (router_kind == ROUTER_SOFTMAX_CHOSEN) {
            float* ex = weights[1];
            if (tid < E) {
                const float mine = z[tid];
                float m = -INFINITY;
                int before = 0;
                for (int o = 0; o < E; ++o) {
                    m = fmaxf(m, z[o]);
                    before += (z[o] > mine || (z[o] == mine && o < tid)) ? 1 : 0;
                }
                ex[tid] = before < top ? expf(mine - m) : 0.f;
            }
            __syncthreads();
            if (tid < E) {
                float sum = 0.f;
                for (int o = 0; o < E; ++o) sum += ex[o];
                wgt[tid] = scale * (ex[tid] / sum);
            }
        } else if (tid < E) {
            expert_weight(z, wgt, E, top, scale, tid, router_kind == ROUTER_SIGMOID);
        }
        __syncthreads();
    }
    const TI* ur = up + static_cast<size_t>(t) * ldu;
    T* orow = out + static_cast<size_t>(t) * ldo;
    const int routed = E * ff, N = routed + shared_ff;
    if (VEC) {
        for (int c = tid * 8; c < N; c += 256 * 8) {
            float g[8], u[8], lim = limit, w_in = 1.f, w_out = 1.f, y[8];
            const TI *gp, *upp;
            bool live = true;
            if (c < routed) {
                const int e = c / ff, j = c - e * ff;
                gp = ur + static_cast<size_t>(e) * 2 * ff + j;
                upp = gp + ff;
                const float we = wgt[e];
                live = we != 0.f;
                if (weight_on_input) w_in = we; else w_out = we;
            } else {
                gp = ur + static_cast<size_t>(routed) * 2 + (c - routed);
                upp = gp + shared_ff;
                lim = shared_limit;
                w_out = sg;
            }
            if (live) {
                if (AHEAD && c < 256 * 8) {
#pragma unroll
                    for (int k = 0; k < 8; ++k) { g[k] = g_first[k]; u[k] = u_first[k]; }
                } else {
                    load8(gp, g);
                    load8(upp, u);
                }
#pragma unroll
                for (int k = 0; k < 8; ++k) {
                    const float gk = fminf(g[k] * w_in, lim), uk = fminf(fmaxf(u[k] * w_in, -lim), lim);
                    const float ex = sizeof(T) == 2 ? __expf(-alpha * gk) : expf(-alpha * gk);
                    y[k] = gk / (1.f + ex) * (uk + up_shift) * w_out;
                }
            } else {
#pragma unroll
                for (int k = 0; k < 8; ++k) y[k] = 0.f;
            }
            if (sizeof(T) == 2) {
                uint4 pk;
                pk.x = pack_bf16x2(y[0], y[1]); pk.y = pack_bf16x2(y[2], y[3]); pk.z = pack_bf16x2(y[4], y[5]); pk.w = pack_bf16x2(y[6], y[7]);
                *reinterpret_cast<uint4*>(orow + c) = pk;
            } else {
                *reinterpret_cast<float4*>(orow + c) = make_float4(y[0], y[1], y[2], y[3]);
                *reinterpret_cast<float4*>(orow + c + 4) = make_float4(y[4], y[5], y[6], y[7]);
            }
        }
        return;
    }
    for (int c = tid; c < N; c += 256) {
        float g, u, lim, w_in = 1.f, w_out = 1.f;
        bool live = true;
        if (c < routed) {
            const int e = c / ff, j = c - e * ff;
            g = to_float(ur[static_cast<size_t>(e) * 2 * ff + j]);
            u = to_float(ur[static_cast<size_t>(e) * 2 * ff + ff + j]);
            lim = limit;
            live = wgt[e] != 0.f;
            if (weight_on_input) w_in = wgt[e]; else w_out = wgt[e];
        } else {
            const int j = c - routed;
            g = to_float(ur[static_cast<size_t>(routed) * 2 + j]);
            u = to_float(ur[static_cast<size_t>(routed) * 2 + shared_ff + j]);
            lim = shared_limit;
            w_out = sg;
        }
        g = fminf(g * w_in, lim);
        u = fminf(fmaxf(u * w_in, -lim), lim);
        const float y = g / (1.f + expf(-alpha * g)) * (u + up_shift) * w_out;
        orow[c] = from_float<T>(live ? y : 0.f);
    }
}

// One workgroup per token: the weights from the token's logits, then
// out[t, e * ff + j] = weight_e * act(up[t, e * ff + j]) for the E experts, and behind them
// out[t, E * ff + j] = act(up[t, E * ff + j]) for the shared expert's columns (N columns in all); act is relu(z)^2, or
// with GELU the exact GELU. With `correction` (E + identity numbers) the experts with the largest score + correction are
// chosen, and the score alone is the weight. The last `identity` of the router's outputs are experts that hand on their
// input: y[t, :] = (the sum of their weights) * h[t, :] (D columns; added to y with y_add).
// VEC: eight columns a thread at a time (16-byte loads of bfloat16, two of float; ff, N and the strides are then
// multiples of 8 and the rows aligned). `weights_out` (optional, [T, E + identity]) receives the weights.
struct MoeChoice {
    const float* correction;
    int identity;
    const void* h;           // [T, ldh], the output's dtype
    int ldh, D, ldy, y_add;
    float* y;                // [T, ldy] fp32
};

template <typename TI, typename T, bool VEC, bool GELU>
__global__ void __launch_bounds__(256)
moe_act_kernel(const TI* __restrict__ up, int ldu, const float* __restrict__ logits, int ldl, int E, int ff, int N, int top, float scale,
               T* __restrict__ out, int ldo, float* __restrict__ weights_out, int ldw, MoeChoice mc) {
    // weights: one copy a wavefront where up to 64 experts let every wavefront work them out by itself, without a barrier
    __shared__ float z[MOE_MAX_EXPERTS], weights[4][MOE_MAX_EXPERTS], choice[MOE_MAX_EXPERTS];
    const int t = blockIdx.x, tid = threadIdx.x, all = E + mc.identity, lane = tid % MLLM_WAVE;
    const int wave = __builtin_amdgcn_readfirstlane(tid / MLLM_WAVE);
    const TI* ur = up + static_cast<size_t>(t) * ldu;
    T* orow = out + static_cast<size_t>(t) * ldo;
    // the first columns are asked for before the weights are worked out
    constexpr int AHEAD = 2;
    float first[AHEAD][8];
    if (VEC) {
#pragma unroll
        for (int u = 0; u < AHEAD; ++u) load8(ur + min(tid * 8 + 2048 * u, N - 8), first[u]);
    }
    float* wgt = weights[all <= MLLM_WAVE ? wave : 0];
    if (all <= MLLM_WAVE) {
        const float mine = logits[static_cast<size_t>(t) * ldl + min(lane, all - 1)];
        const float m = wave_max(mine), ex = lane < all ? expf(mine - m) : 0.f;
        const float score = ex / wave_sum(ex);
        // (without a correction the order of the scores is that of the logits)
        const float key = mc.correction != nullptr ? score + mc.correction[min(lane, all - 1)] : mine;
        int before = 0;
        for (int o = 0; o < all; ++o) {
            const float other = row_lane(key, o);
            before += (other > key || (other == key && o < lane)) ? 1 : 0;
        }
        wgt[lane] = before < top ? scale * score : 0.f;
        wave_lds_sync();
    } else {
        if (tid < all) z[tid] = logits[static_cast<size_t>(t) * ldl + tid];
        __syncthreads();
        if (mc.correction == nullptr) {
            if (tid < all) expert_weight(z, wgt, all, top, scale, tid);
        } else {
            float score = 0.f;
            if (tid < all) {
                float m = -INFINITY, sum = 0.f;
                for (int o = 0; o < all; ++o) m = fmaxf(m, z[o]);
                for (int o = 0; o < all; ++o) sum += expf(z[o] - m);
                score = expf(z[tid] - m) / sum;
                choice[tid] = score + mc.correction[tid];
            }
            __syncthreads();
            if (tid < all) {
                const float mine = choice[tid];
                int before = 0;
                for (int o = 0; o < all; ++o) before += (choice[o] > mine || (choice[o] == mine && o < tid)) ? 1 : 0;
                wgt[tid] = before < top ? scale * score : 0.f;
            }
        }
        __syncthreads();
    }
    if (weights_out != nullptr && tid < all) weights_out[static_cast<size_t>(t) * ldw + tid] = wgt[tid];
    if (VEC) {
        auto columns = [&](int c, float (&v)[8]) {
            const int e = c / ff;                       // (ff is a multiple of 8: the eight columns are one expert's)
            const float wt = e < E ? wgt[e] : 1.f;
            if (GELU) {
                if (wt != 0.f) {                        // (no erf for an expert that was not chosen)
#pragma unroll
                    for (int u = 0; u < 8; ++u) v[u] = wt * gelu_erf(v[u]);
                } else {
#pragma unroll
                    for (int u = 0; u < 8; ++u) v[u] = 0.f;
                }
            } else {
#pragma unroll
                for (int u = 0; u < 8; ++u) v[u] = wt * relu2(v[u]);
            }
            if (sizeof(T) == 2) {
                uint4 pk;
                pk.x = pack_bf16x2(v[0], v[1]); pk.y = pack_bf16x2(v[2], v[3]); pk.z = pack_bf16x2(v[4], v[5]); pk.w = pack_bf16x2(v[6], v[7]);
                *reinterpret_cast<uint4*>(orow + c) = pk;
            } else {
                *reinterpret_cast<float4*>(orow + c) = make_float4(v[0], v[1], v[2], v[3]);
                *reinterpret_cast<float4*>(orow + c + 4) = make_float4(v[4], v[5], v[6], v[7]);
            }
        };
#pragma unroll
        for (int u = 0; u < AHEAD; ++u)
            if (tid * 8 + 2048 * u < N) columns(tid * 8 + 2048 * u, first[u]);
        for (int c = tid * 8 + 2048 * AHEAD; c < N; c += 2048) {
            float v[8];
            load8(ur + c, v);
            columns(c, v);
        }
    } else {
        for (int c = tid; c < N; c += 256) {
            const int e = c / ff;
            const float wt = e < E ? wgt[e] : 1.f;
            const float v = to_float(ur[c]);
            orow[c] = from_float<T>(wt != 0.f ? wt * (GELU ? gelu_erf(v) : relu2(v)) : 0.f);
        }
    }
    if (mc.identity > 0) {
        float w = 0.f;
        for (int o = E; o < all; ++o) w += wgt[o];
        const T* hr = static_cast<const T*>(mc.h) + static_cast<size_t>(t) * mc.ldh;
        float* yr = mc.y + static_cast<size_t>(t) * mc.ldy;
        if (((mc.D | mc.ldh | mc.ldy) & 7) == 0 && ((reinterpret_cast<uintptr_t>(mc.h) | reinterpret_cast<uintptr_t>(mc.y)) & 15) == 0) {
            for (int c = tid * 8; c < mc.D; c += 2048) {
                float v[8], old[8];
                load8(hr + c, v);
                if (mc.y_add) load8(yr + c, old);
#pragma unroll
                for (int u = 0; u < 8; ++u) v[u] = (mc.y_add ? old[u] : 0.f) + w * v[u];
                *reinterpret_cast<float4*>(yr + c) = make_float4(v[0], v[1], v[2], v[3]);
                *reinterpret_cast<float4*>(yr + c + 4) = make_float4(v[4], v[5], v[6], v[7]);
            }
        } else {
            for (int c = tid; c < mc.D; c += 256) yr[c] = (mc.y_add ? yr[c] : 0.f) + w * to_float(hr[c]);
        }
    }
}

// ---------------------------------------------------------------------------------------------
// Grouped products: a slot is a (token, choice) pair, slot = token * top + choice. Routing writes, per expert, the list of
// the slots that chose it (in any order: a row's arithmetic does not depend on its neighbours) and every slot's weight; the
// first products gather the tokens' rows and leave act(gate, up) * weight per slot, the second products multiply those, and
// a last kernel adds a token's slots in their order and takes the sum into the stream.
// ---------------------------------------------------------------------------------------------

// A workgroup takes `tokens` tokens, a thread each; counts are gathered in LDS first, so that an expert's counter sees one
// addition a workgroup. LDS: tokens * (E + 1) logits, then 2 E counters.
__global__ void __launch_bounds__(256)
moe_route_kernel(const float* __restrict__ logits, int ldl, int T, int E, int top, float scale, int kind, int tokens, int* __restrict__ counts,
                 int* __restrict__ lists, int cap, float* __restrict__ weights) {
    extern __shared__ float mr_smem[];
    const int tid = threadIdx.x, first = blockIdx.x * tokens, n = min(tokens, T - first), stride = E + 1;
    int* mine = reinterpret_cast<int*>(mr_smem + tokens * stride);       // [E] slots of this workgroup, then [E] where they start
    for (int i = tid; i < n * E; i += 256) mr_smem[(i / E) * stride + i % E] = logits[static_cast<size_t>(first + i / E) * ldl + i % E];
    for (int i = tid; i < E; i += 256) mine[i] = 0;
    __syncthreads();
    constexpr int KEEP = 8;                          // choices whose places stay in registers; further ones are chosen again
    int chosen[KEEP], place[KEEP];
    float* z = mr_smem + tid * stride;
    float m = -INFINITY, all = 0.f, sum = 0.f;
    if (tid < n) {
        for (int e = 0; e < E; ++e) m = fmaxf(m, z[e]);
        if (kind == ROUTER_SOFTMAX)
            for (int e = 0; e < E; ++e) all += expf(z[e] - m);
#pragma unroll
        for (int j = 0; j < KEEP; ++j) {
            if (j >= top) break;
            int best = 0;
            float value = -INFINITY;
            for (int e = 0; e < E; ++e)
                if (z[e] > value) { value = z[e]; best = e; }
            z[best] = -INFINITY;
            chosen[j] = best;
            place[j] = atomicAdd(&mine[best], 1);
            const float ex = kind == ROUTER_SIGMOID ? 1.f / (1.f + expf(-value)) : expf(value - m);
            sum += ex;
            weights[static_cast<size_t>(first + tid) * top + j] = ex;
        }
    }
    __syncthreads();
    for (int e = tid; e < E; e += 256) mine[E + e] = mine[e] > 0 ? atomicAdd(&counts[e], mine[e]) : 0;
    __syncthreads();
    if (tid >= n) return;
    const float over = kind == ROUTER_SOFTMAX ? all : (kind == ROUTER_SOFTMAX_CHOSEN ? sum : 1.f);
#pragma unroll
    for (int j = 0; j < KEEP; ++j) {
        if (j >= top) break;
        const size_t slot = static_cast<size_t>(first + tid) * top + j;
        weights[slot] = scale * (weights[slot] / over);
        const int at = mine[E + chosen[j]] + place[j];
        if (at < cap) lists[static_cast<size_t>(chosen[j]) * cap + at] = static_cast<int>(slot);
    }
}

typedef __bf16 mbf16x8 __attribute__((ext_vector_type(8)));
typedef float mf32x16 __attribute__((ext_vector_type(16)));
#define MG_BM 64
#define MG_BK 64
#define MG_STRIDE (MG_BK + 8)

struct GroupedArgs {
    const bf16_t* A;             // rows of K: tokens' (FIRST) or slots'
    int lda;
    const bf16_t* W;             // FIRST: expert e's rows [gate: ff | up: ff] from row 2 ff e; else columns ff e .. of [N, ldw]
    int ldw, ff, N, K, E, top, cap;
    const int* counts;
    const int* lists;
    const float* weights;        // per slot (FIRST)
    bf16_t* act;                 // FIRST: [slots, ld_out]
    float* y;                    // else: [slots, ld_out]
    int ld_out;
    float limit, alpha, up_shift;
};

// A tile of 64 slots of one expert x 128 columns (FIRST: 64 gates and the 64 ups of the same columns): four wavefronts, each 32
// slots x 2 tiles of 32. v_mfma_f32_32x32x16_bf16 with the weights as the first operand; LDS double buffer, two k tiles in
// flight in registers. The k loop has no conditions: columns of A beyond K are multiplied with zeros put in for W.
template <bool FIRST>
__global__ void __launch_bounds__(256)
moe_grouped_kernel(GroupedArgs g) {
    constexpr int BN = 128;
    __shared__ __attribute__((aligned(16))) bf16_t As[2][MG_BM * MG_STRIDE];
    __shared__ __attribute__((aligned(16))) bf16_t Ws[2][BN * MG_STRIDE];
    __shared__ int slot_s[MG_BM];
    const int tid = threadIdx.x, lane = tid % MLLM_WAVE, wave = __builtin_amdgcn_readfirstlane(tid / MLLM_WAVE);
    // which expert's row tile this is: a prefix sum over the experts' tiles, 64 experts at a time
    int e = -1, tile = blockIdx.x, count = 0;
    for (int e0 = 0; e0 < g.E && e < 0; e0 += MLLM_WAVE) {
        const int its = e0 + lane < g.E ? min(g.counts[e0 + lane], g.cap) : 0;
        const int nt = (its + MG_BM - 1) / MG_BM;
        int upto = nt;
#pragma unroll
        for (int off = 1; off < MLLM_WAVE; off *= 2) {
            const int other = __shfl_up(upto, off, MLLM_WAVE);
            if (lane >= off) upto += other;
        }
        const unsigned long long here = __ballot(tile < upto);
        if (here != 0) {
            const int l = __ffsll(here) - 1;
            e = e0 + l;
            count = __shfl(its, l, MLLM_WAVE);
            tile -= __shfl(upto, l, MLLM_WAVE) - __shfl(nt, l, MLLM_WAVE);
        } else {
            tile -= __shfl(upto, MLLM_WAVE - 1, MLLM_WAVE);
        }
    }
    if (e < 0) return;                               // (the grid is an upper bound)
    e = __builtin_amdgcn_readfirstlane(e);
    tile = __builtin_amdgcn_readfirstlane(tile);
    count = __builtin_amdgcn_readfirstlane(count);
    const int first = tile * MG_BM, rows = min(MG_BM, count - first), n0 = blockIdx.y * (FIRST ? BN / 2 : BN);
    if (tid < MG_BM) slot_s[tid] = g.lists[static_cast<size_t>(e) * g.cap + first + min(tid, rows - 1)];
    __syncthreads();
    // loads: 16-byte pieces, eight neighbouring threads a row's 128 bytes
    const bf16_t* a_row[2];
    const bf16_t* w_row[4];
    const int piece = (tid % 8) * 8;
#pragma unroll
    for (int u = 0; u < 2; ++u) {
        const int slot = slot_s[tid / 8 + 32 * u];
        a_row[u] = g.A + static_cast<size_t>(FIRST ? slot / g.top : slot) * g.lda;
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
        const int r = tid / 8 + 32 * u;
        if (FIRST) w_row[u] = g.W + (static_cast<size_t>(e) * 2 * g.ff + (r < 64 ? min(n0 + r, g.ff - 1) : g.ff + min(n0 + r - 64, g.ff - 1))) * g.ldw;
        else w_row[u] = g.W + static_cast<size_t>(min(n0 + r, g.N - 1)) * g.ldw + static_cast<size_t>(e) * g.ff;
    }
    mbf16x8 ra[2][2], rw[2][4];
    const int KT = (g.K + MG_BK - 1) / MG_BK;
    auto fetch = [&](auto ring, int kt) {
        constexpr int R = decltype(ring)::value;
        const int k = min(kt * MG_BK + piece, g.K - 8);
#pragma unroll
        for (int u = 0; u < 2; ++u) ra[R][u] = *reinterpret_cast<const mbf16x8*>(a_row[u] + k);
#pragma unroll
        for (int u = 0; u < 4; ++u) rw[R][u] = *reinterpret_cast<const mbf16x8*>(w_row[u] + k);
        __builtin_amdgcn_sched_barrier(0);
    };
    auto stage = [&](auto ring, int kt) {            // tile kt from its registers into its LDS buffer
        constexpr int R = decltype(ring)::value;
        const bool inside = kt * MG_BK + piece < g.K;
        const mbf16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
        for (int u = 0; u < 2; ++u) *reinterpret_cast<mbf16x8*>(&As[R][(tid / 8 + 32 * u) * MG_STRIDE + piece]) = ra[R][u];
#pragma unroll
        for (int u = 0; u < 4; ++u) *reinterpret_cast<mbf16x8*>(&Ws[R][(tid / 8 + 32 * u) * MG_STRIDE + piece]) = inside ? rw[R][u] : zero;
    };
    const int wm = wave / 2, wn = wave % 2;
    const int col[2] = {FIRST ? 32 * wn : 64 * wn, FIRST ? 64 + 32 * wn : 64 * wn + 32};      // this wavefront's rows of Ws
    mf32x16 acc[2];
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
        for (int r = 0; r < 16; ++r) acc[j][r] = 0.f;
    auto multiply = [&](auto ring) {
        constexpr int R = decltype(ring)::value;
#pragma unroll
        for (int ks = 0; ks < MG_BK / 16; ++ks) {
            const int k = ks * 16 + 8 * (lane / 32);
            const mbf16x8 a = *reinterpret_cast<const mbf16x8*>(&As[R][(32 * wm + lane % 32) * MG_STRIDE + k]);
#pragma unroll
            for (int j = 0; j < 2; ++j) {
                const mbf16x8 w = *reinterpret_cast<const mbf16x8*>(&Ws[R][(col[j] + lane % 32) * MG_STRIDE + k]);
                acc[j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(w, a, acc[j], 0, 0, 0);
            }
        }
    };
    std::integral_constant<int, 0> R0;
    std::integral_constant<int, 1> R1;
    fetch(R0, 0);
    fetch(R1, 1);
    stage(R0, 0);
    for (int kt = 0; kt < KT; kt += 2) {
        lds_barrier();                               // tile kt is in LDS, and everybody is done with tile kt - 1
        fetch(R0, kt + 2);
        multiply(R0);
        stage(R1, kt + 1);
        if (kt + 1 >= KT) break;
        lds_barrier();
        fetch(R1, kt + 3);
        multiply(R1);
        stage(R0, kt + 2);
    }
    lds_barrier();                                   // the tiles' LDS is free
    // (register r of lane l: column 8 (r / 4) + 4 (l / 32) + r % 4 of slot l % 32) through LDS into stores of whole rows
    float* epi = reinterpret_cast<float*>(&Ws[0][0]) + wave * (32 * 36);
    constexpr int PASSES = FIRST ? 1 : 2;
    const float my_weight = FIRST ? g.weights[slot_s[32 * wm + lane % 32]] : 1.f;
#pragma unroll
    for (int p = 0; p < PASSES; ++p) {
        wave_lds_sync();
#pragma unroll
        for (int q = 0; q < 4; ++q) {
            float v[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                if (FIRST) {
                    const float gk = fminf(acc[0][4 * q + i], g.limit), uk = fminf(fmaxf(acc[1][4 * q + i], -g.limit), g.limit);
                    v[i] = gk / (1.f + __expf(-g.alpha * gk)) * (uk + g.up_shift) * my_weight;
                } else {
                    v[i] = acc[p][4 * q + i];
                }
            }
            *reinterpret_cast<float4*>(&epi[(lane % 32) * 36 + 8 * q + 4 * (lane / 32)]) = make_float4(v[0], v[1], v[2], v[3]);
        }
        wave_lds_sync();
        const int nb = n0 + (FIRST ? 32 * wn : 64 * wn + 32 * p), last = FIRST ? g.ff : g.N;
#pragma unroll
        for (int it = 0; it < 4; ++it) {
            const int r = it * 8 + lane / 8, n = nb + (lane % 8) * 4;
            if (32 * wm + r >= rows || n >= last) continue;
            const float4 v = *reinterpret_cast<const float4*>(&epi[r * 36 + (lane % 8) * 4]);
            const size_t at = static_cast<size_t>(slot_s[32 * wm + r]) * g.ld_out + n;
            if (FIRST) *reinterpret_cast<uint2*>(g.act + at) = make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w));
            else *reinterpret_cast<float4*>(g.y + at) = v;
        }
    }
}

// What a token's slots sum up to, into the stream: through add (tanh_norm.h; norm and copy) with add_to 1, or with add_to 0 set
// as it is. Zeroes the counters for the next routing.
__global__ void __launch_bounds__(256)
moe_combine_kernel(const float* __restrict__ y, int top, int D, float* __restrict__ x, int add_to, MllmStreamAdd add, int* __restrict__ counts, int E) {
    const int t = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * 4;
    if (t == 0 && blockIdx.x == 0)
        for (int e = threadIdx.x; e < E; e += 256) counts[e] = 0;
    if (c >= D) return;
    const float* row = y + static_cast<size_t>(t) * top * D + c;
    float* xr = x + static_cast<size_t>(t) * D + c;
    float4 old = make_float4(0.f, 0.f, 0.f, 0.f);
    if (add_to) old = *reinterpret_cast<const float4*>(xr);
    float4 sum = *reinterpret_cast<const float4*>(row);
    for (int j = 1; j < top; ++j) {
        const float4 more = *reinterpret_cast<const float4*>(row + static_cast<size_t>(j) * D);
        sum.x += more.x; sum.y += more.y; sum.z += more.z; sum.w += more.w;
    }
    float o[4] = {sum.x, sum.y, sum.z, sum.w};
    const bool has = add.norm.weight != nullptr, has_next = add.next.weight != nullptr;
    if (has) {
        const float a = add.norm.alpha[0];
        const float4 w = *reinterpret_cast<const float4*>(add.norm.weight + c), b = *reinterpret_cast<const float4*>(add.norm.bias + c);
        o[0] = fast_tanh(a * o[0]) * w.x + b.x; o[1] = fast_tanh(a * o[1]) * w.y + b.y; o[2] = fast_tanh(a * o[2]) * w.z + b.z; o[3] = fast_tanh(a * o[3]) * w.w + b.w;
    }
    o[0] += old.x; o[1] += old.y; o[2] += old.z; o[3] += old.w;
    *reinterpret_cast<float4*>(xr) = make_float4(o[0], o[1], o[2], o[3]);
    if (add.copy == nullptr) return;
    if (has_next) {
        const float a = add.next.alpha[0];
        const float4 w = *reinterpret_cast<const float4*>(add.next.weight + c), b = *reinterpret_cast<const float4*>(add.next.bias + c);
        o[0] = fast_tanh(a * o[0]) * w.x + b.x; o[1] = fast_tanh(a * o[1]) * w.y + b.y; o[2] = fast_tanh(a * o[2]) * w.z + b.z; o[3] = fast_tanh(a * o[3]) * w.w + b.w;
    }
    *reinterpret_cast<uint2*>(static_cast<bf16_t*>(add.copy) + static_cast<size_t>(t) * add.ld_copy + c) = make_uint2(pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3]));
}

}  // namespace

extern "C" {

// up [T, E * ff + shared_ff] in up_dtype and out of its shape in `dtype` (out may be up if the dtypes are one; otherwise up is
// fp32); logits [T, E + identity] fp32 (row stride ldl); weights_out (optional) [T, E + identity] fp32. gelu != 0: the exact
// GELU in place of the squared rectified value; correction (optional, [E + identity]), identity, h, y: see the kernel.
// -1: more experts than the kernel holds, or a `top` outside 1..E + identity, or identity experts without h and y.
int mllm_moe_act(const void* up, int ldu, const float* logits, int ldl, int E, int ff, int shared_ff, int top, float scale, void* out, int ldo,
                 float* weights_out, int ldw, int T, int dtype, hipStream_t stream, int up_dtype, int gelu, const float* correction,
                 int identity, const void* h, int ldh, int D, float* y, int ldy, int y_add) {
    if (T <= 0) return 0;
    if (up_dtype < 0) up_dtype = dtype;
    if (E < 1 || identity < 0 || E + identity > MOE_MAX_EXPERTS || top < 1 || top > E + identity || ff < 1 || shared_ff < 0 || logits == nullptr) return -1;
    if (identity > 0 && (h == nullptr || y == nullptr || D < 1)) return -1;
    if (up_dtype != dtype && !(up_dtype == MLLM_F32 && up != out)) return -1;
    const int N = E * ff + shared_ff;
    const int esz = dtype == MLLM_F32 ? 4 : 2, isz = up_dtype == MLLM_F32 ? 4 : 2;
    const bool vec = ff % 8 == 0 && N % 8 == 0 && ldo % 8 == 0 && ((reinterpret_cast<uintptr_t>(up) | reinterpret_cast<uintptr_t>(out)) & 15) == 0 &&
                     (static_cast<size_t>(ldu) * isz) % 16 == 0 && (static_cast<size_t>(ldo) * esz) % 16 == 0;
    const MoeChoice mc{correction, identity, h, ldh, D, ldy, y_add, y};
#define MOE_ACT(TI, TYPE, VEC, GELU)                                                                                                \
    moe_act_kernel<TI, TYPE, VEC, GELU><<<T, 256, 0, stream>>>(static_cast<const TI*>(up), ldu, logits, ldl, E, ff, N, top, scale,   \
                                                               static_cast<TYPE*>(out), ldo, weights_out, ldw, mc)
#define MOE_ACT_G(TI, TYPE)                                                                                                         \
    do {                                                                                                                            \
        if (gelu) { if (vec) MOE_ACT(TI, TYPE, true, true); else MOE_ACT(TI, TYPE, false, true); }                                  \
        else { if (vec) MOE_ACT(TI, TYPE, true, false); else MOE_ACT(TI, TYPE, false, false); }                                     \
    } while (0)
    if (dtype == MLLM_F32) MOE_ACT_G(float, float);
    else if (up_dtype == MLLM_F32) MOE_ACT_G(float, bf16_t);
    else MOE_ACT_G(bf16_t, bf16_t);
#undef MOE_ACT_G
#undef MOE_ACT
    MLLM_LAUNCH_CHECK();
    return 0;
}

// up [T, 2 (E * ff + shared_ff)] in up_dtype (`dtype`, or fp32) and out [T, E * ff + shared_ff] in `dtype`; logits [T, E (+ 1
// with shared_gate)] fp32; router_kind: 0 softmax, 1 sigmoid, 2 softmax over the chosen experts.
// -1: more experts than the kernel holds, a `top` outside 1..E, limits that are not positive, an unknown router_kind.
int mllm_moe_glu_act(const void* up, int ldu, const float* logits, int ldl, int E, int ff, int shared_ff, int top, float scale,
                     int router_kind, float limit, float shared_limit, float alpha, int weight_on_input, int shared_gate, void* out,
                     int ldo, int T, int dtype, hipStream_t stream, float up_shift, int up_dtype) {
    if (T <= 0) return 0;
    if (up_dtype < 0) up_dtype = dtype;
    if (E < 1 || E > MOE_MAX_EXPERTS || top < 1 || top > E || ff < 1 || shared_ff < 0 || logits == nullptr) return -1;
    if (!(limit > 0.f) || (shared_ff > 0 && !(shared_limit > 0.f)) || (shared_gate && shared_ff == 0)) return -1;
    if (router_kind < ROUTER_SOFTMAX || router_kind > ROUTER_SOFTMAX_CHOSEN || (up_dtype != dtype && up_dtype != MLLM_F32)) return -1;
    const int isz = up_dtype == MLLM_F32 ? 4 : 2;
    const bool vec = ff % 8 == 0 && shared_ff % 8 == 0 && ldo % 8 == 0 &&
                     ((reinterpret_cast<uintptr_t>(up) | reinterpret_cast<uintptr_t>(out)) & 15) == 0 && (static_cast<size_t>(ldu) * isz) % 16 == 0;
#define MOE_GLU_V(TI, TYPE, VEC, AHEAD)                                                                                                               \
    moe_glu_act_kernel<TI, TYPE, VEC, AHEAD><<<T, 256, 0, stream>>>(static_cast<const TI*>(up), ldu, logits, ldl, E, ff, shared_ff, top, scale, router_kind, \
                                                             limit, shared_limit, alpha, up_shift, weight_on_input, shared_gate, static_cast<TYPE*>(out), ldo)
#define MOE_GLU(TI, TYPE)                                                                                                                     \
    do {                                                                                                                                       \
        if (vec && T <= 64) MOE_GLU_V(TI, TYPE, true, true); else if (vec) MOE_GLU_V(TI, TYPE, true, false);                                     \
        else MOE_GLU_V(TI, TYPE, false, false);                                                                                                  \
    } while (0)
    if (dtype == MLLM_F32) MOE_GLU(float, float);
    else if (up_dtype == MLLM_F32) MOE_GLU(float, bf16_t);
    else MOE_GLU(bf16_t, bf16_t);
#undef MOE_GLU
#undef MOE_GLU_V
    MLLM_LAUNCH_CHECK();
    return 0;
}

// Gated experts by grouped products (bfloat16). h [T, D] (row stride ldh); logits [T, >= E] fp32; up [2 E ff, D]: expert e's gates
// and ups from row 2 ff e; down [D, E ff]: expert e's from column ff e. router_kind, scale, limit, alpha, up_shift as for
// mllm_moe_glu_act. Room: counts [E] ints, zero (and left zero); lists [E * T] ints, weights [T * top] floats, act [T * top, ff]
// bfloat16, y [T * top, D] fp32. x [T, D] fp32 is set to the result (add_to 0), or grows by it through `add` (add_to 1). -2: sizes
// these kernels do not take (the caller then multiplies densely); -1: operands that are not aligned.
int mllm_moe_grouped_glu(const void* h, int ldh, const float* logits, int ldl, int T, int D, int E, int ff, int top, float scale, int router_kind,
                         float limit, float alpha, float up_shift, const void* up, int ldu, const void* down, int ldd, int* counts, int* lists,
                         float* weights, void* act, float* y, float* x, int add_to, MllmStreamAdd add, hipStream_t stream) {
    if (T <= 0) return 0;
    if (E < 1 || E > MOE_MAX_EXPERTS || top < 1 || top > E || top > 8 || D % 8 != 0 || ff % 8 != 0 || T > 65535 || ldh % 8 != 0 || ldu % 8 != 0 || ldd % 8 != 0) return -2;
    const auto a16 = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
    if (!a16(h) || !a16(up) || !a16(down) || !a16(act) || !a16(y) || !a16(x) || (add.copy != nullptr && (add.ld_copy % 4 != 0 || (reinterpret_cast<uintptr_t>(add.copy) & 7)))) return -1;
    for (const MllmTanhNorm* n : {&add.norm, &add.next})
        if (n->weight != nullptr && (n->alpha == nullptr || n->bias == nullptr || !a16(n->weight) || !a16(n->bias))) return -1;
    if (router_kind < ROUTER_SOFTMAX || router_kind > ROUTER_SOFTMAX_CHOSEN || !(limit > 0.f)) return -1;
    const int tokens = E <= 128 ? 64 : 32;
    const size_t lds = static_cast<size_t>(tokens) * (E + 1) * 4 + static_cast<size_t>(2) * E * 4;
    moe_route_kernel<<<(T + tokens - 1) / tokens, 256, lds, stream>>>(logits, ldl, T, E, top, scale, router_kind, tokens, counts, lists, T, weights);
    MLLM_LAUNCH_CHECK();
    GroupedArgs g{};
    g.A = static_cast<const bf16_t*>(h); g.lda = ldh; g.W = static_cast<const bf16_t*>(up); g.ldw = ldu; g.ff = ff; g.N = 2 * ff; g.K = D; g.E = E;
    g.top = top; g.cap = T; g.counts = counts; g.lists = lists; g.weights = weights; g.act = static_cast<bf16_t*>(act); g.y = y; g.ld_out = ff;
    g.limit = limit; g.alpha = alpha; g.up_shift = up_shift;
    const int row_tiles = static_cast<int>((static_cast<long long>(T) * top) / MG_BM) + E;          // an upper bound
    moe_grouped_kernel<true><<<dim3(row_tiles, (ff + 63) / 64), 256, 0, stream>>>(g);
    MLLM_LAUNCH_CHECK();
    g.A = static_cast<const bf16_t*>(act); g.lda = ff; g.W = static_cast<const bf16_t*>(down); g.ldw = ldd; g.N = D; g.K = ff; g.ld_out = D;
    moe_grouped_kernel<false><<<dim3(row_tiles, (D + 127) / 128), 256, 0, stream>>>(g);
    MLLM_LAUNCH_CHECK();
    moe_combine_kernel<<<dim3((D + 1023) / 1024, T), 256, 0, stream>>>(y, top, D, x, add_to, add, counts, E);
    MLLM_LAUNCH_CHECK();
    return 0;
}

}  // extern "C"
