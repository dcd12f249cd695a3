// The dynamic tanh norm and the small kernels around it, for gfx950: the norm alone, a sub-layer's result added to the
// residual stream through it, something added to the whole stream, and a token's own gated input. Each also leaves, where
// asked, the bfloat16 rows that the next product reads (the new stream, or its norm). All arithmetic is fp32.
#include "common.h"

namespace {

// PRECISE (the 32-bit path): the library's tanh; otherwise one hardware exponential and a reciprocal (absolute error of
// the order of 1e-7).
template <bool PRECISE>
__device__ __forceinline__ float tanh_norm_of(float v, float alpha, float w, float b) {
    return (PRECISE ? tanhf(alpha * v) : fast_tanh(alpha * v)) * w + b;
}

// out[i, :] = norm(x[rows ? rows[i] : i, :]); a thread takes VEC consecutive columns.
template <typename T, int VEC>
__global__ void __launch_bounds__(256)
tanh_norm_kernel(const float* __restrict__ x, int ldx, const int* __restrict__ rows, MllmTanhNorm norm, T* __restrict__ out, int ldo, int D) {
    const int r = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * VEC;
    if (c >= D) return;
    const float* xr = x + static_cast<size_t>(rows ? rows[r] : r) * ldx + c;
    const float a = norm.alpha[0];
    T* o = out + static_cast<size_t>(r) * ldo + c;
    if (VEC == 4) {
        const float4 v = *reinterpret_cast<const float4*>(xr), w = *reinterpret_cast<const float4*>(norm.weight + c), b = *reinterpret_cast<const float4*>(norm.bias + c);
        constexpr bool P = sizeof(T) == 4;
        const float4 y = make_float4(tanh_norm_of<P>(v.x, a, w.x, b.x), tanh_norm_of<P>(v.y, a, w.y, b.y), tanh_norm_of<P>(v.z, a, w.z, b.z),
                                     tanh_norm_of<P>(v.w, a, w.w, b.w));
        if (P) *reinterpret_cast<float4*>(o) = y;
        else *reinterpret_cast<uint2*>(o) = make_uint2(pack_bf16x2(y.x, y.y), pack_bf16x2(y.z, y.w));
    } else {
        *o = from_float<T>(tanh_norm_of<sizeof(T) == 4>(*xr, a, norm.weight[c], norm.bias[c]));
    }
}

// x[r, c] += add.norm(y[r, c]) (y null: nothing) + x0[r, c] (null: nothing) + step[c] (null: nothing), and the copy.
template <bool PRECISE, int VEC>
__global__ void __launch_bounds__(256)
stream_add_kernel(float* __restrict__ x, const float* __restrict__ y, const float* __restrict__ x0, const float* __restrict__ step,
                  int D, MllmStreamAdd add) {
    const int r = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * VEC;
    if (c >= D) return;
    const size_t at = static_cast<size_t>(r) * D + c;
    float v[VEC];
#pragma unroll
    for (int u = 0; u < VEC; ++u) v[u] = x[at + u];
    if (y != nullptr) {
        const float a = add.norm.weight != nullptr ? add.norm.alpha[0] : 0.f;
#pragma unroll
        for (int u = 0; u < VEC; ++u) {
            const float yv = y[at + u];
            v[u] += add.norm.weight != nullptr ? tanh_norm_of<PRECISE>(yv, a, add.norm.weight[c + u], add.norm.bias[c + u]) : yv;
        }
    }
    if (x0 != nullptr) {
#pragma unroll
        for (int u = 0; u < VEC; ++u) v[u] += x0[at + u];
    }
    if (step != nullptr) {
#pragma unroll
        for (int u = 0; u < VEC; ++u) v[u] += step[c + u];
    }
#pragma unroll
    for (int u = 0; u < VEC; ++u) x[at + u] = v[u];
    if (add.copy == nullptr) return;
    if (add.next.weight != nullptr) {
        const float a = add.next.alpha[0];
#pragma unroll
        for (int u = 0; u < VEC; ++u) v[u] = tanh_norm_of<PRECISE>(v[u], a, add.next.weight[c + u], add.next.bias[c + u]);
    }
    bf16_t* o = static_cast<bf16_t*>(add.copy) + static_cast<size_t>(r) * add.ld_copy + c;
    if (VEC == 4) *reinterpret_cast<uint2*>(o) = make_uint2(pack_bf16x2(v[0], v[1 % VEC]), pack_bf16x2(v[2 % VEC], v[3 % VEC]));
    else o[0] = float_to_bf16(v[0]);
}

// out[t, j] = gelu_tanh(z[t, j]) * table[id(t), col0 + j]
template <typename T>
__global__ void __launch_bounds__(256)
token_gate_kernel(const float* __restrict__ z, int ldz, const int* __restrict__ ids, const int* __restrict__ src, const int* __restrict__ prev,
                  int n_prev, const T* __restrict__ table, int ldt, int col0, int dim, T* __restrict__ out, int ldo) {
    const int t = blockIdx.x;
    int id = ids[t];
    if (src != nullptr) {
        const int s = src[t];
        if (s >= 0 && s < n_prev) id = prev[s];
    }
    const T* e = table + static_cast<size_t>(id) * ldt + col0;
    for (int j = threadIdx.x; j < dim; j += blockDim.x) {
        const float v = z[static_cast<size_t>(t) * ldz + j];
        out[static_cast<size_t>(t) * ldo + j] = from_float<T>((sizeof(T) == 4 ? gelu_tanh_precise(v) : gelu_tanh(v)) * to_float(e[j]));
    }
}

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
#define SIDE_WAVES 16

// The token's own gated input in one kernel: for every token t of the workgroup's `rows` (up to 16), with e the dim columns
// from col0 on of the token's table row,
//   g = gelu_tanh(W_gate x_t) * e,  y = W_proj g,  x_t += y / sqrt(mean(y^2) + eps) * weight,
// and the copy (add.copy, add.next). Both maps come as 16 x 32 tiles in operand order ([tile of 16 rows][tile of 32 inputs][lane]
// [8]: lane l holds row l % 16, inputs 8 (l / 16) ..), so a wavefront's load is one kilobyte in a row; both are asked for at the
// start. The weights are the matrix cores' first operand: a lane then holds four consecutive columns of one token. The inputs of
// the first map (the stream, rounded to bfloat16) are dealt over the wavefronts, whose sums meet in LDS in the order of their
// index; of the second the columns are. The first map reads the stream from `xb`, its bfloat16 copy. DT: tiles of 16 over dim; KPW: tiles
// of 32 over the width a wavefront takes of the first map; CPW: tiles of 16 columns it takes of the second.
// SPLIT (few tokens): several workgroups (blockIdx.y) share a token's columns, 16 tiles each; every one works out the first map
// for itself, and the sum of squares comes from g alone, |W_proj g|^2 = g^T (W_proj^T W_proj) g, with that matrix in `gram`:
// fp32 operand tiles [tile of 16 rows][4 inputs][lane] (lane l: row l % 16, input l / 16).
template <int DT, int KPW, int CPW, bool SPLIT>
__global__ void __launch_bounds__(SIDE_WAVES * 64)
token_side_kernel(float* __restrict__ x, const bf16_t* __restrict__ xb, int T, int rows, int D, const bf16x8* __restrict__ gate,
                  const bf16x8* __restrict__ proj, const float* __restrict__ gram, const float* __restrict__ weight, float eps, const int* __restrict__ ids, const int* __restrict__ src,
                  const int* __restrict__ prev, int n_prev, const bf16_t* __restrict__ table, int ldt, int col0, int dim, MllmStreamAdd add) {
    constexpr int DIM = DT * 16, DK = (DIM + 31) / 32, GS = DK * 32 + 8, ZS = DIM + 4;
    // (wide streams: the second map's tiles are asked for behind the first map's products, whose registers they take)
    constexpr bool EARLY = KPW * (DT * 4 + 4) + CPW * (DK * 4 + 4) <= 96;
    static_assert(!SPLIT || CPW == 1, "shared columns: one tile a wavefront");
    constexpr int GU = DT == 4 ? 4 : 1;              // products of g with gram a wavefront takes (DT 1: four wavefronts have one)
    __shared__ __attribute__((aligned(16))) float z_s[SIDE_WAVES][ZS * 16];
    __shared__ __attribute__((aligned(16))) bf16_t g_s[16 * GS];
    __shared__ float ss_s[SIDE_WAVES][16];
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid / 64), lane = tid % 64, tok = lane % 16, q = lane / 16;
    const int first = blockIdx.x * rows, n_rows = min(rows, T - first), KB = D / 32, CB = D / 16;
    const size_t row_at = static_cast<size_t>(first + min(tok, n_rows - 1)) * D;          // (tokens that are not there: the last one, never stored)
    // everything the kernel reads is asked for here: the first map's tiles with the stream, then the table's columns, the
    // second map's tiles and the stream again as the result is laid out
    bf16x8 wg[KPW][DT];
    bf16x8 xa[KPW];
#pragma unroll
    for (int u = 0; u < KPW; ++u) {
        const int kb = min(wave + SIDE_WAVES * u, KB - 1);
        xa[u] = *reinterpret_cast<const bf16x8*>(xb + row_at + kb * 32 + 8 * q);
#pragma unroll
        for (int d = 0; d < DT; ++d) wg[u][d] = gate[(static_cast<size_t>(d) * KB + kb) * 64 + lane];
    }
    // thread -> (token, column of dim) for the step between the maps
    const int e_tok = tid / DIM, e_col = tid % DIM;
    float e_val = 0.f;
    {
        const int t = first + min(min(e_tok, 15), n_rows - 1);
        int id = ids[t];
        if (src != nullptr) {
            const int s = src[t];
            if (s >= 0 && s < n_prev) id = prev[s];
        }
        e_val = to_float(table[static_cast<size_t>(id) * ldt + col0 + min(e_col, dim - 1)]);
    }
    bf16x8 wp[CPW][DK];
    float4 xv[CPW];
    auto fetch_second = [&]() {
#pragma unroll
        for (int c = 0; c < CPW; ++c) {
            const int cb = min(static_cast<int>(blockIdx.y) * SIDE_WAVES + wave + SIDE_WAVES * c, CB - 1);
#pragma unroll
            for (int k = 0; k < DK; ++k) wp[c][k] = proj[(static_cast<size_t>(cb) * DK + k) * 64 + lane];
            xv[c] = *reinterpret_cast<const float4*>(x + row_at + cb * 16 + 4 * q);
        }
        __builtin_amdgcn_sched_barrier(0);
    };
    if (EARLY) fetch_second();
    // (SPLIT: the end's vectors and this wavefront's tiles of gram: row tile, first of its steps of four inputs)
    const int g_row = DT == 1 ? 0 : wave % DT, g_step = DT == 4 ? (wave / 4) * 4 : wave / DT;
    float gm[GU];
    float4 w_first = make_float4(0.f, 0.f, 0.f, 0.f), nw_first = w_first, nb_first = w_first;
    if constexpr (SPLIT) {
#pragma unroll
        for (int u = 0; u < GU; ++u) gm[u] = gram[(static_cast<size_t>(g_row) * (DT * 4) + min(g_step + u, DT * 4 - 1)) * 64 + lane];
        const int n = min(static_cast<int>(blockIdx.y) * SIDE_WAVES + wave, CB - 1) * 16 + 4 * q;
        w_first = *reinterpret_cast<const float4*>(weight + n);
        if (add.copy != nullptr && add.next.weight != nullptr) {
            nw_first = *reinterpret_cast<const float4*>(add.next.weight + n);
            nb_first = *reinterpret_cast<const float4*>(add.next.bias + n);
        }
        __builtin_amdgcn_sched_barrier(0);
    }
    f32x4 acc[DT];
#pragma unroll
    for (int d = 0; d < DT; ++d) acc[d] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int u = 0; u < KPW; ++u) {
        if (wave + SIDE_WAVES * u >= KB) continue;
#pragma unroll
        for (int d = 0; d < DT; ++d) acc[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wg[u][d], xa[u], acc[d], 0, 0, 0);
    }
    // (register r of lane l: column of dim 4 (l / 16) + r, token l % 16)
#pragma unroll
    for (int d = 0; d < DT; ++d) *reinterpret_cast<f32x4*>(&z_s[wave][tok * ZS + d * 16 + 4 * q]) = acc[d];
    if (!EARLY) fetch_second();
    for (int i = tid; i < 16 * GS; i += SIDE_WAVES * 64) g_s[i] = float_to_bf16(0.f);
    lds_barrier();
    if (tid < DIM * 16) {
        float z = 0.f;
#pragma unroll
        for (int w = 0; w < SIDE_WAVES; ++w) z += z_s[w][e_tok * ZS + e_col];
        if (e_col < dim) g_s[e_tok * GS + e_col] = float_to_bf16(gelu_tanh(z) * e_val);
    }
    lds_barrier();
    bf16x8 gb[DK];
#pragma unroll
    for (int k = 0; k < DK; ++k) gb[k] = *reinterpret_cast<const bf16x8*>(g_s + tok * GS + k * 32 + 8 * q);
    f32x4 y[CPW];
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < CPW; ++c) {
        y[c] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < DK; ++k) y[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wp[c][k], gb[k], y[c], 0, 0, 0);
        if (!SPLIT && wave + SIDE_WAVES * c < CB) ss += y[c][0] * y[c][0] + y[c][1] * y[c][1] + y[c][2] * y[c][2] + y[c][3] * y[c][3];
    }
    if constexpr (SPLIT) {
        f32x4 t = f32x4{0.f, 0.f, 0.f, 0.f};
        const bool has = DT > 1 || wave < 4;
#pragma unroll
        for (int u = 0; u < GU; ++u)
            t = __builtin_amdgcn_mfma_f32_16x16x4f32(gm[u], to_float(g_s[tok * GS + 4 * (has ? g_step + u : 0) + q]), t, 0, 0, 0);
        // (register r: row 16 g_row + 4 q + r of gram g, of token `tok`)
#pragma unroll
        for (int r = 0; r < 4; ++r) ss += has ? t[r] * to_float(g_s[tok * GS + 16 * g_row + 4 * q + r]) : 0.f;
    }
    ss = rows_sum(ss);
    if (lane < 16) ss_s[wave][lane] = ss;
    lds_barrier();
    float total = 0.f;
#pragma unroll
    for (int w = 0; w < SIDE_WAVES; ++w) total += ss_s[w][tok];
    const float inv = 1.f / sqrtf(fmaxf(total, 0.f) / static_cast<float>(D) + eps);
    if (tok >= n_rows) return;
    const bool has_next = add.next.weight != nullptr;
    const float alpha = has_next ? add.next.alpha[0] : 0.f;
#pragma unroll
    for (int c = 0; c < CPW; ++c) {
        const int cb = static_cast<int>(blockIdx.y) * SIDE_WAVES + wave + SIDE_WAVES * c;
        if (cb >= CB) continue;
        const int n = cb * 16 + 4 * q;
        const float4 w4 = SPLIT ? w_first : *reinterpret_cast<const float4*>(weight + n);
        float o[4] = {xv[c].x + y[c][0] * inv * w4.x, xv[c].y + y[c][1] * inv * w4.y, xv[c].z + y[c][2] * inv * w4.z, xv[c].w + y[c][3] * inv * w4.w};
        *reinterpret_cast<float4*>(x + row_at + n) = make_float4(o[0], o[1], o[2], o[3]);
        if (add.copy == nullptr) continue;
        if (has_next) {
            const float4 nw = SPLIT ? nw_first : *reinterpret_cast<const float4*>(add.next.weight + n), nb = SPLIT ? nb_first : *reinterpret_cast<const float4*>(add.next.bias + n);
            o[0] = fast_tanh(alpha * o[0]) * nw.x + nb.x; o[1] = fast_tanh(alpha * o[1]) * nw.y + nb.y;
            o[2] = fast_tanh(alpha * o[2]) * nw.z + nb.z; o[3] = fast_tanh(alpha * o[3]) * nw.w + nb.w;
        }
        *reinterpret_cast<uint2*>(static_cast<bf16_t*>(add.copy) + static_cast<size_t>(first + tok) * add.ld_copy + n) =
            make_uint2(pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3]));
    }
}

bool on16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }
bool norm_on16(const MllmTanhNorm& n) { return n.weight == nullptr || (on16(n.weight) && on16(n.bias)); }

}  // namespace

extern "C" {

// x fp32 [.., D] (row stride ldx), out [n, D] in `dtype` (row stride ldo). -1: a norm without its three tensors.
int mllm_tanh_norm(const float* x, int ldx, const int* rows, MllmTanhNorm norm, void* out, int ldo, int n, int D, int dtype, hipStream_t stream) {
    if (n <= 0 || D <= 0) return 0;
    if (norm.alpha == nullptr || norm.weight == nullptr || norm.bias == nullptr || n > 65535 * 16) return -1;
    const bool vec = D % 4 == 0 && ldx % 4 == 0 && ldo % 4 == 0 && on16(x) && on16(out) && norm_on16(norm);
    for (int first = 0; first < n; first += 65535) {
        // (a grid holds 65,535 rows)
        const int m = n - first < 65535 ? n - first : 65535;
        const int* rw = rows ? rows + first : nullptr;
        const float* xs = rows ? x : x + static_cast<size_t>(first) * ldx;
        const dim3 grid((D + (vec ? 1023 : 255)) / (vec ? 1024 : 256), m);
#define TANH_NORM(T, V) tanh_norm_kernel<T, V><<<grid, 256, 0, stream>>>(xs, ldx, rw, norm, static_cast<T*>(out) + static_cast<size_t>(first) * ldo, ldo, D)
        if (dtype == MLLM_F32) { if (vec) TANH_NORM(float, 4); else TANH_NORM(float, 1); }
        else { if (vec) TANH_NORM(bf16_t, 4); else TANH_NORM(bf16_t, 1); }
#undef TANH_NORM
    }
    MLLM_LAUNCH_CHECK();
    return 0;
}

// x fp32 [n, D] contiguous; y, x0 (optional) of its shape, step (optional) [D]. precise != 0: the library's tanh.
int mllm_stream_add(float* x, const float* y, const float* x0, const float* step, int n, int D, MllmStreamAdd add, int precise, hipStream_t stream) {
    if (n <= 0 || D <= 0) return 0;
    const bool vec = D % 4 == 0 && on16(x) && (y == nullptr || on16(y)) && (x0 == nullptr || on16(x0)) && (step == nullptr || on16(step)) &&
                     norm_on16(add.norm) && norm_on16(add.next) && (add.copy == nullptr || (add.ld_copy % 4 == 0 && (reinterpret_cast<uintptr_t>(add.copy) & 7) == 0));
    for (int first = 0; first < n; first += 65535) {
        const int m = n - first < 65535 ? n - first : 65535;
        const size_t off = static_cast<size_t>(first) * D;
        MllmStreamAdd a = add;
        if (a.copy != nullptr) a.copy = static_cast<bf16_t*>(a.copy) + static_cast<size_t>(first) * a.ld_copy;
        const dim3 grid((D + (vec ? 1023 : 255)) / (vec ? 1024 : 256), m);
#define STREAM_ADD(P, V) stream_add_kernel<P, V><<<grid, 256, 0, stream>>>(x + off, y ? y + off : nullptr, x0 ? x0 + off : nullptr, step, D, a)
        if (precise) { if (vec) STREAM_ADD(true, 4); else STREAM_ADD(true, 1); }
        else { if (vec) STREAM_ADD(false, 4); else STREAM_ADD(false, 1); }
#undef STREAM_ADD
    }
    MLLM_LAUNCH_CHECK();
    return 0;
}

// z fp32 [T, dim] (row stride ldz); ids [T], and with `src`: where src[t] is in [0, n_prev), token t's id is prev[src[t]];
// table [vocab, ldt] and out [T, dim] in `dtype`.
int mllm_token_gate(const float* z, int ldz, const int* ids, const int* src, const int* prev, int n_prev, const void* table, int ldt, int col0,
                    int dim, void* out, int ldo, int T, int dtype, hipStream_t stream) {
    if (T <= 0 || dim <= 0) return 0;
    if (ids == nullptr || (src != nullptr && prev == nullptr)) return -1;
    const int threads = dim <= 64 ? 64 : (dim <= 128 ? 128 : 256);
    if (dtype == MLLM_F32)
        token_gate_kernel<float><<<T, threads, 0, stream>>>(z, ldz, ids, src, prev, n_prev, static_cast<const float*>(table), ldt, col0, dim, static_cast<float*>(out), ldo);
    else
        token_gate_kernel<bf16_t><<<T, threads, 0, stream>>>(z, ldz, ids, src, prev, n_prev, static_cast<const bf16_t*>(table), ldt, col0, dim, static_cast<bf16_t*>(out), ldo);
    MLLM_LAUNCH_CHECK();
    return 0;
}

// The sizes token_side_kernel is built for: a width of up to 2,048 in whole tiles of 32, up to 64 columns a token.
int mllm_token_side_fits(int D, int dim) { return D >= 32 && D % 32 == 0 && D <= 2048 && dim >= 1 && dim <= 64 ? 1 : 0; }

// x fp32 [T, D] contiguous; gate and proj bfloat16 in tiles (see the kernel; dim filled up with zeros to a multiple of 16 in the
// gate's rows and of 32 in proj's inputs); xb: the stream's bfloat16 copy [T, D], which add.copy must not be; gram: see the kernel;
// weight [D]; ids, src, prev, table as for mllm_token_gate. Tokens up to
// 2,048 take 8 a workgroup, more take 16. -2: sizes the kernel is not built for; -1: operands that are not aligned.
int mllm_token_side(float* x, const void* xb, int T, int D, const void* gate, const void* proj, const float* gram, const float* weight, float eps, const int* ids, const int* src,
                    const int* prev, int n_prev, const void* table, int ldt, int col0, int dim, MllmStreamAdd add, hipStream_t stream) {
    if (T <= 0) return 0;
    if (!mllm_token_side_fits(D, dim)) return -2;
    if (ids == nullptr || (src != nullptr && prev == nullptr) || !on16(x) || !on16(xb) || xb == add.copy || gram == nullptr || !on16(gate) || !on16(proj) || !on16(weight) || !norm_on16(add.next) ||
        (add.copy != nullptr && (add.ld_copy % 4 != 0 || (reinterpret_cast<uintptr_t>(add.copy) & 7))))
        return -1;
    const int rows = T <= 2048 ? 8 : 16, blocks = (T + rows - 1) / rows;
    const int dt = dim <= 16 ? 1 : (dim <= 32 ? 2 : 4), kpw = D <= 512 ? 1 : (D <= 1024 ? 2 : 4), parts = (D / 16 + SIDE_WAVES - 1) / SIDE_WAVES;
    const bool split = blocks * parts <= 128;
#define TOKEN_SIDE(DT, KPW, CPW, SPLIT)                                                                                                 \
    token_side_kernel<DT, KPW, CPW, SPLIT><<<dim3(blocks, SPLIT ? parts : 1), SIDE_WAVES * 64, 0, stream>>>(x, static_cast<const bf16_t*>(xb), T, rows, D, \
        static_cast<const bf16x8*>(gate), static_cast<const bf16x8*>(proj), gram, weight, eps, ids, src, prev, n_prev,                  \
        static_cast<const bf16_t*>(table), ldt, col0, dim, add)
#define TOKEN_SIDE_K(DT, KPW, CPW) do { if (split) TOKEN_SIDE(DT, KPW, 1, true); else TOKEN_SIDE(DT, KPW, CPW, false); } while (0)
#define TOKEN_SIDE_D(DT) do { if (kpw == 1) TOKEN_SIDE_K(DT, 1, 2); else if (kpw == 2) TOKEN_SIDE_K(DT, 2, 4); else TOKEN_SIDE_K(DT, 4, 8); } while (0)
    if (dt == 1) TOKEN_SIDE_D(1);
    else if (dt == 2) TOKEN_SIDE_D(2);
    else TOKEN_SIDE_D(4);
#undef TOKEN_SIDE_D
#undef TOKEN_SIDE_K
#undef TOKEN_SIDE
    MLLM_LAUNCH_CHECK();
    return 0;
}

}  // extern "C"
