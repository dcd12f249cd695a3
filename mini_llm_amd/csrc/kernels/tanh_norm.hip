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

}  // extern "C"
