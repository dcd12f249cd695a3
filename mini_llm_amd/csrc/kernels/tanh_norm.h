// The dynamic tanh norm, n(v) = tanh(alpha v) * weight + bias (alpha one number, weight and bias per column): no
// statistics, so it can stand inside any kernel that holds a value of the row. And what such a kernel does to the residual
// stream where a sub-layer's result arrives. Plain structures, shared by the kernels and the engine's dispatch.
#pragma once

struct MllmTanhNorm {
    const float* alpha;      // one number, on the device
    const float* weight;     // [columns]; null: no norm
    const float* bias;       // [columns]
};

// x <- x + norm(y) for a result y (with norm.weight null: x <- x + y); then, with `copy` (bfloat16 rows of ld_copy
// elements), copy <- next(x), or x itself if next.weight is null.
struct MllmStreamAdd {
    MllmTanhNorm norm, next;
    void* copy;
    int ld_copy;
};
