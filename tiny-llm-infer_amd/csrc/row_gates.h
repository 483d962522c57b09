// Gates of recurrent layers, one number a row and head, made from float32 sums.
#pragma once
#include "common.h"

// The factor of a row whose norm is still owed to the products that read it: 1 / sqrt(sum of squares / n + eps), the
// sum of squares in `parts` parts [parts][rows].  parts 0: 1.
struct RowFactor {
    const float* ssq;
    int parts, rows;
    float inv_n, eps;
    __device__ __forceinline__ float of_sum(float sum) const { return 1.0f / sqrtf(sum * inv_n + eps); }
    __device__ __forceinline__ float of(int row) const {
        if (parts <= 0) return 1.f;
        float sum = 0.f;
        for (int p = 0; p < parts; ++p) sum += ssq[(size_t)p * rows + row];
        return of_sum(sum);
    }
};

__device__ __forceinline__ float gate_capped(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float gate_log_sigmoid(float u) { return fminf(u, 0.f) - log1pf(expf(-fabsf(u))); }
