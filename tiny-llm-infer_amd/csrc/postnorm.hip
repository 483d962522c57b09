// The residual of a block that norms what a sublayer gives:  x <- x + w * y / sqrt(mean(y^2) + eps).
//
// norm_add:       one workgroup a row: the sublayer's output y (the run's type) is read once into registers,
//                 its mean square summed in float32, the normed row added to the float32 residual, and the
//                 new residual written in the run's type for the next sublayer to read.
// norm_add_norm:  the same with the norm of whoever reads the sum next in the same pass: h = w2 * x / sqrt(mean(x^2) + eps2)
//                 is written instead of x's own rows.  Without y: that norm alone;
//                 without w2: x's own rows.  y may come as float32 partial sums of a product, which are added in order and
//                 rounded as the product would have.  With `rows` only those rows of the
//                 residual are looked at, and it is not written.  With mixes (steps of one row a sequence): h' being the row
//                 that the sequence's slot keeps (zeros at position 0), h + (h' - h) mu_m for every m is written instead, and
//                 h replaces the kept row.
// token_mixes:    those mixes from rows h of portions: h' is the row before in the same sequence.
// residual_rows:  the residual's rows in the run's type (what the first block reads).
#include "common.h"

#define PN_THREADS 256
#define PN_MAX_PER_THREAD 32          // rows of up to 8192 elements stay in registers

template <typename T>
__global__ __launch_bounds__(PN_THREADS) void norm_add_kernel(float* __restrict__ resid, const T* __restrict__ y,
                                                                const float* __restrict__ weight, T* __restrict__ rows_out,
                                                                int n, float eps) {
    __shared__ float red[16];
    const size_t row = blockIdx.x;
    const T* yr = y + row * n;
    float v[PN_MAX_PER_THREAD];
    float ssq = 0.f;
#pragma unroll
    for (int i = 0; i < PN_MAX_PER_THREAD; ++i) {
        const int c = i * PN_THREADS + threadIdx.x;
        v[i] = c < n ? to_f32(yr[c]) : 0.f;
        ssq = fmaf(v[i], v[i], ssq);
    }
    // (beyond what the registers hold: read again below)
    for (int c = PN_MAX_PER_THREAD * PN_THREADS + threadIdx.x; c < n; c += PN_THREADS) {
        const float a = to_f32(yr[c]);
        ssq = fmaf(a, a, ssq);
    }
    const float factor = 1.0f / sqrtf(block_sum(ssq, red) / (float)n + eps);
    float* xr = resid + row * n;
#pragma unroll
    for (int i = 0; i < PN_MAX_PER_THREAD; ++i) {
        const int c = i * PN_THREADS + threadIdx.x;
        if (c < n) {
            const float x = xr[c] + v[i] * factor * weight[c];
            xr[c] = x;
            if (rows_out) from_f32(rows_out + row * n + c, x);
        }
    }
    for (int c = PN_MAX_PER_THREAD * PN_THREADS + threadIdx.x; c < n; c += PN_THREADS) {
        const float x = xr[c] + to_f32(yr[c]) * factor * weight[c];
        xr[c] = x;
        if (rows_out) from_f32(rows_out + row * n + c, x);
    }
}

// The same for bfloat16 rows whose length is a multiple of 8, up to 8192: 16-byte accesses, eight elements a
// thread and round.
#define PN_VEC_ROUNDS 4
__global__ __launch_bounds__(PN_THREADS) void norm_add_vec_kernel(float* __restrict__ resid, const bf16_t* __restrict__ y,
                                                                   const float* __restrict__ weight, bf16_t* __restrict__ rows_out,
                                                                   int n, float eps) {
    __shared__ float red[16];
    const size_t row = blockIdx.x;
    const bf16_t* yr = y + row * n;
    uint4 v[PN_VEC_ROUNDS];
    float ssq = 0.f;
#pragma unroll
    for (int i = 0; i < PN_VEC_ROUNDS; ++i) {
        const int c = (i * PN_THREADS + threadIdx.x) * 8;
        v[i] = make_uint4(0, 0, 0, 0);
        if (c < n) v[i] = *reinterpret_cast<const uint4*>(yr + c);
        const uint32_t w[4] = {v[i].x, v[i].y, v[i].z, v[i].w};
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const float a = __uint_as_float(w[e] << 16), b = __uint_as_float(w[e] & 0xFFFF0000u);
            ssq = fmaf(a, a, ssq);
            ssq = fmaf(b, b, ssq);
        }
    }
    const float factor = 1.0f / sqrtf(block_sum(ssq, red) / (float)n + eps);
    float* xr = resid + row * n;
#pragma unroll
    for (int i = 0; i < PN_VEC_ROUNDS; ++i) {
        const int c = (i * PN_THREADS + threadIdx.x) * 8;
        if (c < n) {
            const uint32_t w[4] = {v[i].x, v[i].y, v[i].z, v[i].w};
            float x[8];
            *reinterpret_cast<float4*>(x) = *reinterpret_cast<const float4*>(xr + c);
            *reinterpret_cast<float4*>(x + 4) = *reinterpret_cast<const float4*>(xr + c + 4);
            float g[8];
            *reinterpret_cast<float4*>(g) = *reinterpret_cast<const float4*>(weight + c);
            *reinterpret_cast<float4*>(g + 4) = *reinterpret_cast<const float4*>(weight + c + 4);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                x[2 * e] += __uint_as_float(w[e] << 16) * factor * g[2 * e];
                x[2 * e + 1] += __uint_as_float(w[e] & 0xFFFF0000u) * factor * g[2 * e + 1];
            }
            *reinterpret_cast<float4*>(xr + c) = *reinterpret_cast<const float4*>(x);
            *reinterpret_cast<float4*>(xr + c + 4) = *reinterpret_cast<const float4*>(x + 4);
            if (rows_out) {
                uint4 st;
                st.x = pack_bf16x2(x[0], x[1]);
                st.y = pack_bf16x2(x[2], x[3]);
                st.z = pack_bf16x2(x[4], x[5]);
                st.w = pack_bf16x2(x[6], x[7]);
                *reinterpret_cast<uint4*>(rows_out + row * n + c) = st;
            }
        }
    }
}

struct MixArgs {
    const float* mu;             // [mixes][n], or null: no mixes
    int mixes;
    void* kept;                  // [slots][n] in the rows' type
    const int* slots;            // [seqs]
    const int* seq_start;        // [seqs]
    size_t stride;               // elements between two mixes of the output
};

// h + (h' - h) mu_m for all m; V elements from column c on, of row `row`
template <typename T, int V>
__device__ __forceinline__ void put_mixes(const float (&h)[V], const float (&prev)[V], const MixArgs& mix, T* __restrict__ out,
                                          size_t at, int c, int n) {
    for (int m = 0; m < mix.mixes; ++m) {
        const float* mu = mix.mu + (size_t)m * n + c;
        T* dst = out + (size_t)m * mix.stride + at;
        float o[V];
#pragma unroll
        for (int e = 0; e < V; ++e) o[e] = h[e] + (prev[e] - h[e]) * mu[e];
        if constexpr (V == 8 && sizeof(T) == 2)
            *reinterpret_cast<uint4*>(dst) = make_uint4(pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3]), pack_bf16x2(o[4], o[5]), pack_bf16x2(o[6], o[7]));
        else
#pragma unroll
            for (int e = 0; e < V; ++e) from_f32(dst + e, o[e]);
    }
}

// V elements of a row as float32: 1, or 8 of an aligned row
template <typename T, int V>
__device__ __forceinline__ void row_load(const T* p, float (&v)[V]) {
    if constexpr (V == 8 && sizeof(T) == 2) {
        const uint4 u = *reinterpret_cast<const uint4*>(p);
        const uint32_t w[4] = {u.x, u.y, u.z, u.w};
#pragma unroll
        for (int e = 0; e < 4; ++e) v[2 * e] = __uint_as_float(w[e] << 16), v[2 * e + 1] = __uint_as_float(w[e] & 0xFFFF0000u);
    } else if constexpr (V == 8) {
        *reinterpret_cast<float4*>(v) = *reinterpret_cast<const float4*>(p);
        *reinterpret_cast<float4*>(v + 4) = *reinterpret_cast<const float4*>(p + 4);
    } else {
        v[0] = to_f32(*p);
    }
}
template <typename T, int V>
__device__ __forceinline__ void row_store(T* p, const float (&v)[V]) {
    if constexpr (V == 8 && sizeof(T) == 2) {
        *reinterpret_cast<uint4*>(p) = make_uint4(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]), pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7]));
    } else if constexpr (V == 8) {
        *reinterpret_cast<float4*>(p) = *reinterpret_cast<const float4*>(v);
        *reinterpret_cast<float4*>(p + 4) = *reinterpret_cast<const float4*>(v + 4);
    } else {
        from_f32(p, v[0]);
    }
}

// ROUNDS x PN_THREADS x V elements of a row are kept in registers between the sums; a row is no longer than that.
template <typename T, int V, int ROUNDS>
__global__ __launch_bounds__(PN_THREADS) void norm_add_norm_kernel(float* __restrict__ resid, const T* __restrict__ y,
                                                                    const float* __restrict__ sums, int parts, size_t plane,
                                                                    const float* __restrict__ w1, float eps1,
                                                                    const float* __restrict__ w2, float eps2, T* __restrict__ out,
                                                                    const int* __restrict__ rows, int n, MixArgs mix) {
    __shared__ float red[16];
    const size_t row = rows ? rows[blockIdx.x] : blockIdx.x;
    float* xr = resid + row * n;
    float v[ROUNDS][V], x[ROUNDS][V], g1[ROUNDS][V], g2[ROUNDS][V];
    float ssq = 0.f;
    const bool add = y || parts > 0;
    // everything but the mixes' weights is asked for before the first sum is taken
#pragma unroll
    for (int i = 0; i < ROUNDS; ++i) {
        const int c = (i * PN_THREADS + threadIdx.x) * V;
#pragma unroll
        for (int e = 0; e < V; ++e) v[i][e] = x[i][e] = g1[i][e] = g2[i][e] = 0.f;
        if (c < n) {
            if (y) row_load<T, V>(y + row * n + c, v[i]);
            for (int p = 0; p < parts; ++p) {
                float a[V];
                row_load<float, V>(sums + p * plane + row * n + c, a);
#pragma unroll
                for (int e = 0; e < V; ++e) v[i][e] += a[e];
            }
            if constexpr (sizeof(T) == 2) {
                if (parts > 0) {
#pragma unroll
                    for (int e = 0; e < V; ++e) v[i][e] = bf16_to_f32(f32_to_bf16(v[i][e]));
                }
            }
            row_load<float, V>(xr + c, x[i]);
            if (add) row_load<float, V>(w1 + c, g1[i]);
            if (w2) row_load<float, V>(w2 + c, g2[i]);
        }
#pragma unroll
        for (int e = 0; e < V; ++e) ssq = fmaf(v[i][e], v[i][e], ssq);
    }
    if (add) {
        const float factor = 1.0f / sqrtf(block_sum(ssq, red) / (float)n + eps1);
#pragma unroll
        for (int i = 0; i < ROUNDS; ++i) {
            const int c = (i * PN_THREADS + threadIdx.x) * V;
            if (c >= n) continue;
#pragma unroll
            for (int e = 0; e < V; ++e) x[i][e] += v[i][e] * factor * g1[i][e];
            if (!rows) row_store<float, V>(xr + c, x[i]);
            if (!w2 && out) row_store<T, V>(out + (size_t)blockIdx.x * n + c, x[i]);
        }
    }
    if (!w2) return;
    T* kept = nullptr;
    bool fresh = true;
    if (mix.mu) {
        kept = (T*)mix.kept + (size_t)mix.slots[row] * n;
        fresh = mix.seq_start[row] <= 0;
#pragma unroll
        for (int i = 0; i < ROUNDS; ++i) {           // (v now holds the kept row)
            const int c = (i * PN_THREADS + threadIdx.x) * V;
#pragma unroll
            for (int e = 0; e < V; ++e) v[i][e] = 0.f;
            if (c < n && !fresh) row_load<T, V>(kept + c, v[i]);
        }
    }
    ssq = 0.f;
#pragma unroll
    for (int i = 0; i < ROUNDS; ++i)
#pragma unroll
        for (int e = 0; e < V; ++e) ssq = fmaf(x[i][e], x[i][e], ssq);
    const float factor = 1.0f / sqrtf(block_sum(ssq, red) / (float)n + eps2);
#pragma unroll
    for (int i = 0; i < ROUNDS; ++i) {
        const int c = (i * PN_THREADS + threadIdx.x) * V;
        if (c >= n) continue;
        float h[V];
#pragma unroll
        for (int e = 0; e < V; ++e) h[e] = x[i][e] * factor * g2[i][e];
        if (!mix.mu) {
            row_store<T, V>(out + (size_t)blockIdx.x * n + c, h);
            continue;
        }
        if constexpr (sizeof(T) == 2) {             // h as it is kept: the mixes are made of rounded rows
#pragma unroll
            for (int e = 0; e < V; ++e) h[e] = bf16_to_f32(f32_to_bf16(h[e]));
        }
        row_store<T, V>(kept + c, h);
        put_mixes<T, V>(h, v[i], mix, out, row * n + c, c, n);
    }
}

template <typename T, int V>
__global__ __launch_bounds__(PN_THREADS) void token_mixes_kernel(const T* __restrict__ h, T* __restrict__ out, const int* __restrict__ seq_of_row,
                                                                 const int* __restrict__ row_start, int n, MixArgs mix) {
    const int row = blockIdx.x;
    const int seq = seq_of_row[row], first = row_start[seq], last = row_start[seq + 1] - 1;
    // the workgroup of a sequence's first row, having read the kept row, replaces it: each element is read and
    // written by the same thread
    T* kept = row == first ? (T*)mix.kept + (size_t)mix.slots[seq] * n : nullptr;
    const bool fresh = row == first && mix.seq_start[seq] <= 0;
    for (int c = threadIdx.x * V; c < n; c += PN_THREADS * V) {
        float cur[V], prev[V];
        row_load<T, V>(h + (size_t)row * n + c, cur);
#pragma unroll
        for (int e = 0; e < V; ++e) prev[e] = 0.f;
        if (!fresh) row_load<T, V>(kept ? kept + c : h + (size_t)(row - 1) * n + c, prev);
        if (kept) {
            float end[V];
            row_load<T, V>(h + (size_t)last * n + c, end);
            row_store<T, V>(kept + c, end);
        }
        put_mixes<T, V>(cur, prev, mix, out, (size_t)row * n + c, c, n);
    }
}

__global__ void residual_rows_kernel(const float* __restrict__ resid, bf16_t* __restrict__ out, long long count) {
    const long long i = ((long long)blockIdx.x * blockDim.x + threadIdx.x) * 4;
    if (i + 3 < count) {
        const float4 v = *reinterpret_cast<const float4*>(resid + i);
        uint2 st;
        st.x = pack_bf16x2(v.x, v.y);
        st.y = pack_bf16x2(v.z, v.w);
        *reinterpret_cast<uint2*>(out + i) = st;
    } else {
        for (long long j = i; j < count; ++j) out[j] = f32_to_bf16(resid[j]);
    }
}

// resid [rows, n] float32 += weight * y / rms(y);  rows_out [rows, n] in the type of y (may be null for float32, where
// the residual itself is what the next sublayer reads)
extern "C" int tli_norm_add(float* resid, const void* y, const float* weight, void* rows_out, int rows, int n, float eps,
                            int dtype, void* stream) {
    if (rows <= 0) return 0;
    if (n <= 0) return tli_fail("norm_add: bad row length %d", n);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == TLI_F32)
        norm_add_kernel<float><<<rows, PN_THREADS, 0, s>>>(resid, (const float*)y, weight, (float*)rows_out, n, eps);
    else if (dtype == TLI_BF16 && n % 8 == 0 && n <= 8 * PN_THREADS * PN_VEC_ROUNDS &&
             !(((uintptr_t)resid | (uintptr_t)y | (uintptr_t)weight | (uintptr_t)rows_out) & 15))
        norm_add_vec_kernel<<<rows, PN_THREADS, 0, s>>>(resid, (const bf16_t*)y, weight, (bf16_t*)rows_out, n, eps);
    else if (dtype == TLI_BF16)
        norm_add_kernel<bf16_t><<<rows, PN_THREADS, 0, s>>>(resid, (const bf16_t*)y, weight, (bf16_t*)rows_out, n, eps);
    else
        return tli_fail("norm_add: unknown dtype %d", dtype);
    return tli_check_launch("norm_add");
}

extern "C" int tli_residual_rows(const float* resid, void* out, long long count, void* stream) {
    if (count <= 0) return 0;
    if (((uintptr_t)resid & 15) || ((uintptr_t)out & 7)) return tli_fail("residual_rows: operands must be 16-byte aligned");
    const long long threads = (count + 3) / 4;
    residual_rows_kernel<<<(unsigned)((threads + 255) / 256), 256, 0, (hipStream_t)stream>>>(resid, (bf16_t*)out, count);
    return tli_check_launch("residual_rows");
}

template <typename T>
static int run_norm_add_norm(float* resid, const T* y, const float* sums, int parts, size_t plane, const float* w1, float eps1, const float* w2, float eps2, T* out, const int* rows,
                             int count, int n, const MixArgs& mix, hipStream_t s) {
    const bool vec = n % 8 == 0 && !(((uintptr_t)resid | (uintptr_t)y | (uintptr_t)sums | (uintptr_t)w1 | (uintptr_t)w2 | (uintptr_t)out | (uintptr_t)mix.mu |
                                      (uintptr_t)mix.kept) & 15);
#define NAN_RUN(V, R) norm_add_norm_kernel<T, V, R><<<count, PN_THREADS, 0, s>>>(resid, y, sums, parts, plane, w1, eps1, w2, eps2, out, rows, n, mix)
    if (vec && n <= 8 * PN_THREADS) NAN_RUN(8, 1);
    else if (vec && n <= 16 * PN_THREADS) NAN_RUN(8, 2);
    else if (vec && n <= 32 * PN_THREADS) NAN_RUN(8, 4);
    else if (n <= 4 * PN_THREADS) NAN_RUN(1, 4);
    else if (n <= 32 * PN_THREADS) NAN_RUN(1, 32);
    else return tli_fail("norm_add_norm: rows of %d elements (at most %d)", n, 32 * PN_THREADS);
#undef NAN_RUN
    return tli_check_launch("norm_add_norm");
}

// resid [total, n] float32 += w1 * y / rms(y) (y null: nothing), out [count, n] = w2 * resid / rms(resid) in the type of y (w2 null:
// resid's rows; out may then be null).  parts > 0: y is float32 partial sums [parts][total][n].  rows (or null): the rows of resid
// and y that `count` counts, resid then unchanged; without them count is total.  mu (or null) [mixes][n], kept [slots][n],
// slots, seq_start [rows]: out is [mixes][count][n] (rows must be null).
extern "C" int tli_norm_add_norm(float* resid, const void* y, int parts, int total, const float* w1, float eps1, const float* w2, float eps2,
                                 void* out, const int* rows, int count, int n, const float* mu, int mixes, void* kept, const int* slots,
                                 const int* seq_start, int dtype, void* stream) {
    if (count <= 0) return 0;
    if (n <= 0 || (y && !w1) || (w2 && !out) || (!w2 && (!y || rows || mu)) || parts < 0 || (parts && !y) || count > total)
        return tli_fail("norm_add_norm: bad arguments");
    if (mu && (rows || mixes <= 0 || !kept || !slots || !seq_start)) return tli_fail("norm_add_norm: bad mixes");
    const MixArgs mix{mu, mixes, kept, slots, seq_start, (size_t)count * n};
    const float* sums = parts ? (const float*)y : nullptr;
    const size_t plane = (size_t)total * n;
    if (parts) y = nullptr;
    hipStream_t s = (hipStream_t)stream;
    if (dtype == TLI_F32)
        return run_norm_add_norm<float>(resid, (const float*)y, sums, parts, plane, w1, eps1, w2, eps2, (float*)out, rows, count, n, mix, s);
    if (dtype == TLI_BF16)
        return run_norm_add_norm<bf16_t>(resid, (const bf16_t*)y, sums, parts, plane, w1, eps1, w2, eps2, (bf16_t*)out, rows, count, n, mix, s);
    return tli_fail("norm_add_norm: unknown dtype %d", dtype);
}

// h [rows, n]; out [mixes][rows][n]; mu [mixes][n]; kept [slots][n] in the type of h
extern "C" int tli_token_mixes(const void* h, const float* mu, int mixes, void* kept, void* out, const int* seq_of_row,
                               const int* row_start, const int* seq_start, const int* slots, int rows, int n, int dtype, void* stream) {
    if (rows <= 0) return 0;
    if (n <= 0 || mixes <= 0) return tli_fail("token_mixes: bad sizes");
    const MixArgs mix{mu, mixes, kept, slots, seq_start, (size_t)rows * n};
    const bool vec = n % 8 == 0 && !(((uintptr_t)h | (uintptr_t)mu | (uintptr_t)kept | (uintptr_t)out) & 15);
    hipStream_t s = (hipStream_t)stream;
#define TM_RUN(T, V) token_mixes_kernel<T, V><<<rows, PN_THREADS, 0, s>>>((const T*)h, (T*)out, seq_of_row, row_start, n, mix)
    if (dtype == TLI_F32) { if (vec) TM_RUN(float, 8); else TM_RUN(float, 1); }
    else if (dtype == TLI_BF16) { if (vec) TM_RUN(bf16_t, 8); else TM_RUN(bf16_t, 1); }
    else return tli_fail("token_mixes: unknown dtype %d", dtype);
#undef TM_RUN
    return tli_check_launch("token_mixes");
}

// out [rows, n] = w * x / sqrt(mean(x^2) + eps) for n elements of rows that lie ld elements apart.  A workgroup a row, V elements
// a thread and round.
template <typename T, int V>
__global__ __launch_bounds__(PN_THREADS) void norm_rows_kernel(const T* __restrict__ x, int ld, const float* __restrict__ w, T* __restrict__ out,
                                                               int n, float eps) {
    __shared__ float red[16];
    const size_t row = blockIdx.x;
    const T* src = x + row * ld;
    float ssq = 0.f;
    for (int c = threadIdx.x * V; c < n; c += PN_THREADS * V) {
        float v[V];
        row_load<T, V>(src + c, v);
#pragma unroll
        for (int e = 0; e < V; ++e) ssq = fmaf(v[e], v[e], ssq);
    }
    const float factor = 1.0f / sqrtf(block_sum(ssq, red) / (float)n + eps);
    for (int c = threadIdx.x * V; c < n; c += PN_THREADS * V) {
        float v[V], g[V];
        row_load<T, V>(src + c, v);
        row_load<float, V>(w + c, g);
#pragma unroll
        for (int e = 0; e < V; ++e) v[e] = v[e] * factor * g[e];
        row_store<T, V>(out + row * n + c, v);
    }
}

extern "C" int tli_norm_rows(const void* x, int ld, const float* w, void* out, int rows, int n, float eps, int dtype, void* stream) {
    if (rows <= 0) return 0;
    if (n <= 0 || ld < n) return tli_fail("norm_rows: bad sizes");
    const bool vec = n % 8 == 0 && ld % 8 == 0 && !(((uintptr_t)x | (uintptr_t)w | (uintptr_t)out) & 15);
    hipStream_t s = (hipStream_t)stream;
#define NR_RUN(T, V) norm_rows_kernel<T, V><<<rows, PN_THREADS, 0, s>>>((const T*)x, ld, w, (T*)out, n, eps)
    if (dtype == TLI_F32) { if (vec) NR_RUN(float, 8); else NR_RUN(float, 1); }
    else if (dtype == TLI_BF16) { if (vec) NR_RUN(bf16_t, 8); else NR_RUN(bf16_t, 1); }
    else return tli_fail("norm_rows: unknown dtype %d", dtype);
#undef NR_RUN
    return tli_check_launch("norm_rows");
}
