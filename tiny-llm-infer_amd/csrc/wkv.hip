// The RWKV's recurrence row by row: for the rows of one sequence, head by head (key size dk, value size dv),
//   o_t = S_(t-1)^T r_t + (r_t . u k_t) v_t,   row c of S_t = d_t(c) (row c of S_(t-1)) + k_t(c) v_t
// float32, S zero before position 0.  d_t = exp(-exp(W2 tanh(z_t) + w0)), a number a channel.
//
// wkv_decays:  d of a step's rows, [T, H dk].
// wkv_rows:    a workgroup a (16 columns of S; head; sequence); a column belongs to 16 lanes of a wave, a lane holding R
//              elements of it.  Rows come through LDS, WR_ROWS at a time.
// Any sizes and both types: what the float32 path runs, and sizes that the chunked form (wkv_chunked.hip) does not take.
#include "recurrence.h"

#define WR_THREADS 256
#define WR_ROWS 8

template <typename T>
__global__ __launch_bounds__(256) void wkv_decays_kernel(const float* __restrict__ z, long long z_row, long long z_col, const T* __restrict__ w2,
                                                         const float* __restrict__ w0, float* __restrict__ decay, int rank, int channels) {
    extern __shared__ float tz[];
    const int t = blockIdx.x;
    for (int i = threadIdx.x; i < rank; i += blockDim.x) tz[i] = tanhf(z[t * z_row + i * z_col]);
    __syncthreads();
    for (int c = threadIdx.x; c < channels; c += blockDim.x) {
        const T* w = w2 + (size_t)c * rank;
        float a = 0.f;
        for (int i = 0; i < rank; ++i) a = fmaf(tz[i], to_f32(w[i]), a);
        decay[(size_t)t * channels + c] = expf(-expf(a + w0[c]));
    }
}

__device__ __forceinline__ float wr_sum16(float v) {     // over the 16 lanes of a DPP row; every lane gets it
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0xB1, 0xF, 0xF, true));
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x4E, 0xF, 0xF, true));
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x141, 0xF, 0xF, true));
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x140, 0xF, 0xF, true));
    return v;
}

template <int R, typename T>
__global__ __launch_bounds__(WR_THREADS) void wkv_rows_kernel(const T* __restrict__ proj, int ld, const float* __restrict__ decay,
                                                              const float* __restrict__ u, float* __restrict__ state,
                                                              float* __restrict__ out, const int* __restrict__ row_start,
                                                              const int* __restrict__ seq_start, const int* __restrict__ slots,
                                                              int H, int dk, int dv) {
    constexpr int L = 16, DKP = L * R, NC = WR_THREADS / L;
    __shared__ float r_s[WR_ROWS][DKP], k_s[WR_ROWS][DKP], d_s[WR_ROWS][DKP], v_s[WR_ROWS][NC];
    const int tid = threadIdx.x, sub = tid % L, jl = tid / L;
    const int h = blockIdx.y, seq = blockIdx.z, j0 = blockIdx.x * NC, j = j0 + jl;
    const int first = row_start[seq], rows = row_start[seq + 1] - first;
    if (rows <= 0) return;
    const bool mine = j < dv;
    float* col = state + (((size_t)slots[seq] * H + h) * dv + (mine ? j : 0)) * dk;
    const bool fresh = seq_start[seq] <= 0;
    float S[R], uu[R];
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int c = r * L + sub;
        S[r] = (mine && !fresh && c < dk) ? col[c] : 0.f;
        uu[r] = c < dk ? u[h * dk + c] : 0.f;
    }
    for (int t0 = 0; t0 < rows; t0 += WR_ROWS) {
        const int n = min(WR_ROWS, rows - t0);
        __syncthreads();
        for (int i = tid; i < n * DKP; i += WR_THREADS) {
            const int t = i / DKP, c = i % DKP;
            const T* src = proj + (size_t)(first + t0 + t) * ld + (size_t)h * dk + c;
            r_s[t][c] = c < dk ? to_f32(src[0]) : 0.f;
            k_s[t][c] = c < dk ? to_f32(src[(size_t)H * dk]) : 0.f;
            d_s[t][c] = c < dk ? decay[((size_t)(first + t0 + t) * H + h) * dk + c] : 0.f;
        }
        for (int i = tid; i < n * NC; i += WR_THREADS) {
            const int t = i / NC, c = i % NC;
            v_s[t][c] = j0 + c < dv ? to_f32(proj[(size_t)(first + t0 + t) * ld + (size_t)2 * H * dk + (size_t)h * dv + j0 + c]) : 0.f;
        }
        __syncthreads();
        for (int t = 0; t < n; ++t) {
            const float v = v_s[t][jl];
            float acc = 0.f;
#pragma unroll
            for (int r = 0; r < R; ++r) {
                const int c = r * L + sub;
                const float kv = k_s[t][c] * v;
                acc = fmaf(fmaf(uu[r], kv, S[r]), r_s[t][c], acc);
                S[r] = fmaf(d_s[t][c], S[r], kv);
            }
            acc = wr_sum16(acc);
            if (mine && sub == 0) out[((size_t)(first + t0 + t) * H + h) * dv + j] = acc;
        }
    }
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int c = r * L + sub;
        if (mine && c < dk) col[c] = S[r];
    }
}

// z: element (t, i) of the decay's inner rows at t * z_row + i * z_col; w2 [channels, rank] in the run's type; w0 [channels]
extern "C" int tli_wkv_decays(const float* z, long long z_row, long long z_col, const void* w2, const float* w0, float* decay, int T,
                              int rank, int channels, int dtype, void* stream) {
    if (T <= 0) return 0;
    if (rank <= 0 || rank > 8192 || channels <= 0) return tli_fail("wkv_decays: bad sizes");
    hipStream_t s = (hipStream_t)stream;
    if (dtype == TLI_F32)
        wkv_decays_kernel<float><<<T, 256, rank * sizeof(float), s>>>(z, z_row, z_col, (const float*)w2, w0, decay, rank, channels);
    else if (dtype == TLI_BF16)
        wkv_decays_kernel<bf16_t><<<T, 256, rank * sizeof(float), s>>>(z, z_row, z_col, (const bf16_t*)w2, w0, decay, rank, channels);
    else
        return tli_fail("wkv_decays: unknown dtype %d", dtype);
    return tli_check_launch("wkv_decays");
}

// proj: rows of ld elements, r (H dk) | k (H dk) | v (H dv) first; decay [T, H dk]; u [H, dk]; state [slots][H][dv][dk]; out [T, H, dv]
extern "C" int tli_wkv_rows(const void* proj, int ld, const float* decay, const float* u, float* state, float* out,
                            const int* row_start, const int* seq_start, const int* slots, int seqs, int H, int dk, int dv,
                            int dtype, void* stream) {
    if (seqs <= 0) return 0;
    if (H <= 0 || H > 65535 || seqs > 65535 || dk <= 0 || dk > TLI_RECURRENCE_MAX_DK || dv <= 0 || ld < H * (2 * dk + dv))
        return tli_fail("wkv_rows: bad sizes (heads %d, keys of %d (at most %d), values of %d)", H, dk, TLI_RECURRENCE_MAX_DK, dv);
    hipStream_t s = (hipStream_t)stream;
    const dim3 grid((dv + 15) / 16, H, seqs);
    int R = 1;
    while (16 * R < dk) R *= 2;
#define WR_RUN(R, T) wkv_rows_kernel<R, T><<<grid, WR_THREADS, 0, s>>>((const T*)proj, ld, decay, u, state, out, row_start, seq_start, slots, H, dk, dv)
#define WR_CASE(R) case R: if (dtype == TLI_F32) WR_RUN(R, float); else if (dtype == TLI_BF16) WR_RUN(R, bf16_t); \
                   else return tli_fail("wkv_rows: unknown dtype %d", dtype); break;
    switch (R) {
        WR_CASE(1) WR_CASE(2) WR_CASE(4) WR_CASE(8) WR_CASE(16)
        default: return tli_fail("wkv_rows: keys of %d", dk);
    }
#undef WR_CASE
#undef WR_RUN
    return tli_check_launch("wkv_rows");
}
