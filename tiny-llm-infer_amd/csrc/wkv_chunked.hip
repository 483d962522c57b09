// Portions of prompts through the RWKV's recurrence (wkv.hip), bfloat16 rows, head sizes in sixteens up to 128: chunks of 64
// rows, products of matrices in float32 on v_mfma_f32_16x16x4_f32 (nothing of the recurrence is rounded to bfloat16).
// With A_t(c) the product of channel c's decays from the chunk's first row to t, and P the state before the chunk,
//   o_t = (A_(t-1) r_t)^T P + sum over s < t of (sum_c r_t(c) k_s(c) A_(t-1)(c) / A_s(c)) v_s + (sum_c r_t u k_t) v_t
//   P'  = diag(A_end) P + sum_s (A_end / A_s) k_s v_s^T
// A_s may be far too small to divide by, so only quotients of later over earlier rows are formed, as exp of differences of
// log A that are never positive: a row's queries and keys are taken to the border of their tile of 16 rows, tiles
// further apart get the decays of the whole tiles between them (a factor a channel), and inside a tile the products of
// decays are formed row by row.
//
// wkv_chunk_local: a workgroup a (chunk; head): the decays' logarithms (the product with W2 on the same instructions), their
//   sums from the chunk's first row (log2 A, left for the next kernel), and the chunk's own term of P'.
// wkv_chunk_scan:  P before every chunk, in place of that term; four elements of S a thread, chunk after chunk.
// wkv_chunk_outputs: a workgroup a (chunk; head), a wave 16 rows: scores inside its tile row by row, those against the tiles
//   before and the product with P as matrices, then the head's norm and its gate.
//
// The matrix instruction's operands: A: lane l has row l % 16, k = l / 16; B: k = l / 16, column l % 16; sums: rows 4 (l / 16) ..
// + 3 of column l % 16.  Of 16 consecutive k, lane group c takes 4 c .. 4 c + 3 in four instructions, so that a lane's
// operands are four consecutive elements.
#include "recurrence.h"

#define WC_ROWS 64
#define WC_THREADS 256
#define WC_KLD (WC_ROWS + 4)
#define WC_LOG2E 1.4426950408889634f
#define WC_LEAST (-127.0f)       // a row's decay is at least 2^-127: as good as 0, and sums of logarithms stay exact enough

typedef float wc_f32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t wc_u32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t wc_u32x2 __attribute__((ext_vector_type(2)));

struct WkvChunks {
    const bf16_t* proj;                                  // [T, ld]: r (H dk) | k (H dk) | v (H dv) | gate (H dv)
    int ld;
    const float* z;                                      // the decays' inner rows, before tanh
    long long z_row, z_col;
    const bf16_t* w2;                                    // [H dk, rank]
    const float* w0;                                     // [H dk]
    int rank;
    const float* u;                                      // [H, dk]
    float* logs;                                         // scratch [T][H dk]: log2 A
    float* before;                                       // scratch [chunks][H][dv][dk]
    float* state;                                        // [slots][H][dv][dk]
    const int* row_start;
    const int* seq_start;
    const int* slots;
    int T, seqs, H, dk, dv;
};

__device__ __forceinline__ int wc_chunks(int rows) { return (rows + WC_ROWS - 1) / WC_ROWS; }

// The sequence, the place in it and the rows of chunk z of the step; false past the last (the grid's slack).
struct WcPlace {
    int seq, index, r0, count;
};
__device__ __forceinline__ bool wc_find(const WkvChunks& a, int z, WcPlace& p) {
    for (int seq = 0; seq < a.seqs; ++seq) {
        const int first = a.row_start[seq], n = a.row_start[seq + 1] - first, c = wc_chunks(n);
        if (z < c) {
            p.seq = seq, p.index = z, p.r0 = first + z * WC_ROWS, p.count = min(WC_ROWS, n - z * WC_ROWS);
            return true;
        }
        z -= c;
    }
    return false;
}

__device__ __forceinline__ void wc_widen(const wc_u32x2& w, float (&v)[4]) {
    v[0] = __uint_as_float(w[0] << 16), v[1] = __uint_as_float(w[0] & 0xFFFF0000u);
    v[2] = __uint_as_float(w[1] << 16), v[3] = __uint_as_float(w[1] & 0xFFFF0000u);
}
__device__ __forceinline__ void wc_widen(const wc_u32x4& w, float (&v)[8]) {
#pragma unroll
    for (int i = 0; i < 4; ++i) v[2 * i] = __uint_as_float(w[i] << 16), v[2 * i + 1] = __uint_as_float(w[i] & 0xFFFF0000u);
}
__device__ __forceinline__ float wc_exp2(float x) { return __builtin_amdgcn_exp2f(x); }
// (absolute error below 2e-7: 1 - 2 / (e^(2x) + 1))
__device__ __forceinline__ float wc_tanh(float x) { return 1.0f - 2.0f * __builtin_amdgcn_rcpf(wc_exp2(2.0f * WC_LOG2E * x) + 1.0f); }

// sum of a lane and those before it in its 16
template <int N>
__device__ __forceinline__ float wc_shifted(float v) {
    return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x110 + N, 0xF, 0xF, true));
}
__device__ __forceinline__ float wc_scan16(float v) {
    v += wc_shifted<1>(v);
    v += wc_shifted<2>(v);
    v += wc_shifted<4>(v);
    v += wc_shifted<8>(v);
    return v;
}

static inline int wc_rank16(int rank) { return (rank + 15) / 16 * 16; }
static inline size_t wc_local_floats(int dk, int dv, int rank) {
    const size_t z = (size_t)WC_ROWS * (wc_rank16(rank) + 4), kt = (size_t)dk * WC_KLD;
    return (z > kt ? z : kt) + (size_t)WC_ROWS * (dv + 4);
}
static inline size_t wc_output_floats(int dk, int dv) {
    const size_t rows = (size_t)2 * WC_ROWS * (dk + 4), kv = (size_t)WC_ROWS * (dk + 4 + dv + 4), p = (size_t)dv * (dk + 4);
    const size_t two = rows > kv ? rows : kv;
    return two > p ? two : p;
}

// N: sixteens of a head's keys and values (EXACT), or their bound
template <int N, bool EXACT>
__global__ __launch_bounds__(WC_THREADS, 2) void wkv_chunk_local_kernel(WkvChunks a) {
    extern __shared__ __align__(16) float wc_lds[];
    constexpr int CT = (N + 3) / 4;                                    // tiles of 16 channels, or of values, a wave
    const int tid = threadIdx.x, lane = tid % TLI_WAVE, wave = __builtin_amdgcn_readfirstlane(tid / TLI_WAVE), col = lane % 16, grp = lane / 16;
    const int nk = EXACT ? N : a.dk / 16, nv = EXACT ? N : a.dv / 16, dk = nk * 16, dv = nv * 16, H = a.H, h = blockIdx.y;
    WcPlace at;
    if (!wc_find(a, blockIdx.x, at)) return;
    const int count = at.count, rank = a.rank, rank16 = (rank + 15) / 16 * 16, ZLD = rank16 + 4, VLD = dv + 4;
    float* tz = wc_lds;                                                // [row][rank16 + 4], then
    float* kt = wc_lds;                                                // [dk][64 + 4]: the weighted keys, transposed
    float* v_s = wc_lds + max(WC_ROWS * ZLD, dk * WC_KLD);             // [row][dv + 4]
    const bf16_t* rows = a.proj + (size_t)at.r0 * a.ld;
    // what comes from memory, asked for together: values, keys (this lane's four channels of four rows), z
    constexpr int VP = (WC_ROWS * N * 2 + WC_THREADS - 1) / WC_THREADS;
    wc_u32x4 vr[VP];
#pragma unroll
    for (int i = 0; i < VP; ++i) {
        const int p = min(tid + i * WC_THREADS, WC_ROWS * nv * 2 - 1), r = p / (nv * 2);
        vr[i] = *reinterpret_cast<const wc_u32x4*>(rows + (size_t)min(r, count - 1) * a.ld + (size_t)2 * H * dk + (size_t)h * dv + (p - r * nv * 2) * 8);
    }
    wc_u32x2 kr[CT][4];
#pragma unroll
    for (int q = 0; q < CT; ++q)
#pragma unroll
        for (int m = 0; m < 4; ++m)
            kr[q][m] = *reinterpret_cast<const wc_u32x2*>(rows + (size_t)min(16 * m + col, count - 1) * a.ld + (size_t)(H + h) * dk +
                                                          16 * min(wave + 4 * q, nk - 1) + 4 * grp);
    for (int i = tid; i < WC_ROWS * rank16; i += WC_THREADS) {
        const int t = i % WC_ROWS, e = i / WC_ROWS;
        float v = 0.f;
        if (e < rank) v = wc_tanh(a.z[(long long)(at.r0 + min(t, count - 1)) * a.z_row + e * a.z_col]);
        tz[t * ZLD + e] = v;
    }
#pragma unroll
    for (int i = 0; i < VP; ++i) {
        const int p = tid + i * WC_THREADS, r = p / (nv * 2);
        if (p >= WC_ROWS * nv * 2) continue;
        float x[8];
        wc_widen(vr[i], x);
        float* dst = v_s + r * VLD + (p - r * nv * 2) * 8;
        *reinterpret_cast<wc_f32x4*>(dst) = (wc_f32x4){x[0], x[1], x[2], x[3]};
        *reinterpret_cast<wc_f32x4*>(dst + 4) = (wc_f32x4){x[4], x[5], x[6], x[7]};
    }
    __syncthreads();
    // log2 of the decays of 16 channels (A) and the chunk's 64 rows (B): lane has channels 4 grp .. + 3 of rows 16 m + col
    wc_f32x4 lw[CT][4];
#pragma unroll
    for (int q = 0; q < CT; ++q) {
#pragma unroll
        for (int m = 0; m < 4; ++m) lw[q][m] = (wc_f32x4){0.f, 0.f, 0.f, 0.f};
        const int ct = min(wave + 4 * q, nk - 1);
        const bf16_t* w_row = a.w2 + (size_t)(h * dk + 16 * ct + col) * rank;
        for (int s = 0; s < rank16; s += 16) {
            const int i = s + 4 * grp;
            wc_u32x2 raw = *reinterpret_cast<const wc_u32x2*>(w_row + (i < rank ? i : 0));       // (rank in fours; past it tz is 0)
            float w[4];
            wc_widen(raw, w);
            wc_f32x4 b[4];
#pragma unroll
            for (int m = 0; m < 4; ++m) b[m] = *reinterpret_cast<const wc_f32x4*>(tz + (16 * m + col) * ZLD + i);
#pragma unroll
            for (int e = 0; e < 4; ++e)
#pragma unroll
                for (int m = 0; m < 4; ++m) lw[q][m] = __builtin_amdgcn_mfma_f32_16x16x4f32(w[e], b[m][e], lw[q][m], 0, 0, 0);
        }
    }
    __syncthreads();                                                   // tz has been read
#pragma unroll
    for (int q = 0; q < CT; ++q) {
        const int ct = wave + 4 * q;
        if (ct >= nk) continue;
        const int c = h * dk + 16 * ct + 4 * grp;
        const wc_f32x4 bias = *reinterpret_cast<const wc_f32x4*>(a.w0 + c);
        wc_f32x4 run = (wc_f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int m = 0; m < 4; ++m) {
            const bool live = 16 * m + col < count;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float x = fmaxf(-WC_LOG2E * expf(lw[q][m][e] + bias[e]), WC_LEAST);
                lw[q][m][e] = run[e] + wc_scan16(live ? x : 0.f);
                run[e] = __shfl(lw[q][m][e], 15, 16);
            }
            if (live) *reinterpret_cast<wc_f32x4*>(a.logs + (size_t)(at.r0 + 16 * m + col) * H * dk + c) = lw[q][m];
        }
#pragma unroll
        for (int m = 0; m < 4; ++m) {
            float k[4];
            wc_widen(kr[q][m], k);
            const bool live = 16 * m + col < count;
#pragma unroll
            for (int e = 0; e < 4; ++e)
                kt[(16 * ct + 4 * grp + e) * WC_KLD + 16 * m + col] = live ? k[e] * wc_exp2(run[e] - lw[q][m][e]) : 0.f;
        }
    }
    __syncthreads();
    wc_f32x4 S[CT][N];
#pragma unroll
    for (int q = 0; q < CT; ++q)
#pragma unroll
        for (int b = 0; b < N; ++b) S[q][b] = (wc_f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < 4; ++s) {
        float v[CT][4];
#pragma unroll
        for (int q = 0; q < CT; ++q)
#pragma unroll
            for (int e = 0; e < 4; ++e) v[q][e] = v_s[(16 * s + 4 * grp + e) * VLD + 16 * min(wave + 4 * q, nv - 1) + col];
#pragma unroll
        for (int b = 0; b < N; ++b) {
            const wc_f32x4 kk = *reinterpret_cast<const wc_f32x4*>(kt + (16 * (EXACT ? b : min(b, nk - 1)) + col) * WC_KLD + 16 * s + 4 * grp);
#pragma unroll
            for (int e = 0; e < 4; ++e)
#pragma unroll
                for (int q = 0; q < CT; ++q) S[q][b] = __builtin_amdgcn_mfma_f32_16x16x4f32(kk[e], v[q][e], S[q][b], 0, 0, 0);
        }
    }
    float* out = a.before + ((size_t)blockIdx.x * H + h) * dv * dk;
#pragma unroll
    for (int q = 0; q < CT; ++q) {
        if (wave + 4 * q >= nv) continue;
#pragma unroll
        for (int b = 0; b < N; ++b)
            if (b < nk) *reinterpret_cast<wc_f32x4*>(out + (size_t)(16 * (wave + 4 * q) + col) * dk + 16 * b + 4 * grp) = S[q][b];
    }
}

// four elements of S a thread
__global__ __launch_bounds__(WC_THREADS) void wkv_chunk_scan_kernel(WkvChunks a) {
    const int H = a.H, dk = a.dk, dv = a.dv, seq = blockIdx.y;
    const size_t per = (size_t)H * dv * dk;
    const size_t i = ((size_t)blockIdx.x * WC_THREADS + threadIdx.x) * 4;
    if (i >= per) return;
    const int first = a.row_start[seq], n = a.row_start[seq + 1] - first, chunks = wc_chunks(n);
    if (n <= 0) return;
    int z0 = 0;
    for (int s = 0; s < seq; ++s) z0 += wc_chunks(a.row_start[s + 1] - a.row_start[s]);
    const int h = (int)(i / ((size_t)dv * dk)), c = (int)(i % dk);
    const float* logs = a.logs + (size_t)h * dk + c;
    const size_t ld = (size_t)H * dk;
    float* slot = a.state + (size_t)a.slots[seq] * per + i;
    float* own = a.before + (size_t)z0 * per + i;
    wc_f32x4 P = (wc_f32x4){0.f, 0.f, 0.f, 0.f};
    if (a.seq_start[seq] > 0) P = *reinterpret_cast<const wc_f32x4*>(slot);
    constexpr int AHEAD = 4;
    wc_f32x4 U[AHEAD], L[AHEAD];
    auto fetch = [&](int z, wc_f32x4& u, wc_f32x4& l) {
        const int zz = min(z, chunks - 1);
        u = *reinterpret_cast<const wc_f32x4*>(own + (size_t)zz * per);
        l = *reinterpret_cast<const wc_f32x4*>(logs + (size_t)(first + min((zz + 1) * WC_ROWS, n) - 1) * ld);
    };
#pragma unroll
    for (int k = 0; k < AHEAD; ++k) fetch(k, U[k], L[k]);
    for (int z = 0; z < chunks; z += AHEAD) {
#pragma unroll
        for (int k = 0; k < AHEAD; ++k) {
            if (z + k < chunks) {
                const wc_f32x4 u = U[k], l = L[k];
                *reinterpret_cast<wc_f32x4*>(own + (size_t)(z + k) * per) = P;
#pragma unroll
                for (int e = 0; e < 4; ++e) P[e] = fmaf(wc_exp2(l[e]), P[e], u[e]);
                if (z + k + AHEAD < chunks) fetch(z + k + AHEAD, U[k], L[k]);
            }
        }
    }
    *reinterpret_cast<wc_f32x4*>(slot) = P;
}

struct WkvOutput {
    bf16_t* out;                                         // rows out_ld elements apart, H dv of each
    int out_ld;
    const float* weight;                                 // [H dv]
    float eps;
};

template <int N, bool EXACT>
__global__ __launch_bounds__(WC_THREADS, 2) void wkv_chunk_outputs_kernel(WkvChunks a, WkvOutput out) {
    extern __shared__ __align__(16) float wc_lds[];
    __shared__ __align__(16) float tile_decay[4][N * 16];              // of a channel over a whole tile of 16 rows
    __shared__ float score_s[4][16 * 17];
    const int tid = threadIdx.x, lane = tid % TLI_WAVE, wave = __builtin_amdgcn_readfirstlane(tid / TLI_WAVE), col = lane % 16, grp = lane / 16;
    const int nk = EXACT ? N : a.dk / 16, nv = EXACT ? N : a.dv / 16, dk = nk * 16, dv = nv * 16, H = a.H, h = blockIdx.y;
    const int KLD = dk + 4, VLD = dv + 4;
    WcPlace at;
    if (!wc_find(a, blockIdx.x, at)) return;
    const int count = at.count, r0 = at.r0;
    const bool from_nothing = at.index == 0 && a.seq_start[at.seq] == 0;
    const bf16_t* rows = a.proj + (size_t)r0 * a.ld;
    const float* logs = a.logs + (size_t)r0 * H * dk + (size_t)h * dk;  // row t's at t * H dk
    const size_t lld = (size_t)H * dk;
    // a wave's tile of 16 rows: the later a tile, the more products it has, so every second round of workgroups deals them
    // out the other way round
    const int rt = ((blockIdx.y * gridDim.x + blockIdx.x) >> 8) & 1 ? WC_ROWS / 16 - 1 - wave : wave;
    const int i = 16 * rt + col, row = min(i, count - 1);              // this lane's row of the chunk
    const bool works = 16 * rt < count;                                // (the same for the whole wave)
    auto k_tile = [&](int b) { return EXACT ? b : min(b, nk - 1); };
    auto v_tile = [&](int t) { return EXACT ? t : min(t, nv - 1); };

    // ---- rows of r and the rows' own decays into LDS; keys, taken to the end of their tile, wait in registers
    float* r_s = wc_lds;                                               // [row][dk + 4]
    float* d_s = wc_lds + WC_ROWS * KLD;                               // [row][dk + 4]
    constexpr int KP = (WC_ROWS * N * 2 + WC_THREADS - 1) / WC_THREADS;
    wc_f32x4 kh[KP][2];
    wc_u32x4 vr[KP];
#pragma unroll
    for (int x = 0; x < KP; ++x) {
        const int p = min(tid + x * WC_THREADS, WC_ROWS * nv * 2 - 1), r = p / (nv * 2);
        vr[x] = *reinterpret_cast<const wc_u32x4*>(rows + (size_t)min(r, count - 1) * a.ld + (size_t)2 * H * dk + (size_t)h * dv + (p - r * nv * 2) * 8);
    }
#pragma unroll
    for (int x = 0; x < KP; ++x) {
        const int p = min(tid + x * WC_THREADS, WC_ROWS * nk * 2 - 1), r = p / (nk * 2), c = (p - r * nk * 2) * 8;
        const int t = min(r, count - 1), last = min(r | 15, count - 1);
        const bf16_t* src = rows + (size_t)t * a.ld + (size_t)h * dk + c;
        const wc_u32x4 rr = *reinterpret_cast<const wc_u32x4*>(src), kk = *reinterpret_cast<const wc_u32x4*>(src + (size_t)H * dk);
        float rv[8], kv[8];
        wc_widen(rr, rv);
        wc_widen(kk, kv);
#pragma unroll
        for (int half = 0; half < 2; ++half) {
            const wc_f32x4 here = *reinterpret_cast<const wc_f32x4*>(logs + t * lld + c + 4 * half);
            const wc_f32x4 end = *reinterpret_cast<const wc_f32x4*>(logs + last * lld + c + 4 * half);
            wc_f32x4 prev = *reinterpret_cast<const wc_f32x4*>(logs + max(t - 1, 0) * lld + c + 4 * half);
            wc_f32x4 d;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                d[e] = wc_exp2(here[e] - (t > 0 ? prev[e] : 0.f));
                kh[x][half][e] = kv[4 * half + e] * wc_exp2(end[e] - here[e]);
            }
            *reinterpret_cast<wc_f32x4*>(r_s + r * KLD + c + 4 * half) = (wc_f32x4){rv[4 * half], rv[4 * half + 1], rv[4 * half + 2], rv[4 * half + 3]};
            *reinterpret_cast<wc_f32x4*>(d_s + r * KLD + c + 4 * half) = d;
        }
    }
    for (int x = tid; x < 4 * dk; x += WC_THREADS) {
        const int b = x / dk, c = x % dk;
        const float end = logs[(size_t)min(16 * b + 15, count - 1) * lld + c], start = b > 0 ? logs[(size_t)min(16 * b - 1, count - 1) * lld + c] : 0.f;
        tile_decay[b][c] = wc_exp2(end - start);
    }
    // this lane's row of r, taken to the start of its tile; the key row of the same number, a quarter of its channels a lane
    float q[N][4], pk[N][4];
#pragma unroll
    for (int b = 0; b < N; ++b) {
        const int c = 16 * k_tile(b) + 4 * grp;
        const wc_f32x4 before = *reinterpret_cast<const wc_f32x4*>(logs + (size_t)max(row - 1, 0) * lld + c);
        const wc_f32x4 start = *reinterpret_cast<const wc_f32x4*>(logs + (size_t)min(max(16 * rt - 1, 0), count - 1) * lld + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) q[b][e] = b < nk ? wc_exp2((row > 0 ? before[e] : 0.f) - (rt > 0 ? start[e] : 0.f)) : 0.f;
        const wc_u32x2 kk = *reinterpret_cast<const wc_u32x2*>(rows + (size_t)row * a.ld + (size_t)(H + h) * dk + grp * 4 * nk + 4 * k_tile(b));
        wc_widen(kk, pk[b]);
    }
    __syncthreads();
    float p[4] = {0.f, 0.f, 0.f, 0.f};                                 // scores of this lane's row against rows 4 grp .. + 3 of its tile
    if (works) {
        float own = 0.f;
#pragma unroll
        for (int b = 0; b < N; ++b) {
            const int c = 16 * k_tile(b) + 4 * grp, cq = grp * 4 * nk + 4 * k_tile(b);
            const wc_f32x4 r = *reinterpret_cast<const wc_f32x4*>(r_s + row * KLD + c);
            const wc_f32x4 rq = *reinterpret_cast<const wc_f32x4*>(r_s + row * KLD + cq), uq = *reinterpret_cast<const wc_f32x4*>(a.u + (size_t)h * dk + cq);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                q[b][e] *= r[e];
                if (b < nk) own = fmaf(rq[e] * uq[e], pk[b][e], own);
            }
        }
        own = quad_rows_sum(own);
        float* sc = score_s[wave];
        for (int s = 1; s < 16; ++s) {                                 // row s of the tile against the rows before it
            float x = 0.f;
            if (col < s) {
                const float* rr = r_s + (16 * rt + s) * KLD + grp * 4 * nk;
                const float* dd = d_s + (16 * rt + s) * KLD + grp * 4 * nk;
#pragma unroll
                for (int b = 0; b < N; ++b) {
                    if (!EXACT && b >= nk) continue;
                    const wc_f32x4 r4 = *reinterpret_cast<const wc_f32x4*>(rr + 4 * b), d4 = *reinterpret_cast<const wc_f32x4*>(dd + 4 * b);
#pragma unroll
                    for (int e = 0; e < 4; ++e) {
                        x = fmaf(r4[e], pk[b][e], x);
                        pk[b][e] *= d4[e];
                    }
                }
            }
            x = quad_rows_sum(x);
            if (grp == 0) sc[s * 17 + col] = x;
        }
        wave_lds_sync();
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int j = 4 * grp + e;
            p[e] = j < col ? sc[col * 17 + j] : j == col ? own : 0.f;
        }
    }
    __syncthreads();                                                   // r_s and d_s have been read
    float* k_s = wc_lds;                                               // [row][dk + 4]
    float* v_s = wc_lds + WC_ROWS * KLD;                               // [row][dv + 4]
#pragma unroll
    for (int x = 0; x < KP; ++x) {
        const int pp = tid + x * WC_THREADS;
        if (pp < WC_ROWS * nk * 2) {
            const int r = pp / (nk * 2), c = (pp - r * nk * 2) * 8;
            *reinterpret_cast<wc_f32x4*>(k_s + r * KLD + c) = kh[x][0];
            *reinterpret_cast<wc_f32x4*>(k_s + r * KLD + c + 4) = kh[x][1];
        }
        if (pp < WC_ROWS * nv * 2) {
            const int r = pp / (nv * 2), c = (pp - r * nv * 2) * 8;
            float v[8];
            wc_widen(vr[x], v);
            *reinterpret_cast<wc_f32x4*>(v_s + r * VLD + c) = (wc_f32x4){v[0], v[1], v[2], v[3]};
            *reinterpret_cast<wc_f32x4*>(v_s + r * VLD + c + 4) = (wc_f32x4){v[4], v[5], v[6], v[7]};
        }
    }
    constexpr int PP = N * N * 16 * 16 / 4 / WC_THREADS;
    const int p_row = dk / 4, p_all = dv * p_row;
    const float* P = a.before + ((size_t)blockIdx.x * H + h) * dv * dk;
    wc_f32x4 pr[PP];
    if (!from_nothing) {
#pragma unroll
        for (int x = 0; x < PP; ++x) pr[x] = *reinterpret_cast<const wc_f32x4*>(P + (size_t)min(tid + x * WC_THREADS, p_all - 1) * 4);
    }
    __syncthreads();
    wc_f32x4 acc[N];
#pragma unroll
    for (int t = 0; t < N; ++t) acc[t] = (wc_f32x4){0.f, 0.f, 0.f, 0.f};
    if (works) {
        auto values = [&](int jt) {                                    // (rows past the chunk's last: a weight of 0 and a real row)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float* v_row = v_s + min(16 * jt + 4 * grp + e, count - 1) * VLD + col;
#pragma unroll
                for (int t = 0; t < N; ++t) acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(v_row[16 * v_tile(t)], p[e], acc[t], 0, 0, 0);
            }
        };
        values(rt);
        for (int jt = rt - 1; jt >= 0; --jt) {
            wc_f32x4 s[2] = {(wc_f32x4){0.f, 0.f, 0.f, 0.f}, (wc_f32x4){0.f, 0.f, 0.f, 0.f}};
            const float* k_row = k_s + (16 * jt + col) * KLD + 4 * grp;
#pragma unroll
            for (int b = 0; b < N; ++b) {
                const wc_f32x4 kk = *reinterpret_cast<const wc_f32x4*>(k_row + 16 * k_tile(b));
                const wc_f32x4 d = *reinterpret_cast<const wc_f32x4*>(&tile_decay[jt][16 * k_tile(b) + 4 * grp]);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    s[e & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(kk[e], q[b][e], s[e & 1], 0, 0, 0);
                    q[b][e] *= d[e];                                   // to the start of tile jt
                }
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) p[e] = s[0][e] + s[1][e];
            values(jt);
        }
    }
    if (!from_nothing) {                                               // (the same for the whole workgroup)
        __syncthreads();                                               // keys and values have been read
#pragma unroll
        for (int x = 0; x < PP; ++x) {
            const int pp = tid + x * WC_THREADS;
            if (pp < p_all) *reinterpret_cast<wc_f32x4*>(wc_lds + (pp / p_row) * KLD + (pp % p_row) * 4) = pr[x];
        }
        __syncthreads();
        if (works) {
#pragma unroll
            for (int b = 0; b < N; ++b) {
                wc_f32x4 s[N];
#pragma unroll
                for (int t = 0; t < N; ++t)
                    s[t] = *reinterpret_cast<const wc_f32x4*>(wc_lds + (16 * v_tile(t) + col) * KLD + 16 * k_tile(b) + 4 * grp);
#pragma unroll
                for (int e = 0; e < 4; ++e)
#pragma unroll
                    for (int t = 0; t < N; ++t) acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(s[t][e], q[b][e], acc[t], 0, 0, 0);
            }
        }
    }
    if (!works) return;
    // the head's norm and gate: this lane has elements 16 t + 4 grp .. + 3 of its row
    float ss = 0.f;
#pragma unroll
    for (int t = 0; t < N; ++t)
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (t < nv) ss = fmaf(acc[t][e], acc[t][e], ss);
    const float factor = 1.0f / sqrtf(quad_rows_sum(ss) / (float)dv + out.eps);
    if (i >= count) return;
    const bf16_t* gate = rows + (size_t)i * a.ld + (size_t)H * (2 * dk + dv) + (size_t)h * dv;
    bf16_t* dst = out.out + (size_t)(r0 + i) * out.out_ld + (size_t)h * dv;
#pragma unroll
    for (int t = 0; t < N; ++t) {
        if (t >= nv) continue;
        const int d = 16 * t + 4 * grp;
        float g[4], y[4];
        wc_widen(*reinterpret_cast<const wc_u32x2*>(gate + d), g);
        const wc_f32x4 wt = *reinterpret_cast<const wc_f32x4*>(out.weight + (size_t)h * dv + d);
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] = acc[t][e] * factor * wt[e] * (g[e] / (1.f + expf(-g[e])));
        *reinterpret_cast<uint2*>(dst + d) = make_uint2(pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3]));
    }
}

// Whether heads of these sizes, their decays through `rank`, go through here (else wkv_rows serves).
extern "C" int tli_wkv_chunked_takes(int dk, int dv, int rank) {
    return dk % 16 == 0 && dv % 16 == 0 && dk >= 16 && dv >= 16 && dk <= 128 && dv <= 128 && rank > 0 && rank % 4 == 0 && rank <= 256;
}

// float32 elements of scratch for T rows in `seqs` sequences
extern "C" long long tli_wkv_chunked_scratch_floats(int T, int seqs, int H, int dk, int dv) {
    return (long long)T * H * dk + ((long long)T / WC_ROWS + seqs) * H * dk * dv;
}

template <int N, bool EXACT>
static int run_wkv_chunked(const WkvChunks& a, const WkvOutput& out, hipStream_t s) {
    const int zs = a.T / WC_ROWS + a.seqs;               // (an upper bound of the chunks; a workgroup past the last leaves)
    const dim3 grid(zs, a.H);
    const size_t local = wc_local_floats(a.dk, a.dv, a.rank) * sizeof(float), outs = wc_output_floats(a.dk, a.dv) * sizeof(float);
    static bool allowed = false;
    if (!allowed) {
        if (hipFuncSetAttribute((const void*)wkv_chunk_local_kernel<N, EXACT>, hipFuncAttributeMaxDynamicSharedMemorySize, 120 * 1024) != hipSuccess ||
            hipFuncSetAttribute((const void*)wkv_chunk_outputs_kernel<N, EXACT>, hipFuncAttributeMaxDynamicSharedMemorySize, 72 * 1024) != hipSuccess)
            return tli_fail("wkv in chunks: cannot have %zu bytes of LDS", local > outs ? local : outs);
        allowed = true;
    }
    wkv_chunk_local_kernel<N, EXACT><<<grid, WC_THREADS, local, s>>>(a);
    const size_t per = (size_t)a.H * a.dv * a.dk / 4;
    wkv_chunk_scan_kernel<<<dim3((unsigned)((per + WC_THREADS - 1) / WC_THREADS), a.seqs), WC_THREADS, 0, s>>>(a);
    wkv_chunk_outputs_kernel<N, EXACT><<<grid, WC_THREADS, outs, s>>>(a, out);
    return tli_check_launch("wkv in chunks");
}

// proj: bfloat16 rows of ld elements, r (H dk) | k (H dk) | v (H dv) | gate (H dv) first; z, w2, w0: as for tli_wkv_decays; u [H, dk];
// state [slots][H][dv][dk]; out: rows out_ld elements apart; scratch: tli_wkv_chunked_scratch_floats(T, ...) floats
extern "C" int tli_wkv_chunked_bf16(const void* proj, int ld, const float* z, long long z_row, long long z_col, const void* w2, const float* w0,
                                    int rank, const float* u, float* state, void* out, int out_ld, const float* weight, float* scratch,
                                    const int* row_start, const int* seq_start, const int* slots, float eps, int T, int seqs, int H,
                                    int dk, int dv, void* stream) {
    if (T <= 0 || seqs <= 0) return 0;
    if (H <= 0 || H > 65535 || seqs > 65535 || !tli_wkv_chunked_takes(dk, dv, rank)) return tli_fail("wkv in chunks: heads of %d and %d through %d", dk, dv, rank);
    if (ld % 8 || ld < 2 * H * (dk + dv) || out_ld % 4 || out_ld < H * dv) return tli_fail("wkv in chunks: rows of %d elements", ld);
    if ((((uintptr_t)proj | (uintptr_t)w0 | (uintptr_t)u | (uintptr_t)state | (uintptr_t)scratch | (uintptr_t)weight) & 15) ||
        (((uintptr_t)out | (uintptr_t)w2) & 7))
        return tli_fail("wkv in chunks: operands must be 16-byte aligned");
    const WkvChunks a{(const bf16_t*)proj, ld, z, z_row, z_col, (const bf16_t*)w2, w0, rank, u, scratch, scratch + (size_t)T * H * dk, state,
                      row_start, seq_start, slots, T, seqs, H, dk, dv};
    const WkvOutput o{(bf16_t*)out, out_ld, weight, eps};
    hipStream_t s = (hipStream_t)stream;
    if (dk == 128 && dv == 128) return run_wkv_chunked<8, true>(a, o, s);
    if (dk == 64 && dv == 64) return run_wkv_chunked<4, true>(a, o, s);
    if (dk <= 64 && dv <= 64) return run_wkv_chunked<4, false>(a, o, s);
    return run_wkv_chunked<8, false>(a, o, s);
}
