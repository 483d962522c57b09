// Portions of prompts through the recurrent layers whose heads are normed one by one (retention.hip, mlstm.hip), bfloat16
// rows, head sizes in sixteens up to 128: the recurrence S_t = a_t S_(t-1) + w_t k_t v_t^T, o_t = S_t^T q_t in chunks of 64
// rows.  With A_t the product of a from the chunk's first row to t and P the state before the chunk,
//   o_t = A_t P^T q_t + sum over s <= t of (A_t / A_s) w_s (q_t . k_s) v_s,        P' = A_end P + sum_s (A_end / A_s) w_s k_s v_s^T
// (the mLSTM's normaliser n is one more column of S whose value is 1), which are products of matrices.  All of them are
// float32 on v_mfma_f32_16x16x4_f32, which takes float32 as it is: nothing of the recurrence is rounded to bfloat16.
//
// chunk_states: a workgroup a (two pairs of pieces of k, 32 elements; 64 of v; head; sequence) walks the sequence's chunks, its part of S in
//   the accumulators of the products, and leaves P of every chunk in scratch; the last S goes to the sequence's slot.
// chunk_outputs: a workgroup a (chunk; head), a wave 16 rows: the two terms of o from P, K and V in LDS (P first, then K
//   and V in its place), the scores and their weights in registers (transposed, S^T = K Q^T, so that they are already the
//   second operand of the product with V), then the head's norm and its gate.
//
// The matrix instruction's operands: A: lane l has row l % 16, k = l / 16; B: k = l / 16, column l % 16; sums: rows 4 (l / 16) ..
// + 3 of column l % 16.  Of 16 consecutive k, lane group c takes 4 c .. 4 c + 3 in four instructions, so that a lane's
// operands are four consecutive elements.
#include "chunked.h"

#define CK_ROWS TLI_CHUNK_ROWS
#define CK_THREADS 256

typedef float ck_f32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t ck_u32x4 __attribute__((ext_vector_type(4)));

struct ChunkRows {                                       // what both kinds read and write
    const bf16_t* proj;                                  // [T, ld]: q (H dk) | k (H dk) | v (H dv) | gate (H dv)
    int ld;
    float* state;                                        // [slots][H][OV][dk], OV = dv, or dv + 1 with a normaliser
    float* before;                                       // scratch [chunks][H][OV][dk]: S before every chunk
    const int* row_start;
    const int* seq_start;
    const int* slots;
    int T, seqs, H, dk, dv;
};

struct ChunkRotation {                                   // of q and k, and the factors behind it
    const float* cos_table;                              // [table_positions, dims / 2] or null
    const float* sin_table;
    int dims, pairing, table_positions;
    float q_scale, k_scale;
};

struct ChunkDecay {
    const float* head;                                   // [H]: one factor a head and w = 1; or null, and then, [H][T]:
    const float* through;                                // log A_t
    const float* take;                                   // w_t
};

// How q and k turn: not at all, pair i being (i, i + dims/2), or (2i, 2i + 1).  Pieces of 4 or 8 elements lie on one side of
// every border (dims and half of it are multiples of 8, for neighbours dims is).  Elements past the turned ones turn by
// an angle of 0, so that no load stands behind a condition.
enum { ROT_NONE = 0, ROT_HALVES = 1, ROT_NEIGHBOURS = 2 };

__device__ __forceinline__ void ck_widen(const uint2& w, float (&v)[4]) {
    v[0] = bf16_to_f32((bf16_t)(w.x & 0xffffu)), v[1] = bf16_to_f32((bf16_t)(w.x >> 16));
    v[2] = bf16_to_f32((bf16_t)(w.y & 0xffffu)), v[3] = bf16_to_f32((bf16_t)(w.y >> 16));
}
__device__ __forceinline__ void ck_widen(const uint4& w, float (&v)[8]) {
    const uint32_t u[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) v[2 * i] = bf16_to_f32((bf16_t)(u[i] & 0xffffu)), v[2 * i + 1] = bf16_to_f32((bf16_t)(u[i] >> 16));
}

// Four elements of a row of q from dim d on and what turns them, as they are loaded.
struct QueryPiece {
    uint2 raw, other;        // halves: the partners
    float4 c, s;             // halves: of four pairs; neighbours: of two
};
template <int ROT>
__device__ __forceinline__ void ck_query_fetch(const bf16_t* head, int d, const ChunkRotation& rot, int pos, QueryPiece& q) {
    q.raw = *reinterpret_cast<const uint2*>(head + d);
    if constexpr (ROT == ROT_NONE) return;
    const int half = rot.dims / 2;
    const bool in = d < rot.dims, second = d >= half;
    if (ROT == ROT_HALVES) {
        q.other = *reinterpret_cast<const uint2*>(head + (!in ? d : second ? d - half : d + half));
        const size_t at = (size_t)pos * half + (!in ? 0 : second ? d - half : d);
        q.c = *reinterpret_cast<const float4*>(rot.cos_table + at);
        q.s = *reinterpret_cast<const float4*>(rot.sin_table + at);
    } else {
        const size_t at = (size_t)pos * half + (in ? d / 2 : 0);
        const float2 c = *reinterpret_cast<const float2*>(rot.cos_table + at), s = *reinterpret_cast<const float2*>(rot.sin_table + at);
        q.c = make_float4(c.x, c.y, 0.f, 0.f);
        q.s = make_float4(s.x, s.y, 0.f, 0.f);
    }
}
template <int ROT>
__device__ __forceinline__ void ck_query_turn(const QueryPiece& q, int d, const ChunkRotation& rot, float (&x)[4]) {
    ck_widen(q.raw, x);
    if constexpr (ROT == ROT_NONE) return;
    if (d >= rot.dims) return;
    const float c[4] = {q.c.x, q.c.y, q.c.z, q.c.w}, s[4] = {q.s.x, q.s.y, q.s.z, q.s.w};
    if (ROT == ROT_HALVES) {
        float other[4];
        ck_widen(q.other, other);
        const bool second = d >= rot.dims / 2;
#pragma unroll
        for (int i = 0; i < 4; ++i)
            x[i] = second ? rotate_second_half(x[i], other[i], c[i], s[i]) : rotate_first_half(x[i], other[i], c[i], s[i]);
    } else {
#pragma unroll
        for (int p = 0; p < 2; ++p) {
            const float a = x[2 * p], b = x[2 * p + 1];
            x[2 * p] = rotate_first_half(a, b, c[p], s[p]);
            x[2 * p + 1] = rotate_second_half(b, a, c[p], s[p]);
        }
    }
}

// Two pieces of 8 elements of a row of K and the rotation's entries for them, as they are loaded: asked for early, made
// into float32 where they are needed.  Pieces that turn together (halves) are one pair; of the others, and of
// neighbours, two pieces side by side are.
struct KeyPair {
    uint4 raw[2];
    float4 c[2], s[2];       // halves: of eight pairs; neighbours: of four for each piece
};
template <int ROT>
__device__ __forceinline__ void ck_pair_dims(int u, const ChunkRotation& rot, int& d1, int& d2) {
    const int together = ROT == ROT_HALVES ? rot.dims / 16 : 0;        // pairs of pieces of the two halves
    d1 = u < together ? 8 * u : (ROT == ROT_HALVES ? rot.dims : 0) + 16 * (u - together);
    d2 = u < together ? d1 + rot.dims / 2 : d1 + 8;
}
template <int ROT>
__device__ __forceinline__ void ck_pair_fetch(const bf16_t* head, int u, const ChunkRotation& rot, KeyPair& k) {
    int d1, d2;
    ck_pair_dims<ROT>(u, rot, d1, d2);
    k.raw[0] = *reinterpret_cast<const uint4*>(head + d1);
    k.raw[1] = *reinterpret_cast<const uint4*>(head + d2);
}
template <int ROT>
__device__ __forceinline__ void ck_pair_angles(int u, const ChunkRotation& rot, int pos, KeyPair& k) {
    if constexpr (ROT == ROT_NONE) return;
    int d1, d2;
    ck_pair_dims<ROT>(u, rot, d1, d2);
    const size_t row = (size_t)pos * (rot.dims / 2);
    size_t first = row, second = row;
    if (ROT == ROT_HALVES) {
        first += d1 < rot.dims ? d1 : 0;
        second = first + 4;
    } else {
        first += d1 < rot.dims ? d1 / 2 : 0;
        second += d2 < rot.dims ? d2 / 2 : 0;
    }
    k.c[0] = *reinterpret_cast<const float4*>(rot.cos_table + first), k.c[1] = *reinterpret_cast<const float4*>(rot.cos_table + second);
    k.s[0] = *reinterpret_cast<const float4*>(rot.sin_table + first), k.s[1] = *reinterpret_cast<const float4*>(rot.sin_table + second);
}
template <int ROT>
__device__ __forceinline__ void ck_pair_turn(const KeyPair& k, int u, const ChunkRotation& rot, int& d1, int& d2, float (&x)[8], float (&y)[8]) {
    ck_pair_dims<ROT>(u, rot, d1, d2);
    ck_widen(k.raw[0], x);
    ck_widen(k.raw[1], y);
    if constexpr (ROT == ROT_NONE) return;
    const float c[8] = {k.c[0].x, k.c[0].y, k.c[0].z, k.c[0].w, k.c[1].x, k.c[1].y, k.c[1].z, k.c[1].w};
    const float s[8] = {k.s[0].x, k.s[0].y, k.s[0].z, k.s[0].w, k.s[1].x, k.s[1].y, k.s[1].z, k.s[1].w};
    if (ROT == ROT_HALVES) {
        if (d1 >= rot.dims) return;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const float a = x[i], b = y[i];
            x[i] = rotate_first_half(a, b, c[i], s[i]);
            y[i] = rotate_second_half(b, a, c[i], s[i]);
        }
    } else {
#pragma unroll
        for (int p = 0; p < 4; ++p) {
            if (d1 < rot.dims) {
                const float a = x[2 * p], b = x[2 * p + 1];
                x[2 * p] = rotate_first_half(a, b, c[p], s[p]);
                x[2 * p + 1] = rotate_second_half(b, a, c[p], s[p]);
            }
            if (d2 < rot.dims) {
                const float a = y[2 * p], b = y[2 * p + 1];
                y[2 * p] = rotate_first_half(a, b, c[4 + p], s[4 + p]);
                y[2 * p + 1] = rotate_second_half(b, a, c[4 + p], s[4 + p]);
            }
        }
    }
}

__device__ __forceinline__ int ck_chunks(int rows) { return (rows + CK_ROWS - 1) / CK_ROWS; }

#define CK_PAIRS 2           // pairs of pieces of k (16 elements each) a workgroup of chunk_states
#define CK_VDIMS 64          // elements of v
#define CK_KLD (CK_ROWS + 4)

template <bool MEMORY, int ROT>
__global__ __launch_bounds__(CK_THREADS) void chunk_states_kernel(ChunkRows a, ChunkRotation rot, ChunkDecay decay) {
    __shared__ __align__(16) float kt[2][CK_PAIRS * 16][CK_KLD];       // the chunk's weighted keys, transposed
    const int tid = threadIdx.x, lane = tid % TLI_WAVE, wave = tid / TLI_WAVE, col = lane % 16, grp = lane / 16;
    const int dk = a.dk, dv = a.dv, H = a.H, OV = dv + (MEMORY ? 1 : 0);
    const int pairs = dk / 16, k_slices = (pairs + CK_PAIRS - 1) / CK_PAIRS;
    const int u0 = (blockIdx.x % k_slices) * CK_PAIRS, dv0 = (blockIdx.x / k_slices) * CK_VDIMS;
    const int h = blockIdx.y, seq = blockIdx.z;
    const int r0 = a.row_start[seq], n = a.row_start[seq + 1] - r0;
    if (n <= 0) return;
    int z0 = 0;
    for (int i = 0; i < seq; ++i) z0 += ck_chunks(a.row_start[i + 1] - a.row_start[i]);
    const int chunks = ck_chunks(n), pos0 = a.seq_start[seq];
    const int j = dv0 + wave * 16 + col;                               // this lane's column of S
    const bool mine = dv0 + wave * 16 < dv;
    const bool norm_too = MEMORY && dv0 == 0 && wave == 0;             // this wave keeps n of these elements of k as well
    const int tiles = min(CK_PAIRS, pairs - u0);                       // of 16 elements of k: tile t's rows of kt are pair u0 + t's pieces
    // element of k that row r (0..15) of a tile's is, and the first of the four consecutive ones from row 4 grp on
    int dim_col[CK_PAIRS], dim_grp[CK_PAIRS];
#pragma unroll
    for (int t = 0; t < CK_PAIRS; ++t) {
        int d1, d2;
        ck_pair_dims<ROT>(min(u0 + t, pairs - 1), rot, d1, d2);
        dim_col[t] = col < 8 ? d1 + col : d2 + col - 8;
        dim_grp[t] = grp < 2 ? d1 + 4 * grp : d2 + 4 * grp - 8;
    }
    float* slot = a.state + ((size_t)a.slots[seq] * H + h) * OV * dk;
    const bool fresh = pos0 == 0;
    ck_f32x4 S[CK_PAIRS];
    float nk[CK_PAIRS];
#pragma unroll
    for (int t = 0; t < CK_PAIRS; ++t) {
        S[t] = (ck_f32x4){0.f, 0.f, 0.f, 0.f};
        nk[t] = 0.f;
        if (fresh || t >= tiles) continue;
        if (mine) S[t] = *reinterpret_cast<const ck_f32x4*>(slot + (size_t)j * dk + dim_grp[t]);
        if (norm_too) nk[t] = slot[(size_t)dv * dk + dim_col[t]];
    }
    const bf16_t* k_head = a.proj + (size_t)r0 * a.ld + (size_t)(H + h) * dk;
    const bf16_t* v_head = a.proj + (size_t)r0 * a.ld + (size_t)2 * H * dk + (size_t)h * dv;      // (the same for all lanes)
    const uint32_t v_lane = (uint32_t)(4 * grp) * a.ld + (mine ? j : 0);
    // half of the threads bring a chunk's keys (a pair of pieces each), the two halves every second chunk
    const int kr = (tid / CK_PAIRS) % CK_ROWS, ku = tid % CK_PAIRS, k_turn = tid / (CK_PAIRS * CK_ROWS);
    const bool k_mine = ku < tiles;
    const float lam = MEMORY ? 0.f : decay.head[h];
    const float* through = MEMORY ? decay.through + (size_t)h * a.T + r0 : nullptr;
    const float* takes = MEMORY ? decay.take + (size_t)h * a.T + r0 : nullptr;
    const float whole = MEMORY ? 0.f : powf(lam, (float)CK_ROWS), w_whole = MEMORY ? 0.f : powf(lam, (float)(CK_ROWS - 1 - kr)) * rot.k_scale;
    const int tail = n - (chunks - 1) * CK_ROWS;                       // rows of the last chunk
    KeyPair kp;
    float w_end = 0.f, w_row = 0.f, w_take = 0.f;
    auto fetch_keys = [&](int z) {
        const int first = z * CK_ROWS, last = min(first + CK_ROWS, n) - 1, r = min(first + kr, last);
        const int u = u0 + min(ku, tiles - 1);
        ck_pair_fetch<ROT>(k_head + (size_t)r * a.ld, u, rot, kp);
        ck_pair_angles<ROT>(u, rot, pos0 + r, kp);
        if (MEMORY) w_end = through[last], w_row = through[r], w_take = takes[r];
    };
    auto store_keys = [&](int z) {
        float x[8], y[8], w = w_whole;
        int d1, d2;
        ck_pair_turn<ROT>(kp, u0 + ku, rot, d1, d2, x, y);
        if (MEMORY) w = expf(w_end - w_row) * w_take;
        else if (z == chunks - 1 && tail < CK_ROWS) w = powf(lam, (float)max(tail - 1 - kr, 0)) * rot.k_scale;
        if (z == chunks - 1 && kr >= tail) w = 0.f;
        if (!k_mine) return;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            kt[z & 1][16 * ku + e][kr] = x[e] * w;
            kt[z & 1][16 * ku + 8 + e][kr] = y[e] * w;
        }
    };
    auto fetch_values = [&](int z, bf16_t (&v)[16], float& end) {
        const int first = z * CK_ROWS;
        if (MEMORY) end = through[min(first + CK_ROWS, n) - 1];
        const bf16_t* base = v_head + (size_t)first * a.ld;
        if (z < chunks - 1 || tail == CK_ROWS) {
#pragma unroll
            for (int s = 0; s < 4; ++s)
#pragma unroll
                for (int i = 0; i < 4; ++i) v[4 * s + i] = (base + (size_t)(16 * s + i) * a.ld)[v_lane];
        } else {
#pragma unroll
            for (int s = 0; s < 4; ++s)
#pragma unroll
                for (int i = 0; i < 4; ++i) v[4 * s + i] = base[(size_t)min(16 * s + 4 * grp + i, tail - 1) * a.ld + (mine ? j : 0)];
        }
    };
    auto walk = [&](int z, const bf16_t (&v)[16], float end) {
        float* P = a.before + ((size_t)(z0 + z) * H + h) * OV * dk;
        const float g = MEMORY ? expf(end) : z == chunks - 1 && tail < CK_ROWS ? powf(lam, (float)tail) : whole;
#pragma unroll
        for (int t = 0; t < CK_PAIRS; ++t) {
            if (t < tiles) {
                if (mine) *reinterpret_cast<ck_f32x4*>(P + (size_t)j * dk + dim_grp[t]) = S[t];
                if (norm_too && grp == 0) P[(size_t)dv * dk + dim_col[t]] = nk[t];
            }
#pragma unroll
            for (int i = 0; i < 4; ++i) S[t][i] *= g;
        }
        float sum[CK_PAIRS] = {};
#pragma unroll
        for (int s = 0; s < 4; ++s) {
#pragma unroll
            for (int t = 0; t < CK_PAIRS; ++t) {
                const ck_f32x4 kk = *reinterpret_cast<const ck_f32x4*>(&kt[z & 1][16 * t + col][16 * s + 4 * grp]);
#pragma unroll
                for (int i = 0; i < 4; ++i) S[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(kk[i], bf16_to_f32(v[4 * s + i]), S[t], 0, 0, 0);
                if (MEMORY) sum[t] += (kk[0] + kk[1]) + (kk[2] + kk[3]);
            }
        }
        if (norm_too) {
#pragma unroll
            for (int t = 0; t < CK_PAIRS; ++t) nk[t] = fmaf(g, nk[t], quad_rows_sum(sum[t]));
        }
    };
    // A chunk's keys are asked for two chunks ahead, each half of the threads having one chunk's on the way, its values
    // one ahead.  (A tile without elements of k, t >= tiles, multiplies what LDS holds and is not stored.)
    bf16_t v0[16], v1[16];
    float end0 = 0.f, end1 = 0.f;                        // the last log A of the chunks whose values are in v0 and v1
    if (k_turn < chunks) fetch_keys(k_turn);
    fetch_values(0, v0, end0);
    if (k_turn == 0) {
        store_keys(0);
        if (2 < chunks) fetch_keys(2);
    }
    __syncthreads();
    for (int z = 0; z < chunks; ++z) {
        // chunk z is in kt[z & 1]; the other buffer was last read before the barrier
        if (z + 1 < chunks) {
            if (z & 1) fetch_values(z + 1, v0, end0);
            else fetch_values(z + 1, v1, end1);
            if (k_turn == ((z + 1) & 1)) {
                store_keys(z + 1);
                if (z + 3 < chunks) fetch_keys(z + 3);
            }
        }
        if (z & 1) walk(z, v1, end1);
        else walk(z, v0, end0);
        __syncthreads();
    }
#pragma unroll
    for (int t = 0; t < CK_PAIRS; ++t) {
        if (t >= tiles) continue;
        if (mine) *reinterpret_cast<ck_f32x4*>(slot + (size_t)j * dk + dim_grp[t]) = S[t];
        if (norm_too && grp == 0) slot[(size_t)dv * dk + dim_col[t]] = nk[t];
    }
}

struct ChunkOutput {
    bf16_t* out;                                         // rows out_ld elements apart, H dv of each
    int out_ld;
    const float* weight;                                 // [H dv] or null
    const float* floors;                                 // [H][T]: exp(-m), with a normaliser
    float eps, scale;
};

static inline size_t ck_lds_floats(int dk, int dv) {
    const size_t state = (size_t)dv * (dk + 4), rows = (size_t)CK_ROWS * (dk + 4 + dv + 4);
    return state > rows ? state : rows;
}

// MEMORY: with a normaliser and the logistic gate; else the silu gate.  NK, NV: sixteens of a head (EXACT), or their
// bound: sixteens past a head's are multiplied all the same, q's as zeros and v's into sums that nobody reads, from
// addresses of the head's last, so that no matrix instruction stands behind a condition
template <bool MEMORY, int ROT, int NK, int NV, bool EXACT>
__global__ __launch_bounds__(CK_THREADS, 2) void chunk_outputs_kernel(ChunkRows a, ChunkRotation rot, ChunkDecay decay, ChunkOutput out) {
    extern __shared__ __align__(16) float ck_lds[];
    __shared__ float log_s[CK_ROWS], take_s[CK_ROWS];                  // mLSTM: log A and w; else the powers of the decay
    const int tid = threadIdx.x, lane = tid % TLI_WAVE, wave = __builtin_amdgcn_readfirstlane(tid / TLI_WAVE), col = lane % 16, grp = lane / 16;
    const int nk = EXACT ? NK : a.dk / 16, nv = EXACT ? NV : a.dv / 16;
    const int dk = nk * 16, dv = nv * 16, H = a.H, OV = dv + (MEMORY ? 1 : 0), KLD = dk + 4, VLD = dv + 4;
    const int h = blockIdx.y;
    int z = blockIdx.x, seq = 0, n = 0;
    for (; seq < a.seqs; ++seq) {
        n = a.row_start[seq + 1] - a.row_start[seq];
        const int c = ck_chunks(n);
        if (z < c) break;
        z -= c;
    }
    if (seq >= a.seqs) return;                                         // (the grid's slack)
    const int r0 = a.row_start[seq] + z * CK_ROWS, count = min(CK_ROWS, n - z * CK_ROWS);
    const bool from_nothing = z == 0 && a.seq_start[seq] == 0;
    const float* P = a.before + ((size_t)blockIdx.x * H + h) * OV * dk;
    const bf16_t* rows = a.proj + (size_t)r0 * a.ld;
    const float lam = MEMORY ? 0.f : decay.head[h];
    // a wave's tile of 16 rows: the later a tile, the more scores it has, so every second round of workgroups deals them out
    // the other way round
    const int rt = ((blockIdx.y * gridDim.x + blockIdx.x) >> 8) & 1 ? CK_ROWS / 16 - 1 - wave : wave;
    const int i = 16 * rt + col;                                       // this lane's row of the chunk
    const int row = min(i, count - 1), pos0 = a.seq_start[seq] + z * CK_ROWS;
    const bool works = 16 * rt < count;                                // (the same for the whole wave)

    // everything that the workgroup reads is asked for at once: P, q, K and V (K's and V's stay in registers until P's place
    // in LDS is free)
    constexpr int PP = (NK * NV * 16 * 16 / 4 + CK_THREADS - 1) / CK_THREADS, KP = (CK_ROWS * NK + CK_THREADS - 1) / CK_THREADS;
    constexpr int VP = (CK_ROWS * NV * 2 + CK_THREADS - 1) / CK_THREADS;
    const int p_row = dk / 4, p_all = dv * p_row;
    ck_f32x4 pr[PP];                                                   // (a native vector type: an array of float4 would go to memory)
    if (!from_nothing) {
#pragma unroll
        for (int u = 0; u < PP; ++u) {
            const int p = tid + u * CK_THREADS;
            pr[u] = *reinterpret_cast<const ck_f32x4*>(P + (size_t)min(p, p_all - 1) * 4);
        }
    }
    KeyPair kp[KP];
    ck_u32x4 vr[VP];
#pragma unroll
    for (int u = 0; u < KP; ++u) {
        const int p = min(tid + u * CK_THREADS, count * nk - 1), r = p / nk;
        ck_pair_fetch<ROT>(rows + (size_t)r * a.ld + (size_t)(H + h) * dk, p - r * nk, rot, kp[u]);
    }
#pragma unroll
    for (int u = 0; u < VP; ++u) {
        const int p = min(tid + u * CK_THREADS, count * nv * 2 - 1), r = p / (nv * 2);
        vr[u] = *reinterpret_cast<const ck_u32x4*>(rows + (size_t)r * a.ld + (size_t)2 * H * dk + (size_t)h * dv + (p - r * nv * 2) * 8);
    }
    if (tid < CK_ROWS) {
        if constexpr (MEMORY) {
            const bool live = tid < count;
            log_s[tid] = live ? decay.through[(size_t)h * a.T + r0 + tid] : 0.f;
            take_s[tid] = live ? decay.take[(size_t)h * a.T + r0 + tid] : 0.f;
        } else {
            log_s[tid] = powf(lam, (float)tid);                        // lam^0 .. lam^63
        }
    }
    auto k_tile = [&](int b) { return EXACT ? b : min(b, nk - 1); };
    auto v_tile = [&](int t) { return EXACT ? t : min(t, nv - 1); };
    float q[NK][4];
    {
        QueryPiece piece[NK];
        const bf16_t* q_row = rows + (size_t)row * a.ld + (size_t)h * dk;
#pragma unroll
        for (int b = 0; b < NK; ++b) ck_query_fetch<ROT>(q_row, 16 * k_tile(b) + 4 * grp, rot, pos0 + row, piece[b]);
#pragma unroll
        for (int b = 0; b < NK; ++b) {
            ck_query_turn<ROT>(piece[b], 16 * k_tile(b) + 4 * grp, rot, q[b]);
#pragma unroll
            for (int e = 0; e < 4; ++e) q[b][e] = b < nk ? q[b][e] * rot.q_scale : 0.f;
        }
    }
    ck_f32x4 acc[NV];
#pragma unroll
    for (int t = 0; t < NV; ++t) acc[t] = (ck_f32x4){0.f, 0.f, 0.f, 0.f};
    float nq = 0.f;                                                    // n . q of this lane's row, this lane group's share
    if (!from_nothing) {                                               // P, [dv][dk]
#pragma unroll
        for (int u = 0; u < PP; ++u) {
            const int p = tid + u * CK_THREADS;
            if (p < p_all) *reinterpret_cast<ck_f32x4*>(ck_lds + (p / p_row) * KLD + (p % p_row) * 4) = pr[u];
        }
    }
#pragma unroll
    for (int u = 0; u < KP; ++u) {                                     // (while the products with P run)
        const int p = min(tid + u * CK_THREADS, count * nk - 1), r = p / nk;
        ck_pair_angles<ROT>(p - r * nk, rot, pos0 + r, kp[u]);
    }
    __syncthreads();
    if (!from_nothing && works) {
        const float g = MEMORY ? expf(log_s[row]) : log_s[row] * lam;  // A of the row
#pragma unroll
        for (int b = 0; b < NK; ++b) {
            if constexpr (MEMORY) {
                const float4 nn = *reinterpret_cast<const float4*>(P + (size_t)dv * dk + 16 * k_tile(b) + 4 * grp);
                nq += q[b][0] * nn.x + q[b][1] * nn.y + q[b][2] * nn.z + q[b][3] * nn.w;
            }
            ck_f32x4 p[NV];
#pragma unroll
            for (int t = 0; t < NV; ++t)
                p[t] = *reinterpret_cast<const ck_f32x4*>(ck_lds + (16 * v_tile(t) + col) * KLD + 16 * k_tile(b) + 4 * grp);
#pragma unroll
            for (int e = 0; e < 4; ++e)
#pragma unroll
                for (int t = 0; t < NV; ++t)
                    acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(p[t][e], q[b][e], acc[t], 0, 0, 0);
        }
        nq *= g;
#pragma unroll
        for (int t = 0; t < NV; ++t)
#pragma unroll
            for (int e = 0; e < 4; ++e) acc[t][e] *= g;
    }
    __syncthreads();                                                   // P has been read
    float* k_s = ck_lds;                                               // [row][dk + 4]
    float* v_s = ck_lds + CK_ROWS * KLD;                               // [row][dv + 4]
#pragma unroll
    for (int u = 0; u < KP; ++u) {
        const int p = tid + u * CK_THREADS, r = p / nk;
        if (p >= count * nk) continue;
        float x[8], y[8];
        int d1, d2;
        ck_pair_turn<ROT>(kp[u], p - r * nk, rot, d1, d2, x, y);
        float* dst = k_s + r * KLD;
#pragma unroll
        for (int e = 0; e < 8; ++e) dst[d1 + e] = x[e] * rot.k_scale;
#pragma unroll
        for (int e = 0; e < 8; ++e) dst[d2 + e] = y[e] * rot.k_scale;
    }
#pragma unroll
    for (int u = 0; u < VP; ++u) {
        const int p = tid + u * CK_THREADS, r = p / (nv * 2);
        if (p >= count * nv * 2) continue;
        float x[8];
        ck_widen(make_uint4(vr[u][0], vr[u][1], vr[u][2], vr[u][3]), x);
        float* dst = v_s + r * VLD + (p - r * nv * 2) * 8;
#pragma unroll
        for (int e = 0; e < 8; ++e) dst[e] = x[e];
    }
    __syncthreads();
    if (!works) return;
    const float my_log = MEMORY ? log_s[row] : 0.f;
    for (int jt = 0; jt <= rt; ++jt) {
        // (rows of K and V past the chunk's last are what was in LDS before: their scores are set to 0, and their
        // values are read from the last row)
        ck_f32x4 s[2] = {(ck_f32x4){0.f, 0.f, 0.f, 0.f}, (ck_f32x4){0.f, 0.f, 0.f, 0.f}};
        const float* k_row = k_s + min(16 * jt + col, count - 1) * KLD + 4 * grp;
#pragma unroll
        for (int b = 0; b < NK; ++b) {
            const ck_f32x4 kk = *reinterpret_cast<const ck_f32x4*>(k_row + 16 * k_tile(b));
#pragma unroll
            for (int e = 0; e < 4; ++e) s[e & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(kk[e], q[b][e], s[e & 1], 0, 0, 0);
        }
        float p[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {                                  // row 16 jt + 4 grp + e of K against this lane's row
            const int j = 16 * jt + 4 * grp + e;
            float w = 0.f;
            if (j <= i && j < count) w = MEMORY ? expf(my_log - log_s[j]) * take_s[j] : log_s[i - j];
            p[e] = (s[0][e] + s[1][e]) * w;
            if (MEMORY) nq += p[e];
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const float* v_row = v_s + min(16 * jt + 4 * grp + e, count - 1) * VLD + col;
#pragma unroll
            for (int t = 0; t < NV; ++t)
                acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(v_row[16 * v_tile(t)], p[e], acc[t], 0, 0, 0);
        }
    }
    // the head's norm and gate: this lane has elements 16 t + 4 grp .. + 3 of its row
    float by = 1.f;
    if constexpr (MEMORY) by = 1.f / (fmaxf(fabsf(quad_rows_sum(nq)), out.floors[(size_t)h * a.T + r0 + row]) + 1e-6f);
    float ss = 0.f;
#pragma unroll
    for (int t = 0; t < NV; ++t)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            acc[t][e] *= by;
            if (t < nv) ss = fmaf(acc[t][e], acc[t][e], ss);
        }
    const float factor = out.scale / sqrtf(quad_rows_sum(ss) / (float)dv + out.eps);
    if (i >= count) return;
    const bf16_t* gate = rows + (size_t)i * a.ld + (size_t)H * (2 * dk + dv) + (size_t)h * dv;
    bf16_t* dst = out.out + (size_t)(r0 + i) * out.out_ld + (size_t)h * dv;
#pragma unroll
    for (int t = 0; t < NV; ++t) {
        if (t >= nv) continue;
        const int d = 16 * t + 4 * grp;
        float g[4], y[4];
        ck_widen(*reinterpret_cast<const uint2*>(gate + d), g);
        float wt[4] = {1.f, 1.f, 1.f, 1.f};
        if (out.weight) {
            const float4 w4 = *reinterpret_cast<const float4*>(out.weight + (size_t)h * dv + d);
            wt[0] = w4.x, wt[1] = w4.y, wt[2] = w4.z, wt[3] = w4.w;
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] = acc[t][e] * factor * wt[e] * ((MEMORY ? 1.f : g[e]) / (1.f + expf(-g[e])));
        *reinterpret_cast<uint2*>(dst + d) = make_uint2(pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3]));
    }
}

// Whether rows of these sizes go through here (else the shared recurrence serves): dims turned elements (0: none).
extern "C" int tli_chunked_takes(int dk, int dv, int dims, int pairing) {
    if (dk % 16 || dv % 16 || dk < 16 || dv < 16 || dk > 128 || dv > 128) return 0;
    return dims % (pairing ? 8 : 16) == 0;
}

// float32 elements of scratch for T rows in `seqs` sequences; OV: dv, or dv + 1 with a normaliser
extern "C" long long tli_chunked_scratch_floats(int T, int seqs, int H, int dk, int OV) {
    return ((long long)T / CK_ROWS + seqs) * H * OV * dk;
}

template <bool MEMORY>
static int run_chunked(const ChunkRows& a, const ChunkRotation& rot, const ChunkDecay& decay, const ChunkOutput& out, hipStream_t s) {
    const int zs = a.T / CK_ROWS + a.seqs;               // (an upper bound of the chunks; a workgroup past the last leaves)
    if (a.H > 65535 || a.seqs > 65535) return tli_fail("chunked recurrence: too many heads or sequences for one launch");
    if (a.ld % 8 || a.ld < 2 * a.H * (a.dk + a.dv)) return tli_fail("chunked recurrence: rows of %d elements", a.ld);
    if (out.out_ld % 4 || out.out_ld < a.H * a.dv) return tli_fail("chunked recurrence: output rows of %d elements", out.out_ld);
    if ((((uintptr_t)a.proj | (uintptr_t)a.state | (uintptr_t)a.before | (uintptr_t)out.weight | (uintptr_t)rot.cos_table | (uintptr_t)rot.sin_table) & 15) ||
        ((uintptr_t)out.out & 7))
        return tli_fail("chunked recurrence: operands must be 16-byte aligned");
    const int slices = ((a.dk / 16 + CK_PAIRS - 1) / CK_PAIRS) * ((a.dv + CK_VDIMS - 1) / CK_VDIMS);
    const dim3 states_grid(slices, a.H, a.seqs);
    const size_t lds = ck_lds_floats(a.dk, a.dv) * sizeof(float);
    const dim3 grid(zs, a.H);
#define CK_RUN(ROT, NK, NV, EXACT)                                                                                          \
    {                                                                                                                       \
        auto kernel = chunk_outputs_kernel<MEMORY, ROT, NK, NV, EXACT>;                                                     \
        static bool allowed = false;                                                                                        \
        if (lds > 60 * 1024 && !allowed) {                                                                                  \
            if (hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 72 * 1024) !=          \
                hipSuccess)                                                                                                 \
                return tli_fail("chunked recurrence: cannot have %zu bytes of LDS", lds);                                   \
            allowed = true;                                                                                                 \
        }                                                                                                                   \
        kernel<<<grid, CK_THREADS, lds, s>>>(a, rot, decay, out);                                                           \
    }
#define CK_SIZES(ROT)                                                                                                       \
    {                                                                                                                       \
        chunk_states_kernel<MEMORY, ROT><<<states_grid, CK_THREADS, 0, s>>>(a, rot, decay);                                 \
        if (a.dk == 128 && a.dv == 128) CK_RUN(ROT, 8, 8, true)                                                             \
        else if (a.dk == 64 && a.dv == 64) CK_RUN(ROT, 4, 4, true)                                                          \
        else if (a.dk <= 32 && a.dv <= 32) CK_RUN(ROT, 2, 2, false)                                                         \
        else if (a.dk <= 64 && a.dv <= 64) CK_RUN(ROT, 4, 4, false)                                                         \
        else CK_RUN(ROT, 8, 8, false)                                                                                       \
    }
    if constexpr (MEMORY) CK_SIZES(ROT_NONE)
    else if (!rot.cos_table) CK_SIZES(ROT_NONE)
    else if (rot.pairing) CK_SIZES(ROT_NEIGHBOURS)
    else CK_SIZES(ROT_HALVES)
#undef CK_SIZES
#undef CK_RUN
    return tli_check_launch("chunked recurrence");
}

// bfloat16 rows; the arguments as for tli_retention_step (recurrent_step.hip), row_start [seqs + 1], seq_start, slots
// [seqs]; scratch: tli_chunked_scratch_floats(T, seqs, H, dk, dv) floats
extern "C" int tli_retention_chunked_bf16(const void* proj, int ld, const float* decay, float* state, void* out, int out_ld,
                                          float* scratch, const int* row_start, const int* seq_start,
                                          const int* slots, const float* cos_table, const float* sin_table, int dims, int pairing,
                                          int table_positions, float k_scale, float eps, float scale, int T, int seqs, int H, int dk,
                                          int dv, void* stream) {
    if (T <= 0 || seqs <= 0) return 0;
    if (H <= 0 || !tli_chunked_takes(dk, dv, cos_table ? dims : 0, pairing) || (cos_table && (dims <= 0 || dims > dk)))
        return tli_fail("retention in chunks: heads of %d and %d with %d turned elements", dk, dv, dims);
    const ChunkRows a{(const bf16_t*)proj, ld, state, scratch, row_start, seq_start, slots, T, seqs, H, dk, dv};
    return run_chunked<false>(a, ChunkRotation{cos_table, sin_table, dims, pairing, table_positions, 1.0f, k_scale},
                              ChunkDecay{decay, nullptr, nullptr}, ChunkOutput{(bf16_t*)out, out_ld, nullptr, nullptr, eps, scale},
                              (hipStream_t)stream);
}

// bfloat16 rows; the arguments as for tli_mlstm (mlstm.hip) and tli_mlstm_step; scratch: tli_chunked_scratch_floats(T, seqs,
// H, dk, dv + 1) floats, rows_scratch: 4 H T floats
extern "C" int tli_mlstm_chunked_bf16(const void* proj, int ld, const float* z, long long z_row, long long z_col, const float* ssq,
                                      int parts, int x_size, float x_eps, const float* bias, float cap, float q_scale,
                                      const float* weight, float* m_state, float* state, void* out, int out_ld, float* scratch,
                                      float* rows_scratch, const int* row_start, const int* seq_start, const int* slots, float eps,
                                      float scale, int T, int seqs, int H, int dk, int dv, void* stream) {
    if (T <= 0 || seqs <= 0) return 0;
    if (H <= 0 || H > 65535 || seqs > 65535 || !tli_chunked_takes(dk, dv, 0, 0)) return tli_fail("mlstm in chunks: heads of %d and %d", dk, dv);
    if (!(cap > 0.f)) return tli_fail("mlstm: the gates' cap must be positive");
    if (ssq && (parts <= 0 || x_size <= 0)) return tli_fail("mlstm: bad sums of squares");
    hipStream_t s = (hipStream_t)stream;
    const size_t per = (size_t)H * T;
    float *keep = rows_scratch, *take = keep + per, *through = take + per, *floors = through + per;
    const MlGates gates{z, z_row, z_col, bias, cap, H, RowFactor{ssq, ssq ? parts : 0, T, 1.0f / (float)(x_size > 0 ? x_size : 1), x_eps}};
    if (tli_mlstm_scan(gates, m_state, keep, take, floors, through, CK_ROWS, row_start, seq_start, slots, T, seqs, s)) return 1;
    const ChunkRows a{(const bf16_t*)proj, ld, state, scratch, row_start, seq_start, slots, T, seqs, H, dk, dv};
    return run_chunked<true>(a, ChunkRotation{nullptr, nullptr, 0, 0, 0, q_scale, 1.0f}, ChunkDecay{nullptr, through, take},
                             ChunkOutput{(bf16_t*)out, out_ld, weight, floors, eps, scale}, s);
}
