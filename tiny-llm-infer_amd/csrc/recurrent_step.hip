// Decode steps of the recurrent layers whose heads are normed one by one (retention.hip, mlstm.hip, wkv.hip): every sequence brings
// one row, and everything between the layer's products is one launch, a workgroup a (head, row).
//   retention:  q, k turned, k scaled; S <- c S + k v^T; o = S^T q; unit RMS; silu gate
//   mLSTM:      the two gates' logits (two dot products over the layer's input, which no other head shares), m, S <- a S +
//               b k v^T, n likewise, o = S^T q / (max(|n q|, exp(-m)) + 1e-6); RMS times the weight; logistic gate
//   wkv:        d = exp(-exp(W2 tanh(z) + w0)) a channel; o = (S + diag(u) k v^T)^T r; S <- diag(d) S + k v^T; RMS times the
//               weight; silu gate
// A column of S belongs to 16 lanes of a wave, a lane holding R elements of it (as in lightning.hip: pieces of up to four
// that lie side by side with the other lanes').  A workgroup takes 16 columns at a time and asks for the first GROUPS x 16
// columns before anything else, so that the state's bytes, which are nearly all that such a step moves, are on their
// way while the row's q, k, v and gates are made.
#include "recurrence.h"
#include "row_gates.h"

#define RS_THREADS 256

__device__ __forceinline__ float rs_sum16(float v) {     // over the 16 lanes of a DPP row; every lane gets it
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0xB1, 0xF, 0xF, true));
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x4E, 0xF, 0xF, true));
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x141, 0xF, 0xF, true));
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x140, 0xF, 0xF, true));
    return v;
}

enum { STEP_RETENTION = 0, STEP_MEMORY = 1, STEP_WKV = 2 };

struct StepRows {                                        // what all kinds read and write
    const void* proj;                                    // [rows, ld]: q (H dk) | k (H dk) | v (H dv) | gate (H dv)
    int ld;
    void* out;                                           // rows out_ld elements apart, H dv of each
    int out_ld;
    float* state;                                        // [slots][H][OV][dk], OV = dv (retention) or dv + 1
    const int* seq_start;
    const int* slots;
    int rows, H, dk, dv;
    float eps, scale;                                    // of the norm; of the output
};

struct StepRetention {
    const int* positions;
    const float* decay;                                  // [H]
    const float* cos_table;                              // [table_positions, dims / 2] or null
    const float* sin_table;
    int dims, pairing, table_positions;
    float k_scale;
};

struct StepMemory {
    const void* x;                                       // [rows, n]: the layer's input
    const void* w;                                       // [2 H, n]: the gates' rows
    int n;
    RowFactor factor;                                    // of x
    const float* bias;                                   // [2 H]
    const float* weight;                                 // [H dv]
    float* m_state;                                      // [slots, H]
    float cap, q_scale;
};

struct StepTimeMix {
    const float* z;                                      // the decays' inner rows, before tanh: element i of row r at r z_row + i z_col
    long long z_row, z_col;
    const void* w2;                                      // [H dk, rank]
    const float* w0;                                     // [H dk]
    int rank;
    const float* u;                                      // [H, dk]
    const float* weight;                                 // [H dv]
};

// elements i .. i + 7 of a row of T where `eight`, else element i alone
template <typename T>
__device__ __forceinline__ float rs_dot8(const T* a, const T* b) {
    if constexpr (sizeof(T) == 2) {
        const uint4 x = *reinterpret_cast<const uint4*>(a), y = *reinterpret_cast<const uint4*>(b);
        const uint32_t u[4] = {x.x, x.y, x.z, x.w}, v[4] = {y.x, y.y, y.z, y.w};
        float s = 0.f;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            s = fmaf(bf16_to_f32((bf16_t)(u[i] & 0xffffu)), bf16_to_f32((bf16_t)(v[i] & 0xffffu)), s);
            s = fmaf(bf16_to_f32((bf16_t)(u[i] >> 16)), bf16_to_f32((bf16_t)(v[i] >> 16)), s);
        }
        return s;
    } else {
        float s = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) s = fmaf(a[i], b[i], s);
        return s;
    }
}

// T: of the projections; TO: of the output and the matrices
template <int KIND, int R, typename T, typename TO>
__global__ __launch_bounds__(RS_THREADS) void recurrent_step_kernel(StepRows a, StepRetention ret, StepMemory mem, StepTimeMix mix) {
    constexpr bool MEMORY = KIND == STEP_MEMORY, WKV = KIND == STEP_WKV;
    constexpr int L = 16, DKP = L * R, NC = RS_THREADS / L;
    constexpr int GROUPS = R >= 16 ? 4 : R >= 8 ? 8 : 8;               // of NC columns, in flight together
    constexpr int VW = R % 4 == 0 ? 4 : R % 2 == 0 ? 2 : 1;
    extern __shared__ __align__(16) float rs_lds[];
    __shared__ float red[16];
    const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, sub = tid % L, jl = tid / L;
    const int dk = a.dk, dv = a.dv, H = a.H, OV = dv + (MEMORY ? 1 : 0);
    float* q_s = rs_lds;
    float* k_s = q_s + DKP;
    float* o_s = k_s + DKP;                                            // [OV]
    float* v_s = o_s + OV;                                             // [OV]
    float* d_s = v_s + OV;                                             // wkv: [DKP] decays,
    float* z_s = d_s + DKP;                                            // [rank]
    auto at = [&](int r) { return (r / VW) * (L * VW) + sub * VW + r % VW; };
    const int slot = a.slots[row];
    const bool fresh = a.seq_start[row] == 0;
    float* S_head = a.state + ((size_t)slot * H + h) * OV * dk;
    const bool whole = dk == DKP && dk % 4 == 0;
    float S[GROUPS][R], n[MEMORY ? R : 1];               // n: the mLSTM's normaliser, column dv, with the first 16 lanes
    auto load_column = [&](int j, auto& c) {
#pragma unroll
        for (int r = 0; r < R; ++r) c[r] = 0.f;
        if (fresh) return;
        const float* col = S_head + (size_t)j * dk;
        if (whole) {
#pragma unroll
            for (int r = 0; r < R; r += VW) {
                if constexpr (VW == 4) {
                    const float4 v = *reinterpret_cast<const float4*>(col + at(r));
                    c[r] = v.x, c[r + 1] = v.y, c[r + 2] = v.z, c[r + 3] = v.w;
                } else if constexpr (VW == 2) {
                    const float2 v = *reinterpret_cast<const float2*>(col + at(r));
                    c[r] = v.x, c[r + 1] = v.y;
                } else {
                    c[r] = col[at(r)];
                }
            }
        } else {
#pragma unroll
            for (int r = 0; r < R; ++r)
                if (at(r) < dk) c[r] = col[at(r)];
        }
    };
    auto store_column = [&](int j, const auto& c) {
        float* col = S_head + (size_t)j * dk;
        if (whole) {
#pragma unroll
            for (int r = 0; r < R; r += VW) {
                if constexpr (VW == 4) *reinterpret_cast<float4*>(col + at(r)) = make_float4(c[r], c[r + 1], c[r + 2], c[r + 3]);
                else if constexpr (VW == 2) *reinterpret_cast<float2*>(col + at(r)) = make_float2(c[r], c[r + 1]);
                else col[at(r)] = c[r];
            }
        } else {
#pragma unroll
            for (int r = 0; r < R; ++r)
                if (at(r) < dk) col[at(r)] = c[r];
        }
    };
    auto load = [&](int j0) {
#pragma unroll
        for (int g = 0; g < GROUPS; ++g)
            if (j0 + g * NC + jl < dv) load_column(j0 + g * NC + jl, S[g]);
    };
    if constexpr (MEMORY) {
        if (jl == 0) load_column(dv, n);
    }
    load(0);
    const T* src = (const T*)a.proj + (size_t)row * a.ld;
    const T* q_src = src + (size_t)h * dk;
    const T* k_src = src + (size_t)(H + h) * dk;
    const T* v_src = src + (size_t)2 * H * dk + (size_t)h * dv;
    float keep = 0.f, floor_ = 0.f;
    if constexpr (WKV) {
        for (int i = tid; i < mix.rank; i += RS_THREADS) z_s[i] = tanhf(mix.z[row * mix.z_row + i * mix.z_col]);
        for (int e = tid; e < DKP; e += RS_THREADS) {
            q_s[e] = e < dk ? to_f32(q_src[e]) : 0.f;
            k_s[e] = e < dk ? to_f32(k_src[e]) : 0.f;
        }
        for (int j = tid; j < OV; j += RS_THREADS) v_s[j] = to_f32(v_src[j]);
        __syncthreads();
        // a channel's decay: P neighbouring threads share out its row of W2
        constexpr int P = RS_THREADS / DKP;
        const int c = tid / P, part = tid % P;
        const TO* w = (const TO*)mix.w2 + (size_t)(h * dk + min(c, dk - 1)) * mix.rank;
        float acc = 0.f;
        if (sizeof(TO) == 2 && mix.rank % 8 == 0) {
            for (int i = part * 8; i < mix.rank; i += 8 * P) {
                const uint4 raw = *reinterpret_cast<const uint4*>(w + i);
                const uint32_t b[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    acc = fmaf(z_s[i + 2 * e], __uint_as_float(b[e] << 16), acc);
                    acc = fmaf(z_s[i + 2 * e + 1], __uint_as_float(b[e] & 0xFFFF0000u), acc);
                }
            }
        } else {
            for (int i = part; i < mix.rank; i += P) acc = fmaf(z_s[i], to_f32(w[i]), acc);
        }
#pragma unroll
        for (int off = 1; off < P; off *= 2) acc += __shfl_xor(acc, off, TLI_WAVE);
        if (part == 0) d_s[c] = c < dk ? expf(-expf(acc + mix.w0[h * dk + c])) : 0.f;
    } else if constexpr (MEMORY) {
        // the gates' logits: every thread a part of the two dot products
        const T* x = (const T*)mem.x + (size_t)row * mem.n;
        const T* wi = (const T*)mem.w + (size_t)h * mem.n;
        const T* wf = (const T*)mem.w + (size_t)(H + h) * mem.n;
        float zi = 0.f, zf = 0.f;
        if (mem.n % 8 == 0) {
            for (int i = tid * 8; i < mem.n; i += RS_THREADS * 8) {
                zi += rs_dot8(x + i, wi + i);
                zf += rs_dot8(x + i, wf + i);
            }
        } else {
            for (int i = tid; i < mem.n; i += RS_THREADS) {
                zi = fmaf(to_f32(x[i]), to_f32(wi[i]), zi);
                zf = fmaf(to_f32(x[i]), to_f32(wf[i]), zf);
            }
        }
        float ss = 0.f;
        for (int p = tid; p < mem.factor.parts; p += RS_THREADS) ss += mem.factor.ssq[(size_t)p * a.rows + row];
        float* m_slot = mem.m_state + (size_t)slot * H + h;
        const float m0 = fresh ? 0.f : *m_slot;
        zi = wave_sum(zi), zf = wave_sum(zf), ss = wave_sum(ss);
        if (tid % TLI_WAVE == 0) red[tid / TLI_WAVE] = zi, red[4 + tid / TLI_WAVE] = zf, red[8 + tid / TLI_WAVE] = ss;
        __syncthreads();                                               // (m0 is read by all as well)
        zi = red[0] + red[1] + red[2] + red[3];
        zf = red[4] + red[5] + red[6] + red[7];
        if (mem.factor.parts > 0) {
            const float f = mem.factor.of_sum(red[8] + red[9] + red[10] + red[11]);
            zi *= f, zf *= f;
        }
        const float gi = gate_capped(zi + mem.bias[h], mem.cap), gf = gate_log_sigmoid(gate_capped(zf + mem.bias[H + h], mem.cap));
        const float m = fmaxf(gf + m0, gi);
        keep = expf(gf + m0 - m);
        floor_ = expf(-m);
        const float take = expf(gi - m);
        if (tid == 0) *m_slot = m;
        for (int e = tid; e < DKP; e += RS_THREADS) {
            q_s[e] = e < dk ? to_f32(q_src[e]) * mem.q_scale : 0.f;
            k_s[e] = e < dk ? to_f32(k_src[e]) : 0.f;
        }
        for (int j = tid; j < OV; j += RS_THREADS) v_s[j] = j < dv ? to_f32(v_src[j]) * take : take;
    } else {
        keep = ret.decay[h];
        const int pos = ret.positions[row], half = ret.dims / 2;
        const bool turn = ret.cos_table && pos >= 0 && pos < ret.table_positions;
        const float* cos_row = turn ? ret.cos_table + (size_t)pos * half : nullptr;
        const float* sin_row = turn ? ret.sin_table + (size_t)pos * half : nullptr;
        for (int e = tid; e < 2 * DKP; e += RS_THREADS) {
            const bool is_k = e >= DKP;
            const int i = is_k ? e - DKP : e;
            const T* head = is_k ? k_src : q_src;
            float x = 0.f;
            if (i < dk) {
                x = to_f32(head[i]);
                if (turn && i < ret.dims) {
                    const bool second = ret.pairing ? (i & 1) : i >= half;
                    const int pair = ret.pairing ? i / 2 : second ? i - half : i;
                    const float other = to_f32(head[ret.pairing ? i ^ 1 : second ? i - half : i + half]);
                    x = second ? rotate_second_half(x, other, cos_row[pair], sin_row[pair])
                               : rotate_first_half(x, other, cos_row[pair], sin_row[pair]);
                }
                if (is_k) x *= ret.k_scale;
            }
            q_s[e] = x;                                                // (k_s lies behind q_s)
        }
        for (int j = tid; j < OV; j += RS_THREADS) v_s[j] = to_f32(v_src[j]);
    }
    __syncthreads();
    float q[R], k[R];
#pragma unroll
    for (int r = 0; r < R; ++r) q[r] = q_s[at(r)], k[r] = k_s[at(r)];
    float d[WKV ? R : 1], bonus = 0.f;                   // wkv: the channels' decays; r diag(u) k
    if constexpr (WKV) {
#pragma unroll
        for (int r = 0; r < R; ++r) {
            d[r] = d_s[at(r)];
            if (at(r) < dk) bonus = fmaf(q[r] * mix.u[h * dk + at(r)], k[r], bonus);
        }
        bonus = rs_sum16(bonus);
    }
    auto walk = [&](int j, auto& c) {                    // (all 16 lanes of a column come here together, or none)
        const float v = v_s[j];
        float acc = 0.f;
#pragma unroll
        for (int r = 0; r < R; ++r) {
            if constexpr (WKV) {
                acc = fmaf(c[r], q[r], acc);
                c[r] = fmaf(d[r], c[r], k[r] * v);
            } else {
                c[r] = fmaf(keep, c[r], k[r] * v);
                acc = fmaf(c[r], q[r], acc);
            }
        }
        acc = rs_sum16(acc);
        if (sub == 0) o_s[j] = WKV ? fmaf(bonus, v, acc) : acc;
        store_column(j, c);
    };
    if constexpr (MEMORY) {
        if (jl == 0) walk(dv, n);
    }
    for (int j0 = 0; j0 < dv; j0 += GROUPS * NC) {
        if (j0 > 0) load(j0);
#pragma unroll
        for (int g = 0; g < GROUPS; ++g)
            if (j0 + g * NC + jl < dv) walk(j0 + g * NC + jl, S[g]);
    }
    __syncthreads();
    const float by = MEMORY ? 1.f / (fmaxf(fabsf(o_s[dv]), floor_) + 1e-6f) : 1.f;
    float ss = 0.f;
    for (int j = tid; j < dv; j += RS_THREADS) {
        const float x = o_s[j] * by;
        ss = fmaf(x, x, ss);
    }
    const float factor = a.scale * by / sqrtf(block_sum(ss, red) / (float)dv + a.eps);
    const T* g_src = src + (size_t)H * (2 * dk + dv) + (size_t)h * dv;
    TO* dst = (TO*)a.out + (size_t)row * a.out_ld + (size_t)h * dv;
    for (int j = tid; j < dv; j += RS_THREADS) {
        const float z = to_f32(g_src[j]);
        const float open = (MEMORY ? mem.weight[h * dv + j] : WKV ? z * mix.weight[h * dv + j] : z) / (1.f + expf(-z));
        from_f32(dst + j, o_s[j] * factor * open);
    }
}

template <int KIND, typename T, typename TO = T>
static int run_step(const StepRows& a, const StepRetention& ret, const StepMemory& mem, const StepTimeMix& mix, hipStream_t s) {
    int R = 1;
    while (16 * R < a.dk) R *= 2;
    const size_t lds = (size_t)(2 * 16 * R + 2 * (a.dv + 1) + (KIND == STEP_WKV ? 16 * R + mix.rank : 0)) * sizeof(float);
    if (lds > 65536) return tli_fail("recurrent_step: values of %d do not fit LDS", a.dv);
    const dim3 grid(a.H, a.rows);
#define RS_CASE(R) case R: recurrent_step_kernel<KIND, R, T, TO><<<grid, RS_THREADS, lds, s>>>(a, ret, mem, mix); break;
    switch (R) {
        RS_CASE(1) RS_CASE(2) RS_CASE(4) RS_CASE(8) RS_CASE(16)
        default: return tli_fail("recurrent_step: keys of %d", a.dk);
    }
#undef RS_CASE
    return tli_check_launch("recurrent_step");
}

static const char* step_fault(const StepRows& a, int rows_need) {
    if (a.H <= 0 || a.H > 65535 || a.rows > 65535 || a.dk <= 0 || a.dk > TLI_RECURRENCE_MAX_DK || a.dv <= 0) return "bad sizes";
    if (a.ld < rows_need) return "the rows do not hold q, k, v and the gate";
    if (a.out_ld < a.H * a.dv) return "the output's rows overlap";
    if ((uintptr_t)a.state & 15) return "the state must be 16-byte aligned";
    return nullptr;
}

// proj: rows of ld elements, q (H dk) | k (H dk) | v (H dv) | gate (H dv) first; the rest as in retention.hip
extern "C" int tli_retention_step(const void* proj, int ld, const float* decay, float* state, void* out, int out_ld,
                                  const int* positions, const int* seq_start, const int* slots, const float* cos_table,
                                  const float* sin_table, int dims, int pairing, int table_positions, float k_scale, float eps,
                                  float scale, int rows, int H, int dk, int dv, int dtype, void* stream) {
    if (rows <= 0) return 0;
    const StepRows a{proj, ld, out, out_ld, state, seq_start, slots, rows, H, dk, dv, eps, scale};
    if (const char* fault = step_fault(a, 2 * H * (dk + dv))) return tli_fail("retention_step: %s", fault);
    if (cos_table && (dims <= 0 || dims % 2 || dims > dk)) return tli_fail("retention_step: %d turned elements of heads of %d", dims, dk);
    const StepRetention ret{positions, decay, cos_table, sin_table, dims, pairing, table_positions, k_scale};
    if (dtype == TLI_F32) return run_step<STEP_RETENTION, float>(a, ret, StepMemory{}, StepTimeMix{}, (hipStream_t)stream);
    if (dtype == TLI_BF16) return run_step<STEP_RETENTION, bf16_t>(a, ret, StepMemory{}, StepTimeMix{}, (hipStream_t)stream);
    return tli_fail("retention_step: unknown dtype %d", dtype);
}

// x: [rows, n] the layer's input (times the rows' factor where ssq is given: row_gates.h); w: [2 H, n]; the rest as in
// mlstm.hip
extern "C" int tli_mlstm_step(const void* proj, int ld, const void* x, const void* w, int n, const float* ssq, int parts, float x_eps,
                              const float* bias, float cap, float q_scale, const float* weight, float* m_state, float* state,
                              void* out, int out_ld, const int* seq_start, const int* slots, float eps, float scale, int rows,
                              int H, int dk, int dv, int dtype, void* stream) {
    if (rows <= 0) return 0;
    const StepRows a{proj, ld, out, out_ld, state, seq_start, slots, rows, H, dk, dv, eps, scale};
    if (const char* fault = step_fault(a, 2 * H * (dk + dv))) return tli_fail("mlstm_step: %s", fault);
    if (n <= 0 || !(cap > 0.f) || (ssq && parts <= 0)) return tli_fail("mlstm_step: bad gates");
    if (((uintptr_t)x | (uintptr_t)w) & 15) return tli_fail("mlstm_step: operands must be 16-byte aligned");
    const StepMemory mem{x, w, n, RowFactor{ssq, ssq ? parts : 0, rows, 1.0f / (float)n, x_eps}, bias, weight, m_state, cap, q_scale};
    if (dtype == TLI_F32) return run_step<STEP_MEMORY, float>(a, StepRetention{}, mem, StepTimeMix{}, (hipStream_t)stream);
    if (dtype == TLI_BF16) return run_step<STEP_MEMORY, bf16_t>(a, StepRetention{}, mem, StepTimeMix{}, (hipStream_t)stream);
    return tli_fail("mlstm_step: unknown dtype %d", dtype);
}

// proj: rows of ld elements of proj_dtype, r (H dk) | k (H dk) | v (H dv) | gate (H dv) first; z, w2, w0, rank: as for tli_wkv_decays
// (wkv.hip); u [H, dk]; weight [H dv]; state [slots][H][dv][dk]; out and w2 in `dtype` (proj_dtype: the same, or float32)
extern "C" int tli_wkv_step(const void* proj, int ld, int proj_dtype, const float* z, long long z_row, long long z_col, const void* w2,
                            const float* w0, int rank, const float* u, const float* weight, float* state, void* out, int out_ld,
                            const int* seq_start, const int* slots, float eps, int rows, int H, int dk, int dv, int dtype, void* stream) {
    if (rows <= 0) return 0;
    const StepRows a{proj, ld, out, out_ld, state, seq_start, slots, rows, H, dk, dv, eps, 1.0f};
    if (const char* fault = step_fault(a, 2 * H * (dk + dv))) return tli_fail("wkv_step: %s", fault);
    if (rank <= 0 || rank > 8192 || ((uintptr_t)w2 & 15)) return tli_fail("wkv_step: bad decays");
    const StepTimeMix mix{z, z_row, z_col, w2, w0, rank, u, weight};
    hipStream_t s = (hipStream_t)stream;
    if (dtype == TLI_F32 && proj_dtype == TLI_F32) return run_step<STEP_WKV, float>(a, StepRetention{}, StepMemory{}, mix, s);
    if (dtype == TLI_BF16 && proj_dtype == TLI_F32) return run_step<STEP_WKV, float, bf16_t>(a, StepRetention{}, StepMemory{}, mix, s);
    if (dtype == TLI_BF16 && proj_dtype == TLI_BF16) return run_step<STEP_WKV, bf16_t>(a, StepRetention{}, StepMemory{}, mix, s);
    return tli_fail("wkv_step: unknown dtypes %d, %d", proj_dtype, dtype);
}
