// The mLSTM's matrix memory.  For the rows of one sequence, head by head (key size dk, value size dv):
//   i = cap tanh((z_i + b_i) / cap),   f = logsigmoid(cap tanh((z_f + b_f) / cap))          (log gates)
//   m_t = max(f_t + m_(t-1), i_t),   m = 0 before position 0
//   S_t = exp(f_t + m_(t-1) - m_t) S_(t-1) + exp(i_t - m_t) k_t v_t^T,   n_t likewise with k_t alone
//   o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6),   q = proj q * q_scale
// S, n, m are state, zero before position 0 (a sequence that starts there does not read its slot).
//
// With a_t = exp(f_t + m_(t-1) - m_t) this is the shared recurrence (recurrence.h) with a factor a row, values times
// exp(i_t - m_t), and n as one more column of S whose value is that factor alone: columns 0..dv-1 of the outputs are
// S_t^T q_t, column dv is n_t . q_t.  The division is left to head_norm_gate (retention.hip), which takes exp(-m_t).
//
// mlstm_scan: a workgroup a (head, sequence) takes 256 rows at a time.  m is a running maximum of sums: a row maps m to
// max(f + m, i), two such maps in a row are one again, (F, M) = (F1 + F2, max(M1 + F2, M2)), so the 256 rows' maps are
// combined by doubling (six exchanges of lanes, then the four waves' through LDS) instead of one after the other.
// m only scales S, n and the floor alike, so in which order its sums are taken does not matter as long as a row's factors
// are made from the same m.
// mlstm_prepare: a workgroup a (row, head) leaves q, k and v in float32 for the recurrence.  In a step of single rows
// (`single`) it makes the gates itself and there is no scan.
#include "chunked.h"

#define ML_THREADS TLI_RECURRENCE_SEGMENT

// (its results: chunked.h)
__global__ __launch_bounds__(ML_THREADS) void mlstm_scan_kernel(MlGates gates, float* __restrict__ m_state,
                                                                float* __restrict__ keep, float* __restrict__ take,
                                                                float* __restrict__ floors, float* __restrict__ through, int unit,
                                                                const int* __restrict__ row_start, const int* __restrict__ seq_start,
                                                                const int* __restrict__ slots, int T) {
    __shared__ float wave_f[ML_THREADS / TLI_WAVE], wave_m[ML_THREADS / TLI_WAVE];
    __shared__ float m_of[ML_THREADS + 1];               // m before the first of the rows, then after each of them
    const int h = blockIdx.x, seq = blockIdx.y, tid = threadIdx.x, lane = tid % TLI_WAVE, wave = tid / TLI_WAVE;
    const int r0 = row_start[seq], n = row_start[seq + 1] - r0;
    float* slot = m_state + (size_t)slots[seq] * gates.H + h;
    float m0 = seq_start[seq] != 0 ? *slot : 0.f;
    for (int first = 0; first < n; first += ML_THREADS) {
        const int r = r0 + first + tid;
        const bool live = first + tid < n;
        const float owed = live ? gates.factor.of(r) : 1.f;
        const float f = live ? gates.forget(r, h, owed) : 0.f;
        const float i = live ? gates.input(r, h, owed) : -INFINITY;          // (a row past the end leaves m alone)
        float F = f, M = i;                                            // the map of this row and those before it in the wave
#pragma unroll
        for (int off = 1; off < TLI_WAVE; off <<= 1) {
            const float Fb = __shfl_up(F, off, TLI_WAVE), Mb = __shfl_up(M, off, TLI_WAVE);
            if (lane >= off) {
                M = fmaxf(Mb + F, M);
                F += Fb;
            }
        }
        if (lane == TLI_WAVE - 1) {
            wave_f[wave] = F;
            wave_m[wave] = M;
        }
        __syncthreads();
        const float F_wave = F;                                        // from the wave's first row on
        float Fw = 0.f, Mw = -INFINITY;                                // the waves before
        for (int w = 0; w < wave; ++w) {
            Mw = fmaxf(Mw + wave_f[w], wave_m[w]);
            Fw += wave_f[w];
        }
        M = fmaxf(Mw + F, M);
        F += Fw;
        const float m = fmaxf(m0 + F, M);
        if (tid == 0) m_of[0] = m0;
        m_of[tid + 1] = m;
        __syncthreads();
        if (live) {
            const size_t at = (size_t)h * T + r;
            keep[at] = expf(f + m_of[tid] - m);
            take[at] = expf(i - m);
            floors[at] = expf(-m);
            through[at] = unit == TLI_WAVE ? F_wave + m_of[wave * TLI_WAVE] - m : F + m0 - m;
        }
        m0 = m_of[min(n - first, ML_THREADS)];
        __syncthreads();
    }
    if (tid == 0 && n > 0) *slot = m0;
}

static_assert(TLI_CHUNK_ROWS == TLI_WAVE, "a chunk's rows are a wave of the scan");

int tli_mlstm_scan(const MlGates& gates, float* m_state, float* keep, float* take, float* floors, float* through, int unit,
                   const int* row_start, const int* seq_start, const int* slots, int T, int seqs, hipStream_t s) {
    if (unit != TLI_CHUNK_ROWS && unit != TLI_RECURRENCE_SEGMENT) return tli_fail("mlstm_scan: units of %d rows", unit);
    mlstm_scan_kernel<<<dim3(gates.H, seqs), ML_THREADS, 0, s>>>(gates, m_state, keep, take, floors, through, unit, row_start,
                                                                 seq_start, slots, T);
    return tli_check_launch("mlstm_scan");
}

template <typename T>
__global__ void mlstm_prepare_kernel(const T* __restrict__ proj, int ld, float q_scale, float* __restrict__ qk, float* __restrict__ v,
                                     MlGates gates, float* __restrict__ m_state, float* __restrict__ keep,
                                     float* __restrict__ take_rows, float* __restrict__ floors, const int* __restrict__ seq_start,
                                     const int* __restrict__ slots, int rows, int single, int dk, int dv, int DKP, int DVP) {
    const size_t row = blockIdx.x;
    const int h = blockIdx.y, H = gates.H;
    const size_t at = (size_t)h * rows + row;
    float take;
    if (single) {                                                      // row r is sequence r
        float* slot = m_state + (size_t)slots[row] * H + h;
        const float m0 = seq_start[row] != 0 ? *slot : 0.f;
        const float owed = gates.factor.of((int)row);
        const float f = gates.forget((int)row, h, owed), i = gates.input((int)row, h, owed);
        const float m = fmaxf(f + m0, i);
        take = expf(i - m);
        __syncthreads();                                               // m0 is read by all before it is replaced
        if (threadIdx.x == 0) {
            keep[at] = expf(f + m0 - m);
            floors[at] = expf(-m);
            *slot = m;
        }
    } else {
        take = take_rows[at];
    }
    const T* src = proj + row * ld;
    float* qk_dst = qk + (row * H + h) * 2 * DKP;
    float* v_dst = v + (row * H + h) * DVP;
    for (int e = threadIdx.x; e < 2 * DKP + DVP; e += blockDim.x) {
        if (e < DKP) {
            qk_dst[e] = e < dk ? to_f32(src[(size_t)h * dk + e]) * q_scale : 0.f;
        } else if (e < 2 * DKP) {
            const int i = e - DKP;
            qk_dst[e] = i < dk ? to_f32(src[(size_t)(H + h) * dk + i]) : 0.f;
        } else {
            const int j = e - 2 * DKP;
            v_dst[j] = j < dv ? to_f32(src[(size_t)2 * H * dk + (size_t)h * dv + j]) * take : j == dv ? take : 0.f;
        }
    }
}

// proj: [T, ld], q (H dk), k (H dk), v (H dv) first; z, z_row, z_col, bias, cap: the gates (MlGates; ssq: [parts][T] sums
// of squares of rows of x_size elements whose factor the logits still owe, or null); m_state: float32
// [slots, H]; state: float32 [slots, H, dv + 1, dk]; out: float32 [T, H, dv + 1]; floors: float32 [H][T] (written);
// scratch: tli_lightning_scratch_floats(T, seqs, longest, H, dk, dv + 1) and 3 H T floats behind it at `rows_scratch`;
// longest: the most rows that a sequence brings; single: every sequence brings one row
extern "C" int tli_mlstm(const void* proj, int ld, const float* z, long long z_row, long long z_col, const float* ssq, int parts,
                         int x_size, float x_eps, const float* bias, float cap,
                         float q_scale, float* m_state, float* state, float* out, float* floors, float* scratch,
                         float* rows_scratch, const int* row_start, const int* seq_start, const int* slots, int T, int seqs,
                         int longest, int single, int H, int dk, int dv, int dtype, int lanes, void* stream) {
    if (seqs <= 0 || T <= 0) return 0;
    if (H <= 0 || H > 65535 || seqs > 65535 || dk <= 0 || dv <= 0 || dk > TLI_RECURRENCE_MAX_DK)
        return tli_fail("mlstm: bad sizes (heads %d, keys of %d (at most %d), values of %d)", H, dk, TLI_RECURRENCE_MAX_DK, dv);
    if (ld < 2 * H * dk + H * dv) return tli_fail("mlstm: rows of %d hold fewer than q, k and v", ld);
    if (!(cap > 0.f)) return tli_fail("mlstm: the gates' cap must be positive");
    if (single && T != seqs) return tli_fail("mlstm: %d rows are not one for each of %d sequences", T, seqs);
    if (lanes != 0 && lanes != 16 && lanes != 64) return tli_fail("mlstm: 16 or 64 lanes a column, not %d", lanes);
    const RecurrencePlan plan = tli_recurrence_plan(longest, dk, dv + 1, lanes);
    float* vals = recurrence_values(plan, scratch, T, H);
    float* keep = rows_scratch;
    float* take = keep + (size_t)H * T;
    float* through = take + (size_t)H * T;
    if (ssq && (parts <= 0 || x_size <= 0)) return tli_fail("mlstm: bad sums of squares");
    const MlGates gates{z, z_row, z_col, bias, cap, H, RowFactor{ssq, ssq ? parts : 0, T, 1.0f / (float)(x_size > 0 ? x_size : 1), x_eps}};
    hipStream_t s = (hipStream_t)stream;
    if (!single && tli_mlstm_scan(gates, m_state, keep, take, floors, through, TLI_RECURRENCE_SEGMENT, row_start, seq_start, slots, T, seqs, s))
        return 1;
    if (dtype == TLI_F32)
        mlstm_prepare_kernel<float><<<dim3(T, H), 256, 0, s>>>((const float*)proj, ld, q_scale, scratch, vals, gates, m_state, keep, take,
                                                               floors, seq_start, slots, T, single, dk, dv, plan.dkp, plan.dvp);
    else if (dtype == TLI_BF16)
        mlstm_prepare_kernel<bf16_t><<<dim3(T, H), 256, 0, s>>>((const bf16_t*)proj, ld, q_scale, scratch, vals, gates, m_state, keep, take,
                                                                floors, seq_start, slots, T, single, dk, dv, plan.dkp, plan.dvp);
    else
        return tli_fail("mlstm: unknown dtype %d", dtype);
    return tli_recurrence_run(plan, scratch, RecurrenceDecay{nullptr, keep, through}, state, out, row_start, seq_start, slots, T, seqs,
                              H, dk, dv + 1, s);
}
