// Retention: linear attention with a fixed decay a head and rotated queries and keys.  For the rows of one sequence,
// head by head (key size dk, value size dv, decay c_h from the caller):
//   q, k turned by the row's position (the first `dims` elements in pairs), k times k_scale behind that;  v as it is
//   S_t = c_h S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t
// retention_prepare leaves q, k and v in float32 as the shared recurrence (recurrence.h) takes them.
#include "recurrence.h"

// pairing 0: pair i is (i, i + dims/2); 1: (2i, 2i + 1)
template <typename T>
__global__ void retention_prepare_kernel(const T* __restrict__ proj, int ld, float* __restrict__ qk, float* __restrict__ v,
                                         const int* __restrict__ positions, const float* __restrict__ cos_table,
                                         const float* __restrict__ sin_table, int dims, int pairing, int table_positions,
                                         float k_scale, int H, int dk, int dv, int DKP, int DVP) {
    const size_t row = blockIdx.x;
    const int h = blockIdx.y;
    const T* src = proj + row * ld;
    float* qk_dst = qk + (row * H + h) * 2 * DKP;
    float* v_dst = v + (row * H + h) * DVP;
    const int pos = positions[row], half = dims / 2;
    const bool turn = cos_table && pos >= 0 && pos < table_positions;
    const float* cos_row = turn ? cos_table + (size_t)pos * half : nullptr;
    const float* sin_row = turn ? sin_table + (size_t)pos * half : nullptr;
    for (int e = threadIdx.x; e < 2 * DKP + DVP; e += blockDim.x) {
        if (e < 2 * DKP) {
            const bool is_k = e >= DKP;
            const int i = is_k ? e - DKP : e;
            float x = 0.f;
            if (i < dk) {
                const T* head = src + (is_k ? (size_t)H * dk : 0) + (size_t)h * dk;
                x = to_f32(head[i]);
                if (turn && i < dims) {
                    const bool second = pairing ? (i & 1) : i >= half;
                    const int pair = pairing ? i / 2 : second ? i - half : i;
                    const float other = to_f32(head[pairing ? i ^ 1 : second ? i - half : i + half]);
                    x = second ? rotate_second_half(x, other, cos_row[pair], sin_row[pair])
                               : rotate_first_half(x, other, cos_row[pair], sin_row[pair]);
                }
                if (is_k) x *= k_scale;
            }
            qk_dst[e] = x;
        } else {
            const int j = e - 2 * DKP;
            v_dst[j] = j < dv ? to_f32(src[(size_t)2 * H * dk + (size_t)h * dv + j]) : 0.f;
        }
    }
}

// proj: [T, ld], q (H dk), k (H dk), v (H dv) first; decay [H]; cos, sin: float32 [table_positions, dims / 2] or null;
// state, out, scratch, longest, lanes: as for tli_lightning_recurrence
extern "C" int tli_retention(const void* proj, int ld, const float* decay, float* state, float* out, float* scratch,
                             const int* positions, const int* row_start, const int* seq_start, const int* slots,
                             const float* cos_table, const float* sin_table, int dims, int pairing, int table_positions,
                             float k_scale, int T, int seqs, int longest, int H, int dk, int dv, int dtype, int lanes,
                             void* stream) {
    if (seqs <= 0 || T <= 0) return 0;
    if (H <= 0 || H > 65535 || dk <= 0 || dv <= 0 || dk > TLI_RECURRENCE_MAX_DK)
        return tli_fail("retention: bad sizes (heads %d, keys of %d (at most %d), values of %d)", H, dk, TLI_RECURRENCE_MAX_DK, dv);
    if (ld < 2 * H * dk + H * dv) return tli_fail("retention: rows of %d hold fewer than q, k and v", ld);
    if (cos_table && (dims <= 0 || dims % 2 || dims > dk)) return tli_fail("retention: %d turned elements of heads of %d", dims, dk);
    if (lanes != 0 && lanes != 16 && lanes != 64) return tli_fail("retention: 16 or 64 lanes a column, not %d", lanes);
    const RecurrencePlan plan = tli_recurrence_plan(longest, dk, dv, lanes);
    float* vals = recurrence_values(plan, scratch, T, H);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == TLI_F32)
        retention_prepare_kernel<float><<<dim3(T, H), 256, 0, s>>>((const float*)proj, ld, scratch, vals, positions, cos_table, sin_table,
                                                                   dims, pairing, table_positions, k_scale, H, dk, dv, plan.dkp, plan.dvp);
    else if (dtype == TLI_BF16)
        retention_prepare_kernel<bf16_t><<<dim3(T, H), 256, 0, s>>>((const bf16_t*)proj, ld, scratch, vals, positions, cos_table, sin_table,
                                                                    dims, pairing, table_positions, k_scale, H, dk, dv, plan.dkp, plan.dvp);
    else
        return tli_fail("retention: unknown dtype %d", dtype);
    return tli_recurrence_run(plan, scratch, RecurrenceDecay{decay, nullptr, nullptr}, state, out, row_start, seq_start, slots, T,
                              seqs, H, dk, dv, s);
}

// What stands behind a recurrence whose heads are normed one by one.  One wave a (row, head):
//   x = o                                     or, with `floors`, o / (max(|o[dv]|, floor) + 1e-6): element dv of the
//                                             head's outputs is what its normaliser gave
//   y = x / sqrt(mean(x^2) + eps) * weight[h dv + i] * gate(g) * scale     gate: silu (0) or the logistic function (1)
template <typename T>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(
    const float* __restrict__ o, int ov, const float* __restrict__ floors, int rows, const float* __restrict__ weight,
    const T* __restrict__ gate, int gate_ld, T* __restrict__ out, int out_ld, int heads, int dv, float eps, int kind,
    float scale) {
    const int lane = threadIdx.x % TLI_WAVE;
    const size_t unit = (size_t)blockIdx.x * (blockDim.x / TLI_WAVE) + threadIdx.x / TLI_WAVE;
    if (unit >= (size_t)rows * heads) return;
    const size_t row = unit / heads;
    const int h = (int)(unit % heads);
    const float* x = o + unit * ov;
    float by = 1.f;
    if (floors) by = 1.f / (fmaxf(fabsf(x[dv]), floors[(size_t)h * rows + row]) + 1e-6f);
    constexpr int KEEP = 4;                              // elements of a head that a lane keeps for the second pass
    float kept[KEEP];
    float ss = 0.f;
#pragma unroll
    for (int u = 0; u < KEEP; ++u) {
        const int i = lane + u * TLI_WAVE;
        kept[u] = i < dv ? x[i] * by : 0.f;
        ss = fmaf(kept[u], kept[u], ss);
    }
    for (int i = lane + KEEP * TLI_WAVE; i < dv; i += TLI_WAVE) {
        const float v = x[i] * by;
        ss = fmaf(v, v, ss);
    }
    const float factor = scale / sqrtf(wave_sum(ss) / (float)dv + eps);
    const T* g = gate + row * gate_ld + (size_t)h * dv;
    T* dst = out + row * out_ld + (size_t)h * dv;
    auto put = [&](int i, float v) {
        const float z = to_f32(g[i]);
        const float open = (kind == 0 ? z : 1.f) / (1.f + expf(-z));
        from_f32(dst + i, v * factor * (weight ? weight[h * dv + i] : 1.f) * open);
    };
#pragma unroll
    for (int u = 0; u < KEEP; ++u)
        if (lane + u * TLI_WAVE < dv) put(lane + u * TLI_WAVE, kept[u]);
    for (int i = lane + KEEP * TLI_WAVE; i < dv; i += TLI_WAVE) put(i, x[i] * by);
}

// o: float32 [rows, heads, ov], ov = dv, or dv + 1 with `floors` (float32 [heads][rows]); weight: float32 [heads dv] or
// null; gate: [rows, gate_ld], its first heads * dv columns; out: rows out_ld elements apart
extern "C" int tli_head_norm_gate(const float* o, const float* floors, const float* weight, const void* gate, int gate_ld,
                                  void* out, int out_ld, int rows, int heads, int dv, float eps, int kind, float scale,
                                  int dtype, void* stream) {
    if (rows <= 0) return 0;
    if (heads <= 0 || dv <= 0 || gate_ld < heads * dv || out_ld < heads * dv) return tli_fail("head_norm_gate: bad sizes");
    if (kind < 0 || kind > 1) return tli_fail("head_norm_gate: unknown gate %d", kind);
    const int ov = floors ? dv + 1 : dv;
    const size_t units = (size_t)rows * heads;
    if ((units + 3) / 4 > 0x7fffffffULL) return tli_fail("head_norm_gate: too many rows for one launch");
    const unsigned blocks = (unsigned)((units + 3) / 4);
    hipStream_t s = (hipStream_t)stream;
    if (dtype == TLI_F32)
        head_norm_gate_kernel<float><<<blocks, 256, 0, s>>>(o, ov, floors, rows, weight, (const float*)gate, gate_ld, (float*)out, out_ld,
                                                            heads, dv, eps, kind, scale);
    else if (dtype == TLI_BF16)
        head_norm_gate_kernel<bf16_t><<<blocks, 256, 0, s>>>(o, ov, floors, rows, weight, (const bf16_t*)gate, gate_ld, (bf16_t*)out,
                                                             out_ld, heads, dv, eps, kind, scale);
    else
        return tli_fail("head_norm_gate: unknown dtype %d", dtype);
    return tli_check_launch("head_norm_gate");
}
