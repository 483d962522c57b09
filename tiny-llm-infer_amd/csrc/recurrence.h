// The recurrence over a step's rows that several recurrent layers share (its kernels are in lightning.hip):
//   S_t = a_t S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t      head by head, S [dk, dv], float32, zero before position 0
// with one factor a head, or one a row and head.  A caller leaves the rows' q, k and v in float32, padded:
//   qk [T][H][2][dkp] (q, then k; zeros from dk on)   at scratch
//   v  [T][H][dvp] (zeros from dv on)                 behind it
#pragma once
#include "common.h"

// Rows of a segment of a long portion (tli_recurrence_plan says whether a step's portions are cut into segments).
#define TLI_RECURRENCE_SEGMENT 256
#define TLI_RECURRENCE_MAX_DK 256

struct RecurrencePlan {
    int lanes;               // lanes that hold a column of S
    int dkp, dvp;            // padded sizes of a head's q or k, and of its v
    int segment;             // rows of a segment, or 0: every sequence's rows are walked whole
};

struct RecurrenceDecay {
    const float* head;       // [H]: one factor a head; or null, and then
    const float* row;        // [H][T]: a_t
    const float* log_through;// [H][T]: log of the product of a_s over the rows s from t's segment's first to t (only read
};                           //         where the plan has segments, which start at the sequence's first row of the step)

// lanes 0: the launch rule (16), else 16 or 64; longest: the most rows that a sequence of the step has
RecurrencePlan tli_recurrence_plan(int longest, int dk, int dv, int lanes);

// state: [slots][H][dv][dk]; out: [T, H dv]; scratch: tli_lightning_scratch_floats(T, ...) elements, q, k and v in place
int tli_recurrence_run(const RecurrencePlan& plan, float* scratch, const RecurrenceDecay& decay, float* state, float* out,
                       const int* row_start, const int* seq_start, const int* slots, int T, int seqs, int H, int dk, int dv,
                       hipStream_t s);

static inline float* recurrence_values(const RecurrencePlan& p, float* scratch, int T, int H) {
    return scratch + (size_t)T * H * 2 * p.dkp;
}
