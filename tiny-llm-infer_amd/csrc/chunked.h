// Shared by mlstm.hip (whose gates and scan they are) and chunked.hip.
#pragma once
#include "recurrence.h"
#include "row_gates.h"

#define TLI_CHUNK_ROWS 64    // rows of a chunk of chunked.hip

struct MlGates {
    const float* z;          // logits: head h's input gate of row r at z[r z_row + h z_col], its forget gate H columns on
    long long z_row, z_col;
    const float* bias;       // [2 H]
    float cap;
    int H;
    RowFactor factor;        // of the rows that the logits were made from
    __device__ __forceinline__ float input(int r, int h, float f) const { return gate_capped(z[r * z_row + h * z_col] * f + bias[h], cap); }
    __device__ __forceinline__ float forget(int r, int h, float f) const {
        return gate_log_sigmoid(gate_capped(z[r * z_row + (H + h) * z_col] * f + bias[H + h], cap));
    }
};

// keep, take, floors, through: [H][T]: a_t; exp(i_t - m_t); exp(-m_t); log of the product of a from the first of the row's
// unit of rows on (units of TLI_CHUNK_ROWS or of TLI_RECURRENCE_SEGMENT, counted from the sequence's first row of the step)
int tli_mlstm_scan(const MlGates& gates, float* m_state, float* keep, float* take, float* floors, float* through, int unit,
                   const int* row_start, const int* seq_start, const int* slots, int T, int seqs, hipStream_t s);
