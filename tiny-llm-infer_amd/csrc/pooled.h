// Pooled blocks beside a window: block b of `pool` positions, b pool .. b pool + pool - 1, has one key and one value a
// head, in a cache of their own with the layout of the tokens' ([page][kv head][slot][key_dim] and [page][kv head]
// [value_dim][slot]; slot b % page_size of the table's page b / page_size).  A row at p with a window of w sees the
// blocks that end at or before p - w, beside the tokens j <= p with p - j < w.
#pragma once

struct PooledKeys {
    const void* k;
    const void* v;
    const int* tables;       // [sequences][width]
    int width, pages;
    int pool;                // 0: there are none
};

// how many blocks a row at `pos` sees
__host__ __device__ __forceinline__ int pooled_blocks_seen(int pos, int window, int pool) {
    const int before = pos - window + 1;                 // positions before the window
    return before > 0 ? before / pool : 0;
}
