// What stands before the attention over a window and pooled blocks (pooled.h).
//
// projection_norm_prepare, one workgroup a row, float32 arithmetic, from the raw projections q | k | v of the row:
//   q = proj q + bias,  k = proj k + bias,  v = proj v + bias
//   q, k: x / sqrt(mean(x^2) + eps) * weight over ALL heads' elements together (null weight: no norm)
//   q, k: the first `dims` elements of every head turned by the position in pairs, (i, i + dims/2) or (2i, 2i + 1)
//   q -> q_out [rows, heads, key_dim];  k -> [page][kv head][slot][key_dim];  v -> [page][kv head][value_dim][slot]
//   In a step of single rows (`single`), a row that ends a block of `pool` positions also leaves the block's means.
// pool_blocks, a workgroup a (block that this step ends, kv head): the means of the block's keys and values as the cache
//   holds them, added up in the order of their positions, into the blocks' own cache.
#include "common.h"
#include "pooled.h"

#define PN_THREADS 256

// the mean of element (key: d of kv head g; value likewise) over the block's positions, read from the tokens' pages
template <typename T, bool VALUE>
__device__ __forceinline__ float block_mean(const T* __restrict__ cache, const int* __restrict__ table, int page_size, int num_pages,
                                            int kv_heads, int g, int dim, int d, int first, int pool) {
    float sum = 0.f;
    for (int j = 0; j < pool; ++j) {
        const int pos = first + j, slot = pos % page_size;
        const int page = table[pos / page_size];
        if (page < 0 || page >= num_pages) continue;
        const size_t head = ((size_t)page * kv_heads + g) * page_size * dim;
        sum += to_f32(VALUE ? cache[head + (size_t)d * page_size + slot] : cache[head + (size_t)slot * dim + d]);
    }
    return sum / (float)pool;
}

template <typename T>
__device__ __forceinline__ void store_block_means(const T* __restrict__ k_cache, const T* __restrict__ v_cache,
                                                  const int* __restrict__ table, int page_size, int num_pages, int kv_heads,
                                                  int key_dim, int value_dim, int g, int block, const PooledKeys& pooled,
                                                  const int* __restrict__ pooled_table, int first_thread, int threads) {
    const int page = pooled_table[block / page_size], slot = block % page_size;
    if (page < 0 || page >= pooled.pages) return;
    T* k_dst = (T*)pooled.k + (((size_t)page * kv_heads + g) * page_size + slot) * key_dim;
    T* v_dst = (T*)pooled.v + ((size_t)page * kv_heads + g) * page_size * value_dim + slot;
    for (int e = first_thread; e < key_dim + value_dim; e += threads) {
        T m;
        if (e < key_dim) {
            from_f32(&m, block_mean<T, false>(k_cache, table, page_size, num_pages, kv_heads, g, key_dim, e, block * pooled.pool, pooled.pool));
            k_dst[e] = cache_value(m);
        } else {
            const int d = e - key_dim;
            from_f32(&m, block_mean<T, true>(v_cache, table, page_size, num_pages, kv_heads, g, value_dim, d, block * pooled.pool, pooled.pool));
            v_dst[(size_t)d * page_size] = cache_value(m);
        }
    }
}

template <typename T>
__global__ __launch_bounds__(PN_THREADS) void projection_norm_prepare_kernel(
    const T* __restrict__ proj, int ld, const float* __restrict__ bias, T* __restrict__ q_out, T* k_cache, T* v_cache,
    const int* __restrict__ positions, const int* __restrict__ seq_of_row, const int* __restrict__ tables, int table_width,
    int page_size, int num_pages, int heads, int kv_heads, int key_dim, int value_dim, const float* __restrict__ q_weight,
    const float* __restrict__ k_weight, float eps, const float* __restrict__ cos_table, const float* __restrict__ sin_table,
    int dims, int pairing, int table_positions, PooledKeys pooled, int single) {
    extern __shared__ float pn_row[];                    // q and k of the row, all heads
    __shared__ float red[16];
    const int row = blockIdx.x, tid = threadIdx.x;
    const int qn = heads * key_dim, kn = kv_heads * key_dim;
    const T* src = proj + (size_t)row * ld;
    float ssq = 0.f, ssk = 0.f;
    for (int i = tid; i < qn + kn; i += PN_THREADS) {
        const float x = to_f32(src[i]) + (bias ? bias[i] : 0.f);
        pn_row[i] = x;
        if (i < qn) ssq = fmaf(x, x, ssq);
        else ssk = fmaf(x, x, ssk);
    }
    const float q_factor = q_weight ? 1.0f / sqrtf(block_sum(ssq, red) / (float)qn + eps) : 1.f;
    const float k_factor = k_weight ? 1.0f / sqrtf(block_sum(ssk, red) / (float)kn + eps) : 1.f;
    __syncthreads();
    const int pos = positions[row];
    const int* table = tables + (size_t)seq_of_row[row] * table_width;
    const int page = table[pos / page_size], slot = pos % page_size;
    const bool kept = page >= 0 && page < num_pages;
    const int half = dims / 2;
    const bool turn = cos_table && pos >= 0 && pos < table_positions;
    const float* cos_row = turn ? cos_table + (size_t)pos * half : nullptr;
    const float* sin_row = turn ? sin_table + (size_t)pos * half : nullptr;
    for (int i = tid; i < qn + kn; i += PN_THREADS) {
        const bool is_q = i < qn;
        const float* w = is_q ? q_weight : k_weight;
        const int base = is_q ? 0 : qn;
        const float factor = is_q ? q_factor : k_factor;
        auto normed = [&](int j) { return w ? pn_row[j] * factor * w[j - base] : pn_row[j]; };
        const int d = (i - base) % key_dim;
        float x = normed(i);
        if (turn && d < dims) {
            const bool second = pairing ? (d & 1) : d >= half;
            const int pair = pairing ? d / 2 : second ? d - half : d;
            const float other = normed(pairing ? (second ? i - 1 : i + 1) : second ? i - half : i + half);
            x = second ? rotate_second_half(x, other, cos_row[pair], sin_row[pair])
                       : rotate_first_half(x, other, cos_row[pair], sin_row[pair]);
        }
        if (is_q) {
            from_f32(q_out + (size_t)row * qn + i, x);
        } else if (kept) {
            T k;
            from_f32(&k, x);
            k_cache[(((size_t)page * kv_heads + (i - qn) / key_dim) * page_size + slot) * key_dim + d] = cache_value(k);
        }
    }
    const int vn = kv_heads * value_dim;
    if (kept)
        for (int i = tid; i < vn; i += PN_THREADS) {
            T v;
            from_f32(&v, to_f32(src[qn + kn + i]) + (bias ? bias[qn + kn + i] : 0.f));
            v_cache[((size_t)page * vn + i) * page_size + slot] = cache_value(v);      // (kv head, dim) is i
        }
    if (single && pooled.pool > 0 && (pos + 1) % pooled.pool == 0) {
        __syncthreads();                                 // the row's own key and value are in their page
        const int* pooled_table = pooled.tables + (size_t)seq_of_row[row] * pooled.width;
        for (int g = 0; g < kv_heads; ++g)
            store_block_means<T>(k_cache, v_cache, table, page_size, num_pages, kv_heads, key_dim, value_dim, g, pos / pooled.pool,
                                 pooled, pooled_table, tid, PN_THREADS);
    }
}

template <typename T>
__global__ __launch_bounds__(PN_THREADS) void pool_blocks_kernel(
    const T* __restrict__ k_cache, const T* __restrict__ v_cache, const int* __restrict__ row_start,
    const int* __restrict__ seq_start, int num_seqs, const int* __restrict__ tables, int table_width, int page_size, int num_pages,
    int kv_heads, int key_dim, int value_dim, PooledKeys pooled) {
    int block = blockIdx.x, seq = 0;
    for (; seq < num_seqs; ++seq) {
        const int start = seq_start[seq], end = start + row_start[seq + 1] - row_start[seq];
        const int first = start / pooled.pool, count = end / pooled.pool - first;      // blocks that end within the step
        if (block < count) {
            block += first;
            break;
        }
        block -= count;
    }
    if (seq >= num_seqs) return;                         // (the grid's slack)
    store_block_means<T>(k_cache, v_cache, tables + (size_t)seq * table_width, page_size, num_pages, kv_heads, key_dim, value_dim,
                         blockIdx.y, block, pooled, pooled.tables + (size_t)seq * pooled.width, threadIdx.x, blockDim.x);
}

// proj: [rows, ld], q (heads key_dim) | k (kv_heads key_dim) | v (kv_heads value_dim) first; bias: float32 over these or
// null; q_weight [heads key_dim], k_weight [kv_heads key_dim]: float32 or null; cos, sin: float32 [table_positions, dims / 2]
// or null; pooled caches and tables as in pooled.h (pool 0: none); single: every sequence brings one row
extern "C" int tli_pooled_prepare(const void* proj, int ld, const float* bias, void* q_out, void* k_cache, void* v_cache,
                                  const int* positions, const int* seq_of_row, const int* row_start, const int* seq_start,
                                  int num_seqs, const int* tables, int table_width, int page_size, int num_pages, int rows,
                                  int heads, int kv_heads, int key_dim, int value_dim, const float* q_weight,
                                  const float* k_weight, float eps, const float* cos_table, const float* sin_table, int dims,
                                  int pairing, int table_positions, void* pooled_k, void* pooled_v, const int* pooled_tables,
                                  int pooled_width, int pooled_pages, int pool, int single, int dtype, void* stream) {
    if (rows <= 0) return 0;
    if (heads <= 0 || kv_heads <= 0 || key_dim <= 0 || value_dim <= 0) return tli_fail("pooled_prepare: bad sizes");
    if (ld < (heads + kv_heads) * key_dim + kv_heads * value_dim) return tli_fail("pooled_prepare: rows of %d do not hold the projections", ld);
    if (cos_table && (dims <= 0 || dims % 2 || dims > key_dim)) return tli_fail("pooled_prepare: %d turned elements of heads of %d", dims, key_dim);
    if (page_size <= 0 || table_width <= 0 || num_pages <= 0) return tli_fail("pooled_prepare: bad cache geometry");
    if (pool < 0 || (pool > 0 && (pooled_width <= 0 || pooled_pages <= 0))) return tli_fail("pooled_prepare: bad blocks of %d", pool);
    if (single && rows != num_seqs) return tli_fail("pooled_prepare: %d rows are not one for each of %d sequences", rows, num_seqs);
    if (kv_heads > 65535) return tli_fail("pooled_prepare: too many heads");
    const size_t lds = (size_t)(heads + kv_heads) * key_dim * sizeof(float);
    if (lds > 150 * 1024) return tli_fail("pooled_prepare: q and k of %zu bytes do not fit LDS", lds);
    const PooledKeys pooled{pooled_k, pooled_v, pooled_tables, pooled_width, pooled_pages, pool};
    hipStream_t s = (hipStream_t)stream;
#define PN_RUN(T)                                                                                                              \
    {                                                                                                                          \
        auto kernel = projection_norm_prepare_kernel<T>;                                                                       \
        static bool allowed = false;                                                                                           \
        if (lds > 65536 && !allowed) {                                                                                         \
            if (hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024) != hipSuccess) \
                return tli_fail("pooled_prepare: cannot have %zu bytes of LDS", lds);                                          \
            allowed = true;                                                                                                    \
        }                                                                                                                      \
        kernel<<<rows, PN_THREADS, lds, s>>>((const T*)proj, ld, bias, (T*)q_out, (T*)k_cache, (T*)v_cache, positions,          \
                                             seq_of_row, tables, table_width, page_size, num_pages, heads, kv_heads, key_dim,  \
                                             value_dim, q_weight, k_weight, eps, cos_table, sin_table, dims, pairing,          \
                                             table_positions, pooled, single);                                                 \
        if (pool > 0 && !single)                                                                                               \
            pool_blocks_kernel<T><<<dim3(rows / pool + num_seqs, kv_heads), PN_THREADS, 0, s>>>(                               \
                (const T*)k_cache, (const T*)v_cache, row_start, seq_start, num_seqs, tables, table_width, page_size,          \
                num_pages, kv_heads, key_dim, value_dim, pooled);                                                              \
    }
    if (dtype == TLI_F32) PN_RUN(float)
    else if (dtype == TLI_BF16) PN_RUN(bf16_t)
    else return tli_fail("pooled_prepare: unknown dtype %d", dtype);
#undef PN_RUN
    return tli_check_launch("pooled_prepare");
}
