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

#define PN_THREADS 512
#define PB_AHEAD 8             // positions of a block whose loads are under way together

// the mean of element (key: d of kv head g; value likewise) over the block's positions, read from the tokens' pages
template <typename T, bool VALUE>
__device__ __forceinline__ float block_mean(const T* __restrict__ cache, const int* __restrict__ table, int page_size, int num_pages,
                                            int kv_heads, int g, int dim, int d, int first, int pool) {
    float sum = 0.f;
    int at = first / page_size, slot = first - at * page_size;
    for (int j0 = 0; j0 < pool; j0 += PB_AHEAD) {        // every load of eight positions is issued before one is used
        int page[PB_AHEAD], where[PB_AHEAD];
        float v[PB_AHEAD];
#pragma unroll
        for (int j = 0; j < PB_AHEAD; ++j) {
            page[j] = table[at];
            where[j] = slot;
            if (j0 + j + 1 < pool) ++slot;               // (past the block's end: its last position again, not added)
            if (slot == page_size) slot = 0, ++at;
        }
#pragma unroll
        for (int j = 0; j < PB_AHEAD; ++j) {
            const bool have = page[j] >= 0 && page[j] < num_pages;
            const size_t head = ((size_t)(have ? page[j] : 0) * kv_heads + g) * page_size * dim;
            v[j] = to_f32(VALUE ? cache[head + (size_t)d * page_size + where[j]] : cache[head + (size_t)where[j] * dim + d]);
        }
#pragma unroll
        for (int j = 0; j < PB_AHEAD; ++j) asm volatile("" : "+v"(v[j]));       // (not loaded under the conditions below)
#pragma unroll
        for (int j = 0; j < PB_AHEAD; ++j) sum += page[j] >= 0 && page[j] < num_pages && j0 + j < pool ? v[j] : 0.f;
    }
    return sum / (float)pool;
}

// element e of a block's means of kv head g: e < key_dim the key's, then the value's
template <typename T>
__device__ __forceinline__ void store_block_mean(const T* __restrict__ k_cache, const T* __restrict__ v_cache,
                                                 const int* __restrict__ table, int page_size, int num_pages, int kv_heads,
                                                 int key_dim, int value_dim, int g, int e, int block, const PooledKeys& pooled,
                                                 const int* __restrict__ pooled_table) {
    const int page = pooled_table[block / page_size], slot = block % page_size;
    if (page < 0 || page >= pooled.pages) return;
    const size_t head = ((size_t)page * kv_heads + g) * page_size;
    T m;
    if (e < key_dim) {
        from_f32(&m, block_mean<T, false>(k_cache, table, page_size, num_pages, kv_heads, g, key_dim, e, block * pooled.pool, pooled.pool));
        ((T*)pooled.k)[(head + slot) * key_dim + e] = cache_value(m);
    } else {
        const int d = e - key_dim;
        from_f32(&m, block_mean<T, true>(v_cache, table, page_size, num_pages, kv_heads, g, value_dim, d, block * pooled.pool, pooled.pool));
        ((T*)pooled.v)[head * value_dim + (size_t)d * page_size + slot] = cache_value(m);
    }
}

// N consecutive elements at once: 8 where sizes and addresses allow 16-byte accesses of bfloat16, else 1
template <int N, typename T>
__device__ __forceinline__ void pn_load(const T* p, float (&v)[N]) {
    if constexpr (N == 8) {
        const uint4 w = *reinterpret_cast<const uint4*>(p);
        const uint32_t u[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
        for (int i = 0; i < 4; ++i) v[2 * i] = bf16_to_f32((bf16_t)(u[i] & 0xffffu)), v[2 * i + 1] = bf16_to_f32((bf16_t)(u[i] >> 16));
    } else {
        v[0] = to_f32(p[0]);
    }
}
template <int N>
__device__ __forceinline__ void pn_load_f32(const float* p, float (&v)[N]) {
    if constexpr (N == 8) {
        const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
        v[0] = a.x, v[1] = a.y, v[2] = a.z, v[3] = a.w, v[4] = b.x, v[5] = b.y, v[6] = b.z, v[7] = b.w;
    } else {
        v[0] = p[0];
    }
}
template <int N, bool CACHE, typename T>
__device__ __forceinline__ void pn_store(T* p, const float (&v)[N]) {
    T o[N];
#pragma unroll
    for (int i = 0; i < N; ++i) {
        from_f32(o + i, v[i]);
        if (CACHE) o[i] = cache_value(o[i]);
    }
    if constexpr (N == 8)
        *reinterpret_cast<uint4*>(p) = make_uint4(o[0] | (uint32_t)o[1] << 16, o[2] | (uint32_t)o[3] << 16, o[4] | (uint32_t)o[5] << 16,
                                                  o[6] | (uint32_t)o[7] << 16);
    else
        p[0] = o[0];
}

// any sizes
template <typename T>
__global__ __launch_bounds__(PN_THREADS) void projection_norm_prepare_kernel(
    const T* __restrict__ proj, int ld, const float* __restrict__ bias, T* __restrict__ q_out, T* k_cache, T* v_cache,
    const int* __restrict__ positions, const int* __restrict__ seq_of_row, const int* __restrict__ tables, int table_width,
    int page_size, int num_pages, int heads, int kv_heads, int key_dim, int value_dim, const float* __restrict__ q_weight,
    const float* __restrict__ k_weight, float eps, const float* __restrict__ cos_table, const float* __restrict__ sin_table,
    int dims, int pairing, int table_positions, PooledKeys pooled, int single) {
    constexpr int N = 1;
    extern __shared__ __align__(16) float pn_row[];      // q and k of the row, all heads, times their norm's weights
    __shared__ float red[16];
    const int row = blockIdx.x, tid = threadIdx.x;
    const int qn = heads * key_dim, kn = kv_heads * key_dim, vn = kv_heads * value_dim;
    const T* src = proj + (size_t)row * ld;
    const int pos = positions[row];
    const int* table = tables + (size_t)seq_of_row[row] * table_width;
    const int page = table[pos / page_size], slot = pos % page_size;
    const bool kept = page >= 0 && page < num_pages;
    float ssq = 0.f, ssk = 0.f;
    for (int i = tid * N; i < qn + kn; i += PN_THREADS * N) {
        float x[N], w[N];
        pn_load<N>(src + i, x);
        if (bias) {
            pn_load_f32<N>(bias + i, w);
#pragma unroll
            for (int j = 0; j < N; ++j) x[j] += w[j];
        }
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < N; ++j) ss = fmaf(x[j], x[j], ss);
        const bool is_q = i < qn;
        const float* weight = is_q ? q_weight : k_weight;
        (is_q ? ssq : ssk) += ss;
        if (weight) {
            pn_load_f32<N>(weight + (is_q ? i : i - qn), w);
#pragma unroll
            for (int j = 0; j < N; ++j) x[j] *= w[j];
        }
#pragma unroll
        for (int j = 0; j < N; ++j) pn_row[i + j] = x[j];
    }
    if (kept)
        for (int i = tid * N; i < vn; i += PN_THREADS * N) {
            float x[N], w[N];
            pn_load<N>(src + qn + kn + i, x);
            if (bias) {
                pn_load_f32<N>(bias + qn + kn + i, w);
#pragma unroll
                for (int j = 0; j < N; ++j) x[j] += w[j];
            }
#pragma unroll
            for (int j = 0; j < N; ++j) {
                T v;
                from_f32(&v, x[j]);
                v_cache[((size_t)page * vn + i + j) * page_size + slot] = cache_value(v);      // (kv head, dim) is i + j
            }
        }
    // (the sums of q and of k in one exchange)
    {
        const float a = wave_sum(ssq), b = wave_sum(ssk);
        if (tid % TLI_WAVE == 0) red[tid / TLI_WAVE] = a, red[8 + tid / TLI_WAVE] = b;
    }
    __syncthreads();                                     // (pn_row as well)
    float q_factor = 1.f, k_factor = 1.f;
    {
        float a = 0.f, b = 0.f;
#pragma unroll
        for (int w = 0; w < PN_THREADS / TLI_WAVE; ++w) a += red[w], b += red[8 + w];
        if (q_weight) q_factor = 1.0f / sqrtf(a / (float)qn + eps);
        if (k_weight) k_factor = 1.0f / sqrtf(b / (float)kn + eps);
    }
    const int half = dims / 2;
    const bool turn = cos_table && pos >= 0 && pos < table_positions;
    const float* cos_row = turn ? cos_table + (size_t)pos * half : nullptr;
    const float* sin_row = turn ? sin_table + (size_t)pos * half : nullptr;
    for (int i = tid * N; i < qn + kn; i += PN_THREADS * N) {
        const bool is_q = i < qn;
        const int base = is_q ? 0 : qn, d0 = (i - base) % key_dim;
        const float factor = is_q ? q_factor : k_factor;
        float x[N];
#pragma unroll
        for (int j = 0; j < N; ++j) {
            const int d = d0 + j;
            x[j] = pn_row[i + j] * factor;
            if (turn && d < dims) {
                const bool second = pairing ? (d & 1) : d >= half;
                const int pair = pairing ? d / 2 : second ? d - half : d;
                const int at = i + j;
                const float other = pn_row[pairing ? (second ? at - 1 : at + 1) : second ? at - half : at + half] * factor;
                x[j] = second ? rotate_second_half(x[j], other, cos_row[pair], sin_row[pair])
                              : rotate_first_half(x[j], other, cos_row[pair], sin_row[pair]);
            }
        }
        if (is_q) pn_store<N, false>(q_out + (size_t)row * qn + i, x);
        else if (kept) pn_store<N, true>(k_cache + (((size_t)page * kv_heads + (i - qn) / key_dim) * page_size + slot) * key_dim + d0, x);
    }
    if (single && pooled.pool > 0 && (pos + 1) % pooled.pool == 0) {
        __syncthreads();                                 // the row's own key and value are in their page
        const int* pooled_table = pooled.tables + (size_t)seq_of_row[row] * pooled.width;
        const int each = key_dim + value_dim;
        for (int u = tid; u < kv_heads * each; u += PN_THREADS)
            store_block_mean<T>(k_cache, v_cache, table, page_size, num_pages, kv_heads, key_dim, value_dim, u / each, u % each,
                                pos / pooled.pool, pooled, pooled_table);
    }
}

// Sizes in eights, bfloat16: a thread takes pieces of 8 elements (16 bytes) of the row q | k | v, up to KEEP of them,
// and asks for all it needs before it waits for anything: projections, biases, weights, and (neighbours: the partner
// is in the piece) the rotation's cosines and sines.
template <int KEEP>
__global__ __launch_bounds__(PN_THREADS) void projection_norm_prepare8_kernel(
    const bf16_t* __restrict__ proj, int ld, const float* __restrict__ bias, bf16_t* __restrict__ q_out, bf16_t* k_cache,
    bf16_t* v_cache, const int* __restrict__ positions, const int* __restrict__ seq_of_row, const int* __restrict__ tables,
    int table_width, int page_size, int num_pages, int heads, int kv_heads, int key_dim, int value_dim,
    const float* __restrict__ q_weight, const float* __restrict__ k_weight, float eps, const float* __restrict__ cos_table,
    const float* __restrict__ sin_table, int dims, int pairing, int table_positions, PooledKeys pooled, int single) {
    extern __shared__ __align__(16) float pn_row[];      // pairing 0: q and k of the row times their norm's weights
    __shared__ float red[16];
    const int row = blockIdx.x, tid = threadIdx.x;
    const int qn = heads * key_dim, kn = kv_heads * key_dim, vn = kv_heads * value_dim, all = qn + kn + vn;
    const bf16_t* src = proj + (size_t)row * ld;
    const int pos = positions[row];
    const int* table = tables + (size_t)seq_of_row[row] * table_width;
    const int half = dims / 2;
    const bool turn = cos_table && pos >= 0 && pos < table_positions;
    const float* cos_row = turn ? cos_table + (size_t)pos * half : nullptr;
    const float* sin_row = turn ? sin_table + (size_t)pos * half : nullptr;
    float x[KEEP][8];
    float cs[KEEP][4], sn[KEEP][4];
    int dim0[KEEP];
    float ssq = 0.f, ssk = 0.f;
#pragma unroll
    for (int u = 0; u < KEEP; ++u) {
        const int i = (tid + u * PN_THREADS) * 8;
        dim0[u] = i < qn + kn ? (i < qn ? i : i - qn) % key_dim : 0;
        if (i >= all) continue;
        pn_load<8>(src + i, x[u]);
        if (bias) {
            float w[8];
            pn_load_f32<8>(bias + i, w);
#pragma unroll
            for (int j = 0; j < 8; ++j) x[u][j] += w[j];
        }
        if (i >= qn + kn) continue;
        if (turn && pairing && dim0[u] < dims) {
            const float4 c = *reinterpret_cast<const float4*>(cos_row + dim0[u] / 2), s = *reinterpret_cast<const float4*>(sin_row + dim0[u] / 2);
            cs[u][0] = c.x, cs[u][1] = c.y, cs[u][2] = c.z, cs[u][3] = c.w;
            sn[u][0] = s.x, sn[u][1] = s.y, sn[u][2] = s.z, sn[u][3] = s.w;
        }
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < 8; ++j) ss = fmaf(x[u][j], x[u][j], ss);
        (i < qn ? ssq : ssk) += ss;
        const float* weight = i < qn ? q_weight : k_weight;
        if (weight) {
            float w[8];
            pn_load_f32<8>(weight + (i < qn ? i : i - qn), w);
#pragma unroll
            for (int j = 0; j < 8; ++j) x[u][j] *= w[j];
        }
        if (!pairing) {
            *reinterpret_cast<float4*>(pn_row + i) = make_float4(x[u][0], x[u][1], x[u][2], x[u][3]);
            *reinterpret_cast<float4*>(pn_row + i + 4) = make_float4(x[u][4], x[u][5], x[u][6], x[u][7]);
        }
    }
    const int page = table[pos / page_size], slot = pos % page_size;
    const bool kept = page >= 0 && page < num_pages;
    {
        const float a = wave_sum(ssq), b = wave_sum(ssk);
        if (tid % TLI_WAVE == 0) red[tid / TLI_WAVE] = a, red[8 + tid / TLI_WAVE] = b;
    }
    __syncthreads();                                     // (pn_row as well)
    float q_factor = 1.f, k_factor = 1.f;
    {
        float a = 0.f, b = 0.f;
#pragma unroll
        for (int w = 0; w < PN_THREADS / TLI_WAVE; ++w) a += red[w], b += red[8 + w];
        if (q_weight) q_factor = 1.0f / sqrtf(a / (float)qn + eps);
        if (k_weight) k_factor = 1.0f / sqrtf(b / (float)kn + eps);
    }
#pragma unroll
    for (int u = 0; u < KEEP; ++u) {
        const int i = (tid + u * PN_THREADS) * 8;
        if (i >= all) continue;
        if (i >= qn + kn) {
            if (kept) {
                const int e = i - qn - kn;                             // (kv head, dim) is e + j
#pragma unroll
                for (int j = 0; j < 8; ++j) v_cache[((size_t)page * vn + e + j) * page_size + slot] = cache_value(f32_to_bf16(x[u][j]));
            }
            continue;
        }
        const float factor = i < qn ? q_factor : k_factor;
        const int d0 = dim0[u];
        float y[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) y[j] = x[u][j] * factor;
        if (turn && d0 < dims) {
            if (pairing) {
#pragma unroll
                for (int p = 0; p < 4; ++p) {
                    const float a = y[2 * p], b = y[2 * p + 1];
                    y[2 * p] = rotate_first_half(a, b, cs[u][p], sn[u][p]);
                    y[2 * p + 1] = rotate_second_half(b, a, cs[u][p], sn[u][p]);
                }
            } else {
                const bool second = d0 >= half;                        // (half is in eights: a piece lies in one of them)
                float other[8], c[8], s[8];
                pn_load_f32<8>(pn_row + (second ? i - half : i + half), other);
                pn_load_f32<8>(cos_row + (second ? d0 - half : d0), c);
                pn_load_f32<8>(sin_row + (second ? d0 - half : d0), s);
#pragma unroll
                for (int j = 0; j < 8; ++j)
                    y[j] = second ? rotate_second_half(y[j], other[j] * factor, c[j], s[j]) : rotate_first_half(y[j], other[j] * factor, c[j], s[j]);
            }
        }
        if (i < qn) pn_store<8, false>(q_out + (size_t)row * qn + i, y);
        else if (kept) pn_store<8, true>(k_cache + (((size_t)page * kv_heads + (i - qn) / key_dim) * page_size + slot) * key_dim + d0, y);
    }
    if (single && pooled.pool > 0 && (pos + 1) % pooled.pool == 0) {
        __syncthreads();                                 // the row's own key and value are in their page
        const int* pooled_table = pooled.tables + (size_t)seq_of_row[row] * pooled.width;
        const int each = key_dim + value_dim;
        for (int u = tid; u < kv_heads * each; u += PN_THREADS)
            store_block_mean<bf16_t>(k_cache, v_cache, table, page_size, num_pages, kv_heads, key_dim, value_dim, u / each, u % each,
                                     pos / pooled.pool, pooled, pooled_table);
    }
}

#define PB_THREADS 256

template <typename T>
__global__ __launch_bounds__(PB_THREADS) void pool_blocks_kernel(
    const T* __restrict__ k_cache, const T* __restrict__ v_cache, const int* __restrict__ row_start,
    const int* __restrict__ seq_start, int num_seqs, const int* __restrict__ tables, int table_width, int page_size, int num_pages,
    int kv_heads, int key_dim, int value_dim, PooledKeys pooled) {
    // which sequence's: 64 sequences at a time, a lane each
    const int lane = threadIdx.x % 64;
    int block = blockIdx.x, seq = -1;
    for (int base = 0; base < num_seqs && seq < 0; base += 64) {
        int first = 0, count = 0;
        if (base + lane < num_seqs) {
            const int start = seq_start[base + lane], end = start + row_start[base + lane + 1] - row_start[base + lane];
            first = start / pooled.pool;
            count = end / pooled.pool - first;           // blocks that end within the step
        }
        int upto = count;
        for (int off = 1; off < 64; off *= 2) {
            const int before = __shfl_up(upto, off);
            if (lane >= off) upto += before;
        }
        const unsigned long long beyond = __ballot(block < upto);
        if (beyond) {
            const int at = __ffsll(beyond) - 1;
            block += __shfl(first - (upto - count), at);
            seq = base + at;
        } else {
            block -= __shfl(upto, 63);
        }
    }
    if (seq < 0) return;                                 // (the grid's slack)
    seq = __builtin_amdgcn_readfirstlane(seq);
    block = __builtin_amdgcn_readfirstlane(block);
    for (int e = threadIdx.x; e < key_dim + value_dim; e += blockDim.x)
        store_block_mean<T>(k_cache, v_cache, tables + (size_t)seq * table_width, page_size, num_pages, kv_heads, key_dim, value_dim,
                            blockIdx.y, e, block, pooled, pooled.tables + (size_t)seq * pooled.width);
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
#define PN_RUN(T, KERNEL)                                                                                                           \
    {                                                                                                                          \
        auto kernel = KERNEL;                                                                                                  \
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
            pool_blocks_kernel<T><<<dim3(rows / pool + num_seqs, kv_heads), PB_THREADS, 0, s>>>(                               \
                (const T*)k_cache, (const T*)v_cache, row_start, seq_start, num_seqs, tables, table_width, page_size,          \
                num_pages, kv_heads, key_dim, value_dim, pooled);                                                              \
    }
    const int pieces = ((heads + kv_heads) * key_dim + kv_heads * value_dim) / 8;
    const bool eights = ld % 8 == 0 && key_dim % 8 == 0 && value_dim % 8 == 0 && pieces <= 8 * PN_THREADS &&
                        (!cos_table || dims % (pairing ? 8 : 16) == 0) &&
                        !(((uintptr_t)proj | (uintptr_t)bias | (uintptr_t)q_out | (uintptr_t)k_cache | (uintptr_t)q_weight |
                           (uintptr_t)k_weight | (uintptr_t)cos_table | (uintptr_t)sin_table) & 15);
    if (dtype == TLI_F32) PN_RUN(float, projection_norm_prepare_kernel<float>)
    else if (dtype == TLI_BF16 && eights && pieces <= 2 * PN_THREADS) PN_RUN(bf16_t, projection_norm_prepare8_kernel<2>)
    else if (dtype == TLI_BF16 && eights) PN_RUN(bf16_t, projection_norm_prepare8_kernel<8>)
    else if (dtype == TLI_BF16) PN_RUN(bf16_t, projection_norm_prepare_kernel<bf16_t>)
    else return tli_fail("pooled_prepare: unknown dtype %d", dtype);
#undef PN_RUN
    return tli_check_launch("pooled_prepare");
}
