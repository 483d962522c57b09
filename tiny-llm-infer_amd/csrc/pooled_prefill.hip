// Portions of prompts through the attention over a window and pooled blocks (pooled.h), on the matrix cores: bfloat16,
// key and value heads of 64 or of 128.  What it computes is what attention_sized_plain.hip computes with pooled blocks.
//
// A workgroup of four waves; a wave has one query head and a tile of 32 consecutive rows of one sequence (two column tiles
// of 16 of the transposed products S^T = K Q^T and O^T = V^T P^T), and the four read the same key head, so that they share
// every tile of 32 keys.  Tiles are numbered row tile by row tile and, within one, head by head of the key head's query
// heads.  The 256 threads bring a tile's keys [32][dim] and its values, transposed [dim][32] as the cache has them, into
// LDS with 16-byte loads, the next two tiles' on their way meanwhile (the pages of everything that is seen are looked up
// once, into LDS), two buffers taking turns with one barrier a tile.  A
// fragment of K or V^T read from LDS serves both column tiles.
//
// v_mfma_f32_16x16x32_bf16: A: lane l has row l % 16, k = 8 (l / 16) .. + 7; B: the same k of column l % 16; sums: rows
// 4 (l / 16) .. + 3 of column l % 16.  The scores of two tiles of 16 keys leave lane group c with keys 4 c .. + 3 and
// 16 + 4 c .. + 3, which are taken as its eight k of the second product as they are; V^T's fragment takes the same keys.
#include "common.h"
#include "pooled.h"

typedef __attribute__((ext_vector_type(8))) __bf16 pp_bf16x8;
typedef __attribute__((ext_vector_type(4))) float pp_f32x4;
typedef __attribute__((ext_vector_type(4))) uint32_t pp_u32x4;     // (arrays of uint4 that lambdas fill would go to memory)

union PpFrag {
    uint4 q;
    uint2 d[2];
    uint32_t w[4];
    pp_bf16x8 v;
};

#define PP_WAVES 4
#define PP_ROWS 32
#define PP_KEYS 32
#define PP_VLD (PP_KEYS + 8)         // bfloat16 elements a row of V^T in LDS
#define PP_TABLE 6144                // the most pages that a workgroup's rows may see

// NK, NV: sixteens of a key and of a value
template <int NK, int NV>
__global__ __launch_bounds__(64 * PP_WAVES, 2) void pooled_prefill_kernel(
    const bf16_t* __restrict__ q, bf16_t* __restrict__ out, int out_ld, const bf16_t* __restrict__ k_cache,
    const bf16_t* __restrict__ v_cache, const int* __restrict__ row_start, const int* __restrict__ seq_start, int num_seqs,
    const int* __restrict__ tables, int table_width, int page_size, int num_pages, int heads, int kv_heads, float scale_log2,
    int window, const float* __restrict__ sinks, PooledKeys pooled, float out_scale, int table_room) {
    constexpr int DK = NK * 16, DV = NV * 16, LD = DK + 8, C = PP_ROWS / 16;
    constexpr int KP = PP_KEYS * DK / 8 / (64 * PP_WAVES), VP = DV * PP_KEYS / 8 / (64 * PP_WAVES);      // 16-byte pieces a thread brings
    static_assert(KP * 64 * PP_WAVES * 8 == PP_KEYS * DK && VP * 64 * PP_WAVES * 8 == DV * PP_KEYS, "a tile is shared out evenly");
    __shared__ __align__(16) bf16_t k_lds[2][PP_KEYS * LD];
    __shared__ __align__(16) bf16_t v_lds[2][DV * PP_VLD];
    extern __shared__ int pages_s[];                                   // of the tokens from k_low on, then of the blocks
    const int tid = threadIdx.x, lane = tid % 64, wave = __builtin_amdgcn_readfirstlane(tid / 64), col = lane % 16, grp = lane / 16;
    const int per_kv = heads / kv_heads, g = blockIdx.y;
    int wg = blockIdx.x, seq = 0, first_row = 0, count = 0, units = 0;
    for (; seq < num_seqs; ++seq) {
        first_row = row_start[seq];
        count = row_start[seq + 1] - first_row;
        units = ((count + PP_ROWS - 1) / PP_ROWS) * per_kv;
        const int n_wg = (units + PP_WAVES - 1) / PP_WAVES;
        if (wg < n_wg) {
            wg = n_wg - 1 - wg;                                        // (the rows that see the most keys start first)
            break;
        }
        wg -= n_wg;
    }
    if (seq >= num_seqs) return;                                       // (the whole workgroup)
    const int unit = min(wg * PP_WAVES + wave, units - 1);
    const bool works = wg * PP_WAVES + wave < units;
    const int rt = unit / per_kv, head = g * per_kv + unit % per_kv;
    const int rt_first = wg * PP_WAVES / per_kv, rt_last = min(wg * PP_WAVES + PP_WAVES - 1, units - 1) / per_kv;
    const int base = seq_start[seq];
    // what the workgroup's rows see: tokens lo .. hi and the first blocks_hi blocks; and this wave's
    const int hi = base + min(count, (rt_last + 1) * PP_ROWS) - 1, lo = max(0, base + rt_first * PP_ROWS - window + 1);
    const int blocks_hi = pooled_blocks_seen(hi, window, pooled.pool);
    const int w_first = base + rt * PP_ROWS, w_last = base + min(count, (rt + 1) * PP_ROWS) - 1;
    const int w_lo = max(0, w_first - window + 1), w_blocks = pooled_blocks_seen(w_last, window, pooled.pool);
    const int blocks_all = pooled_blocks_seen(w_first, window, pooled.pool);                // seen by every row of the wave
    const int* table = tables + (size_t)seq * table_width;
    const int* block_table = pooled.tables + (size_t)seq * pooled.width;
    const size_t k_page = (size_t)kv_heads * page_size * DK, v_page = (size_t)kv_heads * page_size * DV;
    const int shift = __builtin_ctz(page_size), mask = page_size - 1;
    const int k_low = lo / PP_KEYS * PP_KEYS, k_top = hi / PP_KEYS * PP_KEYS;
    const int n_tokens = (k_top - k_low) / PP_KEYS + 1, n_tiles = n_tokens + (blocks_hi + PP_KEYS - 1) / PP_KEYS;
    auto is_block = [&](int i) { return i >= n_tokens; };
    auto tile_key = [&](int i) { return is_block(i) ? (i - n_tokens) * PP_KEYS : k_top - i * PP_KEYS; };

    const int page_low = k_low >> shift, token_pages = (hi >> shift) - page_low + 1;
    const int block_pages = blocks_hi > 0 ? ((blocks_hi - 1) >> shift) + 1 : 0;
    if (token_pages + block_pages > table_room) return;                // (the host makes room for all)
    for (int i = tid; i < token_pages + block_pages; i += 64 * PP_WAVES) {
        const bool block = i >= token_pages;
        const int page = block ? block_table[i - token_pages] : table[page_low + i];
        pages_s[i] = page >= 0 && page < (block ? pooled.pages : num_pages) ? page : 0;
    }
    __syncthreads();
    static_assert(64 * PP_WAVES == 8 * PP_KEYS, "eight threads a key");
    struct Tile {
        pp_u32x4 k[KP], v[VP];
    };
    const int k_key = tid / 8, k_piece = tid % 8;                      // of a tile's keys; pieces k_piece + 8 ps of it
    auto fetch = [&](int i, Tile& tile) {
        const bool block = is_block(i);
        const bf16_t* kc = block ? (const bf16_t*)pooled.k : k_cache;
        const bf16_t* vc = block ? (const bf16_t*)pooled.v : v_cache;
        const int limit = block ? blocks_hi - 1 : hi, k0 = tile_key(i), from = block ? token_pages : -page_low;
        // (a key past the last that is seen is read as the last one: its page is there)
        auto page_of = [&](int key) { return pages_s[(key >> shift) + from]; };
        {
            const int key = min(k0 + k_key, limit);
            const bf16_t* src = kc + (size_t)page_of(key) * k_page + ((size_t)g * page_size + (key & mask)) * DK;
#pragma unroll
            for (int ps = 0; ps < KP; ++ps) tile.k[ps] = *reinterpret_cast<const pp_u32x4*>(src + (k_piece + 8 * ps) * 8);
        }
#pragma unroll
        for (int ps = 0; ps < VP; ++ps) {
            const int c = tid + ps * 64 * PP_WAVES, key = min(k0 + (c % 4) * 8, limit & ~7);        // eight slots in a row lie in one page
            tile.v[ps] = *reinterpret_cast<const pp_u32x4*>(vc + (size_t)page_of(key) * v_page + ((size_t)g * DV + c / 4) * page_size + (key & mask));
        }
    };
    auto store = [&](int buf, const Tile& tile) {
#pragma unroll
        for (int ps = 0; ps < KP; ++ps) *reinterpret_cast<pp_u32x4*>(k_lds[buf] + k_key * LD + (k_piece + 8 * ps) * 8) = tile.k[ps];
#pragma unroll
        for (int ps = 0; ps < VP; ++ps) {
            const int c = tid + ps * 64 * PP_WAVES;
            *reinterpret_cast<pp_u32x4*>(v_lds[buf] + (c / 4) * PP_VLD + (c % 4) * 8) = tile.v[ps];
        }
    };
    Tile even, odd;                                                    // tiles 0, 2, .. and 1, 3, .. on their way
    fetch(0, even);
    if (n_tiles > 1) fetch(1, odd);

    PpFrag qf[C][NK / 2];
    int qpos[C], qlo[C], qblocks[C], row[C];
    float m[C], l[C];
    pp_f32x4 acc[C][NV];
#pragma unroll
    for (int c = 0; c < C; ++c) {
        const int r = min(rt * PP_ROWS + c * 16 + col, count - 1);     // (idle columns repeat the last row; never stored)
        row[c] = first_row + r;
        qpos[c] = base + r;
        qlo[c] = max(0, qpos[c] - window + 1);
        qblocks[c] = pooled_blocks_seen(qpos[c], window, pooled.pool);
        m[c] = -INFINITY;
        l[c] = 0.f;
#pragma unroll
        for (int j = 0; j < NK / 2; ++j)
            qf[c][j].q = *reinterpret_cast<const uint4*>(q + ((size_t)row[c] * heads + head) * DK + 32 * j + 8 * grp);
#pragma unroll
        for (int t = 0; t < NV; ++t) acc[c][t] = (pp_f32x4){0.f, 0.f, 0.f, 0.f};
    }
    store(0, even);
    __syncthreads();
    // tile `it` is in LDS, `next` is tile it + 1 on its way; `free` takes tile it + 2
    auto step = [&](int it, Tile& free, const Tile& next) {
        const int k0 = tile_key(it);
        const bool block = is_block(it), more = it + 1 < n_tiles;
        if (it + 2 < n_tiles) fetch(it + 2, free);
        // (the same for the whole wave)
        if (works && (block ? k0 < w_blocks : k0 <= w_last && k0 + PP_KEYS > w_lo)) {
            const bf16_t* kt = k_lds[it & 1];
            const bf16_t* vt = v_lds[it & 1];
            pp_f32x4 s[C][2];
#pragma unroll
            for (int c = 0; c < C; ++c)
#pragma unroll
                for (int t = 0; t < 2; ++t) s[c][t] = (pp_f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int j = 0; j < NK / 2; ++j)
#pragma unroll
                for (int t = 0; t < 2; ++t) {
                    PpFrag a;
                    a.q = *reinterpret_cast<const uint4*>(kt + (16 * t + col) * LD + 32 * j + 8 * grp);
#pragma unroll
                    for (int c = 0; c < C; ++c) s[c][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, qf[c][j].v, s[c][t], 0, 0, 0);
                }
            const bool all = block ? k0 + PP_KEYS <= blocks_all : k0 + PP_KEYS - 1 <= w_first && k0 >= w_last - window + 1;
            PpFrag p[C];
            bool rescale = false;
            float corr[C];
#pragma unroll
            for (int c = 0; c < C; ++c) {
                const int s_hi = block ? qblocks[c] - 1 : qpos[c], s_lo = block ? 0 : qlo[c];
                float w[8], mx = -INFINITY;
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    const int key = k0 + (e < 4 ? 0 : 16) + 4 * grp + (e & 3);
                    const float v = s[c][e / 4][e & 3] * scale_log2;
                    w[e] = all | ((key <= s_hi) & (key >= s_lo)) ? v : -INFINITY;
                    mx = fmaxf(mx, w[e]);
                }
                const float m_new = fmaxf(m[c], quad_rows_max(mx));
                // (a column whose keys so far are all hidden keeps m = -inf: its weights and its correction are 0)
                const float base_m = m_new == -INFINITY ? 0.f : m_new;
                corr[c] = __builtin_amdgcn_exp2f(m[c] - base_m);
                float sum = 0.f;
#pragma unroll
                for (int e = 0; e < 8; e += 2) {
                    const float a = __builtin_amdgcn_exp2f(w[e] - base_m), b = __builtin_amdgcn_exp2f(w[e + 1] - base_m);
                    const uint32_t both = pack_bf16x2(a, b);
                    p[c].w[e / 2] = both;
                    // the weights as the values meet them
                    sum += __uint_as_float(both << 16) + __uint_as_float(both & 0xffff0000u);
                }
                l[c] = fmaf(l[c], corr[c], sum);                       // (this lane group's keys; the groups are added up at the end)
                m[c] = m_new;
                rescale |= corr[c] != 1.0f;
            }
            if (__any(rescale)) {
#pragma unroll
                for (int c = 0; c < C; ++c)
#pragma unroll
                    for (int t = 0; t < NV; ++t)
#pragma unroll
                        for (int i = 0; i < 4; ++i) acc[c][t][i] *= corr[c];
            }
#pragma unroll
            for (int t = 0; t < NV; ++t) {
                PpFrag a;
                a.d[0] = *reinterpret_cast<const uint2*>(vt + (16 * t + col) * PP_VLD + 4 * grp);
                a.d[1] = *reinterpret_cast<const uint2*>(vt + (16 * t + col) * PP_VLD + 16 + 4 * grp);
#pragma unroll
                for (int c = 0; c < C; ++c) acc[c][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, p[c].v, acc[c][t], 0, 0, 0);
            }
        }
        if (more) store((it + 1) & 1, next);
        __syncthreads();                                               // the next tile is written; this one is read by all
    };
    for (int it = 0; it < n_tiles; it += 2) {
        step(it, even, odd);
        if (it + 1 < n_tiles) step(it + 1, odd, even);
    }
    if (!works) return;
#pragma unroll
    for (int c = 0; c < C; ++c) {
        const float total = quad_rows_sum(l[c]);
        float inv = out_scale / total;                                 // (a row sees itself: total > 0)
        if (sinks) {
            const float sink = sinks[head] * 1.4426950408889634f, top = fmaxf(m[c], sink), keys = __builtin_amdgcn_exp2f(m[c] - top);
            inv = out_scale * keys / (total * keys + __builtin_amdgcn_exp2f(sink - top));
        }
        if (rt * PP_ROWS + c * 16 + col >= count) continue;
        bf16_t* dst = out + (size_t)row[c] * out_ld + (size_t)head * DV + 4 * grp;
#pragma unroll
        for (int t = 0; t < NV; ++t)
            *reinterpret_cast<uint2*>(dst + 16 * t) = make_uint2(pack_bf16x2(acc[c][t][0] * inv, acc[c][t][1] * inv),
                                                                 pack_bf16x2(acc[c][t][2] * inv, acc[c][t][3] * inv));
    }
}

// The most pages that a workgroup's rows see in sequences of up to `longest` tokens: their windows', and all blocks'
static int pp_pages(int longest, int window, int pool, int page_size) {
    const long long tokens = ((long long)window + PP_WAVES * PP_ROWS + PP_KEYS < longest ? (long long)window + PP_WAVES * PP_ROWS + PP_KEYS : longest) / page_size + 2;
    return (int)(tokens + longest / ((long long)pool * page_size) + 2);
}

// Whether these sizes have a kernel here (else attention_sized_mfma.hip or the plain kernel serves).
extern "C" int tli_pooled_prefill_takes(int key_dim, int value_dim, int page_size, int longest, int window, int pool) {
    return pp_pages(longest, window, pool, page_size) <= PP_TABLE && ((key_dim == 64 && value_dim == 64) || (key_dim == 128 && value_dim == 128)) && page_size >= 8 && !(page_size & (page_size - 1));
}

// The arguments as for tli_attention_pooled_mfma_bf16 (attention_sized_mfma.hip); row_tiles: an upper bound of the sum over
// the sequences of ceil(rows / 32); longest: an upper bound of the sequences' tokens
extern "C" int tli_pooled_prefill_bf16(const void* q, void* out, const void* k_cache, const void* v_cache, const int* row_start,
                                       const int* seq_start, int num_seqs, int row_tiles, const int* tables, int table_width,
                                       int page_size, int num_pages, int heads, int kv_heads, int key_dim, int value_dim, float scale,
                                       int window, const void* pooled_k, const void* pooled_v, const int* pooled_tables,
                                       int pooled_width, int pooled_pages, int pool, int longest, const float* sinks, int out_ld, float out_scale,
                                       void* stream) {
    if (num_seqs <= 0 || row_tiles <= 0) return 0;
    if (window <= 0 || pool <= 0 || page_size <= 0 || longest <= 0) return tli_fail("pooled_prefill: blocks of %d beside a window of %d", pool, window);
    if (!tli_pooled_prefill_takes(key_dim, value_dim, page_size, longest, window, pool))
        return tli_fail("pooled_prefill: keys of %d and values of %d in pages of %d", key_dim, value_dim, page_size);
    if (heads <= 0 || kv_heads <= 0 || heads % kv_heads || kv_heads > 65535) return tli_fail("pooled_prefill: %d heads over %d", heads, kv_heads);
    if (table_width <= 0 || num_pages <= 0 || pooled_width <= 0 || pooled_pages <= 0)
        return tli_fail("pooled_prefill: bad cache geometry");
    if (out_ld % 4 || out_ld < heads * value_dim) return tli_fail("pooled_prefill: output rows of %d elements", out_ld);
    if ((((uintptr_t)q | (uintptr_t)k_cache | (uintptr_t)v_cache | (uintptr_t)pooled_k | (uintptr_t)pooled_v) & 15) || ((uintptr_t)out & 7))
        return tli_fail("pooled_prefill: operands must be 16-byte aligned");
    const PooledKeys pooled{pooled_k, pooled_v, pooled_tables, pooled_width, pooled_pages, pool};
    // (a sequence's tiles are rounded up to whole workgroups: at most one more a sequence; a workgroup past the last leaves)
    const long long wgs = ((long long)row_tiles * (heads / kv_heads) + PP_WAVES - 1) / PP_WAVES + num_seqs;
    if (wgs > 0x7fffffffLL) return tli_fail("pooled_prefill: too many tiles for one launch");
    const dim3 grid((unsigned)wgs, kv_heads);
    hipStream_t s = (hipStream_t)stream;
    const int room = pp_pages(longest, window, pool, page_size);
    const float scale_log2 = scale * 1.4426950408889634f;
#define PP_RUN(NK, NV)                                                                                                            \
    pooled_prefill_kernel<NK, NV><<<grid, 64 * PP_WAVES, (size_t)room * sizeof(int), s>>>((const bf16_t*)q, (bf16_t*)out, out_ld, (const bf16_t*)k_cache, \
                                                                 (const bf16_t*)v_cache, row_start, seq_start, num_seqs, tables, \
                                                                 table_width, page_size, num_pages, heads, kv_heads, scale_log2, \
                                                                 window, sinks, pooled, out_scale, room)
    if (key_dim == 128) PP_RUN(8, 8);
    else PP_RUN(4, 4);
#undef PP_RUN
    return tli_check_launch("pooled_prefill");
}
