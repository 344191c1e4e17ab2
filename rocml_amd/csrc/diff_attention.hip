// Differential attention over the paged key/value cache for gfx950: every head has two softmax maps over the same values,
//     o = a1 - lambda a2,   a_i = softmax over the visible keys of (q_i . k_i * scale) applied to v,
// and the head's output is o / sqrt(mean(o^2) + eps) * out_scale.
//
// A query head's two maps count as two query heads and a key head's two maps as two key heads that share one value head.  Query
// rows stand in the order (key/value head, map, head of the group), so that a map's query heads of one key head are
// neighbours; keys are [page, 2 G, 64, d], values transposed inside a page [page, G, dv, 64].  H heads, G key/value heads,
// R = H / G.
//
// Prompts: a block takes 64 query rows of one head, two waves of 32 rows per map; keys of both maps and the values go through
// LDS once for all four waves, and the waves of the second map hand their outputs to those of the first through LDS, which
// combine, norm and round.  Decode steps: a block takes a token, a key/value head and a split of its pages; columns 0 .. 7 of the matrix
// products are the first map's query heads, columns 8 .. 15 the second's, the scores of both maps add up in one accumulator (each map's
// query operand is zero in the other's columns), and one product with the values serves all 16.  It reads the
// projection itself: rotation, append of the new keys and value and attention are one launch.  Everything else (32-bit, other
// sizes) runs the plain kernel per map and a combining kernel behind it.
//
// The algebra is the online softmax of the other attention kernels; scores, weights, the combination and the norm are 32-bit.
#include "common.h"
#include "attention_generic.h"

ROCML_LAST_ERROR_FN(diff_attention)

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;
typedef __attribute__((ext_vector_type(16))) float f32x16_t;
typedef __attribute__((ext_vector_type(4))) uint32_t u32x4_t;

constexpr int DA_PAGE = 64;
constexpr int DA_THREADS = 256;
constexpr int DA_QTILE = 64;            // query rows of a prompt block
constexpr int DA_ROUND = 256;           // blocks that start together: one per CU
constexpr float DA_LAZY_MAX = 8.0f;     // how far a row's maximum may run ahead of its exponents' reference (powers of two)
constexpr int DA_MAX_GROUP = 8;         // query heads per key/value head in a decode block
static const float DA_LOG2E = 1.4426950408889634f;

__device__ __forceinline__ float da_exp2(float x) { return __builtin_amdgcn_exp2f(x); }

__device__ __forceinline__ float da_across_halves(float v, bool is_max) {
    typedef __attribute__((ext_vector_type(2))) unsigned u32x2_;
    u32x2_ r = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    float a = __uint_as_float(r[0]), b = __uint_as_float(r[1]);
    return is_max ? fmaxf(a, b) : a + b;
}

struct DiffArgs {
    const bf16_t* q;                    // prompts: [T, 2 H, d]
    bf16_t* out;                        // [T, H dv]
    bf16_t* kcache; bf16_t* vcache;
    const int* block_table; int bt_width; const int* token_pos;
    const int* cu_seqlens; int n_seqs;
    int heads, kv; int d, dv; float scale_log2e; int window;
    float lambda, out_scale, eps;
};

// ---- prompts ---------------------------------------------------------------------------------
template <int DK, int DV>
struct DiffPrefillLds {
    static constexpr int K_ROW = DK + 8, V_ROW = DA_PAGE + 8;                   // 16 bytes of padding a row
    static constexpr int TILES = (2 * DA_PAGE * K_ROW + DV * V_ROW) * 2;
    static constexpr int EXCHANGE = DA_QTILE * DV * 4;                          // the second map's outputs, 32-bit
    static constexpr int BYTES = TILES > EXCHANGE ? TILES : EXCHANGE;
};

// DK, DV: the sizes rounded up to what the kernel is made for (what lies beyond d and dv is zero).
template <int DK, int DV>
__global__ void __launch_bounds__(DA_THREADS, DV <= 128 ? 2 : 1)
diff_prefill_kernel(DiffArgs a) {
    using L = DiffPrefillLds<DK, DV>;
    constexpr int KK = DK / 16;      // matrix steps along d for the scores
    constexpr int DT = DV / 32;      // 32-row tiles of the output
    extern __shared__ uint4 da_smem[];
    bf16_t* sk = (bf16_t*)da_smem;                      // [map][64][K_ROW]
    bf16_t* sv = sk + 2 * DA_PAGE * L::K_ROW;           // [DV][V_ROW]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int map = wave >> 1, part = wave & 1;
    const int h2 = lane >> 5, col = lane & 31;
    // heavy tiles (the last of a sequence) first, every other round of blocks backwards: the CUs then carry equal sums
    int n_blocks = gridDim.x, total_tiles = n_blocks / a.heads;
    int round0 = (blockIdx.x / DA_ROUND) * DA_ROUND, in_round = blockIdx.x - round0;
    int round_size = min(DA_ROUND, n_blocks - round0);
    int s = round0 + (((blockIdx.x / DA_ROUND) & 1) ? round_size - 1 - in_round : in_round);
    const int h = s % a.heads, group = a.heads / a.kv, g = h / group;
    int tile = total_tiles - 1 - s / a.heads, b = 0, tok0 = 0, n_new = 0;
    for (; b < a.n_seqs; ++b) {
        tok0 = a.cu_seqlens[b];
        n_new = a.cu_seqlens[b + 1] - tok0;
        int tiles = (n_new + DA_QTILE - 1) / DA_QTILE;
        if (tile < tiles) break;
        tile -= tiles;
    }
    if (b >= a.n_seqs) return;
    const int* pages = a.block_table + (size_t)b * a.bt_width;
    const int pos0 = a.token_pos[tok0];
    auto first_key = [&](int pos) { return a.window > 0 ? max(0, pos - a.window + 1) : 0; };
    const int row_lo = tile * DA_QTILE, row_hi = min(n_new, row_lo + DA_QTILE) - 1;      // the block's query rows
    const int w_lo = row_lo + part * 32, w_hi = min(n_new - 1, w_lo + 31);               // the wave's
    const bool wave_active = w_lo < n_new;
    const int my_row = w_lo + col;
    const bool row_ok = my_row < n_new;
    const int my_pos = pos0 + my_row, my_lo = first_key(my_pos);
    const int wave_first_key = first_key(pos0 + w_lo), wave_last_key = pos0 + w_hi;
    const int wave_min_pos = pos0 + w_lo, wave_max_lo = first_key(pos0 + w_hi);
    const bool wave_full = w_hi - w_lo == 31;

    bf16x8_t qf[KK];                 // column = query row, 8 values of d per lane and step
    {
        int qh = (g * 2 + map) * group + h % group;
        const bf16_t* qrow = a.q + ((size_t)(tok0 + (row_ok ? my_row : 0)) * 2 * a.heads + qh) * a.d + h2 * 8;
#pragma unroll
        for (int kk = 0; kk < KK; ++kk) {
            uint4 v = make_uint4(0u, 0u, 0u, 0u);
            if (row_ok && kk * 16 + h2 * 8 < a.d) v = *(const uint4*)(qrow + kk * 16);
            qf[kk] = __builtin_bit_cast(bf16x8_t, v);
        }
    }
    float m = -INFINITY, l = 0.f;
    f32x16_t o[DT];
#pragma unroll
    for (int i = 0; i < DT; ++i)
#pragma unroll
        for (int e = 0; e < 16; ++e) o[i][e] = 0.f;

    // A page's keys and values wait in registers while the page before it is multiplied out of LDS.
    constexpr int K_PIECES = 2 * DA_PAGE * DK / 8 / DA_THREADS, V_PIECES = DV * DA_PAGE / 8 / DA_THREADS;
    u32x4_t kreg[K_PIECES], vreg[V_PIECES];
    const u32x4_t zero = {0u, 0u, 0u, 0u};
    const int first_page = first_key(pos0 + row_lo) / DA_PAGE, last_page = (pos0 + row_hi) / DA_PAGE;
    auto load_page = [&](int lp) {
        int phys = pages[lp];
        const bf16_t* gk = a.kcache + ((size_t)phys * 2 * a.kv + 2 * g) * DA_PAGE * a.d;      // both maps' rows, one behind the other
        const bf16_t* gv = a.vcache + ((size_t)phys * a.kv + g) * a.dv * DA_PAGE;
#pragma unroll
        for (int i = 0; i < K_PIECES; ++i) {
            int piece = tid + i * DA_THREADS, row = piece / (DK / 8), dc = piece % (DK / 8);
            kreg[i] = dc * 8 < a.d ? *(const u32x4_t*)(gk + (size_t)row * a.d + dc * 8) : zero;
        }
#pragma unroll
        for (int i = 0; i < V_PIECES; ++i) {
            int piece = tid + i * DA_THREADS;
            vreg[i] = piece / 8 < a.dv ? *(const u32x4_t*)(gv + (size_t)piece * 8) : zero;
        }
    };
    load_page(first_page);
    for (int lpage = first_page; lpage <= last_page; ++lpage) {
        __syncthreads();                                // the page before has been consumed
#pragma unroll
        for (int i = 0; i < K_PIECES; ++i) {
            int piece = tid + i * DA_THREADS, row = piece / (DK / 8), dc = piece % (DK / 8);
            *(u32x4_t*)(sk + row * L::K_ROW + dc * 8) = kreg[i];
        }
#pragma unroll
        for (int i = 0; i < V_PIECES; ++i) {
            // within 16 keys the four groups of 4 stand in the order 0, 2, 1, 3: the second product wants keys
            // {4h .. 4h+3, 8+4h .. 8+4h+3} per lane, the order the scores come in, as one 16-byte read
            int piece = tid + i * DA_THREADS, d = piece / 8, kc = piece % 8;
            uint2* dst = (uint2*)(sv + d * L::V_ROW + (kc >> 1) * 16 + (kc & 1) * 4);
            dst[0] = make_uint2(vreg[i][0], vreg[i][1]);
            dst[2] = make_uint2(vreg[i][2], vreg[i][3]);
        }
        __syncthreads();
        if (lpage < last_page) load_page(lpage + 1);
        if (!wave_active) continue;
        const int page_key0 = lpage * DA_PAGE;
        bool live[2];
        f32x16_t sc[2];              // element e is key 8 (e / 4) + 4 h2 + e % 4, column = query row
#pragma unroll
        for (int half = 0; half < 2; ++half) {
            int key0 = page_key0 + half * 32;
            live[half] = !(key0 > wave_last_key || key0 + 31 < wave_first_key);          // the same for the whole wave
            if (!live[half]) continue;
#pragma unroll
            for (int e = 0; e < 16; ++e) sc[half][e] = 0.f;
            const bf16_t* krow = sk + (map * DA_PAGE + half * 32 + col) * L::K_ROW + h2 * 8;
#pragma unroll
            for (int kk = 0; kk < KK; ++kk)
                sc[half] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, *(const uint4*)(krow + kk * 16)), qf[kk], sc[half], 0, 0, 0);
        }
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int half = 0; half < 2; ++half) {
            if (!live[half]) continue;
            int key0 = page_key0 + half * 32;
            f32x16_t& sh = sc[half];
            if (!wave_full || key0 + 31 > wave_min_pos || key0 < wave_max_lo) {          // some key is out of some row's sight
#pragma unroll
                for (int e = 0; e < 16; ++e) {
                    int key = key0 + 8 * (e >> 2) + 4 * h2 + (e & 3);
                    sh[e] = (row_ok && key <= my_pos && key >= my_lo) ? sh[e] : -INFINITY;
                }
            }
            float mx = sh[0];
#pragma unroll
            for (int e = 1; e < 16; ++e) mx = fmaxf(mx, sh[e]);
            mx = da_across_halves(mx, true) * a.scale_log2e;        // the scale is positive
            // the exponents' reference follows a row's maximum only when that has grown by more than DA_LAZY_MAX
            if (__builtin_amdgcn_ballot_w64(mx > m + DA_LAZY_MAX)) {
                float m_new = fmaxf(m, mx);
                float corr = da_exp2(m - (m_new == -INFINITY ? 0.f : m_new));
                l *= corr;
#pragma unroll
                for (int dt = 0; dt < DT; ++dt)
#pragma unroll
                    for (int e = 0; e < 16; ++e) o[dt][e] *= corr;
                m = m_new;
            }
            float m_use = m == -INFINITY ? 0.f : m, sum = 0.f;
#pragma unroll
            for (int e = 0; e < 16; ++e) {
                sh[e] = da_exp2(fmaf(sh[e], a.scale_log2e, -m_use));
                sum += sh[e];
            }
            l += da_across_halves(sum, false);
            bf16x8_t pf[2];
#pragma unroll
            for (int u = 0; u < 2; ++u)
                pf[u] = __builtin_bit_cast(bf16x8_t, make_uint4(f32x2_to_bf16x2(sh[8 * u + 0], sh[8 * u + 1]), f32x2_to_bf16x2(sh[8 * u + 2], sh[8 * u + 3]),
                                                                f32x2_to_bf16x2(sh[8 * u + 4], sh[8 * u + 5]), f32x2_to_bf16x2(sh[8 * u + 6], sh[8 * u + 7])));
#pragma unroll
            for (int u = 0; u < 2; ++u)
#pragma unroll
                for (int dt = 0; dt < DT; ++dt) {
                    const bf16_t* vrow = sv + (dt * 32 + col) * L::V_ROW + half * 32 + 16 * u + 8 * h2;
                    o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, *(const uint4*)vrow), pf[u], o[dt], 0, 0, 0);
                }
        }
    }
    // The second map's outputs go to the first's waves: a lane of either holds the same rows and values.
    __syncthreads();                                    // the last page has been consumed: its LDS is free
    float* exchange = (float*)da_smem;                  // [part][DT * 16][64 lanes]
    float inv = 1.0f / l;
    if (map == 1 && wave_active) {
#pragma unroll
        for (int dt = 0; dt < DT; ++dt)
#pragma unroll
            for (int e = 0; e < 16; ++e) exchange[((part * DT + dt) * 16 + e) * 64 + lane] = o[dt][e] * inv;
    }
    __syncthreads();
    if (map == 1 || !row_ok) return;
    float ss = 0.f;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
        for (int e = 0; e < 16; ++e) {
            float v = o[dt][e] * inv - a.lambda * exchange[((part * DT + dt) * 16 + e) * 64 + lane];
            o[dt][e] = v;
            ss = fmaf(v, v, ss);
        }
    // (both lanes of a row are active or neither is; a row's values are spread over lanes col and col + 32)
    float f = a.out_scale / sqrtf((ss + __shfl_xor(ss, 32, 64)) / (float)a.dv + a.eps);
    bf16_t* orow = a.out + ((size_t)(tok0 + my_row) * a.heads + h) * a.dv;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
        for (int e4 = 0; e4 < 4; ++e4) {
            int d = dt * 32 + 8 * e4 + 4 * h2;
            if (d < a.dv)                               // (dv is a multiple of 4)
                *(uint2*)(orow + d) = make_uint2(f32x2_to_bf16x2(o[dt][4 * e4] * f, o[dt][4 * e4 + 1] * f),
                                                 f32x2_to_bf16x2(o[dt][4 * e4 + 2] * f, o[dt][4 * e4 + 3] * f));
        }
}

// ---- decode: one query token per sequence ------------------------------------------------------
// The projection's rows: [2 H d query columns in the order above | 2 G d key columns | G dv value columns], 32-bit sums or
// n_splits K pieces of them, added in order.
struct DiffProj {
    const float* qkv; int ld; int n_splits; long long split_stride;
    const float* cos_t; const float* sin_t; int rot;        // [T, rot / 2], or null
};

template <int DK, int DV, int AHEAD>
__global__ void __launch_bounds__(DA_THREADS)
diff_decode_kernel(DiffArgs a, DiffProj pj, int n_splits, float* __restrict__ part_o, float* __restrict__ part_ml) {
    constexpr int KD = DK / 32;      // matrix steps along d for the scores
    constexpr int DT = DV / 16;      // 16-row tiles of the output
    constexpr int WAVES = DA_THREADS / 64;
    extern __shared__ float da_sm_o[];                  // [WAVES][16][DV + 4]
    __shared__ float sm_m[WAVES][16], sm_l[WAVES][16];
    __shared__ __attribute__((aligned(16))) bf16_t sm_q[16 * DK];
    __shared__ __attribute__((aligned(16))) bf16_t sm_knew[2 * DK];
    __shared__ __attribute__((aligned(16))) bf16_t sm_vnew[DV];
    const int split = blockIdx.x, kvh = blockIdx.y, t = blockIdx.z;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int g = lane >> 4, col = lane & 15;
    const int group = a.heads / a.kv;
    const int* pages = a.block_table + (size_t)t * a.bt_width;
    const int len = a.token_pos[t] + 1, new_pos = len - 1;
    const int lo = a.window > 0 ? max(0, len - a.window) : 0;
    const int first_page = lo / DA_PAGE, last_page = new_pos / DA_PAGE;
    const int n_pages = last_page - first_page + 1;
    // split s takes the pages s, s + n_splits, ... of the visible ones
    const int my_pages = split < n_pages ? (n_pages - split + n_splits - 1) / n_splits : 0;
    const int n_pieces = my_pages * 2;                  // of 32 keys, taken by the waves in turn
    const bool owner = (last_page - first_page) % n_splits == split;        // appends the new keys and value

    uint4 kbuf[AHEAD][2][2][KD], vbuf[AHEAD][DT];
    auto request_piece = [&](int piece, uint4 (&kreg)[2][2][KD], uint4 (&vreg)[DT]) {
        int round = __builtin_amdgcn_readfirstlane(piece >> 1), half = piece & 1;
        int phys = pages[first_page + split + round * n_splits];
        const bf16_t* vbase = a.vcache + ((size_t)phys * a.kv + kvh) * a.dv * DA_PAGE + half * 32;
        // row r of score tile u is key 8 (r / 4) + 4 u + r % 4 of the piece: the 8 keys whose weights a lane holds after the
        // softmax are then consecutive, and its values for them are one 16-byte load
#pragma unroll
        for (int mp = 0; mp < 2; ++mp)
#pragma unroll
            for (int u = 0; u < 2; ++u) {
                const bf16_t* krow = a.kcache + (((size_t)phys * 2 * a.kv + 2 * kvh + mp) * DA_PAGE + half * 32 + 8 * (col >> 2) + 4 * u + (col & 3)) * a.d + g * 8;
#pragma unroll
                for (int kd = 0; kd < KD; ++kd) {
                    kreg[mp][u][kd] = make_uint4(0u, 0u, 0u, 0u);
                    if (kd * 32 + g * 8 < a.d) kreg[mp][u][kd] = *(const uint4*)(krow + kd * 32);
                }
            }
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) {
            vreg[dt] = make_uint4(0u, 0u, 0u, 0u);
            if (dt * 16 + col < a.dv) vreg[dt] = *(const uint4*)(vbase + (size_t)(dt * 16 + col) * DA_PAGE + g * 8);
        }
    };
    if (wave < n_pieces) request_piece(wave, kbuf[0], vbuf[0]);
    if (AHEAD == 2 && wave + WAVES < n_pieces) request_piece(wave + WAVES, kbuf[AHEAD - 1], vbuf[AHEAD - 1]);

    // Query heads, and in the owner the new keys and value, from the projection.
    {
        const float* tok = pj.qkv + (size_t)t * pj.ld;
        const int page_new = pages[last_page], in_page = new_pos % DA_PAGE;
        auto value = [&](int c) {
            float v = tok[c];
            for (int sp = 1; sp < pj.n_splits; ++sp) v += tok[sp * pj.split_stride + c];
            return v;
        };
        const int half = pj.cos_t ? pj.rot / 2 : 0;
        const int n_rows = 2 * group + (owner ? 2 : 0);
        for (int idx = tid; idx < n_rows * DK; idx += DA_THREADS) {
            int r = idx / DK, e = idx % DK;
            bool is_k = r >= 2 * group;
            int mp = is_k ? r - 2 * group : r / group, q_in = r - mp * group;
            int col0 = is_k ? 2 * a.heads * a.d + (2 * kvh + mp) * a.d : ((kvh * 2 + mp) * group + q_in) * a.d;
            float x = 0.f;
            if (e < a.d) {
                x = value(col0 + e);
                if (e < 2 * half) {
                    int i = e < half ? e : e - half;
                    float other = value(col0 + (e < half ? e + half : e - half));
                    float c = pj.cos_t[(size_t)t * half + i], sn = pj.sin_t[(size_t)t * half + i];
                    x = e < half ? x * c - other * sn : other * sn + x * c;
                }
            }
            bf16_t xb = f32_to_bf16(x);
            if (is_k) {
                sm_knew[mp * DK + e] = xb;
                if (e < a.d && page_new >= 0)
                    a.kcache[(((size_t)page_new * 2 * a.kv + 2 * kvh + mp) * DA_PAGE + in_page) * a.d + e] = xb;
            } else {
                sm_q[(mp * DA_MAX_GROUP + q_in) * DK + e] = xb;
            }
        }
        if (owner) {
            const int v0 = 2 * (a.heads + a.kv) * a.d + kvh * a.dv;
            for (int e = tid; e < DV; e += DA_THREADS) {
                bf16_t xb = f32_to_bf16(e < a.dv ? value(v0 + e) : 0.f);
                sm_vnew[e] = xb;
                if (e < a.dv && page_new >= 0) a.vcache[(((size_t)page_new * a.kv + kvh) * a.dv + e) * DA_PAGE + in_page] = xb;
            }
        }
        __syncthreads();
    }
    bf16x8_t qf[2][KD];              // a map's query operand is zero in the other map's columns
    {
        const int mine = col >> 3;
        const bool head_ok = (col & 7) < group;
#pragma unroll
        for (int mp = 0; mp < 2; ++mp)
#pragma unroll
            for (int kd = 0; kd < KD; ++kd) {
                uint4 v = make_uint4(0u, 0u, 0u, 0u);
                if (head_ok && mine == mp) v = *(const uint4*)(sm_q + col * DK + kd * 32 + g * 8);
                qf[mp][kd] = __builtin_bit_cast(bf16x8_t, v);
            }
    }
    float m = -INFINITY, l = 0.f;
    f32x4_t o[DT];
#pragma unroll
    for (int i = 0; i < DT; ++i) o[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    // keys [key0, key0 + 32) of which those in [from, to) count
    auto multiply_piece = [&](int key0, int from, int to, const uint4 (&kreg)[2][2][KD], const uint4 (&vreg)[DT]) {
        __builtin_amdgcn_sched_barrier(0);
        f32x4_t s[2];                // element i of s[u] is key 8 g + 4 u + i, column = map and head
#pragma unroll
        for (int u = 0; u < 2; ++u) {
            s[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int mp = 0; mp < 2; ++mp)
#pragma unroll
                for (int kd = 0; kd < KD; ++kd)
                    s[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, kreg[mp][u][kd]), qf[mp][kd], s[u], 0, 0, 0);
        }
        float mx = -INFINITY;
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                int key = key0 + g * 8 + u * 4 + i;
                float v = s[u][i] * a.scale_log2e;
                v = (key >= from && key < to) ? v : -INFINITY;
                s[u][i] = v;
                mx = fmaxf(mx, v);
            }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        float m_new = fmaxf(m, mx);
        float m_use = m_new == -INFINITY ? 0.f : m_new;
        float corr = da_exp2(m - m_use), sum = 0.f;
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                s[u][i] = da_exp2(s[u][i] - m_use);
                sum += s[u][i];
            }
        sum += __shfl_xor(sum, 16, 64);
        sum += __shfl_xor(sum, 32, 64);
        l = l * corr + sum;
        m = m_new;
        uint4 pv = make_uint4(f32x2_to_bf16x2(s[0][0], s[0][1]), f32x2_to_bf16x2(s[0][2], s[0][3]),
                              f32x2_to_bf16x2(s[1][0], s[1][1]), f32x2_to_bf16x2(s[1][2], s[1][3]));
        bf16x8_t pf = __builtin_bit_cast(bf16x8_t, pv);
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) {
            o[dt] = o[dt] * corr;
            o[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, vreg[dt]), pf, o[dt], 0, 0, 0);
        }
    };
    // (the new key is not yet in the cache where a block reads it: the owner multiplies it last, from LDS)
    const int cached = owner ? new_pos : len;
    auto key_of = [&](int piece) { return (first_page + split + (piece >> 1) * n_splits) * DA_PAGE + (piece & 1) * 32; };
    for (int piece = wave; piece < n_pieces; piece += WAVES * AHEAD) {
        multiply_piece(key_of(piece), lo, cached, kbuf[0], vbuf[0]);
        if (piece + WAVES * AHEAD < n_pieces) request_piece(piece + WAVES * AHEAD, kbuf[0], vbuf[0]);
        if (AHEAD == 2 && piece + WAVES < n_pieces) {
            multiply_piece(key_of(piece + WAVES), lo, cached, kbuf[AHEAD - 1], vbuf[AHEAD - 1]);
            if (piece + 3 * WAVES < n_pieces) request_piece(piece + 3 * WAVES, kbuf[AHEAD - 1], vbuf[AHEAD - 1]);
        }
    }
    if (owner && wave == n_pieces % WAVES) {            // the new key: row 0 of score tile 0
        bool krow = col == 0, vrow = g == 0;
#pragma unroll
        for (int mp = 0; mp < 2; ++mp)
#pragma unroll
            for (int u = 0; u < 2; ++u)
#pragma unroll
                for (int kd = 0; kd < KD; ++kd) {
                    kbuf[0][mp][u][kd] = make_uint4(0u, 0u, 0u, 0u);
                    if (krow && u == 0) kbuf[0][mp][u][kd] = *(const uint4*)(sm_knew + mp * DK + kd * 32 + g * 8);
                }
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) vbuf[0][dt] = make_uint4(vrow ? (uint32_t)sm_vnew[dt * 16 + col] : 0u, 0u, 0u, 0u);
        multiply_piece(new_pos, new_pos, new_pos + 1, kbuf[0], vbuf[0]);
    }
    // merge the waves in wave order; element i of o[dt] is value 16 dt + 4 g + i, column = map and head
    {
        float* mine = da_sm_o + ((size_t)wave * 16 + col) * (DV + 4);
#pragma unroll
        for (int dt = 0; dt < DT; ++dt)
#pragma unroll
            for (int i = 0; i < 4; ++i) mine[dt * 16 + g * 4 + i] = o[dt][i];
    }
    if (g == 0) {
        sm_m[wave][col] = m;
        sm_l[wave][col] = l;
    }
    __syncthreads();
    static_assert(WAVES == 4, "the waves' weights are the parts of one vector");
    auto merged = [&](int c, float& mm, float& ll) {
        mm = fmaxf(fmaxf(sm_m[0][c], sm_m[1][c]), fmaxf(sm_m[2][c], sm_m[3][c]));
        auto weight = [&](int w) { return sm_m[w][c] == -INFINITY ? 0.f : da_exp2(sm_m[w][c] - mm); };
        float4 wgt = make_float4(weight(0), weight(1), weight(2), weight(3));
        ll = sm_l[0][c] * wgt.x + sm_l[1][c] * wgt.y + sm_l[2][c] * wgt.z + sm_l[3][c] * wgt.w;
        return wgt;
    };
    auto merged_value = [&](int c, float4 wgt, int d) {
        const float* p = da_sm_o + (size_t)c * (DV + 4) + d;
        constexpr int next = 16 * (DV + 4);
        return p[0] * wgt.x + p[next] * wgt.y + p[2 * next] * wgt.z + p[3 * next] * wgt.w;
    };
    if (n_splits == 1) {
        for (int r = wave; r < group; r += WAVES) {
            float m1, m2, l1, l2, val[DV / 64], ss = 0.f;
            float4 w1 = merged(r, m1, l1), w2 = merged(DA_MAX_GROUP + r, m2, l2);
#pragma unroll
            for (int j = 0; j < DV / 64; ++j) {
                int d = lane + j * 64;
                val[j] = merged_value(r, w1, d) / l1 - a.lambda * (merged_value(DA_MAX_GROUP + r, w2, d) / l2);
                ss = fmaf(val[j], val[j], ss);          // (values beyond dv are zero)
            }
            float f = a.out_scale / sqrtf(wave_sum(ss) / (float)a.dv + a.eps);
            bf16_t* orow = a.out + ((size_t)t * a.heads + kvh * group + r) * a.dv;
#pragma unroll
            for (int j = 0; j < DV / 64; ++j)
                if (lane + j * 64 < a.dv) orow[lane + j * 64] = f32_to_bf16(val[j] * f);
        }
        return;
    }
    for (int r = wave; r < 2 * group; r += WAVES) {     // rows (map, head) of partial results
        float mm, ll;
        int c = (r / group) * DA_MAX_GROUP + r % group;
        float4 wgt = merged(c, mm, ll);
        size_t slot = (((size_t)t * a.kv + kvh) * 2 * group + r) * n_splits + split;
        for (int d = lane; d < a.dv; d += 64) part_o[slot * a.dv + d] = merged_value(c, wgt, d);
        if (lane == 0) {
            part_ml[slot * 2] = mm;
            part_ml[slot * 2 + 1] = ll;
        }
    }
}

// Merge of the splits in split order for both maps of a head, their combination and its norm.  grid (H, T); at most 64 splits.
__global__ void __launch_bounds__(DA_THREADS)
diff_decode_reduce_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml, DiffArgs a, int n_splits) {
    __shared__ float wgt[2][64];
    __shared__ float scratch[DA_THREADS / WAVE];
    int h = blockIdx.x, t = blockIdx.y, group = a.heads / a.kv, g = h / group;
    int lane = threadIdx.x & 63, d = threadIdx.x < a.dv ? threadIdx.x : 0;
    float map_out[2];
    size_t row[2];
    float first[2][4];
#pragma unroll
    for (int mp = 0; mp < 2; ++mp) {
        row[mp] = (((size_t)t * a.kv + g) * 2 + mp) * group + h % group;
        const float* po = part_o + row[mp] * n_splits * a.dv;
#pragma unroll
        for (int s = 0; s < 4; ++s) first[mp][s] = po[(size_t)min(s, n_splits - 1) * a.dv + d];
    }
    float inv_l[2];
#pragma unroll
    for (int mp = 0; mp < 2; ++mp) {
        const float* ml = part_ml + row[mp] * n_splits * 2;
        bool has = lane < n_splits;
        float ms = has ? ml[lane * 2] : -INFINITY, ls = has ? ml[lane * 2 + 1] : 0.f;
        float mm = wave_max(ms);
        float w = ms == -INFINITY ? 0.f : da_exp2(ms - mm);
        if (threadIdx.x < 64) wgt[mp][lane] = w;
        inv_l[mp] = 1.0f / wave_sum(ls * w);            // every wave computes the same sum
    }
    __syncthreads();
#pragma unroll
    for (int mp = 0; mp < 2; ++mp) {
        const float* po = part_o + row[mp] * n_splits * a.dv;
        float acc = 0.f;
#pragma unroll
        for (int s = 0; s < 4; ++s) acc += s < n_splits ? first[mp][s] * wgt[mp][s] : 0.f;
        for (int s0 = 4; s0 < n_splits; s0 += 8) {
            float more[8];
#pragma unroll
            for (int s = 0; s < 8; ++s) more[s] = po[(size_t)min(s0 + s, n_splits - 1) * a.dv + d];
#pragma unroll
            for (int s = 0; s < 8; ++s) acc += s0 + s < n_splits ? more[s] * wgt[mp][s0 + s] : 0.f;
        }
        map_out[mp] = acc * inv_l[mp];
    }
    float v = threadIdx.x < a.dv ? map_out[0] - a.lambda * map_out[1] : 0.f;
    float ss = wave_sum(v * v);
    if (lane == 0) scratch[threadIdx.x / WAVE] = ss;
    __syncthreads();
    float total = 0.f;
    for (int w = 0; w < (int)blockDim.x / WAVE; ++w) total += scratch[w];
    if (threadIdx.x < a.dv)
        a.out[((size_t)t * a.heads + h) * a.dv + threadIdx.x] = f32_to_bf16(v * (a.out_scale / sqrtf(total / (float)a.dv + a.eps)));
}

// ---- the plain path's last step ----------------------------------------------------------------
// maps [T, 2 H, dv] 32-bit in the order of the query rows -> out [T, H dv]; a wave per (token, head).
template <typename TO>
__global__ void __launch_bounds__(DA_THREADS)
diff_combine_kernel(const float* __restrict__ maps, TO* __restrict__ out, int n_tokens, int heads, int kv, int dv, float lambda, float out_scale,
                    float eps) {
    long long row = (long long)blockIdx.x * (DA_THREADS / WAVE) + threadIdx.x / WAVE;
    if (row >= (long long)n_tokens * heads) return;
    int lane = threadIdx.x & (WAVE - 1);
    long long t = row / heads;
    int h = (int)(row - t * heads), group = heads / kv, g = h / group, r = h - g * group;
    const float* a1 = maps + ((size_t)t * 2 * heads + (g * 2) * group + r) * dv;
    const float* a2 = a1 + (size_t)group * dv;
    float ss = 0.f;
    for (int d = lane; d < dv; d += WAVE) {
        float v = a1[d] - lambda * a2[d];
        ss = fmaf(v, v, ss);
    }
    float f = out_scale / sqrtf(wave_sum(ss) / (float)dv + eps);
    for (int d = lane; d < dv; d += WAVE) Elem<TO>::store(out + (size_t)row * dv + d, (a1[d] - lambda * a2[d]) * f);
}

// ---- launches ----------------------------------------------------------------------------------
template <typename K>
static int da_allow_lds(K kernel, int bytes) {
    hipError_t e = hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
    if (e != hipSuccess) return rocml_fail("diff_attention: cannot reserve %d bytes of LDS: %s", bytes, hipGetErrorString(e));
    return 0;
}

template <int DK, int DV>
static int launch_diff_prefill(const DiffArgs& a, int tiles, hipStream_t stream) {
    static bool ready = false;
    if (!ready) {
        if (da_allow_lds(diff_prefill_kernel<DK, DV>, DiffPrefillLds<DK, DV>::BYTES)) return 1;
        ready = true;
    }
    diff_prefill_kernel<DK, DV><<<tiles * a.heads, DA_THREADS, DiffPrefillLds<DK, DV>::BYTES, stream>>>(a);
    return 0;
}

template <int DK, int DV>
static int launch_diff_decode(const DiffArgs& a, const DiffProj& pj, int n_tokens, int n_splits, float* part_o, float* part_ml, hipStream_t stream) {
    constexpr int AHEAD = DK <= 64 && DV <= 128 ? 2 : 1;
    constexpr int LDS = DA_THREADS / 64 * 16 * (DV + 4) * 4;
    static bool ready = false;
    if (!ready) {
        if (da_allow_lds(diff_decode_kernel<DK, DV, AHEAD>, LDS)) return 1;
        ready = true;
    }
    diff_decode_kernel<DK, DV, AHEAD><<<dim3(n_splits, a.kv, n_tokens), DA_THREADS, LDS, stream>>>(a, pj, n_splits, part_o, part_ml);
    return 0;
}

// the instantiation for head sizes d and dv, rounded up
#define DA_BY_SIZES(fn, d_, dv_, ...)                                                                                           \
    ((d_) <= 32 ? ((dv_) <= 64 ? fn<32, 64>(__VA_ARGS__) : (dv_) <= 128 ? fn<32, 128>(__VA_ARGS__) : fn<32, 256>(__VA_ARGS__))  \
     : (d_) <= 64 ? ((dv_) <= 64 ? fn<64, 64>(__VA_ARGS__) : (dv_) <= 128 ? fn<64, 128>(__VA_ARGS__) : fn<64, 256>(__VA_ARGS__)) \
                  : ((dv_) <= 64 ? fn<128, 64>(__VA_ARGS__) : (dv_) <= 128 ? fn<128, 128>(__VA_ARGS__) : fn<128, 256>(__VA_ARGS__)))

static bool da_mfma_sizes(int d, int dv, int page_size) {
    return page_size == DA_PAGE && d % 8 == 0 && d <= 128 && dv % 4 == 0 && dv <= 256;
}

ROCML_EXPORT int rocml_diff_attention_sizes_ok(int d, int dv, int page_size) { return d > 0 && dv > 0 && da_mfma_sizes(d, dv, page_size) ? 1 : 0; }
ROCML_EXPORT int rocml_diff_attention_max_group() { return DA_MAX_GROUP; }

// Attention of a step whose keys and values are in the cache.  q [T, 2 H, d] in the order above; maps (32-bit [T, 2 H, dv], the plain
// path only); plain != 0: the plain path whatever the sizes.  q_counts (host): query tokens of each sequence.
ROCML_EXPORT int rocml_diff_attention(const void* q, void* out, const void* kcache, const void* vcache, int dtype, const int* block_table,
                                      int bt_width, const int* token_seq, const int* token_pos, int n_tokens, int heads, int kv, int d, int dv,
                                      int page_size, float scale, int window, float lambda, float out_scale, float eps, const int* cu_seqlens,
                                      int n_seqs, const int* q_counts, float* maps, int plain, hipStream_t stream) {
    ROCML_REQUIRE(n_tokens >= 0 && heads > 0 && kv > 0 && heads % kv == 0 && d > 0 && dv > 0 && page_size > 0 && bt_width > 0 && window >= 0,
                  "diff_attention: bad sizes T=%d heads=%d/%d d=%d dv=%d page=%d width=%d window=%d", n_tokens, heads, kv, d, dv, page_size,
                  bt_width, window);
    ROCML_REQUIRE(dtype == ROCML_F32 || dtype == ROCML_BF16, "diff_attention: unknown dtype code %d", dtype);
    ROCML_REQUIRE(scale > 0.f && eps > 0.f, "diff_attention: scale and eps must be positive");
    ROCML_REQUIRE(d <= AG_BLOCK * AG_MAX_D_PER_THREAD && dv <= AG_BLOCK * AG_MAX_D_PER_THREAD, "diff_attention: head sizes %d and %d exceed %d", d,
                  dv, AG_BLOCK * AG_MAX_D_PER_THREAD);
    ROCML_REQUIRE(q && out && kcache && vcache && block_table && token_seq && token_pos && cu_seqlens && q_counts && n_seqs > 0,
                  "diff_attention: missing arguments");
    long long tiles = 0, counted = 0;
    for (int b = 0; b < n_seqs; ++b) {
        ROCML_REQUIRE(q_counts[b] >= 0, "diff_attention: sequence %d has %d query tokens", b, q_counts[b]);
        tiles += (q_counts[b] + DA_QTILE - 1) / DA_QTILE;
        counted += q_counts[b];
    }
    ROCML_REQUIRE(counted == n_tokens && tiles * heads < (1ll << 31), "diff_attention: the sequences' query counts add up to %lld, the step has %d tokens",
                  counted, n_tokens);
    if (n_tokens == 0) return 0;
    if (!plain && dtype == ROCML_BF16 && da_mfma_sizes(d, dv, page_size)) {
        DiffArgs a{(const bf16_t*)q, (bf16_t*)out, (bf16_t*)const_cast<void*>(kcache), (bf16_t*)const_cast<void*>(vcache), block_table, bt_width,
                   token_pos, cu_seqlens, n_seqs, heads, kv, d, dv, scale * DA_LOG2E, window, lambda, out_scale, eps};
        int rc = DA_BY_SIZES(launch_diff_prefill, d, dv, a, (int)tiles, stream);
        if (rc) return rc;
        ROCML_CHECK_LAUNCH("diff_attention");
        return 0;
    }
    ROCML_REQUIRE(maps, "diff_attention: the plain path needs room for the maps' outputs");
    dim3 grid(n_tokens, 2 * heads);
    size_t lds = (size_t)(d + AG_BLOCK) * sizeof(float);
    AttnExtra ex{dv, 0, 0, nullptr, 0, nullptr, 0.f, 0, 2};
    int rows = ceil_div((long long)n_tokens * heads, DA_THREADS / WAVE);
    if (dtype == ROCML_F32) {
        attn_generic_kernel<float, float><<<grid, AG_BLOCK, lds, stream>>>((const float*)q, maps, (const float*)kcache, (const float*)vcache,
            block_table, bt_width, token_seq, token_pos, 2 * heads, 2 * kv, d, page_size, scale, window, ex);
        diff_combine_kernel<float><<<rows, DA_THREADS, 0, stream>>>(maps, (float*)out, n_tokens, heads, kv, dv, lambda, out_scale, eps);
    } else {
        attn_generic_kernel<bf16_t, float><<<grid, AG_BLOCK, lds, stream>>>((const bf16_t*)q, maps, (const bf16_t*)kcache, (const bf16_t*)vcache,
            block_table, bt_width, token_seq, token_pos, 2 * heads, 2 * kv, d, page_size, scale, window, ex);
        diff_combine_kernel<bf16_t><<<rows, DA_THREADS, 0, stream>>>(maps, (bf16_t*)out, n_tokens, heads, kv, dv, lambda, out_scale, eps);
    }
    ROCML_CHECK_LAUNCH("diff_attention");
    return 0;
}

// A decode step straight from the projection: rotation, append and attention in one launch (and the merge of the splits in a
// second).  Token t is the one token of the step's sequence t.
ROCML_EXPORT int rocml_diff_attention_decode(const float* qkv, int ld, int qkv_splits, long long qkv_split_stride, const float* cos_t,
                                             const float* sin_t, int rot, void* out, void* kcache, void* vcache, const int* block_table,
                                             int bt_width, const int* token_pos, int n_tokens, int heads, int kv, int d, int dv, int page_size,
                                             float scale, int window, float lambda, float out_scale, float eps, int n_splits, void* workspace,
                                             long long workspace_bytes, hipStream_t stream) {
    ROCML_REQUIRE(n_tokens >= 0 && heads > 0 && kv > 0 && heads % kv == 0 && heads / kv <= DA_MAX_GROUP && bt_width > 0 && window >= 0 && qkv_splits >= 1,
                  "diff_attention_decode: bad sizes T=%d heads=%d/%d width=%d splits=%d", n_tokens, heads, kv, bt_width, qkv_splits);
    ROCML_REQUIRE(d > 0 && dv > 0 && da_mfma_sizes(d, dv, page_size), "diff_attention_decode: head sizes %d and %d or pages of %d do not fit", d, dv, page_size);
    ROCML_REQUIRE(scale > 0.f && eps > 0.f, "diff_attention_decode: scale and eps must be positive");
    ROCML_REQUIRE(qkv && out && kcache && vcache && block_table && token_pos, "diff_attention_decode: missing arguments");
    ROCML_REQUIRE(ld >= 2 * (heads + kv) * d + kv * dv && (qkv_splits == 1 || qkv_split_stride >= (long long)n_tokens * ld),
                  "diff_attention_decode: projection rows of %d numbers are too short", ld);
    ROCML_REQUIRE((cos_t == nullptr) == (sin_t == nullptr) && (!cos_t || (rot > 0 && rot % 2 == 0 && rot <= d)),
                  "diff_attention_decode: %d of %d values of a head turn", rot, d);
    if (n_tokens == 0) return 0;
    if (n_splits > 64) n_splits = 64;
    if (n_splits < 1) n_splits = 1;
    long long per_split = (long long)n_tokens * 2 * heads * (dv + 2) * (long long)sizeof(float);
    if (n_splits > 1 && per_split * n_splits > workspace_bytes) n_splits = workspace ? (int)(workspace_bytes / per_split) : 1;
    if (n_splits < 1) n_splits = 1;
    float* part_o = (float*)workspace;
    float* part_ml = part_o ? part_o + (size_t)n_tokens * 2 * heads * n_splits * dv : nullptr;
    DiffArgs a{nullptr, (bf16_t*)out, (bf16_t*)kcache, (bf16_t*)vcache, block_table, bt_width, token_pos, nullptr, 0, heads, kv, d, dv,
               scale * DA_LOG2E, window, lambda, out_scale, eps};
    DiffProj pj{qkv, ld, qkv_splits, qkv_split_stride, cos_t, sin_t, rot};
    int rc = DA_BY_SIZES(launch_diff_decode, d, dv, a, pj, n_tokens, n_splits, part_o, part_ml, stream);
    if (rc) return rc;
    if (n_splits > 1)
        diff_decode_reduce_kernel<<<dim3(heads, n_tokens), (dv + 63) / 64 * 64, 0, stream>>>(part_o, part_ml, a, n_splits);
    ROCML_CHECK_LAUNCH("diff_attention_decode");
    return 0;
}
