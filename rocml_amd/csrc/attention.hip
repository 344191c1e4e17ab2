// Attention over the paged key/value cache for gfx950.  One entry point for any step: the
// query tokens of a step carry their sequence and position, keys and values are read from
// the cache (the step's own keys were appended before), so prefill, decode and any cut of a
// prompt run the same code.  bfloat16 with a head size that is a multiple of 32 runs on the
// matrix cores; everything else, and the whole 32-bit path, runs the plain kernel.
#include "common.h"
#include "attention_generic.h"
#include "attention_mfma.h"
#include "attention_latent.h"

ROCML_LAST_ERROR_FN(attention)

enum AttnAlgo : int { ATTN_AUTO = 0, ATTN_PLAIN = 1, ATTN_MFMA = 2 };

static const float LOG2E = 1.4426950408889634f;

template <typename K>
static int allow_lds(K kernel, int bytes) {
    hipError_t e = hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
    if (e != hipSuccess)
        return rocml_fail("attention: cannot reserve %d bytes of LDS: %s", bytes, hipGetErrorString(e));
    return 0;
}

struct AttnArgs {
    const bf16_t* q; bf16_t* out; const bf16_t* kcache; const bf16_t* vcache;
    const int* block_table; int bt_width; const int* token_seq; const int* token_pos;
    const int* cu_seqlens; int n_seqs; int n_tokens; int total_q_tiles; int max_len;
    int hq, hkv; float scale; int window; void* workspace; long long workspace_bytes;
    int n_splits_hint;
    const DecodeProj* proj;     // decode only: the step's q/k/v projection instead of q and an appended cache
    const PrefillProj* prefill_proj = nullptr;      // prompts: the projection instead of prepared queries
    MaskExtra extra = MaskExtra{};                  // blocks of positions, distance slopes, sink
    bool has_extra = false;
};

template <int D, bool FUSED, int AHEAD, int WAVES>
static int launch_decode_kernel(const AttnArgs& a, int n_splits, float* part_o, float* part_ml, hipStream_t stream) {
    int group = a.hq / a.hkv;
    int lds = WAVES * group * (D + 4) * (int)sizeof(float);
    dim3 grid(n_splits, a.hkv, a.n_tokens);
    if (a.has_extra) {
        static int allowed_extra = 0;
        if (lds > allowed_extra) {
            if (allow_lds(attn_decode_mfma_kernel<D, FUSED, AHEAD, WAVES, true>, lds)) return 1;
            allowed_extra = lds;
        }
        attn_decode_mfma_kernel<D, FUSED, AHEAD, WAVES, true><<<grid, 64 * WAVES, lds, stream>>>(
            a.q, a.out, const_cast<bf16_t*>(a.kcache), const_cast<bf16_t*>(a.vcache), a.block_table, a.bt_width,
            a.token_seq, a.token_pos, a.hq, a.hkv, a.scale * LOG2E, a.window, n_splits, part_o, part_ml,
            FUSED ? *a.proj : DecodeProj{}, a.extra);
        return 0;
    }
    static int allowed = 0;
    if (lds > allowed) {
        if (allow_lds(attn_decode_mfma_kernel<D, FUSED, AHEAD, WAVES>, lds)) return 1;
        allowed = lds;
    }
    attn_decode_mfma_kernel<D, FUSED, AHEAD, WAVES><<<grid, 64 * WAVES, lds, stream>>>(
        a.q, a.out, const_cast<bf16_t*>(a.kcache), const_cast<bf16_t*>(a.vcache), a.block_table, a.bt_width,
        a.token_seq, a.token_pos, a.hq, a.hkv, a.scale * LOG2E, a.window, n_splits, part_o, part_ml,
        FUSED ? *a.proj : DecodeProj{});
    return 0;
}

constexpr int WIDE_BLOCK_MIN_PIECES = 8;         // of a block: more than two a wave of four

template <int D, bool FUSED>
static int launch_decode(const AttnArgs& a, hipStream_t stream) {
    // Enough blocks to fill the chip, at most one split per page of the longest sequence.
    int n_splits = a.n_splits_hint;
    if (n_splits <= 0) {
        n_splits = 2 * cu_count() / (a.n_tokens * a.hkv);
        int max_pages = (a.max_len + AM_PAGE - 1) / AM_PAGE;
        if (n_splits > max_pages) n_splits = max_pages;
    }
    if (n_splits > 64) n_splits = 64;
    if (n_splits < 1) n_splits = 1;
    long long per_split = (long long)a.n_tokens * a.hq * (D + 2) * sizeof(float);
    if (n_splits > 1 && per_split * n_splits > a.workspace_bytes)
        n_splits = a.workspace ? (int)(a.workspace_bytes / per_split) : 1;
    if (n_splits < 1) n_splits = 1;
    float* part_o = (float*)a.workspace;
    float* part_ml = part_o ? part_o + (size_t)a.n_tokens * a.hq * n_splits * D : nullptr;
    // Many splits mean few pieces per block: then two of a wave's pieces travel at a time; so they
    // do when the chip holds at most one block a CU (a long loop then gains from it what a second
    // block would bring).  The choice follows the launch's shape, not the lengths, as the number of
    // splits does.
    // Eight waves a block where the chip holds at most one block a CU and a block of four waves
    // could give a wave more pieces than two trips bring (the pages the block table has room for,
    // two pieces each, over the splits and the waves: the launch's shape again, not the lengths).
    int rc;
    if constexpr (D <= 128) {
        bool one_a_cu = (long long)a.n_tokens * a.hkv * n_splits <= cu_count();
        long long pieces = 2ll * ((a.bt_width + n_splits - 1) / n_splits);
        if (one_a_cu && pieces > WIDE_BLOCK_MIN_PIECES)
            rc = launch_decode_kernel<D, FUSED, 2, 8>(a, n_splits, part_o, part_ml, stream);
        else
            rc = n_splits >= 4 || one_a_cu ? launch_decode_kernel<D, FUSED, 2, 4>(a, n_splits, part_o, part_ml, stream)
                                           : launch_decode_kernel<D, FUSED, 1, 4>(a, n_splits, part_o, part_ml, stream);
    } else {
        rc = launch_decode_kernel<D, FUSED, 1, 4>(a, n_splits, part_o, part_ml, stream);
    }
    if (rc) return rc;
    if (n_splits > 1)
        // whole waves: the kernel's reductions exchange values between all 64 lanes
        attn_decode_reduce_kernel<D><<<a.n_tokens * a.hq, (D + 63) / 64 * 64, 0, stream>>>(part_o, part_ml, a.out, n_splits);
    return 0;
}

template <int D> static int launch_decode_plain(const AttnArgs& a, hipStream_t s) { return launch_decode<D, false>(a, s); }
template <int D> static int launch_decode_fused(const AttnArgs& a, hipStream_t s) { return launch_decode<D, true>(a, s); }

template <int D>
static int launch_prefill(const AttnArgs& a, hipStream_t stream) {
    static bool ready = false;
    if (!ready) {
        if (allow_lds(attn_prefill_mfma_kernel<D, false>, PrefillLds<D>::BYTES)) return 1;
        if (allow_lds(attn_prefill_mfma_kernel<D, true>, PrefillLds<D>::BYTES)) return 1;
        if (allow_lds(attn_prefill_mfma_kernel<D, false, true>, PrefillLds<D>::BYTES)) return 1;
        ready = true;
    }
    dim3 grid(a.total_q_tiles * a.hq);
    if (a.has_extra)
        attn_prefill_mfma_kernel<D, false, true><<<grid, AM_THREADS, PrefillLds<D>::BYTES, stream>>>(
            a.q, a.out, a.kcache, a.vcache, a.block_table, a.bt_width, a.cu_seqlens, a.n_seqs, a.token_pos,
            a.hq, a.hkv, a.scale * LOG2E, a.window, PrefillProj{}, a.extra);
    else if (a.prefill_proj)
        attn_prefill_mfma_kernel<D, true><<<grid, AM_THREADS, PrefillLds<D>::BYTES, stream>>>(
            nullptr, a.out, a.kcache, a.vcache, a.block_table, a.bt_width, a.cu_seqlens, a.n_seqs, a.token_pos,
            a.hq, a.hkv, a.scale * LOG2E, a.window, *a.prefill_proj);
    else
        attn_prefill_mfma_kernel<D, false><<<grid, AM_THREADS, PrefillLds<D>::BYTES, stream>>>(
            a.q, a.out, a.kcache, a.vcache, a.block_table, a.bt_width, a.cu_seqlens, a.n_seqs, a.token_pos,
            a.hq, a.hkv, a.scale * LOG2E, a.window, PrefillProj{});
    return 0;
}

// Attention over latent rows (attention_latent.h): a block per 64 rows of work and key split.
struct LatentArgs {
    const bf16_t* q; bf16_t* out; const bf16_t* cache; const int* block_table; int bt_width;
    const int* cu_seqlens; int n_seqs; const int* token_pos; int n_tokens; int n_heads; int dk; int dv;
    float scale; int window; int tiles; void* workspace; long long workspace_bytes;
};

template <int KD, int DT, int RT>
static int launch_latent(const LatentArgs& a, hipStream_t stream) {
    using L = LatentLds<KD, DT>;
    static bool ready = false;
    if (!ready) {
        if (allow_lds(attn_latent_mfma_kernel<KD, DT, RT>, L::BYTES)) return 1;
        ready = true;
    }
    // Splits of the key range: enough blocks for one a CU, at most one per two pieces the rows can see
    // (a block's first piece costs it four trips to memory, a further one about one).
    // The choice follows the launch's shape (rows, window, width of the block table), not the lengths.
    int cus = cu_count();
    int pieces = a.window > 0 ? a.window / AL_KEYS + 2 : a.bt_width * (AM_PAGE / AL_KEYS);
    int n_splits = cus / a.tiles;
    if (n_splits > (pieces + 1) / 2) n_splits = (pieces + 1) / 2;
    if (n_splits > 64) n_splits = 64;
    long long rows = (long long)a.n_tokens * a.n_heads;
    long long per_split = rows * (a.dv + 2) * (long long)sizeof(float);
    if (n_splits > 1 && per_split * n_splits > a.workspace_bytes) n_splits = a.workspace ? (int)(a.workspace_bytes / per_split) : 1;
    if (n_splits < 1) n_splits = 1;
    float* part_o = (float*)a.workspace;
    float* part_ml = part_o ? part_o + rows * n_splits * a.dv : nullptr;
    attn_latent_mfma_kernel<KD, DT, RT><<<dim3(a.tiles, n_splits), 256, L::BYTES, stream>>>(
        a.q, a.out, a.cache, a.block_table, a.bt_width, a.cu_seqlens, a.n_seqs, a.token_pos, a.n_heads, a.dk, a.dv,
        a.scale * LOG2E, a.window, n_splits, part_o, part_ml);
    if (n_splits > 1)
        attn_latent_reduce_kernel<<<(unsigned)rows, a.dv > 256 ? 256 : a.dv > 128 ? 128 : 64, 0, stream>>>(part_o, part_ml, a.out, n_splits, a.dv);
    return 0;
}

static bool mfma_head_dim(int d) { return d == 32 || d == 64 || d == 96 || d == 128 || d == 192 || d == 256; }

#define BY_HEAD_DIM(fn, d, ...)                       \
    ((d) == 32 ? fn<32>(__VA_ARGS__)                  \
     : (d) == 64 ? fn<64>(__VA_ARGS__)                \
     : (d) == 96 ? fn<96>(__VA_ARGS__)                \
     : (d) == 128 ? fn<128>(__VA_ARGS__)              \
     : (d) == 192 ? fn<192>(__VA_ARGS__) : fn<256>(__VA_ARGS__))

// algo: 0 = choose, 1 = plain kernel, 2 = MFMA kernels (error if they cannot take the shapes).
// cu_seqlens [n_seqs + 1] gives where each sequence's query tokens start (tokens of a sequence
// are consecutive and in position order) and q_counts, an array in host memory, how many each has
// (the prefill kernel's grid is sized from it); max_new is the most query tokens of any
// sequence, max_len the longest context.
// workspace holds the partial results of split decode attention.
ROCML_EXPORT int rocml_attention(const void* q, void* out, const void* kcache, const void* vcache,
                                 int dtype, const int* block_table, int bt_width,
                                 const int* token_seq, const int* token_pos, int n_tokens, int hq,
                                 int hkv, int d, int page_size, float scale, int window, int algo,
                                 const int* cu_seqlens, int n_seqs, int max_new, const int* q_counts,
                                 int max_len, int n_splits, void* workspace, long long workspace_bytes,
                                 int dv, int v_in_k, int chunk, const float* slopes, int sink,
                                 const float* sinks, float softcap, int keep_first, hipStream_t stream) {
    // dv (0: the key head's size), v_in_k, chunk, slopes, sink, sinks, softcap and keep_first: see AttnExtra in attention_generic.h.
    ROCML_REQUIRE(!sinks || sink, "attention: learned sinks need the sink switched on");
    ROCML_REQUIRE(softcap >= 0.f, "attention: negative soft cap %g", (double)softcap);
    if (dv <= 0) dv = d;
    ROCML_REQUIRE(chunk >= 0 && (chunk == 0 || window == 0), "attention: a layer has a window or blocks of positions, not both");
    ROCML_REQUIRE(!v_in_k || dv <= d, "attention: values taken from the key rows need dv <= d (dv=%d d=%d)", dv, d);
    ROCML_REQUIRE(v_in_k || vcache, "attention: no value cache");
    ROCML_REQUIRE(dv <= AG_BLOCK * AG_MAX_D_PER_THREAD, "attention: value head size %d exceeds %d", dv,
                  AG_BLOCK * AG_MAX_D_PER_THREAD);
    bool plain_features = dv == d && !v_in_k;          // what the matrix-core kernels need
    ROCML_REQUIRE(keep_first >= 0, "attention: %d kept first positions", keep_first);
    if (window == 0) keep_first = 0;                   // (everything is seen anyway)
    ROCML_REQUIRE(keep_first == 0 || chunk == 0, "attention: kept first positions go with a window");
    bool has_extra = chunk > 0 || slopes || sink || softcap > 0.f || keep_first > 0;
    ROCML_REQUIRE(n_tokens >= 0 && hq > 0 && hkv > 0 && d > 0 && page_size > 0 && bt_width > 0,
                  "attention: bad sizes T=%d Hq=%d Hkv=%d D=%d page=%d width=%d", n_tokens, hq, hkv,
                  d, page_size, bt_width);
    ROCML_REQUIRE(hq % hkv == 0, "attention: %d query heads are not a multiple of %d kv heads", hq, hkv);
    ROCML_REQUIRE(window >= 0, "attention: negative window %d", window);
    ROCML_REQUIRE(d <= AG_BLOCK * AG_MAX_D_PER_THREAD, "attention: head_dim %d exceeds %d", d,
                  AG_BLOCK * AG_MAX_D_PER_THREAD);
    ROCML_REQUIRE(algo >= ATTN_AUTO && algo <= ATTN_MFMA, "attention: unknown algorithm %d", algo);
    if (n_tokens == 0) return 0;
    bool decode = max_new == 1;
    long long total_q_tiles = 0, counted = 0;
    if (q_counts && n_seqs > 0)
        for (int b = 0; b < n_seqs; ++b) {
            ROCML_REQUIRE(q_counts[b] >= 0, "attention: sequence %d has %d query tokens", b, q_counts[b]);
            total_q_tiles += (q_counts[b] + AM_QTILE - 1) / AM_QTILE;
            counted += q_counts[b];
        }
    ROCML_REQUIRE(!q_counts || n_seqs <= 0 || counted == n_tokens,
                  "attention: the sequences' query counts add up to %lld, the step has %d tokens", counted, n_tokens);
    ROCML_REQUIRE(total_q_tiles * hq < (1ll << 31), "attention: too many query tiles");
    bool mfma_ok = plain_features && dtype == ROCML_BF16 && page_size == AM_PAGE && mfma_head_dim(d) && max_new >= 1 &&
                   (decode ? hq / hkv <= 16 : (cu_seqlens != nullptr && n_seqs > 0 && total_q_tiles > 0));
    if (algo == ATTN_MFMA && !v_in_k)
        ROCML_REQUIRE(mfma_ok, "attention: the MFMA kernels need bfloat16, pages of 64 positions, a head size "
                               "of 32, 64, 96, 128, 192 or 256, at most 16 query heads per kv head in decode and "
                               "the sequence offsets in prefill (D=%d page=%d group=%d)", d, page_size, hq / hkv);
    // one shared key/value head whose values lie in its key rows: the kernel for latent rows
    bool latent_ok = v_in_k && !has_extra && dtype == ROCML_BF16 && page_size == AM_PAGE && hkv == 1 && d % 8 == 0 &&
                     dv % 8 == 0 && d <= 576 && dv <= 512 && max_new >= 1 && cu_seqlens && n_seqs > 0 && q_counts;
    if (algo == ATTN_MFMA && v_in_k)
        ROCML_REQUIRE(latent_ok, "attention: the matrix-core kernel for values in the key rows needs bfloat16, pages of 64, one "
                                 "key/value head, sizes that are multiples of 8 up to 576 and 512, and the sequence offsets "
                                 "(D=%d Dv=%d Hkv=%d)", d, dv, hkv);
    if (latent_ok && algo != ATTN_PLAIN) {
        // two tiles of rows a wave where the sequences bring at least 128 rows each on average (prompts)
        // and the sizes leave the registers for it
        int kd = (d + 31) / 32, dt = (dv + 15) / 16;
        int rt = (long long)n_tokens * hq >= 128ll * n_seqs && kd <= 10 && dt <= 16 ? 2 : 1;
        long long tiles = 0;
        for (int b = 0; b < n_seqs; ++b) tiles += ((long long)q_counts[b] * hq + AL_ROWS * rt - 1) / (AL_ROWS * rt);
        ROCML_REQUIRE(tiles > 0 && tiles < (1ll << 31), "attention: %lld row tiles", tiles);
        LatentArgs a{(const bf16_t*)q, (bf16_t*)out, (const bf16_t*)kcache, block_table, bt_width, cu_seqlens, n_seqs,
                     token_pos, n_tokens, hq, d, dv, scale, window, (int)tiles, workspace, workspace_bytes};
#define BY_ROW_TILES(KD_, DT_) (rt == 2 ? launch_latent<KD_, DT_, 2>(a, stream) : launch_latent<KD_, DT_, 1>(a, stream))
        int rc = kd <= 3 && dt <= 4     ? BY_ROW_TILES(3, 4)
                 : kd <= 6 && dt <= 8   ? BY_ROW_TILES(6, 8)
                 : kd <= 10 && dt <= 16 ? BY_ROW_TILES(10, 16)
                                        : launch_latent<18, 32, 1>(a, stream);
#undef BY_ROW_TILES
        if (rc) return rc;
        ROCML_CHECK_LAUNCH("attention over latent rows");
        return 0;
    }
    if (mfma_ok && algo != ATTN_PLAIN) {
        AttnArgs a{(const bf16_t*)q, (bf16_t*)out, (const bf16_t*)kcache, (const bf16_t*)vcache, block_table,
                   bt_width, token_seq, token_pos, cu_seqlens, n_seqs, n_tokens, (int)total_q_tiles, max_len, hq, hkv,
                   scale, window, workspace, workspace_bytes, n_splits, nullptr};
        a.extra = MaskExtra{chunk, slopes, sink, sinks, softcap, keep_first};
        a.has_extra = has_extra;
        int rc = decode ? BY_HEAD_DIM(launch_decode_plain, d, a, stream) : BY_HEAD_DIM(launch_prefill, d, a, stream);
        if (rc) return rc;
        ROCML_CHECK_LAUNCH("attention");
        return 0;
    }
    dim3 grid(n_tokens, hq);
    size_t lds = (size_t)(d + AG_BLOCK) * sizeof(float);
    AttnExtra ex{dv, v_in_k, chunk, slopes, sink, sinks, softcap, keep_first};
    if (dtype == ROCML_F32)
        attn_generic_kernel<float><<<grid, AG_BLOCK, lds, stream>>>(
            (const float*)q, (float*)out, (const float*)kcache, (const float*)vcache, block_table,
            bt_width, token_seq, token_pos, hq, hkv, d, page_size, scale, window, ex);
    else if (dtype == ROCML_BF16)
        attn_generic_kernel<bf16_t><<<grid, AG_BLOCK, lds, stream>>>(
            (const bf16_t*)q, (bf16_t*)out, (const bf16_t*)kcache, (const bf16_t*)vcache, block_table,
            bt_width, token_seq, token_pos, hq, hkv, d, page_size, scale, window, ex);
    else
        return rocml_fail("attention: unknown dtype code %d", dtype);
    ROCML_CHECK_LAUNCH("attention");
    return 0;
}

// A decode step's attention straight from the q/k/v projection: per-head norm, rotation, append
// to the cache and attention in one launch (and the merge of the splits in a second), instead of
// a kernel for the first three and rocml_attention for the rest.  One token per sequence;
// bfloat16 cache with pages of 64 positions; a head size of 64, 128, 192 or 256; at most 16
// query heads per kv head.  qkv is the projection's 32-bit output [tokens, ld] with q, k and v
// side by side (k and v are not read when write_kv is 0: the cache then holds this step's row
// already), or its split-K partial sums [qkv_splits][tokens][ld], which are added in split
// order.  q_gain/k_gain null: no norm; cos/sin null: no rotation, else [tokens, D/2].
// token_seq null: token t is the one token of the step's sequence t (row t of the block table).
// row_ssq (may be null): the projection's operand lacked its norm's scale (see DecodeProj).
ROCML_EXPORT int rocml_attention_decode_fused(const float* qkv, int ld, int qkv_splits, long long qkv_split_stride,
                                              const float* q_gain, const float* k_gain, float eps,
                                              const float* cos_t, const float* sin_t, int write_kv, void* out,
                                              void* kcache, void* vcache, const int* block_table, int bt_width,
                                              const int* token_seq, const int* token_pos, int n_tokens, int hq,
                                              int hkv, int d, int page_size, float scale, int window,
                                              int max_len, int n_splits, void* workspace,
                                              long long workspace_bytes, const float* row_ssq, int row_parts,
                                              float row_eps, int row_width, const float* bias, int chunk,
                                              const float* slopes, int sink, const float* sinks, int keep_first, int rot,
                                              int v_is_k, hipStream_t stream) {
    // bias (may be null): [ld] numbers added to the projection's sums; chunk, slopes, sink, sinks, keep_first: see
    // MaskExtra.  rot: leading values of a head that turn (with tables [tokens, rot/2]; D or 0: all of them).  v_is_k:
    // the rows hold no value columns, a value is the projected key.
    if (rot <= 0) rot = d;
    ROCML_REQUIRE(rot <= d && rot % 2 == 0, "fused decode attention: %d of %d values of a head turn", rot, d);
    ROCML_REQUIRE(keep_first >= 0 && (keep_first == 0 || chunk == 0), "fused decode attention: kept first positions go with a window");
    ROCML_REQUIRE(!sinks || sink, "fused decode attention: learned sinks need the sink switched on");
    if (window == 0) keep_first = 0;
    ROCML_REQUIRE(chunk >= 0 && (chunk == 0 || window == 0), "fused decode attention: a window or blocks of positions, not both");
    ROCML_REQUIRE(n_tokens >= 0 && hq > 0 && hkv > 0 && bt_width > 0 && qkv_splits >= 1,
                  "fused decode attention: bad sizes T=%d Hq=%d Hkv=%d width=%d splits=%d", n_tokens, hq, hkv,
                  bt_width, qkv_splits);
    ROCML_REQUIRE(hq % hkv == 0 && hq / hkv <= 16,
                  "fused decode attention: %d query heads over %d kv heads (at most 16 per kv head)", hq, hkv);
    ROCML_REQUIRE(page_size == AM_PAGE && (d == 64 || d == 128 || d == 192 || d == 256),
                  "fused decode attention: needs pages of 64 positions and a head size of 64, 128, 192 or 256 "
                  "(page=%d D=%d)", page_size, d);
    ROCML_REQUIRE(window >= 0, "fused decode attention: negative window %d", window);
    int rows = write_kv ? hq + (v_is_k ? 1 : 2) * hkv : hq;
    ROCML_REQUIRE(ld >= rows * d && ld % 4 == 0 && ((uintptr_t)qkv & 15) == 0 &&
                      (qkv_splits == 1 || (qkv_split_stride >= (long long)n_tokens * ld && qkv_split_stride % 4 == 0)),
                  "fused decode attention: projection rows of %d values (need %d, a multiple of 4, 16-byte aligned), "
                  "split stride %lld", ld, rows * d, qkv_split_stride);
    ROCML_REQUIRE((q_gain == nullptr) == (k_gain == nullptr) && (cos_t == nullptr) == (sin_t == nullptr),
                  "fused decode attention: gains and rotation tables come in pairs");
    if (n_tokens == 0) return 0;
    ROCML_REQUIRE(!row_ssq || (row_parts > 0 && row_eps > 0.f && row_width > 0),
                  "fused decode attention: a row scale needs parts, eps and the norm's width");
    DecodeProj pj{qkv, ld, qkv_splits, qkv_split_stride, q_gain, k_gain, eps, cos_t, sin_t, write_kv,
                  row_ssq, row_parts, row_eps, row_ssq ? 1.0f / (float)row_width : 0.f, bias, rot, v_is_k};
    AttnArgs a{nullptr, (bf16_t*)out, (const bf16_t*)kcache, (const bf16_t*)vcache, block_table, bt_width,
               token_seq, token_pos, nullptr, 0, n_tokens, 0, max_len, hq, hkv, scale, window, workspace,
               workspace_bytes, n_splits, &pj};
    a.extra = MaskExtra{chunk, slopes, sink, sinks, 0.f, keep_first};
    // (the bias, a rotation of a part of the head and values taken from the keys ride in the same instantiation)
    a.has_extra = chunk > 0 || slopes || sink || bias || keep_first > 0 || rot != d || v_is_k;
    int rc = d == 64 ? launch_decode_fused<64>(a, stream)
             : d == 128 ? launch_decode_fused<128>(a, stream)
             : d == 192 ? launch_decode_fused<192>(a, stream) : launch_decode_fused<256>(a, stream);
    if (rc) return rc;
    ROCML_CHECK_LAUNCH("fused decode attention");
    return 0;
}

// Prompts: attention of a step's new tokens over the cache, with the queries taken from the step's
// q/k/v projection (32-bit, complete sums: a token's q heads first) and prepared by the kernel
// itself: per-head norm (q_gain null: none), rotation of the whole head with pairs (e, e + D/2)
// (cos/sin null: none, else [tokens, D/2]), rounding to bfloat16.  The keys and values of the new
// tokens are in the cache already.  bfloat16 caches with pages of 64 positions and the MFMA
// kernels' head sizes; cu_seqlens, q_counts as in rocml_attention.
ROCML_EXPORT int rocml_attention_prefill_fused(const float* qkv, int ld, const float* q_gain, float eps,
                                               const float* cos_t, const float* sin_t, void* out,
                                               const void* kcache, const void* vcache, const int* block_table,
                                               int bt_width, const int* token_pos, int n_tokens, int hq, int hkv,
                                               int d, int page_size, float scale, int window,
                                               const int* cu_seqlens, int n_seqs, const int* q_counts,
                                               hipStream_t stream) {
    ROCML_REQUIRE(n_tokens >= 0 && hq > 0 && hkv > 0 && bt_width > 0 && n_seqs > 0 && cu_seqlens && q_counts,
                  "fused prefill attention: bad sizes T=%d Hq=%d Hkv=%d width=%d sequences=%d", n_tokens, hq, hkv,
                  bt_width, n_seqs);
    ROCML_REQUIRE(hq % hkv == 0, "fused prefill attention: %d query heads are not a multiple of %d kv heads", hq, hkv);
    ROCML_REQUIRE(page_size == AM_PAGE && mfma_head_dim(d),
                  "fused prefill attention: needs pages of 64 positions and a head size of 32, 64, 96, 128, 192 or 256 "
                  "(page=%d D=%d)", page_size, d);
    ROCML_REQUIRE(window >= 0, "fused prefill attention: negative window %d", window);
    ROCML_REQUIRE(ld >= hq * d && ld % 4 == 0 && ((uintptr_t)qkv & 15) == 0,
                  "fused prefill attention: projection rows of %d values (need %d, a multiple of 4, 16-byte aligned)",
                  ld, hq * d);
    ROCML_REQUIRE((cos_t == nullptr) == (sin_t == nullptr), "fused prefill attention: rotation tables come in pairs");
    ROCML_REQUIRE(!q_gain || ((uintptr_t)q_gain & 15) == 0, "fused prefill attention: the gain must be 16-byte aligned");
    ROCML_REQUIRE(!cos_t || ((((uintptr_t)cos_t | (uintptr_t)sin_t) & 15) == 0),
                  "fused prefill attention: the rotation tables must be 16-byte aligned");
    if (n_tokens == 0) return 0;
    long long total_q_tiles = 0, counted = 0;
    for (int b = 0; b < n_seqs; ++b) {
        ROCML_REQUIRE(q_counts[b] >= 0, "fused prefill attention: sequence %d has %d query tokens", b, q_counts[b]);
        total_q_tiles += (q_counts[b] + AM_QTILE - 1) / AM_QTILE;
        counted += q_counts[b];
    }
    ROCML_REQUIRE(counted == n_tokens, "fused prefill attention: the sequences' query counts add up to %lld, the step has %d tokens",
                  counted, n_tokens);
    ROCML_REQUIRE(total_q_tiles > 0 && total_q_tiles * hq < (1ll << 31), "fused prefill attention: %lld query tiles", total_q_tiles);
    PrefillProj pj{qkv, ld, q_gain, eps, cos_t, sin_t};
    AttnArgs a{nullptr, (bf16_t*)out, (const bf16_t*)kcache, (const bf16_t*)vcache, block_table, bt_width,
               nullptr, token_pos, cu_seqlens, n_seqs, n_tokens, (int)total_q_tiles, 0, hq, hkv, scale, window, nullptr,
               0, 0, nullptr};
    a.prefill_proj = &pj;
    int rc = BY_HEAD_DIM(launch_prefill, d, a, stream);
    if (rc) return rc;
    ROCML_CHECK_LAUNCH("fused prefill attention");
    return 0;
}
