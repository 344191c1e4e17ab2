// A residual path of several streams (gfx950, wave64): what a sublayer reads is a weighted sum of the streams, and behind it
// every stream is formed anew from all the old ones and the sublayer's output.  All 32-bit.
//
// One kernel does everything that lies between two sublayers in one pass over a token's row:
//     y      the sublayer's output (a product's K pieces are added here, in split order),
//     new_t  = sum_s mix[s][t] x_s + w_out[t] y            (without y: new_t = x_t),
//     total  = sum_t new_t                                   (where the streams end), and
//     normed = rms(sum_t w_in[t] new_t) * gain              (what the next sublayer reads, in the compute type).
// Streams lie token by token, [T, S, n].  A source of one stream ([T, n], src_stride 0) stands for S equal ones: how the
// streams begin.  The new streams may be written over the old ones (a thread reads and writes the same columns of all
// streams).
#include "common.h"

ROCML_LAST_ERROR_FN(streams)

constexpr int SM_MAX = 16;           // streams
constexpr int SM_BLOCK = 1024;       // most threads of a block

struct StreamArgs {
    const float* src; long long src_row; long long src_stride;      // numbers between tokens and between streams
    const float* y; const float* partials; int n_splits; long long split_stride; int replace;
    const float* mix; const float* w_out;                           // [S][S] from, to; [S]
    float* dst;                                                     // [T, S, n] or null
    float* total;                                                   // [T, n] or null
    const float* w_in; const float* gain; float eps; void* normed;  // normed null: no read of the new streams
    int n; int n_streams;
};

__device__ __forceinline__ float sm_block_sum(float v, float* scratch) {
    v = wave_sum(v);
    int waves = (blockDim.x + WAVE - 1) / WAVE;
    if ((threadIdx.x & (WAVE - 1)) == 0) scratch[threadIdx.x / WAVE] = v;
    __syncthreads();
    float r = 0.f;
    for (int w = 0; w < waves; ++w) r += scratch[w];
    return r;
}

__device__ __forceinline__ void sm_store4(float* p, float4 v) { *(float4*)p = v; }
__device__ __forceinline__ void sm_store4(bf16_t* p, float4 v) { *(uint2*)p = make_uint2(f32x2_to_bf16x2(v.x, v.y), f32x2_to_bf16x2(v.z, v.w)); }

__device__ __forceinline__ void sm_fma(float4& a, float w, float4 v) {
    a.x = fmaf(w, v.x, a.x); a.y = fmaf(w, v.y, a.y); a.z = fmaf(w, v.z, a.z); a.w = fmaf(w, v.w, a.w);
}

// Rows that are whole 16-byte pieces, NV pieces a thread; exactly S streams.  UPDATE: there is a sublayer's output to add.
template <typename TO, int S, int NV, bool UPDATE>
__global__ void __launch_bounds__(SM_BLOCK)
stream_links_vec_kernel(StreamArgs a) {
    __shared__ float scratch[SM_BLOCK / WAVE];
    const int nv = a.n / 4;
    const size_t row = blockIdx.x;
    const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
    const float* src = a.src + row * a.src_row;
    float4 u[NV], gain[NV];
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        int i = threadIdx.x + j * blockDim.x;
        u[j] = zero;
        gain[j] = zero;
        if (i >= nv) continue;
        float4 x[S];
#pragma unroll
        for (int s = 0; s < S; ++s) x[s] = *(const float4*)(src + s * a.src_stride + 4 * i);
        if (a.normed) gain[j] = *(const float4*)(a.gain + 4 * i);
        if constexpr (UPDATE) {
            float4 y = zero;
            if (!a.replace) y = *(const float4*)(a.y + row * a.n + 4 * i);
            for (int sp = 0; sp < a.n_splits; sp += 4) {          // (four pieces' loads on their way at a time, added in order)
                float4 p0, p1, p2, p3;
                const float* base = a.partials + row * a.n + 4 * i;
                p0 = *(const float4*)(base + sp * a.split_stride);
                p1 = *(const float4*)(base + min(sp + 1, a.n_splits - 1) * a.split_stride);
                p2 = *(const float4*)(base + min(sp + 2, a.n_splits - 1) * a.split_stride);
                p3 = *(const float4*)(base + min(sp + 3, a.n_splits - 1) * a.split_stride);
                sm_fma(y, 1.f, p0);
                if (sp + 1 < a.n_splits) sm_fma(y, 1.f, p1);
                if (sp + 2 < a.n_splits) sm_fma(y, 1.f, p2);
                if (sp + 3 < a.n_splits) sm_fma(y, 1.f, p3);
            }
            float4 out[S];
#pragma unroll
            for (int t = 0; t < S; ++t) {
                out[t] = zero;
#pragma unroll
                for (int s = 0; s < S; ++s) sm_fma(out[t], a.mix[s * S + t], x[s]);
                sm_fma(out[t], a.w_out[t], y);
            }
#pragma unroll
            for (int t = 0; t < S; ++t) x[t] = out[t];
        }
        if (a.dst) {
#pragma unroll
            for (int t = 0; t < S; ++t) *(float4*)(a.dst + (row * S + t) * a.n + 4 * i) = x[t];
        }
        if (a.total) {
            float4 v = zero;
#pragma unroll
            for (int t = 0; t < S; ++t) { v.x += x[t].x; v.y += x[t].y; v.z += x[t].z; v.w += x[t].w; }
            *(float4*)(a.total + row * a.n + 4 * i) = v;
        }
        if (a.normed) {
#pragma unroll
            for (int t = 0; t < S; ++t) sm_fma(u[j], a.w_in[t], x[t]);
            ss = fmaf(u[j].x, u[j].x, fmaf(u[j].y, u[j].y, fmaf(u[j].z, u[j].z, fmaf(u[j].w, u[j].w, ss))));
        }
    }
    if (!a.normed) return;
    float inv = 1.0f / sqrtf(sm_block_sum(ss, scratch) / (float)a.n + a.eps);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        int i = threadIdx.x + j * blockDim.x;
        if (i < nv)
            sm_store4((TO*)a.normed + row * a.n + 4 * i, make_float4(u[j].x * inv * gain[j].x, u[j].y * inv * gain[j].y,
                                                                     u[j].z * inv * gain[j].z, u[j].w * inv * gain[j].w));
    }
}

// Any width and up to SM_MAX streams: the sublayer's input is formed twice, the second time from what this thread stored
// (or from the source where nothing is updated).
template <typename TO>
__global__ void __launch_bounds__(256)
stream_links_kernel(StreamArgs a) {
    __shared__ float scratch[SM_BLOCK / WAVE];
    const size_t row = blockIdx.x;
    const int S = a.n_streams;
    const float* src = a.src + row * a.src_row;
    const bool update = a.mix != nullptr;
    float ss = 0.f;
    for (int i = threadIdx.x; i < a.n; i += blockDim.x) {
        float x[SM_MAX];
#pragma unroll
        for (int s = 0; s < SM_MAX; ++s) x[s] = s < S ? src[s * a.src_stride + i] : 0.f;
        float y = 0.f;
        if (update) {
            y = a.replace ? 0.f : a.y[row * a.n + i];
            for (int sp = 0; sp < a.n_splits; ++sp) y += a.partials[sp * a.split_stride + row * a.n + i];
        }
        float u = 0.f, sum = 0.f;
        for (int t = 0; t < S; ++t) {
            float v = 0.f;
            if (update) {
#pragma unroll
                for (int s = 0; s < SM_MAX; ++s)
                    if (s < S) v = fmaf(a.mix[s * S + t], x[s], v);
                v = fmaf(a.w_out[t], y, v);
            } else {
                v = src[t * a.src_stride + i];
            }
            if (a.dst) a.dst[(row * S + t) * a.n + i] = v;
            sum += v;
            if (a.normed) u = fmaf(a.w_in[t], v, u);
        }
        if (a.total) a.total[row * a.n + i] = sum;
        ss = fmaf(u, u, ss);
    }
    if (!a.normed) return;
    float inv = 1.0f / sqrtf(sm_block_sum(ss, scratch) / (float)a.n + a.eps);
    const float* again = update ? a.dst + row * S * a.n : src;
    const long long stride = update ? a.n : a.src_stride;
    for (int i = threadIdx.x; i < a.n; i += blockDim.x) {
        float u = 0.f;
        for (int t = 0; t < S; ++t) u = fmaf(a.w_in[t], again[t * stride + i], u);
        Elem<TO>::store((TO*)a.normed + row * a.n + i, u * inv * a.gain[i]);
    }
}

template <typename TO, int S, bool UPDATE>
static void launch_stream_links_vec(const StreamArgs& a, int rows, hipStream_t stream) {
    int nv = a.n / 4;
    int per = ceil_div(nv, SM_BLOCK);
    int pieces = per <= 1 ? 1 : per <= 2 ? 2 : 4;
    int threads = ceil_div(ceil_div(nv, pieces), WAVE) * WAVE;
    if (pieces == 1) stream_links_vec_kernel<TO, S, 1, UPDATE><<<rows, threads, 0, stream>>>(a);
    else if (pieces == 2) stream_links_vec_kernel<TO, S, 2, UPDATE><<<rows, threads, 0, stream>>>(a);
    else stream_links_vec_kernel<TO, S, 4, UPDATE><<<rows, threads, 0, stream>>>(a);
}

template <typename TO, int S>
static void launch_stream_links(const StreamArgs& a, int rows, hipStream_t stream) {
    if (a.mix) launch_stream_links_vec<TO, S, true>(a, rows, stream);
    else launch_stream_links_vec<TO, S, false>(a, rows, stream);
}

template <typename TO>
static void launch_stream_links_any(const StreamArgs& a, int rows, bool vec, hipStream_t stream) {
    if (!vec || a.n_streams > 4) stream_links_kernel<TO><<<rows, 256, 0, stream>>>(a);
    else if (a.n_streams == 1) launch_stream_links<TO, 1>(a, rows, stream);
    else if (a.n_streams == 2) launch_stream_links<TO, 2>(a, rows, stream);
    else if (a.n_streams == 3) launch_stream_links<TO, 3>(a, rows, stream);
    else launch_stream_links<TO, 4>(a, rows, stream);
}

ROCML_EXPORT int rocml_stream_links(const float* src, int src_streams, const float* y, const float* partials, int n_splits,
                                    long long split_stride, int replace, const float* mix, const float* w_out, float* dst, float* total,
                                    const float* w_in, const float* gain, float eps, void* normed, int normed_dtype, int rows, int n,
                                    int n_streams, hipStream_t stream) {
    ROCML_REQUIRE(rows >= 0 && n > 0 && n_streams >= 1 && n_streams <= SM_MAX, "stream_links: bad sizes rows=%d n=%d streams=%d (at most %d)",
                  rows, n, n_streams, SM_MAX);
    ROCML_REQUIRE(src && (src_streams == n_streams || src_streams == 1), "stream_links: a source of %d streams for %d", src_streams, n_streams);
    ROCML_REQUIRE((mix == nullptr) == (w_out == nullptr), "stream_links: the streams' update needs both of its weights");
    ROCML_REQUIRE(mix ? (replace ? n_splits > 0 : y != nullptr) : (!y && n_splits == 0),
                  "stream_links: an update goes with a sublayer's output (or its K pieces), a plain read without");
    ROCML_REQUIRE(n_splits >= 0 && (n_splits == 0 || (partials && split_stride >= (long long)rows * n)), "stream_links: K pieces need a pointer and a stride");
    ROCML_REQUIRE((normed == nullptr) == (w_in == nullptr) && (normed == nullptr) == (gain == nullptr) && (!normed || eps > 0.f),
                  "stream_links: a read of the streams needs weights, a gain, a positive eps and a place");
    ROCML_REQUIRE(normed || total || dst, "stream_links: nothing to write");
    ROCML_REQUIRE(!(mix && normed) || dst, "stream_links: streams that are read on have to be stored");
    ROCML_REQUIRE(normed_dtype == ROCML_F32 || normed_dtype == ROCML_BF16, "stream_links: unknown dtype code %d", normed_dtype);
    if (rows == 0) return 0;
    StreamArgs a{src, (long long)src_streams * n, src_streams == 1 ? 0ll : (long long)n, y, partials, n_splits, split_stride, replace,
                 mix, w_out, dst, total, w_in, gain, eps, normed, n, n_streams};
    uintptr_t all = (uintptr_t)src | (uintptr_t)y | (uintptr_t)partials | (uintptr_t)dst | (uintptr_t)total | (uintptr_t)gain | (uintptr_t)normed;
    bool vec = n % 4 == 0 && n <= 16 * SM_BLOCK && (all & 15) == 0 && split_stride % 4 == 0;
    if (normed_dtype == ROCML_BF16) launch_stream_links_any<bf16_t>(a, rows, vec, stream);
    else launch_stream_links_any<float>(a, rows, vec, stream);
    ROCML_CHECK_LAUNCH("stream_links");
    return 0;
}
