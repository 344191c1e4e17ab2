// Plain attention over the paged cache for any head size and either storage type: one
// 256-thread block per (query token, query head).  It serves the 32-bit path (prefill and
// decode) and every head size the fast kernels refuse.  The algebra is the reference's
// (rocml-kernels/kernels/attn_decode.hip:151-170, attn_prefill.hip:167-190): s_j = (q . k_j) *
// scale, running maximum m, l = l * e^(m - m') + sum e^(s - m'), acc likewise, out = acc / l.
// A query at position p sees keys [lo, p], lo = 0 or p - window + 1.  Keys are taken 256 at a
// time: every thread scores one key, then the threads split the head's values.
// Cache layout: keys [page, Hkv, page_size, D], values transposed in a page [page, Hkv, Dv, page_size].
//
// What a layer may add to this, all of it parameters (AttnExtra):
//  * dv: the size of a value head, when it is not the size of a key head;
//  * v_in_k: there is no value cache, the value of a key is the first dv numbers of its row (keys
//    and values expanded from one latent vector, with the expansion folded into the queries and
//    into the product after the attention: one key/value head [latent, rotated part]);
//  * chunk: positions are cut into blocks of `chunk`, counted from 0; a query sees its own block
//    up to itself (lo = pos - pos % chunk) instead of a window;
//  * slopes[h]: slope * (pos - j) is taken off the score of key j;
//  * sink: one more term exp(0) in the denominator, with no value: the running maximum starts at 0
//    and the running sum at 1;
//  * sinks[h]: with sink, the term is exp(sinks[h]) instead: the running maximum starts there;
//  * softcap: the scaled score s becomes softcap * tanh(s / softcap), before the mask and the slope;
//  * keep_first: with a window, the first keep_first positions are seen whatever their distance;
//  * key_heads_per_value: so many neighbouring key heads share one value head (the value cache then has fewer heads).
// The output may be of another type than the queries (TO).
#pragma once
#include "common.h"

constexpr int AG_BLOCK = 256;
constexpr int AG_MAX_D_PER_THREAD = 4;   // head_dim <= 1024

__device__ __forceinline__ float ag_block_max(float v, float* scratch) {
    v = wave_max(v);
    __syncthreads();
    if ((threadIdx.x & (WAVE - 1)) == 0) scratch[threadIdx.x / WAVE] = v;
    __syncthreads();
    float r = scratch[0];
#pragma unroll
    for (int w = 1; w < AG_BLOCK / WAVE; ++w) r = fmaxf(r, scratch[w]);
    return r;
}

__device__ __forceinline__ float ag_block_sum(float v, float* scratch) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & (WAVE - 1)) == 0) scratch[threadIdx.x / WAVE] = v;
    __syncthreads();
    float r = 0.f;
#pragma unroll
    for (int w = 0; w < AG_BLOCK / WAVE; ++w) r += scratch[w];
    return r;
}

struct AttnExtra {
    int dv;                 // value head size
    int v_in_k;             // values are the leading dv numbers of the key rows
    int chunk;              // 0: none
    const float* slopes;    // [Hq] or null
    int sink;
    const float* sinks;     // [Hq] or null
    float softcap;          // 0: none
    int keep_first;         // 0: none
    int key_heads_per_value = 1;
};

__device__ __forceinline__ int attn_first_key(int pos, int window, int chunk) {
    if (chunk > 0) return pos - pos % chunk;
    return window > 0 ? max(0, pos - window + 1) : 0;
}

template <typename T, typename TO = T>
__global__ void __launch_bounds__(AG_BLOCK)
attn_generic_kernel(const T* __restrict__ q, TO* __restrict__ out, const T* __restrict__ kcache,
                    const T* __restrict__ vcache, const int* __restrict__ block_table, int bt_width,
                    const int* __restrict__ token_seq, const int* __restrict__ token_pos, int hq,
                    int hkv, int d, int page_size, float scale, int window, AttnExtra ex) {
    extern __shared__ float smem[];
    float* qs = smem;                 // [d]
    float* ps = smem + d;             // [AG_BLOCK]
    __shared__ float red[AG_BLOCK / WAVE];
    int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
    int pos = token_pos[t];
    const int* pages = block_table + (size_t)token_seq[t] * bt_width;
    int kvh = h / (hq / hkv);
    int lo = attn_first_key(pos, window, ex.chunk);
    // the keys to visit, numbered 0 .. n_seen - 1: kept first positions before the window, then the window
    int n_kept = min(ex.keep_first, lo), n_seen = n_kept + pos - lo + 1;
    auto key_of = [&](int i) { return i < n_kept ? i : lo + i - n_kept; };
    int dv = ex.dv;
    int hv = hkv / ex.key_heads_per_value, vh = kvh / ex.key_heads_per_value;
    float slope = ex.slopes ? ex.slopes[h] : 0.f;
    const T* qrow = q + ((size_t)t * hq + h) * d;
    for (int e = tid; e < d; e += AG_BLOCK) qs[e] = Elem<T>::load(qrow + e);
    __syncthreads();
    float m = ex.sink ? (ex.sinks ? ex.sinks[h] : 0.f) : -INFINITY, l = ex.sink ? 1.f : 0.f;
    float acc[AG_MAX_D_PER_THREAD] = {};
    for (int c0 = 0; c0 < n_seen; c0 += AG_BLOCK) {
        int j = key_of(c0 + tid);
        bool seen = c0 + tid < n_seen;
        float s = -INFINITY;
        if (seen) {
            int page = pages[j / page_size];
            const T* krow = kcache + (((size_t)page * hkv + kvh) * page_size + j % page_size) * d;
            float dot = 0.f;
            for (int e = 0; e < d; ++e) dot = fmaf(qs[e], Elem<T>::load(krow + e), dot);
            s = dot * scale;
            if (ex.softcap > 0.f) s = ex.softcap * tanhf(s / ex.softcap);
            s -= slope * (float)(pos - j);
        }
        float m_new = fmaxf(m, ag_block_max(s, red));
        float corr = expf(m - m_new);            // first chunk: exp(-inf) = 0
        float p = seen ? expf(s - m_new) : 0.f;
        ps[tid] = p;
        l = l * corr + ag_block_sum(p, red);     // barrier inside also publishes ps
        int n_keys = min(AG_BLOCK, n_seen - c0);
#pragma unroll
        for (int r = 0; r < AG_MAX_D_PER_THREAD; ++r) {
            int e = tid + r * AG_BLOCK;
            if (e >= dv) break;
            float a = acc[r] * corr;
            if (ex.v_in_k) {
                for (int jj = 0; jj < n_keys; ++jj) {
                    int key = key_of(c0 + jj);
                    int page = pages[key / page_size];
                    const T* krow = kcache + (((size_t)page * hkv + kvh) * page_size + key % page_size) * d;
                    a = fmaf(ps[jj], Elem<T>::load(krow + e), a);
                }
            } else {
                for (int jj = 0; jj < n_keys; ++jj) {
                    int key = key_of(c0 + jj);
                    int page = pages[key / page_size];
                    const T* vcol = vcache + ((size_t)page * hv + vh) * dv * page_size + key % page_size;
                    a = fmaf(ps[jj], Elem<T>::load(vcol + (size_t)e * page_size), a);
                }
            }
            acc[r] = a;
        }
        m = m_new;
        __syncthreads();                         // ps is rewritten by the next chunk
    }
    TO* orow = out + ((size_t)t * hq + h) * dv;
#pragma unroll
    for (int r = 0; r < AG_MAX_D_PER_THREAD; ++r) {
        int e = tid + r * AG_BLOCK;
        if (e < dv) Elem<TO>::store(orow + e, acc[r] / l);
    }
}
