// What the kernels that make queries, keys and values ready for the cache share: eight neighbours at once, and a
// prompt's values into their pages a page at a time.
#pragma once
#include "common.h"

template <typename T> struct Eight;
template <> struct Eight<float> {
    __device__ static void load(const float* p, float* o) {
        const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
        o[0] = a.x; o[1] = a.y; o[2] = a.z; o[3] = a.w; o[4] = b.x; o[5] = b.y; o[6] = b.z; o[7] = b.w;
    }
    __device__ static void store(float* p, const float* v) {
        *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
        *reinterpret_cast<float4*>(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
    }
};
template <> struct Eight<bf16_t> {
    __device__ static void load(const bf16_t* p, float* o) {
        const uint4 v = *reinterpret_cast<const uint4*>(p);
        const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            o[2 * i] = __uint_as_float(w[i] << 16);
            o[2 * i + 1] = __uint_as_float(w[i] & 0xFFFF0000u);
        }
    }
    __device__ static void store(bf16_t* p, const float* v) {
        *reinterpret_cast<uint4*>(p) = make_uint4(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]),
                                                  pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7]));
    }
};

// Values into their pages, a page at a time: one workgroup per (32 positions touched by this step, sequence, kv
// head) reads the new tokens' value heads as rows, turns them through LDS and writes channel rows.
#define QT_TOKENS 32
template <typename TA, typename TC>
__global__ void __launch_bounds__(256)
values_to_pages_kernel(const TA* __restrict__ qkv, size_t row_len, size_t v_off, const int32_t* __restrict__ cu_seqlens,
                       const int32_t* __restrict__ tok_pos, const int32_t* __restrict__ page_table, int table_width,
                       TC* __restrict__ v_pages, int kv_heads, int vdim, int page_size, const float* __restrict__ bias) {
    extern __shared__ float tile[];                          // [QT_TOKENS][vdim + 1]
    const int b = blockIdx.y, kvh = blockIdx.z;
    const int t_begin = cu_seqlens[b], n = cu_seqlens[b + 1] - t_begin;
    if (n <= 0) return;
    const int start = tok_pos[t_begin];                      // the sequence's new tokens sit at start .. start + n - 1
    const int first = (start / QT_TOKENS + blockIdx.x) * QT_TOKENS;
    const int lo = max(first, start), hi = min(first + QT_TOKENS - 1, start + n - 1);
    if (lo > hi) return;
    const int stride = vdim + 1;
    const TA* from = qkv + v_off + (size_t)kvh * vdim;
    const float* add = bias ? bias + (size_t)kvh * vdim : nullptr;
    const bool whole = lo == first && hi == first + QT_TOKENS - 1;
    if (sizeof(TA) == 2 && whole && vdim % 8 == 0 && (row_len % 8) == 0 && (v_off % 8) == 0) {
        const int pieces = vdim / 8;
        for (int e = threadIdx.x; e < QT_TOKENS * pieces; e += blockDim.x) {
            const int tt = e / pieces, d = (e - tt * pieces) * 8;
            float v[8];
            Eight<TA>::load(from + (size_t)(t_begin + first - start + tt) * row_len + d, v);
#pragma unroll
            for (int j = 0; j < 8; ++j) tile[tt * stride + d + j] = v[j];
        }
    } else {
        for (int e = threadIdx.x; e < (hi - lo + 1) * vdim; e += blockDim.x) {
            const int tt = e / vdim, d = e - tt * vdim;
            tile[(lo - first + tt) * stride + d] = to_f32(from[(size_t)(t_begin + lo - start + tt) * row_len + d]);
        }
    }
    __syncthreads();
    const int page = page_table[(size_t)b * table_width + first / page_size];
    TC* base = v_pages + ((size_t)page * kv_heads + kvh) * page_size * vdim + first % page_size;
    if (whole && page_size % 8 == 0) {
        for (int e = threadIdx.x; e < vdim * (QT_TOKENS / 8); e += blockDim.x) {
            const int d = e / (QT_TOKENS / 8), t8 = (e - d * (QT_TOKENS / 8)) * 8;
            const float b = add ? add[d] : 0.f;
            float v[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) v[j] = tile[(t8 + j) * stride + d] + b;
            Eight<TC>::store(base + (size_t)d * page_size + t8, v);
        }
    } else {
        for (int e = threadIdx.x; e < vdim * QT_TOKENS; e += blockDim.x) {
            const int d = e / QT_TOKENS, tt = e - d * QT_TOKENS;
            if (first + tt >= lo && first + tt <= hi) from_f32(base + (size_t)d * page_size + tt, tile[tt * stride + d] + (add ? add[d] : 0.f));
        }
    }
}
