// Queries, keys and values of an attention whose projections have biases and whose rotation turns the halves of the
// first part of a head, in one pass over the projection's rows (q heads at q_off, k heads at k_off, v heads at v_off
// of rows of row_len elements; the biases float32, one per column of q, k and v):
//
//   q, k: x += bias; with gains, x <- x / sqrt(mean(x^2) + eps) * gain over a head (one gain of dim for all q heads, one for
//         all k heads); the elements (i, i + half), i < half, turn by pos * inv_freq[i], cosine and sine times `amplitude`;
//         what lies behind 2 half passes; q in place, k into k_pages [pages][kv_heads][page_size][dim];
//   v:    v + bias into v_pages [pages][kv_heads][vdim][page_size] (transposed inside a page).
//
// Bias, norm, angle, sine and cosine are float32; an element is rounded once.  kv_heads 0: a layer that reads another one's
// keys and values, queries alone.
#include "api.h"
#include "common.h"
#include "kv_pages.h"

// One wavefront per (token, head): the general form, and that of single tokens.
template <typename T>
__global__ void __launch_bounds__(256)
qk_half_bias_kv_write_kernel(T* __restrict__ proj, size_t row_len, int q_off, int k_off, int v_off,
                             const float* __restrict__ q_bias, const float* __restrict__ k_bias,
                             const float* __restrict__ v_bias, const float* __restrict__ q_gain,
                             const float* __restrict__ k_gain, float eps, const float* __restrict__ inv_freq, int half,
                             float amplitude, const int32_t* __restrict__ tok_pos, const int32_t* __restrict__ tok_seq,
                             const int32_t* __restrict__ page_table, int table_width, T* __restrict__ k_pages,
                             T* __restrict__ v_pages, int tokens, int heads, int kv_heads, int dim, int vdim, int page_size,
                             int write_values) {
    const int lane = threadIdx.x & (RI_WAVE - 1);
    const int all_heads = heads + (write_values ? 2 : 1) * kv_heads;
    const long item = (long)blockIdx.x * (blockDim.x / RI_WAVE) + threadIdx.x / RI_WAVE;
    if (item >= (long)tokens * all_heads) return;          // whole wavefront leaves together
    const int t = (int)(item / all_heads), hh = (int)(item % all_heads);
    T* row = proj + (size_t)t * row_len;
    const int pos = tok_pos[t];
    const int kvh = hh < heads + kv_heads ? hh - heads : hh - heads - kv_heads;      // of a key or value head
    const size_t page_head =
        hh < heads ? 0 : (size_t)page_table[(size_t)tok_seq[t] * table_width + pos / page_size] * kv_heads + kvh;
    if (hh >= heads + kv_heads) {
        const T* x = row + v_off + (size_t)kvh * vdim;
        T* vt = v_pages + page_head * page_size * vdim + pos % page_size;
        for (int d = lane; d < vdim; d += RI_WAVE)
            from_f32(vt + (size_t)d * page_size, to_f32(x[d]) + (v_bias ? v_bias[(size_t)kvh * vdim + d] : 0.f));
        return;
    }
    const bool is_q = hh < heads;
    T* x = row + (is_q ? q_off + (size_t)hh * dim : k_off + (size_t)kvh * dim);
    const float* bias = is_q ? q_bias : k_bias;
    if (bias) bias += (size_t)(is_q ? hh : kvh) * dim;
    T* to = is_q ? x : k_pages + (page_head * page_size + pos % page_size) * dim;
    const float* gain = is_q ? q_gain : k_gain;
    float inv = 1.f;
    if (gain) {
        float ss = 0.f;
        for (int i = lane; i < dim; i += RI_WAVE) {
            const float v = to_f32(x[i]) + (bias ? bias[i] : 0.f);
            ss += v * v;
        }
        inv = 1.f / sqrtf(wave_sum(ss) / (float)dim + eps);
    }
    for (int i = lane; i < half; i += RI_WAVE) {
        float u = to_f32(x[i]), v = to_f32(x[i + half]);
        if (bias) {
            u += bias[i];
            v += bias[i + half];
        }
        if (gain) {
            u = u * inv * gain[i];
            v = v * inv * gain[i + half];
        }
        float sn, cs;
        sincosf((float)pos * inv_freq[i], &sn, &cs);
        sn *= amplitude;
        cs *= amplitude;
        from_f32(to + i, u * cs - v * sn);
        from_f32(to + i + half, v * cs + u * sn);
    }
    for (int i = 2 * half + lane; i < dim; i += RI_WAVE) {
        const float v = to_f32(x[i]) + (bias ? bias[i] : 0.f);
        from_f32(to + i, gain ? v * inv * gain[i] : v);
    }
}

// A prompt whose halves and head sizes 16-byte pieces divide: a workgroup a token.  The token's sines and cosines are
// made once, in LDS; with gains a head's norm meets over the lanes that hold its pieces, where they are a power of two (`lanes`),
// and else in a pass of its own ahead (a wavefront a head, lanes 0); a thread takes a piece of eight from each half of a head (or one of the part that passes), every
// load and store 16 bytes (32 for float32).  The values go a page at a time (values_to_pages_kernel).
template <typename T>
__global__ void __launch_bounds__(512)
qk_half_bias_k_write_vec_kernel(T* __restrict__ proj, size_t row_len, int q_off, int k_off, const float* __restrict__ q_bias,
                                const float* __restrict__ k_bias, const float* __restrict__ q_gain,
                                const float* __restrict__ k_gain, float eps, const float* __restrict__ inv_freq, int half,
                                float amplitude, const int32_t* __restrict__ tok_pos, const int32_t* __restrict__ tok_seq,
                                const int32_t* __restrict__ page_table, int table_width, T* __restrict__ k_pages, int heads,
                                int kv_heads, int dim, int page_size, int lanes) {
    extern __shared__ __align__(16) float turn[];          // [half] cosines, [half] sines, [heads + kv_heads] factors
    const int t = blockIdx.x, pos = tok_pos[t];
    T* row = proj + (size_t)t * row_len;
    if (q_gain && !lanes) {
        for (int hh = threadIdx.x / RI_WAVE; hh < heads + kv_heads; hh += blockDim.x / RI_WAVE) {
            const bool is_q = hh < heads;
            const T* x = row + (is_q ? q_off + (size_t)hh * dim : k_off + (size_t)(hh - heads) * dim);
            const float* bias = is_q ? q_bias : k_bias;
            if (bias) bias += (size_t)(is_q ? hh : hh - heads) * dim;
            float ss = 0.f;
            for (int i = (threadIdx.x & (RI_WAVE - 1)) * 8; i < dim; i += RI_WAVE * 8) {
                float u[8], b[8];
                Eight<T>::load(x + i, u);
                if (bias) {
                    Eight<float>::load(bias + i, b);
#pragma unroll
                    for (int k = 0; k < 8; ++k) u[k] += b[k];
                }
#pragma unroll
                for (int k = 0; k < 8; ++k) ss += u[k] * u[k];
            }
            ss = wave_sum(ss);
            if ((threadIdx.x & (RI_WAVE - 1)) == 0) turn[2 * half + hh] = 1.f / sqrtf(ss / (float)dim + eps);
        }
    }
    for (int i = threadIdx.x; i < half; i += blockDim.x) {
        float sn, cs;
        sincosf((float)pos * inv_freq[i], &sn, &cs);
        turn[i] = cs * amplitude;
        turn[half + i] = sn * amplitude;
    }
    __syncthreads();
    const long page = kv_heads > 0 ? page_table[(size_t)tok_seq[t] * table_width + pos / page_size] : 0;
    const int turning = half / 8, pieces = turning + (dim - 2 * half) / 8;      // of a head
    for (int e = threadIdx.x; e < (heads + kv_heads) * pieces; e += blockDim.x) {
        const int hh = e / pieces, piece = e - hh * pieces;
        const bool is_q = hh < heads;
        T* x = row + (is_q ? q_off + (size_t)hh * dim : k_off + (size_t)(hh - heads) * dim);
        const float* bias = is_q ? q_bias : k_bias;
        if (bias) bias += (size_t)(is_q ? hh : hh - heads) * dim;
        T* to = is_q ? x : k_pages + ((page * kv_heads + (hh - heads)) * page_size + pos % page_size) * dim;
        const int i = piece < turning ? piece * 8 : 2 * half + (piece - turning) * 8;
        const bool turns = piece < turning;
        float u[8], v[8], b[8];
        Eight<T>::load(x + i, u);
        Eight<T>::load(x + (turns ? i + half : i), v);
        if (bias) {
            Eight<float>::load(bias + i, b);
#pragma unroll
            for (int k = 0; k < 8; ++k) u[k] += b[k];
            Eight<float>::load(bias + (turns ? i + half : i), b);
#pragma unroll
            for (int k = 0; k < 8; ++k) v[k] += b[k];
        }
        const float* gain = is_q ? q_gain : k_gain;
        if (gain) {
            float inv;
            if (lanes) {                                      // (the lanes of a head run this loop together)
                float ss = 0.f;
#pragma unroll
                for (int k = 0; k < 8; ++k) ss += u[k] * u[k] + (turns ? v[k] * v[k] : 0.f);
                for (int m = lanes / 2; m > 0; m >>= 1) ss += __shfl_xor(ss, m, RI_WAVE);
                inv = 1.f / sqrtf(ss / (float)dim + eps);
            } else {
                inv = turn[2 * half + hh];
            }
            Eight<float>::load(gain + i, b);
#pragma unroll
            for (int k = 0; k < 8; ++k) u[k] = u[k] * inv * b[k];
            Eight<float>::load(gain + (turns ? i + half : i), b);
#pragma unroll
            for (int k = 0; k < 8; ++k) v[k] = v[k] * inv * b[k];
        }
        if (turns) {
            float cs[8], sn[8];
            Eight<float>::load(turn + i, cs);
            Eight<float>::load(turn + half + i, sn);
#pragma unroll
            for (int k = 0; k < 8; ++k) {
                const float a = u[k] * cs[k] - v[k] * sn[k];
                v[k] = v[k] * cs[k] + u[k] * sn[k];
                u[k] = a;
            }
            Eight<T>::store(to + i + half, v);
        }
        Eight<T>::store(to + i, u);
    }
}

template <typename T>
static void launch_qk_half(T* proj, size_t row_len, int q_off, int k_off, int v_off, const float* q_bias, const float* k_bias,
                           const float* v_bias, const float* q_gain, const float* k_gain, float eps, const float* inv_freq, int half,
                           float amplitude, const int32_t* tok_pos, const int32_t* tok_seq, const int32_t* cu_seqlens, int seqs, int max_new,
                           const int32_t* page_table, int table_width, T* k_pages, T* v_pages, int tokens, int heads,
                           int kv_heads, int dim, int vdim, int page_size, hipStream_t s) {
    const bool prompt = cu_seqlens && max_new > 1;
    const bool paged_values = prompt && kv_heads > 0 && page_size % QT_TOKENS == 0 && seqs <= 65535 && kv_heads <= 65535 &&
                              (size_t)QT_TOKENS * (vdim + 1) * sizeof(float) <= 65536;
    // (a piece of eight starts on a 16-byte boundary where every head, half and row does)
    const int unit = 16 / (int)sizeof(T);
    const bool pieces = prompt && (paged_values || kv_heads == 0) && half % 8 == 0 && dim % 8 == 0 &&
                        (row_len | q_off | k_off) % unit == 0 && (uintptr_t)proj % 16 == 0 && (uintptr_t)k_pages % 16 == 0 &&
                        ((uintptr_t)q_bias | (uintptr_t)k_bias | (uintptr_t)q_gain | (uintptr_t)k_gain) % 16 == 0 &&
                        (2L * half + heads + kv_heads + 4) * (long)sizeof(float) <= 65536;
    if (pieces) {
        const int of_head = half / 8 + (dim - 2 * half) / 8, all = (heads + kv_heads) * of_head;
        const int lanes = of_head <= RI_WAVE && (of_head & (of_head - 1)) == 0 ? of_head : 0;
        const int threads = all <= 512 && all > 256 ? (all + RI_WAVE - 1) / RI_WAVE * RI_WAVE : 256;      // (a token in one turn where that fits)
        qk_half_bias_k_write_vec_kernel<T><<<tokens, threads, (2 * half + heads + kv_heads + 4) * sizeof(float), s>>>(
            proj, row_len, q_off, k_off, q_bias, k_bias, q_gain, k_gain, eps, inv_freq, half, amplitude, tok_pos, tok_seq, page_table, table_width,
            k_pages, heads, kv_heads, dim, page_size, lanes);
    } else {
        const long items = (long)tokens * (heads + (paged_values ? 1 : 2) * kv_heads);
        qk_half_bias_kv_write_kernel<T><<<(unsigned)((items + 3) / 4), 256, 0, s>>>(
            proj, row_len, q_off, k_off, v_off, q_bias, k_bias, v_bias, q_gain, k_gain, eps, inv_freq, half, amplitude, tok_pos, tok_seq, page_table,
            table_width, k_pages, v_pages, tokens, heads, kv_heads, dim, vdim, page_size, !paged_values);
    }
    if (paged_values) {
        dim3 grid((max_new + QT_TOKENS - 2) / QT_TOKENS + 1, seqs, kv_heads);      // the 32-position pieces a sequence may touch
        values_to_pages_kernel<T, T><<<grid, 256, QT_TOKENS * (vdim + 1) * sizeof(float), s>>>(
            proj, row_len, (size_t)v_off, cu_seqlens, tok_pos, page_table, table_width, v_pages, kv_heads, vdim, page_size, v_bias);
    }
}

extern "C" int ri_qk_half_bias_kv_write(void* proj, int act_dtype, long row_len, int q_off, int k_off, int v_off,
                                        const float* q_bias, const float* k_bias, const float* v_bias, const float* q_gain,
                                        const float* k_gain, float eps, const float* inv_freq, int half, float amplitude, const int32_t* tok_pos, const int32_t* tok_seq,
                                        const int32_t* cu_seqlens, int seqs, int max_new, const int32_t* page_table,
                                        int table_width, void* k_pages, void* v_pages, int cache_dtype, int tokens, int heads,
                                        int kv_heads, int dim, int vdim, int page_size, void* stream) {
    RI_REQUIRE(tokens > 0 && heads > 0 && kv_heads >= 0, "qk_half_bias_kv_write: tokens %d, heads %d, kv heads %d", tokens, heads,
               kv_heads);
    RI_REQUIRE(dim >= 1 && vdim >= 1 && half >= 0 && 2 * half <= dim && half <= 8192 && (half == 0 || inv_freq),
               "qk_half_bias_kv_write: heads of %d and %d, %d pairs turn", dim, vdim, half);
    RI_REQUIRE(q_off >= 0 && q_off + (long)heads * dim <= row_len, "qk_half_bias_kv_write: q at %d does not fit rows of %ld", q_off, row_len);
    RI_REQUIRE(kv_heads == 0 || (k_off >= 0 && v_off >= 0 && k_off + (long)kv_heads * dim <= row_len &&
                                 v_off + (long)kv_heads * vdim <= row_len),
               "qk_half_bias_kv_write: k and v at %d and %d do not fit rows of %ld", k_off, v_off, row_len);
    RI_REQUIRE((act_dtype == RI_F32 || act_dtype == RI_BF16) && (kv_heads == 0 || act_dtype == cache_dtype),
               "qk_half_bias_kv_write: activations (%d) and cache (%d) must share float32 or bfloat16", act_dtype, cache_dtype);
    RI_REQUIRE(kv_heads == 0 || (page_size > 0 && table_width > 0 && k_pages && v_pages), "qk_half_bias_kv_write: page geometry");
    RI_REQUIRE(((long)tokens * (heads + 2 * kv_heads) + 3) / 4 <= 2147483647L, "qk_half_bias_kv_write: %ld heads exceed one launch",
               (long)tokens * (heads + 2 * kv_heads));
    RI_REQUIRE(kv_heads == 0 || (q_gain == nullptr) == (k_gain == nullptr), "qk_half_bias_kv_write: gains of q and k come together");
    RI_REQUIRE(!cu_seqlens || (seqs > 0 && max_new > 0), "qk_half_bias_kv_write: seqs %d, max_new %d", seqs, max_new);
    hipStream_t s = (hipStream_t)stream;
#define RI_GO(T)                                                                                                          \
    launch_qk_half<T>((T*)proj, (size_t)row_len, q_off, kv_heads ? k_off : 0, kv_heads ? v_off : 0, q_bias, k_bias, v_bias, \
                      q_gain, k_gain, eps, inv_freq, half, amplitude, tok_pos, tok_seq, cu_seqlens, seqs, max_new, page_table, table_width,      \
                      (T*)k_pages, (T*)v_pages, tokens, heads, kv_heads, dim, vdim, page_size, s)
    if (act_dtype == RI_F32) RI_GO(float); else RI_GO(bf16_t);
#undef RI_GO
    RI_LAUNCH_CHECK("qk_half_bias_kv_write");
    return 0;
}
