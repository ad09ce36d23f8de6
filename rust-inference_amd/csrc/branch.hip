// Row-wise kernels around a sublayer whose norm sits on its output, and around mixers that run side by side:
//
//   embed_scaled:     r = E[id] * scale (float32), and a copy of r in the activations' format;
//   embed_bigram:     r = E[id] + B[row of the pair (token before, token)], the token before kept per sequence;
//   branch_norm_add:  r += layer_scale * norm(y), the norm (layer norm with gain and bias, or RMS norm with gain) over the
//                     sublayer's output y, which may come as parts of a split product that are added in order;
//                     again with a copy of the new r in the activations' format, which the next sublayer reads
//                     (the sublayers read r itself: there is no norm before them), or, where a norm sits in front of the
//                     next sublayer too, with that norm of the new r: act = r / sqrt(mean(r^2) + next_eps) * next_gain;
//   gate_rows:        out = scale * x * gate(g), element by element, into columns of a wider row (the heads of
//                     several mixers side by side, for one output product);
//   row_norm_gate:    out = scale * x / sqrt(mean(x^2) + eps) * gain * gate(g), the mean over the whole row (all heads
//                     of a mixer together), likewise into columns of a wider row.
//   normed_sum:       out = a_scale * norm(a) + b_scale * norm(b), RMS norms of two mixers' results over the model's width.
//
// The residual, the statistics of every norm, the layer scale and the gates' sigmoids are float32; a value is
// rounded once, when it is stored in the activations' format.  One workgroup a row; a row's sums are taken in an
// order that depends on the row's width alone.
#include "api.h"
#include "common.h"

#define BR_NORM_RMS 1
#define BR_NORM_LAYER 2
#define BR_GATE_SIGMOID 0
#define BR_GATE_SILU 1

// 16 bytes of float32 or 8 of bfloat16 at once, as four floats.
__device__ __forceinline__ float4 ld4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 ld4(const bf16_t* p) {
    const uint2 w = *reinterpret_cast<const uint2*>(p);
    return make_float4(__uint_as_float(w.x << 16), __uint_as_float(w.x & 0xFFFF0000u), __uint_as_float(w.y << 16),
                       __uint_as_float(w.y & 0xFFFF0000u));
}
__device__ __forceinline__ void st4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void st4(bf16_t* p, float4 v) {
    uint2 w;
    w.x = pack_bf16x2(v.x, v.y);
    w.y = pack_bf16x2(v.z, v.w);
    *reinterpret_cast<uint2*>(p) = w;
}

// Rows whose width is a multiple of 4: a thread takes four neighbours, a workgroup 1,024 columns of one row.
template <typename TW, typename TA>
__global__ void __launch_bounds__(256)
embed_scaled_vec_kernel(float* __restrict__ out, TA* __restrict__ act, const TW* __restrict__ table,
                        const int32_t* __restrict__ ids, float scale, int dim) {
    const int t = blockIdx.x, c = (blockIdx.y * 256 + threadIdx.x) * 4;
    if (c >= dim) return;
    float4 v = ld4(table + (size_t)ids[t] * dim + c);
    v = make_float4(v.x * scale, v.y * scale, v.z * scale, v.w * scale);
    st4(out + (size_t)t * dim + c, v);
    if (act) st4(act + (size_t)t * dim + c, v);
}

template <typename TW, typename TA>
__global__ void __launch_bounds__(256)
embed_scaled_kernel(float* __restrict__ out, TA* __restrict__ act, const TW* __restrict__ table,
                    const int32_t* __restrict__ ids, float scale, int dim) {
    const int t = blockIdx.x;
    const TW* row = table + (size_t)ids[t] * dim;
    for (int d = threadIdx.x; d < dim; d += blockDim.x) {
        const float v = to_f32(row[d]) * scale;
        out[(size_t)t * dim + d] = v;
        if (act) from_f32(act + (size_t)t * dim + d, v);
    }
}

extern "C" int ri_embed_scaled(float* out, void* act, int act_dtype, const void* table, int table_dtype, const int32_t* ids,
                               float scale, int tokens, int dim, void* stream) {
    RI_REQUIRE(tokens > 0 && dim > 0, "embed_scaled: tokens %d, dim %d", tokens, dim);
    RI_REQUIRE((table_dtype == RI_F32 || table_dtype == RI_BF16) && (act_dtype == RI_F32 || act_dtype == RI_BF16),
               "embed_scaled: table dtype %d, activations %d", table_dtype, act_dtype);
    hipStream_t s = (hipStream_t)stream;
    const dim3 vgrid(tokens, (dim / 4 + 255) / 256);
#define RI_GO(TW, TA)                                                                                                   \
    if (dim % 4 == 0 && vgrid.y <= 65535)                                                                               \
        embed_scaled_vec_kernel<TW, TA><<<vgrid, 256, 0, s>>>(out, (TA*)act, (const TW*)table, ids, scale, dim);        \
    else                                                                                                                \
        embed_scaled_kernel<TW, TA><<<tokens, 256, 0, s>>>(out, (TA*)act, (const TW*)table, ids, scale, dim)
    if (table_dtype == RI_F32) { if (act_dtype == RI_F32) RI_GO(float, float); else RI_GO(float, bf16_t); }
    else                       { if (act_dtype == RI_F32) RI_GO(bf16_t, float); else RI_GO(bf16_t, bf16_t); }
#undef RI_GO
    RI_LAUNCH_CHECK("embed_scaled");
    return 0;
}

// Row `buckets` (the last) for a sequence's first token; else row (before * mul_prev + id * mul_cur) mod buckets, both
// factors already reduced modulo buckets (every product then fits 64 bits).  A workgroup a token; the workgroup of a
// sequence's first new token alone reads the token kept from the step before, and it alone puts the step's last token in
// its place, after it has read.
template <typename TW, bool VEC>
__global__ void __launch_bounds__(1024)
embed_bigram_kernel(float* __restrict__ out, const TW* __restrict__ table, const TW* __restrict__ pairs,
                    const int32_t* __restrict__ ids, const int32_t* __restrict__ tok_pos, const int32_t* __restrict__ tok_seq,
                    const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ slots, int32_t* __restrict__ last,
                    long buckets, long mul_prev, long mul_cur, int dim) {
    const int t = blockIdx.x, b = tok_seq[t], slot = slots[b];
    const bool opens = t == cu_seqlens[b];                   // the sequence's first token of this step
    const long id = ids[t];
    long row = buckets;
    if (tok_pos[t] > 0) {
        const long before = opens ? last[slot] : ids[t - 1];
        row = (before * mul_prev + id * mul_cur) % buckets;
    }
    const TW* a = table + (size_t)id * dim;
    const TW* p = pairs + (size_t)row * dim;
    float* o = out + (size_t)t * dim;
    if (VEC) {
        for (int d = threadIdx.x * 4; d < dim; d += blockDim.x * 4) {
            const float4 u = ld4(a + d), v = ld4(p + d);
            st4(o + d, make_float4(u.x + v.x, u.y + v.y, u.z + v.z, u.w + v.w));
        }
    } else {
        for (int d = threadIdx.x; d < dim; d += blockDim.x) o[d] = to_f32(a[d]) + to_f32(p[d]);
    }
    if (!opens) return;
    __syncthreads();                                         // every thread has read the kept token
    if (threadIdx.x == 0) last[slot] = ids[cu_seqlens[b + 1] - 1];
}

extern "C" int ri_embed_bigram(float* out, const void* table, const void* pairs, int table_dtype, const int32_t* ids,
                               const int32_t* tok_pos, const int32_t* tok_seq, const int32_t* cu_seqlens, const int32_t* slots,
                               int32_t* last, long buckets, long mul_prev, long mul_cur, int tokens, int dim, void* stream) {
    RI_REQUIRE(tokens > 0 && dim > 0, "embed_bigram: tokens %d, dim %d", tokens, dim);
    RI_REQUIRE(buckets >= 1 && buckets <= 2147483647L && mul_prev >= 0 && mul_prev < buckets && mul_cur >= 0 && mul_cur < buckets,
               "embed_bigram: %ld buckets, factors %ld and %ld (reduced modulo the buckets)", buckets, mul_prev, mul_cur);
    RI_REQUIRE(table_dtype == RI_F32 || table_dtype == RI_BF16, "embed_bigram: table dtype %d", table_dtype);
    hipStream_t s = (hipStream_t)stream;
    // a row of up to 4,096 elements in one pass of the workgroup: every load of both rows in flight at once
    const int threads = dim % 4 != 0 || dim <= 1024 ? 256 : dim <= 2048 ? 512 : 1024;
#define RI_GO(TW, VEC)                                                                                                  \
    embed_bigram_kernel<TW, VEC><<<tokens, threads, 0, s>>>(out, (const TW*)table, (const TW*)pairs, ids, tok_pos, tok_seq,    \
                                                       cu_seqlens, slots, last, buckets, mul_prev, mul_cur, dim)
    if (table_dtype == RI_F32) { if (dim % 4 == 0) RI_GO(float, true); else RI_GO(float, false); }
    else                       { if (dim % 4 == 0) RI_GO(bf16_t, true); else RI_GO(bf16_t, false); }
#undef RI_GO
    RI_LAUNCH_CHECK("embed_bigram");
    return 0;
}

// The row's y is kept in LDS as float32 between the passes (parts added once, in order).
template <typename TY, typename TA>
__global__ void __launch_bounds__(256)
branch_norm_add_kernel(float* __restrict__ residual, TA* __restrict__ act, const TY* __restrict__ y, int parts,
                       size_t part_stride, const float* __restrict__ gain, const float* __restrict__ bias, float eps,
                       int kind, const float* __restrict__ layer_scale, int dim, const float* __restrict__ next_gain,
                       float next_eps) {
    extern __shared__ float row[];                           // dim floats
    __shared__ float scratch[16];
    const size_t at = (size_t)blockIdx.x * dim;
    float sum = 0.f;
    for (int d = threadIdx.x; d < dim; d += blockDim.x) {
        float v = to_f32(y[at + d]);
        for (int p = 1; p < parts; ++p) v += to_f32(y[p * part_stride + at + d]);
        row[d] = v;
        sum += v;
    }
    float mean = 0.f;
    if (kind == BR_NORM_LAYER) mean = block_sum(sum, scratch) / (float)dim;
    float ss = 0.f;
    for (int d = threadIdx.x; d < dim; d += blockDim.x) {
        const float c = row[d] - mean;
        ss += c * c;
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)dim + eps);
    float rr = 0.f;
    for (int d = threadIdx.x; d < dim; d += blockDim.x) {
        float v = (row[d] - mean) * inv * gain[d];
        if (bias) v += bias[d];
        if (layer_scale) v *= layer_scale[d];
        const float r = residual[at + d] + v;
        residual[at + d] = r;
        if (next_gain) {                                     // (a thread's own columns: no barrier needed for them)
            row[d] = r;
            rr += r * r;
        } else if (act) from_f32(act + at + d, r);
    }
    if (!next_gain) return;
    const float next_inv = 1.0f / sqrtf(block_sum(rr, scratch) / (float)dim + next_eps);
    for (int d = threadIdx.x; d < dim; d += blockDim.x) from_f32(act + at + d, row[d] * next_inv * next_gain[d]);
}

// The same for rows of up to 8,192 elements, a multiple of 4: a thread asks for all its 16-byte pieces of the residual
// and of every part of y up front and keeps them in registers, so that a row is one trip to memory and not one an
// element; the parts are added in their order, the row's sums taken in an order that the width alone fixes.  `tiled`
// (with NEXT): act in the order of tiled_at.
template <typename TY, typename TA, int VPT, bool NEXT>
__global__ void __launch_bounds__(256)
branch_norm_add_vec_kernel(float* __restrict__ residual, TA* __restrict__ act, const TY* __restrict__ y, int parts,
                           size_t part_stride, const float* __restrict__ gain, const float* __restrict__ bias, float eps,
                           int kind, const float* __restrict__ layer_scale, int dim, const float* __restrict__ next_gain,
                           float next_eps, int tiled) {
    __shared__ float scratch[16];
    const size_t at = (size_t)blockIdx.x * dim;
    float4 r[VPT], v[VPT], ng[NEXT ? VPT : 1];
    int col[VPT];
    bool ok[VPT];
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        const int c = (threadIdx.x + i * 256) * 4;
        ok[i] = c < dim;
        col[i] = ok[i] ? c : 0;                              // a column pulled back inside the row: the load is issued anyway
        r[i] = ld4(residual + at + col[i]);
        v[i] = ld4(y + at + col[i]);
        if (NEXT) ng[i] = ld4(next_gain + col[i]);
    }
    for (int p = 1; p < parts; ++p) {
#pragma unroll
        for (int i = 0; i < VPT; ++i) {
            const float4 w = ld4(y + p * part_stride + at + col[i]);
            v[i] = make_float4(v[i].x + w.x, v[i].y + w.y, v[i].z + w.z, v[i].w + w.w);
        }
    }
    float mean = 0.f;
    if (kind == BR_NORM_LAYER) {
        float sum = 0.f;
#pragma unroll
        for (int i = 0; i < VPT; ++i)
            if (ok[i]) sum += (v[i].x + v[i].y) + (v[i].z + v[i].w);
        mean = block_sum(sum, scratch) / (float)dim;
    }
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        if (ok[i]) {
            const float a = v[i].x - mean, b = v[i].y - mean, c = v[i].z - mean, d = v[i].w - mean;
            ss += (a * a + b * b) + (c * c + d * d);
        }
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)dim + eps);
    float rr = 0.f;
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        if (!ok[i]) continue;
        const float4 g = ld4(gain + col[i]);
        float4 o = make_float4((v[i].x - mean) * inv * g.x, (v[i].y - mean) * inv * g.y, (v[i].z - mean) * inv * g.z,
                               (v[i].w - mean) * inv * g.w);
        if (bias) {
            const float4 b = ld4(bias + col[i]);
            o = make_float4(o.x + b.x, o.y + b.y, o.z + b.z, o.w + b.w);
        }
        if (layer_scale) {
            const float4 l = ld4(layer_scale + col[i]);
            o = make_float4(o.x * l.x, o.y * l.y, o.z * l.z, o.w * l.w);
        }
        o = make_float4(r[i].x + o.x, r[i].y + o.y, r[i].z + o.z, r[i].w + o.w);
        st4(residual + at + col[i], o);
        if (NEXT) {
            r[i] = o;
            rr += (o.x * o.x + o.y * o.y) + (o.z * o.z + o.w * o.w);
        } else if (act) st4(act + at + col[i], o);
    }
    if (!NEXT) return;
    const float next_inv = 1.0f / sqrtf(block_sum(rr, scratch) / (float)dim + next_eps);
#pragma unroll
    for (int i = 0; i < VPT; ++i)
        if (ok[i])                                           // four columns of one chunk of eight, tiled or not
            st4(tiled ? act + tiled_at(blockIdx.x, col[i], (dim + 31) / 32) : act + at + col[i],
                make_float4(r[i].x * next_inv * ng[NEXT ? i : 0].x, r[i].y * next_inv * ng[NEXT ? i : 0].y,
                            r[i].z * next_inv * ng[NEXT ? i : 0].z, r[i].w * next_inv * ng[NEXT ? i : 0].w));
}

extern "C" int ri_branch_norm_add_norm(float* residual, void* act, int act_dtype, const void* y, int y_dtype, int parts,
                                       const float* gain, const float* bias, float eps, int kind, const float* layer_scale,
                                       const float* next_gain, float next_eps, int tiled, int rows, int dim, void* stream) {
    RI_REQUIRE(rows > 0 && dim > 0 && parts >= 1, "branch_norm_add: %d rows of %d in %d parts", rows, dim, parts);
    RI_REQUIRE(kind == BR_NORM_RMS || kind == BR_NORM_LAYER, "branch_norm_add: norm kind %d", kind);
    RI_REQUIRE(gain && residual && y, "branch_norm_add: a gain, a residual and a branch output are needed");
    RI_REQUIRE(!next_gain || act, "branch_norm_add: the next norm's rows need a place");
    RI_REQUIRE(!tiled || (next_gain && act_dtype == RI_BF16 && rows <= 64 && dim % 4 == 0 && dim <= 8192),
               "branch_norm_add: tiled rows are the next norm's, at most 64 (%d of %d), in bfloat16", rows, dim);
    RI_REQUIRE((size_t)dim * sizeof(float) <= 64 * 1024, "branch_norm_add: rows of %d exceed the kernel's 16384", dim);
    RI_REQUIRE((y_dtype == RI_F32 || y_dtype == RI_BF16) && (act_dtype == RI_F32 || act_dtype == RI_BF16),
               "branch_norm_add: dtypes %d and %d", y_dtype, act_dtype);
    RI_REQUIRE(parts == 1 || y_dtype == RI_F32, "branch_norm_add: parts of a product are float32");
    hipStream_t s = (hipStream_t)stream;
    const size_t lds = (size_t)dim * sizeof(float), stride = (size_t)rows * dim;
#define RI_VEC(TY, TA, VPT)                                                                                             \
    do {                                                                                                                \
        if (next_gain)                                                                                                  \
            branch_norm_add_vec_kernel<TY, TA, VPT, true><<<rows, 256, 0, s>>>(                                           \
                residual, (TA*)act, (const TY*)y, parts, stride, gain, bias, eps, kind, layer_scale, dim, next_gain,      \
                next_eps, tiled);                                                                                       \
        else                                                                                                            \
            branch_norm_add_vec_kernel<TY, TA, VPT, false><<<rows, 256, 0, s>>>(                                          \
                residual, (TA*)act, (const TY*)y, parts, stride, gain, bias, eps, kind, layer_scale, dim, nullptr, 0.f, 0); \
    } while (0)
#define RI_GO(TY, TA)                                                                                                   \
    do {                                                                                                                \
        if (dim % 4 == 0 && dim <= 1024) RI_VEC(TY, TA, 1);                                                             \
        else if (dim % 4 == 0 && dim <= 2048) RI_VEC(TY, TA, 2);                                                        \
        else if (dim % 4 == 0 && dim <= 4096) RI_VEC(TY, TA, 4);                                                        \
        else if (dim % 4 == 0 && dim <= 8192) RI_VEC(TY, TA, 8);                                                        \
        else                                                                                                            \
            branch_norm_add_kernel<TY, TA><<<rows, 256, lds, s>>>(residual, (TA*)act, (const TY*)y, parts, stride, gain,  \
                                                                 bias, eps, kind, layer_scale, dim, next_gain, next_eps); \
    } while (0)
    if (lds > 48 * 1024) {
        static bool asked = false;
        if (!asked) {
            hipFuncSetAttribute((const void*)branch_norm_add_kernel<float, float>, hipFuncAttributeMaxDynamicSharedMemorySize, 64 * 1024);
            hipFuncSetAttribute((const void*)branch_norm_add_kernel<float, bf16_t>, hipFuncAttributeMaxDynamicSharedMemorySize, 64 * 1024);
            hipFuncSetAttribute((const void*)branch_norm_add_kernel<bf16_t, float>, hipFuncAttributeMaxDynamicSharedMemorySize, 64 * 1024);
            hipFuncSetAttribute((const void*)branch_norm_add_kernel<bf16_t, bf16_t>, hipFuncAttributeMaxDynamicSharedMemorySize, 64 * 1024);
            asked = true;
        }
    }
    if (y_dtype == RI_F32) { if (act_dtype == RI_F32) RI_GO(float, float); else RI_GO(float, bf16_t); }
    else                   { if (act_dtype == RI_F32) RI_GO(bf16_t, float); else RI_GO(bf16_t, bf16_t); }
#undef RI_GO
#undef RI_VEC
    RI_LAUNCH_CHECK("branch_norm_add");
    return 0;
}

extern "C" int ri_branch_norm_add(float* residual, void* act, int act_dtype, const void* y, int y_dtype, int parts,
                                  const float* gain, const float* bias, float eps, int kind, const float* layer_scale,
                                  int rows, int dim, void* stream) {
    return ri_branch_norm_add_norm(residual, act, act_dtype, y, y_dtype, parts, gain, bias, eps, kind, layer_scale, nullptr, 0.f,
                                   0, rows, dim, stream);
}

__device__ __forceinline__ float gate_of(float g, int kind) {
    const float sg = 1.0f / (1.0f + expf(-g));
    return kind == BR_GATE_SILU ? g * sg : sg;
}

template <typename TX, typename TA>
__global__ void __launch_bounds__(256)
gate_rows_kernel(TA* __restrict__ out, int out_stride, const TX* __restrict__ x, const TA* __restrict__ gate, int gate_stride,
                 float scale, int kind, int width) {
    const size_t t = blockIdx.x;
    for (int d = threadIdx.x; d < width; d += blockDim.x)
        from_f32(out + t * out_stride + d,
                 scale * to_f32(x[t * width + d]) * (gate ? gate_of(to_f32(gate[t * gate_stride + d]), kind) : 1.0f));
}

// Widths, offsets and row lengths that are multiples of 4: a thread takes four neighbours, a workgroup 1,024 columns.
template <typename TX, typename TA>
__global__ void __launch_bounds__(256)
gate_rows_vec_kernel(TA* __restrict__ out, int out_stride, const TX* __restrict__ x, const TA* __restrict__ gate,
                     int gate_stride, float scale, int kind, int width) {
    const size_t t = blockIdx.x;
    const int d = (blockIdx.y * 256 + threadIdx.x) * 4;
    if (d >= width) return;
    float4 v = ld4(x + t * width + d);
    v = make_float4(v.x * scale, v.y * scale, v.z * scale, v.w * scale);
    if (gate) {
        const float4 g = ld4(gate + t * gate_stride + d);
        v = make_float4(v.x * gate_of(g.x, kind), v.y * gate_of(g.y, kind), v.z * gate_of(g.z, kind), v.w * gate_of(g.w, kind));
    }
    st4(out + t * out_stride + d, v);
}

// out[t, out_off + d] = scale * x[t, d] * gate(g[t, g_off + d]); x: [rows, width] in its own format; g and out share
// the activations' format.  gate NULL: the scaled copy alone.
extern "C" int ri_gate_rows(void* out, int out_stride, int out_off, const void* x, int x_dtype, const void* gate,
                            int gate_stride, int g_off, int act_dtype, float scale, int kind, int rows, int width,
                            void* stream) {
    RI_REQUIRE(rows > 0 && width > 0, "gate_rows: %d rows of %d", rows, width);
    RI_REQUIRE(out_off >= 0 && out_off + width <= out_stride && (!gate || (g_off >= 0 && g_off + width <= gate_stride)),
               "gate_rows: columns %d..+%d of rows of %d, gates %d..+%d of rows of %d", out_off, width, out_stride, g_off,
               width, gate_stride);
    RI_REQUIRE(kind == BR_GATE_SIGMOID || kind == BR_GATE_SILU, "gate_rows: gate kind %d", kind);
    RI_REQUIRE((x_dtype == RI_F32 || x_dtype == RI_BF16) && (act_dtype == RI_F32 || act_dtype == RI_BF16),
               "gate_rows: dtypes %d and %d", x_dtype, act_dtype);
    hipStream_t s = (hipStream_t)stream;
    const bool vec = (width | out_off | out_stride) % 4 == 0 && (!gate || (g_off | gate_stride) % 4 == 0) &&
                     (width / 4 + 255) / 256 <= 65535;
    const dim3 vgrid(rows, (width / 4 + 255) / 256);
#define RI_GO(TX, TA)                                                                                                  \
    if (vec)                                                                                                           \
        gate_rows_vec_kernel<TX, TA><<<vgrid, 256, 0, s>>>((TA*)out + out_off, out_stride, (const TX*)x,                  \
                                                           gate ? (const TA*)gate + g_off : nullptr, gate_stride, scale, \
                                                           kind, width);                                                \
    else                                                                                                               \
    gate_rows_kernel<TX, TA><<<rows, 256, 0, s>>>((TA*)out + out_off, out_stride, (const TX*)x,                             \
                                                  gate ? (const TA*)gate + g_off : nullptr,                              \
                                                  gate_stride, scale, kind, width)
    if (x_dtype == RI_F32) { if (act_dtype == RI_F32) RI_GO(float, float); else RI_GO(float, bf16_t); }
    else                   { if (act_dtype == RI_F32) RI_GO(bf16_t, float); else RI_GO(bf16_t, bf16_t); }
#undef RI_GO
    RI_LAUNCH_CHECK("gate_rows");
    return 0;
}

template <typename TA>
__global__ void __launch_bounds__(256)
row_norm_gate_kernel(TA* __restrict__ out, int out_stride, const float* __restrict__ x, const float* __restrict__ gain,
                     float eps, const TA* __restrict__ gate, int gate_stride, float scale, int kind, int width) {
    __shared__ float scratch[16];
    const size_t t = blockIdx.x;
    float ss = 0.f;
    for (int d = threadIdx.x; d < width; d += blockDim.x) {
        const float v = x[t * width + d];
        ss += v * v;
    }
    const float inv = 1.0f / sqrtf(block_sum(ss, scratch) / (float)width + eps);
    for (int d = threadIdx.x; d < width; d += blockDim.x) {
        float v = x[t * width + d] * inv;
        if (gain) v *= gain[d];
        if (gate) v *= gate_of(to_f32(gate[t * gate_stride + d]), kind);
        from_f32(out + t * out_stride + d, scale * v);
    }
}

// Rows of up to 8,192 elements whose width, offsets and row lengths are multiples of 4: a row in registers, one trip.
template <typename TA, int VPT>
__global__ void __launch_bounds__(256)
row_norm_gate_vec_kernel(TA* __restrict__ out, int out_stride, const float* __restrict__ x, const float* __restrict__ gain,
                         float eps, const TA* __restrict__ gate, int gate_stride, float scale, int kind, int width) {
    __shared__ float scratch[16];
    const size_t t = blockIdx.x;
    float4 v[VPT], g[VPT];
    int col[VPT];
    bool ok[VPT];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        const int c = (threadIdx.x + i * 256) * 4;
        ok[i] = c < width;
        col[i] = ok[i] ? c : 0;
        v[i] = ld4(x + t * width + col[i]);
        g[i] = gate ? ld4(gate + t * gate_stride + col[i]) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
#pragma unroll
    for (int i = 0; i < VPT; ++i)
        if (ok[i]) ss += (v[i].x * v[i].x + v[i].y * v[i].y) + (v[i].z * v[i].z + v[i].w * v[i].w);
    const float f = scale / sqrtf(block_sum(ss, scratch) / (float)width + eps);
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        if (!ok[i]) continue;
        float4 o = make_float4(v[i].x * f, v[i].y * f, v[i].z * f, v[i].w * f);
        if (gain) {
            const float4 w = ld4(gain + col[i]);
            o = make_float4(o.x * w.x, o.y * w.y, o.z * w.z, o.w * w.w);
        }
        if (gate)
            o = make_float4(o.x * gate_of(g[i].x, kind), o.y * gate_of(g[i].y, kind), o.z * gate_of(g[i].z, kind),
                            o.w * gate_of(g[i].w, kind));
        st4(out + t * out_stride + col[i], o);
    }
}

// out[t, out_off + d] = scale * x[t, d] / sqrt(mean_d(x[t, :]^2) + eps) * gain[d] * gate(g[t, g_off + d]); x float32.
extern "C" int ri_row_norm_gate(void* out, int out_stride, int out_off, const float* x, const float* gain, float eps,
                                const void* gate, int gate_stride, int g_off, int act_dtype, float scale, int kind,
                                int rows, int width, void* stream) {
    RI_REQUIRE(rows > 0 && width > 0, "row_norm_gate: %d rows of %d", rows, width);
    RI_REQUIRE(out_off >= 0 && out_off + width <= out_stride, "row_norm_gate: columns %d..+%d of rows of %d", out_off,
               width, out_stride);
    RI_REQUIRE(!gate || (g_off >= 0 && g_off + width <= gate_stride), "row_norm_gate: gates %d..+%d of rows of %d", g_off,
               width, gate_stride);
    RI_REQUIRE(kind == BR_GATE_SIGMOID || kind == BR_GATE_SILU, "row_norm_gate: gate kind %d", kind);
    RI_REQUIRE(act_dtype == RI_F32 || act_dtype == RI_BF16, "row_norm_gate: dtype %d", act_dtype);
    hipStream_t s = (hipStream_t)stream;
    if ((width | out_off | out_stride) % 4 == 0 && (!gate || (g_off | gate_stride) % 4 == 0) && width <= 8192) {
#define RI_VEC(TA, VPT)                                                                                                 \
    row_norm_gate_vec_kernel<TA, VPT><<<rows, 256, 0, s>>>((TA*)out + out_off, out_stride, x, gain, eps,                   \
                                                           gate ? (const TA*)gate + g_off : nullptr, gate_stride, scale,  \
                                                           kind, width)
#define RI_GO(TA)                                                                                                       \
    if (width <= 1024) RI_VEC(TA, 1); else if (width <= 2048) RI_VEC(TA, 2); else if (width <= 4096) RI_VEC(TA, 4);       \
    else RI_VEC(TA, 8)
        if (act_dtype == RI_F32) { RI_GO(float); } else { RI_GO(bf16_t); }
#undef RI_GO
#undef RI_VEC
        RI_LAUNCH_CHECK("row_norm_gate");
        return 0;
    }
    if (act_dtype == RI_F32)
        row_norm_gate_kernel<float><<<rows, 256, 0, s>>>((float*)out + out_off, out_stride, x, gain, eps,
                                                         gate ? (const float*)gate + g_off : nullptr, gate_stride, scale, kind, width);
    else
        row_norm_gate_kernel<bf16_t><<<rows, 256, 0, s>>>((bf16_t*)out + out_off, out_stride, x, gain, eps,
                                                          gate ? (const bf16_t*)gate + g_off : nullptr, gate_stride, scale, kind, width);
    RI_LAUNCH_CHECK("row_norm_gate");
    return 0;
}

// ------------------------------------------------------------------ normed results of mixers side by side, added
// out (+)= a_scale * rms_norm(a) * a_gain + b_scale * rms_norm(b) * b_gain: a and b are the results of two output products,
// each [parts, rows, dim] (the parts added in order) or one part in the activations' format; b may be absent.
// (four parts are asked for together, each from an address that exists, and added in their order)
template <typename T, int VPT>
__device__ __forceinline__ void parts4(float4 (&v)[VPT], const T* x, int parts, size_t stride, size_t row, const int (&at)[VPT]) {
    for (int q0 = 0; q0 < parts; q0 += 4) {
        float4 p[4][VPT];
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int i = 0; i < VPT; ++i) p[j][i] = ld4(x + (size_t)min(q0 + j, parts - 1) * stride + row + at[i]);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const bool live = q0 + j < parts;
#pragma unroll
            for (int i = 0; i < VPT; ++i) {
                v[i].x = live ? v[i].x + p[j][i].x : v[i].x;
                v[i].y = live ? v[i].y + p[j][i].y : v[i].y;
                v[i].z = live ? v[i].z + p[j][i].z : v[i].z;
                v[i].w = live ? v[i].w + p[j][i].w : v[i].w;
            }
        }
    }
}

// Rows of up to 4 THREADS VPT elements in a multiple of 4: both rows in registers, one trip; one workgroup a row, whose threads
// depend on the width alone.
template <typename TX, typename TY, int VPT, int THREADS>
__global__ void __launch_bounds__(THREADS)
normed_sum_vec_kernel(float* __restrict__ out, int accumulate, const TX* __restrict__ a, int a_parts, const float* __restrict__ a_gain,
                      float a_scale, const TY* __restrict__ b, int b_parts, const float* __restrict__ b_gain, float b_scale,
                      float eps, size_t stride, int dim) {
    __shared__ float scratch[16];
    const size_t t = (size_t)blockIdx.x * dim;
    float4 va[VPT], vb[VPT], ga[VPT], gb[VPT];
    int at[VPT];
    bool ok[VPT];
    const float* b_gain_there = b ? b_gain : a_gain;
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        const int c = (threadIdx.x + i * THREADS) * 4;
        ok[i] = c < dim;
        at[i] = ok[i] ? c : 0;
        va[i] = vb[i] = make_float4(0.f, 0.f, 0.f, 0.f);
        ga[i] = ld4(a_gain + at[i]);
        gb[i] = ld4(b_gain_there + at[i]);
    }
    parts4<TX, VPT>(va, a, a_parts, stride, t, at);
    if (b) parts4<TY, VPT>(vb, b, b_parts, stride, t, at);
    float sa = 0.f, sb = 0.f;
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        if (!ok[i]) continue;
        sa += (va[i].x * va[i].x + va[i].y * va[i].y) + (va[i].z * va[i].z + va[i].w * va[i].w);
        sb += (vb[i].x * vb[i].x + vb[i].y * vb[i].y) + (vb[i].z * vb[i].z + vb[i].w * vb[i].w);
    }
    const float fa = a_scale / sqrtf(block_sum(sa, scratch) / (float)dim + eps);
    const float fb = b ? b_scale / sqrtf(block_sum(sb, scratch) / (float)dim + eps) : 0.f;
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
        if (!ok[i]) continue;
        float4 v = make_float4(fa * va[i].x * ga[i].x, fa * va[i].y * ga[i].y, fa * va[i].z * ga[i].z, fa * va[i].w * ga[i].w);
        if (b) v = make_float4(v.x + fb * vb[i].x * gb[i].x, v.y + fb * vb[i].y * gb[i].y, v.z + fb * vb[i].z * gb[i].z,
                               v.w + fb * vb[i].w * gb[i].w);
        if (accumulate) {
            const float4 o = ld4(out + t + at[i]);
            v = make_float4(v.x + o.x, v.y + o.y, v.z + o.z, v.w + o.w);
        }
        st4(out + t + at[i], v);
    }
}

template <typename T>
__device__ __forceinline__ float parts1(const T* x, int parts, size_t stride, size_t at) {
    float v = to_f32(x[at]);
    for (int p = 1; p < parts; ++p) v += to_f32(x[p * stride + at]);
    return v;
}

template <typename TX, typename TY>
__global__ void __launch_bounds__(256)
normed_sum_kernel(float* __restrict__ out, int accumulate, const TX* __restrict__ a, int a_parts, const float* __restrict__ a_gain,
                  float a_scale, const TY* __restrict__ b, int b_parts, const float* __restrict__ b_gain, float b_scale, float eps,
                  size_t stride, int dim) {
    __shared__ float scratch[16];
    const size_t t = (size_t)blockIdx.x * dim;
    float sa = 0.f, sb = 0.f;
    for (int d = threadIdx.x; d < dim; d += blockDim.x) {
        const float x = parts1(a, a_parts, stride, t + d), y = b ? parts1(b, b_parts, stride, t + d) : 0.f;
        sa += x * x;
        sb += y * y;
    }
    const float fa = a_scale / sqrtf(block_sum(sa, scratch) / (float)dim + eps);
    const float fb = b ? b_scale / sqrtf(block_sum(sb, scratch) / (float)dim + eps) : 0.f;
    for (int d = threadIdx.x; d < dim; d += blockDim.x) {
        float v = fa * parts1(a, a_parts, stride, t + d) * a_gain[d];
        if (b) v += fb * parts1(b, b_parts, stride, t + d) * b_gain[d];
        out[t + d] = accumulate ? out[t + d] + v : v;
    }
}

extern "C" int ri_normed_sum(float* out, int accumulate, const void* a, int a_dtype, int a_parts, const float* a_gain, float a_scale,
                             const void* b, int b_dtype, int b_parts, const float* b_gain, float b_scale, float eps, int rows,
                             int dim, void* stream) {
    RI_REQUIRE(out && a && a_gain && rows > 0 && dim > 0 && a_parts >= 1 && (!b || (b_gain && b_parts >= 1)),
               "normed_sum: %d rows of %d, %d and %d parts", rows, dim, a_parts, b_parts);
    RI_REQUIRE((a_dtype == RI_F32 || (a_dtype == RI_BF16 && a_parts == 1)) && (!b || b_dtype == RI_F32 || (b_dtype == RI_BF16 && b_parts == 1)),
               "normed_sum: parts of a product are float32");
    hipStream_t s = (hipStream_t)stream;
    const size_t stride = (size_t)rows * dim;
    const bool vec = dim % 4 == 0 && dim <= 8192;
#define RI_ARGS(TX, TY) out, accumulate, (const TX*)a, a_parts, a_gain, a_scale, (const TY*)b, b_parts, b_gain, b_scale, eps, stride, dim
#define RI_GO(TX, TY)                                                                                       if (!vec) normed_sum_kernel<TX, TY><<<rows, 256, 0, s>>>(RI_ARGS(TX, TY));                               \
    else if (dim <= 1024) normed_sum_vec_kernel<TX, TY, 1, 256><<<rows, 256, 0, s>>>(RI_ARGS(TX, TY));       \
    else if (dim <= 2048) normed_sum_vec_kernel<TX, TY, 1, 512><<<rows, 512, 0, s>>>(RI_ARGS(TX, TY));       \
    else if (dim <= 4096) normed_sum_vec_kernel<TX, TY, 1, 1024><<<rows, 1024, 0, s>>>(RI_ARGS(TX, TY));     \
    else normed_sum_vec_kernel<TX, TY, 2, 1024><<<rows, 1024, 0, s>>>(RI_ARGS(TX, TY))
    if (a_dtype == RI_F32) { if (!b || b_dtype == RI_F32) { RI_GO(float, float); } else { RI_GO(float, bf16_t); } }
    else                   { if (!b || b_dtype == RI_F32) { RI_GO(bf16_t, float); } else { RI_GO(bf16_t, bf16_t); } }
#undef RI_GO
#undef RI_ARGS
    RI_LAUNCH_CHECK("normed_sum");
    return 0;
}
