// The gated delta rule: a mixer that keeps, per sequence and head, a float32 state S of dim x vdim and the last
// inputs of three short convolutions.
//
// Per token, with q and k shared by heads / kv_heads value heads each:
//     x <- silu(causal convolution over time of the projection, per channel)       for q, k and v
//     q <- q / sqrt(sum q^2 + 1e-6) * dim^(-1/2),   k <- k / sqrt(sum k^2 + 1e-6)      per head
//     beta = sigmoid(b),   g = exp(-exp(A_log) * softplus(a + dt_bias))               per value head
//     S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q.
// With a decay per key channel (CH in the kernels) g is a number per head and row of S, g = exp(-exp(A_log_h) *
// softplus(z + dt_bias)) of z [heads * dim], S <- diag(g) S, and the output gate is the sigmoid of a product's float32 result.
// Everything after the projections is float32.  ri_delta_prepare makes q, k, v, g and beta of all tokens of a step
// (a workgroup a token and head), ri_delta_tails then moves the convolutions' last inputs into the sequences' state, and
// ri_delta_scan walks every sequence's tokens in order.  A token's sums are taken in the same order whatever step
// or block of tokens it falls into.
#include "api.h"
#include "common.h"

#define DELTA_MAX_TAPS 16

__device__ __forceinline__ float silu_f(float v) { return v / (1.f + expf(-v)); }
__device__ __forceinline__ float softplus_f(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }

// A token's row of gates: g then beta per head; with CH the decays of every head and the betas, padded to a multiple of 4.
template <bool CH>
__host__ __device__ __forceinline__ int delta_gate_row(int heads, int dim) {
    return CH ? heads * dim + ((heads + 3) & ~3) : 2 * heads;
}

// A workgroup takes one token and one unit of its channels: a q or k head (units 0 .. 2 kv_heads - 1), which it
// norms, or a stretch of DELTA_V_UNIT channels of v.  conv[] (dynamic LDS, max(dim, DELTA_V_UNIT) floats) holds the
// unit's activated convolutions.  (One workgroup a token walked its thousands of channels in turns of 256, each
// turn waiting for its own loads: 22 us for a single token.)
#define DELTA_V_UNIT 256

// CH: ab holds z, rows of z_row elements, the logits of beta are those of bsrc (rows of b_row), and the units behind
// those of v are stretches of DELTA_V_UNIT of the decays; gates is [heads * dim decays, heads betas] a token.
template <typename T, bool CH>
__global__ void __launch_bounds__(256)
delta_prepare_kernel(float* __restrict__ qkv, float* __restrict__ gates, const T* __restrict__ proj, int row, int q_off,
                     const float* __restrict__ taps, int ntaps, const float* __restrict__ tails,
                     const float* __restrict__ ab, const float* __restrict__ a_log, const float* __restrict__ dt_bias,
                     const int32_t* __restrict__ tok_seq, const int32_t* __restrict__ cu_seqlens,
                     const int32_t* __restrict__ slots, int heads, int kv_heads, int dim, int vdim, int z_row,
                     const T* __restrict__ bsrc, int b_row) {
    extern __shared__ float conv[];
    __shared__ float scratch[16];
    const int t = blockIdx.x, unit = blockIdx.y, b = tok_seq[t];
    const int i = t - cu_seqlens[b];                          // the token's place among its sequence's new tokens
    const int qk = kv_heads * dim, channels = 2 * qk + heads * vdim;
    if (CH) {
        const int decays = heads * dim, at = (unit - 2 * kv_heads - (heads * vdim + DELTA_V_UNIT - 1) / DELTA_V_UNIT) * DELTA_V_UNIT;
        float* to = gates + (size_t)t * delta_gate_row<CH>(heads, dim);
        if (at >= 0) {                                        // a stretch of decays (the whole workgroup)
            const int e = at + threadIdx.x;
            if (e < decays) to[e] = expf(-expf(a_log[e / dim]) * softplus_f(ab[(size_t)t * z_row + e] + dt_bias[e]));
            return;
        }
        if (unit == 0)
            for (int h = threadIdx.x; h < heads; h += blockDim.x) to[decays + h] = 1.f / (1.f + expf(-to_f32(bsrc[(size_t)t * b_row + h])));
    }
    const bool normed = unit < 2 * kv_heads;
    const int first = normed ? unit * dim : 2 * qk + (unit - 2 * kv_heads) * DELTA_V_UNIT;
    const int count = normed ? dim : min(DELTA_V_UNIT, channels - first);
    const float* tail = tails + (size_t)slots[b] * (ntaps - 1) * channels;
    if (ntaps <= 4) {
        // the usual few taps: all inputs asked for at once, whatever their place (an address that is not used is
        // pulled back to one that exists), so that no load waits for another
        const float* tail_safe = ntaps > 1 ? tail : taps;
        for (int e = threadIdx.x; e < count; e += blockDim.x) {
            const int c = first + e;
            float x[4], w[4];
#pragma unroll
            for (int d = 0; d < 4; ++d) {
                const int at = i - d;
                const float a = to_f32(proj[(size_t)(t - min(d, i)) * row + q_off + c]);
                const float bb = tail_safe[(size_t)min(max(ntaps - 1 + at, 0), max(ntaps - 2, 0)) * channels + c];
                x[d] = at >= 0 ? a : bb;
                w[d] = d < ntaps ? taps[(size_t)c * ntaps + max(ntaps - 1 - d, 0)] : 0.f;
            }
            float y = 0.f;
#pragma unroll
            for (int d = 3; d >= 0; --d) y += d < ntaps ? w[d] * x[d] : 0.f;           // oldest input first
            conv[e] = silu_f(y);
        }
    } else {
        for (int e = threadIdx.x; e < count; e += blockDim.x) {
            const int c = first + e;
            float y = 0.f;
            for (int d = ntaps - 1; d >= 0; --d) {                // oldest input first
                const int at = i - d;
                const float x = at >= 0 ? to_f32(proj[(size_t)(t - d) * row + q_off + c])
                                        : tail[(size_t)(ntaps - 1 + at) * channels + c];
                y += taps[(size_t)c * ntaps + (ntaps - 1 - d)] * x;
            }
            conv[e] = silu_f(y);
        }
    }
    __syncthreads();
    float* out = qkv + (size_t)t * channels + first;
    if (normed) {                                             // a q head (also times dim^(-1/2)) or a k head
        float ss = 0.f;
        for (int e = threadIdx.x; e < count; e += blockDim.x) ss += conv[e] * conv[e];
        ss = block_sum(ss, scratch);
        const float f = (unit < kv_heads ? rsqrtf((float)dim) : 1.f) / sqrtf(ss + 1e-6f);
        for (int e = threadIdx.x; e < count; e += blockDim.x) out[e] = conv[e] * f;
    } else {
        for (int e = threadIdx.x; e < count; e += blockDim.x) out[e] = conv[e];
    }
    if (!CH && unit == 0 && threadIdx.x < heads) {
        const int h = threadIdx.x;
        const float a = ab[(size_t)t * 2 * heads + h], bb = ab[(size_t)t * 2 * heads + heads + h];
        gates[(size_t)t * 2 * heads + h] = expf(-expf(a_log[h]) * softplus_f(a + dt_bias[h]));
        gates[(size_t)t * 2 * heads + heads + h] = 1.f / (1.f + expf(-bb));
    }
}

// The same for q/k heads whose four-channel pieces are a power of two that divides a wavefront, up to four taps: a thread takes
// four neighbouring channels (or decays) of TT tokens in turn and keeps the inputs before its token in registers, so that a row
// is read once; a head's norm meets over its dim / 4 lanes, without a barrier.  (The form above reads every row once per tap and
// leaves threads idle where a head has fewer channels than a workgroup threads: 64 us against 32 for 2,048 tokens of 8 heads of 128 with their decays.)
__device__ __forceinline__ float4 delta_ld4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 delta_ld4(const bf16_t* p) {
    const uint2 w = *reinterpret_cast<const uint2*>(p);
    return make_float4(__uint_as_float(w.x << 16), __uint_as_float(w.x & 0xFFFF0000u), __uint_as_float(w.y << 16),
                       __uint_as_float(w.y & 0xFFFF0000u));
}

template <typename T, bool CH, int TT>
__global__ void __launch_bounds__(256)
delta_prepare_pieces_kernel(float* __restrict__ qkv, float* __restrict__ gates, const T* __restrict__ proj, int row, int q_off,
                            const float* __restrict__ taps, int ntaps, const float* __restrict__ tails,
                            const float* __restrict__ ab, const float* __restrict__ a_log, const float* __restrict__ dt_bias,
                            const int32_t* __restrict__ tok_seq, const int32_t* __restrict__ cu_seqlens,
                            const int32_t* __restrict__ slots, int heads, int kv_heads, int dim, int vdim, int z_row,
                            const T* __restrict__ bsrc, int b_row, int tokens) {
    const int qk = kv_heads * dim, channels = 2 * qk + heads * vdim, decays = CH ? heads * dim : 0;
    const int pieces = channels / 4, lanes = dim / 4, t0 = blockIdx.y * TT, gate_row = delta_gate_row<CH>(heads, dim);
    if (blockIdx.x == 0) {                                    // a number a head: the betas and, without CH, the decays
        for (int e = threadIdx.x; e < TT * heads; e += 256) {
            const int t = t0 + e / heads, h = e % heads;
            if (t >= tokens) break;
            if (CH) {
                gates[(size_t)t * gate_row + decays + h] = 1.f / (1.f + expf(-to_f32(bsrc[(size_t)t * b_row + h])));
            } else {
                const float a = ab[(size_t)t * 2 * heads + h], bb = ab[(size_t)t * 2 * heads + heads + h];
                gates[(size_t)t * 2 * heads + h] = expf(-expf(a_log[h]) * softplus_f(a + dt_bias[h]));
                gates[(size_t)t * 2 * heads + heads + h] = 1.f / (1.f + expf(-bb));
            }
        }
    }
    const int piece = blockIdx.x * 256 + threadIdx.x;
    if (blockIdx.x * 256 + (threadIdx.x & ~(RI_WAVE - 1)) >= pieces + decays / 4) return;      // whole wavefronts without work leave
    if (piece >= pieces) {                                    // four decays, or nothing
        const int c = (piece - pieces) * 4;
        if (!CH || c >= decays) return;
        const float4 bias = make_float4(dt_bias[c], dt_bias[c + 1], dt_bias[c + 2], dt_bias[c + 3]);
        const float rate = expf(a_log[c / dim]);
        float4 zs[TT];
#pragma unroll
        for (int k = 0; k < TT; ++k) zs[k] = delta_ld4(ab + (size_t)min(t0 + k, tokens - 1) * z_row + c);
#pragma unroll
        for (int k = 0; k < TT; ++k) {
            if (t0 + k >= tokens) break;
            const float4 z = zs[k];
            float* to = gates + (size_t)(t0 + k) * gate_row + c;
            to[0] = expf(-rate * softplus_f(z.x + bias.x));
            to[1] = expf(-rate * softplus_f(z.y + bias.y));
            to[2] = expf(-rate * softplus_f(z.z + bias.z));
            to[3] = expf(-rate * softplus_f(z.w + bias.w));
        }
        return;
    }
    const int c = piece * 4;
    float4 w[4], x[4];                                        // w[d], x[d]: the tap and the input d tokens back
#pragma unroll
    for (int d = 0; d < 4; ++d) {
        const float* p = taps + (size_t)c * ntaps + max(ntaps - 1 - d, 0);
        const float4 v = make_float4(p[0], p[ntaps], p[2 * ntaps], p[3 * ntaps]);
        w[d] = d < ntaps ? v : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    float4 next[TT];                                          // the tokens' own inputs, all asked for at once
#pragma unroll
    for (int k = 0; k < TT; ++k) next[k] = delta_ld4(proj + (size_t)min(t0 + k, tokens - 1) * row + q_off + c);
    int seq[TT], place[TT];                                   // ... and whose they are (the same for the whole workgroup)
#pragma unroll
    for (int k = 0; k < TT; ++k) seq[k] = tok_seq[min(t0 + k, tokens - 1)];
#pragma unroll
    for (int k = 0; k < TT; ++k) place[k] = min(t0 + k, tokens - 1) - cu_seqlens[seq[k]];
    const bool normed = c < 2 * qk;
    const float scale = c < qk ? rsqrtf((float)dim) : 1.f;
#pragma unroll
    for (int k = 0; k < TT; ++k) {
        const int t = t0 + k, i = place[k];
        if (t >= tokens) break;
        if (k == 0 || i == 0) {
            const float* tail = ntaps > 1 ? tails + (size_t)slots[seq[k]] * (ntaps - 1) * channels + c : nullptr;
#pragma unroll
            for (int d = 1; d < 4; ++d) {
                x[d] = make_float4(0.f, 0.f, 0.f, 0.f);
                if (d < ntaps) x[d] = i - d >= 0 ? delta_ld4(proj + (size_t)(t - d) * row + q_off + c) : delta_ld4(tail + (size_t)(ntaps - 1 + i - d) * channels);
            }
        }
        x[0] = next[k];
        float4 y = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int d = 3; d >= 0; --d) {                        // oldest input first
            y.x += w[d].x * x[d].x;
            y.y += w[d].y * x[d].y;
            y.z += w[d].z * x[d].z;
            y.w += w[d].w * x[d].w;
        }
        y = make_float4(silu_f(y.x), silu_f(y.y), silu_f(y.z), silu_f(y.w));
        float ss = (y.x * y.x + y.y * y.y) + (y.z * y.z + y.w * y.w);
        float f = 1.f;
        if (normed) {                                         // (a head's lanes come here together)
            for (int m = lanes / 2; m > 0; m >>= 1) ss += __shfl_xor(ss, m, RI_WAVE);
            f = scale / sqrtf(ss + 1e-6f);
        }
        *reinterpret_cast<float4*>(qkv + (size_t)t * channels + c) = make_float4(y.x * f, y.y * f, y.z * f, y.w * f);
#pragma unroll
        for (int d = 3; d > 0; --d) x[d] = x[d - 1];
    }
}

// The last ntaps - 1 inputs of every sequence after this step's n tokens: row r of the new tail is entry n + r of
// (old tail, then the step's inputs).  One thread a (sequence, channel): it reads all it needs before it writes.
template <typename T>
__global__ void __launch_bounds__(256)
delta_tails_kernel(float* __restrict__ tails, const T* __restrict__ proj, int row, int q_off, int ntaps,
                   const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ slots, int channels) {
    const int b = blockIdx.y, c = blockIdx.x * blockDim.x + threadIdx.x;
    if (c >= channels) return;
    const int t0 = cu_seqlens[b], n = cu_seqlens[b + 1] - t0, keep = ntaps - 1;
    float* tail = tails + (size_t)slots[b] * keep * channels;
    float v[DELTA_MAX_TAPS];
    for (int r = 0; r < keep; ++r) {
        const int at = n + r;                                 // place in (old tail, new inputs)
        v[r] = at < keep ? tail[(size_t)at * channels + c] : to_f32(proj[(size_t)(t0 + at - keep) * row + q_off + c]);
    }
    for (int r = 0; r < keep; ++r) tail[(size_t)r * channels + c] = v[r];
}

// The sum over the four lanes of a quad, in each of them, by two quad permutations of the vector unit's own data
// path (DPP): [1, 0, 3, 2] then [2, 3, 0, 1].  A shuffle goes through the LDS crossbar instead, and the walk waits
// for four of them in a row at every token.
__device__ __forceinline__ float quad_sum(float v) {
    v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xB1, 0xF, 0xF, true));
    v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x4E, 0xF, 0xF, true));
    return v;
}

// The same over the SL = 4, 8 or 16 lanes of a column: after the quads, the mirror image inside every eight lanes
// (lane i takes lane 7 - i: the other quad, all of whose lanes hold its sum), then inside every sixteen.
template <int SL>
__device__ __forceinline__ float slices_sum(float v) {
    v = quad_sum(v);
    if (SL >= 8) v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x141, 0xF, 0xF, true));
    if (SL == 16) v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x140, 0xF, 0xF, true));
    return v;
}

// The walk.  A workgroup owns one (sequence, value head) and 256 / SL columns of its state: that many columns x SL
// slices of rows (4 or 8); a thread keeps RPT rows of one column in registers (rows r * RPT ..+RPT of slice r; rows
// past dim are zeros that stay zeros).  Tokens come through LDS in blocks of DELTA_BLOCK, the next block's loads in
// flight while a block is walked.  The two sums over rows of a token meet over the SL lanes of a column.  A token costs
// a wavefront 4 RPT vector instructions and nothing hides them, so eight slices halve a token's time; they also
// double the workgroups that each stage q and k, which is what counts once the machine is full: the launch chooses.
template <int RPT, int SL, bool CH>
struct DeltaLds {
    static constexpr int DELTA_BLOCK = RPT * SL >= (CH ? 128 : 256) ? 8 : 16;    // tokens a block: two buffers stay inside 64 KB
    static constexpr int QS = RPT + 4;                        // stride of a slice of q or k: no bank conflicts between the slices
    static constexpr int COLS = 256 / SL;
    float q[DELTA_BLOCK][SL][QS];
    float k[DELTA_BLOCK][SL][QS];
    float v[DELTA_BLOCK][COLS];
    float g[CH ? 1 : DELTA_BLOCK], beta[DELTA_BLOCK];
    float gk[CH ? DELTA_BLOCK : 1][SL][CH ? QS : 1];          // a decay a row
};

template <int RPT, int SL, bool CH>
__global__ void __launch_bounds__(256)
delta_scan_kernel(float* __restrict__ out, const float* __restrict__ qkv, const float* __restrict__ gates,
                  float* __restrict__ state, const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ slots,
                  int heads, int kv_heads, int dim, int vdim) {
    __shared__ DeltaLds<RPT, SL, CH> lds[2];
    constexpr int DELTA_BLOCK = DeltaLds<RPT, SL, CH>::DELTA_BLOCK, COLS = DeltaLds<RPT, SL, CH>::COLS;
    constexpr int QR = DELTA_BLOCK * SL * RPT / 256;          // elements of q (and of k) a thread fetches per block
    constexpr int VR = DELTA_BLOCK * COLS / 256;
    const int b = blockIdx.x / heads, h = blockIdx.x % heads, col0 = blockIdx.y * COLS;
    const int hq = h / (heads / kv_heads);
    const int tid = threadIdx.x, r = tid & (SL - 1), col = col0 + tid / SL;
    const bool has_col = col < vdim;
    const int t0 = cu_seqlens[b], n = cu_seqlens[b + 1] - t0;
    if (n <= 0) return;
    const int qk = kv_heads * dim, channels = 2 * qk + heads * vdim;
    float* st = state + (((size_t)slots[b] * heads + h) * dim) * vdim;

    float S[RPT];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        // (no load in a branch: the address is pulled back inside the state and the value dropped afterwards)
        const int rw = r * RPT + i;
        const float v = st[(size_t)min(rw, dim - 1) * vdim + min(col, vdim - 1)];
        S[i] = (has_col && rw < dim) ? v : 0.f;
    }

    const int gate_row = delta_gate_row<CH>(heads, dim);
    float fq[QR], fk[QR], fgk[CH ? QR : 1], fv[VR], fg = 0.f;
    auto fetch = [&](int first) {                             // the block of tokens first ..+DELTA_BLOCK, into registers
#pragma unroll
        for (int e = 0; e < QR; ++e) {
            const int at = e * 256 + tid, tk = at / (SL * RPT), rw = at % (SL * RPT);
            const bool ok = first + tk < n && rw < dim;
            const float* p = qkv + (size_t)(t0 + min(first + tk, n - 1)) * channels + (size_t)hq * dim + min(rw, dim - 1);
            const float a = p[0], c = p[qk];
            fq[e] = ok ? a : 0.f;
            fk[e] = ok ? c : 0.f;
            if (CH) fgk[e] = gates[(size_t)(t0 + min(first + tk, n - 1)) * gate_row + h * dim + min(rw, dim - 1)];
        }
#pragma unroll
        for (int e = 0; e < VR; ++e) {
            const int at = e * 256 + tid, tk = at / COLS, cc = col0 + at % COLS;
            const float a = qkv[(size_t)(t0 + min(first + tk, n - 1)) * channels + 2 * qk + (size_t)h * vdim + min(cc, vdim - 1)];
            fv[e] = a;
        }
        if (tid < 2 * DELTA_BLOCK) {
            const int tk = tid >> 1;
            fg = gates[(size_t)(t0 + min(first + tk, n - 1)) * gate_row + (CH ? heads * dim : (tid & 1) * heads) + h];
        }
    };
    auto stage = [&](DeltaLds<RPT, SL, CH>& l) {
#pragma unroll
        for (int e = 0; e < QR; ++e) {
            const int at = e * 256 + tid, tk = at / (SL * RPT), rw = at % (SL * RPT);
            l.q[tk][rw / RPT][rw % RPT] = fq[e];
            l.k[tk][rw / RPT][rw % RPT] = fk[e];
            if (CH) l.gk[tk][rw / RPT][rw % RPT] = fgk[e];
        }
#pragma unroll
        for (int e = 0; e < VR; ++e) {
            const int at = e * 256 + tid;
            l.v[at / COLS][at % COLS] = fv[e];
        }
        if (tid < 2 * DELTA_BLOCK) {
            if (tid & 1) l.beta[tid >> 1] = fg; else if (!CH) l.g[tid >> 1] = fg;
        }
    };

    fetch(0);
    stage(lds[0]);
    __syncthreads();
    int cur = 0;
    for (int first = 0; first < n; first += DELTA_BLOCK) {
        const bool more = first + DELTA_BLOCK < n;
        fetch(more ? first + DELTA_BLOCK : first);            // (always issued: no load in a branch)
        const DeltaLds<RPT, SL, CH>& l = lds[cur];
        const int count = min(DELTA_BLOCK, n - first);
#pragma unroll 2
        for (int tk = 0; tk < count; ++tk) {
            const float g = CH ? 1.f : l.g[tk], beta = l.beta[tk];
            // four partial sums each: a single one would be a chain of RPT dependent additions
            float kk[RPT], d4[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int i = 0; i < RPT; ++i) {
                kk[i] = l.k[tk][r][i];
                S[i] *= CH ? l.gk[tk][r][i] : g;
                d4[i & 3] += S[i] * kk[i];
            }
            const float dot = slices_sum<SL>((d4[0] + d4[1]) + (d4[2] + d4[3]));
            const float u = beta * (l.v[tk][tid / SL] - dot);
            float o4[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int i = 0; i < RPT; ++i) {
                S[i] += kk[i] * u;
                o4[i & 3] += S[i] * l.q[tk][r][i];
            }
            const float o = slices_sum<SL>((o4[0] + o4[1]) + (o4[2] + o4[3]));
            if (r == 0 && has_col) out[(size_t)(t0 + first + tk) * heads * vdim + (size_t)h * vdim + col] = o;
        }
        stage(lds[cur ^ 1]);
        __syncthreads();
        cur ^= 1;
    }
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int rw = r * RPT + i;
        if (has_col && rw < dim) st[(size_t)rw * vdim + col] = S[i];
    }
}

// The walk of a launch of few heads: a workgroup is one wavefront with four columns and sixteen slices of rows, so that a head of
// 128 columns is 32 workgroups, each on a vector unit of its own, and a token costs 5 RPT vector instructions of one wavefront.
// What the chain from token to token waits for is short: with S' = g S, both sums of a token run over S' side by side (S'^T k
// and S'^T q, beside k . q), then u = beta (v - S'^T k) and o = S'^T q + (k . q) u, and S = S' + k u is ready for the next token
// without a sum of its own.  q, k and the decays come in 16-byte pieces (dim and the rows a multiple of 4), a block of tokens at a
// time, the next block's in flight; a token's values are read from LDS while the token before it is walked.  A block's results
// wait in LDS and leave before the next loads are asked for: a store among the walk's tokens would be waited for with those loads.
template <int RPT, bool CH>
struct DeltaToken {
    float k[RPT], q[RPT], gk[CH ? RPT : 1], g, beta, v;
};

template <int RPT, bool CH>
__global__ void __launch_bounds__(64)
delta_scan_narrow_kernel(float* __restrict__ out, const float* __restrict__ qkv, const float* __restrict__ gates,
                         float* __restrict__ state, const int32_t* __restrict__ cu_seqlens, const int32_t* __restrict__ slots,
                         int heads, int kv_heads, int dim, int vdim) {
    constexpr int B = RPT <= 8 ? 16 : 8, SL = 16, COLS = 4, PIECES = SL * RPT / 4, PR = B * PIECES / 64, QS = RPT + 4;
    __shared__ __attribute__((aligned(16))) float lq[B][SL][QS], lk[B][SL][QS], lg[CH ? B : 1][SL][CH ? QS : 4];
    __shared__ float lv[B][COLS], lo[B][COLS], lbeta[B], lgs[B];
    const int b = blockIdx.x / heads, h = blockIdx.x % heads, col0 = blockIdx.y * COLS, hq = h / (heads / kv_heads);
    const int tid = threadIdx.x, r = tid & (SL - 1), mine = tid / SL, col = col0 + mine;
    const bool has_col = col < vdim;
    const int t0 = cu_seqlens[b], n = cu_seqlens[b + 1] - t0;
    if (n <= 0) return;
    const int qk = kv_heads * dim, channels = 2 * qk + heads * vdim, gate_row = delta_gate_row<CH>(heads, dim);
    float* st = state + (((size_t)slots[b] * heads + h) * dim) * vdim;

    float S[RPT];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int rw = r * RPT + i;
        const float v = st[(size_t)min(rw, dim - 1) * vdim + min(col, vdim - 1)];
        S[i] = (has_col && rw < dim) ? v : 0.f;
    }

    float4 fq[PR], fk[PR], fg[CH ? PR : 1];
    float fv, fbeta, fgs = 0.f;
    auto fetch = [&](int first) {                             // the block of tokens first ..+B, into registers
#pragma unroll
        for (int e = 0; e < PR; ++e) {
            const int at = e * 64 + tid, tk = at / PIECES, rw = (at % PIECES) * 4;
            const int t = t0 + min(first + tk, n - 1), row = min(rw, dim - 4);
            const float* p = qkv + (size_t)t * channels + hq * dim + row;
            fq[e] = delta_ld4(p);
            fk[e] = delta_ld4(p + qk);
            if (CH) fg[e] = delta_ld4(gates + (size_t)t * gate_row + h * dim + row);
        }
        const int vt = t0 + min(first + (tid & (B * COLS - 1)) / COLS, n - 1);
        fv = qkv[(size_t)vt * channels + 2 * qk + h * vdim + min(col0 + tid % COLS, vdim - 1)];
        const float* gp = gates + (size_t)(t0 + min(first + (tid & (B - 1)), n - 1)) * gate_row + (CH ? heads * dim : heads) + h;
        fbeta = gp[0];
        if (!CH) fgs = gp[-heads];
    };
    auto stage = [&]() {
#pragma unroll
        for (int e = 0; e < PR; ++e) {
            const int at = e * 64 + tid, tk = at / PIECES, rw = (at % PIECES) * 4;
            const bool ok = rw < dim;                         // rows past dim: a state of zeros that stays so
            // (component by component: a choice between whole structures would put the arrays into memory)
            auto kept = [&](const float4& v) { return make_float4(ok ? v.x : 0.f, ok ? v.y : 0.f, ok ? v.z : 0.f, ok ? v.w : 0.f); };
            *reinterpret_cast<float4*>(&lq[tk][rw / RPT][rw % RPT]) = kept(fq[e]);
            *reinterpret_cast<float4*>(&lk[tk][rw / RPT][rw % RPT]) = kept(fk[e]);
            if (CH) *reinterpret_cast<float4*>(&lg[tk][rw / RPT][rw % RPT]) = kept(fg[e]);
        }
        if (tid < B * COLS) lv[tid / COLS][tid % COLS] = fv;
        if (tid < B) {
            lbeta[tid] = fbeta;
            if (!CH) lgs[tid] = fgs;
        }
    };
    typedef DeltaToken<RPT, CH> Token;
    auto read = [&](Token& x, int tk) {
#pragma unroll
        for (int i = 0; i < RPT; i += 4) {
            const float4 k = delta_ld4(&lk[tk][r][i]), q = delta_ld4(&lq[tk][r][i]);
            x.k[i] = k.x; x.k[i + 1] = k.y; x.k[i + 2] = k.z; x.k[i + 3] = k.w;
            x.q[i] = q.x; x.q[i + 1] = q.y; x.q[i + 2] = q.z; x.q[i + 3] = q.w;
            if (CH) {
                const float4 g = delta_ld4(&lg[tk][r][i]);
                x.gk[i] = g.x; x.gk[i + 1] = g.y; x.gk[i + 2] = g.z; x.gk[i + 3] = g.w;
            }
        }
        x.g = CH ? 1.f : lgs[tk];
        x.beta = lbeta[tk];
        x.v = lv[tk][mine];
    };
    auto walk = [&](const Token& x, int tk) {
        float a[2] = {0.f, 0.f}, o[2] = {0.f, 0.f}, c[2] = {0.f, 0.f};
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
            S[i] *= CH ? x.gk[i] : x.g;
            a[i & 1] += S[i] * x.k[i];
            o[i & 1] += S[i] * x.q[i];
            c[i & 1] += x.k[i] * x.q[i];
        }
        const float sa = slices_sum<16>(a[0] + a[1]), so = slices_sum<16>(o[0] + o[1]), sc = slices_sum<16>(c[0] + c[1]);
        const float u = x.beta * (x.v - sa);
#pragma unroll
        for (int i = 0; i < RPT; ++i) S[i] += x.k[i] * u;
        if (r == 0) lo[tk][mine] = so + sc * u;
    };
    auto hand_on = [&](int first, int count) {                // the results of a block that was walked
        if (tid < count * COLS && col0 + tid % COLS < vdim)
            out[(size_t)(t0 + first + tid / COLS) * heads * vdim + (size_t)h * vdim + col0 + tid % COLS] = lo[tid / COLS][tid % COLS];
    };

    fetch(0);
    for (int first = 0; first < n; first += B) {
        stage();
        if (first > 0) hand_on(first - B, B);
        __syncthreads();                                      // (one wavefront: what it wrote is in place)
        const int count = min(B, n - first);
        fetch(first + B < n ? first + B : first);             // (always issued: no load in a branch)
        Token x, y;
        read(x, 0);
        for (int tk = 0; tk < count; tk += 2) {               // (the last token's successor is read from its own place and not used)
            read(y, min(tk + 1, B - 1));
            walk(x, tk);
            read(x, min(tk + 2, B - 1));
            if (tk + 1 < count) walk(y, tk + 1);
        }
        __syncthreads();
    }
    hand_on((n - 1) / B * B, (n - 1) % B + 1);
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int rw = r * RPT + i;
        if (has_col && rw < dim) st[(size_t)rw * vdim + col] = S[i];
    }
}

// One new token a sequence: the convolutions, the unit norms, the gates, the step on the state, the per-head norm
// and the output gate in one kernel.  A workgroup owns one (sequence, head): `groups` threads across a row of the
// state, four columns each (16-byte loads and stores of whole lines), x 256 / groups slices of rows, a thread RPT rows
// in registers.  The sums over rows meet through LDS, slice after slice.  The convolutions' tails are read here and
// moved on by delta_tails_kernel afterwards (the heads that share a q/k head all read its tail).
// CH: ab holds z (rows of z_row elements, the gate's pre-activations from column gate_at of them on), the logits of beta
// are those of bsrc, the gate is a sigmoid.
template <typename T, int RPT, bool CH>
__global__ void __launch_bounds__(256)
delta_step_kernel(T* __restrict__ out, const T* __restrict__ proj, int row, int q_off, int g_off,
                  const float* __restrict__ taps, int ntaps, const float* __restrict__ tails, const float* __restrict__ ab,
                  const float* __restrict__ a_log, const float* __restrict__ dt_bias, float* __restrict__ state,
                  const int32_t* __restrict__ slots, const float* __restrict__ gain, float eps, int heads, int kv_heads,
                  int dim, int vdim, int groups, int z_row, int gate_at, const T* __restrict__ bsrc, int b_row) {
    __shared__ float qs[256], ks[256], vs[256], gs[CH ? 256 : 1], scratch[16];
    __shared__ float4 part[256];
    const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
    const int hq = h / (heads / kv_heads), slot = slots[b];
    const int grp = tid % groups, r = tid / groups, slices = 256 / groups, c0 = grp * 4;
    const bool has_col = c0 < vdim;                           // vdim is a multiple of 4: all four columns or none
    const int qk = kv_heads * dim, channels = 2 * qk + heads * vdim;
    float* st = state + (((size_t)slot * heads + h) * dim) * vdim;
    float4 S[RPT];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        // (no load in a branch: the address is pulled back inside the state and the value dropped afterwards)
        const int rw = r * RPT + i;
        const float4 v = *reinterpret_cast<const float4*>(st + (size_t)min(rw, dim - 1) * vdim + min(c0, vdim - 4));
        S[i] = (has_col && rw < dim) ? v : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    const T* x = proj + (size_t)b * row;
    const float* tail = tails + (size_t)slot * (ntaps - 1) * channels;
    // everything the end of the kernel reads from memory is asked for here, so that no load is waited for on its own
    const float* zr = ab + (size_t)b * (CH ? z_row : 2 * heads);
    const float a_in = CH ? 0.f : zr[h], b_in = CH ? to_f32(bsrc[(size_t)b * b_row + h]) : zr[heads + h];
    const float a_exp = a_log[h], a_bias = CH ? 0.f : dt_bias[h];
    float gate[4], gain_c[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        gate[j] = CH ? zr[gate_at + h * vdim + min(c0, vdim - 4) + j] : to_f32(x[g_off + h * vdim + min(c0, vdim - 4) + j]);
        gain_c[j] = gain[min(c0, vdim - 4) + j];
    }
    if (CH && tid < dim) gs[tid] = expf(-expf(a_exp) * softplus_f(zr[h * dim + tid] + dt_bias[h * dim + tid]));      // (dim <= 256)
    for (int e = tid; e < 2 * dim + vdim; e += 256) {
        const int ch = e < dim ? hq * dim + e : e < 2 * dim ? qk + hq * dim + (e - dim) : 2 * qk + h * vdim + (e - 2 * dim);
        float y = 0.f;
        if (ntaps <= 4) {                                     // the usual few taps: every load asked for before any is used
            const float* tail_safe = ntaps > 1 ? tail : taps;
            float xv[3], wv[3];
#pragma unroll
            for (int d = 1; d <= 3; ++d) {
                xv[d - 1] = tail_safe[(size_t)max(ntaps - 1 - d, 0) * channels + ch];
                wv[d - 1] = taps[(size_t)ch * ntaps + max(ntaps - 1 - d, 0)];
            }
            const float w0 = taps[(size_t)ch * ntaps + ntaps - 1], x0 = to_f32(x[q_off + ch]);
#pragma unroll
            for (int d = 3; d >= 1; --d) y += d < ntaps ? wv[d - 1] * xv[d - 1] : 0.f;
            y += w0 * x0;
        } else {
            for (int d = ntaps - 1; d >= 1; --d) y += taps[(size_t)ch * ntaps + (ntaps - 1 - d)] * tail[(size_t)(ntaps - 1 - d) * channels + ch];
            y += taps[(size_t)ch * ntaps + ntaps - 1] * to_f32(x[q_off + ch]);
        }
        const float a = silu_f(y);
        if (e < dim) qs[e] = a; else if (e < 2 * dim) ks[e - dim] = a; else vs[e - 2 * dim] = a;
    }
    __syncthreads();
    float sq = 0.f, sk = 0.f;
    for (int e = tid; e < dim; e += 256) {
        sq += qs[e] * qs[e];
        sk += ks[e] * ks[e];
    }
    sq = block_sum(sq, scratch);
    sk = block_sum(sk, scratch);
    const float fq = rsqrtf((float)dim) / sqrtf(sq + 1e-6f), fk = 1.f / sqrtf(sk + 1e-6f);
    const float g_head = CH ? 1.f : expf(-expf(a_exp) * softplus_f(a_in + a_bias));
    const float beta = 1.f / (1.f + expf(-b_in));
    float kk[RPT];
    float4 d = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int rw = r * RPT + i;
        kk[i] = rw < dim ? ks[rw] * fk : 0.f;
        const float g = CH ? gs[min(rw, dim - 1)] : g_head;
        S[i].x *= g; S[i].y *= g; S[i].z *= g; S[i].w *= g;
        d.x += S[i].x * kk[i]; d.y += S[i].y * kk[i]; d.z += S[i].z * kk[i]; d.w += S[i].w * kk[i];
    }
    part[tid] = d;
    __syncthreads();
    float4 dot = make_float4(0.f, 0.f, 0.f, 0.f);
    for (int j = 0; j < slices; ++j) {                        // slice after slice: the same order for every column
        const float4 p = part[j * groups + grp];
        dot.x += p.x; dot.y += p.y; dot.z += p.z; dot.w += p.w;
    }
    const int cv = min(c0, vdim - 4);
    const float4 u = make_float4(beta * (vs[cv] - dot.x), beta * (vs[cv + 1] - dot.y), beta * (vs[cv + 2] - dot.z),
                                 beta * (vs[cv + 3] - dot.w));
    __syncthreads();                                          // part is written again
    float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int rw = r * RPT + i;
        const float qq = rw < dim ? qs[rw] * fq : 0.f;
        S[i].x += kk[i] * u.x; S[i].y += kk[i] * u.y; S[i].z += kk[i] * u.z; S[i].w += kk[i] * u.w;
        o.x += S[i].x * qq; o.y += S[i].y * qq; o.z += S[i].z * qq; o.w += S[i].w * qq;
        if (has_col && rw < dim) *reinterpret_cast<float4*>(st + (size_t)rw * vdim + c0) = S[i];
    }
    part[tid] = o;
    __syncthreads();
    o = make_float4(0.f, 0.f, 0.f, 0.f);
    for (int j = 0; j < slices; ++j) {
        const float4 p = part[j * groups + grp];
        o.x += p.x; o.y += p.y; o.z += p.z; o.w += p.w;
    }
    const float ss = block_sum((r == 0 && has_col) ? (o.x * o.x + o.y * o.y) + (o.z * o.z + o.w * o.w) : 0.f, scratch);
    if (r == 0 && has_col) {
        const float inv = 1.f / sqrtf(ss / (float)vdim + eps);
        T* to = out + (size_t)b * heads * vdim + (size_t)h * vdim + c0;
        auto open = [](float z) { return CH ? 1.f / (1.f + expf(-z)) : silu_f(z); };
        from_f32(to, o.x * inv * gain_c[0] * open(gate[0]));
        from_f32(to + 1, o.y * inv * gain_c[1] * open(gate[1]));
        from_f32(to + 2, o.z * inv * gain_c[2] * open(gate[2]));
        from_f32(to + 3, o.w * inv * gain_c[3] * open(gate[3]));
    }
}

static int delta_step_cols(int vdim) {
    int cols = 32;
    while (cols < vdim) cols *= 2;
    return cols;
}

extern "C" int ri_delta_step_fits(int dim, int vdim) {
    if (dim < 1 || dim > 256 || vdim < 4 || vdim > 256 || vdim % 4) return 0;
    const int slices = 256 / (delta_step_cols(vdim) / 4);
    return (dim + slices - 1) / slices <= 16;
}

template <bool CH>
static int launch_delta_step(void* out, const void* proj, int act_dtype, int row, int q_off, int g_off, const float* taps,
                             int ntaps, float* tails, const float* ab, const float* a_log, const float* dt_bias,
                             float* state, const int32_t* cu_seqlens, const int32_t* slots, const float* gain, float eps,
                             int seqs, int heads, int kv_heads, int dim, int vdim, int z_row, int gate_at, const void* bsrc,
                             int b_row, void* stream) {
    RI_REQUIRE(seqs > 0 && seqs <= 65535 && heads > 0 && heads <= 65535 && kv_heads > 0 && heads % kv_heads == 0,
               "delta_step: %d sequences, %d heads, %d kv heads", seqs, heads, kv_heads);
    RI_REQUIRE(ri_delta_step_fits(dim, vdim), "delta_step: heads of %d x %d", dim, vdim);
    RI_REQUIRE(ntaps >= 1 && ntaps <= DELTA_MAX_TAPS, "delta_step: %d taps, the kernels take 1 to %d", ntaps, DELTA_MAX_TAPS);
    const long channels = 2L * kv_heads * dim + (long)heads * vdim;
    RI_REQUIRE(q_off >= 0 && q_off + channels <= row && (CH || (g_off >= 0 && g_off + (long)heads * vdim <= row)),
               "delta_step: %ld channels at column %d and the gate at %d of rows of %d", channels, q_off, g_off, row);
    RI_REQUIRE(act_dtype == RI_F32 || act_dtype == RI_BF16, "delta_step: dtype %d", act_dtype);
    hipStream_t s = (hipStream_t)stream;
    const int groups = delta_step_cols(vdim) / 4, slices = 256 / groups, rpt = (dim + slices - 1) / slices;
    const dim3 grid(heads, seqs);
#define RI_DSTEP_GO(T, R) delta_step_kernel<T, R, CH><<<grid, 256, 0, s>>>((T*)out, (const T*)proj, row, q_off, g_off, taps, ntaps, \
                                                                    tails, ab, a_log, dt_bias, state, slots, gain, eps, heads,   \
                                                                    kv_heads, dim, vdim, groups, z_row, gate_at, (const T*)bsrc, b_row)
    if (act_dtype == RI_F32) {
        if (rpt <= 4) RI_DSTEP_GO(float, 4); else if (rpt <= 8) RI_DSTEP_GO(float, 8); else RI_DSTEP_GO(float, 16);
    } else {
        if (rpt <= 4) RI_DSTEP_GO(bf16_t, 4); else if (rpt <= 8) RI_DSTEP_GO(bf16_t, 8); else RI_DSTEP_GO(bf16_t, 16);
    }
#undef RI_DSTEP_GO
    RI_LAUNCH_CHECK("delta_step");
    if (ntaps > 1) {
        const dim3 tgrid((unsigned)((channels + 255) / 256), seqs);
        if (act_dtype == RI_F32)
            delta_tails_kernel<float><<<tgrid, 256, 0, s>>>(tails, (const float*)proj, row, q_off, ntaps, cu_seqlens, slots, (int)channels);
        else
            delta_tails_kernel<bf16_t><<<tgrid, 256, 0, s>>>(tails, (const bf16_t*)proj, row, q_off, ntaps, cu_seqlens, slots, (int)channels);
        RI_LAUNCH_CHECK("delta_tails");
    }
    return 0;
}

extern "C" int ri_delta_step(void* out, const void* proj, int act_dtype, int row, int q_off, int g_off, const float* taps,
                             int ntaps, float* tails, const float* ab, const float* a_log, const float* dt_bias,
                             float* state, const int32_t* cu_seqlens, const int32_t* slots, const float* gain, float eps,
                             int seqs, int heads, int kv_heads, int dim, int vdim, void* stream) {
    return launch_delta_step<false>(out, proj, act_dtype, row, q_off, g_off, taps, ntaps, tails, ab, a_log, dt_bias, state,
                                    cu_seqlens, slots, gain, eps, seqs, heads, kv_heads, dim, vdim, 0, 0, nullptr, 0, stream);
}

// Rows of pre-activations of a decay per key channel: what both entry points below ask of them.
static int check_channels(const char* name, const void* z, int z_row, const void* b, int b_row, int heads, int dim) {
    RI_REQUIRE(z && b && z_row >= heads * dim && b_row >= heads, "%s: decays in rows of %d, betas in rows of %d for %d heads of %d", name,
               z_row, b_row, heads, dim);
    return 0;
}

extern "C" int ri_delta_step_channels(void* out, const void* proj, int act_dtype, int row, int q_off, const float* taps, int ntaps,
                                      float* tails, const float* z, int z_row, int gate_at, const void* b, int b_row,
                                      const float* a_log, const float* dt_bias, float* state, const int32_t* cu_seqlens,
                                      const int32_t* slots, const float* gain, float eps, int seqs, int heads, int kv_heads,
                                      int dim, int vdim, void* stream) {
    if (check_channels("delta_step_channels", z, z_row, b, b_row, heads, dim)) return 1;
    RI_REQUIRE(gate_at >= 0 && gate_at + (long)heads * vdim <= z_row, "delta_step_channels: the gate at %d of rows of %d", gate_at, z_row);
    return launch_delta_step<true>(out, proj, act_dtype, row, q_off, 0, taps, ntaps, tails, z, a_log, dt_bias, state, cu_seqlens,
                                   slots, gain, eps, seqs, heads, kv_heads, dim, vdim, z_row, gate_at, b, b_row, stream);
}

template <bool CH>
static int launch_delta_prepare(float* qkv, float* gates, const void* proj, int act_dtype, int row, int q_off,
                                const float* taps, int ntaps, float* tails, const float* ab, const float* a_log,
                                const float* dt_bias, const int32_t* tok_seq, const int32_t* cu_seqlens,
                                const int32_t* slots, int seqs, int tokens, int heads, int kv_heads, int dim, int vdim,
                                int z_row, const void* bsrc, int b_row, void* stream) {
    RI_REQUIRE(tokens > 0 && seqs > 0 && heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && vdim > 0,
               "delta_prepare: tokens %d, sequences %d, heads %d, kv heads %d of %d x %d", tokens, seqs, heads, kv_heads,
               dim, vdim);
    RI_REQUIRE(CH || heads <= 256, "delta_prepare: %d heads, the kernel takes up to 256", heads);
    RI_REQUIRE(ntaps >= 1 && ntaps <= DELTA_MAX_TAPS, "delta_prepare: %d taps, the kernels take 1 to %d", ntaps, DELTA_MAX_TAPS);
    const long channels = 2L * kv_heads * dim + (long)heads * vdim;
    RI_REQUIRE(q_off >= 0 && q_off + channels <= row, "delta_prepare: %ld channels at column %d of rows of %d", channels, q_off, row);
    RI_REQUIRE(dim <= 8192, "delta_prepare: heads of %d exceed the workgroup's memory", dim);
    RI_REQUIRE(act_dtype == RI_F32 || act_dtype == RI_BF16, "delta_prepare: dtype %d", act_dtype);
    hipStream_t s = (hipStream_t)stream;
    const size_t shared = (size_t)(dim > DELTA_V_UNIT ? dim : DELTA_V_UNIT) * sizeof(float);
    const int units = 2 * kv_heads + (heads * vdim + DELTA_V_UNIT - 1) / DELTA_V_UNIT + (CH ? (heads * dim + DELTA_V_UNIT - 1) / DELTA_V_UNIT : 0);
    RI_REQUIRE(units <= 65535, "delta_prepare: %d units of channels exceed one launch", units);
    const dim3 pgrid(tokens, units);
    const int lanes = dim / 4;
    // (the form depends on the sizes alone, so that a token's sums are the same in every step)
    const bool in_pieces = dim % 4 == 0 && lanes <= RI_WAVE && (lanes & (lanes - 1)) == 0 && ntaps <= 4 && (heads * vdim) % 4 == 0 &&
                           (row | q_off) % 4 == 0 && (uintptr_t)proj % 16 == 0 && (uintptr_t)tails % 16 == 0 &&
                           (!CH || (z_row % 4 == 0 && (uintptr_t)ab % 16 == 0));
    if (in_pieces) {
        const int pieces = (int)(channels + (CH ? (long)heads * dim : 0)) / 4, tt = tokens >= 1024 ? 8 : 2;
        const dim3 grid((pieces + 255) / 256, (tokens + tt - 1) / tt);
        RI_REQUIRE((tokens + tt - 1) / tt <= 65535, "delta_prepare: %d tokens exceed one launch", tokens);
#define RI_GO(T, TT)                                                                                                            \
    delta_prepare_pieces_kernel<T, CH, TT><<<grid, 256, 0, s>>>(qkv, gates, (const T*)proj, row, q_off, taps, ntaps, tails, ab,  \
                                                                a_log, dt_bias, tok_seq, cu_seqlens, slots, heads, kv_heads, dim, \
                                                                vdim, z_row, (const T*)bsrc, b_row, tokens)
        if (act_dtype == RI_F32) { if (tt == 8) RI_GO(float, 8); else RI_GO(float, 2); }
        else                     { if (tt == 8) RI_GO(bf16_t, 8); else RI_GO(bf16_t, 2); }
#undef RI_GO
    } else if (act_dtype == RI_F32) {
        delta_prepare_kernel<float, CH><<<pgrid, 256, shared, s>>>(qkv, gates, (const float*)proj, row, q_off, taps, ntaps, tails,
                                                                   ab, a_log, dt_bias, tok_seq, cu_seqlens, slots, heads,
                                                                   kv_heads, dim, vdim, z_row, (const float*)bsrc, b_row);
    } else {
        delta_prepare_kernel<bf16_t, CH><<<pgrid, 256, shared, s>>>(qkv, gates, (const bf16_t*)proj, row, q_off, taps, ntaps,
                                                                    tails, ab, a_log, dt_bias, tok_seq, cu_seqlens, slots,
                                                                    heads, kv_heads, dim, vdim, z_row, (const bf16_t*)bsrc, b_row);
    }
    RI_LAUNCH_CHECK("delta_prepare");
    if (ntaps > 1) {
        const dim3 grid((unsigned)((channels + 255) / 256), seqs);
        if (act_dtype == RI_F32)
            delta_tails_kernel<float><<<grid, 256, 0, s>>>(tails, (const float*)proj, row, q_off, ntaps, cu_seqlens, slots, (int)channels);
        else
            delta_tails_kernel<bf16_t><<<grid, 256, 0, s>>>(tails, (const bf16_t*)proj, row, q_off, ntaps, cu_seqlens, slots, (int)channels);
        RI_LAUNCH_CHECK("delta_tails");
    }
    return 0;
}

extern "C" int ri_delta_prepare(float* qkv, float* gates, const void* proj, int act_dtype, int row, int q_off,
                                const float* taps, int ntaps, float* tails, const float* ab, const float* a_log,
                                const float* dt_bias, const int32_t* tok_seq, const int32_t* cu_seqlens,
                                const int32_t* slots, int seqs, int tokens, int heads, int kv_heads, int dim, int vdim,
                                void* stream) {
    return launch_delta_prepare<false>(qkv, gates, proj, act_dtype, row, q_off, taps, ntaps, tails, ab, a_log, dt_bias, tok_seq,
                                       cu_seqlens, slots, seqs, tokens, heads, kv_heads, dim, vdim, 0, nullptr, 0, stream);
}

extern "C" int ri_delta_prepare_channels(float* qkv, float* gates, const void* proj, int act_dtype, int row, int q_off,
                                         const float* taps, int ntaps, float* tails, const float* z, int z_row, const void* b,
                                         int b_row, const float* a_log, const float* dt_bias, const int32_t* tok_seq,
                                         const int32_t* cu_seqlens, const int32_t* slots, int seqs, int tokens, int heads,
                                         int kv_heads, int dim, int vdim, void* stream) {
    if (check_channels("delta_prepare_channels", z, z_row, b, b_row, heads, dim)) return 1;
    return launch_delta_prepare<true>(qkv, gates, proj, act_dtype, row, q_off, taps, ntaps, tails, z, a_log, dt_bias, tok_seq,
                                      cu_seqlens, slots, seqs, tokens, heads, kv_heads, dim, vdim, z_row, b, b_row, stream);
}

extern "C" int ri_delta_max_dim() { return 256; }

template <bool CH>
static int launch_delta_scan(float* out, const float* qkv, const float* gates, float* state, const int32_t* cu_seqlens,
                             const int32_t* slots, int seqs, int tokens, int heads, int kv_heads, int dim, int vdim,
                             int slices, void* stream) {
    RI_REQUIRE(slices == 0 || slices == 4 || slices == 8 || slices == 16,
               "delta_scan: %d slices of rows (4, 8, 16, or 0 for the launch's choice)", slices);
    RI_REQUIRE(tokens > 0 && seqs > 0 && heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && vdim > 0,
               "delta_scan: tokens %d, sequences %d, heads %d, kv heads %d", tokens, seqs, heads, kv_heads);
    RI_REQUIRE(dim >= 1 && dim <= 256, "delta_scan: key heads of %d, the kernel takes 1 to 256", dim);
    RI_REQUIRE((long)seqs * heads <= 2147483647L && (vdim + 3) / 4 <= 65535, "delta_scan: the grid");
    hipStream_t s = (hipStream_t)stream;
    // sixteen slices of rows in workgroups of one wavefront while every wavefront has a vector unit of its own; else eight slices
    // while the workgroups of four would leave compute units idle (a token's time halves), four once they fill the machine (half
    // the workgroups stage q and k)
    const long cus = ri_compute_units(), narrow = (long)seqs * heads * ((vdim + 3) / 4);
    const bool pieces = dim % 4 == 0 && (heads * vdim) % 4 == 0 && ((uintptr_t)qkv | (uintptr_t)gates) % 16 == 0;
    RI_REQUIRE(slices != 16 || pieces, "delta_scan: sixteen slices take heads in 16-byte pieces, not %d x %d", dim, vdim);
    const int sl = slices ? slices : narrow <= 4 * cus && pieces && dim >= 16 ? 16
                   : (long)seqs * heads * ((vdim + 63) / 64) <= cus && dim >= 8 ? 8 : 4;
    const int cols = sl == 16 ? 4 : 256 / sl;
    const dim3 grid((unsigned)(seqs * heads), (unsigned)((vdim + cols - 1) / cols));
    const int need = (dim + sl - 1) / sl;
#define RI_DELTA_GO(R, SL) delta_scan_kernel<R, SL, CH><<<grid, 256, 0, s>>>(out, qkv, gates, state, cu_seqlens, slots, heads, kv_heads, dim, vdim)
#define RI_DELTA_NARROW(R) delta_scan_narrow_kernel<R, CH><<<grid, 64, 0, s>>>(out, qkv, gates, state, cu_seqlens, slots, heads, kv_heads, dim, vdim)
    if (sl == 16) {
        if (need <= 4) RI_DELTA_NARROW(4);
        else if (need <= 8) RI_DELTA_NARROW(8);
        else RI_DELTA_NARROW(16);
    } else if (sl == 8) {
        if (need <= 4) RI_DELTA_GO(4, 8);
        else if (need <= 8) RI_DELTA_GO(8, 8);
        else if (need <= 16) RI_DELTA_GO(16, 8);
        else RI_DELTA_GO(32, 8);
    } else {
        if (need <= 4) RI_DELTA_GO(4, 4);
        else if (need <= 8) RI_DELTA_GO(8, 4);
        else if (need <= 16) RI_DELTA_GO(16, 4);
        else if (need <= 32) RI_DELTA_GO(32, 4);
        else RI_DELTA_GO(64, 4);
    }
#undef RI_DELTA_GO
#undef RI_DELTA_NARROW
    RI_LAUNCH_CHECK("delta_scan");
    return 0;
}

extern "C" int ri_delta_scan(float* out, const float* qkv, const float* gates, float* state, const int32_t* cu_seqlens,
                             const int32_t* slots, int seqs, int tokens, int heads, int kv_heads, int dim, int vdim,
                             int slices, void* stream) {
    return launch_delta_scan<false>(out, qkv, gates, state, cu_seqlens, slots, seqs, tokens, heads, kv_heads, dim, vdim, slices, stream);
}

extern "C" int ri_delta_scan_channels(float* out, const float* qkv, const float* gates, float* state, const int32_t* cu_seqlens,
                                      const int32_t* slots, int seqs, int tokens, int heads, int kv_heads, int dim, int vdim,
                                      int slices, void* stream) {
    return launch_delta_scan<true>(out, qkv, gates, state, cu_seqlens, slots, seqs, tokens, heads, kv_heads, dim, vdim, slices, stream);
}
