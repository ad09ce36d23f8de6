// The matrix-core attention (attention_mfma.h) for heads of any multiple of 8 elements up to 128 and value heads of any
// multiple of 4 up to 256, the two of their own sizes: kernels built for key heads of 64 and 128 and value heads of 64, 96,
// 128, 192 and 256, each taking what fits below it.  What lies behind a head's end is zero in the operands.
#include "attention_mfma.h"

#define PAD_MAX_DIM 128
#define PAD_MAX_VDIM 256
#define PAD_WIDE_VDIM 128         // value heads above it: one tile of columns a wavefront, and no streaming (registers)

static int check_padded(const char* name, int heads, int kv_heads, int dim, int vdim, int page_size, int q_stride,
                        int table_width, float scale) {
    RI_REQUIRE(heads > 0 && kv_heads > 0 && heads % kv_heads == 0, "%s: heads %d, kv heads %d", name, heads, kv_heads);
    RI_REQUIRE(dim >= 8 && dim <= PAD_MAX_DIM && dim % 8 == 0 && vdim >= 4 && vdim <= PAD_MAX_VDIM && vdim % 4 == 0,
               "%s: heads of %d and %d (multiples of 8 up to %d, and of 4 up to %d)", name, dim, vdim, PAD_MAX_DIM, PAD_MAX_VDIM);
    RI_REQUIRE(page_size == PAGE, "%s: pages of %d tokens (this kernel takes %d)", name, page_size, PAGE);
    RI_REQUIRE(q_stride >= heads * dim && q_stride % 8 == 0, "%s: q row stride %d", name, q_stride);
    RI_REQUIRE(table_width > 0, "%s: page table width %d", name, table_width);
    RI_REQUIRE(kv_heads <= 65535, "%s: %d kv heads exceed one launch", name, kv_heads);
    RI_REQUIRE(scale > 0.f, "%s: the scale %g must be positive", name, (double)scale);
    return 0;
}

// The smallest built sizes that hold a head: what the switches below run over.
static int padded_dim(int dim) { return dim <= 64 ? 64 : 128; }
static int padded_vdim(int vdim) { return vdim <= 64 ? 64 : vdim <= 96 ? 96 : vdim <= 128 ? 128 : vdim <= 192 ? 192 : 256; }

// Whether the kernels take these sizes and this many query heads a kv head.
extern "C" int ri_attention_padded_fits(int dim, int vdim, int group, int decode) {
    const bool sizes = dim >= 8 && dim <= PAD_MAX_DIM && dim % 8 == 0 && vdim >= 4 && vdim <= PAD_MAX_VDIM && vdim % 4 == 0;
    return sizes && group >= 1 && group <= (decode || vdim > PAD_WIDE_VDIM ? 16 : 32);
}

extern "C" int ri_attention_prefill_padded_bf16(void* out, const void* qkv, int q_stride, const void* k_pages,
                                                const void* v_pages, const int32_t* cu_seqlens, const int32_t* tok_pos,
                                                const int32_t* page_table, int table_width, int seqs, int max_new,
                                                int heads, int kv_heads, int dim, int vdim, int page_size, int window, int chunk,
                                                float scale, float softcap, const float* slopes, int keep_first,
                                                const float* sinks, void* stream) {
    RI_REQUIRE(chunk >= 0 && (chunk == 0 || window <= 0), "attention_prefill_padded: chunks of %d beside a window of %d", chunk, window);
    const Reach reach = {window, chunk};
    RI_REQUIRE(keep_first >= 0, "attention_prefill_padded: %d first tokens kept", keep_first);
    if (check_padded("attention_prefill_padded", heads, kv_heads, dim, vdim, page_size, q_stride, table_width, scale)) return 1;
    const float cap_pre = softcap > 0.f ? scale / softcap : 0.f, cap_post = softcap > 0.f ? softcap / scale : 0.f;
    const int group = heads / kv_heads;
    RI_REQUIRE(seqs > 0 && seqs <= 65535 && max_new > 0, "attention_prefill_padded: seqs %d, max_new %d", seqs, max_new);
    int nt_tiles = vdim > PAD_WIDE_VDIM ? 1 : 2;             // halved while that leaves the machine unfilled, as for equal sizes
    if (nt_tiles == 2 && group <= 16) {
        const int tile_tokens = 32 / group;
        const long wgs = (long)((max_new + 4 * tile_tokens - 1) / (4 * tile_tokens)) * seqs * kv_heads;
        if (wgs < 3L * ri_compute_units()) nt_tiles = 1;
    }
    RI_REQUIRE(group <= 16 * nt_tiles, "attention_prefill_padded: %d query heads per kv head (at most %d)", group, 16 * nt_tiles);
    const int tile_tokens = (16 * nt_tiles) / group;
    const int tiles = (max_new + 4 * tile_tokens - 1) / (4 * tile_tokens);
    RI_REQUIRE(tiles <= 65535, "attention_prefill_padded: %d tiles of tokens exceed one launch", tiles);
    dim3 grid(kv_heads, tiles, seqs);
    const float scale_log2 = scale * 1.4426950408889634f;
    hipStream_t s = (hipStream_t)stream;
#define RI_CASE(DH, NT, DV)                                                                                       \
    case (DH * 8 + NT) * 512 + DV:                                                                                \
        attn_prefill_mfma_kernel<DH, NT, DV, true><<<grid, 256, 0, s>>>(                                           \
            (bf16_t*)out, (const bf16_t*)qkv, q_stride, (const bf16_t*)k_pages, (const bf16_t*)v_pages,          \
            cu_seqlens, tok_pos, page_table, table_width, heads, kv_heads, reach, scale_log2, cap_pre,          \
            cap_post, slopes, 1.f / scale, keep_first, sinks, dim, vdim);                                         \
        break;
#define RI_CASES(DH)                                                                                              \
    RI_CASE(DH, 2, 64) RI_CASE(DH, 1, 64) RI_CASE(DH, 2, 96) RI_CASE(DH, 1, 96) RI_CASE(DH, 2, 128) RI_CASE(DH, 1, 128) \
    RI_CASE(DH, 1, 192) RI_CASE(DH, 1, 256)
    switch ((padded_dim(dim) * 8 + nt_tiles) * 512 + padded_vdim(vdim)) {
        RI_CASES(64)
        RI_CASES(128)
    }
#undef RI_CASES
#undef RI_CASE
    RI_LAUNCH_CHECK("attention_prefill_padded");
    return 0;
}

// One new token a sequence; the workspace has room for max_chunks * ri_attention_decode_pieces results of vdim + 2 floats
// a sequence and head.
extern "C" int ri_attention_decode_padded_bf16(void* out, float* workspace, const void* qkv, int q_stride,
                                               const void* k_pages, const void* v_pages, const int32_t* tok_pos,
                                               const int32_t* page_table, int table_width, int seqs, int max_chunks,
                                               int heads, int kv_heads, int dim, int vdim, int page_size, int window, int chunk,
                                               float scale, float softcap, const float* slopes, int tiled_out,
                                               int keep_first, const float* sinks, void* stream) {
    RI_REQUIRE(chunk >= 0 && (chunk == 0 || window <= 0), "attention_decode_padded: chunks of %d beside a window of %d", chunk, window);
    const Reach reach = {window, chunk};
    RI_REQUIRE(keep_first >= 0, "attention_decode_padded: %d first tokens kept", keep_first);
    if (check_padded("attention_decode_padded", heads, kv_heads, dim, vdim, page_size, q_stride, table_width, scale)) return 1;
    const float cap_pre = softcap > 0.f ? scale / softcap : 0.f, cap_post = softcap > 0.f ? softcap / scale : 0.f;
    RI_REQUIRE(!tiled_out || seqs <= 64, "attention_decode_padded: tiled rows are at most 64 (%d)", seqs);
    const int group = heads / kv_heads;
    RI_REQUIRE(group <= 16, "attention_decode_padded: %d query heads per kv head (at most 16)", group);
    RI_REQUIRE(seqs > 0 && max_chunks > 0 && max_chunks <= 65535 && heads <= 65535,
               "attention_decode_padded: seqs %d, chunks %d, heads %d", seqs, max_chunks, heads);
    const float scale_log2 = scale * 1.4426950408889634f;
    hipStream_t s = (hipStream_t)stream;
    // (the streaming kernel does not keep first tokens, and holds two pages in registers: not for wide value heads)
    const int splits = keep_first > 0 || vdim > PAD_WIDE_VDIM ? 0 : stream_splits(seqs, kv_heads, max_chunks);
    if (splits > 0) {
        const bool wide = stream_wide(seqs, kv_heads, max_chunks);
        dim3 sgrid(seqs, kv_heads, splits);
#define RI_STREAM(DH, W, DV)                                                                                      \
    attn_decode_stream_kernel<DH, false, W, DV, true><<<sgrid, W * 64, 0, s>>>(                                    \
        (bf16_t*)out, workspace, (const bf16_t*)qkv, q_stride, nullptr, nullptr, 0.f, nullptr, (bf16_t*)k_pages,  \
        (bf16_t*)v_pages, tok_pos, page_table, table_width, heads, kv_heads, reach, scale_log2, splits,          \
        tiled_out, cap_pre, cap_post, slopes, 1.f / scale, sinks, dim, vdim)
#define RI_CASE(DH, DV)                                                                                           \
    case DH * 512 + DV:                                                                                           \
        if (wide) RI_STREAM(DH, 8, DV);                                                                           \
        else RI_STREAM(DH, 4, DV);                                                                                \
        if (splits > 1)                                                                                           \
            launch_join<DV, true>((bf16_t*)out, workspace, tok_pos, seqs, heads, Reach{-1, 0}, splits, tiled_out, s, DECODE_CHUNK, 0, \
                                  sinks, vdim);                                                                   \
        break;
        switch (padded_dim(dim) * 512 + padded_vdim(vdim)) {
            RI_CASE(64, 64) RI_CASE(64, 96) RI_CASE(64, 128) RI_CASE(128, 64) RI_CASE(128, 96) RI_CASE(128, 128)
        }
#undef RI_CASE
#undef RI_STREAM
        RI_LAUNCH_CHECK("attention_decode_padded (streaming)");
        return 0;
    }
    const int pieces = decode_pieces(seqs, kv_heads, group, max_chunks), all = max_chunks * pieces;
    const dim3 pgrid(seqs, kv_heads, all);
#define RI_CHUNKS(DH, CW, DV)                                                                                     \
    case (DH * 16 + CW) * 512 + DV:                                                                               \
        attn_decode_mfma_kernel<DH, CW, DV, true><<<pgrid, CW * 64, 0, s>>>(                                       \
            workspace, (const bf16_t*)qkv, q_stride, (const bf16_t*)k_pages, (const bf16_t*)v_pages, tok_pos,     \
            page_table, table_width, heads, kv_heads, reach, scale_log2, all, cap_pre, cap_post, slopes,         \
            1.f / scale, keep_first, dim, vdim);                                                                  \
        launch_join<DV, true>((bf16_t*)out, workspace, tok_pos, seqs, heads, reach, all, tiled_out, s, CW * PAGE,  \
                              keep_first, sinks, vdim);                                                           \
        break;
#define RI_CASE(DH, DV) RI_CHUNKS(DH, 8, DV) RI_CHUNKS(DH, 4, DV) RI_CHUNKS(DH, 2, DV)
    switch ((padded_dim(dim) * 16 + DECODE_WAVES / pieces) * 512 + padded_vdim(vdim)) {
        RI_CASE(64, 64) RI_CASE(64, 96) RI_CASE(64, 128) RI_CASE(64, 192) RI_CASE(64, 256)
        RI_CASE(128, 64) RI_CASE(128, 96) RI_CASE(128, 128) RI_CASE(128, 192) RI_CASE(128, 256)
    }
#undef RI_CASE
#undef RI_CHUNKS
    RI_LAUNCH_CHECK("attention_decode_padded");
    return 0;
}
