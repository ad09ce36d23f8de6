// The matrix-core attention (attention_mfma.h) for heads of 32, 64 and 128 elements whose value heads have the same
// size: the launches.
#include "attention_mfma.h"

extern "C" int ri_attention_decode_streams(int seqs, int kv_heads, int max_chunks) {
    return stream_splits(seqs, kv_heads, max_chunks);
}

// ------------------------------------------------------------------ host side
static int check_common(const char* name, int heads, int kv_heads, int head_dim, int page_size, int q_stride,
                        int table_width) {
    RI_REQUIRE(heads > 0 && kv_heads > 0 && heads % kv_heads == 0, "%s: heads %d, kv heads %d", name, heads, kv_heads);
    RI_REQUIRE(head_dim == 32 || head_dim == 64 || head_dim == 128,
               "%s: head_dim %d (this kernel is built for 32, 64 and 128)", name, head_dim);
    RI_REQUIRE(page_size == PAGE, "%s: pages of %d tokens (this kernel takes %d)", name, page_size, PAGE);
    RI_REQUIRE(q_stride >= heads * head_dim && q_stride % 8 == 0, "%s: q row stride %d", name, q_stride);
    RI_REQUIRE(table_width > 0, "%s: page table width %d", name, table_width);
    RI_REQUIRE(kv_heads <= 65535, "%s: %d kv heads exceed one launch", name, kv_heads);
    return 0;
}

// Column tiles per wavefront: at most 64 columns for head_dim up to 64, 32 for 128 (registers); fewer when
// that leaves the launch with less than four workgroups a compute unit (few query heads per kv head, a
// prompt of a few thousand tokens: at 32 query and 8 kv heads of 128, 2,048 tokens take 81 us with 1,024
// workgroups of half the columns against 95 us with 512; from 4,096 tokens on the full tiles win).  A
// column's arithmetic does not depend on the tile it sits in, only the grid does.
// Tiles are halved while the launch has fewer workgroups than this many for each compute unit (measured with
// 256 of them: a prompt of 3,072 tokens at Qwen3-8B sizes takes 105 us with two tiles a wavefront in 768
// workgroups, 126 us with one tile in 1,536; at 2,048 tokens one tile in 1,024 workgroups takes 57 us, two in
// 512 take 67).
#define PREFILL_MIN_WGS_PER_CU 3
static int prefill_tiles(int head_dim, int group, int max_new, int seqs, int kv_heads) {
    int nt = head_dim <= 64 ? 4 : 2;
    while (nt > 1 && group <= 16 * (nt / 2)) {
        const int tile_tokens = (16 * nt) / group;
        const long wgs = (long)((max_new + 4 * tile_tokens - 1) / (4 * tile_tokens)) * seqs * kv_heads;
        if (wgs >= (long)PREFILL_MIN_WGS_PER_CU * ri_compute_units()) break;
        nt /= 2;
    }
    return nt;
}

extern "C" int ri_attention_prefill_kept_bf16(void* out, const void* qkv, int q_stride, const void* k_pages,
                                              const void* v_pages, const int32_t* cu_seqlens, const int32_t* tok_pos,
                                              const int32_t* page_table, int table_width, int seqs, int max_new,
                                              int heads, int kv_heads, int head_dim, int page_size, int window, int chunk,
                                              float scale, float softcap, const float* slopes, int keep_first,
                                              const float* sinks, void* stream) {
    RI_REQUIRE(chunk >= 0 && (chunk == 0 || window <= 0), "attention_prefill: chunks of %d beside a window of %d", chunk, window);
    const Reach reach = {window, chunk};
    RI_REQUIRE(keep_first >= 0, "attention_prefill_bf16: %d first tokens kept", keep_first);
    const float cap_pre = softcap > 0.f ? scale / softcap : 0.f, cap_post = softcap > 0.f ? softcap / scale : 0.f;
    RI_REQUIRE(scale > 0.f, "attention_prefill_bf16: the scale %g must be positive", (double)scale);
    if (check_common("attention_prefill_bf16", heads, kv_heads, head_dim, page_size, q_stride, table_width)) return 1;
    const int group = heads / kv_heads;
    RI_REQUIRE(seqs > 0 && seqs <= 65535 && max_new > 0, "attention_prefill_bf16: seqs %d, max_new %d", seqs, max_new);
    const int nt_tiles = prefill_tiles(head_dim, group, max_new, seqs, kv_heads);
    RI_REQUIRE(group <= 16 * nt_tiles, "attention_prefill_bf16: %d query heads per kv head (at most %d)", group,
               16 * nt_tiles);
    const int tile_tokens = (16 * nt_tiles) / group;
    const int tiles = (max_new + 4 * tile_tokens - 1) / (4 * tile_tokens);
    RI_REQUIRE(tiles <= 65535, "attention_prefill_bf16: %d tiles of tokens exceed one launch", tiles);
    dim3 grid(kv_heads, tiles, seqs);
    const float scale_log2 = scale * 1.4426950408889634f;
    hipStream_t s = (hipStream_t)stream;
#define RI_PREFILL_CASE(DH, NT)                                                                                  \
    case DH * 8 + NT:                                                                                            \
        attn_prefill_mfma_kernel<DH, NT><<<grid, 256, 0, s>>>(                                                   \
            (bf16_t*)out, (const bf16_t*)qkv, q_stride, (const bf16_t*)k_pages, (const bf16_t*)v_pages,          \
            cu_seqlens, tok_pos, page_table, table_width, heads, kv_heads, reach, scale_log2, cap_pre,          \
            cap_post, slopes, 1.f / scale, keep_first, sinks);                                                   \
        break;
    switch (head_dim * 8 + nt_tiles) {
        RI_PREFILL_CASE(32, 4)
        RI_PREFILL_CASE(32, 2)
        RI_PREFILL_CASE(32, 1)
        RI_PREFILL_CASE(64, 4)
        RI_PREFILL_CASE(64, 2)
        RI_PREFILL_CASE(64, 1)
        RI_PREFILL_CASE(128, 2)
        RI_PREFILL_CASE(128, 1)
    }
#undef RI_PREFILL_CASE
    RI_LAUNCH_CHECK("attention_prefill_bf16");
    return 0;
}

extern "C" int ri_attention_prefill_bf16(void* out, const void* qkv, int q_stride, const void* k_pages,
                                         const void* v_pages, const int32_t* cu_seqlens, const int32_t* tok_pos,
                                         const int32_t* page_table, int table_width, int seqs, int max_new,
                                         int heads, int kv_heads, int head_dim, int page_size, int window,
                                         float scale, float softcap, const float* slopes, void* stream) {
    return ri_attention_prefill_kept_bf16(out, qkv, q_stride, k_pages, v_pages, cu_seqlens, tok_pos, page_table, table_width,
                                          seqs, max_new, heads, kv_heads, head_dim, page_size, window, 0, scale, softcap, slopes,
                                          0, nullptr, stream);
}

extern "C" int ri_attention_decode_chunks(int max_len) { return (max_len + DECODE_CHUNK - 1) / DECODE_CHUNK; }

// The workspace of a decode attention call has room for max_chunks times this many results a sequence and head.
extern "C" int ri_attention_decode_pieces(int seqs, int kv_heads, int heads, int max_chunks) {
    return decode_pieces(seqs, kv_heads, heads / (kv_heads > 0 ? kv_heads : 1), max_chunks);
}

// keep_first, sinks: the first keys that stay visible behind a window, and a number per head whose exponential joins
// the softmax's denominator; only the kernels that work in chunks take kept keys (where ri_attention_decode_streams says
// the step streams, the caller takes the prompt kernel).
extern "C" int ri_attention_decode_kept_bf16(void* out, float* workspace, const void* qkv, int q_stride,
                                             const void* k_pages, const void* v_pages, const int32_t* cu_seqlens,
                                             const int32_t* tok_pos, const int32_t* page_table, int table_width, int seqs,
                                             int max_chunks, int heads, int kv_heads, int head_dim, int page_size,
                                             int window, int chunk, float scale, float softcap, const float* slopes, int tiled_out,
                                             int keep_first, const float* sinks, void* stream) {
    RI_REQUIRE(chunk >= 0 && (chunk == 0 || window <= 0), "attention_decode: chunks of %d beside a window of %d", chunk, window);
    const Reach reach = {window, chunk};
    RI_REQUIRE(keep_first >= 0, "attention_decode_bf16: %d first tokens kept", keep_first);
    RI_REQUIRE(keep_first == 0 || stream_splits(seqs, kv_heads, max_chunks) == 0,
               "attention_decode_bf16: kept first tokens in a step that streams (%d sequences)", seqs);
    const float cap_pre = softcap > 0.f ? scale / softcap : 0.f, cap_post = softcap > 0.f ? softcap / scale : 0.f;
    RI_REQUIRE(scale > 0.f, "attention_decode_bf16: the scale %g must be positive", (double)scale);
    if (check_common("attention_decode_bf16", heads, kv_heads, head_dim, page_size, q_stride, table_width)) return 1;
    RI_REQUIRE(!tiled_out || (seqs <= 64 && head_dim % 32 == 0), "attention_decode_bf16: tiled rows are at most 64 (%d)", seqs);
    const int group = heads / kv_heads;
    RI_REQUIRE(group <= 16, "attention_decode_bf16: %d query heads per kv head (at most 16)", group);
    RI_REQUIRE(seqs > 0 && max_chunks > 0 && max_chunks <= 65535 && heads <= 65535,
               "attention_decode_bf16: seqs %d, chunks %d, heads %d", seqs, max_chunks, heads);
    dim3 grid(seqs, kv_heads, max_chunks);
    const float scale_log2 = scale * 1.4426950408889634f;
    hipStream_t s = (hipStream_t)stream;
    const int splits = stream_splits(seqs, kv_heads, max_chunks);
    const bool wide = stream_wide(seqs, kv_heads, max_chunks);
    if (splits > 0) {
        dim3 sgrid(seqs, kv_heads, splits);
#define RI_STREAM_CASE(DH)                                                                                        \
    case DH:                                                                                                      \
        if (wide)                                                                                                 \
            attn_decode_stream_kernel<DH, false, 8><<<sgrid, 8 * 64, 0, s>>>(                                     \
                (bf16_t*)out, workspace, (const bf16_t*)qkv, q_stride, nullptr, nullptr, 0.f, nullptr,            \
                (bf16_t*)k_pages, (bf16_t*)v_pages, tok_pos, page_table, table_width, heads, kv_heads, reach,     \
                scale_log2, splits, tiled_out, cap_pre, cap_post, slopes, 1.f / scale, sinks);                           \
        else                                                                                                      \
            attn_decode_stream_kernel<DH, false, 4><<<sgrid, 4 * 64, 0, s>>>(                                     \
                (bf16_t*)out, workspace, (const bf16_t*)qkv, q_stride, nullptr, nullptr, 0.f, nullptr,            \
                (bf16_t*)k_pages, (bf16_t*)v_pages, tok_pos, page_table, table_width, heads, kv_heads, reach,     \
                scale_log2, splits, tiled_out, cap_pre, cap_post, slopes, 1.f / scale, sinks);                           \
        if (splits > 1)                                                                                          \
            launch_join<DH>((bf16_t*)out, workspace, tok_pos, seqs, heads, Reach{-1, 0}, splits, tiled_out, s, DECODE_CHUNK, 0, sinks); \
        break;
        switch (head_dim) {
            RI_STREAM_CASE(32)
            RI_STREAM_CASE(64)
            RI_STREAM_CASE(128)
        }
#undef RI_STREAM_CASE
        RI_LAUNCH_CHECK("attention_decode_bf16 (streaming)");
        return 0;
    }
    const int pieces = decode_pieces(seqs, kv_heads, group, max_chunks), all = max_chunks * pieces;
    const dim3 pgrid(seqs, kv_heads, all);
#define RI_DECODE_CASE(DH, CW)                                                                                    \
    case DH * 16 + CW:                                                                                            \
        attn_decode_mfma_kernel<DH, CW><<<pgrid, CW * 64, 0, s>>>(                                                \
            workspace, (const bf16_t*)qkv, q_stride, (const bf16_t*)k_pages, (const bf16_t*)v_pages,             \
            tok_pos, page_table, table_width, heads, kv_heads, reach, scale_log2, all, cap_pre, cap_post,       \
            slopes, 1.f / scale, keep_first);                                                                     \
        launch_join<DH>((bf16_t*)out, workspace, tok_pos, seqs, heads, reach, all, tiled_out, s, CW * PAGE,      \
                        keep_first, sinks);                                                                       \
        break;
    switch (head_dim * 16 + DECODE_WAVES / pieces) {
        RI_DECODE_CASE(32, 8)
        RI_DECODE_CASE(32, 4)
        RI_DECODE_CASE(32, 2)
        RI_DECODE_CASE(64, 8)
        RI_DECODE_CASE(64, 4)
        RI_DECODE_CASE(64, 2)
        RI_DECODE_CASE(128, 8)
        RI_DECODE_CASE(128, 4)
        RI_DECODE_CASE(128, 2)
    }
#undef RI_DECODE_CASE
    RI_LAUNCH_CHECK("attention_decode_bf16");
    return 0;
}

extern "C" int ri_attention_decode_bf16(void* out, float* workspace, const void* qkv, int q_stride,
                                        const void* k_pages, const void* v_pages, const int32_t* cu_seqlens,
                                        const int32_t* tok_pos, const int32_t* page_table, int table_width, int seqs,
                                        int max_chunks, int heads, int kv_heads, int head_dim, int page_size,
                                        int window, float scale, float softcap, const float* slopes, int tiled_out,
                                        void* stream) {
    return ri_attention_decode_kept_bf16(out, workspace, qkv, q_stride, k_pages, v_pages, cu_seqlens, tok_pos, page_table,
                                         table_width, seqs, max_chunks, heads, kv_heads, head_dim, page_size, window, 0, scale,
                                         softcap, slopes, tiled_out, 0, nullptr, stream);
}

// The decode attention of a layer from the raw fused projection (which is not changed): q/k norm, rotation,
// the new token's k and v into their pages and attention in chunks in one kernel, then the join.
extern "C" int ri_attention_decode_fused_bf16(void* out, float* workspace, const void* qkv, int q_stride,
                                              const float* q_gain, const float* k_gain, float eps,
                                              const float* inv_freq, void* k_pages, void* v_pages,
                                              const int32_t* tok_pos, const int32_t* page_table, int table_width,
                                              int seqs, int max_chunks, int heads, int kv_heads, int head_dim,
                                              int page_size, int window, float scale, int tiled_out, void* stream) {
    const Reach reach = {window, 0};
    if (check_common("attention_decode_fused_bf16", heads, kv_heads, head_dim, page_size, q_stride, table_width))
        return 1;
    RI_REQUIRE(!tiled_out || (seqs <= 64 && head_dim % 32 == 0), "attention_decode_fused_bf16: tiled rows are at most 64 (%d)", seqs);
    const int group = heads / kv_heads;
    RI_REQUIRE(group <= 16, "attention_decode_fused_bf16: %d query heads per kv head (at most 16)", group);
    RI_REQUIRE(seqs > 0 && max_chunks > 0 && max_chunks <= 65535 && heads <= 65535,
               "attention_decode_fused_bf16: seqs %d, chunks %d, heads %d", seqs, max_chunks, heads);
    RI_REQUIRE(q_stride >= (heads + 2 * kv_heads) * head_dim, "attention_decode_fused_bf16: qkv row stride %d",
               q_stride);
    dim3 grid(seqs, kv_heads, max_chunks);
    const float scale_log2 = scale * 1.4426950408889634f;
    hipStream_t s = (hipStream_t)stream;
    const int splits = stream_splits(seqs, kv_heads, max_chunks);
    const bool wide = stream_wide(seqs, kv_heads, max_chunks);
    if (splits > 0) {
        dim3 sgrid(seqs, kv_heads, splits);
#define RI_STREAM_CASE(DH)                                                                                        \
    case DH:                                                                                                      \
        if (wide)                                                                                                 \
            attn_decode_stream_kernel<DH, true, 8><<<sgrid, 8 * 64, 0, s>>>(                                      \
                (bf16_t*)out, workspace, (const bf16_t*)qkv, q_stride, q_gain, k_gain, eps, inv_freq,             \
                (bf16_t*)k_pages, (bf16_t*)v_pages, tok_pos, page_table, table_width, heads, kv_heads, reach,     \
                scale_log2, splits, tiled_out, 0.f, 0.f, nullptr, 0.f, nullptr);                                           \
        else                                                                                                      \
            attn_decode_stream_kernel<DH, true, 4><<<sgrid, 4 * 64, 0, s>>>(                                      \
                (bf16_t*)out, workspace, (const bf16_t*)qkv, q_stride, q_gain, k_gain, eps, inv_freq,             \
                (bf16_t*)k_pages, (bf16_t*)v_pages, tok_pos, page_table, table_width, heads, kv_heads, reach,     \
                scale_log2, splits, tiled_out, 0.f, 0.f, nullptr, 0.f, nullptr);                                           \
        if (splits > 1) launch_join<DH>((bf16_t*)out, workspace, tok_pos, seqs, heads, Reach{-1, 0}, splits, tiled_out, s); \
        break;
        switch (head_dim) {
            RI_STREAM_CASE(32)
            RI_STREAM_CASE(64)
            RI_STREAM_CASE(128)
        }
#undef RI_STREAM_CASE
        RI_LAUNCH_CHECK("attention_decode_fused_bf16 (streaming)");
        return 0;
    }
    const int pieces = decode_pieces(seqs, kv_heads, group, max_chunks), all = max_chunks * pieces;
    const dim3 pgrid(seqs, kv_heads, all);
#define RI_FUSED_CASE(DH, CW)                                                                                     \
    case DH * 16 + CW:                                                                                            \
        attn_decode_fused_kernel<DH, CW><<<pgrid, CW * 64, 0, s>>>(                                               \
            workspace, (const bf16_t*)qkv, q_stride, q_gain, k_gain, eps, inv_freq, (bf16_t*)k_pages,             \
            (bf16_t*)v_pages, tok_pos, page_table, table_width, heads, kv_heads, reach, scale_log2, all);        \
        launch_join<DH>((bf16_t*)out, workspace, tok_pos, seqs, heads, reach, all, tiled_out, s, CW * PAGE);     \
        break;
    switch (head_dim * 16 + DECODE_WAVES / pieces) {
        RI_FUSED_CASE(32, 8)
        RI_FUSED_CASE(32, 4)
        RI_FUSED_CASE(32, 2)
        RI_FUSED_CASE(64, 8)
        RI_FUSED_CASE(64, 4)
        RI_FUSED_CASE(64, 2)
        RI_FUSED_CASE(128, 8)
        RI_FUSED_CASE(128, 4)
        RI_FUSED_CASE(128, 2)
    }
#undef RI_FUSED_CASE
    RI_LAUNCH_CHECK("attention_decode_fused_bf16");
    return 0;
}
