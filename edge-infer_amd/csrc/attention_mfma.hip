// bfloat16 attention on the matrix cores for head sizes 64 and 128: the forms without a cap on the
// scores (kernels and launches: attention_mfma.h).
#define EI_ATTN_CAPPED 0
#include "attention_mfma.h"

// Positions of one sequence that a prefill work item of this file holds for a group ratio
// (with key_ways = 2, half as many: two waves then share the keys of every page for the same
// rows, which gives a short prompt twice the blocks).
extern "C" int ei_attn_prefill_mfma_positions(int G) {
  const int HB = G % 4 == 0 ? 4 : (G % 2 == 0 ? 2 : 1);
  return kWideRows * (kPrefillWaves / HB);
}

extern "C" int ei_attention_prefill_mfma(const void* q, const void* k_pages, const void* v_pages,
                                         const int32_t* item_seq, const int32_t* item_row0,
                                         const int32_t* item_npos, int n_items,
                                         const int32_t* row_pos, const int32_t* page_table,
                                         int table_width, void* out, int nq, int nkv, int D,
                                         int window, float scale, int key_ways, int pair_items,
                                         hipStream_t stream) {
  return prefill_launch(q, k_pages, v_pages, item_seq, item_row0, item_npos, n_items, row_pos,
                        page_table, table_width, out, nq, nkv, D, window, scale, key_ways,
                        pair_items, nullptr, stream);
}

// The same with the options of `AttnExtra`: chunk (0: none), slopes and sinks (float32 [nq] on
// the device, or null), another source's sums, the gates a head, kept first positions (0: none)
// and the gates an element.
extern "C" int ei_attention_prefill_mfma_ext(
    const void* q, const void* k_pages, const void* v_pages, const int32_t* item_seq,
    const int32_t* item_row0, const int32_t* item_npos, int n_items, const int32_t* row_pos,
    const int32_t* page_table, int table_width, void* out, int nq, int nkv, int D, int window,
    float scale, int key_ways, int pair_items, int chunk, const float* slopes,
    const float* sinks, const float* pool_o, const float* pool_ml, const float* gate, int keep,
    const void* wide, int wide_dtype, int wide_slices, long long wide_slice, long long wide_row,
    hipStream_t stream) {
  EI_REQUIRE(chunk >= 0, "attention_prefill: negative chunk");
  EI_REQUIRE(keep >= 0 && (keep == 0 || chunk == 0), "attention_prefill: kept first positions with chunks");
  EI_REQUIRE(wide_fits(wide, wide_dtype, wide_slices, wide_slice, wide_row, nq, D),
             "attention_prefill: the elements' gates have the wrong shape");
  EI_REQUIRE(scale > 0.f, "attention_prefill: the scale must be positive");
  EI_REQUIRE((pool_o == nullptr) == (pool_ml == nullptr),
             "attention_prefill: the other source's sums and their weights come together");
  const AttnExtra extra{chunk, slopes, sinks, pool_o, pool_ml, gate, keep, wide, wide_dtype,
                        wide_slices, static_cast<size_t>(wide_slice), static_cast<size_t>(wide_row), 0.f};
  return prefill_launch(q, k_pages, v_pages, item_seq, item_row0, item_npos, n_items, row_pos,
                        page_table, table_width, out, nq, nkv, D, window, scale, key_ways,
                        pair_items, &extra, stream);
}

// Whether the decode kernel of this file takes a head size and group ratio.
extern "C" int ei_attn_decode_mfma_supported(int D, int G) {
  return (D == 64 || D == 128) && G >= 1 ? 1 : 0;
}

// q, out: [rows, nq, D] bfloat16, one row per sequence (row_seq < 0: padding row);
// pages: [n_pages, nkv, 64, D]; n_splits > 1 needs part_o [rows, nq, n_splits, D] and
// part_ml [rows, nq, n_splits, 2] float32.  longest (or null): one int32 on the device, the most
// tokens that a sequence of this step holds; slices are then that sequence's share for all.
// heads: query heads of a kv group that one block takes (a power of two; 0: as many as a
// block of `waves` waves can, 4 for 16 waves, 8 for 8, else 16); a group of more has several
// blocks.
extern "C" int ei_attention_decode_mfma(const void* q, const void* k_pages, const void* v_pages,
                                        const int32_t* row_pos, const int32_t* row_seq,
                                        const int32_t* page_table, int table_width, void* out,
                                        float* part_o, float* part_ml, int rows, int nq, int nkv,
                                        int D, int window, float scale, int n_splits,
                                        int waves, int heads, const int32_t* longest,
                                        hipStream_t stream) {
  return decode_launch(q, k_pages, v_pages, row_pos, row_seq, page_table, table_width, out,
                       part_o, part_ml, rows, nq, nkv, D, window, scale, n_splits, waves, heads,
                       longest, nullptr, stream);
}

// The same with the options of `AttnExtra`: chunk (0: none), slopes and sinks (float32 [nq] on
// the device, or null), another source's sums, the gates a head, kept first positions (0: none)
// and the gates an element.
extern "C" int ei_attention_decode_mfma_ext(const void* q, const void* k_pages,
                                            const void* v_pages, const int32_t* row_pos,
                                            const int32_t* row_seq, const int32_t* page_table,
                                            int table_width, void* out, float* part_o,
                                            float* part_ml, int rows, int nq, int nkv, int D,
                                            int window, float scale, int n_splits, int waves,
                                            int heads, const int32_t* longest, int chunk,
                                            const float* slopes, const float* sinks,
                                            const float* pool_o, const float* pool_ml,
                                            const float* gate, int keep, const void* wide,
                                            int wide_dtype, int wide_slices, long long wide_slice,
                                            long long wide_row, hipStream_t stream) {
  EI_REQUIRE(chunk >= 0, "attention_decode: negative chunk");
  EI_REQUIRE(keep >= 0 && (keep == 0 || chunk == 0), "attention_decode: kept first positions with chunks");
  EI_REQUIRE(wide_fits(wide, wide_dtype, wide_slices, wide_slice, wide_row, nq, D),
             "attention_decode: the elements' gates have the wrong shape");
  const AttnExtra extra{chunk, slopes, sinks, pool_o, pool_ml, gate, keep, wide, wide_dtype,
                        wide_slices, static_cast<size_t>(wide_slice), static_cast<size_t>(wide_row), 0.f};
  return decode_launch(q, k_pages, v_pages, row_pos, row_seq, page_table, table_width, out,
                       part_o, part_ml, rows, nq, nkv, D, window, scale, n_splits, waves, heads,
                       longest, nullptr, stream, &extra);
}

// The same from the fused projection instead of q: qkv float32 [nsplit][rows, (nq + 2 nkv) * D]
// (partial sums, added in slice order); the kernel norms and rotates its queries itself and,
// with write_cache, also the position's key, and stores that key and the value in the pages
// (so the separate norm-rotate-store kernel is not needed for these rows).  q_norm_w, k_norm_w
// (float32 [D]) and rope_table (float32 [positions, rot_dim], rot_dim even and at most D) may
// each be null.
extern "C" int ei_attention_decode_mfma_fused(
    const float* qkv, int nsplit, long long split_stride, const float* q_norm_w,
    const float* k_norm_w, float eps, const float* rope_table, int rot_dim, int write_cache,
    void* k_pages,
    void* v_pages, const int32_t* row_pos, const int32_t* row_seq, const int32_t* page_table,
    int table_width, void* out, float* part_o, float* part_ml, int rows, int nq, int nkv, int D,
    int window, float scale, int n_splits, int waves, int heads, const int32_t* longest,
    hipStream_t stream) {
  EI_REQUIRE(qkv && nsplit >= 1 && split_stride >= 0, "attention_decode_fused: bad projection");
  EI_REQUIRE(!rope_table || (rot_dim >= 2 && rot_dim % 2 == 0 && rot_dim <= D),
             "attention_decode_fused: the rotated width must be even and at most head_dim");
  DecodePrep prep{};
  prep.qkv = qkv;
  prep.nsplit = nsplit;
  prep.split_stride = split_stride;
  prep.q_norm_w = q_norm_w;
  prep.k_norm_w = k_norm_w;
  prep.eps = eps;
  prep.rope_table = rope_table;
  prep.rot_dim = rope_table ? rot_dim : D;
  prep.k_store = write_cache ? static_cast<bf16_t*>(k_pages) : nullptr;
  prep.v_store = write_cache ? static_cast<bf16_t*>(v_pages) : nullptr;
  return decode_launch(nullptr, k_pages, v_pages, row_pos, row_seq, page_table, table_width, out,
                       part_o, part_ml, rows, nq, nkv, D, window, scale, n_splits, waves, heads,
                       longest, &prep, stream);
}
