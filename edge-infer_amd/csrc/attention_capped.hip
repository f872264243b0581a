// bfloat16 attention on the matrix cores for head sizes 64 and 128 with a cap on the scores: the
// scaled score s becomes cap tanh(s / cap) (kernels and launches: attention_mfma.h).
#define EI_ATTN_CAPPED 1
#include "attention_mfma.h"

// Arguments as ei_attention_prefill_mfma_ext's (without kept first positions and gates an element),
// and the cap.
extern "C" int ei_attention_prefill_capped(
    const void* q, const void* k_pages, const void* v_pages, const int32_t* item_seq,
    const int32_t* item_row0, const int32_t* item_npos, int n_items, const int32_t* row_pos,
    const int32_t* page_table, int table_width, void* out, int nq, int nkv, int D, int window,
    float scale, int key_ways, int pair_items, int chunk, const float* slopes,
    const float* sinks, const float* pool_o, const float* pool_ml, const float* gate, float cap,
    hipStream_t stream) {
  EI_REQUIRE(chunk >= 0 && cap > 0.f && scale > 0.f,
             "attention_prefill: cap and scale must be positive, the chunk not negative");
  EI_REQUIRE((pool_o == nullptr) == (pool_ml == nullptr),
             "attention_prefill: the other source's sums and their weights come together");
  const AttnExtra extra{chunk, slopes, sinks, pool_o, pool_ml, gate, 0, nullptr, EI_F32, 1, 0, 0, cap};
  return prefill_launch(q, k_pages, v_pages, item_seq, item_row0, item_npos, n_items, row_pos,
                        page_table, table_width, out, nq, nkv, D, window, scale, key_ways,
                        pair_items, &extra, stream);
}

// Arguments as ei_attention_decode_mfma_ext's, with the same differences.
extern "C" int ei_attention_decode_capped(
    const void* q, const void* k_pages, const void* v_pages, const int32_t* row_pos,
    const int32_t* row_seq, const int32_t* page_table, int table_width, void* out, float* part_o,
    float* part_ml, int rows, int nq, int nkv, int D, int window, float scale, int n_splits,
    int waves, int heads, const int32_t* longest, int chunk, const float* slopes,
    const float* sinks, const float* pool_o, const float* pool_ml, const float* gate, float cap,
    hipStream_t stream) {
  EI_REQUIRE(chunk >= 0 && cap > 0.f, "attention_decode: the cap must be positive, the chunk not negative");
  const AttnExtra extra{chunk, slopes, sinks, pool_o, pool_ml, gate, 0, nullptr, EI_F32, 1, 0, 0, cap};
  return decode_launch(q, k_pages, v_pages, row_pos, row_seq, page_table, table_width, out, part_o,
                       part_ml, rows, nq, nkv, D, window, scale, n_splits, waves, heads, longest,
                       nullptr, stream, &extra);
}
