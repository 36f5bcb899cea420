#include "elem.h"
extern "C" int infer_talking_prefill_supported(int64_t, int64_t, int64_t, int64_t) { return 0; }
extern "C" int infer_talking_prefill(const void* q, int64_t q_stride, const void* keys, const void* values, int64_t key_pad,
                          int64_t vdim_pad, const int32_t* block_table, int64_t bt_stride, int64_t table_cols,
                          int64_t block_size, int64_t num_blocks, const int32_t* seqs, const int32_t* cu_q,
                          const int32_t* cu_k, int64_t num_seqs, int64_t tokens, int64_t max_seqlen_q, int64_t heads,
                          int64_t kv_heads, int64_t dim, int64_t vdim, float scale, const void* talk, float out_scale,
                          void* out, int64_t out_stride, float* workspace, int64_t workspace_floats, void* stream) { return -1; }
