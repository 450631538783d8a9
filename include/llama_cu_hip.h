/*
 * C ABI of the MI355X (gfx950) device layer behind the llama_cu host interface.
 *
 * The reference (eiz/llama.cu) has no FFI: its forward pass, llama_context_impl::next_token
 * (llama_cu.cu:1073-1210), launches CUDA kernels directly.  This header declares one entry point
 * per launch site of that function, plus the buffer calls of llama_cu.h:109-134, so that the host
 * code (and any other language) reaches the GPU through plain pointers and sizes.
 *
 * Conventions
 *   - every pointer named *_dev is device memory; fp16 tensors are IEEE binary16, row-major
 *   - `stream` is a hipStream_t passed as void* (NULL = the default stream); work is asynchronous
 *     unless stated
 *   - every function returns 0 on success and a negative code on failure, never throws, never
 *     exits; lcu_last_error() describes the last failure of the calling thread
 *   - shapes the kernels do not support are rejected before any launch (LCU_E_SHAPE)
 *   - one host thread per stream.  Operators that work in two launches keep partial results in
 *     a 32 MiB workspace: every stream made by lcu_stream_create owns one (so contexts, which each
 *     create a stream, never share scratch), the default stream and streams made elsewhere use one
 *     per device created by lcu_init - calls on those that overlap on one device race
 */
#ifndef LLAMA_CU_HIP_H
#define LLAMA_CU_HIP_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define LCU_OK 0
#define LCU_E_HIP (-1)      /* a HIP runtime call failed */
#define LCU_E_SHAPE (-2)    /* unsupported or inconsistent shape / null pointer */
#define LCU_E_NOINIT (-3)   /* lcu_init has not run on this device */

typedef struct lcu_device_props {
  char name[128];
  int compute_units;
  int lds_bytes_per_block;
  int l2_bytes;
  int clock_khz;
  int memory_clock_khz;
  int memory_bus_bits;
  size_t total_memory;
  size_t free_memory;
} lcu_device_props;

/* ---- runtime: llama_cu.cu:1525-1542 (initialize), 691-736 (scoped_gpu, gpu_buffer[_view]) ---- */
int lcu_init(int device);
const char* lcu_last_error(void);
int lcu_device_get_props(int device, lcu_device_props* out);
int lcu_get_device(int* out_device);                                            /* scoped_gpu, 691-697 */
int lcu_set_device(int device);
int lcu_malloc(void** out_dev, size_t bytes);                                   /* gpu_buffer ctor, 712-715 */
int lcu_free(void* dev);                                                        /* gpu_buffer dtor, 732-736 */
int lcu_memset(void* dev, int byte_value, size_t bytes, void* stream);          /* llama_cu.h:239-241 */
int lcu_h2d(void* dst_dev, const void* src_host, size_t bytes, void* stream);   /* copy_from, 699-706; async */
int lcu_d2h(void* dst_host, const void* src_dev, size_t bytes, void* stream);   /* copy_to, 707-710; blocks */
int lcu_d2d(void* dst_dev, const void* src_dev, size_t bytes, void* stream);
int lcu_stream_create(void** out_stream);
int lcu_stream_destroy(void* stream);
/* bounded in-launch waits that ran out on this stream's workspace so far (0 in any healthy run) */
int lcu_sync_timeouts(void* stream, unsigned* out_count);
/* Adds `count` to that counter (stream-ordered), as a wait that ran out would: lets a caller rehearse its
 * handling of a failed hand-over without making any kernel wait.  No counterpart in the reference. */
int lcu_sync_add_timeouts(void* stream, unsigned count);

/* Clears the stream's hand-over words (stream-ordered, not under capture).  A hand-over word is taken for new
 * when it carries the launch's epoch, 21 bits of *seq_dev and the salt: a caller whose step counter has run
 * through 2^21 values clears the words before the epochs repeat, and never uses a counter whose low 21 bits
 * are zero with salt 0 (the epoch of a cleared word).  No counterpart in the reference. */
int lcu_sync_reset(void* stream);
int lcu_sync(void* stream);                                                     /* NULL = whole device */
/* HIP graph capture of the launches made on `stream` between begin and end; every lcu_* kernel
 * entry point may be captured (none of them records a memset node or allocates).  No counterpart
 * in the reference, whose host loop launches ~480 kernels per token one by one. */
int lcu_graph_begin_capture(void* stream);
int lcu_graph_end_capture(void* stream, void** out_graph_exec);
int lcu_graph_launch(void* graph_exec, void* stream);
int lcu_graph_destroy(void* graph_exec);
int lcu_event_create(void** out_event);
int lcu_event_destroy(void* event);
int lcu_event_record(void* event, void* stream);
int lcu_event_elapsed_ms(float* out_ms, void* start_event, void* stop_event);   /* waits for stop */

/* ---- matmul: out[M,N] = lhs[M,K] * rhs[N,K]^T + beta * out ----
 * lcu_gemm_f16_nt replaces matmul_nt(tensor4d_view) and the kernels it selects
 * (llama_cu.cu:1463-1496, 150-220, 225-285): M == 1 runs the streaming GEMV, larger M the MFMA
 * GEMM.  K must be a multiple of 8.  fp32 accumulation, one rounding to fp16 of acc + beta*out.
 * With 2 <= M <= 64 (short prompts) and K a multiple of 128 the K range is split over workgroups
 * and the fp32 partial sums pass through the stream's workspace (both GEMM entry points). */
int lcu_gemm_f16_nt(void* out_dev, const void* lhs_dev, const void* rhs_dev, int M, int K, int N,
                    float beta, void* stream);
/* lcu_gemm_f16u8_nt replaces matmul_nt(generic_tensor&) for quantised weights and
 * matmul_nt_wmma_16x128x256_fp16u8 (llama_cu.cu:1498-1523, 287-366): codes [N,K] uint8, scales
 * [N,K/block] fp16, each weight dequantised as fp16((code - 127.5) * scale) before it is used.
 * K % 16 == 0, block % 16 == 0, K % block == 0. */
int lcu_gemm_f16u8_nt(void* out_dev, const void* lhs_dev, const void* codes_dev,
                      const void* scales_dev, int M, int K, int N, int block, float beta,
                      void* stream);
/* Up to three such products with one lhs and weight matrices of one shape in a single launch
 * (Wq, Wk, Wv at launch sites 1144-1156; W1, W3 at 1180-1181): out_dev, rhs_dev (codes_dev,
 * scales_dev) are host arrays of n_mats device pointers.  Same results as n_mats separate calls;
 * with M == 1 it is n_mats separate calls. */
int lcu_gemm_f16_nt_multi(void* const* out_dev, const void* lhs_dev, const void* const* rhs_dev, int n_mats, int M,
                          int K, int N, float beta, void* stream);
int lcu_gemm_f16u8_nt_multi(void* const* out_dev, const void* lhs_dev, const void* const* codes_dev,
                            const void* const* scales_dev, int n_mats, int M, int K, int N, int block, float beta,
                            void* stream);

/* ---- int8 absmax quantiser: transform.cu:28-72 and 74-87; block in {32, 64, 128, 256, 512, 1024} */
int lcu_quantize_absmax_u8(void* codes_dev, void* scales_dev, const void* in_dev, size_t rows,
                           size_t cols, int block, void* stream);
int lcu_dequantize_absmax_u8(void* out_dev, const void* scales_dev, const void* codes_dev,
                             size_t rows, size_t cols, int block, void* stream);

/* ---- row and element-wise kernels ---- */
/* rms_norm, llama_cu.cu:66-107 (launch sites 1129, 1176, 1191) */
int lcu_rmsnorm(void* out_dev, const void* in_dev, const void* weights_dev, int rows, int cols,
                float eps, void* stream);
/* rotary, llama_cu.cu:368-389 (launch sites 1146, 1152).  The angles cos/sin(pos / theta^(c/head_dim))
 * come from a table built once on the host with the C library's powf/cosf/sinf:
 * table_dev[pos][pair] = {cos, sin} as float2, pair = (c mod head_dim) / 2. */
int lcu_rope_table_create(void** out_table_dev, int positions, int head_dim, float theta);
int lcu_rope(void* out_dev, const void* in_dev, int rows, int cols, int n_heads, int pos_offset,
             const void* table_dev, int table_positions, void* stream);
/* lcu_rope in place on two tensors of one shape in one launch: the new rows of Q and of K of a prompt
 * (launch sites 1146 and 1152; the reference rotates the whole K cache into a scratch copy on every call) */
int lcu_rope_pair(void* a_dev, void* b_dev, int rows, int cols, int n_heads, int pos_offset, const void* table_dev,
                  int table_positions, void* stream);
/* softmax_rows, llama_cu.cu:433-499 (launch sites 1166, 1196); in place allowed */
int lcu_softmax_rows(void* out_dev, const void* in_dev, int rows, int w, float temp, void* stream);
/* e^x on n fp32 values with the exponential that every softmax and SiLU of this library takes
 * (IEEE operations only, within one ulp; the reference calls CUDA's expf at llama_cu.cu:463, 497,
 * 537).  Exported so that the host restatement of the same steps can be held to it bit for bit. */
int lcu_exp_f32(void* out_dev, const void* in_dev, size_t n, void* stream);
/* silu, llama_cu.cu:533-539 (launch site 1183) */
int lcu_silu_mul(void* out_dev, const void* a_dev, const void* b_dev, size_t size, void* stream);
/* embed / embed_uint8, llama_cu.cu:32-62 (launch sites 1090, 1094); ids are int16 */
int lcu_embed(void* out_dev, const void* ids_dev, int n_ids, int dim, const void* table_dev,
              int n_vocab, void* stream);
int lcu_embed_u8(void* out_dev, const void* ids_dev, int n_ids, int dim, const void* codes_dev,
                 const void* scales_dev, int block, int n_vocab, void* stream);
/* embed / embed_uint8 (launch sites 1090, 1094) and the first layer's rms_norm (1129) of the same rows in
 * one launch: x_out gets the rows, norm_out their norm under weights_dev.  block 0: table_dev is the fp16
 * table and scales_dev is ignored; else table_dev holds codes (block a multiple of 8 dividing dim).
 * dim a multiple of 8, at most 8192.  Same values as lcu_embed[_u8] followed by lcu_rmsnorm. */
int lcu_embed_rmsnorm(void* x_out_dev, void* norm_out_dev, const void* ids_dev, int n_ids, int dim,
                      const void* table_dev, const void* scales_dev, int block, int n_vocab,
                      const void* weights_dev, float eps, void* stream);
/* the host argmax of llama_cu.cu:1205-1209 done on the device: index of the first maximum of n
 * fp16 values compared as float, written as int32 */
int lcu_argmax_f16(void* out_index_dev, const void* values_dev, int n, void* stream);
/* softmax_rows over one row of n logits with temperature (launch site 1196) and the argmax of
 * 1205-1209 on its rounded output, in one launch; probs_dev must not alias logits_dev */
int lcu_softmax_argmax(void* probs_dev, void* out_index_dev, const void* logits_dev, int n, float temp,
                       void* stream);
/* lcu_softmax_argmax whose output is two int32: the index, then the stream's count of bounded in-launch
 * waits that ran out (what lcu_sync_timeouts reads) as it stands when this launch runs.  A step that ends
 * with this launch brings its own health back in the copy that fetches the token: a count that has moved
 * since the last step means hand-over words of this step were stale and its token must not be used
 * (the fail-loud rule of llama_cu.h:48-56 applied to the in-launch hand-overs). */
int lcu_softmax_argmax_status(void* probs_dev, void* out_index2_dev, const void* logits_dev, int n, float temp,
                              void* stream);

/* the sampler the reference leaves commented out at llama_cu.cu:1202-1203
 * (std::discrete_distribution over the probabilities): int32 index i drawn with probability
 * p[i] / sum(p) from n fp16 values and 64 random bits, in integer arithmetic (weight = p * 2^24,
 * r = floor(random * total / 2^64), the smallest i whose running weight sum exceeds r; 0 when all
 * weights are 0).  random_dev, when not NULL, points at the 64 bits on the device and replaces
 * `random`, so a captured launch can draw a new number on every replay. */
int lcu_sample_row(void* out_index_dev, const void* probs_dev, int n, uint64_t random, const void* random_dev,
                   void* stream);

/* ---- attention: matmul_qk + softmax_rows + matmul_qkv, llama_cu.cu:400-531, launch sites
 * 1161-1171, without the [n_heads, n, T] score tensor in memory.  q [n_new, dim]; k (already
 * rotated) and v are the first T rows of a [*, dim] cache; causal: row r sees columns
 * c <= r + start_pos.  Scores are rounded to fp16, probabilities are rounded to fp16, the
 * weighted sum runs in fp32: the reference's three rounding points.  head_dim must be 128,
 * T <= 4096 (the multi-row kernel keeps a strip of 16 or 32 rows of scores in LDS).  A call with
 * n_new == 1 hands scores over between workgroups inside its launch when `stream` was made by
 * lcu_stream_create (such a stream owns its hand-over words); on the default stream and on streams
 * made elsewhere, which share the device's, it takes launches that hand nothing over. */
int lcu_attention(void* out_dev, const void* q_dev, const void* k_dev, const void* v_dev,
                  int n_new, int T, int start_pos, int dim, int n_heads, void* stream);

/* lcu_attention for one new token whose position (= T - 1) is read from the device int32 pos_dev
 * when the kernel runs; max_T bounds it (at most the cache length; the position is clamped to it).
 * A bound of 1024 or less selects the single-launch kernel, a larger one the two-launch form that
 * spreads long rows over the chip, so a caller that replays a captured graph keeps the bound at
 * 1024 while the position allows it.  Uses the stream's workspace when max_T > 1024. */
int lcu_attention_decode(void* out_dev, const void* q_dev, const void* k_dev, const void* v_dev,
                         const void* pos_dev, int max_T, int dim, int n_heads, void* stream);

/* lcu_attention_decode with the work of a head spread over eight workgroups, which hand their scores
 * to one another inside the launch through the stream's workspace (same bits as
 * lcu_attention_decode).  Every score travels with the launch's epoch, *seq_dev << 10 | salt: seq_dev is a device
 * uint32 that the caller changes (counts up) before every run of the call, also before every replay
 * of a graph that holds it; salt (0..1023) tells the calls of one such run apart (the layer index).
 * Two consecutive launches on a stream must never have the same epoch.  A hand-over that does not
 * arrive (it cannot on an otherwise idle device) is given up after a bounded wait and counted:
 * lcu_sync_timeouts.  No counterpart in the reference (its score tensor goes through memory
 * between three launches, llama_cu.cu:1161-1171). */
int lcu_attention_decode_spread(void* out_dev, const void* q_dev, const void* k_dev, const void* v_dev,
                                const void* pos_dev, const void* seq_dev, int salt, int max_T, int dim, int n_heads,
                                void* stream);

/* lcu_attention_decode_spread, then x += att . Wo^T (llama_cu.cu:1174, fp16 Wo [dim, dim]) and
 * norm_out = rms_norm(x) with norm_w (1176), in one launch of one 1024-thread workgroup per compute
 * unit: each owns 16 rows of everything, holds its rows of Wo in registers while the attention
 * runs, and takes part in three more hand-overs like the scores' (same epoch rule, same bounded
 * waits).  Same bits as lcu_attention_decode + lcu_gemm_f16_nt (beta 1) + lcu_rmsnorm.  max_T <= 1024;
 * 8 * n_heads workgroups wait for one another and must all be resident, one per compute unit: more
 * heads than a eighth of the compute units are refused (LCU_E_SHAPE), and on a device whose compute
 * units other work holds for good the waits run out (lcu_sync_timeouts) and the result is undefined.
 * Two launches of this entry point must not run at the same time (two streams): each could hold compute
 * units the other is waiting for; the host layer runs one decode step at a time for that reason.
 * x_io_dev: the residual row, updated in place. */
int lcu_decode_attention_wo_norm(void* x_io_dev, void* norm_out_dev, const void* q_dev, const void* k_dev,
                                 const void* v_dev, const void* wo_dev, const void* norm_w_dev, float eps,
                                 const void* pos_dev, const void* seq_dev, int salt, int max_T, int dim, int n_heads,
                                 void* stream);

/* ---- one decode step of several sequences (batching is a TODO of the reference, README.md:34):
 * the GEMMs take the n_seq rows as M; these three handle what differs per sequence.  The caches
 * are given as device arrays of n_seq pointers ([positions][dim] fp16 each), positions as n_seq
 * int32 on the device (row pos[b] is the new one of sequence b). ---- */
/* rotary of row b of q (in place) and of k_new at position pos[b]; rotated k and v_new row b are
 * stored in row pos[b] of sequence b's caches (launch sites 1144-1156 with a position per row) */
int lcu_rope_store_batch(void* q_dev, const void* k_new_dev, const void* v_new_dev, const void* k_cache_ptrs_dev,
                         const void* v_cache_ptrs_dev, const void* pos_dev, int n_seq, int dim, int n_heads,
                         const void* table_dev, int table_positions, void* stream);
/* lcu_attention for one new token (n_new == 1, T cached rows, start_pos = T - 1) that allocates
 * nothing and touches no workspace: no counterpart in the reference; for callers that cannot
 * call hipMalloc (code under HIP graph capture, serving loops and harnesses that forbid it).  The
 * scores of rows longer than 1024 go through a static device array of 64 heads x 4096 rows of
 * fp16 (512 KiB per GPU, held until the process ends): T beyond 4096 or more than 64 heads are
 * rejected (LCU_E_SHAPE), lcu_init must have run on the current device (LCU_E_NOINIT).  Same bits
 * as lcu_attention.  Every call on a GPU uses that GPU's one array: calls that overlap on one GPU
 * (two streams, two threads) race. */
int lcu_attention_decode_static(void* out_dev, const void* q_dev, const void* k_dev, const void* v_dev, int T,
                                int dim, int n_heads, void* stream);
/* lcu_attention_decode for every sequence in one launch: row b of q against rows 0..pos[b] of
 * sequence b's caches -> row b of out; max_T bounds pos[b] + 1 */
int lcu_attention_decode_batch(void* out_dev, const void* q_dev, const void* k_cache_ptrs_dev,
                               const void* v_cache_ptrs_dev, const void* pos_dev, int n_seq, int max_T, int dim,
                               int n_heads, void* stream);
/* The products of a batched step fused with what follows them (for 2..64 sequences the partial sums
 * of the split-K product are added up by the kernel that goes on with them; any other shape runs
 * the separate operators above).  w_dev / scales_dev: host arrays of device pointers (scales NULL
 * and block 0 for fp16 weights); *_tmp_dev: [n_seq][dim] / [n_seq][ffn] fp16 scratch.
 *   lcu_batch_qkv: Wq, Wk, Wv products of lhs [n_seq][dim], then lcu_rope_store_batch (1144-1156)
 *   lcu_batch_ffn_up: W1, W3 products, then fp16(silu(w1) * w3) (1180-1183)
 *   lcu_batch_proj_norm: x += lhs [n_seq][K] * W^T (1174 / 1185), then norm_out = rms_norm(x) with
 *     norm_w (1176, or 1129 of the next layer, or 1191) */
int lcu_batch_qkv(void* q_out_dev, void* k_tmp_dev, void* v_tmp_dev, const void* lhs_dev, const void* const* w_dev,
                  const void* const* scales_dev, int block, int n_seq, int dim, int n_heads,
                  const void* k_cache_ptrs_dev, const void* v_cache_ptrs_dev, const void* pos_dev,
                  const void* table_dev, int table_positions, void* stream);
int lcu_batch_ffn_up(void* out_dev, void* w1_tmp_dev, void* w3_tmp_dev, const void* lhs_dev, const void* const* w_dev,
                     const void* const* scales_dev, int block, int n_seq, int dim, int ffn, void* stream);
int lcu_batch_proj_norm(void* x_dev, void* norm_out_dev, const void* lhs_dev, const void* w_dev, const void* scales_dev,
                        int block, int n_seq, int K, int dim, const void* norm_w_dev, float eps, void* stream);
/* lcu_softmax_argmax on `rows` rows of n logits (n a multiple of 8): probabilities [rows][n],
 * one int32 index per row */
int lcu_softmax_argmax_rows(void* probs_dev, void* out_index_dev, const void* logits_dev, int rows, int n, float temp,
                            void* stream);

/* ---- fused decode steps (n_new == 1), each replacing several launch sites of next_token ---- */
/* rms_norm(x, attn_norm) -> Wq/Wk/Wv GEMV -> RoPE(q, k at position pos) -> q to q_out, k and v into
 * row pos of the caches: llama_cu.cu:1129-1156.  Weight pointers are fp16 [dim, dim], or uint8 codes
 * with fp16 scales when block > 0.  norm_w_dev == NULL means x_dev is already normalised
 * (lcu_rmsnorm ran first); the same holds for lcu_decode_ffn_up.  pos_dev != NULL: the position is
 * read from that device int32 when the kernel runs (`pos` is ignored), so that one captured graph
 * serves every decode step. */
int lcu_decode_qkv(void* q_out_dev, void* k_cache_dev, void* v_cache_dev, const void* x_dev,
                   const void* norm_w_dev, const void* wq_dev, const void* wk_dev, const void* wv_dev,
                   const void* sq_dev, const void* sk_dev, const void* sv_dev, int block, int dim,
                   int n_heads, int pos, const void* pos_dev, float eps, const void* rope_table_dev,
                   int table_positions, void* stream);
/* x += lhs [1, K] . W^T (W [N, K], fp16 or uint8 codes with scales; llama_cu.cu:1185) and then
 * norm_out = rms_norm(x) with norm_w (1129 of the next layer), in one launch: one more workgroup
 * than the GEMV has waits inside the launch for the rows of the new x, which reach it as
 * {two halves, epoch} words through the stream's workspace, and writes x and its norm.  The epoch is
 * *seq_dev << 10 | salt, as for lcu_attention_decode_spread (same rule, same bounded wait).  Same
 * bits as lcu_gemm_f16_nt / lcu_gemm_f16u8_nt (beta 1) + lcu_rmsnorm.  N <= 8192. */
int lcu_decode_proj_norm(void* x_io_dev, void* norm_out_dev, const void* lhs_dev, const void* w_dev,
                         const void* scales_dev, int block, int K, int N, const void* norm_w_dev, float eps,
                         const void* seq_dev, int salt, void* stream);
/* rms_norm(x, ffn_norm) -> W1 and W3 GEMV -> silu(w1) * w3: llama_cu.cu:1176-1183 */
int lcu_decode_ffn_up(void* out_dev, const void* x_dev, const void* norm_w_dev, const void* w1_dev,
                      const void* w3_dev, const void* s1_dev, const void* s3_dev, int block, int dim,
                      int ffn, float eps, void* stream);
/* rms_norm(x, norm) -> output GEMV: llama_cu.cu:1191-1195 for the single row that is used */
int lcu_decode_logits(void* logits_dev, const void* x_dev, const void* norm_w_dev,
                      const void* wout_dev, const void* sout_dev, int block, int dim, int n_vocab,
                      float eps, void* stream);

/* ---- synthetic tensors (no counterpart in the reference, which reads weights from files):
 * value[i] = fp16(float(S - 262140) * scale), S = sum of the eight 16-bit fields of two chained
 * splitmix64 hashes of (seed, stream_id, i), scale = float(std / sqrt(8 * (65536^2 - 1) / 12)).
 * Integer-exact, so any host restating the recipe gets the same bits. */
int lcu_fill_normal_f16(void* out_dev, size_t n, uint64_t seed, uint64_t stream_id, float std,
                        void* stream);
int lcu_fill_f16(void* out_dev, size_t n, uint16_t bits, void* stream);

/* error_stats, transform.cu:99-150 (launch site 175): out3 = {mean squared difference, largest
 * absolute difference, mean absolute difference} of two fp16 arrays of n elements, as fp32.
 * Deterministic (partials are added in index order, where the reference uses atomics).  Uses the
 * stream's workspace. */
int lcu_error_stats(void* out3_dev, const void* a_dev, const void* b_dev, size_t n, void* stream);

/* ---- layered decoders: models built from a list of layers (no counterpart in the reference, whose only
 * model is the LLaMA above).  Element type: activations and weights are bfloat16 or fp32; products
 * accumulate in fp32; the residual stream, norms, router, gates, recurrent state, scores and softmax are
 * fp32 whatever the element type.  Vectors (biases, norm weights, decays) are fp32.  Rows of activations
 * and weights are padded with zeros to a multiple of 64 elements ("ld"), so every K is one. ---- */
#define LCU_BF16 0
#define LCU_F32 1

/* out[M,N] (row stride ldo) = lhs[M,K] . w[N,K]^T + bias; columns below gelu_cols then pass through the tanh
 * GELU.  Output of the element type, or fp32 when out_f32. */
int lcu_linear(void* out_dev, int out_f32, int ldo, const void* lhs_dev, const void* w_dev, const void* bias_dev,
               int gelu_cols, int dtype, int M, int K, int N, void* stream);

/* the same without bias; columns from tail_from on go to fp32 rows tail [M][ld_tail] instead */
int lcu_linear_tail(void* out_dev, int ldo, void* tail_f32_dev, int ld_tail, int tail_from, const void* lhs_dev, const void* w_dev,
                    int dtype, int M, int K, int N, void* stream);

/* clamped gated unit: g = min(gate, limit), u = clamp(up, +-limit), g sigmoid(alpha g) (u + up_shift) */
typedef struct lcu_gate_params {
  float limit, alpha, up_shift;
} lcu_gate_params;
/* out[M][N/2] = gated unit of lhs . w^T; w holds, in blocks of 64 rows, 32 gate rows and then the 32 up rows
 * of the same outputs (N a multiple of 64) */
int lcu_linear_gated(void* out_dev, int ldo, const void* lhs_dev, const void* w_dev, const lcu_gate_params* gate, int dtype,
                     int M, int K, int N, void* stream);

/* Mixture of experts.  lcu_router: per token the `top` experts with the largest scores sigmoid(z), z = w . h
 * in fp32 (int32 [n][top], fp32 [n][top]), and sigmoid of row n_experts of w (one more row) when
 * shared_gate_dev is given.  lcu_experts_plan sorts the choices by expert: row r of the sorted order is
 * token row_token[r] with weight row_weight[r], choice k of token t lies at row inverse[t * top + k], and
 * tiles of at most tile_rows rows of one expert are listed.  lcu_experts_up: gated unit of
 * row_weight[r] * h[row_token[r]] through expert e's matrix (w_dev + e * expert_stride bytes);
 * lcu_experts_down: the rows' second product, fp32.  Arrays of the plan are device memory: row_* and
 * inverse n * top entries, tile_* max_tiles, expert_end n_experts, n_tiles one.  tile_rows is 64, 128
 * or 256 (bfloat16), 32 (fp32). */
typedef struct lcu_expert_plan {
  void* row_token_dev;
  void* row_weight_dev;
  void* inverse_dev;
  void* tile_expert_dev;
  void* tile_row_dev;
  void* expert_end_dev;
  void* n_tiles_dev;
  int tile_rows;
  int max_tiles;
} lcu_expert_plan;
int lcu_router(void* expert_dev, void* weight_dev, void* shared_gate_dev, const void* h_dev, const void* w_dev, int n_experts,
               int top, int dtype, int n, int K, void* stream);
int lcu_experts_plan(const lcu_expert_plan* plan, const void* expert_dev, const void* weight_dev, int n, int top, int n_experts,
                     void* stream);
int lcu_experts_up(void* out_dev, int ldo, const void* lhs_dev, const void* w_dev, size_t expert_stride,
                   const lcu_gate_params* gate, const lcu_expert_plan* plan, int dtype, int n_tokens, int K, int N,
                   void* stream);
int lcu_experts_down(void* out_f32_dev, int ldo, const void* lhs_dev, const void* w_dev, size_t expert_stride,
                     const lcu_expert_plan* plan, int dtype, int n_rows, int K, int N, void* stream);

/* Row kernels; a row is `width` of ld elements, its RMS norm taken over `groups` equal consecutive parts.
 * Norm weights are fp32 vectors of ld entries.  lcu_embed_pos_norm: x = norm(table[id] + pos_table[*start + row]) under w_embed, h = norm(x) under w_next
 * (NULL: none).  lcu_residual_norm: m = per token the sum of `top` fp32 rows of out (rows
 * inverse[token * top + k], or token * top + k when inverse is NULL) and shared_gate[row] times the shared
 * expert's row; x += norm(m) under w_after; h =
 * norm(x) under w_next.  Where w_next is NULL and h is given, h = x as it is.  lcu_embed_scaled: x = scale *
 * table[id], h likewise.  lcu_group_norm: h[i] = norm(x[row_index[i]]). */
int lcu_embed_pos_norm(void* x_dev, void* h_dev, const void* ids_i32_dev, int n_ids, const void* table_dev, int n_vocab,
                       const void* pos_table_dev, int n_pos, const void* start_dev, const void* w_embed_dev,
                       const void* w_next_dev, int dtype, int width, int ld, int groups, float eps, void* stream);
int lcu_embed_scaled(void* x_dev, void* h_dev, const void* ids_i32_dev, int n_ids, const void* table_dev, int n_vocab, float scale,
                     const void* w_next_dev, int dtype, int width, int ld, int groups, float eps, void* stream);
int lcu_residual_norm(void* x_dev, void* h_dev, const void* out_f32_dev, const void* inverse_dev, int top,
                      const void* shared_f32_dev, const void* shared_gate_dev, const void* w_after_dev,
                      const void* w_next_dev, int dtype, int rows, int width, int ld, int groups, float eps, void* stream);
int lcu_group_norm(void* h_dev, const void* x_f32_dev, const void* row_index_dev, const void* w_dev, int dtype, int rows,
                   int width, int ld, int groups, float eps, void* stream);
/* index = first maximum of n fp32 values; probs = fp16(softmax(logits / temp)) of one row of n */
int lcu_argmax_f32(void* out_index_dev, const void* values_dev, int n, void* stream);
int lcu_softmax_f32(void* probs_f16_dev, const void* logits_dev, int n, float temp, void* stream);

/* Gated linear recurrence.  Channels lie block by block, each block padded to a multiple of 32.
 * lcu_conv_causal: u[t] = bias + sum over taps of w[k] z[t - (taps - 1) + k] per channel (w fp32
 * [taps][ld], bias NULL: none), then silu when asked; inputs before this call come from state [taps - 1][ld] (element type), which is then
 * brought up to date.  lcu_gated_recurrence: r, i = sigmoid of the block-diagonal products of u (w
 * [blocks][block_width][block_width]) plus bias, log a = decay r, S = a S + sqrt(1 - a^2) i u from the fp32
 * state [ld], which is brought up to date; out = S * y.  scratch: lcu_gated_recurrence_scratch bytes. */
int lcu_conv_causal(void* u_dev, const void* z_dev, int ldz, const void* w_dev, const void* bias_dev, void* state_dev, int taps,
                    int silu, int dtype, int n, int channels, int ld, void* stream);
size_t lcu_gated_recurrence_scratch(int n, int ld);
int lcu_gated_recurrence(void* out_dev, const void* u_dev, const void* y_dev, int ldy, const void* wr_dev, const void* wi_dev,
                         const void* br_dev, const void* bi_dev, const void* decay_dev, void* state_dev, void* scratch_dev,
                         int dtype, int n, int channels, int block_width, int ld, void* stream);

/* Sliding-window attention with kept first tokens, grouped heads and a per-head distance bias: key j of
 * position i is visible when j <= i and (i - j < window or j < keep), its score scale q.k - r1 ln(1 + r2
 * (i - j)).  dk: head size padded to a multiple of 32 (at most 256); dv: value size padded to 32, 64, 128 or
 * 256.  Caches [positions][kv_heads * dk] and [positions][kv_heads * dv]. */
typedef struct lcu_window_params {
  int heads, kv_heads, dk, dv, window, keep;
  float scale;
  const void* r1_dev; /* fp32 [heads]; NULL: no distance bias */
  const void* r2_dev;
  /* lcu_attention_windowed only; zeros: nothing of this.  The last dk_shared columns of a key come from
   * k_shared [position][dk_shared], the same for all heads; k_ld, v_ld: elements from position to position (0:
   * kv_heads times the own columns); first_position: that of row 0 of k, v and k_shared, at or before the first
   * window's begin; sink: fp32 [heads], exp(sink) is added to the denominator; gate [n][ldg]: the result is
   * multiplied with sigmoid(gate). */
  int dk_shared, k_ld, v_ld, first_position;
  const void* k_shared_dev;
  const void* sink_dev;
  const void* gate_dev;
  int ldg;
} lcu_window_params;
/* Rows q | k | v of a projection: k and v of row t into cache row *start + t.  v_mode 0: v as it is; 1: and
 * a copy into v_first [n][v_cols]; 2: (1 - lambda) v + lambda v_first. */
int lcu_kv_store(void* k_cache_dev, void* v_cache_dev, const void* qkv_dev, int ldq, int q_cols, int k_cols, int v_cols,
                 void* v_first_dev, int v_mode, const void* lambda_dev, const void* start_dev, int max_positions, int dtype, int n,
                 void* stream);
int lcu_attention_windowed(void* out_dev, int ldo, const void* q_dev, int ldq, const void* k_cache_dev, const void* v_cache_dev,
                           int start, const lcu_window_params* window, int dtype, int n, void* stream);
/* one new token at position *pos_dev (bfloat16), the visible keys spread over the chip; arrived_dev: kv_heads
 * uint32, zero before the call and after it (the workgroup that arrives last adds the parts up; nobody waits).
 * Uses the stream's workspace. */
int lcu_attention_windowed_decode(void* out_dev, const void* q_dev, const void* k_cache_dev, const void* v_cache_dev,
                                  const void* pos_dev, int max_positions, const lcu_window_params* window, void* arrived_dev,
                                  void* stream);

/* Latent attention: keys and values of all heads are products of one normed latent c per token (and a rotated key
 * part that the heads share).  Head parts are padded to multiples of 32 (dn unrotated, dr rotated of which the
 * first rot are turned in pairs (2i, 2i + 1); dr 0: no rotated part), values to dv, the latent to ldc (a multiple
 * of 64); window INT_MAX: every key before.  A query head is [dn | dr]. */
typedef struct lcu_latent_params {
  int heads, dn, dr, rot, dv, rank, ldc, window;
  float scale;
} lcu_latent_params;
/* Projected rows [n][ld] of tokens *start ...: c (rank columns from latent_at) is normed into row *start + t of
 * latents [max_positions][ldc]; the shared key part (from key_at) is rotated into keys [max_positions][dr]; when
 * rotate_queries, the rotated part of head h (from query_at + h (dn + dr)) is rotated in place; when low_rank > 0 the
 * first low_rank columns are normed into low [n][low_ld].  Angle of pair i at position p: p freq[i]; gain: factor
 * on cosine and sine.  Norm weights are fp32, padded like what they scale. */
typedef struct lcu_latent_rows_args {
  void* rows_dev;
  int ld, n, latent_at, key_at, query_at, rotate_queries, low_rank, low_ld, max_positions;
  const void* latent_norm_dev;
  const void* low_norm_dev;
  void* low_dev;
  void* latents_dev;
  void* keys_dev;
  const void* freq_dev; /* fp32 [rot / 2] */
  float gain, eps;
  const void* start_dev;
} lcu_latent_rows_args;
int lcu_latent_rows(const lcu_latent_rows_args* rows, const lcu_latent_params* p, int dtype, void* stream);
/* Few tokens, bfloat16, without keys and values multiplied out.  lcu_latent_queries: out [n][heads * ldc], head h =
 * uk_t[h] [ldc][dn] times the unrotated part of the query; with rows, lcu_latent_rows in the same launch (the
 * unrotated parts do not depend on it).  lcu_latent_attention: scores and softmax over the latents (sink as above,
 * NULL: none), then uv [heads * dv][ldc] and the gate (NULL: none).  scratch: lcu_latent_attention_scratch bytes;
 * lcu_latent_attention_fits: 0 where the sizes are too large for its kernels (ldc above 512). */
int lcu_latent_queries(void* out_dev, const void* q_dev, int ldq, const void* uk_t_dev, const lcu_latent_params* p,
                       const lcu_latent_rows_args* rows, int n, void* stream);
int lcu_latent_attention_fits(const lcu_latent_params* p);
int lcu_latent_slices(const lcu_latent_params* p, int n, int max_positions);
size_t lcu_latent_attention_scratch(const lcu_latent_params* p, int n, int max_positions);
int lcu_latent_attention(void* out_dev, int ldo, const void* q_latent_dev, const void* q_rot_dev, int ldq, const void* latents_dev,
                         const void* keys_dev, const void* start_dev, int max_positions, const void* uv_dev, const void* sink_dev,
                         const void* gate_dev, int ldg, const lcu_latent_params* p, void* scratch_dev, int n, void* stream);

/* Gated delta rule.  Channels q [kv_heads * dk] | k [kv_heads * dk] | v [heads * dv] of a token (after their convolution,
 * rows of ld), dim in dk (32, 64, 128 or 256) and vdim in dv (a multiple of 32, at most 256), padding zero; query/key
 * head h / (heads / kv_heads).  q and k are made unit vectors (eps 1e-6), q times dim^-1/2; beta = sigmoid(b), g =
 * exp(-exp(a_log) softplus(a + dt_bias)), from fp32 rows [b | a]; S = g S, S += k (beta (v - S^T k))^T, o = S^T q; out
 * = rms norm of o over vdim, times norm, times silu(gate).  state: fp32 [heads][dk][dv], brought up to date. */
typedef struct lcu_delta_params {
  int heads, kv_heads, dk, dv, dim, vdim;
  float eps;
  const void* a_log_dev;   /* fp32 [heads] */
  const void* dt_bias_dev; /* fp32 [heads] */
  const void* norm_dev;    /* fp32 [vdim] */
} lcu_delta_params;
size_t lcu_delta_rule_scratch(const lcu_delta_params* d, int n);
int lcu_delta_rule(void* out_dev, int ldo, const void* qkv_dev, int ld, const void* gate_dev, int ldg, const void* ba_f32_dev, int ld_ba,
                   const lcu_delta_params* d, void* state_dev, void* scratch_dev, int dtype, int n, void* stream);

/* One new token, bfloat16, fused.  x is normalised already.
 *   lcu_decode_linear: fp32 out = w . x + bias
 *   lcu_decode_linear_bf16: the same without bias, bfloat16 out
 *   lcu_decode_delta_in: the first `channels` rows through the step of the convolution and silu (w [taps][channels],
 *     state [taps - 1][channels]) to u, `plain` rows to plain, the rest to tail in fp32
 *   lcu_decode_delta_step: lcu_delta_rule for one token
 *   lcu_decode_gated: lcu_linear_gated for one token (ld hidden units)
 *   lcu_decode_recurrent_in: rows y (GELU) and x of a recurrent block, the latter through the convolution
 *   lcu_decode_recurrent_step: gates and state of lcu_gated_recurrence for one token
 *   lcu_decode_kv: rows q | k | v, then lcu_kv_store at position *pos
 *   lcu_decode_experts_up: hidden activations of the chosen experts (w at up + choice * up_stride bytes,
 *     packed as for lcu_linear_gated, K columns; ld hidden units each) and of the shared one
 *   lcu_decode_experts_down: slot s: fp32 row out + s * ldo = w[choice[s]] . hidden[s]; the shared product is
 *     slot `slots`
 *   lcu_decode_residual_router: lcu_residual_norm of the row (the sum of `top` rows of out and the gated shared
 *     row), then lcu_router of it when router_w is given */
int lcu_decode_linear(void* out_f32_dev, const void* x_dev, const void* w_dev, const void* bias_dev, int K, int N, void* stream);
int lcu_decode_linear_bf16(void* out_dev, const void* x_dev, const void* w_dev, int K, int N, void* stream);
int lcu_decode_delta_in(void* u_dev, void* plain_dev, void* tail_f32_dev, void* conv_state_dev, const void* x_dev, const void* w_dev,
                        const void* conv_dev, int taps, int K, int channels, int plain, int N, void* stream);
int lcu_decode_delta_step(void* out_dev, const void* qkv_dev, const void* gate_dev, const void* ba_f32_dev, const lcu_delta_params* d,
                          void* state_dev, void* stream);
int lcu_decode_gated(void* hidden_dev, const void* h_dev, const void* w_dev, const lcu_gate_params* gate, int ld, int K, void* stream);
int lcu_decode_recurrent_in(void* y_dev, void* u_dev, void* conv_state_dev, const void* x_dev, const void* w_dev,
                            const void* bias_dev, const void* conv_dev, const void* conv_bias_dev, int taps, int K, int ld,
                            void* stream);
int lcu_decode_recurrent_step(void* out_dev, const void* u_dev, const void* y_dev, const void* wr_dev, const void* wi_dev,
                              const void* br_dev, const void* bi_dev, const void* decay_dev, void* state_dev, int channels,
                              int block_width, void* stream);
int lcu_decode_kv(void* q_out_dev, void* k_cache_dev, void* v_cache_dev, const void* x_dev, const void* w_dev, const void* bias_dev,
                  int q_cols, int k_cols, int v_cols, void* v_first_dev, int v_mode, const void* lambda_dev, const void* pos_dev,
                  int max_positions, int K, void* stream);
int lcu_decode_experts_up(void* hidden_dev, void* shared_hidden_dev, const void* h_dev, const void* choice_dev,
                          const void* weight_dev, const void* up_dev, size_t up_stride, const lcu_gate_params* gate,
                          const void* shared_up_dev, const lcu_gate_params* shared_gate, int top, int ld, int shared_ld, int K,
                          void* stream);
int lcu_decode_experts_down(void* out_f32_dev, int ldo, const void* hidden_dev, const void* choice_dev, const void* w_dev,
                            size_t stride, int slots, int K, const void* shared_hidden_dev, const void* shared_w_dev, int shared_K,
                            int N, void* stream);
int lcu_decode_residual_router(void* x_dev, void* h_dev, const void* out_f32_dev, int top, const void* shared_f32_dev,
                               const void* shared_gate_dev, const void* w_after_dev, const void* w_next_dev, int width, int ld,
                               int groups, float eps, const void* router_w_dev, int n_experts, int choose, void* expert_dev,
                               void* weight_dev, void* router_gate_dev, void* stream);

/* pseudo-random matrix (synthetic weights): mean + std * N(0, 1) (the hash of lcu_fill_normal_f16) into
 * columns 0 .. cols - 1 of rows of ld elements */
int lcu_fill_normal_matrix(void* out_dev, size_t rows, int cols, int ld, int dtype, uint64_t seed, uint64_t stream_id, float mean,
                           float std, void* stream);

#ifdef __cplusplus
}
#endif
#endif
