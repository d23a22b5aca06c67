// Python bindings for the omnia_amd gfx950 kernels.  Each entry validates the
// operand shapes/dtypes on the host BEFORE launching (a bad launch on the box
// can take every GPU of the host down), then launches on the current HIP
// stream so the calls are capturable into hipGraphs by the engine.
#include <chrono>
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>
#include <hip/hip_runtime.h>

// the layout of mask.h's struct: (window, kept first positions, chunk)
struct Mask { int window, keep, chunk; };
// of score.h's: (scale, cap, r1, r2)
struct Score { float scale, cap; const float *r1, *r2; };

extern "C" {
int omnia_pgemm(int epi, void* out, const void* X, const void* W, int M, int N, int K, int ldo,
                const float* ss_in, int ss_in_n, float inv_d, float eps, float* ss_out,
                const int* positions, const float* cos_sin, void* k_cache, void* v_cache,
                const int64_t* slots, int hq, int hkv, int block_size, const float* bias,
                int gelu, hipStream_t s);
int omnia_row_sumsq(float* ss, const void* x, int rows, int d, int64_t stride, hipStream_t s);
int omnia_ar_alltoall(void* out, const void* in, void* const* regions, int* epochs, int* err,
                      int64_t chunk, int64_t slot_bytes, int rank, int world, hipStream_t s);
int omnia_ar_sendrecv(void* out, const void* in, void* const* regions, int* epochs, int* err,
                      int64_t nbytes, int64_t slot_bytes, int rank, int world, int src_rank,
                      hipStream_t s);
int omnia_pgemm_set_schedule(int sched);
int omnia_pgemm_splitk(void* parts, const void* X, const void* W, int M, int N, int K, int S,
                       int sched, hipStream_t s);
int omnia_pgemm_moe(int mode, void* out, const void* A, const void* W, const int* sorted,
                    const int* blk_expert, const int* n_blocks, const float* route_w, int K,
                    int N, int topk, int n_assign, int e_lo, int max_blocks, float alpha,
                    float limit, hipStream_t s);
int omnia_pgemm_variant(int variant, void* out, const void* X, const void* W, int M, int N,
                        int K, hipStream_t s);
int omnia_rmsnorm(void* out, const void* x, void* residual, const void* w, int rows, int d,
                  int64_t x_stride, int64_t out_stride, float eps, hipStream_t s);
int omnia_rope_kv(void* q, void* k, const void* v, const int* positions, const float* cos_sin,
                  void* k_cache, void* v_cache, const int64_t* slots, int T, int hq, int hkv,
                  int head_dim, int64_t q_stride, int64_t kv_stride, int block_size,
                  hipStream_t s);
int omnia_silu_mul(void* out, const void* x, int64_t T, int inter, hipStream_t s);
int omnia_embedding(void* out, const int* ids, const void* w, int T, int d, int vocab_start,
                    int vocab_end, const int64_t* src, const int* tok_slots, hipStream_t s);
int omnia_decode_attention(void* out, float* part_o, float* part_ml, const void* q,
                           const void* k_cache, const void* v_cache, const int* block_tables,
                           int bt_stride, const int* seq_lens, int B, int hq, int hkv,
                           int head_dim, int block_size, int64_t q_stride, int part_size,
                           int max_parts, float scale, int split_t, int split_min,
                           hipStream_t s);
int omnia_prefill_attention(void* out, const void* q, const void* k_cache, const void* v_cache,
                            const int* block_tables, int bt_stride, const int* q_start_loc,
                            const int* seq_lens, const int* tile_seq, const int* tile_q0,
                            int n_tiles, int hq, int hkv, int head_dim, int block_size,
                            int64_t q_stride, int64_t out_stride, float scale, int hp,
                            int q_tile, float* lse_out, const int* kv_lens, hipStream_t s);
int omnia_apply_token_mask(void* logits, int logits_is_bf16, int rows, int64_t row_stride,
                           int vocab, const uint32_t* mask, int words, hipStream_t s);
int omnia_sample(int* out_tok, float* out_logprob, const void* logits, int logits_is_bf16,
                 int rows, int64_t row_stride, int vocab, const float* temperature,
                 const int* top_k, const float* top_p, const uint64_t* seeds,
                 const int64_t* steps, int* counts, const float* freq_pen, const float* pres_pen,
                 const float* rep_pen, int* tok_slots, const int64_t* dst, hipStream_t s);
int omnia_tp_gumbel(float* pack, int64_t ld, int col, const void* logits, int rows,
                    int64_t row_stride, int vocab, int vocab_start, const float* temperature,
                    const int* top_k, const float* top_p, const int64_t* seeds,
                    const int64_t* steps, hipStream_t s);
int omnia_tp_pack(float* pack, int64_t ld, int K, const void* logits, int rows,
                  int64_t row_stride, int vocab, int vocab_start, const float* temperature,
                  const int* top_k, const float* top_p, const int64_t* seeds,
                  const int64_t* steps, hipStream_t s);
int omnia_tp_merge(int* out, int* tok_slots, const int64_t* dst_slot, const float* allp, int W,
                   int B, int64_t ld, int K, const float* temperature, const int* top_k,
                   const float* top_p, const int64_t* seeds, const int64_t* steps,
                   hipStream_t s);
int omnia_mean_pool_l2(float* out, const void* hidden, int64_t stride, const int* cu, int B,
                       int D, hipStream_t s);
int omnia_cosine_scores(float* scores, const float* q, int nq, const void* m, int64_t N, int D,
                        const uint8_t* valid, hipStream_t s);
int omnia_topk(int* out_idx, float* out_val, const float* scores, int nq, int64_t N, int k,
               hipStream_t s);
int omnia_moe_topk(int* ids, float* wts, const void* logits, int logits_bf16, int n_tok, int E,
                   int k, int renorm, hipStream_t s);
int omnia_moe_max_blocks(int n_assign, int n_experts, int bm);
int omnia_moe_router_topk(int* ids, float* wts, const void* x, const void* router, int n_tok,
                          int d, int E, int k, int renorm, hipStream_t s);
int omnia_moe_align(int* sorted, int* blk_expert, int* n_blocks, const int* ids, int n, int E,
                    int e_lo, int e_hi, int max_blocks, int bm, hipStream_t s);
int omnia_moe_route(int* ids, float* wts, const void* x, const void* router, int f32, int n_tok,
                    int d, int E, int k, int sigmoid, int renorm, const float* corr, int groups,
                    int keep, const float* bias, hipStream_t s);
int omnia_moe_gemm(int mode, void* out, const void* A, const void* W, int f32, const int* sorted,
                   const int* blk_expert, const int* n_blocks, const float* route_w, int K, int N,
                   int topk, int n_assign, int e_lo, int max_blocks, float alpha, float limit,
                   hipStream_t s);
int omnia_moe_combine(void* out, const void* Y, const int* ids, int n_tok, int d, int topk,
                      int e_lo, int e_hi, hipStream_t s);
int omnia_ipc_handle_size();
int omnia_ipc_alloc(void** ptr, int64_t bytes);
int omnia_ipc_free(void* ptr);
int omnia_ipc_get_handle(void* ptr, void* handle_out);
int omnia_ipc_open(const void* handle, void** ptr);
int omnia_ipc_close(void* ptr);
int omnia_ar_blocks();
int omnia_ar_max_ranks();
int omnia_ar_oneshot(void* out, const void* in, void* const* regions, int* epochs, int* err,
                     int64_t n, int64_t slot_bytes, int rank, int world, hipStream_t s);
int omnia_splitk_add_rmsnorm(void* out, const void* parts, int half, void* residual, const void* w, int S,
                             int M, int d, float eps, hipStream_t s);
int omnia_splitk_rope_kv(void* q, const void* parts, int half, int S, int T, const int* positions,
                         const float* cos_sin, void* k_cache, void* v_cache, const int64_t* slots,
                         int hq, int hkv, int head_dim, int block_size, hipStream_t s);
int omnia_splitk_swiglu(void* out, const void* parts, int half, int S, int M, int inter, hipStream_t s);
int omnia_splitk_reduce(void* out, const void* parts, int half, int S, int64_t n, hipStream_t s);
int64_t omnia_ar_region_bytes(int64_t slot_bytes);
int omnia_ar_twoshot(void* out, const void* in, void* residual, const void* w,
                     void* const* regions, int* epochs, int* err, int M, int d,
                     int64_t slot_bytes, int rank, int world, float eps, hipStream_t s);
int omnia_wgemm(int mode, void* out, const void* X, const void* W, int M, int N, int K, int S,
                int nw, int nwaves, int ldo, hipStream_t s);
int omnia_wgemm_wide(int mode, void* out, const void* X, const void* W, int M, int N, int K,
                     int S, int wt, int ldo, hipStream_t s);
int omnia_dgemm(int mode, void* out, const void* X, const void* W, float* ws, int* cnt, int M,
                int N, int K, int S, int wm, int wn, int ldo, int64_t ws_floats, int cnt_len,
                hipStream_t s);
int omnia_ar_allgather(void* out, const void* in, void* const* regions, int* epochs, int* err,
                       int64_t nbytes, int64_t slot_bytes, int rank, int world, hipStream_t s);
int omnia_tgemm(int mode, void* out, const void* X, const void* W, int M, int N, int K, int S,
                int bn, int wnt, int ldo, hipStream_t s);
int omnia_tanh_norm_embed(void* h, float* x, const int* ids, const void* table, int f32, int T,
                          int d, int vocab, float alpha, const float* w, const float* b,
                          const int64_t* src, const int* tok_slots, hipStream_t s);
int omnia_tanh_norm_residual(void* h, int f32, float* x, const void* m, int ptype, int S,
                             int64_t row, int64_t slab, int rows, int d, const float* bias,
                             float a1, const float* w1, const float* b1, float a2,
                             const float* w2, const float* b2, const int* ids, const float* wts,
                             const void* in, int first, hipStream_t s);
int omnia_glu(void* out, int f32, const void* m, int ptype, int S, int rows, int inter,
              const float* bias, int gelu, hipStream_t s);
int omnia_branch_residual(void* h, int f32, float* x, int rows, int d, const void* a, int at,
                          int aS, int64_t arow, int64_t aslab, const float* abias,
                          const float* aw, const void* b, int bt, int bS, int64_t brow,
                          int64_t bslab, const float* bbias, const float* bw, float inv_n,
                          float eps, float alpha, const float* nw, const float* nb,
                          hipStream_t s);
int omnia_lightning_pow_cols();
int64_t omnia_lightning_scratch(int n_rows, int nseq, int H, int Dp, int Vp);
int omnia_lightning_step(float* o, float* state, const void* x, int ptype, int S, int64_t ld,
                         int64_t slab, const float* pw, const int* positions, const int* slots,
                         int T, int H, int Dp, int Vp, hipStream_t s);
int omnia_lightning_scan(float* o, float* state, float* seg, const void* x, int f32, int64_t ldx,
                         const float* pw, const int* q_start, int nseq, const int* positions,
                         const int* slots, int n_rows, int H, int Dp, int Vp, hipStream_t s);
int omnia_lightning_norm(void* y, int f32, const float* o, const void* x, int ptype, int S,
                         int64_t ld, int64_t slab, int goff, const float* w, int T, int n,
                         float inv_n, float eps, hipStream_t s);
int omnia_delta_prep(float* qn, float* kn, void* vc, float* decay, float* beta, const void* x,
                     int f32, int64_t ldx, const void* conv_w, const void* conv_state,
                     const float* a_log, const float* dt_bias, const int* q_start, int nseq,
                     const int* positions, const int* slots, int T, int KH, int H, int D, int Dp,
                     int V, int taps, hipStream_t s);
int omnia_delta_step(void* y, float* state, void* conv_state, const float* qn, const float* kn,
                     const void* vc, const float* decay, const float* beta, const void* x, int f32,
                     int64_t ldx, const float* norm_w, const int* positions, const int* slots,
                     int T, int KH, int H, int D, int Dp, int V, int Vs, int Vp, int taps,
                     float eps, hipStream_t s);
int64_t omnia_delta_records(int n_rows, int nseq, int H);
int omnia_delta_scan(float* o, float* state, void* conv_state, float* rec, const float* qn,
                     const float* kn, const void* vc, const float* decay, const float* beta,
                     const void* x, int f32, int64_t ldx, const int* q_start, int nseq,
                     const int* positions, const int* slots, int n_rows, int KH, int H, int D, int Dp, int V, int Vs, int taps,
                     hipStream_t s);
int omnia_delta_norm(void* y, const float* o, const void* x, int f32, int64_t ldx, int zoff,
                     const float* norm_w, int T, int H, int V, int Vs, int Vp, float eps,
                     hipStream_t s);
int omnia_rms_embed(void* h, float* x, const int* ids, const void* table, int f32, int T, int d,
                    int vocab, const float* we, const float* wp, float inv_n, float eps,
                    const int64_t* src, const int* tok_slots, hipStream_t s);
int omnia_rms_residual(void* h, int f32, float* x, const void* m, int ptype, int S,
                       int64_t row_stride, int64_t part_stride, int rows, int d,
                       const float* bias, const float* w_post, const float* w_pre, float inv_n, float eps,
                       hipStream_t s);
int omnia_softcap(void* z, int f32, int64_t n, float cap, hipStream_t s);
int omnia_gqa_prep(void* q, void* kc, void* vc, int f32, const void* x, int ptype, int S,
                   int64_t slab, int64_t ldx, const float* wq, const float* wk,
                   const float* bias, const int* positions, const int64_t* slots,
                   const float* cos_sin, int pairs, int T, int H, int G, int D, int Dp, int Vp,
                   int R, int page, float eps, const float* temp, float* gate, hipStream_t s);
int omnia_gqa_attend(void* out, int f32, const void* q, const void* kc, const void* vc,
                     const int* block_tables, int bt_stride, const int* q_start, int nseq,
                     const int* positions, int T, int page, int H, int G, int Dp, int Vp,
                     Mask mask, Score score, const float* sinks, const float* gate,
                     hipStream_t s);
int omnia_gqa_decode(void* out, float* part_o, float* part_ml, const void* q, const void* kc,
                     const void* vc, const int* block_tables, int bt_stride, const int* positions,
                     int T, int page, int H, int G, int Dp, int Vp, Mask mask, Score score,
                     const float* sinks, const float* gate, int splits, int max_ctx,
                     hipStream_t s);
int omnia_gqa_prefill(void* out, const void* q, const void* kc, const void* vc,
                      const int* block_tables, int bt_stride, const int* q_start,
                      const int* seq_lens, const int* tile_seq, const int* tile_q0, int n_tiles,
                      int page, int H, int G, int Dp, int Vp, Mask mask, Score score,
                      const float* sinks, const float* gate, int bounded, hipStream_t s);
int omnia_joined_residual(void* h1, void* h2, int f32, float* x, int fresh, int rows, int d,
                          const void* am, int at, int aS, int64_t arow, int64_t apart,
                          const void* bm, int bS, int64_t brow, int64_t bpart, const void* cm,
                          int ct, int cS, int64_t crow, int64_t cpart, const int* ids,
                          const void* table, int vocab, float scale, const float* step,
                          const int64_t* src, const int* tok_slots, const float* w1, float g1,
                          const float* w2, float g2, float inv_n, float eps, hipStream_t s);
int omnia_latent_prep(void* cq, void* cache, const void* x, int f32, int64_t ldx, const float* wq,
                      const float* wc, const int* positions, const int64_t* slots,
                      const float* cos_sin, int T, int Q, int Qp, int C, int Cp, int R, int Lp,
                      float eps, hipStream_t s);
int omnia_latent_rotate(void* q, int f32, int64_t ldq, int hstride, int off, const int* positions,
                        const float* cos_sin, int T, int H, int R, hipStream_t s);
int omnia_latent_heads(void* out, int f32, int64_t ldo, int ho, const void* x, int64_t ldx, int hx,
                       const void* W, int T, int H, int N, int K, const void* gate, int64_t ldg,
                       const int* positions, const float* cos_sin, int R, int Rp, int rotx,
                       int tail, hipStream_t s);
int omnia_latent_attend(void* out, int f32, const void* q, const void* cache,
                        const int* block_tables, int bt_stride, const int* q_start, int nseq,
                        const int* positions, int T, int page, int H, int Cp, int Lp, int window,
                        float scale, hipStream_t s);
int omnia_latent_decode_covers(int Cp, int Lp);
int omnia_latent_decode(void* out, float* part_o, float* part_ml, const void* q, const void* cache,
                        const int* block_tables, int bt_stride, const int* positions, int T,
                        int page, int H, int Cp, int Lp, int window, float scale, int splits,
                        hipStream_t s);
int omnia_latent_gather(void* c, void* kr, const void* cache, const int* block_tables,
                        int bt_stride, const int* kv_start, const int* kv_first,
                        const int* seq_lens, int nseq, int page, int Tk, int Cp, int Rp, int Lp,
                        hipStream_t s);
int omnia_latent_prefill(void* out, const void* q, const void* kx, const void* kr, const void* vt,
                         const int* q_start, const int* seq_lens, const int* kv_start,
                         const int* kv_first, const int* tile_seq, const int* tile_q0, int n_tiles,
                         int H, int QW, int Da, int Rp, int VW, int Tk, int window, float scale,
                         const void* gate, int64_t ldg, hipStream_t s);
int omnia_stage_copy(void* dst, const void* src, int64_t head_bytes, int64_t bt_off,
                     int64_t row_stride, int rows, int64_t row_bytes, hipStream_t s);
int64_t omnia_host_device_ptr(void* host);
}

namespace {

hipStream_t cur_stream() { return c10::hip::getCurrentHIPStream().stream(); }

#define CHECK_GPU(t) TORCH_CHECK((t).is_cuda(), #t " must be a GPU tensor")
#define CHECK_BF16(t) TORCH_CHECK((t).scalar_type() == at::kBFloat16, #t " must be bf16")
#define CHECK_I32(t) TORCH_CHECK((t).scalar_type() == at::kInt, #t " must be int32")
#define CHECK_RC(rc, what) TORCH_CHECK((rc) == 0, what " launch failed rc=", (rc))

template <typename T>
T* opt_ptr(const c10::optional<at::Tensor>& t) {
  return t.has_value() && t->defined() ? reinterpret_cast<T*>(t->data_ptr()) : nullptr;
}

void rmsnorm(at::Tensor out, at::Tensor x, at::Tensor w, double eps) {
  CHECK_GPU(x); CHECK_BF16(x); CHECK_BF16(out); CHECK_BF16(w);
  TORCH_CHECK(x.dim() == 2 && out.dim() == 2, "rmsnorm expects 2-D");
  TORCH_CHECK(x.stride(1) == 1 && out.stride(1) == 1 && w.is_contiguous(), "inner dim contiguous");
  const int d = x.size(1);
  TORCH_CHECK(w.numel() == d && out.size(1) == d && out.size(0) == x.size(0), "shape mismatch");
  CHECK_RC(omnia_rmsnorm(out.data_ptr(), x.data_ptr(), nullptr, w.data_ptr(), x.size(0), d,
                         x.stride(0), out.stride(0), (float)eps, cur_stream()), "rmsnorm");
}

// residual += x ; x = rmsnorm(residual) * w      (both in place)
void fused_add_rmsnorm(at::Tensor x, at::Tensor residual, at::Tensor w, double eps) {
  CHECK_GPU(x); CHECK_BF16(x); CHECK_BF16(residual); CHECK_BF16(w);
  TORCH_CHECK(x.dim() == 2 && x.is_contiguous() && residual.is_contiguous(), "contiguous 2-D");
  TORCH_CHECK(residual.sizes() == x.sizes() && w.numel() == x.size(1), "shape mismatch");
  CHECK_RC(omnia_rmsnorm(x.data_ptr(), x.data_ptr(), residual.data_ptr(), w.data_ptr(),
                         x.size(0), x.size(1), x.stride(0), x.stride(0), (float)eps,
                         cur_stream()), "fused_add_rmsnorm");
}

void rope_kv(at::Tensor q, at::Tensor k, at::Tensor v, at::Tensor positions, at::Tensor cos_sin,
             c10::optional<at::Tensor> k_cache, c10::optional<at::Tensor> v_cache,
             c10::optional<at::Tensor> slots, int64_t hq, int64_t hkv, int64_t block_size) {
  CHECK_GPU(q); CHECK_BF16(q); CHECK_BF16(k); CHECK_BF16(v); CHECK_I32(positions);
  TORCH_CHECK(cos_sin.scalar_type() == at::kFloat && cos_sin.is_contiguous(), "cos_sin f32");
  TORCH_CHECK(q.dim() == 2 && k.dim() == 2 && v.dim() == 2, "q/k/v as [T, H*D] views");
  TORCH_CHECK(q.stride(1) == 1 && k.stride(1) == 1 && v.stride(1) == 1, "inner contiguous");
  TORCH_CHECK(k.stride(0) == v.stride(0), "k/v share row stride");
  const int T = q.size(0);
  const int D = q.size(1) / hq;
  TORCH_CHECK(D == 128 && k.size(1) == hkv * D && v.size(1) == hkv * D, "head_dim 128");
  TORCH_CHECK(positions.numel() == T && k.size(0) == T, "T mismatch");
  TORCH_CHECK(cos_sin.size(1) == D, "cos_sin width");
  const int64_t* sl = nullptr;
  void *kc = nullptr, *vc = nullptr;
  if (slots.has_value() && slots->defined()) {
    TORCH_CHECK(slots->scalar_type() == at::kLong && slots->numel() == T, "slots int64[T]");
    TORCH_CHECK(k_cache.has_value() && v_cache.has_value(), "caches required with slots");
    CHECK_BF16(*k_cache);
    TORCH_CHECK(k_cache->dim() == 4 && k_cache->size(1) == hkv && k_cache->size(2) == block_size &&
                k_cache->size(3) == D && k_cache->is_contiguous() && v_cache->is_contiguous(),
                "cache layout [NB, Hkv, BS, D]");
    sl = slots->data_ptr<int64_t>();
    kc = k_cache->data_ptr();
    vc = v_cache->data_ptr();
  }
  CHECK_RC(omnia_rope_kv(q.data_ptr(), k.data_ptr(), v.data_ptr(), positions.data_ptr<int>(),
                         cos_sin.data_ptr<float>(), kc, vc, sl, T, hq, hkv, D, q.stride(0),
                         k.stride(0), block_size, cur_stream()), "rope_kv");
}

void silu_mul(at::Tensor out, at::Tensor x) {
  CHECK_GPU(x); CHECK_BF16(x); CHECK_BF16(out);
  TORCH_CHECK(x.is_contiguous() && out.is_contiguous(), "contiguous");
  const int64_t inter = out.size(-1);
  TORCH_CHECK(x.size(-1) == 2 * inter && x.numel() == 2 * out.numel(), "shape mismatch");
  CHECK_RC(omnia_silu_mul(out.data_ptr(), x.data_ptr(), out.numel() / inter, inter,
                          cur_stream()), "silu_mul");
}

// src / tok_slots (optional, decode): row t's token is tok_slots[src[t]] when
// src[t] >= 0 (sampled on the device by an earlier step), else ids[t]
void embedding(at::Tensor out, at::Tensor ids, at::Tensor w, int64_t vocab_start,
               c10::optional<at::Tensor> src, c10::optional<at::Tensor> tok_slots) {
  CHECK_GPU(ids); CHECK_I32(ids); CHECK_BF16(w); CHECK_BF16(out);
  TORCH_CHECK(w.is_contiguous() && out.is_contiguous(), "contiguous");
  TORCH_CHECK(out.size(0) == ids.numel() && out.size(1) == w.size(1), "shape mismatch");
  const bool has_src = src.has_value() && src->defined();
  if (has_src) {
    CHECK_I32(*tok_slots);
    TORCH_CHECK(src->scalar_type() == at::kLong && src->numel() == ids.numel() &&
                src->is_contiguous() && tok_slots->is_contiguous(),
                "src [T] int64, tok_slots int32");
  }
  CHECK_RC(omnia_embedding(out.data_ptr(), ids.data_ptr<int>(), w.data_ptr(), ids.numel(),
                           w.size(1), vocab_start, vocab_start + w.size(0),
                           has_src ? src->data_ptr<int64_t>() : nullptr,
                           has_src ? tok_slots->data_ptr<int>() : nullptr, cur_stream()),
           "embedding");
}

void decode_attention(at::Tensor out, at::Tensor q, at::Tensor k_cache, at::Tensor v_cache,
                      at::Tensor block_tables, at::Tensor seq_lens, at::Tensor part_o,
                      at::Tensor part_ml, int64_t part_size, double scale, int64_t splits,
                      int64_t split_min) {
  CHECK_GPU(q); CHECK_BF16(q); CHECK_BF16(out); CHECK_BF16(k_cache); CHECK_BF16(v_cache);
  CHECK_I32(block_tables); CHECK_I32(seq_lens);
  TORCH_CHECK(k_cache.dim() == 4 && k_cache.is_contiguous() && v_cache.is_contiguous(),
              "cache [NB, Hkv, BS, D]");
  const int hkv = k_cache.size(1), bs = k_cache.size(2), D = k_cache.size(3);
  TORCH_CHECK(q.dim() == 3 && q.stride(2) == 1 && q.stride(1) == D, "q [B, Hq, D]");
  const int B = q.size(0), hq = q.size(1);
  TORCH_CHECK(out.is_contiguous() && out.size(0) == B && out.size(1) == hq, "out [B, Hq, D]");
  TORCH_CHECK(block_tables.dim() == 2 && block_tables.size(0) >= B && block_tables.stride(1) == 1,
              "block_tables [B, max_blocks]");
  TORCH_CHECK(seq_lens.numel() >= B, "seq_lens");
  const int max_ctx = block_tables.size(1) * bs;
  // splits > 0: length-balanced split into up to `splits` partitions (>= split_min keys)
  TORCH_CHECK(splits >= 0 && (splits == 0 || split_min > 0), "splits / split_min");
  const int max_parts = std::max<int>((max_ctx + part_size - 1) / part_size, (int)splits);
  TORCH_CHECK(part_o.scalar_type() == at::kFloat && part_ml.scalar_type() == at::kFloat,
              "workspace f32");
  TORCH_CHECK(part_o.numel() >= (int64_t)B * hq * max_parts * D &&
              part_ml.numel() >= (int64_t)B * hq * max_parts * 2, "workspace too small");
  CHECK_RC(omnia_decode_attention(out.data_ptr(), part_o.data_ptr<float>(),
                                  part_ml.data_ptr<float>(), q.data_ptr(), k_cache.data_ptr(),
                                  v_cache.data_ptr(), block_tables.data_ptr<int>(),
                                  block_tables.stride(0), seq_lens.data_ptr<int>(), B, hq, hkv, D,
                                  bs, q.stride(0), part_size, max_parts, (float)scale,
                                  (int)splits, (int)split_min, cur_stream()),
           "decode_attention");
}

void prefill_attention(at::Tensor out, at::Tensor q, at::Tensor k_cache, at::Tensor v_cache,
                       at::Tensor block_tables, at::Tensor q_start_loc, at::Tensor seq_lens,
                       at::Tensor tile_seq, at::Tensor tile_q0, double scale, int64_t hp,
                       int64_t q_tile, c10::optional<at::Tensor> lse,
                       c10::optional<at::Tensor> kv_lens) {
  CHECK_GPU(q); CHECK_BF16(q); CHECK_BF16(out); CHECK_BF16(k_cache);
  CHECK_I32(block_tables); CHECK_I32(q_start_loc); CHECK_I32(seq_lens); CHECK_I32(tile_seq);
  CHECK_I32(tile_q0);
  const int hkv = k_cache.size(1), bs = k_cache.size(2), D = k_cache.size(3);
  TORCH_CHECK(q.dim() == 3 && q.stride(2) == 1 && q.stride(1) == D, "q [T, Hq, D]");
  TORCH_CHECK(out.dim() == 3 && out.stride(2) == 1 && out.stride(1) == D, "out [T, Hq, D]");
  TORCH_CHECK(tile_seq.numel() == tile_q0.numel(), "tiles");
  TORCH_CHECK(block_tables.stride(1) == 1, "block_tables rows contiguous");
  float* lse_p = nullptr;
  if (lse.has_value()) {
    TORCH_CHECK(lse->scalar_type() == at::kFloat && lse->is_contiguous() && lse->dim() == 2 &&
                    lse->size(0) >= q.size(0) && lse->size(1) == q.size(1),
                "lse fp32 [T, Hq] contiguous");
    lse_p = lse->data_ptr<float>();
  }
  const int* kvl_p = nullptr;
  if (kv_lens.has_value()) {
    CHECK_I32((*kv_lens));
    TORCH_CHECK(kv_lens->numel() == seq_lens.numel(), "kv_lens [B]");
    kvl_p = kv_lens->data_ptr<int>();
  }
  CHECK_RC(omnia_prefill_attention(out.data_ptr(), q.data_ptr(), k_cache.data_ptr(),
                                   v_cache.data_ptr(), block_tables.data_ptr<int>(),
                                   block_tables.stride(0), q_start_loc.data_ptr<int>(),
                                   seq_lens.data_ptr<int>(), tile_seq.data_ptr<int>(),
                                   tile_q0.data_ptr<int>(), tile_seq.numel(), q.size(1), hkv, D,
                                   bs, q.stride(0), out.stride(0), (float)scale, (int)hp,
                                   (int)q_tile, lse_p, kvl_p, cur_stream()),
           "prefill_attention");
}

void sample(at::Tensor out_tok, c10::optional<at::Tensor> out_logprob, at::Tensor logits,
            at::Tensor temperature, c10::optional<at::Tensor> top_k,
            c10::optional<at::Tensor> top_p, c10::optional<at::Tensor> seeds,
            c10::optional<at::Tensor> steps, c10::optional<at::Tensor> counts,
            c10::optional<at::Tensor> freq_pen, c10::optional<at::Tensor> pres_pen,
            c10::optional<at::Tensor> rep_pen, c10::optional<at::Tensor> tok_slots,
            c10::optional<at::Tensor> dst) {
  CHECK_GPU(logits); CHECK_I32(out_tok);
  TORCH_CHECK(logits.dim() == 2 && logits.stride(1) == 1, "logits [B, V]");
  TORCH_CHECK(logits.scalar_type() == at::kBFloat16 || logits.scalar_type() == at::kFloat,
              "logits bf16/f32");
  const int rows = logits.size(0), vocab = logits.size(1);
  TORCH_CHECK(out_tok.numel() >= rows && temperature.numel() >= rows, "per-row params");
  if (counts.has_value() && counts->defined())
    TORCH_CHECK(counts->scalar_type() == at::kInt && counts->size(0) >= rows &&
                counts->size(1) == vocab && counts->is_contiguous(), "counts int32 [B, V]");
  if (tok_slots.has_value() && tok_slots->defined()) {
    CHECK_I32(*tok_slots);
    TORCH_CHECK(dst.has_value() && dst->defined() && dst->scalar_type() == at::kLong &&
                dst->numel() >= rows && dst->is_contiguous() && tok_slots->is_contiguous(),
                "tok_slots int32 + dst int64 [B]");
  }
  CHECK_RC(omnia_sample(out_tok.data_ptr<int>(), opt_ptr<float>(out_logprob), logits.data_ptr(),
                        logits.scalar_type() == at::kBFloat16, rows, logits.stride(0), vocab,
                        temperature.data_ptr<float>(), opt_ptr<int>(top_k), opt_ptr<float>(top_p),
                        opt_ptr<uint64_t>(seeds), opt_ptr<int64_t>(steps), opt_ptr<int>(counts),
                        opt_ptr<float>(freq_pen), opt_ptr<float>(pres_pen),
                        opt_ptr<float>(rep_pen), opt_ptr<int>(tok_slots), opt_ptr<int64_t>(dst),
                        cur_stream()), "sample");
}

// K13: grammar mask -> -inf logits (mask int32 [rows, ceil(V/32)], bit v = allowed)
// TP sampling: per-row Gumbel-max winner of this rank's vocab slice, written
// into columns col, col+1 of the fp32 candidate pack [B, ld]
void tp_gumbel(at::Tensor pack, int64_t col, at::Tensor logits, int64_t vocab_start,
               at::Tensor temperature, c10::optional<at::Tensor> top_k,
               c10::optional<at::Tensor> top_p, at::Tensor seeds,
               c10::optional<at::Tensor> steps) {
  CHECK_GPU(pack); CHECK_GPU(logits); CHECK_BF16(logits);
  TORCH_CHECK(logits.dim() == 2 && logits.stride(1) == 1, "logits [B, V] inner-contiguous");
  const int rows = logits.size(0), vocab = logits.size(1);
  TORCH_CHECK(pack.scalar_type() == at::kFloat && pack.dim() == 2 && pack.stride(1) == 1 &&
              pack.size(0) == rows && col >= 0 && col + 2 <= pack.size(1), "pack fp32 [B, ld]");
  TORCH_CHECK(temperature.scalar_type() == at::kFloat && temperature.numel() >= rows &&
              temperature.is_cuda(), "temperature fp32 [B]");
  TORCH_CHECK(seeds.scalar_type() == at::kLong && seeds.numel() >= rows && seeds.is_cuda(),
              "seeds int64 [B]");
  if (top_k.has_value() && top_k->defined())
    TORCH_CHECK(top_k->scalar_type() == at::kInt && top_k->numel() >= rows, "top_k int32 [B]");
  if (top_p.has_value() && top_p->defined())
    TORCH_CHECK(top_p->scalar_type() == at::kFloat && top_p->numel() >= rows, "top_p fp32 [B]");
  if (steps.has_value() && steps->defined())
    TORCH_CHECK(steps->scalar_type() == at::kLong && steps->numel() >= rows, "steps int64 [B]");
  CHECK_RC(omnia_tp_gumbel(pack.data_ptr<float>(), pack.stride(0), (int)col, logits.data_ptr(),
                           rows, logits.stride(0), vocab, (int)vocab_start,
                           temperature.data_ptr<float>(), opt_ptr<int>(top_k),
                           opt_ptr<float>(top_p), seeds.data_ptr<int64_t>(),
                           opt_ptr<int64_t>(steps), cur_stream()), "tp_gumbel");
}

// TP sampler, per rank: candidate pack of this rank's vocab slice (sampling.hip)
void tp_pack(at::Tensor pack, int64_t K, at::Tensor logits, int64_t vocab_start,
             at::Tensor temperature, c10::optional<at::Tensor> top_k,
             c10::optional<at::Tensor> top_p, at::Tensor seeds, c10::optional<at::Tensor> steps) {
  CHECK_GPU(pack); CHECK_GPU(logits); CHECK_BF16(logits);
  TORCH_CHECK(logits.dim() == 2 && logits.stride(1) == 1, "logits [B, V] inner-contiguous");
  const int rows = logits.size(0), vocab = logits.size(1);
  TORCH_CHECK(pack.scalar_type() == at::kFloat && pack.dim() == 2 && pack.is_contiguous() &&
              pack.size(0) == rows && pack.size(1) >= 2 * K + 4 && K >= 1 && K <= vocab,
              "pack fp32 [B, >= 2K+4] contiguous, 1 <= K <= V");
  TORCH_CHECK(temperature.is_cuda() && temperature.scalar_type() == at::kFloat &&
              temperature.numel() >= rows, "temperature fp32 [B]");
  TORCH_CHECK(seeds.is_cuda() && seeds.scalar_type() == at::kLong && seeds.numel() >= rows,
              "seeds int64 [B]");
  if (top_k.has_value() && top_k->defined())
    TORCH_CHECK(top_k->is_cuda() && top_k->scalar_type() == at::kInt && top_k->numel() >= rows,
                "top_k int32 [B]");
  if (top_p.has_value() && top_p->defined())
    TORCH_CHECK(top_p->is_cuda() && top_p->scalar_type() == at::kFloat && top_p->numel() >= rows,
                "top_p fp32 [B]");
  if (steps.has_value() && steps->defined())
    TORCH_CHECK(steps->is_cuda() && steps->scalar_type() == at::kLong && steps->numel() >= rows,
                "steps int64 [B]");
  CHECK_RC(omnia_tp_pack(pack.data_ptr<float>(), pack.stride(0), (int)K, logits.data_ptr(), rows,
                         logits.stride(0), vocab, (int)vocab_start, temperature.data_ptr<float>(),
                         opt_ptr<int>(top_k), opt_ptr<float>(top_p), seeds.data_ptr<int64_t>(),
                         opt_ptr<int64_t>(steps), cur_stream()), "tp_pack");
}

// TP sampler, every rank: token of each row from the all-gathered packs [W, B, ld];
// with tok_slots / dst, also tok_slots[dst[r]] = token (device token hand-off)
void tp_merge(at::Tensor out, c10::optional<at::Tensor> tok_slots, c10::optional<at::Tensor> dst,
              at::Tensor allp, int64_t K, at::Tensor temperature, c10::optional<at::Tensor> top_k,
              c10::optional<at::Tensor> top_p, at::Tensor seeds, c10::optional<at::Tensor> steps) {
  CHECK_GPU(out); CHECK_GPU(allp); CHECK_I32(out);
  TORCH_CHECK(allp.scalar_type() == at::kFloat && allp.dim() == 3 && allp.is_contiguous(),
              "allp fp32 [W, B, ld] contiguous");
  const int W = allp.size(0), B = allp.size(1);
  const int64_t ld = allp.size(2);
  TORCH_CHECK(out.numel() >= B && out.is_contiguous(), "out int32 [B]");
  TORCH_CHECK(K >= 1 && ld >= 2 * K + 4 && W * K <= 512, "W * K <= 512, ld >= 2K+4");
  TORCH_CHECK(temperature.is_cuda() && temperature.scalar_type() == at::kFloat &&
              temperature.numel() >= B, "temperature fp32 [B]");
  TORCH_CHECK(seeds.is_cuda() && seeds.scalar_type() == at::kLong && seeds.numel() >= B,
              "seeds int64 [B]");
  if (top_k.has_value() && top_k->defined())
    TORCH_CHECK(top_k->scalar_type() == at::kInt && top_k->numel() >= B, "top_k int32 [B]");
  if (top_p.has_value() && top_p->defined())
    TORCH_CHECK(top_p->scalar_type() == at::kFloat && top_p->numel() >= B, "top_p fp32 [B]");
  if (steps.has_value() && steps->defined())
    TORCH_CHECK(steps->scalar_type() == at::kLong && steps->numel() >= B, "steps int64 [B]");
  const bool slots = tok_slots.has_value() && tok_slots->defined();
  if (slots) {
    TORCH_CHECK(dst.has_value() && dst->defined() && dst->scalar_type() == at::kLong &&
                dst->numel() >= B && dst->is_cuda(), "dst int64 [B] with tok_slots");
    CHECK_I32(*tok_slots);
    TORCH_CHECK(tok_slots->is_cuda() && tok_slots->is_contiguous(), "tok_slots int32 on device");
  }
  CHECK_RC(omnia_tp_merge(out.data_ptr<int>(), slots ? tok_slots->data_ptr<int>() : nullptr,
                          slots ? dst->data_ptr<int64_t>() : nullptr, allp.data_ptr<float>(), W, B,
                          ld, (int)K, temperature.data_ptr<float>(), opt_ptr<int>(top_k),
                          opt_ptr<float>(top_p), seeds.data_ptr<int64_t>(),
                          opt_ptr<int64_t>(steps), cur_stream()), "tp_merge");
}

void apply_token_mask(at::Tensor logits, at::Tensor mask) {
  CHECK_GPU(logits); CHECK_GPU(mask); CHECK_I32(mask);
  TORCH_CHECK(logits.dim() == 2 && logits.stride(1) == 1, "logits [B, V]");
  TORCH_CHECK(logits.scalar_type() == at::kBFloat16 || logits.scalar_type() == at::kFloat,
              "logits bf16/f32");
  const int rows = logits.size(0), vocab = logits.size(1), words = (vocab + 31) / 32;
  TORCH_CHECK(mask.dim() == 2 && mask.size(0) == rows && mask.size(1) == words &&
              mask.is_contiguous(), "mask int32 [B, ceil(V/32)] contiguous");
  CHECK_RC(omnia_apply_token_mask(logits.data_ptr(), logits.scalar_type() == at::kBFloat16, rows,
                                  logits.stride(0), vocab,
                                  reinterpret_cast<const uint32_t*>(mask.data_ptr<int>()), words,
                                  cur_stream()), "apply_token_mask");
}

// K17: out[b] = normalize(mean(hidden[cu[b]:cu[b+1]]))   fp32
void mean_pool_l2(at::Tensor out, at::Tensor hidden, at::Tensor cu) {
  CHECK_GPU(hidden); CHECK_BF16(hidden); CHECK_I32(cu);
  TORCH_CHECK(out.scalar_type() == at::kFloat && out.is_contiguous(), "out fp32 contiguous");
  TORCH_CHECK(hidden.dim() == 2 && hidden.stride(1) == 1, "hidden [T, D] inner-contiguous");
  TORCH_CHECK(cu.dim() == 1 && cu.is_contiguous() && cu.is_cuda(), "cu [B+1] on device");
  const int B = cu.size(0) - 1, D = hidden.size(1);
  TORCH_CHECK(out.dim() == 2 && out.size(0) == B && out.size(1) == D, "out [B, D]");
  TORCH_CHECK(D % 8 == 0 && D <= 8192, "D must be a multiple of 8, <= 8192");
  CHECK_RC(omnia_mean_pool_l2(out.data_ptr<float>(), hidden.data_ptr(), hidden.stride(0),
                              cu.data_ptr<int>(), B, D, cur_stream()), "mean_pool_l2");
}

// K18: scores[q, n] = Q[q] . M[n]  (fp32 out, -inf where valid[n] == 0)
void cosine_scores(at::Tensor scores, at::Tensor q, at::Tensor m,
                   c10::optional<at::Tensor> valid) {
  CHECK_GPU(m); CHECK_BF16(m);
  TORCH_CHECK(q.scalar_type() == at::kFloat && q.is_contiguous() && q.is_cuda(), "q fp32");
  TORCH_CHECK(m.dim() == 2 && m.is_contiguous(), "m [N, D] contiguous");
  TORCH_CHECK(q.dim() == 2 && q.size(1) == m.size(1), "q [NQ, D]");
  const int nq = q.size(0), D = m.size(1);
  const int64_t N = m.size(0);
  TORCH_CHECK(nq == 1 || nq == 2 || nq == 4 || nq == 8, "NQ must be 1/2/4/8 (pad on host)");
  TORCH_CHECK((int64_t)nq * D * 4 <= 64 * 1024, "NQ*D too large for the LDS stage");
  TORCH_CHECK(D % 8 == 0, "D % 8");
  TORCH_CHECK(scores.scalar_type() == at::kFloat && scores.is_contiguous() &&
              scores.size(0) == nq && scores.size(1) == N, "scores [NQ, N] fp32");
  const uint8_t* vp = nullptr;
  if (valid.has_value() && valid->defined()) {
    TORCH_CHECK(valid->scalar_type() == at::kByte && valid->numel() >= N && valid->is_cuda(),
                "valid uint8 [>= N]");
    vp = valid->data_ptr<uint8_t>();
  }
  CHECK_RC(omnia_cosine_scores(scores.data_ptr<float>(), q.data_ptr<float>(), nq, m.data_ptr(),
                               N, D, vp, cur_stream()), "cosine_scores");
}

void topk(at::Tensor out_idx, at::Tensor out_val, at::Tensor scores, int64_t k) {
  CHECK_GPU(scores);
  TORCH_CHECK(scores.scalar_type() == at::kFloat && scores.is_contiguous() && scores.dim() == 2,
              "scores [NQ, N] fp32 contiguous");
  const int nq = scores.size(0);
  const int64_t N = scores.size(1);
  TORCH_CHECK(k >= 1 && k <= 1024 && k <= N, "1 <= k <= min(1024, N)");
  CHECK_I32(out_idx);
  TORCH_CHECK(out_val.scalar_type() == at::kFloat, "out_val fp32");
  TORCH_CHECK(out_idx.numel() == nq * k && out_val.numel() == nq * k && out_idx.is_contiguous() &&
              out_val.is_contiguous(), "outputs [NQ, k]");
  CHECK_RC(omnia_topk(out_idx.data_ptr<int>(), out_val.data_ptr<float>(),
                      scores.data_ptr<float>(), nq, N, (int)k, cur_stream()), "topk");
}

// ---------------------------------------------------------------- MoE (K14)
void moe_topk(at::Tensor ids, at::Tensor wts, at::Tensor logits, int64_t k, bool renorm) {
  CHECK_GPU(logits); CHECK_I32(ids);
  TORCH_CHECK(logits.dim() == 2 && logits.is_contiguous(), "logits [T, E] contiguous");
  const bool bf = logits.scalar_type() == at::kBFloat16;
  TORCH_CHECK(bf || logits.scalar_type() == at::kFloat, "logits bf16/fp32");
  const int T = logits.size(0), E = logits.size(1);
  TORCH_CHECK(E <= 64 && k >= 1 && k <= E, "E <= 64, 1 <= k <= E");
  TORCH_CHECK(ids.numel() == (int64_t)T * k && wts.numel() == (int64_t)T * k &&
              wts.scalar_type() == at::kFloat && ids.is_contiguous() && wts.is_contiguous(),
              "ids/wts [T, k]");
  CHECK_RC(omnia_moe_topk(ids.data_ptr<int>(), wts.data_ptr<float>(), logits.data_ptr(), bf, T,
                          E, k, renorm, cur_stream()), "moe_topk");
}

// router GEMM + top-k in one kernel: x [T, d] bf16, router [E, d] bf16 -> ids / wts [T, k]
void moe_router_topk(at::Tensor ids, at::Tensor wts, at::Tensor x, at::Tensor router, int64_t k,
                     bool renorm) {
  CHECK_GPU(x); CHECK_BF16(x); CHECK_BF16(router); CHECK_I32(ids);
  TORCH_CHECK(x.dim() == 2 && x.is_contiguous() && router.dim() == 2 && router.is_contiguous() &&
              router.size(1) == x.size(1) && x.size(1) % 8 == 0, "x [T, d], router [E, d]");
  const int T = x.size(0), E = router.size(0);
  TORCH_CHECK(E <= 64 && k >= 1 && k <= E, "E <= 64, 1 <= k <= E");
  TORCH_CHECK(ids.numel() == (int64_t)T * k && wts.numel() == (int64_t)T * k &&
              wts.scalar_type() == at::kFloat && ids.is_contiguous() && wts.is_contiguous(),
              "ids/wts [T, k]");
  CHECK_RC(omnia_moe_router_topk(ids.data_ptr<int>(), wts.data_ptr<float>(), x.data_ptr(),
                                 router.data_ptr(), T, x.size(1), E, k, renorm, cur_stream()),
           "moe_router_topk");
}

int64_t moe_max_blocks(int64_t n_assign, int64_t n_experts, int64_t bm) {
  return omnia_moe_max_blocks(n_assign, n_experts, bm);
}

// segments aligned to bm = sorted.numel() / blk_expert.numel() rows (64: moe_gemm,
// 256: the pgemm_moe prefill tile)
void moe_align(at::Tensor sorted, at::Tensor blk_expert, at::Tensor n_blocks, at::Tensor ids,
               int64_t E, int64_t e_lo, int64_t e_hi) {
  CHECK_GPU(ids); CHECK_I32(ids); CHECK_I32(sorted); CHECK_I32(blk_expert); CHECK_I32(n_blocks);
  const int n = ids.numel();
  const int mb = blk_expert.numel();
  TORCH_CHECK(mb > 0 && (sorted.numel() == (int64_t)mb * 64 || sorted.numel() == (int64_t)mb * 256),
              "sorted must hold max_blocks*64 (or *256) rows");
  const int bm = (int)(sorted.numel() / mb);
  TORCH_CHECK(mb >= omnia_moe_max_blocks(n, e_hi - e_lo, bm), "blk_expert too small");
  TORCH_CHECK(E <= 256 && 0 <= e_lo && e_lo < e_hi && e_hi <= E, "expert range");
  CHECK_RC(omnia_moe_align(sorted.data_ptr<int>(), blk_expert.data_ptr<int>(),
                           n_blocks.data_ptr<int>(), ids.data_ptr<int>(), n, E, e_lo, e_hi, mb,
                           bm, cur_stream()), "moe_align");
}

// the 256x256-tile grouped MoE GEMMs (pgemm.hip EPI 5 / 6) over 256-row segments
void pgemm_moe(int64_t mode, at::Tensor out, at::Tensor A, at::Tensor W, at::Tensor sorted,
               at::Tensor blk_expert, at::Tensor n_blocks, c10::optional<at::Tensor> route_w,
               int64_t topk, int64_t n_assign, int64_t e_lo, double alpha, double limit) {
  CHECK_GPU(A); CHECK_BF16(A); CHECK_BF16(W); CHECK_BF16(out);
  CHECK_I32(sorted); CHECK_I32(blk_expert); CHECK_I32(n_blocks);
  if (route_w.has_value())
    TORCH_CHECK(route_w->is_cuda() && route_w->is_contiguous() && route_w->numel() == n_assign &&
                route_w->scalar_type() == at::kFloat, "route weights fp32 [T*k]");
  TORCH_CHECK(A.is_contiguous() && W.is_contiguous() && out.is_contiguous(), "contiguous");
  TORCH_CHECK(W.dim() == 3, "W [E_local, rows, K]");
  const int K = W.size(2);
  const int mb = blk_expert.numel();
  TORCH_CHECK(sorted.numel() == (int64_t)mb * 256, "sorted must hold max_blocks*256 rows");
  TORCH_CHECK(A.size(-1) == K && K % 128 == 0, "K mismatch / K % 128");
  int N;
  if (mode != 1) {
    N = mode == 3 ? W.size(1) : W.size(1) / 2;
    TORCH_CHECK(N % 128 == 0 && out.size(0) == (int64_t)mb * 256 && out.size(1) == N,
                "act [max_blocks*256, I]");
    TORCH_CHECK(A.size(0) * topk == n_assign, "x rows * topk == n_assign");
  } else {
    N = W.size(1);
    TORCH_CHECK(N % 256 == 0 && out.size(0) == n_assign && out.size(1) == N, "Y [T*k, d]");
    TORCH_CHECK(A.size(0) == (int64_t)mb * 256, "act rows");
  }
  CHECK_RC(omnia_pgemm_moe((int)mode, out.data_ptr(), A.data_ptr(), W.data_ptr(),
                           sorted.data_ptr<int>(), blk_expert.data_ptr<int>(),
                           n_blocks.data_ptr<int>(), opt_ptr<float>(route_w), K, N, topk,
                           n_assign, e_lo, mb, (float)alpha, (float)limit, cur_stream()),
           "pgemm_moe");
}

// router: fp32 logits, sigmoid / softmax scores; x [T, d] and router [E, d] bf16 or fp32
void moe_route(at::Tensor ids, at::Tensor wts, at::Tensor x, at::Tensor router, int64_t k,
               bool sigmoid, bool renorm, c10::optional<at::Tensor> corr, int64_t groups,
               int64_t keep, c10::optional<at::Tensor> bias) {
  CHECK_GPU(x); CHECK_I32(ids);
  const bool f32 = x.scalar_type() == at::kFloat;
  TORCH_CHECK((f32 || x.scalar_type() == at::kBFloat16) && router.scalar_type() == x.scalar_type(),
              "x and router: bf16 or fp32");
  TORCH_CHECK(x.dim() == 2 && x.is_contiguous() && router.is_cuda() && router.dim() == 2 &&
              router.is_contiguous() && router.size(1) == x.size(1),
              "x [T, d], router [E, d]");
  const int T = x.size(0), E = router.size(0);
  TORCH_CHECK(ids.numel() == (int64_t)T * k && wts.numel() == (int64_t)T * k && wts.is_cuda() &&
              wts.scalar_type() == at::kFloat && ids.is_contiguous() && wts.is_contiguous(),
              "ids/wts [T, k]");
  if (corr.has_value())
    TORCH_CHECK(corr->is_cuda() && corr->scalar_type() == at::kFloat && corr->is_contiguous() &&
                corr->numel() == E, "correction fp32 [E]");
  if (bias.has_value())
    TORCH_CHECK(bias->is_cuda() && bias->scalar_type() == at::kFloat && bias->is_contiguous() &&
                bias->numel() == E, "bias fp32 [E]");
  CHECK_RC(omnia_moe_route(ids.data_ptr<int>(), wts.data_ptr<float>(), x.data_ptr(),
                           router.data_ptr(), f32, T, x.size(1), E, k, sigmoid, renorm,
                           opt_ptr<float>(corr), groups, keep, opt_ptr<float>(bias),
                           cur_stream()), "moe_route");
}

// modes in moe.hip; A, W and out all bf16 or all fp32
void moe_gemm(int64_t mode, at::Tensor out, at::Tensor A, at::Tensor W, at::Tensor sorted,
              at::Tensor blk_expert, at::Tensor n_blocks, c10::optional<at::Tensor> route_w,
              int64_t topk, int64_t n_assign, int64_t e_lo, double alpha, double limit) {
  CHECK_GPU(A); CHECK_GPU(W); CHECK_GPU(out);
  const bool f32 = A.scalar_type() == at::kFloat;
  TORCH_CHECK((f32 || A.scalar_type() == at::kBFloat16) && W.scalar_type() == A.scalar_type() &&
              out.scalar_type() == A.scalar_type(), "A, W, out: bf16 or fp32");
  CHECK_I32(sorted); CHECK_I32(blk_expert); CHECK_I32(n_blocks);
  TORCH_CHECK(A.is_contiguous() && W.is_contiguous() && out.is_contiguous(), "contiguous");
  TORCH_CHECK(W.dim() == 3, "W [E_local, rows, K]");
  const int K = W.size(2);
  const int mb = blk_expert.numel();
  TORCH_CHECK(sorted.numel() == (int64_t)mb * 64, "sorted must hold max_blocks*64 rows");
  TORCH_CHECK(A.size(-1) == K && K % 64 == 0, "K mismatch / K % 64");
  if (route_w.has_value())
    TORCH_CHECK(route_w->is_cuda() && route_w->is_contiguous() && route_w->numel() == n_assign &&
                route_w->scalar_type() == at::kFloat, "route weights fp32 [T*k]");
  int N;
  if (mode != 1) {
    N = mode == 3 ? W.size(1) : W.size(1) / 2;
    TORCH_CHECK(N % 32 == 0 && out.size(0) == (int64_t)mb * 64 && out.size(1) == N,
                "act [max_blocks*64, I]");
    TORCH_CHECK(A.size(0) * topk == n_assign, "x rows * topk == n_assign");
  } else {
    N = W.size(1);
    TORCH_CHECK(N % 64 == 0 && out.size(0) == n_assign && out.size(1) == N, "Y [T*k, d]");
    TORCH_CHECK(A.size(0) == (int64_t)mb * 64, "act rows");
  }
  CHECK_RC(omnia_moe_gemm((int)mode, out.data_ptr(), A.data_ptr(), W.data_ptr(), f32,
                          sorted.data_ptr<int>(), blk_expert.data_ptr<int>(),
                          n_blocks.data_ptr<int>(), opt_ptr<float>(route_w), K, N, topk,
                          n_assign, e_lo, mb, (float)alpha, (float)limit, cur_stream()),
           "moe_gemm");
}

void moe_combine(at::Tensor out, at::Tensor Y, at::Tensor ids, int64_t topk, int64_t e_lo,
                 int64_t e_hi) {
  CHECK_GPU(Y); CHECK_BF16(Y); CHECK_BF16(out); CHECK_I32(ids);
  const int T = out.size(0), d = out.size(1);
  TORCH_CHECK(Y.size(0) == (int64_t)T * topk && Y.size(1) == d && ids.numel() == T * topk,
              "Y [T*k, d]");
  CHECK_RC(omnia_moe_combine(out.data_ptr(), Y.data_ptr(), ids.data_ptr<int>(), T, d, topk,
                             e_lo, e_hi, cur_stream()), "moe_combine");
}

// decode projection GEMM: mode 0 out[M,N] = x W^T (W [N,K]); mode 1 out[M,I] =
// silu(x Wg^T) * (x Wu^T) with W = [Wg; Wu] ([2I, K]).  Shapes are validated
// here AND in omnia_dgemm before anything is launched.
void dgemm(int64_t mode, at::Tensor out, at::Tensor x, at::Tensor W, at::Tensor ws, at::Tensor cnt,
           int64_t splits, int64_t wm, int64_t wn) {
  CHECK_GPU(x); CHECK_BF16(x); CHECK_BF16(W); CHECK_BF16(out);
  TORCH_CHECK(ws.scalar_type() == at::kFloat && ws.is_cuda(), "ws fp32");
  CHECK_I32(cnt);
  TORCH_CHECK(x.dim() == 2 && W.dim() == 2 && out.dim() == 2, "2-D operands");
  TORCH_CHECK(x.is_contiguous() && W.is_contiguous() && out.stride(1) == 1, "contiguous");
  const int M = x.size(0), K = x.size(1);
  TORCH_CHECK(W.size(1) == K, "K mismatch");
  const int N = mode == 0 ? W.size(0) : W.size(0) / 2;
  TORCH_CHECK(mode == 0 || W.size(0) % 2 == 0, "gate_up rows even");
  TORCH_CHECK(out.size(0) == M && out.size(1) == N, "out shape");
  CHECK_RC(omnia_dgemm((int)mode, out.data_ptr(), x.data_ptr(), W.data_ptr(),
                       ws.data_ptr<float>(), cnt.data_ptr<int>(), M, N, K, (int)splits, (int)wm,
                       (int)wn, (int)out.stride(0), ws.numel(), (int)cnt.numel(), cur_stream()),
           "dgemm");
}

// weight-streaming decode GEMM (wgemm.hip): mode 0 bf16 out[M,N] = x W^T; mode 1
// SwiGLU bf16 out[M,I] from W = [Wg; Wu]; mode 2 fp32 split-K slabs out[S,M,N].
void wgemm(int64_t mode, at::Tensor out, at::Tensor x, at::Tensor W, int64_t splits, int64_t nw,
           int64_t nwaves) {
  CHECK_GPU(x); CHECK_BF16(x); CHECK_BF16(W);
  TORCH_CHECK(x.dim() == 2 && W.dim() == 2, "2-D operands");
  TORCH_CHECK(x.is_contiguous() && W.is_contiguous(), "contiguous x / W");
  const int M = x.size(0), K = x.size(1);
  TORCH_CHECK(W.size(1) == K, "K mismatch");
  TORCH_CHECK(mode == 0 || mode == 1 || mode == 2, "mode");
  TORCH_CHECK(mode != 1 || W.size(0) % 2 == 0, "gate_up rows even");
  const int N = mode == 1 ? W.size(0) / 2 : W.size(0);
  int ldo;
  if (mode == 2) {
    TORCH_CHECK(out.scalar_type() == at::kFloat && out.is_cuda() && out.is_contiguous(),
                "mode 2: fp32 contiguous slabs");
    TORCH_CHECK(out.dim() == 3 && out.size(0) == splits && out.size(1) == M && out.size(2) == N,
                "mode 2: out [S, M, N]");
    ldo = N;
  } else {
    CHECK_BF16(out);
    TORCH_CHECK(out.dim() == 2 && out.size(0) == M && out.size(1) == N && out.stride(1) == 1,
                "out [M, N]");
    ldo = out.stride(0);
  }
  CHECK_RC(omnia_wgemm((int)mode, out.data_ptr(), x.data_ptr(), W.data_ptr(), M, N, K,
                       (int)splits, (int)nw, (int)nwaves, ldo, cur_stream()),
           "wgemm");
}

// wide-batch weight-streaming decode GEMM (wgemm_wide.hip, 128 < M <= 256):
// same modes / out shapes as wgemm; wt = 32-column MFMA tiles per wave (1 or 2)
void wgemm_wide(int64_t mode, at::Tensor out, at::Tensor x, at::Tensor W, int64_t splits,
                int64_t wt) {
  CHECK_BF16(x); CHECK_BF16(W);
  TORCH_CHECK(x.dim() == 2 && W.dim() == 2, "2-D operands");
  TORCH_CHECK(x.is_contiguous() && W.is_contiguous(), "contiguous x / W");
  const int M = x.size(0), K = x.size(1);
  TORCH_CHECK(W.size(1) == K, "K mismatch");
  TORCH_CHECK(mode == 0 || mode == 1 || mode == 2, "mode");
  TORCH_CHECK(mode != 1 || W.size(0) % 2 == 0, "gate_up rows even");
  const int N = mode == 1 ? W.size(0) / 2 : W.size(0);
  int ldo;
  if (mode == 2) {
    TORCH_CHECK(out.scalar_type() == at::kFloat && out.is_cuda() && out.is_contiguous(),
                "mode 2: fp32 contiguous slabs");
    TORCH_CHECK(out.dim() == 3 && out.size(0) == splits && out.size(1) == M && out.size(2) == N,
                "mode 2: out [S, M, N]");
    ldo = N;
  } else {
    CHECK_BF16(out);
    TORCH_CHECK(out.dim() == 2 && out.size(0) == M && out.size(1) == N && out.stride(1) == 1,
                "out [M, N]");
    ldo = out.stride(0);
  }
  CHECK_RC(omnia_wgemm_wide((int)mode, out.data_ptr(), x.data_ptr(), W.data_ptr(), M, N, K,
                            (int)splits, (int)wt, ldo, cur_stream()),
           "wgemm_wide");
}

// full-batch tile decode GEMM (tgemm.hip, M <= 256): same modes / out shapes as
// wgemm; bn = weight rows per block (64/128/256), wnt = non-temporal weight loads
void tgemm(int64_t mode, at::Tensor out, at::Tensor x, at::Tensor W, int64_t splits, int64_t bn,
           int64_t wnt) {
  CHECK_GPU(x); CHECK_BF16(x); CHECK_BF16(W);
  TORCH_CHECK(x.dim() == 2 && W.dim() == 2, "2-D operands");
  TORCH_CHECK(x.is_contiguous() && W.is_contiguous(), "contiguous x / W");
  TORCH_CHECK(x.device() == W.device() && x.device() == out.device(), "same device");
  const int M = x.size(0), K = x.size(1);
  TORCH_CHECK(W.size(1) == K, "K mismatch");
  TORCH_CHECK(mode >= 0 && mode <= 3, "mode");
  TORCH_CHECK(mode != 1 || W.size(0) % 2 == 0, "gate_up rows even");
  const int N = mode == 1 ? W.size(0) / 2 : W.size(0);
  int ldo;
  if (mode >= 2) {
    TORCH_CHECK(out.scalar_type() == (mode == 2 ? at::kFloat : at::kHalf) && out.is_contiguous(),
                "mode 2 / 3: fp32 / fp16 contiguous slabs");
    TORCH_CHECK(out.dim() == 3 && out.size(0) == splits && out.size(1) == M && out.size(2) == N,
                "mode 2 / 3: out [S, M, N]");
    ldo = N;
  } else {
    CHECK_BF16(out);
    TORCH_CHECK(out.dim() == 2 && out.size(0) == M && out.size(1) == N && out.stride(1) == 1,
                "out [M, N]");
    ldo = out.stride(0);
  }
  CHECK_RC(omnia_tgemm((int)mode, out.data_ptr(), x.data_ptr(), W.data_ptr(), M, N, K,
                       (int)splits, (int)bn, (int)wnt, ldo, cur_stream()),
           "tgemm");
}

// prefill GEMM with fused epilogues (pgemm.hip, 256x256 tiles): epi 0 plain
// (optionally row-scaled), 1 gate_up + SwiGLU, 2 residual add + row sum of
// squares, 3 QKV + RoPE + paged KV write.  ss_in = partial row sums of squares
// [M, n] of x (row scale rsqrt(sum / d + eps)), ss_out = [M, N / 256].
void pgemm(int64_t epi, at::Tensor out, at::Tensor x, at::Tensor W,
           c10::optional<at::Tensor> ss_in, double inv_d, double eps,
           c10::optional<at::Tensor> ss_out, c10::optional<at::Tensor> positions,
           c10::optional<at::Tensor> cos_sin, c10::optional<at::Tensor> k_cache,
           c10::optional<at::Tensor> v_cache, c10::optional<at::Tensor> slots, int64_t hq,
           int64_t hkv, int64_t block_size, c10::optional<at::Tensor> bias, bool gelu) {
  CHECK_GPU(x); CHECK_BF16(x); CHECK_BF16(W); CHECK_BF16(out);
  TORCH_CHECK(x.dim() == 2 && W.dim() == 2 && out.dim() == 2, "2-D operands");
  TORCH_CHECK(x.is_contiguous() && W.is_contiguous(), "contiguous x / W");
  TORCH_CHECK(out.stride(1) == 1, "out rows contiguous");
  TORCH_CHECK(x.device() == W.device() && x.device() == out.device(), "same device");
  TORCH_CHECK(epi >= 0 && epi <= 3, "epi");
  const int M = x.size(0), K = x.size(1);
  TORCH_CHECK(W.size(1) == K, "K mismatch");
  TORCH_CHECK(epi != 1 || W.size(0) % 2 == 0, "gate_up rows even");
  const int N = epi == 1 ? W.size(0) / 2 : W.size(0);
  TORCH_CHECK(out.size(0) == M, "out rows");
  TORCH_CHECK(out.size(1) == (epi == 3 ? hq * 128 : N), "out [M, N] (q [M, hq*128] for epi 3)");
  const float* ssi = nullptr;
  int ssn = 0;
  if (ss_in.has_value() && ss_in->defined()) {
    TORCH_CHECK(ss_in->scalar_type() == at::kFloat && ss_in->is_contiguous() && ss_in->dim() == 2 &&
                ss_in->size(0) == M && ss_in->device() == x.device(), "ss_in fp32 [M, n]");
    ssi = ss_in->data_ptr<float>();
    ssn = ss_in->size(1);
  }
  float* sso = nullptr;
  if (epi == 2) {
    TORCH_CHECK(ss_out.has_value() && ss_out->defined(), "epi 2 needs ss_out");
    TORCH_CHECK(ss_out->scalar_type() == at::kFloat && ss_out->is_contiguous() &&
                ss_out->dim() == 2 && ss_out->size(0) == M && ss_out->size(1) == N / 256 &&
                ss_out->device() == x.device(), "ss_out fp32 [M, N/256]");
    sso = ss_out->data_ptr<float>();
  }
  const int* pos = nullptr;
  const float* cs = nullptr;
  void *kc = nullptr, *vc = nullptr;
  const int64_t* sl = nullptr;
  if (epi == 3) {
    TORCH_CHECK(positions.has_value() && cos_sin.has_value() && k_cache.has_value() &&
                v_cache.has_value() && slots.has_value(), "epi 3 needs rope / cache operands");
    TORCH_CHECK(positions->scalar_type() == at::kInt && positions->numel() == M &&
                positions->is_contiguous(), "positions int32 [M]");
    TORCH_CHECK(cos_sin->scalar_type() == at::kFloat && cos_sin->is_contiguous() &&
                cos_sin->dim() == 2 && cos_sin->size(1) == 128, "cos_sin f32 [P, 128]");
    TORCH_CHECK(slots->scalar_type() == at::kLong && slots->numel() == M && slots->is_contiguous(),
                "slots int64 [M]");
    CHECK_BF16(*k_cache); CHECK_BF16(*v_cache);
    TORCH_CHECK(k_cache->dim() == 4 && k_cache->size(1) == hkv && k_cache->size(2) == block_size &&
                k_cache->size(3) == 128 && k_cache->is_contiguous() && v_cache->is_contiguous() &&
                v_cache->sizes() == k_cache->sizes(), "cache layout [NB, Hkv, BS, 128]");
    for (const at::Tensor* t : {&*positions, &*cos_sin, &*k_cache, &*v_cache, &*slots})
      TORCH_CHECK(t->device() == x.device(), "same device");
    pos = positions->data_ptr<int>();
    cs = cos_sin->data_ptr<float>();
    kc = k_cache->data_ptr();
    vc = v_cache->data_ptr();
    sl = slots->data_ptr<int64_t>();
  }
  const float* bp = nullptr;
  if (bias.has_value() && bias->defined()) {
    TORCH_CHECK(epi == 1 && bias->is_cuda() && bias->scalar_type() == at::kFloat &&
                bias->is_contiguous() && bias->numel() == 2 * N, "bias fp32 [2N] (epi 1)");
    bp = bias->data_ptr<float>();
  }
  if (M == 0) return;
  CHECK_RC(omnia_pgemm((int)epi, out.data_ptr(), x.data_ptr(), W.data_ptr(), M, N, K,
                       out.stride(0), ssi, ssn, (float)inv_d, (float)eps, sso, pos, cs, kc, vc, sl,
                       (int)hq, (int)hkv, (int)block_size, bp, gelu, cur_stream()),
           "pgemm");
}

void pgemm_variant(int64_t variant, at::Tensor out, at::Tensor x, at::Tensor W) {
  CHECK_GPU(x); CHECK_BF16(x); CHECK_BF16(W); CHECK_BF16(out);
  TORCH_CHECK(x.is_contiguous() && W.is_contiguous() && out.is_contiguous(), "contiguous");
  TORCH_CHECK(x.dim() == 2 && W.dim() == 2 && W.size(1) == x.size(1) && out.size(0) == x.size(0) &&
              out.size(1) == W.size(0), "shapes");
  CHECK_RC(omnia_pgemm_variant((int)variant, out.data_ptr(), x.data_ptr(), W.data_ptr(),
                               x.size(0), W.size(0), x.size(1), cur_stream()),
           "pgemm_variant");
}

// split-K 256x256 MFMA GEMM (pgemm.hip EPI 4): parts fp16 [S, M, N] whose sum
// over S is x @ W^T; sched 0 / 1 = 8-wave / 4-wave main loop
void pgemm_splitk(at::Tensor parts, at::Tensor x, at::Tensor W, int64_t sched) {
  CHECK_GPU(x); CHECK_BF16(x); CHECK_BF16(W);
  TORCH_CHECK(x.dim() == 2 && W.dim() == 2 && W.size(1) == x.size(1), "x [M, K], W [N, K]");
  TORCH_CHECK(x.is_contiguous() && W.is_contiguous(), "contiguous x / W");
  TORCH_CHECK(parts.scalar_type() == at::kHalf && parts.is_contiguous() && parts.dim() == 3 &&
              parts.size(1) == x.size(0) && parts.size(2) == W.size(0), "parts fp16 [S, M, N]");
  TORCH_CHECK(x.device() == W.device() && x.device() == parts.device(), "same device");
  if (x.size(0) == 0) return;
  CHECK_RC(omnia_pgemm_splitk(parts.data_ptr(), x.data_ptr(), W.data_ptr(), x.size(0), W.size(0),
                              x.size(1), parts.size(0), (int)sched, cur_stream()),
           "pgemm_splitk");
}

void row_sumsq(at::Tensor ss, at::Tensor x) {
  CHECK_GPU(x); CHECK_BF16(x);
  TORCH_CHECK(x.dim() == 2 && x.stride(1) == 1, "x [M, d] rows contiguous");
  TORCH_CHECK(ss.scalar_type() == at::kFloat && ss.is_contiguous() && ss.numel() == x.size(0) &&
              ss.device() == x.device(), "ss fp32 [M]");
  CHECK_RC(omnia_row_sumsq(ss.data_ptr<float>(), x.data_ptr(), x.size(0), x.size(1), x.stride(0),
                           cur_stream()),
           "row_sumsq");
}

// ------------------------------------------------- split-K consumers (splitk.hip)
// fp32 slabs, or fp16 ones (tgemm mode 3); returns 1 for fp16
static int check_parts(const at::Tensor& p) {
  TORCH_CHECK(p.is_cuda() && (p.scalar_type() == at::kFloat || p.scalar_type() == at::kHalf) &&
              p.is_contiguous() && p.dim() == 3, "parts: contiguous fp32 / fp16 [S, M, N]");
  TORCH_CHECK(p.size(0) >= 1 && p.size(0) <= 16, "1 <= S <= 16");
  return p.scalar_type() == at::kHalf ? 1 : 0;
}

void splitk_add_rmsnorm(at::Tensor out, at::Tensor parts, at::Tensor residual, at::Tensor w,
                        double eps) {
  const int half = check_parts(parts);
  CHECK_BF16(out); CHECK_BF16(residual); CHECK_BF16(w);
  const int M = parts.size(1), d = parts.size(2);
  TORCH_CHECK(residual.is_contiguous() && residual.size(0) == M && residual.size(1) == d,
              "residual [M, d]");
  TORCH_CHECK(out.is_contiguous() && out.size(0) == M && out.size(1) == d, "out [M, d]");
  TORCH_CHECK(w.numel() == d, "w [d]");
  CHECK_RC(omnia_splitk_add_rmsnorm(out.data_ptr(), parts.data_ptr(), half, residual.data_ptr(),
                                    w.data_ptr(), parts.size(0), M, d, (float)eps, cur_stream()),
           "splitk_add_rmsnorm");
}

void splitk_rope_kv(at::Tensor q, at::Tensor parts, at::Tensor positions, at::Tensor cos_sin,
                    at::Tensor k_cache, at::Tensor v_cache, at::Tensor slots, int64_t hq,
                    int64_t hkv, int64_t block_size) {
  const int half = check_parts(parts);
  CHECK_BF16(q); CHECK_BF16(k_cache); CHECK_BF16(v_cache); CHECK_I32(positions);
  const int T = parts.size(1);
  TORCH_CHECK(parts.size(2) == (hq + 2 * hkv) * 128, "parts N = (hq + 2 hkv) * 128");
  TORCH_CHECK(q.is_contiguous() && q.size(0) == T && q.size(1) == hq * 128, "q [T, hq*128]");
  TORCH_CHECK(positions.numel() == T && slots.numel() == T, "positions / slots [T]");
  TORCH_CHECK(slots.scalar_type() == at::kLong, "slots int64");
  TORCH_CHECK(cos_sin.scalar_type() == at::kFloat && cos_sin.size(1) == 128, "cos_sin");
  TORCH_CHECK(k_cache.dim() == 4 && k_cache.size(1) == hkv && k_cache.size(2) == block_size &&
              k_cache.size(3) == 128 && k_cache.is_contiguous() && v_cache.is_contiguous(),
              "cache [NB, Hkv, BS, 128]");
  CHECK_RC(omnia_splitk_rope_kv(q.data_ptr(), parts.data_ptr(), half, parts.size(0), T,
                                positions.data_ptr<int>(), cos_sin.data_ptr<float>(),
                                k_cache.data_ptr(), v_cache.data_ptr(),
                                slots.data_ptr<int64_t>(), hq, hkv, 128, block_size,
                                cur_stream()),
           "splitk_rope_kv");
}

void splitk_swiglu(at::Tensor out, at::Tensor parts) {
  const int half = check_parts(parts);
  CHECK_BF16(out);
  const int M = parts.size(1), I = parts.size(2) / 2;
  TORCH_CHECK(parts.size(2) % 2 == 0 && out.is_contiguous() && out.size(0) == M &&
              out.size(1) == I, "out [M, I] for parts [S, M, 2I]");
  CHECK_RC(omnia_splitk_swiglu(out.data_ptr(), parts.data_ptr(), half, parts.size(0), M, I,
                               cur_stream()), "splitk_swiglu");
}

void splitk_reduce(at::Tensor out, at::Tensor parts) {
  const int half = check_parts(parts);
  CHECK_BF16(out);
  TORCH_CHECK(out.is_contiguous() && out.numel() == parts.size(1) * parts.size(2), "out [M, N]");
  CHECK_RC(omnia_splitk_reduce(out.data_ptr(), parts.data_ptr(), half, parts.size(0),
                               out.numel(), cur_stream()), "splitk_reduce");
}

// ------------------------------------------------- one-shot IPC all-reduce (K16)
int64_t ipc_alloc(int64_t bytes) {
  void* p = nullptr;
  CHECK_RC(omnia_ipc_alloc(&p, bytes), "ipc_alloc");
  return reinterpret_cast<int64_t>(p);
}
void ipc_free(int64_t ptr) { CHECK_RC(omnia_ipc_free(reinterpret_cast<void*>(ptr)), "ipc_free"); }
py::bytes ipc_get_handle(int64_t ptr) {
  std::string h(omnia_ipc_handle_size(), '\0');
  CHECK_RC(omnia_ipc_get_handle(reinterpret_cast<void*>(ptr), &h[0]), "ipc_get_handle");
  return py::bytes(h);
}
int64_t ipc_open(py::bytes handle) {
  std::string h = handle;
  TORCH_CHECK((int)h.size() == omnia_ipc_handle_size(), "bad IPC handle size");
  void* p = nullptr;
  CHECK_RC(omnia_ipc_open(h.data(), &p), "ipc_open");
  return reinterpret_cast<int64_t>(p);
}
void ipc_close(int64_t ptr) { CHECK_RC(omnia_ipc_close(reinterpret_cast<void*>(ptr)), "ipc_close"); }

// regions: int64 CPU tensor [world] of region base pointers (own + opened peers)
void ar_oneshot(at::Tensor out, at::Tensor in, at::Tensor regions, at::Tensor epochs,
                at::Tensor err, int64_t slot_bytes, int64_t rank) {
  CHECK_GPU(in); CHECK_BF16(in); CHECK_BF16(out); CHECK_I32(epochs); CHECK_I32(err);
  TORCH_CHECK(in.is_contiguous() && out.is_contiguous() && in.numel() == out.numel(), "contig");
  TORCH_CHECK(regions.device().is_cpu() && regions.scalar_type() == at::kLong, "regions cpu i64");
  TORCH_CHECK(epochs.numel() >= omnia_ar_blocks(), "epochs per block");
  const int world = regions.numel();
  TORCH_CHECK(world <= omnia_ar_max_ranks(), "world too large");
  std::vector<void*> regs(world);
  for (int p = 0; p < world; ++p) regs[p] = reinterpret_cast<void*>(regions.data_ptr<int64_t>()[p]);
  CHECK_RC(omnia_ar_oneshot(out.data_ptr(), in.data_ptr(), regs.data(), epochs.data_ptr<int>(),
                            err.data_ptr<int>(), in.numel(), slot_bytes, (int)rank, world,
                            cur_stream()), "ar_oneshot");
}

// all-gather of any contiguous tensor's bytes over the IPC regions: out holds
// world x in.nbytes (rank order)
void ar_allgather(at::Tensor out, at::Tensor in, at::Tensor regions, at::Tensor epochs,
                  at::Tensor err, int64_t slot_bytes, int64_t rank) {
  CHECK_GPU(in); CHECK_GPU(out); CHECK_I32(epochs); CHECK_I32(err);
  TORCH_CHECK(in.is_contiguous() && out.is_contiguous(), "contiguous");
  TORCH_CHECK(regions.device().is_cpu() && regions.scalar_type() == at::kLong, "regions cpu i64");
  TORCH_CHECK(epochs.numel() >= omnia_ar_blocks(), "epochs per block");
  const int world = regions.numel();
  TORCH_CHECK(world <= omnia_ar_max_ranks(), "world too large");
  const int64_t nb = in.numel() * in.element_size();
  TORCH_CHECK(out.numel() * out.element_size() == nb * world, "out must hold world x in bytes");
  std::vector<void*> regs(world);
  for (int p = 0; p < world; ++p) regs[p] = reinterpret_cast<void*>(regions.data_ptr<int64_t>()[p]);
  CHECK_RC(omnia_ar_allgather(out.data_ptr(), in.data_ptr(), regs.data(), epochs.data_ptr<int>(),
                              err.data_ptr<int>(), nb, slot_bytes, (int)rank, world,
                              cur_stream()), "ar_allgather");
}

// IPC all-to-all: in / out [world][chunk] (any dtype, chunk bytes % 16 == 0)
void ar_alltoall(at::Tensor out, at::Tensor in, at::Tensor regions, at::Tensor epochs,
                 at::Tensor err, int64_t slot_bytes, int64_t rank) {
  CHECK_GPU(in); CHECK_GPU(out); CHECK_I32(epochs); CHECK_I32(err);
  TORCH_CHECK(in.is_contiguous() && out.is_contiguous(), "contiguous");
  TORCH_CHECK(in.device() == out.device() && epochs.device() == in.device() &&
              err.device() == in.device(), "same device");
  TORCH_CHECK(regions.device().is_cpu() && regions.scalar_type() == at::kLong, "regions cpu i64");
  TORCH_CHECK(epochs.numel() >= omnia_ar_blocks(), "epochs per block");
  const int world = regions.numel();
  TORCH_CHECK(world <= omnia_ar_max_ranks(), "world too large");
  const int64_t nb = in.numel() * in.element_size();
  TORCH_CHECK(out.numel() * out.element_size() == nb && nb % world == 0,
              "in / out: [world][chunk] bytes");
  std::vector<void*> regs(world);
  for (int p = 0; p < world; ++p) regs[p] = reinterpret_cast<void*>(regions.data_ptr<int64_t>()[p]);
  CHECK_RC(omnia_ar_alltoall(out.data_ptr(), in.data_ptr(), regs.data(), epochs.data_ptr<int>(),
                             err.data_ptr<int>(), nb / world, slot_bytes, (int)rank, world,
                             cur_stream()), "ar_alltoall");
}

// IPC point-to-point: out <- rank src's `in` (same bytes on every rank)
void ar_sendrecv(at::Tensor out, at::Tensor in, at::Tensor regions, at::Tensor epochs,
                 at::Tensor err, int64_t slot_bytes, int64_t rank, int64_t src) {
  CHECK_GPU(in); CHECK_GPU(out); CHECK_I32(epochs); CHECK_I32(err);
  TORCH_CHECK(in.is_contiguous() && out.is_contiguous(), "contiguous");
  TORCH_CHECK(in.device() == out.device() && epochs.device() == in.device() &&
              err.device() == in.device(), "same device");
  TORCH_CHECK(regions.device().is_cpu() && regions.scalar_type() == at::kLong, "regions cpu i64");
  TORCH_CHECK(epochs.numel() >= omnia_ar_blocks(), "epochs per block");
  const int world = regions.numel();
  TORCH_CHECK(world <= omnia_ar_max_ranks(), "world too large");
  const int64_t nb = in.numel() * in.element_size();
  TORCH_CHECK(out.numel() * out.element_size() == nb, "out bytes == in bytes");
  std::vector<void*> regs(world);
  for (int p = 0; p < world; ++p) regs[p] = reinterpret_cast<void*>(regions.data_ptr<int64_t>()[p]);
  CHECK_RC(omnia_ar_sendrecv(out.data_ptr(), in.data_ptr(), regs.data(), epochs.data_ptr<int>(),
                             err.data_ptr<int>(), nb, slot_bytes, (int)rank, world, (int)src,
                             cur_stream()), "ar_sendrecv");
}

// two-shot (reduce-scatter + all-gather) over the same IPC regions; with w the
// fused residual add + RMSNorm variant (residual updated in place)
void ar_twoshot(at::Tensor out, at::Tensor in, c10::optional<at::Tensor> residual,
                c10::optional<at::Tensor> w, at::Tensor regions, at::Tensor epochs, at::Tensor err,
                int64_t slot_bytes, int64_t rank, double eps) {
  CHECK_GPU(in); CHECK_BF16(in); CHECK_BF16(out); CHECK_I32(epochs); CHECK_I32(err);
  TORCH_CHECK(in.dim() == 2 && in.is_contiguous() && out.is_contiguous() &&
              out.sizes() == in.sizes(), "in/out contiguous [M, d]");
  TORCH_CHECK(regions.device().is_cpu() && regions.scalar_type() == at::kLong, "regions cpu i64");
  TORCH_CHECK(epochs.numel() >= omnia_ar_blocks(), "epochs per block");
  const bool norm = w.has_value() && w->defined();
  if (norm) {
    TORCH_CHECK(residual.has_value() && residual->defined(), "NORM needs the residual");
    CHECK_BF16((*residual)); CHECK_BF16((*w));
    TORCH_CHECK(residual->sizes() == in.sizes() && residual->is_contiguous(), "residual [M, d]");
    TORCH_CHECK(w->numel() == in.size(1), "w [d]");
  }
  const int world = regions.numel();
  TORCH_CHECK(world <= omnia_ar_max_ranks(), "world too large");
  std::vector<void*> regs(world);
  for (int p = 0; p < world; ++p) regs[p] = reinterpret_cast<void*>(regions.data_ptr<int64_t>()[p]);
  CHECK_RC(omnia_ar_twoshot(out.data_ptr(), in.data_ptr(), opt_ptr<void>(residual),
                            opt_ptr<void>(w), regs.data(), epochs.data_ptr<int>(),
                            err.data_ptr<int>(), in.size(0), in.size(1), slot_bytes, (int)rank,
                            world, (float)eps, cur_stream()), "ar_twoshot");
}

// ------------------------------------------------- host step launch (no GIL churn)
// One decode step = H2D staging copy + graph launch + D2H token copy + event
// record, enqueued back to back on the current stream inside ONE Python call.
// Each separate torch call would drop and re-take the GIL; with a busy asyncio
// serving thread every re-take can wait a full switch interval, starving the
// engine thread and idling the GPU between steps.
void graph_launch_step(int64_t graph_exec, int64_t h2d_dst, int64_t h2d_src, int64_t h2d_bytes,
                       int64_t d2h_dst, int64_t d2h_src, int64_t d2h_bytes, int64_t event) {
  hipStream_t s = cur_stream();
  if (h2d_bytes > 0)
    TORCH_CHECK(hipMemcpyAsync(reinterpret_cast<void*>(h2d_dst),
                               reinterpret_cast<const void*>(h2d_src), h2d_bytes,
                               hipMemcpyHostToDevice, s) == hipSuccess, "H2D staging copy");
  TORCH_CHECK(hipGraphLaunch(reinterpret_cast<hipGraphExec_t>(graph_exec), s) == hipSuccess,
              "hipGraphLaunch");
  if (d2h_bytes > 0)
    TORCH_CHECK(hipMemcpyAsync(reinterpret_cast<void*>(d2h_dst),
                               reinterpret_cast<const void*>(d2h_src), d2h_bytes,
                               hipMemcpyDeviceToHost, s) == hipSuccess, "D2H token copy");
  if (event)
    TORCH_CHECK(hipEventRecord(reinterpret_cast<hipEvent_t>(event), s) == hipSuccess,
                "hipEventRecord");
}

// Same step, but the staging upload is a compute-queue kernel reading the
// mapped pinned buffer (`src_dev` = omnia_host_device_ptr of it) instead of an
// SDMA copy the compute queue would have to wait on; only the scalar head and
// the [rows x row_bytes] block-table window the graph bucket reads are moved.
void graph_launch_staged(int64_t graph_exec, int64_t dst, int64_t src_dev, int64_t head_bytes,
                         int64_t bt_off, int64_t row_stride, int64_t rows, int64_t row_bytes,
                         int64_t d2h_dst, int64_t d2h_src, int64_t d2h_bytes, int64_t event) {
  hipStream_t s = cur_stream();
  TORCH_CHECK(dst && src_dev && rows >= 0 && rows <= (1 << 20), "bad staging operands");
  CHECK_RC(omnia_stage_copy(reinterpret_cast<void*>(dst), reinterpret_cast<const void*>(src_dev),
                            head_bytes, bt_off, row_stride, (int)rows, row_bytes, s),
           "stage_copy");
  TORCH_CHECK(hipGraphLaunch(reinterpret_cast<hipGraphExec_t>(graph_exec), s) == hipSuccess,
              "hipGraphLaunch");
  if (d2h_bytes > 0)
    TORCH_CHECK(hipMemcpyAsync(reinterpret_cast<void*>(d2h_dst),
                               reinterpret_cast<const void*>(d2h_src), d2h_bytes,
                               hipMemcpyDeviceToHost, s) == hipSuccess, "D2H token copy");
  if (event)
    TORCH_CHECK(hipEventRecord(reinterpret_cast<hipEvent_t>(event), s) == hipSuccess,
                "hipEventRecord");
}

// standalone staged upload (tests / non-graph paths)
void stage_copy(int64_t dst, int64_t src_dev, int64_t head_bytes, int64_t bt_off,
                int64_t row_stride, int64_t rows, int64_t row_bytes) {
  TORCH_CHECK(dst && src_dev && rows >= 0 && rows <= (1 << 20), "bad staging operands");
  CHECK_RC(omnia_stage_copy(reinterpret_cast<void*>(dst), reinterpret_cast<const void*>(src_dev),
                            head_bytes, bt_off, row_stride, (int)rows, row_bytes, cur_stream()),
           "stage_copy");
}

int64_t host_device_ptr(at::Tensor host) {
  TORCH_CHECK(host.is_pinned(), "host_device_ptr needs a pinned tensor");
  return omnia_host_device_ptr(host.data_ptr());
}

int64_t event_create() {
  hipEvent_t e;
  TORCH_CHECK(hipEventCreateWithFlags(&e, hipEventDisableTiming) == hipSuccess,
              "hipEventCreate");
  return reinterpret_cast<int64_t>(e);
}

void event_destroy(int64_t e) { (void)hipEventDestroy(reinterpret_cast<hipEvent_t>(e)); }

bool event_query(int64_t e) {
  return hipEventQuery(reinterpret_cast<hipEvent_t>(e)) == hipSuccess;
}

// wait for an event; the GIL is released only if it has not completed yet.
// Returns the nanoseconds spent re-acquiring the GIL after the event fired
// (the serving thread's hold time -- a direct measure of GIL contention).
int64_t event_sync(int64_t e) {
  auto ev = reinterpret_cast<hipEvent_t>(e);
  if (hipEventQuery(ev) == hipSuccess) return 0;
  std::chrono::steady_clock::time_point done;
  {
    py::gil_scoped_release rel;
    TORCH_CHECK(hipEventSynchronize(ev) == hipSuccess, "hipEventSynchronize");
    done = std::chrono::steady_clock::now();
  }
  return std::chrono::duration_cast<std::chrono::nanoseconds>(
             std::chrono::steady_clock::now() - done).count();
}

// ------------------------------------------------- layer-list models (bf16 or fp32)
using OptT = c10::optional<at::Tensor>;

// 1: fp32 storage, 0: bf16
int is_f32(const at::Tensor& t, const char* what) {
  CHECK_GPU(t);
  TORCH_CHECK(t.scalar_type() == at::kBFloat16 || t.scalar_type() == at::kFloat, what,
              " must be bf16 or fp32");
  return t.scalar_type() == at::kFloat;
}
void like(const at::Tensor& t, const at::Tensor& ref, int64_t numel, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == ref.scalar_type() && t.is_contiguous() &&
              t.numel() == numel, what, ": want ", numel, " contiguous elements of the model dtype");
}
const float* vecf(const at::Tensor& t, int64_t n, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kFloat && t.is_contiguous() && t.numel() == n,
              what, ": want fp32 [", n, "]");
  return t.data_ptr<float>();
}
const int* veci(const at::Tensor& t, int64_t n, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kInt && t.is_contiguous() && t.numel() == n,
              what, ": want int32 [", n, "]");
  return t.data_ptr<int>();
}
float* outf(const at::Tensor& t, int64_t n, const char* what) {
  return const_cast<float*>(vecf(t, n, what));
}
// a row view [T, >= width] with contiguous columns; returns the row stride
int64_t rows2(const at::Tensor& t, int64_t T, int64_t width, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.dim() == 2 && t.stride(1) == 1 && t.size(0) == T &&
              t.size(1) >= width, what, ": want [", T, ", >= ", width, "] rows");
  return t.stride(0);
}

// a projection: [M, N] in bf16 / fp32, or split-K slabs [S, M, N] in fp32 / fp16; rows may
// be columns of a wider projection (row stride ld, slab stride slab)
struct Proj { int type, S; int64_t M, N, ld, slab; };
Proj proj(const at::Tensor& m, bool strided = false) {
  CHECK_GPU(m);
  const bool p = m.dim() == 3;
  TORCH_CHECK((m.dim() == 2 || p) && (strided ? m.stride(-1) == 1 : m.is_contiguous()),
              "projection [M, N] or [S, M, N]");
  const auto st = m.scalar_type();
  TORCH_CHECK(st == at::kBFloat16 || st == at::kFloat || st == at::kHalf, "projection dtype");
  return {st == at::kBFloat16 ? 0 : st == at::kFloat ? 1 : 2, p ? (int)m.size(0) : 1,
          p ? m.size(1) : m.size(0), m.size(-1), m.stride(-2), p ? m.stride(0) : 0};
}

void tanh_norm_embed(at::Tensor h, at::Tensor x, at::Tensor ids, at::Tensor table, int64_t vocab,
                     double alpha, at::Tensor w, at::Tensor b, OptT src, OptT tok_slots) {
  const int f32 = is_f32(table, "table");
  TORCH_CHECK(table.dim() == 2 && table.is_contiguous() && table.size(0) >= vocab, "table [V, d]");
  const int64_t T = ids.numel(), d = table.size(1);
  like(h, table, T * d, "h");
  const int64_t* sp = nullptr;
  if (src.has_value() && src->defined()) {
    TORCH_CHECK(src->is_cuda() && src->scalar_type() == at::kLong && src->is_contiguous() &&
                src->numel() == T && tok_slots.has_value(), "src int64 [T] with tok_slots");
    CHECK_I32(*tok_slots);
    sp = src->data_ptr<int64_t>();
  }
  CHECK_RC(omnia_tanh_norm_embed(h.data_ptr(), outf(x, T * d, "x"), veci(ids, T, "ids"),
                                 table.data_ptr(), f32, T, d, vocab, (float)alpha, vecf(w, d, "w"),
                                 vecf(b, d, "b"), sp, opt_ptr<int>(tok_slots), cur_stream()),
           "tanh_norm_embed");
}

// m: a projection [M, d], split-K slabs [S, M, d], or (slots) per-row parts [M, S, d]
struct ResidParts { int type; int64_t S, M, d, row, part; };
ResidParts resid_parts(const at::Tensor& m, bool slots) {
  const Proj p = proj(m);
  TORCH_CHECK(!slots || m.dim() == 3, "slots [M, S, d]");
  const int64_t S = slots ? p.M : p.S, M = slots ? m.size(0) : p.M;
  return {p.type, S, M, p.N, slots ? S * p.N : p.N, slots ? p.N : M * p.N};
}
const float* opt_vecf(const OptT& t, int64_t n, const char* what) {
  return t.has_value() && t->defined() ? vecf(*t, n, what) : nullptr;
}

// w1 null: no post-norm.  ids / wts [M, S], in [M, d]: parts of identity experts (ids >=
// first) stand for wts * in
void tanh_norm_residual(at::Tensor h, at::Tensor x, at::Tensor m, bool slots, OptT bias, double a1,
                        OptT w1, OptT b1, double a2, at::Tensor w2, at::Tensor b2, OptT ids,
                        OptT wts, OptT in, int64_t first) {
  const int f32 = is_f32(h, "h");
  const ResidParts p = resid_parts(m, slots);
  const int64_t d = p.d;
  like(h, h, p.M * d, "h");
  const float* w1p = opt_vecf(w1, d, "w1");
  TORCH_CHECK(!w1p || (b1.has_value() && b1->defined()), "w1 comes with b1");
  const int* idp = nullptr;
  if (ids.has_value() && ids->defined()) {
    TORCH_CHECK(slots && wts.has_value() && in.has_value(), "identity parts: slots, wts, in");
    idp = veci(*ids, p.M * p.S, "ids");
    vecf(*wts, p.M * p.S, "wts");
    like(*in, h, p.M * d, "in");
  }
  CHECK_RC(omnia_tanh_norm_residual(
               h.data_ptr(), f32, outf(x, p.M * d, "x"), m.data_ptr(), p.type, p.S, p.row, p.part,
               p.M, d, opt_vecf(bias, d, "bias"), (float)a1, w1p, opt_vecf(b1, d, "b1"),
               (float)a2, vecf(w2, d, "w2"), vecf(b2, d, "b2"), idp,
               idp ? wts->data_ptr<float>() : nullptr, idp ? in->data_ptr() : nullptr, first,
               cur_stream()),
           "tanh_norm_residual");
}

// x += rms(a + abias) aw + rms(b + bbias) bw; h = x (nw null), RMS (nb null) or tanh norm
void branch_residual(at::Tensor h, at::Tensor x, at::Tensor a, OptT abias, at::Tensor aw,
                     at::Tensor b, OptT bbias, at::Tensor bw, double inv_n, double eps,
                     double alpha, OptT nw, OptT nb) {
  const int f32 = is_f32(h, "h");
  const Proj pa = proj(a), pb = proj(b);
  const int64_t M = pa.M, d = pa.N;
  TORCH_CHECK(pb.M == M && pb.N == d, "branches of one shape");
  like(h, h, M * d, "h");
  CHECK_RC(omnia_branch_residual(
               h.data_ptr(), f32, outf(x, M * d, "x"), M, d, a.data_ptr(), pa.type, pa.S, pa.ld,
               pa.slab, opt_vecf(abias, d, "abias"), vecf(aw, d, "aw"), b.data_ptr(), pb.type,
               pb.S, pb.ld, pb.slab, opt_vecf(bbias, d, "bbias"), vecf(bw, d, "bw"), (float)inv_n,
               (float)eps, (float)alpha, opt_vecf(nw, d, "nw"), opt_vecf(nb, d, "nb"),
               cur_stream()),
           "branch_residual");
}

// x (+)= parts + scale * table[token] + step; h1 / h2 = rms(x) g w.  Parts: [M, d], slabs
// [S, M, d], or (slots) [M, S, d]; table null: no embedding
void joined_residual(at::Tensor h1, OptT h2, at::Tensor x, bool fresh, OptT m0, bool slots0,
                     OptT m1, bool slots1, OptT m2, bool slots2, OptT ids, OptT table,
                     int64_t vocab, double scale, OptT step, OptT src, OptT tok_slots, OptT w1,
                     double g1, OptT w2, double g2, double inv_n, double eps) {
  const int f32 = is_f32(h1, "h1");
  TORCH_CHECK(x.dim() == 2 && x.size(0) == h1.size(0) && x.size(1) == h1.size(1), "x [M, d]");
  const int64_t M = x.size(0), d = x.size(1);
  like(h1, h1, M * d, "h1");
  const bool two = h2.has_value() && h2->defined();
  if (two) like(*h2, h1, M * d, "h2");
  // kernel slots a, b, c: b takes a part stored in the model's type, expert slots first
  const int own = f32 ? 1 : 0;
  const OptT* ms[3] = {&m0, &m1, &m2};
  const bool sl[3] = {slots0, slots1, slots2};
  ResidParts p[3];
  int n = 0, at_b = -1;
  const void* ptr[3];
  for (int i = 0; i < 3; ++i) {
    if (!ms[i]->has_value() || !(*ms[i])->defined()) continue;
    p[n] = resid_parts(**ms[i], sl[i]);
    TORCH_CHECK(p[n].M == M && p[n].d == d, "part [M, d]");
    ptr[n] = (*ms[i])->data_ptr();
    if (p[n].type == own && (at_b < 0 || sl[i])) at_b = n;
    ++n;
  }
  TORCH_CHECK(n < 3 || at_b >= 0, "one of three parts is stored in the model's type");
  const ResidParts none{own, 0, M, d, 0, 0};
  ResidParts k[3] = {none, none, none};
  const void* kp[3] = {nullptr, nullptr, nullptr};
  for (int i = 0, at = 0; i < n; ++i) {
    const int to = i == at_b ? 1 : at;
    if (i != at_b) at += 2;
    k[to] = p[i];
    kp[to] = ptr[i];
  }
  const void* tp = nullptr;
  const int* idp = nullptr;
  const int64_t* sp = nullptr;
  if (table.has_value() && table->defined() && scale != 0.0) {
    TORCH_CHECK(table->is_cuda() && table->dim() == 2 && table->is_contiguous() &&
                table->scalar_type() == h1.scalar_type() && table->size(0) >= vocab &&
                table->size(1) == d && ids.has_value(), "table [V, d] with ids");
    tp = table->data_ptr();
    idp = veci(*ids, M, "ids");
    if (src.has_value() && src->defined()) {
      TORCH_CHECK(src->is_cuda() && src->scalar_type() == at::kLong && src->is_contiguous() &&
                  src->numel() == M && tok_slots.has_value(), "src int64 [M] with tok_slots");
      CHECK_I32(*tok_slots);
      sp = src->data_ptr<int64_t>();
    }
  }
  CHECK_RC(omnia_joined_residual(
               h1.data_ptr(), two ? h2->data_ptr() : nullptr, f32, outf(x, M * d, "x"), fresh, M,
               d, kp[0], k[0].type, k[0].S, k[0].row, k[0].part, kp[1], k[1].S, k[1].row,
               k[1].part, kp[2], k[2].type, k[2].S, k[2].row, k[2].part, idp, tp, vocab,
               (float)scale, opt_vecf(step, d, "step"), sp, opt_ptr<int>(tok_slots),
               opt_vecf(w1, d, "w1"), (float)g1, opt_vecf(w2, d, "w2"), (float)g2, (float)inv_n,
               (float)eps, cur_stream()),
           "joined_residual");
}

// act(g + bg) * (u + bu): silu, or the tanh form of gelu
void glu(at::Tensor out, at::Tensor m, OptT bias, bool gelu) {
  const int f32 = is_f32(out, "out");
  const Proj p = proj(m);
  TORCH_CHECK(p.N % 2 == 0, "gate | up columns");
  like(out, out, p.M * (p.N / 2), "out");
  CHECK_RC(omnia_glu(out.data_ptr(), f32, m.data_ptr(), p.type, p.S, p.M, p.N / 2,
                     opt_vecf(bias, p.N, "bias"), gelu, cur_stream()), "glu");
}

// ------------------------------------------------------- fixed-decay linear attention
// state fp32 [slots, H, Dp, Vp]; pw [H, pow cols]; x rows [q | k | v | g] (possibly slabs)
struct Lightning { int64_t H, Dp, Vp, cols; };
Lightning lightning_sizes(const at::Tensor& state, const at::Tensor& pw, const Proj& p,
                          int64_t T, const at::Tensor& o) {
  TORCH_CHECK(state.is_cuda() && state.scalar_type() == at::kFloat && state.is_contiguous() &&
              state.dim() == 4, "state fp32 [slots, H, Dp, Vp]");
  const int64_t H = state.size(1), Dp = state.size(2), Vp = state.size(3);
  vecf(pw, H * omnia_lightning_pow_cols(), "pw");
  TORCH_CHECK(p.M == T && p.N >= 2 * H * (Dp + Vp), "projection rows [q | k | v | g]");
  vecf(o, T * H * Vp, "o");
  return {H, Dp, Vp, 2 * H * (Dp + Vp)};
}

void lightning_step(at::Tensor o, at::Tensor state, at::Tensor x, at::Tensor pw,
                    at::Tensor positions, at::Tensor slots) {
  const Proj p = proj(x, true);
  const int64_t T = positions.numel();
  const Lightning l = lightning_sizes(state, pw, p, T, o);
  CHECK_RC(omnia_lightning_step(o.data_ptr<float>(), state.data_ptr<float>(), x.data_ptr(), p.type,
                                p.S, p.ld, p.slab, pw.data_ptr<float>(),
                                veci(positions, T, "positions"), veci(slots, T, "slots"), T, l.H,
                                l.Dp, l.Vp, cur_stream()), "lightning_step");
}

void lightning_scan(at::Tensor o, at::Tensor state, OptT seg, at::Tensor x, at::Tensor pw,
                    at::Tensor q_start, at::Tensor positions, at::Tensor slots) {
  const int f32 = is_f32(x, "x");
  const Proj p = proj(x, true);
  const int64_t T = positions.numel(), nseq = slots.numel();
  TORCH_CHECK(p.S == 1 && x.dim() == 2, "plain projection rows");
  const Lightning l = lightning_sizes(state, pw, p, T, o);
  const int64_t need = omnia_lightning_scratch(T, nseq, l.H, l.Dp, l.Vp);
  CHECK_RC(omnia_lightning_scan(o.data_ptr<float>(), state.data_ptr<float>(),
                                need ? outf(seg.value(), need, "seg") : nullptr, x.data_ptr(), f32,
                                p.ld, pw.data_ptr<float>(), veci(q_start, nseq + 1, "q_start"),
                                nseq, veci(positions, T, "positions"),
                                veci(slots, nseq, "slots"), T, l.H, l.Dp, l.Vp, cur_stream()),
           "lightning_scan");
}

void lightning_norm(at::Tensor y, at::Tensor o, at::Tensor x, int64_t goff, at::Tensor w,
                    double inv_n, double eps) {
  const int f32 = is_f32(y, "y");
  const Proj p = proj(x, true);
  const int64_t n = w.numel();
  TORCH_CHECK(p.N >= goff + n, "gate columns");
  like(y, y, p.M * n, "y");
  CHECK_RC(omnia_lightning_norm(y.data_ptr(), f32, vecf(o, p.M * n, "o"), x.data_ptr(), p.type,
                                p.S, p.ld, p.slab, goff, vecf(w, n, "w"), p.M, n, (float)inv_n,
                                (float)eps, cur_stream()), "lightning_norm");
}

// rows of a step: q_start null = decode (row = sequence), else prefill portions
void delta_prep(at::Tensor qn, at::Tensor kn, at::Tensor vc, at::Tensor decay, at::Tensor beta,
                at::Tensor x, at::Tensor conv_w, at::Tensor conv_state, at::Tensor a_log,
                at::Tensor dt_bias, OptT q_start, at::Tensor positions, at::Tensor slots,
                int64_t KH, int64_t H, int64_t D, int64_t Dp, int64_t V, int64_t taps) {
  const int f32 = is_f32(x, "x");
  const int64_t T = positions.numel(), C = 2 * KH * D + H * V;
  const bool pre = q_start.has_value() && q_start->defined();
  const int64_t nseq = slots.numel();
  TORCH_CHECK(pre || nseq == T, "decode: one slot per row");
  const int64_t ld = rows2(x, T, C + H * V + 2 * H, "x");
  like(conv_w, x, C * taps, "conv_w");
  like(vc, x, T * H * V, "vc");
  TORCH_CHECK(conv_state.is_contiguous() && conv_state.scalar_type() == x.scalar_type() &&
              conv_state.dim() == 3 && conv_state.size(1) == taps - 1 && conv_state.size(2) == C,
              "conv_state [slots, taps-1, C]");
  CHECK_RC(omnia_delta_prep(outf(qn, T * KH * Dp, "qn"), outf(kn, T * KH * Dp, "kn"),
                            vc.data_ptr(), outf(decay, T * H, "decay"), outf(beta, T * H, "beta"),
                            x.data_ptr(), f32, ld, conv_w.data_ptr(), conv_state.data_ptr(),
                            vecf(a_log, H, "a_log"), vecf(dt_bias, H, "dt_bias"),
                            pre ? veci(*q_start, nseq + 1, "q_start") : nullptr, nseq,
                            veci(positions, T, "positions"), veci(slots, nseq, "slots"), T, KH, H,
                            D, Dp, V, taps, cur_stream()), "delta_prep");
}

void check_state(const at::Tensor& state, const at::Tensor& conv_state, const at::Tensor& x,
                 int64_t H, int64_t D, int64_t Vs, int64_t taps, int64_t C) {
  TORCH_CHECK(state.is_cuda() && state.scalar_type() == at::kFloat && state.is_contiguous() &&
              state.dim() == 4 && state.size(1) == H && state.size(2) == D && state.size(3) == Vs,
              "state fp32 [slots, H, D, Vs]");
  TORCH_CHECK(conv_state.is_contiguous() && conv_state.scalar_type() == x.scalar_type() &&
              conv_state.dim() == 3 && conv_state.size(0) == state.size(0) &&
              conv_state.size(1) == taps - 1 && conv_state.size(2) == C,
              "conv_state [slots, taps-1, C]");
}

void delta_step(at::Tensor y, at::Tensor state, at::Tensor conv_state, at::Tensor qn,
                at::Tensor kn, at::Tensor vc, at::Tensor decay, at::Tensor beta, at::Tensor x,
                at::Tensor norm_w, at::Tensor positions, at::Tensor slots, int64_t KH, int64_t H,
                int64_t D, int64_t Dp, int64_t V, int64_t Vp, int64_t taps, double eps) {
  const int f32 = is_f32(x, "x");
  const int64_t T = positions.numel(), C = 2 * KH * D + H * V, Vs = state.size(-1);
  const int64_t ld = rows2(x, T, C + H * V + 2 * H, "x");
  check_state(state, conv_state, x, H, D, Vs, taps, C);
  like(y, x, T * H * Vp, "y");
  like(vc, x, T * H * V, "vc");
  CHECK_RC(omnia_delta_step(y.data_ptr(), state.data_ptr<float>(), conv_state.data_ptr(),
                            vecf(qn, T * KH * Dp, "qn"), vecf(kn, T * KH * Dp, "kn"),
                            vc.data_ptr(), vecf(decay, T * H, "decay"), vecf(beta, T * H, "beta"),
                            x.data_ptr(), f32, ld, vecf(norm_w, V, "norm_w"),
                            veci(positions, T, "positions"), veci(slots, T, "slots"), T, KH, H, D,
                            Dp, V, Vs, Vp, taps, (float)eps, cur_stream()), "delta_step");
}

void delta_scan(at::Tensor o, at::Tensor state, at::Tensor conv_state, at::Tensor rec, at::Tensor qn,
                at::Tensor kn, at::Tensor vc, at::Tensor decay, at::Tensor beta, at::Tensor x,
                at::Tensor q_start, at::Tensor positions, at::Tensor slots, int64_t KH, int64_t H,
                int64_t D, int64_t Dp, int64_t V, int64_t taps) {
  const int f32 = is_f32(x, "x");
  const int64_t T = positions.numel(), C = 2 * KH * D + H * V, Vs = state.size(-1);
  const int64_t ld = rows2(x, T, C + H * V + 2 * H, "x"), nseq = slots.numel();
  check_state(state, conv_state, x, H, D, Vs, taps, C);
  like(vc, x, T * H * V, "vc");
  CHECK_RC(omnia_delta_scan(outf(o, T * H * Vs, "o"), state.data_ptr<float>(),
                            conv_state.data_ptr(),
                            outf(rec, omnia_delta_records(T, nseq, H), "rec"),
                            vecf(qn, T * KH * Dp, "qn"), vecf(kn, T * KH * Dp, "kn"), vc.data_ptr(),
                            vecf(decay, T * H, "decay"), vecf(beta, T * H, "beta"), x.data_ptr(),
                            f32, ld, veci(q_start, nseq + 1, "q_start"), nseq,
                            veci(positions, T, "positions"), veci(slots, nseq, "slots"), T, KH, H,
                            D, Dp, V, Vs, taps, cur_stream()), "delta_scan");
}

void delta_norm(at::Tensor y, at::Tensor o, at::Tensor x, int64_t zoff, at::Tensor norm_w,
                int64_t H, int64_t V, int64_t Vs, int64_t Vp, double eps) {
  const int f32 = is_f32(x, "x");
  const int64_t T = x.size(0), ld = rows2(x, T, zoff + H * V, "x");
  like(y, x, T * H * Vp, "y");
  CHECK_RC(omnia_delta_norm(y.data_ptr(), vecf(o, T * H * Vs, "o"), x.data_ptr(), f32, ld, zoff,
                            vecf(norm_w, V, "norm_w"), T, H, V, Vs, Vp, (float)eps, cur_stream()),
           "delta_norm");
}

// latent pages [NB, page, Lp]
void check_latent(const at::Tensor& cache, const at::Tensor& ref) {
  TORCH_CHECK(cache.is_cuda() && cache.dim() == 3 && cache.is_contiguous() &&
              cache.scalar_type() == ref.scalar_type(), "latent cache [NB, page, Lp]");
}
const int* tables(const at::Tensor& bt, int64_t nseq) {
  TORCH_CHECK(bt.is_cuda() && bt.dim() == 2 && bt.scalar_type() == at::kInt && bt.stride(1) == 1 &&
              bt.size(0) >= nseq, "block_tables int32 [nseq, pages]");
  return bt.data_ptr<int>();
}
const float* rot_table(const at::Tensor& cs, int64_t R) {
  TORCH_CHECK(cs.is_cuda() && cs.scalar_type() == at::kFloat && cs.is_contiguous() &&
              cs.dim() == 2 && cs.size(1) == R, "cos_sin fp32 [positions, R]");
  return cs.data_ptr<float>();
}

void latent_prep(at::Tensor cq, at::Tensor cache, at::Tensor x, at::Tensor wq, at::Tensor wc,
                 at::Tensor positions, at::Tensor slots, at::Tensor cos_sin, int64_t Cp, int64_t R,
                 double eps) {
  const int f32 = is_f32(x, "x");
  check_latent(cache, x);
  const int64_t T = positions.numel(), Q = wq.numel(), C = wc.numel();
  TORCH_CHECK(cq.dim() == 2, "cq [T, Qp]");
  const int64_t Qp = cq.size(1), ld = rows2(x, T, Qp + Cp + R, "x");
  like(cq, x, T * Qp, "cq");
  TORCH_CHECK(slots.is_cuda() && slots.scalar_type() == at::kLong && slots.is_contiguous() &&
              slots.numel() == T, "slots int64 [T]");
  CHECK_RC(omnia_latent_prep(cq.data_ptr(), cache.data_ptr(), x.data_ptr(), f32, ld,
                             vecf(wq, Q, "wq"), vecf(wc, C, "wc"),
                             veci(positions, T, "positions"), slots.data_ptr<int64_t>(),
                             rot_table(cos_sin, R), T, Q, Qp, C, Cp, R, cache.size(2), (float)eps,
                             cur_stream()), "latent_prep");
}

void latent_rotate(at::Tensor q, int64_t hstride, int64_t off, at::Tensor positions,
                   at::Tensor cos_sin, int64_t H, int64_t R) {
  const int f32 = is_f32(q, "q");
  const int64_t T = positions.numel(), ld = rows2(q, T, H * hstride, "q");
  CHECK_RC(omnia_latent_rotate(q.data_ptr(), f32, ld, hstride, off,
                               veci(positions, T, "positions"), rot_table(cos_sin, R), T, H, R,
                               cur_stream()), "latent_rotate");
}

// x [T, H*hx] -> out [T, H*ho]; W [H, N, K]
void latent_heads(at::Tensor out, int64_t ho, at::Tensor x, int64_t hx, at::Tensor W, OptT gate,
                  OptT positions, OptT cos_sin, int64_t R, int64_t Rp, int64_t rotx) {
  const int f32 = is_f32(x, "x");
  TORCH_CHECK(W.dim() == 3, "W [H, N, K]");
  const int64_t T = x.size(0), H = W.size(0), N = W.size(1), K = W.size(2);
  like(W, x, W.numel(), "W");
  const int64_t ldx = rows2(x, T, H * hx, "x"), ldo = rows2(out, T, H * ho, "out");
  TORCH_CHECK(out.scalar_type() == x.scalar_type() && K <= hx && N <= ho, "widths");
  int64_t ldg = 0;
  if (gate.has_value() && gate->defined()) {
    ldg = rows2(*gate, T, H, "gate");
    TORCH_CHECK(gate->scalar_type() == x.scalar_type(), "gate dtype");
  }
  const bool rot = positions.has_value() && positions->defined();
  if (rot) TORCH_CHECK(N + Rp <= ho && R <= Rp && rotx + R <= hx && cos_sin.has_value(), "rotated part");
  CHECK_RC(omnia_latent_heads(out.data_ptr(), f32, ldo, ho, x.data_ptr(), ldx, hx, W.data_ptr(), T,
                              H, N, K, opt_ptr<void>(gate), ldg,
                              rot ? veci(*positions, T, "positions") : nullptr,
                              rot ? rot_table(*cos_sin, R) : nullptr, R, Rp, rotx,
                              rot ? ho - N - Rp : 0, cur_stream()), "latent_heads");
}

void latent_attend(at::Tensor out, at::Tensor q, at::Tensor cache, at::Tensor block_tables,
                   OptT q_start, at::Tensor positions, int64_t H, int64_t Cp, int64_t window,
                   double scale) {
  const int f32 = is_f32(q, "q");
  check_latent(cache, q);
  const int64_t T = positions.numel(), Lp = cache.size(2);
  const bool pre = q_start.has_value() && q_start->defined();
  const int64_t nseq = pre ? q_start->numel() - 1 : T;
  like(q, q, T * H * Lp, "q");
  like(out, q, T * H * Cp, "out");
  CHECK_RC(omnia_latent_attend(out.data_ptr(), f32, q.data_ptr(), cache.data_ptr(),
                               tables(block_tables, nseq), block_tables.stride(0),
                               pre ? veci(*q_start, nseq + 1, "q_start") : nullptr, nseq,
                               veci(positions, T, "positions"), T, cache.size(1), H, Cp, Lp,
                               window, (float)scale, cur_stream()), "latent_attend");
}

void latent_decode(at::Tensor out, OptT part_o, OptT part_ml, at::Tensor q, at::Tensor cache,
                   at::Tensor block_tables, at::Tensor positions, int64_t H, int64_t Cp,
                   int64_t window, double scale, int64_t splits) {
  CHECK_GPU(q); CHECK_BF16(q);
  check_latent(cache, q);
  const int64_t T = positions.numel(), Lp = cache.size(2);
  like(q, q, T * H * Lp, "q");
  like(out, q, T * H * Cp, "out");
  float *po = nullptr, *pm = nullptr;
  if (splits > 1) {
    TORCH_CHECK(part_o.has_value() && part_ml.has_value(), "partials for splits > 1");
    TORCH_CHECK(part_o->scalar_type() == at::kFloat && part_o->numel() >= T * H * splits * Cp &&
                part_ml->scalar_type() == at::kFloat && part_ml->numel() >= T * H * splits * 2,
                "partial sizes");
    po = part_o->data_ptr<float>();
    pm = part_ml->data_ptr<float>();
  }
  CHECK_RC(omnia_latent_decode(out.data_ptr(), po, pm, q.data_ptr(), cache.data_ptr(),
                               tables(block_tables, T), block_tables.stride(0),
                               veci(positions, T, "positions"), T, cache.size(1), H, Cp, Lp,
                               window, (float)scale, splits, cur_stream()), "latent_decode");
}

void latent_gather(at::Tensor c, at::Tensor kr, at::Tensor cache, at::Tensor block_tables,
                   at::Tensor kv_start, at::Tensor kv_first, at::Tensor seq_lens) {
  CHECK_GPU(c); CHECK_BF16(c);
  check_latent(cache, c);
  TORCH_CHECK(c.dim() == 2 && kr.dim() == 2 && c.size(0) == kr.size(0), "c [Tk, Cp], kr [Tk, Rp]");
  like(c, c, c.numel(), "c");
  like(kr, c, kr.numel(), "kr");
  const int64_t nseq = kv_first.numel(), Tk = c.size(0);
  CHECK_RC(omnia_latent_gather(c.data_ptr(), kr.data_ptr(), cache.data_ptr(),
                               tables(block_tables, nseq), block_tables.stride(0),
                               veci(kv_start, nseq + 1, "kv_start"),
                               veci(kv_first, nseq, "kv_first"), veci(seq_lens, nseq, "seq_lens"),
                               nseq, cache.size(1), Tk, c.size(1), kr.size(1), cache.size(2),
                               cur_stream()), "latent_gather");
}

// q / out [T, H, QW | VW], kx [Tk, H*Da], kr [Tk, Rp], vt [H*VW, Tk], gate [T, H] rows
void latent_prefill(at::Tensor out, at::Tensor q, at::Tensor kx, at::Tensor kr, at::Tensor vt,
                    at::Tensor q_start, at::Tensor seq_lens, at::Tensor kv_start,
                    at::Tensor kv_first, at::Tensor tile_seq, at::Tensor tile_q0, int64_t window,
                    double scale, at::Tensor gate) {
  CHECK_GPU(q); CHECK_BF16(q);
  TORCH_CHECK(q.dim() == 3 && out.dim() == 3, "q / out [T, H, w]");
  const int64_t T = q.size(0), H = q.size(1), QW = q.size(2), VW = out.size(2);
  const int64_t Tk = kx.size(0), Da = kx.size(1) / H, Rp = kr.size(1);
  like(q, q, T * H * QW, "q");
  like(out, q, T * H * VW, "out");
  like(kx, q, Tk * H * Da, "kx");
  like(kr, q, Tk * Rp, "kr");
  like(vt, q, H * VW * Tk, "vt");
  CHECK_BF16(gate);
  const int64_t ldg = rows2(gate, T, H, "gate"), nseq = seq_lens.numel(), nt = tile_seq.numel();
  CHECK_RC(omnia_latent_prefill(
               out.data_ptr(), q.data_ptr(), kx.data_ptr(), kr.data_ptr(), vt.data_ptr(),
               veci(q_start, nseq + 1, "q_start"), veci(seq_lens, nseq, "seq_lens"),
               veci(kv_start, nseq + 1, "kv_start"), veci(kv_first, nseq, "kv_first"),
               veci(tile_seq, nt, "tile_seq"), veci(tile_q0, nt, "tile_q0"), nt, H, QW, Da, Rp, VW,
               Tk, window, (float)scale, gate.data_ptr(), ldg, cur_stream()), "latent_prefill");
}

// ------------------------------------------- RMS norms around an fp32 residual stream
void rms_embed(at::Tensor h, at::Tensor x, at::Tensor ids, at::Tensor table, int64_t vocab,
               OptT w_embed, OptT w_pre, double inv_n, double eps, OptT src, OptT tok_slots) {
  const int f32 = is_f32(table, "table");
  TORCH_CHECK(table.dim() == 2 && table.is_contiguous() && table.size(0) >= vocab, "table [V, d]");
  const int64_t T = ids.numel(), d = table.size(1);
  like(h, table, T * d, "h");
  const int64_t* sp = nullptr;
  if (src.has_value() && src->defined()) {
    TORCH_CHECK(src->is_cuda() && src->scalar_type() == at::kLong && src->is_contiguous() &&
                src->numel() == T && tok_slots.has_value(), "src int64 [T] with tok_slots");
    CHECK_I32(*tok_slots);
    sp = src->data_ptr<int64_t>();
  }
  CHECK_RC(omnia_rms_embed(h.data_ptr(), outf(x, T * d, "x"), veci(ids, T, "ids"),
                           table.data_ptr(), f32, T, d, vocab, opt_vecf(w_embed, d, "w_embed"),
                           opt_vecf(w_pre, d, "w_pre"), (float)inv_n, (float)eps, sp,
                           opt_ptr<int>(tok_slots), cur_stream()), "rms_embed");
}

void rms_residual(at::Tensor h, at::Tensor x, at::Tensor m, bool slots, OptT bias,
                  at::Tensor w_post, OptT w_pre, double inv_n, double eps) {
  const int f32 = is_f32(h, "h");
  const ResidParts p = resid_parts(m, slots);
  const int64_t d = p.d;
  like(h, h, p.M * d, "h");
  CHECK_RC(omnia_rms_residual(h.data_ptr(), f32, outf(x, p.M * d, "x"), m.data_ptr(), p.type, p.S,
                              p.row, p.part, p.M, d, opt_vecf(bias, d, "bias"),
                              vecf(w_post, d, "w_post"), opt_vecf(w_pre, d, "w_pre"),
                              (float)inv_n, (float)eps, cur_stream()), "rms_residual");
}

void softcap(at::Tensor z, double cap) {
  const int f32 = is_f32(z, "logits");
  TORCH_CHECK(z.is_contiguous() && cap > 0, "contiguous logits, cap > 0");
  CHECK_RC(omnia_softcap(z.data_ptr(), f32, z.numel(), (float)cap, cur_stream()), "softcap");
}

// ------------------------------------------------------------ grouped-query attention
// k pages [NB, G, page, Dp], v pages [NB, G, page, Vp]
void check_kv(const at::Tensor& k, const at::Tensor& v, const at::Tensor& ref) {
  TORCH_CHECK(k.is_cuda() && k.dim() == 4 && k.is_contiguous() && v.is_cuda() && v.dim() == 4 &&
              v.is_contiguous() && k.scalar_type() == ref.scalar_type() &&
              v.scalar_type() == ref.scalar_type() && k.size(0) == v.size(0) &&
              k.size(1) == v.size(1) && k.size(2) == v.size(2), "k / v pages [NB, G, page, width]");
}

// x: [T, (H*Dp | G*Dp | G*Vp) + padding] or its slabs; k / v pages absent: q only
// wq null: no norms; cos_sin null: no rotation; pairs: neighbours turn together; temp
// [positions] or null; gate [T, H] or null: H more columns behind v
void gqa_prep(at::Tensor q, OptT k, OptT v, at::Tensor x, OptT wq, OptT wk, OptT bias,
              at::Tensor positions, at::Tensor slots, OptT cos_sin, bool pairs, int64_t H,
              int64_t D, int64_t Dp, double eps, OptT temp, OptT gate) {
  const int f32 = is_f32(q, "q");
  const Proj p = proj(x, true);
  const bool rot = cos_sin.has_value() && cos_sin->defined();
  const int64_t T = positions.numel(), R = rot ? cos_sin->size(1) : 0;
  const float* wqp = opt_vecf(wq, Dp, "wq");
  const bool own = k.has_value() && k->defined();
  int64_t G = 0, Vp = 0, page = 1;
  if (own) {
    TORCH_CHECK(v.has_value() && (!wqp || wk.has_value()), "k pages come with v pages and a k norm");
    check_kv(*k, *v, q);
    G = k->size(1);
    page = k->size(2);
    Vp = v->size(3);
    TORCH_CHECK(k->size(3) == Dp, "k page width");
  }
  float* gp = nullptr;
  if (gate.has_value() && gate->defined()) gp = outf(*gate, T * H, "gate");
  TORCH_CHECK(p.M == T && p.N >= H * Dp + G * (Dp + Vp) + (gp ? H : 0), "projection row width");
  like(q, q, T * H * Dp, "q");
  TORCH_CHECK(slots.is_cuda() && slots.scalar_type() == at::kLong && slots.is_contiguous() &&
              slots.numel() == T, "slots int64 [T]");
  CHECK_RC(omnia_gqa_prep(q.data_ptr(), own ? k->data_ptr() : nullptr,
                          own ? v->data_ptr() : nullptr, f32, x.data_ptr(), p.type, p.S,
                          p.slab, p.ld, wqp, own && wqp ? vecf(*wk, Dp, "wk") : nullptr,
                          opt_vecf(bias, H * Dp + G * (Dp + Vp), "bias"),
                          veci(positions, T, "positions"), slots.data_ptr<int64_t>(),
                          rot ? rot_table(*cos_sin, R) : nullptr, pairs, T, H, G, D, Dp, Vp, R,
                          page, (float)eps,
                          temp.has_value() && temp->defined() ?
                              vecf(*temp, temp->numel(), "temp") : nullptr, gp, cur_stream()),
           "gqa_prep");
}

struct KV { int64_t G, page, Dp, Vp; };
KV kv_sizes(const at::Tensor& out, const at::Tensor& q, const at::Tensor& k, const at::Tensor& v,
            int64_t T, int64_t H, const OptT& sinks) {
  check_kv(k, v, q);
  const KV s{k.size(1), k.size(2), k.size(3), v.size(3)};
  TORCH_CHECK(H % s.G == 0, "query heads over key/value heads");
  like(q, q, T * H * s.Dp, "q");
  like(out, q, T * H * s.Vp, "out");
  opt_vecf(sinks, H, "sinks");
  return s;
}

using MaskT = std::tuple<int64_t, int64_t, int64_t>;  // (window, kept first, chunk)
Mask mask_of(const MaskT& m) {
  return {(int)std::get<0>(m), (int)std::get<1>(m), (int)std::get<2>(m)};
}

// dist [2, H]: the heads' distance biases (r1 | r2), or null
Score score_of(double scale, double cap, const OptT& dist, int64_t H) {
  const float* r = opt_vecf(dist, 2 * H, "dist");
  TORCH_CHECK(cap >= 0, "cap");
  return {(float)scale, (float)cap, r, r ? r + H : nullptr};
}

void gqa_attend(at::Tensor out, at::Tensor q, at::Tensor k, at::Tensor v, at::Tensor block_tables,
                OptT q_start, at::Tensor positions, int64_t H, MaskT mask, double scale,
                OptT sinks, double cap, OptT dist, OptT gate) {
  const int f32 = is_f32(q, "q");
  const int64_t T = positions.numel();
  const KV s = kv_sizes(out, q, k, v, T, H, sinks);
  const bool pre = q_start.has_value() && q_start->defined();
  const int64_t nseq = pre ? q_start->numel() - 1 : T;
  CHECK_RC(omnia_gqa_attend(out.data_ptr(), f32, q.data_ptr(), k.data_ptr(), v.data_ptr(),
                            tables(block_tables, nseq), block_tables.stride(0),
                            pre ? veci(*q_start, nseq + 1, "q_start") : nullptr, nseq,
                            veci(positions, T, "positions"), T, s.page, H, s.G, s.Dp, s.Vp,
                            mask_of(mask), score_of(scale, cap, dist, H),
                            opt_ptr<float>(sinks), opt_vecf(gate, T * H, "gate"), cur_stream()),
           "gqa_attend");
}

void gqa_decode(at::Tensor out, OptT part_o, OptT part_ml, at::Tensor q, at::Tensor k,
                at::Tensor v, at::Tensor block_tables, at::Tensor positions, int64_t H,
                MaskT mask, double scale, OptT sinks, int64_t splits, double cap, OptT dist,
                OptT gate) {
  CHECK_GPU(q); CHECK_BF16(q);
  const int64_t T = positions.numel();
  const KV s = kv_sizes(out, q, k, v, T, H, sinks);
  float *po = nullptr, *pm = nullptr;
  if (splits > 1) {
    TORCH_CHECK(part_o.has_value() && part_ml.has_value(), "partials for splits > 1");
    po = outf(*part_o, T * H * splits * s.Vp, "part_o");
    pm = outf(*part_ml, T * H * splits * 2, "part_ml");
  }
  const int64_t ctx = block_tables.size(1) * s.page;  // a row's context fits its table row
  CHECK_RC(omnia_gqa_decode(out.data_ptr(), po, pm, q.data_ptr(), k.data_ptr(), v.data_ptr(),
                            tables(block_tables, T), block_tables.stride(0),
                            veci(positions, T, "positions"), T, s.page, H, s.G, s.Dp, s.Vp,
                            mask_of(mask), score_of(scale, cap, dist, H),
                            opt_ptr<float>(sinks), opt_vecf(gate, T * H, "gate"), splits, ctx,
                            cur_stream()),
           "gqa_decode");
}

void gqa_prefill(at::Tensor out, at::Tensor q, at::Tensor k, at::Tensor v, at::Tensor block_tables,
                 at::Tensor q_start, at::Tensor seq_lens, at::Tensor tile_seq, at::Tensor tile_q0,
                 int64_t H, MaskT mask, double scale, OptT sinks, double cap, OptT dist,
                 OptT gate, bool bounded) {
  CHECK_GPU(q); CHECK_BF16(q);
  TORCH_CHECK(q.dim() == 2, "q [T, H*Dp]");
  const KV s = kv_sizes(out, q, k, v, q.size(0), H, sinks);
  const int64_t nseq = seq_lens.numel(), nt = tile_seq.numel();
  CHECK_RC(omnia_gqa_prefill(out.data_ptr(), q.data_ptr(), k.data_ptr(), v.data_ptr(),
                             tables(block_tables, nseq), block_tables.stride(0),
                             veci(q_start, nseq + 1, "q_start"), veci(seq_lens, nseq, "seq_lens"),
                             veci(tile_seq, nt, "tile_seq"), veci(tile_q0, nt, "tile_q0"), nt,
                             s.page, H, s.G, s.Dp, s.Vp, mask_of(mask),
                             score_of(scale, cap, dist, H), opt_ptr<float>(sinks),
                             opt_vecf(gate, q.size(0) * H, "gate"), bounded, cur_stream()),
           "gqa_prefill");
}

}  // namespace

PYBIND11_MODULE(_omnia_kernels, m) {
  m.doc() = "omnia_amd hand-written CDNA4 (gfx950) HIP kernels";
  m.def("rmsnorm", &rmsnorm);
  m.def("tanh_norm_embed", &tanh_norm_embed);
  m.def("rms_embed", &rms_embed);
  m.def("rms_residual", &rms_residual);
  m.def("softcap", &softcap);
  m.def("gqa_prep", &gqa_prep);
  m.def("gqa_attend", &gqa_attend);
  m.def("gqa_decode", &gqa_decode);
  m.def("gqa_prefill", &gqa_prefill);
  m.def("tanh_norm_residual", &tanh_norm_residual);
  m.def("branch_residual", &branch_residual);
  m.def("joined_residual", &joined_residual);
  m.def("glu", &glu);
  m.def("lightning_step", &lightning_step);
  m.def("lightning_scan", &lightning_scan);
  m.def("lightning_norm", &lightning_norm);
  m.def("lightning_pow_cols", &omnia_lightning_pow_cols);
  m.def("lightning_scratch", &omnia_lightning_scratch);
  m.def("delta_prep", &delta_prep);
  m.def("delta_step", &delta_step);
  m.def("delta_scan", &delta_scan);
  m.def("delta_norm", &delta_norm);
  m.def("latent_prep", &latent_prep);
  m.def("latent_rotate", &latent_rotate);
  m.def("latent_heads", &latent_heads);
  m.def("latent_attend", &latent_attend);
  m.def("latent_decode", &latent_decode);
  m.def("latent_gather", &latent_gather);
  m.def("latent_prefill", &latent_prefill);
  m.def("delta_records", &omnia_delta_records);
  m.def("latent_decode_covers", &omnia_latent_decode_covers);
  m.def("fused_add_rmsnorm", &fused_add_rmsnorm);
  m.def("rope_kv", &rope_kv);
  m.def("silu_mul", &silu_mul);
  m.def("embedding", &embedding, py::arg("out"), py::arg("ids"), py::arg("w"),
        py::arg("vocab_start"), py::arg("src") = py::none(), py::arg("tok_slots") = py::none());
  m.def("decode_attention", &decode_attention);
  m.def("prefill_attention", &prefill_attention, py::arg("out"), py::arg("q"),
        py::arg("k_cache"), py::arg("v_cache"), py::arg("block_tables"), py::arg("q_start_loc"),
        py::arg("seq_lens"), py::arg("tile_seq"), py::arg("tile_q0"), py::arg("scale"),
        py::arg("hp") = 0, py::arg("q_tile") = 64, py::arg("lse") = py::none(),
        py::arg("kv_lens") = py::none());
  m.def("sample", &sample, py::arg("out_tok"), py::arg("out_logprob"), py::arg("logits"),
        py::arg("temperature"), py::arg("top_k"), py::arg("top_p"), py::arg("seeds"),
        py::arg("steps"), py::arg("counts"), py::arg("freq_pen"), py::arg("pres_pen"),
        py::arg("rep_pen"), py::arg("tok_slots") = py::none(), py::arg("dst") = py::none());
  m.def("mean_pool_l2", &mean_pool_l2);
  m.def("cosine_scores", &cosine_scores);
  m.def("topk", &topk);
  m.def("moe_topk", &moe_topk);
  m.def("moe_router_topk", &moe_router_topk);
  m.def("moe_max_blocks", &moe_max_blocks, py::arg("n_assign"), py::arg("n_experts"),
        py::arg("bm") = 64);
  m.def("pgemm_moe", &pgemm_moe, py::arg("mode"), py::arg("out"), py::arg("A"), py::arg("W"),
        py::arg("sorted"), py::arg("blk_expert"), py::arg("n_blocks"), py::arg("route_w"),
        py::arg("topk"), py::arg("n_assign"), py::arg("e_lo"), py::arg("alpha") = 0.0,
        py::arg("limit") = 0.0);
  m.def("moe_route", &moe_route, py::arg("ids"), py::arg("wts"), py::arg("x"), py::arg("router"),
        py::arg("k"), py::arg("sigmoid"), py::arg("renorm"), py::arg("corr") = py::none(),
        py::arg("groups") = 1, py::arg("keep") = 1, py::arg("bias") = py::none());
  m.def("moe_align", &moe_align);
  m.def("moe_gemm", &moe_gemm, py::arg("mode"), py::arg("out"), py::arg("A"), py::arg("W"),
        py::arg("sorted"), py::arg("blk_expert"), py::arg("n_blocks"), py::arg("route_w"),
        py::arg("topk"), py::arg("n_assign"), py::arg("e_lo"), py::arg("alpha") = 0.0,
        py::arg("limit") = 0.0);
  m.def("moe_combine", &moe_combine);
  m.def("dgemm", &dgemm);
  m.def("wgemm", &wgemm);
  m.def("wgemm_wide", &wgemm_wide);
  m.def("tgemm", &tgemm);
  m.def("pgemm", &pgemm);
  m.def("row_sumsq", &row_sumsq);
  m.def("pgemm_variant", &pgemm_variant);
  m.def("pgemm_splitk", &pgemm_splitk);
  m.def("pgemm_set_schedule", [](int64_t sched) {
    TORCH_CHECK(omnia_pgemm_set_schedule((int)sched) == 0, "pgemm schedule must be 0 or 1");
  });
  m.def("ar_twoshot", &ar_twoshot);
  m.def("ar_region_bytes", &omnia_ar_region_bytes);
  m.def("splitk_add_rmsnorm", &splitk_add_rmsnorm);
  m.def("splitk_rope_kv", &splitk_rope_kv);
  m.def("splitk_swiglu", &splitk_swiglu);
  m.def("splitk_reduce", &splitk_reduce);
  m.def("ipc_alloc", &ipc_alloc);
  m.def("ipc_free", &ipc_free);
  m.def("ipc_get_handle", &ipc_get_handle);
  m.def("ipc_open", &ipc_open);
  m.def("ipc_close", &ipc_close);
  m.def("ar_oneshot", &ar_oneshot);
  m.def("ar_allgather", &ar_allgather);
  m.def("ar_alltoall", &ar_alltoall);
  m.def("ar_sendrecv", &ar_sendrecv);
  m.def("ar_blocks", &omnia_ar_blocks);
  m.def("ar_max_ranks", &omnia_ar_max_ranks);
  m.def("apply_token_mask", &apply_token_mask);
  m.def("tp_gumbel", &tp_gumbel);
  m.def("tp_pack", &tp_pack);
  m.def("tp_merge", &tp_merge);
  m.def("graph_launch_step", &graph_launch_step);
  m.def("graph_launch_staged", &graph_launch_staged);
  m.def("stage_copy", &stage_copy);
  m.def("host_device_ptr", &host_device_ptr);
  m.def("event_create", &event_create);
  m.def("event_destroy", &event_destroy);
  m.def("event_query", &event_query);
  m.def("event_sync", &event_sync);
  m.attr("arch") = "gfx950";
}
