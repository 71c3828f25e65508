/* ktx_gla.h — C ABI of the kernels (libktx_hip.so / libktx_seq.so) for decoders whose residual is several parallel streams mixed by
 * learned weights around every sublayer (hyper-connections) and whose layers carry a matrix state per head that decays and takes in
 * outer products: gated linear attention (a decay per key channel, from a low-rank projection), lightning attention (a constant decay per
 * head, silu on queries, keys and values) and the state-space-dual scan of Mamba-2
 * (one decay per head, keys and queries shared by the heads of a group, behind a short causal convolution).  Plus the output stage such
 * mixers share: heads gated and RMS-normed in either order, the results of several mixers laid side by side for one output product.
 *
 * Batching contract: that of ktx_seq.h — the T tokens of all scheduled requests are flattened, request b owns rows
 * q_indptr[b] .. q_indptr[b+1], starts at position pos0[b] and keeps its state in slot slot[b].  The residual streams, norms, decays,
 * steps, gates of a recurrence and its state are fp32 whatever the storage type (KTX_SEQ_BF16 / KTX_SEQ_F32).  DEVICE pointers,
 * enqueue-only on `stream`, 0 = success (ktx_last_error()). */
#ifndef KTX_GLA_H
#define KTX_GLA_H
#include <stddef.h>
#include <stdint.h>

#include "ktx_seq.h"

#ifdef __cplusplus
extern "C" {
#endif

/* ---- hyper-connections ------------------------------------------------------------------------------------------------------------- */
/* One launch between two sublayers, per token t (n streams of W entries):
 *   write (y != NULL):   x'_j = sum_s mix[s][j] x_s + out[j] y        for every stream j, all from the old ones; otherwise x' = x
 *   read  (h != NULL):   u = sum_s in[s] x'_s  (in NULL: the plain sum);  h = (u - mean) / sqrt(var + eps) * norm_w + norm_b
 * x_out (optional, may be x when x is laid out [T][n][W]) receives x'.  With rows (int32 [T], optional): output i is token rows[i]'s, and
 * x_out must be NULL. */
typedef struct ktx_hyper_args {
  const float* x;     /* stream s of token t: x + t * x_tok + s * x_str; x_str == 0: all streams are equal (the model's first layer) */
  int64_t x_tok, x_str;
  const float* y;     /* fp32 rows of stride ldy: the sublayer's result */
  int64_t ldy;
  const float* mix;   /* fp32 [n][n], [from][to] */
  const float* out;   /* fp32 [n] */
  float* x_out;       /* fp32 [T][n][W] */
  const float* in;    /* fp32 [n] */
  const float* norm_w;
  const float* norm_b; /* fp32 [W]; norm_b may be NULL */
  float eps;
  const int32_t* rows;
  void* h;            /* [T][W] of out_dtype */
  int32_t out_dtype;
} ktx_hyper_args;
enum { KTX_HYPER_MAX_STREAMS = 16 };
int ktx_hyper_mix(int T, int W, int n, const ktx_hyper_args* a, ktx_stream_t stream);

/* ---- inputs of the two recurrences ---------------------------------------------------------------------------------------------------- */
/* alpha[t][c] = sigmoid(z)^inv_tau, z = bias[c] + sum_r low[t][r] w[r][c], c < C: fp32 throughout; low fp32 rows of stride ldl, w fp32
 * [R][C] (the low-rank factor TRANSPOSED), bias fp32 [C] or NULL.  alpha fp32 [T][C]. */
int ktx_lowrank_decay(int T, int C, int R, const float* d_low, int64_t ldl, const float* d_w, const float* d_bias, float inv_tau,
                      float* d_alpha, ktx_stream_t stream);

/* u[t][c] = silu(bias[c] + sum_j w[c][j] xin[t - taps + 1 + j][c]) for the C channels at column c_off of proj (fp32 rows of stride ldp;
 * w fp32 [C][taps], the last column multiplies the current token; bias fp32 [C] or NULL); inputs before a request's first new token come
 * from its slot of conv_state fp32 [slots][taps - 1][C] when pos0 > 0 and are zero otherwise; the slot's state moves on (with
 * max_q_len == 1 inside the launch, otherwise in a second one).  With H > 0: dt = softplus(proj[t][dt_off + h] + dt_bias[h]),
 * gates[t][h] = dt, gates[t][H + h] = exp(-exp(A_log[h]) dt).  u fp32 [T][C], gates fp32 [T][2H]; 1 <= taps <= 16. */
int ktx_ssd_prep(int B, int T, int max_q_len, int C, int taps, int H, const float* d_proj, int64_t ldp, int c_off, int dt_off,
                 const float* d_w, const float* d_bias, const float* d_dt_bias, const float* d_A_log, const int32_t* d_q_indptr,
                 const int32_t* d_pos0, const int32_t* d_slot, const int32_t* d_tok_req, float* d_conv_state, float* d_u, float* d_gates,
                 ktx_stream_t stream);

/* ---- the decayed outer-product scan --------------------------------------------------------------------------------------------------- */
/* Per head h (key / query head g = h / heads_per_key), token by token from the slot's state S fp32 [slots][heads][dim][vdim] (zero when
 * pos0 == 0, whatever the slot holds):
 *   S <- diag(a_t) S + k_t (m_t v_t)^T;   o[t][h] = q_scale S^T q_t + skip[h] v_t
 * a: per key channel, a[t * lda + h * dim + d], or (a_per_head) one number a[t * lda + h]; m = vmul[t * ldm + h] (NULL: 1); skip fp32
 * [heads] or NULL.  q, k, v: fp32 rows with strides ldq, ldk, ldv, head g's dim entries at g * dim, head h's vdim entries at h * vdim.
 * 0 <= a <= 1 is assumed.  o fp32 [T][heads * vdim].  Steps of a few tokens, and dim > 128, run token by token on the vector ALUs; prompts
 * with dim <= 128 run 16 tokens at a time on the fp32 matrix cores.  dim <= 512.
 * Requests longer than chunk_len tokens are cut into chunks that run side by side: every chunk's own state from zero, a pass over the
 * chunks' states, then every chunk from the state it starts with.  Scratch for that (needed when max_q_len > chunk_len):
 * ktx_decay_scan_scratch() floats; n = ceil(max_q_len / chunk_len) chunks per request are launched.  A decay
 * that never changes is one row with stride lda = 0. */
typedef struct ktx_decay_scan_args {
  int32_t heads, dim, vdim, heads_per_key;
  const float *q, *k, *v, *a, *vmul, *skip;
  int64_t ldq, ldk, ldv, lda, ldm;
  int32_t a_per_head;
  float q_scale;
  int32_t qkv_act;    /* != 0: q, k and v are silu of what q, k, v hold */
  float* S;
  float* o;
  float* scratch;
  int32_t chunk_len;
} ktx_decay_scan_args;
size_t ktx_decay_scan_scratch(const ktx_decay_scan_args* a, int B, int max_q_len);
int ktx_decay_scan(int B, int T, int max_q_len, const int32_t* d_q_indptr, const int32_t* d_pos0, const int32_t* d_slot,
                   const ktx_decay_scan_args* a, ktx_stream_t stream);

/* ---- gate / norm segments side by side ------------------------------------------------------------------------------------------------ */
/* out[t][out_off + c] = scale * f(o[t][c], gate[t][c]), c < n, for up to KTX_GATE_SEGS segments in one launch; per segment
 *   group == 0:                 f = o act(gate)
 *   gate_first == 0:            f = o r w act(gate), r = 1 / sqrt(mean(o^2 over the group of c) + eps)
 *   gate_first != 0:            f = p r w,           p = o act(gate), r = 1 / sqrt(mean(p^2 over the group of c) + eps)
 * groups of `group` consecutive columns (dividing n); w fp32, entry c % w_mod (w_mod = group: shared by the groups; n: one each).
 * act: 0 sigmoid, 1 silu.  o: rows of stride ldo of o_dtype; gate fp32 rows of stride ldg.  out: rows of stride ldout of out_dtype. */
enum { KTX_GATE_SEGS = 2 };
typedef struct ktx_gate_seg {
  const void* o;
  int64_t ldo;
  int32_t o_dtype;
  const float* gate;
  int64_t ldg;
  const float* w;
  int32_t n, group, w_mod, act, gate_first;
  float eps, scale;
  int32_t out_off;
} ktx_gate_seg;
int ktx_gate_segments(int T, int n_segs, const ktx_gate_seg* segs, void* d_out, int out_dtype, int64_t ldout, ktx_stream_t stream);

#ifdef __cplusplus
}
#endif
#endif
