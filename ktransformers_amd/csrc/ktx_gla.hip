// ktx_gla.hip — kernels behind include/ktx_gla.h: the hyper-connection step (residual streams mixed around a sublayer, read and layer-
// normed for the next one in the same launch), the low-rank decay of gated linear attention, the convolved inputs, steps and decays of
// the state-space-dual scan, the decayed outer-product scan the recurrences share (chunks of a prompt run side by side; silu on the way in for lightning attention), and the gate /
// norm segments in front of an output product.
//
// Streams, norms, decays, steps and the state are fp32; element types only select how activations are stored.
#include "ktx_common.h"
#include "../../include/ktx_gla.h"

#include <math.h>

#include <algorithm>

namespace {

#include "ktx_seq_dev.inc"
#include "ktx_conv_dev.inc"

__device__ __forceinline__ float silu_f32(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f32(float z) { return z > 20.f ? z : log1pf(expf(z)); }

bool aligned16(const void* p) { return ((uintptr_t)p & 15u) == 0; }
int dtype_ok(int d) { return d == KTX_SEQ_F32 || d == KTX_SEQ_BF16; }

// ---------------------------------------------------------------------------------------------------------------------
// hyper-connections.  One token per workgroup; a thread owns 4 neighbouring entries per EV of ALL streams in registers, every load of the
// token (streams, the sublayer's row, then the norm's weights) is requested before the first is used.
__device__ __forceinline__ float4 f4_fma(float s, const float4& v, const float4& c) {
  return make_float4(fmaf(s, v.x, c.x), fmaf(s, v.y, c.y), fmaf(s, v.z, c.z), fmaf(s, v.w, c.w));
}
__device__ __forceinline__ void st4(float* p, const float4& v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void st4(bf16_t* p, const float4& v) { *reinterpret_cast<uint2*>(p) = make_uint2(ktx_pk_bf16(v.x, v.y), ktx_pk_bf16(v.z, v.w)); }

template <typename OT, int NS, int EV>
__global__ void __launch_bounds__(256) hyper_vec_kernel(int W, ktx_hyper_args a) {
  __shared__ float red[4];
  const int tid = threadIdx.x;
  const int t = a.rows ? a.rows[blockIdx.x] : blockIdx.x;
  const float* x = a.x + (size_t)t * a.x_tok;
  const float4 zero4 = make_float4(0.f, 0.f, 0.f, 0.f);
  float4 xs[EV][NS], u[EV];
#pragma unroll
  for (int v = 0; v < EV; v++) {
    const int e = (v * 256 + tid) * 4;
#pragma unroll
    for (int s = 0; s < NS; s++) xs[v][s] = e < W ? *reinterpret_cast<const float4*>(x + s * a.x_str + e) : zero4;
    u[v] = a.y && e < W ? *reinterpret_cast<const float4*>(a.y + (size_t)t * a.ldy + e) : zero4;
  }
  if (a.y) {
    float m[NS][NS], o[NS];
#pragma unroll
    for (int j = 0; j < NS; j++) {
      o[j] = a.out[j];
#pragma unroll
      for (int s = 0; s < NS; s++) m[s][j] = a.mix[s * NS + j];
    }
#pragma unroll
    for (int v = 0; v < EV; v++) {
      float4 nx[NS];
#pragma unroll
      for (int j = 0; j < NS; j++) {
        nx[j] = make_float4(o[j] * u[v].x, o[j] * u[v].y, o[j] * u[v].z, o[j] * u[v].w);
#pragma unroll
        for (int s = 0; s < NS; s++) nx[j] = f4_fma(m[s][j], xs[v][s], nx[j]);
      }
#pragma unroll
      for (int j = 0; j < NS; j++) xs[v][j] = nx[j];
    }
  }
  // the norm's weights are on their way while the streams are written and the row is reduced
  float4 w[EV], b[EV];
  if (a.h) {
#pragma unroll
    for (int v = 0; v < EV; v++) {
      const int e = (v * 256 + tid) * 4;
      w[v] = e < W ? *reinterpret_cast<const float4*>(a.norm_w + e) : zero4;
      b[v] = a.norm_b && e < W ? *reinterpret_cast<const float4*>(a.norm_b + e) : zero4;
    }
  }
  if (a.x_out) {
#pragma unroll
    for (int v = 0; v < EV; v++) {
      const int e = (v * 256 + tid) * 4;
      if (e < W) {
#pragma unroll
        for (int j = 0; j < NS; j++) st4(a.x_out + ((size_t)t * NS + j) * W + e, xs[v][j]);
      }
    }
  }
  if (!a.h) return;
  float sum = 0.f;
#pragma unroll
  for (int v = 0; v < EV; v++) {
    u[v] = zero4;
#pragma unroll
    for (int s = 0; s < NS; s++) u[v] = f4_fma(a.in ? a.in[s] : 1.0f, xs[v][s], u[v]);
    sum += (u[v].x + u[v].y) + (u[v].z + u[v].w);                 // (entries beyond W are 0)
  }
  const float mean = block_sum256(sum, red) / (float)W;
  float q = 0.f;
#pragma unroll
  for (int v = 0; v < EV; v++) {
    if ((v * 256 + tid) * 4 < W) {
      u[v] = make_float4(u[v].x - mean, u[v].y - mean, u[v].z - mean, u[v].w - mean);
      q += (u[v].x * u[v].x + u[v].y * u[v].y) + (u[v].z * u[v].z + u[v].w * u[v].w);
    }
  }
  const float r = 1.0f / sqrtf(block_sum256(q, red) / (float)W + a.eps);
  OT* h = reinterpret_cast<OT*>(a.h) + (size_t)blockIdx.x * W;
#pragma unroll
  for (int v = 0; v < EV; v++) {
    const int e = (v * 256 + tid) * 4;
    if (e < W) st4(h + e, make_float4(u[v].x * r * w[v].x + b[v].x, u[v].y * r * w[v].y + b[v].y, u[v].z * r * w[v].z + b[v].z, u[v].w * r * w[v].w + b[v].w));
  }
}

// any width and up to KTX_HYPER_MAX_STREAMS streams: entry by entry, the read row in LDS between the passes
template <typename OT>
__global__ void __launch_bounds__(256) hyper_any_kernel(int W, int n, ktx_hyper_args a) {
  extern __shared__ float row[];
  __shared__ float red[4];
  const int tid = threadIdx.x;
  const int t = a.rows ? a.rows[blockIdx.x] : blockIdx.x;
  const float* x = a.x + (size_t)t * a.x_tok;
  float sum = 0.f;
  for (int e = tid; e < W; e += 256) {
    float xs[KTX_HYPER_MAX_STREAMS], nx[KTX_HYPER_MAX_STREAMS];
#pragma unroll
    for (int s = 0; s < KTX_HYPER_MAX_STREAMS; s++) xs[s] = s < n ? x[s * a.x_str + e] : 0.f;
    const float y = a.y ? a.y[(size_t)t * a.ldy + e] : 0.f;
    float u = 0.f;
#pragma unroll
    for (int j = 0; j < KTX_HYPER_MAX_STREAMS; j++) {
      if (j < n) {
        nx[j] = xs[j];
        if (a.y) {
          float v = a.out[j] * y;
#pragma unroll
          for (int s = 0; s < KTX_HYPER_MAX_STREAMS; s++)
            if (s < n) v = fmaf(a.mix[s * n + j], xs[s], v);
          nx[j] = v;
        }
        u = fmaf(a.in ? a.in[j] : 1.0f, nx[j], u);
      }
    }
    if (a.x_out) {
#pragma unroll
      for (int j = 0; j < KTX_HYPER_MAX_STREAMS; j++)
        if (j < n) a.x_out[((size_t)t * n + j) * W + e] = nx[j];
    }
    row[e] = u;
    sum += u;
  }
  if (!a.h) return;
  const float mean = block_sum256(sum, red) / (float)W;
  float q = 0.f;
  for (int e = tid; e < W; e += 256) {      // (each thread re-reads only what it wrote)
    const float d = row[e] - mean;
    q += d * d;
  }
  const float r = 1.0f / sqrtf(block_sum256(q, red) / (float)W + a.eps);
  OT* h = reinterpret_cast<OT*>(a.h) + (size_t)blockIdx.x * W;
  for (int e = tid; e < W; e += 256) st_elem(h, e, (row[e] - mean) * r * a.norm_w[e] + (a.norm_b ? a.norm_b[e] : 0.f));
}

// ---------------------------------------------------------------------------------------------------------------------
// the decay of gated linear attention: thread = channel, LD_TT tokens per workgroup share a read of the transposed factor
constexpr int LD_TT = 8;
__global__ void __launch_bounds__(256) lowrank_decay_kernel(int T, int C, int R, const float* __restrict__ low, int64_t ldl,
                                                            const float* __restrict__ w, const float* __restrict__ bias, float inv_tau,
                                                            float* __restrict__ alpha) {
  extern __shared__ float lt[];            // [LD_TT][R]
  const int t0 = blockIdx.x * LD_TT, c = blockIdx.y * 256 + threadIdx.x, nt = min(LD_TT, T - t0);
  for (int e = threadIdx.x; e < LD_TT * R; e += 256) {
    const int tt = e / R;
    lt[e] = tt < nt ? low[(size_t)(t0 + tt) * ldl + e % R] : 0.f;
  }
  __syncthreads();
  if (c >= C) return;
  float z[LD_TT];
  const float b = bias ? bias[c] : 0.f;
#pragma unroll
  for (int i = 0; i < LD_TT; i++) z[i] = b;
#pragma unroll 8
  for (int r = 0; r < R; r++) {
    const float wv = w[(size_t)r * C + c];
#pragma unroll
    for (int i = 0; i < LD_TT; i++) z[i] = fmaf(lt[i * R + r], wv, z[i]);
  }
#pragma unroll
  for (int i = 0; i < LD_TT; i++)
    if (i < nt) alpha[(size_t)(t0 + i) * C + c] = expf(log_sigmoid_f32(z[i]) * inv_tau);
}

// ---------------------------------------------------------------------------------------------------------------------
// the state-space-dual scan's inputs: short convolution + silu, steps, decays.  blockIdx = (token, 1024 channels)
constexpr int SP_MAX_TAPS = 16;
__device__ __forceinline__ void ssd_gates(int t, int H, const float* __restrict__ proj, int64_t ldp, int dt_off, const float* __restrict__ dt_bias,
                                          const float* __restrict__ A_log, float* __restrict__ gates) {
  for (int h = threadIdx.x; h < H; h += 256) {
    const float dt = softplus_f32(proj[(size_t)t * ldp + dt_off + h] + dt_bias[h]);
    gates[(size_t)t * 2 * H + h] = dt;
    gates[(size_t)t * 2 * H + H + h] = expf(-expf(A_log[h]) * dt);
  }
}

// 1 .. 4 taps, everything 16-byte aligned: a thread owns four neighbouring channels; `one_token` (no request brings more than one): the
// slot's state moves on here — the token's workgroups are the only readers of its slot, a thread touches only its own channels
template <int TAPS>
__global__ void __launch_bounds__(256) ssd_prep_vec_kernel(int C, int H, const float* __restrict__ proj, int64_t ldp, int c_off, int dt_off,
                                                           const float* __restrict__ cw, const float* __restrict__ bias,
                                                           const float* __restrict__ dt_bias, const float* __restrict__ A_log,
                                                           const int32_t* __restrict__ q_indptr, const int32_t* __restrict__ pos0,
                                                           const int32_t* __restrict__ slot, const int32_t* __restrict__ tok_req,
                                                           float* __restrict__ conv_state, int one_token, float* __restrict__ uo,
                                                           float* __restrict__ gates) {
  const int t = blockIdx.x, e = (blockIdx.y * 256 + threadIdx.x) * 4;
  const float4 zero4 = make_float4(0.f, 0.f, 0.f, 0.f);
  if (e < C) {
    float4 u[TAPS], w[4];
    float4 y = bias ? *reinterpret_cast<const float4*>(bias + e) : zero4;
    float* st = nullptr;
    if constexpr (TAPS > 1) {
      const int b = tok_req[t], i = t - q_indptr[b];
      const bool carried = pos0[b] > 0;
      st = conv_state + (size_t)slot[b] * (TAPS - 1) * C;
#pragma unroll
      for (int j = 0; j < TAPS; j++) {
        const int ii = i - (TAPS - 1) + j;
        if (ii >= 0) u[j] = *reinterpret_cast<const float4*>(proj + (size_t)(t - (TAPS - 1) + j) * ldp + c_off + e);
        else if (carried) u[j] = *reinterpret_cast<const float4*>(st + (size_t)(TAPS - 1 + ii) * C + e);
        else u[j] = zero4;
      }
    } else {
      u[0] = *reinterpret_cast<const float4*>(proj + (size_t)t * ldp + c_off + e);
    }
#pragma unroll
    for (int n = 0; n < 4; n++) {      // the taps of channel e + n: TAPS consecutive floats
      if constexpr (TAPS == 4) {
        w[n] = *reinterpret_cast<const float4*>(cw + (size_t)(e + n) * 4);
      } else {
        const float* wp = cw + (size_t)(e + n) * TAPS;
        w[n] = make_float4(wp[0], TAPS > 1 ? wp[1] : 0.f, TAPS > 2 ? wp[2] : 0.f, 0.f);
      }
    }
    auto tap = [](const float4& v, int j) { return j == 0 ? v.x : j == 1 ? v.y : j == 2 ? v.z : v.w; };
#pragma unroll
    for (int j = 0; j < TAPS; j++) {
      y.x = fmaf(tap(w[0], j), u[j].x, y.x);
      y.y = fmaf(tap(w[1], j), u[j].y, y.y);
      y.z = fmaf(tap(w[2], j), u[j].z, y.z);
      y.w = fmaf(tap(w[3], j), u[j].w, y.w);
    }
    *reinterpret_cast<float4*>(uo + (size_t)t * C + e) = make_float4(silu_f32(y.x), silu_f32(y.y), silu_f32(y.z), silu_f32(y.w));
    if constexpr (TAPS > 1) {
      if (one_token) {
#pragma unroll
        for (int j = 0; j < TAPS - 1; j++) *reinterpret_cast<float4*>(st + (size_t)j * C + e) = u[j + 1];
      }
    }
  }
  if (blockIdx.y == 0) ssd_gates(t, H, proj, ldp, dt_off, dt_bias, A_log, gates);
}

__global__ void __launch_bounds__(256) ssd_prep_kernel(int C, int taps, int H, const float* __restrict__ proj, int64_t ldp, int c_off,
                                                       int dt_off, const float* __restrict__ cw, const float* __restrict__ bias,
                                                       const float* __restrict__ dt_bias, const float* __restrict__ A_log,
                                                       const int32_t* __restrict__ q_indptr, const int32_t* __restrict__ pos0,
                                                       const int32_t* __restrict__ slot, const int32_t* __restrict__ tok_req,
                                                       const float* __restrict__ conv_state, float* __restrict__ uo, float* __restrict__ gates) {
  const int t = blockIdx.x, b = tok_req[t], i = t - q_indptr[b];
  const bool carried = pos0[b] > 0;
  const float* st = taps > 1 ? conv_state + (size_t)slot[b] * (taps - 1) * C : nullptr;
  for (int e = blockIdx.y * 1024 + threadIdx.x; e < min(C, (int)(blockIdx.y + 1) * 1024); e += 256) {
    float y = bias ? bias[e] : 0.f;
    for (int j = 0; j < taps; j++) {
      const int ii = i - (taps - 1) + j;
      float u = 0.f;
      if (ii >= 0) u = proj[(size_t)(t - (taps - 1) + j) * ldp + c_off + e];
      else if (carried) u = st[(size_t)(taps - 1 + ii) * C + e];
      y = fmaf(cw[(size_t)e * taps + j], u, y);
    }
    uo[(size_t)t * C + e] = silu_f32(y);
  }
  if (blockIdx.y == 0) ssd_gates(t, H, proj, ldp, dt_off, dt_bias, A_log, gates);
}

// ---------------------------------------------------------------------------------------------------------------------
// the decayed outer-product scan.  Workgroup = (request, chunk of its tokens) x head x 64 value columns; lane = value column, wavefront =
// R rows of the state, held in registers.  k, q and a are the same for all lanes of a wavefront: they come through the scalar cache as
// operands of the vector instructions, and so do the per-head numbers; a group of SC_TG tokens' values is requested a group ahead.  The
// wavefronts' partial read-outs of a group meet in LDS behind ONE barrier.
constexpr int SC_TG = 8;
struct ScanDims {
  int heads, dim, vdim, hpk, L, nch;
  int64_t ldq, ldk, ldv, lda, ldm;
  float q_scale;
  int act;                                 // != 0: q, k and v pass silu on their way in
};
__device__ __forceinline__ float silu_fast(float z) { return z * sigmoid_fast(z); }

template <int R, bool PH, bool OUT, bool FULL>
__device__ __forceinline__ void scan_token(const ScanDims& c, float (&S)[R], int live, const float* __restrict__ kr, const float* __restrict__ qr,
                                           const float* __restrict__ ar, float vv, float& acc0, float& acc1) {
  const float ah = PH ? ar[0] : 0.f;
#pragma unroll
  for (int i = 0; i < R; i++) {
    const bool ok = FULL || i < live;
    const float kk = ok ? kr[i] : 0.f;
    const float aa = PH ? ah : (ok ? ar[i] : 0.f);
    S[i] = fmaf(kk, vv, aa * S[i]);
    if constexpr (OUT) {
      const float qq = ok ? qr[i] : 0.f;
      if (i & 1) acc1 = fmaf(S[i], qq, acc1);
      else acc0 = fmaf(S[i], qq, acc0);
    }
  }
}

// the same with silu on keys and queries: lanes 0 .. R - 1 take the keys, lanes R .. 2 R - 1 the queries of the wavefront's rows, one activation
// per lane, and hand them out
template <int R, bool PH, bool OUT, bool FULL>
__device__ __forceinline__ void scan_token_act(const ScanDims& c, float (&S)[R], int live, int lane, const float* __restrict__ kr,
                                               const float* __restrict__ qr, const float* __restrict__ ar, float vv, float& acc0, float& acc1) {
  const int i0 = lane & (R - 1);           // (R is a power of two up to 32)
  const bool isq = OUT && (lane & R);
  const float z = FULL || i0 < live ? (isq ? qr[i0] : kr[i0]) : 0.f;
  const int s = __builtin_bit_cast(int, silu_fast(z));
  const float ah = PH ? ar[0] : 0.f;
#pragma unroll
  for (int i = 0; i < R; i++) {
    const bool ok = FULL || i < live;
    const float kk = __builtin_bit_cast(float, __builtin_amdgcn_readlane(s, i));
    const float aa = PH ? ah : (ok ? ar[i] : 0.f);
    S[i] = fmaf(kk, vv, aa * S[i]);
    if constexpr (OUT) {
      const float qq = __builtin_bit_cast(float, __builtin_amdgcn_readlane(s, R + i));
      if (i & 1) acc1 = fmaf(S[i], qq, acc1);
      else acc0 = fmaf(S[i], qq, acc0);
    }
  }
}

template <int R, bool PH, bool OUT, bool FULL>
__global__ void __launch_bounds__(1024) decay_scan_kernel(ScanDims c, const int32_t* __restrict__ q_indptr, const int32_t* __restrict__ pos0,
                                                          const int32_t* __restrict__ slot, const float* __restrict__ q,
                                                          const float* __restrict__ k, const float* __restrict__ v, const float* __restrict__ a,
                                                          const float* __restrict__ vmul, const float* __restrict__ skip, float* Sg,
                                                          float* delta, float* __restrict__ o) {
  extern __shared__ float red[];           // [2][wavefronts][SC_TG][64]
  const int b = blockIdx.x / c.nch, ch = blockIdx.x % c.nch, h = blockIdx.y, lane = threadIdx.x & 63;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), NW = blockDim.x >> 6;
  const int q1 = q_indptr[b + 1], t0 = q_indptr[b] + ch * c.L, t1 = min(q1, t0 + c.L);
  if (t0 >= t1 || (!OUT && t1 == q1)) return;      // (the last chunk's own state is nobody's start)
  const int D = c.dim, V = c.vdim, col = blockIdx.z * 64 + lane, d0 = wave * R, live = D - d0;
  const bool vok = col < V;
  const size_t chunk_row = (size_t)blockIdx.x * c.heads + h;
  float* dl = delta ? delta + chunk_row * D * V : nullptr;                            // this chunk's state rows in the scratch
  float* Sp = Sg + ((size_t)slot[b] * c.heads + h) * D * V;
  float S[R];
  const float* init = OUT ? (dl ? dl : (pos0[b] > 0 ? Sp : nullptr)) : nullptr;
#pragma unroll
  for (int i = 0; i < R; i++) S[i] = init && vok && (FULL || i < live) ? init[(size_t)(d0 + i) * V + col] : 0.f;
  const float* kb = k + (h / c.hpk) * D + d0;
  const float* qb = OUT ? q + (h / c.hpk) * D + d0 : nullptr;
  const float* ab = PH ? a + h : a + h * D + d0;
  const float* vb = v + h * V + (vok ? col : 0);
  const float sk = OUT && skip && wave == 0 ? skip[h] : 0.f;
  float nv[SC_TG];
#pragma unroll
  for (int i = 0; i < SC_TG; i++) nv[i] = vok && t0 + i < t1 ? vb[(size_t)(t0 + i) * c.ldv] : 0.f;
  int buf = 0;
  for (int tb = t0; tb < t1; tb += SC_TG, buf ^= 1) {
    const int nt = min(SC_TG, t1 - tb);
    float cv[SC_TG], po[SC_TG];
#pragma unroll
    for (int i = 0; i < SC_TG; i++) {
      cv[i] = nv[i];
      nv[i] = vok && tb + SC_TG + i < t1 ? vb[(size_t)(tb + SC_TG + i) * c.ldv] : 0.f;
      po[i] = 0.f;
    }
#pragma unroll
    for (int i = 0; i < SC_TG; i++) {
      if (i < nt) {                        // (uniform over the workgroup)
        const size_t t = tb + i;
        const float m = vmul ? vmul[t * c.ldm + h] : 1.0f;
        float a0 = 0.f, a1 = 0.f;
        if (c.act) {
          cv[i] = silu_fast(cv[i]);
          scan_token_act<R, PH, OUT, FULL>(c, S, live, lane, kb + t * c.ldk, OUT ? qb + t * c.ldq : nullptr, ab + t * c.lda, cv[i] * m, a0, a1);
        } else {
          scan_token<R, PH, OUT, FULL>(c, S, live, kb + t * c.ldk, OUT ? qb + t * c.ldq : nullptr, ab + t * c.lda, cv[i] * m, a0, a1);
        }
        if constexpr (OUT) po[i] = fmaf(a0 + a1, c.q_scale, sk * cv[i]);
      }
    }
    if constexpr (OUT) {
      if (NW == 1) {
#pragma unroll
        for (int i = 0; i < SC_TG; i++)
          if (i < nt && vok) o[((size_t)(tb + i) * c.heads + h) * V + col] = po[i];
      } else {
        float* rb = red + (size_t)buf * NW * SC_TG * 64;
#pragma unroll
        for (int i = 0; i < SC_TG; i++) rb[(wave * SC_TG + i) * 64 + lane] = po[i];
        __syncthreads();                   // (the other half is rewritten only behind the next group's barrier)
        for (int i = wave; i < nt; i += NW) {
          float s = 0.f;
          for (int w = 0; w < NW; w++) s += rb[(w * SC_TG + i) * 64 + lane];
          if (vok) o[((size_t)(tb + i) * c.heads + h) * V + col] = s;
        }
      }
    }
  }
  if (OUT && t1 != q1) return;
  float* dst = OUT ? Sp : dl;
#pragma unroll
  for (int i = 0; i < R; i++)
    if (vok && (FULL || i < live)) dst[(size_t)(d0 + i) * V + col] = S[i];
}

// The same scan for prompts on the fp32 matrix cores, SM_T tokens at a time.  Workgroup = (request, chunk) x head x NT / 64 tiles of 16 value
// columns; a wavefront keeps its columns of the state, all key rows, as the accumulators of v_mfma_f32_16x16x4_f32.  With p_t the product
// of the decays of the block's tokens up to t and s_t that of the tokens behind t — products of factors that are at most 1: nothing is divided
// by a decay and nothing overflows —
//   o_t = (q_t p_t)^T S + sum_{i <= t} A[t][i] v_i,   A[t][i] = m_i sum_d q_td k_id prod_{i < j <= t} a_jd  (+ skip where i = t)
//   S  <- diag(p_last) S + sum_t (k_t s_t m_t) v_t^T
// With one decay per head A is a matrix product (key rows dealt out to the wavefronts) times the products of decays; with a decay per key
// channel it is formed on the vector ALUs, thread = (token i, a slice of the channels) that walks t with k_i's running product.  An accumulator
// holds rows 4 g + r of a tile in lane group g, register r: with the contraction visiting rows in the order (r, g) it is the next product's
// operand as it stands.
constexpr int SM_T = 16, SM_AST = 20, SCAN_MFMA_MIN = 8;
typedef float f32x4 __attribute__((ext_vector_type(4)));

// v[j] and v[j + N] meet across the lane pairs CTRL joins: a lane keeps the one its bit names
template <int N, int CTRL>
__device__ __forceinline__ void fold_pairs(float (&v)[SM_T], bool upper) {
#pragma unroll
  for (int j = 0; j < N; j++) {
    const float give = upper ? v[j] : v[j + N], keep = upper ? v[j + N] : v[j];
    v[j] = keep + ktx_dpp_f<CTRL>(give);
  }
}

template <int DT, int NT, bool PH>
struct ScanTile {
  static constexpr int DW = DT * 16, DP = DW + 4;              // row stride: lane groups four rows apart meet different LDS banks
  static constexpr int RAW_A = PH ? SM_T : SM_T * DP;
  static constexpr int PARTS = !PH ? 1 : DT < NT / 64 ? DT : NT / 64;      // partial products of A
  // raw q | k | a | m, then q p | k s m | p_last | A (its parts), and with one decay per head the products of decays
  static constexpr int QR = 0, KR = SM_T * DP, AR = 2 * SM_T * DP, MR = AR + RAW_A, QP = MR + SM_T, KP = QP + SM_T * DP, PL = KP + SM_T * DP,
                       AS = PL + DP, RT = AS + PARTS * SM_T * SM_AST, FLOATS = RT + (PH ? SM_T * SM_AST : 0);
};

template <int DT, int NT, bool PH, bool OUT>
__global__ void __launch_bounds__(NT, DT == 8 && NT == 256 && !PH && OUT ? 3 : 4) decay_scan_mfma_kernel(ScanDims c, const int32_t* __restrict__ q_indptr, const int32_t* __restrict__ pos0,
                                                             const int32_t* __restrict__ slot, const float* __restrict__ q,
                                                             const float* __restrict__ k, const float* __restrict__ v, const float* __restrict__ a,
                                                             const float* __restrict__ vmul, const float* __restrict__ skip, float* Sg,
                                                             float* delta, float* __restrict__ o) {
  typedef ScanTile<DT, NT, PH> L;
  constexpr int DW = L::DW, DP = L::DP, E = SM_T * DW / NT, SL = NT / SM_T, CPS = DW / SL, VW = CPS >= 4 ? 4 : CPS;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, g = lane >> 4;
  const int b = blockIdx.x / c.nch, ch = blockIdx.x % c.nch, h = blockIdx.y;
  const int q1 = q_indptr[b + 1], t0 = q_indptr[b] + ch * c.L, t1 = min(q1, t0 + c.L);
  if (t0 >= t1 || (!OUT && t1 == q1)) return;      // (the last chunk's own state is nobody's start)
  const int D = c.dim, V = c.vdim, col = (blockIdx.z * (NT / 64) + wave) * 16 + l16;
  const bool vok = col < V;
  float* dl = delta ? delta + ((size_t)blockIdx.x * c.heads + h) * D * V : nullptr;
  float* Sp = Sg + ((size_t)slot[b] * c.heads + h) * D * V;
  const float* init = OUT ? (dl ? dl : (pos0[b] > 0 ? Sp : nullptr)) : nullptr;
  const uint32_t off_s = g * 4 * (uint32_t)V + col;
  f32x4 S[DT];
#pragma unroll
  for (int d = 0; d < DT; d++)
#pragma unroll
    for (int r = 0; r < 4; r++) S[d][r] = init && vok && g * 4 < D - (d * 16 + r) ? (init + (size_t)(d * 16 + r) * V)[off_s] : 0.f;
  const float* kb = k + (h / c.hpk) * D;
  const float* qb = OUT ? q + (h / c.hpk) * D : nullptr;
  const float* ab = PH ? a + h : a + h * D;
  const float* vb = v + (size_t)h * V;
  float* ob = o + (size_t)h * V;
  const float sk = OUT && skip ? skip[h] : 0.f;
  // a thread's elements lie RS rows apart: one 32-bit offset per operand, the rest of every address is uniform
  constexpr int RS = NT / DW;
  const int row0 = tid / DW, cc0 = tid % DW;
  const uint32_t off_k = row0 * (uint32_t)c.ldk + cc0, off_q = row0 * (uint32_t)c.ldq + cc0, off_a = PH ? tid * (uint32_t)c.lda : row0 * (uint32_t)c.lda + cc0,
                 off_v = g * 4 * (uint32_t)c.ldv + col, off_o = g * 4 * (uint32_t)(c.heads * V) + col, off_m = tid * (uint32_t)c.ldm;
  float rq[OUT ? E : 1], rk[E], ra[PH ? 1 : E], rm = 0.f, rv[4];
  auto fetch = [&](int tb) {
#pragma unroll
    for (int n = 0; n < E; n++) {
      const int t = tb + n * RS;
      const bool ok = t + row0 < t1 && cc0 < D;
      rk[n] = ok ? (kb + (size_t)t * c.ldk)[off_k] : 0.f;
      if constexpr (OUT) rq[n] = ok ? (qb + (size_t)t * c.ldq)[off_q] : 0.f;
      if constexpr (!PH) ra[n] = ok ? (ab + (size_t)t * c.lda)[off_a] : 1.f;
    }
    if (tid < SM_T) {
      rm = tb + tid < t1 ? (vmul ? (vmul + (size_t)tb * c.ldm + h)[off_m] : 1.f) : 0.f;
      if constexpr (PH) ra[0] = tb + tid < t1 ? (ab + (size_t)tb * c.lda)[off_a] : 1.f;
    }
#pragma unroll
    for (int s = 0; s < 4; s++) rv[s] = vok && tb + g * 4 + s < t1 ? (vb + (size_t)(tb + s) * c.ldv)[off_v] : 0.f;
  };
  auto put = [&]() {
#pragma unroll
    for (int n = 0; n < E; n++) {
      const int at = (row0 + n * RS) * DP + cc0;
      lds[L::KR + at] = c.act ? silu_fast(rk[n]) : rk[n];
      if constexpr (OUT) lds[L::QR + at] = (c.act ? silu_fast(rq[n]) : rq[n]) * c.q_scale;
      if constexpr (!PH) lds[L::AR + at] = ra[n];
    }
    if (tid < SM_T) {
      lds[L::MR + tid] = rm;
      if constexpr (PH) lds[L::AR + tid] = ra[0];
    }
  };
  fetch(t0);
  put();
  for (int tb = t0; tb < t1; tb += SM_T) {
    float cv[4];
#pragma unroll
    for (int s = 0; s < 4; s++) cv[s] = c.act ? silu_fast(rv[s]) : rv[s];
    if (tb + SM_T < t1) fetch(tb + SM_T);
    __syncthreads();                       // the block's rows are there; the last block's products have been read
    if constexpr (OUT) {
      // (what follows compares the thread's place with constants: an opaque copy of it keeps those masks from being held across the loop)
      int tl = tid;
      asm volatile("" : "+v"(tl));
      if constexpr (PH) {
        if (wave < L::PARTS) {
          f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int d = wave; d < DT; d += L::PARTS) {
            const float4 x = *reinterpret_cast<const float4*>(lds + L::QR + l16 * DP + d * 16 + g * 4);
            const float4 y = *reinterpret_cast<const float4*>(lds + L::KR + l16 * DP + d * 16 + g * 4);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, y.x, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, y.y, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, y.z, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, y.w, acc, 0, 0, 0);
          }
#pragma unroll
          for (int r = 0; r < 4; r++) lds[L::AS + (wave * SM_T + g * 4 + r) * SM_AST + l16] = acc[r];
        }
        if (tid < SM_T * SM_T) {           // m_i prod_{i < j <= t} a_j, 0 for i > t
          const int t = tl / SM_T, i = tl % SM_T;
          float p = i <= t ? lds[L::MR + i] : 0.f;
#pragma unroll
          for (int j = 1; j < SM_T; j++) p *= j > i && j <= t ? lds[L::AR + j] : 1.f;
          lds[L::RT + t * SM_AST + i] = p;
        }
      } else {
        const int i = tl / SL, sl = tl % SL, i0 = wave * 64 / SL;
        float kk[CPS], w[CPS], sum[SM_T];
#pragma unroll
        for (int m = 0; m < CPS; m++) {
          kk[m] = lds[L::KR + i * DP + (m / VW) * SL * VW + sl * VW + m % VW];
          w[m] = 0.f;
        }
#pragma unroll
        for (int t = 0; t < SM_T; t++) {
          sum[t] = 0.f;
          if (t >= i0) {                   // (uniform over the wavefront)
#pragma unroll
            for (int m = 0; m < CPS; m++) {
              const int cc = (m / VW) * SL * VW + sl * VW + m % VW;
              w[m] = t == i ? kk[m] : w[m] * lds[L::AR + t * DP + cc];
              sum[t] = fmaf(lds[L::QR + t * DP + cc], w[m], sum[t]);
            }
          }
        }
        // the 16 sums over the row's 16 lanes: every step halves the sums a lane carries (partners 8, 7, 2, 1 lanes' bits away)
        fold_pairs<8, KTX_DPP_ROW_ROR8>(sum, tl & 8);
        fold_pairs<4, KTX_DPP_ROW_HALF_MIRROR>(sum, tl & 4);
        fold_pairs<2, KTX_DPP_QUAD_2301>(sum, tl & 2);
        fold_pairs<1, KTX_DPP_QUAD_1032>(sum, tl & 1);
        float st = sum[0];
        if constexpr (SL == 32) st += __shfl_xor(st, 16);
        if (sl < 16) lds[L::AS + sl * SM_AST + i] = fmaf(st, lds[L::MR + i], sl == i ? sk : 0.f);
      }
    }
    if (row0 == 0) {                       // thread = key channel, one group of threads per operand
      float p = 1.f;
#pragma unroll
      for (int t = SM_T - 1; t >= 0; t--) {
        lds[L::KP + t * DP + cc0] = lds[L::KR + t * DP + cc0] * (lds[L::MR + t] * p);
        p *= lds[L::AR + (PH ? t : t * DP + cc0)];
      }
      lds[L::PL + cc0] = p;
    } else if (OUT && row0 == 1) {
      float p = 1.f;
#pragma unroll
      for (int t = 0; t < SM_T; t++) {
        p *= lds[L::AR + (PH ? t : t * DP + cc0)];
        lds[L::QP + t * DP + cc0] = lds[L::QR + t * DP + cc0] * p;
      }
    }
    __syncthreads();
    if (tb + SM_T < t1) put();             // (the raw rows have been read)
    if constexpr (OUT) {
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int d = 0; d < DT; d++) {
        const float4 x = *reinterpret_cast<const float4*>(lds + L::QP + l16 * DP + d * 16 + g * 4);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, S[d][0], acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, S[d][1], acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, S[d][2], acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, S[d][3], acc, 0, 0, 0);
        if (d & 1) __builtin_amdgcn_sched_barrier(0);      // (all tiles' operands requested at once would cost the registers of a wavefront)
      }
      float4 y = *reinterpret_cast<const float4*>(lds + L::AS + l16 * SM_AST + g * 4);
      if constexpr (PH) {
#pragma unroll
        for (int n = 1; n < L::PARTS; n++) {
          const float4 z = *reinterpret_cast<const float4*>(lds + L::AS + (n * SM_T + l16) * SM_AST + g * 4);
          y = make_float4(y.x + z.x, y.y + z.y, y.z + z.z, y.w + z.w);
        }
        const float4 w = *reinterpret_cast<const float4*>(lds + L::RT + l16 * SM_AST + g * 4);
        const int i = l16 - g * 4;
        y = make_float4(fmaf(y.x, w.x, i == 0 ? sk : 0.f), fmaf(y.y, w.y, i == 1 ? sk : 0.f), fmaf(y.z, w.z, i == 2 ? sk : 0.f), fmaf(y.w, w.w, i == 3 ? sk : 0.f));
      }
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(y.x, cv[0], acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(y.y, cv[1], acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(y.z, cv[2], acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(y.w, cv[3], acc, 0, 0, 0);
#pragma unroll
      for (int r = 0; r < 4; r++) {
        if (vok && tb + g * 4 + r < t1) (ob + (size_t)(tb + r) * c.heads * V)[off_o] = acc[r];
      }
    }
#pragma unroll
    for (int d = 0; d < DT; d++) {
      const float4 p = *reinterpret_cast<const float4*>(lds + L::PL + d * 16 + g * 4);
      S[d][0] *= p.x;
      S[d][1] *= p.y;
      S[d][2] *= p.z;
      S[d][3] *= p.w;
#pragma unroll
      for (int s = 0; s < 4; s++) S[d] = __builtin_amdgcn_mfma_f32_16x16x4f32(lds[L::KP + (g * 4 + s) * DP + d * 16 + l16], cv[s], S[d], 0, 0, 0);
      if (d & 1) __builtin_amdgcn_sched_barrier(0);
    }
  }
  if (OUT && t1 != q1) return;
  float* dst = OUT ? Sp : dl;
  int gl = g * 4;
  asm volatile("" : "+v"(gl));
#pragma unroll
  for (int d = 0; d < DT; d++)
#pragma unroll
    for (int r = 0; r < 4; r++)
      if (vok && gl < D - (d * 16 + r)) (dst + (size_t)(d * 16 + r) * V)[off_s] = S[d][r];
}

// between the two passes over the chunks: (i) the product of a chunk's decays, thread = key row (or the head), (ii) thread = 4 (or 1)
// state entries walks the request's chunks and replaces every chunk's own state by the one it starts from
__global__ void __launch_bounds__(256) chunk_decay_kernel(ScanDims c, int cols, const int32_t* __restrict__ q_indptr, const float* __restrict__ a,
                                                          float* __restrict__ lam) {
  const int b = blockIdx.x / c.nch, ch = blockIdx.x % c.nch, e = blockIdx.y * 256 + threadIdx.x;      // e < cols = heads * dim, or heads
  const int q1 = q_indptr[b + 1], t0 = q_indptr[b] + ch * c.L, t1 = min(q1, t0 + c.L);
  if (t0 >= t1 || t1 == q1 || e >= cols) return;
  float p = 1.f;
#pragma unroll 16
  for (int t = t0; t < t1; t++) p *= a[(size_t)t * c.lda + e];
  lam[(size_t)blockIdx.x * cols + e] = p;
}

template <typename VT>
__device__ __forceinline__ VT vt_fma(float s, const VT& v, const VT& d);
template <>
__device__ __forceinline__ float vt_fma<float>(float s, const float& v, const float& d) { return fmaf(s, v, d); }
template <>
__device__ __forceinline__ float4 vt_fma<float4>(float s, const float4& v, const float4& d) { return f4_fma(s, v, d); }

constexpr int CC_U = 8;
template <typename VT, bool PH>
__global__ void __launch_bounds__(256) chunk_chain_kernel(ScanDims c, const int32_t* __restrict__ q_indptr, const int32_t* __restrict__ pos0,
                                                          const int32_t* __restrict__ slot, const float* __restrict__ Sg,
                                                          const float* __restrict__ lam, float* delta) {
  constexpr int N = sizeof(VT) / 4;
  const int e = (blockIdx.x * 256 + threadIdx.x) * N, h = blockIdx.y, b = blockIdx.z, DV = c.dim * c.vdim;
  if (e >= DV) return;
  const int n = q_indptr[b + 1] - q_indptr[b], nc = (n + c.L - 1) / c.L;
  if (nc == 0) return;
  VT S = VT();
  if (pos0[b] > 0) S = *reinterpret_cast<const VT*>(Sg + ((size_t)slot[b] * c.heads + h) * DV + e);
  const size_t step = (size_t)c.heads * DV, lstep = PH ? c.heads : (size_t)c.heads * c.dim;
  float* dp = delta + ((size_t)b * c.nch * c.heads + h) * DV + e;
  const float* lp = lam + (size_t)b * c.nch * lstep + (PH ? h : h * c.dim + e / c.vdim);
  for (int c0 = 0; c0 < nc; c0 += CC_U) {
    VT d[CC_U];
    float l[CC_U];
#pragma unroll
    for (int i = 0; i < CC_U; i++) {
      const bool ok = c0 + i < nc - 1;
      d[i] = ok ? *reinterpret_cast<const VT*>(dp + (size_t)(c0 + i) * step) : VT();
      l[i] = ok ? lp[(size_t)(c0 + i) * lstep] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < CC_U; i++) {
      if (c0 + i < nc) *reinterpret_cast<VT*>(dp + (size_t)(c0 + i) * step) = S;
      S = vt_fma<VT>(l[i], S, d[i]);
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------------
// gate / norm segments: a wavefront takes a unit — one norm group of at most GS_WAVE columns, or GS_WAVE columns of an un-normed segment —,
// wider groups take a workgroup
constexpr int GS_PER = 8, GS_WAVE = 64 * GS_PER, GS_WIDE = 2;
struct GateSegs {
  ktx_gate_seg s[KTX_GATE_SEGS];
  bool vec[KTX_GATE_SEGS];                 // aligned pieces of eight columns: a lane owns consecutive columns
};
// eight columns of a row, 16-byte aligned
__device__ __forceinline__ void f8_ld(const float* p, float (&v)[8]) {
  const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
  v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}
__device__ __forceinline__ void seg_o8(const ktx_gate_seg& s, int t, int c, float (&v)[8]) {
  if (s.o_dtype == KTX_SEQ_F32) {
    f8_ld(reinterpret_cast<const float*>(s.o) + (size_t)t * s.ldo + c, v);
  } else {
    const uint4 u = *reinterpret_cast<const uint4*>(reinterpret_cast<const bf16_t*>(s.o) + (size_t)t * s.ldo + c);
    v[0] = ktx_lo_f32(u.x); v[1] = ktx_hi_f32(u.x); v[2] = ktx_lo_f32(u.y); v[3] = ktx_hi_f32(u.y);
    v[4] = ktx_lo_f32(u.z); v[5] = ktx_hi_f32(u.z); v[6] = ktx_lo_f32(u.w); v[7] = ktx_hi_f32(u.w);
  }
}
__device__ __forceinline__ void st8(float* p, const float (&v)[8]) {
  *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  *reinterpret_cast<float4*>(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
}
__device__ __forceinline__ void st8(bf16_t* p, const float (&v)[8]) {
  *reinterpret_cast<uint4*>(p) = make_uint4(ktx_pk_bf16(v[0], v[1]), ktx_pk_bf16(v[2], v[3]), ktx_pk_bf16(v[4], v[5]), ktx_pk_bf16(v[6], v[7]));
}
__device__ __forceinline__ float seg_o(const ktx_gate_seg& s, int t, int c) {
  return s.o_dtype == KTX_SEQ_F32 ? reinterpret_cast<const float*>(s.o)[(size_t)t * s.ldo + c]
                                  : bf16_to_f32(reinterpret_cast<const bf16_t*>(s.o)[(size_t)t * s.ldo + c]);
}
__device__ __forceinline__ float seg_act(const ktx_gate_seg& s, float g) { return s.act ? silu_f32(g) : sigmoid_f32(g); }

template <typename OT>
__global__ void __launch_bounds__(256) gate_segments_kernel(int n_segs, GateSegs sg, OT* __restrict__ out, int64_t ldout) {
  extern __shared__ float row[];
  __shared__ float red[4];
  const int t = blockIdx.x, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int unit0 = blockIdx.y * 4 + wave, ustep = gridDim.y * 4;
  int base = 0;                            // units of the segments in front
  for (int si = 0; si < n_segs; si++) {
    const ktx_gate_seg& s = sg.s[si];
    OT* orow = out + (size_t)t * ldout + s.out_off;
    if (s.group <= GS_WAVE) {
      const int width = s.group ? s.group : GS_WAVE, units = (s.n + width - 1) / width;
      for (int u = unit0; u < base + units; u += ustep) {
        if (u < base) continue;
        const int c0 = (u - base) * width, nc = min(width, s.n - c0);
        float p[GS_PER], g[GS_PER], w[GS_PER];
        float ss = 0.f;
        const bool vec = sg.vec[si];
        if (vec) {                         // (whole pieces: nc, c0 and w_mod are multiples of 8)
          const int c = lane * 8;
#pragma unroll
          for (int i = 0; i < GS_PER; i++) {
            p[i] = g[i] = 0.f;
            w[i] = 1.f;
          }
          if (c < nc) {
            seg_o8(s, t, c0 + c, p);
            f8_ld(s.gate + (size_t)t * s.ldg + c0 + c, g);
            if (s.group) f8_ld(s.w + (c0 + c) % s.w_mod, w);
          }
        } else {
#pragma unroll
          for (int i = 0; i < GS_PER; i++) {
            const int c = lane + i * 64;
            const bool ok = c < nc;
            p[i] = ok ? seg_o(s, t, c0 + c) : 0.f;
            g[i] = ok ? s.gate[(size_t)t * s.ldg + c0 + c] : 0.f;
            w[i] = ok && s.group ? s.w[(c0 + c) % s.w_mod] : 1.f;
          }
        }
#pragma unroll
        for (int i = 0; i < GS_PER; i++) {
          g[i] = seg_act(s, g[i]);
          if (s.gate_first) p[i] *= g[i];
          ss += p[i] * p[i];
        }
        const float r = s.group ? 1.0f / sqrtf(wave_sum(ss) / (float)s.group + s.eps) : 1.0f;
        if (vec) {
#pragma unroll
          for (int i = 0; i < GS_PER; i++) p[i] = p[i] * r * w[i] * (s.gate_first ? 1.f : g[i]) * s.scale;
          if (lane * 8 < nc) st8(orow + c0 + lane * 8, p);
          continue;
        }
#pragma unroll
        for (int i = 0; i < GS_PER; i++) {
          const int c = lane + i * 64;
          if (c < nc) st_elem(orow, c0 + c, p[i] * r * w[i] * (s.gate_first ? 1.f : g[i]) * s.scale);
        }
      }
      base += units;
    } else {
      for (int gI = blockIdx.y; gI < s.n / s.group; gI += gridDim.y) {
        const int c0 = gI * s.group;
        float ss = 0.f;
        if (sg.vec[si] && s.group <= 8 * 256 * GS_WIDE) {      // a thread's pieces stay in registers, all requested before the first is used
          float p[GS_WIDE][8], g[GS_WIDE][8], w[8];
#pragma unroll
          for (int k = 0; k < GS_WIDE; k++) {
            const int c = (tid + k * 256) * 8;
            if (c < s.group) {
              seg_o8(s, t, c0 + c, p[k]);
              f8_ld(s.gate + (size_t)t * s.ldg + c0 + c, g[k]);
            } else {
#pragma unroll
              for (int i = 0; i < 8; i++) p[k][i] = g[k][i] = 0.f;
            }
          }
#pragma unroll
          for (int k = 0; k < GS_WIDE; k++)
#pragma unroll
            for (int i = 0; i < 8; i++) {
              g[k][i] = seg_act(s, g[k][i]);
              if (s.gate_first) p[k][i] *= g[k][i];
              ss += p[k][i] * p[k][i];
            }
          const float r = 1.0f / sqrtf(block_sum256(ss, red) / (float)s.group + s.eps) * s.scale;
#pragma unroll
          for (int k = 0; k < GS_WIDE; k++) {
            const int c = (tid + k * 256) * 8;
            if (c < s.group) {
              f8_ld(s.w + (c0 + c) % s.w_mod, w);
#pragma unroll
              for (int i = 0; i < 8; i++) p[k][i] *= r * w[i] * (s.gate_first ? 1.f : g[k][i]);
              st8(orow + c0 + c, p[k]);
            }
          }
          continue;
        }
#pragma unroll 4
        for (int c = tid; c < s.group; c += 256) {
          float p = seg_o(s, t, c0 + c);
          if (s.gate_first) p *= seg_act(s, s.gate[(size_t)t * s.ldg + c0 + c]);
          row[c] = p;
          ss += p * p;
        }
        const float r = 1.0f / sqrtf(block_sum256(ss, red) / (float)s.group + s.eps) * s.scale;
#pragma unroll 4
        for (int c = tid; c < s.group; c += 256) {      // (each thread re-reads only what it wrote)
          float p = row[c] * r * s.w[(c0 + c) % s.w_mod];
          if (!s.gate_first) p *= seg_act(s, s.gate[(size_t)t * s.ldg + c0 + c]);
          st_elem(orow, c0 + c, p);
        }
      }
    }
  }
}

}  // namespace

extern "C" {

int ktx_hyper_mix(int T, int W, int n, const ktx_hyper_args* a, ktx_stream_t stream) {
  KTX_REQUIRE(a && T >= 0 && W > 0 && n > 0 && n <= KTX_HYPER_MAX_STREAMS && a->x && a->x_tok > 0 && a->x_str >= 0,
              "ktx_hyper_mix: 1 .. 16 streams, the streams and their strides");
  KTX_REQUIRE(!a->y || (a->mix && a->out && a->ldy >= W), "ktx_hyper_mix: writing needs its weights");
  KTX_REQUIRE(!a->h || (a->norm_w && dtype_ok(a->out_dtype)), "ktx_hyper_mix: reading needs the norm and a known result type");
  KTX_REQUIRE(!a->rows || !a->x_out, "ktx_hyper_mix: a row gather does not write the streams");
  KTX_REQUIRE(a->h || a->x_out, "ktx_hyper_mix: nothing to do");
  if (T == 0) return 0;
  hipStream_t st = (hipStream_t)stream;
  auto al = [](const void* p) { return !p || aligned16(p); };
  const bool vec = W % 4 == 0 && W <= 4096 && a->x_tok % 4 == 0 && a->x_str % 4 == 0 && (!a->y || a->ldy % 4 == 0) && al(a->x) && al(a->y) &&
                   al(a->x_out) && al(a->norm_w) && al(a->norm_b) && al(a->h) && (n <= 4 || (n <= 8 && W <= 2048));
  const int ev = W <= 1024 ? 1 : W <= 2048 ? 2 : 4;
  const bool lp = a->h && a->out_dtype == KTX_SEQ_BF16;
  if (vec) {
#define KTX_HY_GO(NS, EV)                                                    \
  do {                                                                       \
    if (lp) hyper_vec_kernel<bf16_t, NS, EV><<<T, 256, 0, st>>>(W, *a);      \
    else hyper_vec_kernel<float, NS, EV><<<T, 256, 0, st>>>(W, *a);          \
  } while (0)
#define KTX_HY_EV(NS)                     \
  do {                                    \
    if (ev == 1) KTX_HY_GO(NS, 1);        \
    else if (ev == 2) KTX_HY_GO(NS, 2);   \
    else KTX_HY_GO(NS, 4);                \
  } while (0)
#define KTX_HY_EV2(NS)                    \
  do {                                    \
    if (ev == 1) KTX_HY_GO(NS, 1);        \
    else KTX_HY_GO(NS, 2);                \
  } while (0)
    switch (n) {
      case 1: KTX_HY_EV(1); break;
      case 2: KTX_HY_EV(2); break;
      case 3: KTX_HY_EV(3); break;
      case 4: KTX_HY_EV(4); break;
      case 5: KTX_HY_EV2(5); break;
      case 6: KTX_HY_EV2(6); break;
      case 7: KTX_HY_EV2(7); break;
      default: KTX_HY_EV2(8); break;
    }
#undef KTX_HY_EV2
#undef KTX_HY_EV
#undef KTX_HY_GO
  } else {
    const size_t lds = (size_t)W * 4;
    KTX_REQUIRE(lds <= 150 * 1024, "ktx_hyper_mix: a row must fit the LDS");
    KTX_HIP(ktx_set_max_lds((const void*)hyper_any_kernel<bf16_t>, 150 * 1024));
    KTX_HIP(ktx_set_max_lds((const void*)hyper_any_kernel<float>, 150 * 1024));
    if (lp) hyper_any_kernel<bf16_t><<<T, 256, lds, st>>>(W, n, *a);
    else hyper_any_kernel<float><<<T, 256, lds, st>>>(W, n, *a);
  }
  KTX_HIP(hipGetLastError());
  return 0;
}

int ktx_lowrank_decay(int T, int C, int R, const float* d_low, int64_t ldl, const float* d_w, const float* d_bias, float inv_tau,
                      float* d_alpha, ktx_stream_t stream) {
  KTX_REQUIRE(T >= 0 && C > 0 && R > 0 && ldl >= R && d_low && d_w && d_alpha, "ktx_lowrank_decay: sizes and pointers");
  KTX_REQUIRE((size_t)LD_TT * R * 4 <= 150 * 1024, "ktx_lowrank_decay: rank <= 4800");
  if (T == 0) return 0;
  KTX_HIP(ktx_set_max_lds((const void*)lowrank_decay_kernel, 150 * 1024));
  lowrank_decay_kernel<<<dim3((T + LD_TT - 1) / LD_TT, (C + 255) / 256), 256, (size_t)LD_TT * R * 4, (hipStream_t)stream>>>(T, C, R, d_low, ldl, d_w,
                                                                                                                       d_bias, inv_tau, d_alpha);
  KTX_HIP(hipGetLastError());
  return 0;
}

int ktx_ssd_prep(int B, int T, int max_q_len, int C, int taps, int H, const float* d_proj, int64_t ldp, int c_off, int dt_off,
                 const float* d_w, const float* d_bias, const float* d_dt_bias, const float* d_A_log, const int32_t* d_q_indptr,
                 const int32_t* d_pos0, const int32_t* d_slot, const int32_t* d_tok_req, float* d_conv_state, float* d_u, float* d_gates,
                 ktx_stream_t stream) {
  KTX_REQUIRE(B >= 0 && T >= 0 && max_q_len >= 0 && C > 0 && H >= 0 && taps >= 1 && taps <= SP_MAX_TAPS && c_off >= 0 && ldp >= c_off + C,
              "ktx_ssd_prep: 1 .. 16 taps, rows that hold the channels");
  KTX_REQUIRE(d_proj && d_w && d_q_indptr && d_pos0 && d_slot && d_tok_req && d_u && (taps == 1 || d_conv_state), "ktx_ssd_prep: null pointer");
  KTX_REQUIRE(H == 0 || (d_dt_bias && d_A_log && d_gates && dt_off >= 0 && ldp >= dt_off + H), "ktx_ssd_prep: the steps' inputs");
  if (T == 0 || B == 0) return 0;
  hipStream_t st = (hipStream_t)stream;
  const dim3 grid(T, (C + 1023) / 1024);
  const bool vec = taps <= 4 && C % 4 == 0 && ldp % 4 == 0 && c_off % 4 == 0 && aligned16(d_proj) && aligned16(d_w) && (!d_bias || aligned16(d_bias)) &&
                   aligned16(d_u) && (taps == 1 || aligned16(d_conv_state));
  const int one = vec && max_q_len == 1 ? 1 : 0;
  if (vec) {
#define KTX_SP_GO(TAPS)                                                                                                               \
  ssd_prep_vec_kernel<TAPS><<<grid, 256, 0, st>>>(C, H, d_proj, ldp, c_off, dt_off, d_w, d_bias, d_dt_bias, d_A_log, d_q_indptr, d_pos0, \
                                                  d_slot, d_tok_req, d_conv_state, one, d_u, d_gates)
    if (taps == 1) KTX_SP_GO(1);
    else if (taps == 2) KTX_SP_GO(2);
    else if (taps == 3) KTX_SP_GO(3);
    else KTX_SP_GO(4);
#undef KTX_SP_GO
  } else {
    ssd_prep_kernel<<<grid, 256, 0, st>>>(C, taps, H, d_proj, ldp, c_off, dt_off, d_w, d_bias, d_dt_bias, d_A_log, d_q_indptr, d_pos0, d_slot,
                                          d_tok_req, d_conv_state, d_u, d_gates);
  }
  KTX_HIP(hipGetLastError());
  if (taps > 1 && !one) {      // second launch: the state moves on only after every token of the step has read it
    conv_state_update_kernel<<<dim3((C + 255) / 256, B), 256, 0, st>>>(C, taps, d_q_indptr, d_pos0, d_slot, d_proj + c_off, ldp, nullptr, d_conv_state);
    KTX_HIP(hipGetLastError());
  }
  return 0;
}

static int scan_chunks(const ktx_decay_scan_args* a, int max_q_len) {
  return a->chunk_len > 0 && max_q_len > a->chunk_len ? (max_q_len + a->chunk_len - 1) / a->chunk_len : 1;
}

size_t ktx_decay_scan_scratch(const ktx_decay_scan_args* a, int B, int max_q_len) {
  const int nch = scan_chunks(a, max_q_len);
  if (nch == 1) return 0;
  return (size_t)B * nch * a->heads * ((size_t)a->dim * a->vdim + (a->a_per_head ? 1 : a->dim));
}

int ktx_decay_scan(int B, int T, int max_q_len, const int32_t* d_q_indptr, const int32_t* d_pos0, const int32_t* d_slot,
                   const ktx_decay_scan_args* a, ktx_stream_t stream) {
  KTX_REQUIRE(a && B >= 0 && T >= 0 && max_q_len >= 0 && a->heads > 0 && a->dim > 0 && a->vdim > 0 && a->heads_per_key > 0 &&
                  a->heads % a->heads_per_key == 0,
              "ktx_decay_scan: positive sizes, heads a multiple of heads_per_key");
  KTX_REQUIRE(d_q_indptr && d_pos0 && d_slot && a->q && a->k && a->v && a->a && a->S && a->o, "ktx_decay_scan: null pointer");
  KTX_REQUIRE(a->heads <= 65535 && a->dim <= 512, "ktx_decay_scan: dim <= 512");
  if (B == 0 || T == 0 || max_q_len == 0) return 0;
  const int nch = scan_chunks(a, max_q_len);
  KTX_REQUIRE(nch == 1 || a->scratch, "ktx_decay_scan: chunks need scratch");
  hipStream_t st = (hipStream_t)stream;
  ScanDims c{a->heads, a->dim, a->vdim, a->heads_per_key, nch == 1 ? max_q_len : a->chunk_len, nch, a->ldq, a->ldk, a->ldv, a->lda, a->ldm, a->q_scale, a->qkv_act};
  // few tokens: many short wavefronts, so that the state streams in and out side by side; prompts: long ones, whose fixed work per token
  // (values, read-out) is shared by more rows
  const int R = a->dim > 256 ? 32 : max_q_len <= 4 ? 8 : (a->dim > 128 || a->dim % 32 == 0) ? 32 : a->dim % 16 == 0 ? 16 : 8;
  const int R2 = (a->dim + R - 1) / R > 16 ? 32 : R;
  const int NW = (a->dim + R2 - 1) / R2;
  const bool full = a->dim % R2 == 0;
  const dim3 grid((unsigned)B * nch, a->heads, (a->vdim + 63) / 64);
  float* delta = nch > 1 ? a->scratch : nullptr;
  float* lam = nch > 1 ? a->scratch + (size_t)B * nch * a->heads * a->dim * a->vdim : nullptr;
  // prompts: the matrix cores, as many value columns per workgroup as a head has (up to 128)
  const bool mfma = a->dim <= 128 && max_q_len > SCAN_MFMA_MIN;
#define KTX_SCANM_GO(DT, NT, PH, OUT)                                                                                                              \
  do {                                                                                                                                          \
    const size_t lds = (size_t)ScanTile<DT, NT, PH>::FLOATS * 4;                                                                                 \
    KTX_HIP(ktx_set_max_lds((const void*)decay_scan_mfma_kernel<DT, NT, PH, OUT>, 128 * 1024));                                                   \
    decay_scan_mfma_kernel<DT, NT, PH, OUT><<<dim3((unsigned)B * nch, a->heads, (a->vdim + NT / 4 - 1) / (NT / 4)), NT, lds, st>>>(              \
        c, d_q_indptr, d_pos0, d_slot, a->q, a->k, a->v, a->a, a->vmul, a->skip, a->S, delta, a->o);                                              \
  } while (0)
#define KTX_SCANM_P(DT, NT, OUT)                       \
  do {                                                 \
    if (a->a_per_head) KTX_SCANM_GO(DT, NT, true, OUT); \
    else KTX_SCANM_GO(DT, NT, false, OUT);             \
  } while (0)
#define KTX_SCANM_N(DT, OUT)                        \
  do {                                              \
    if (a->vdim > 64) KTX_SCANM_P(DT, 512, OUT);    \
    else KTX_SCANM_P(DT, 256, OUT);                 \
  } while (0)
#define KTX_SCANM(OUT)                              \
  do {                                              \
    if (a->dim <= 32) KTX_SCANM_N(2, OUT);          \
    else if (a->dim <= 64) KTX_SCANM_N(4, OUT);     \
    else KTX_SCANM_N(8, OUT);                       \
  } while (0)
#define KTX_SCAN_GO(RR, PH, OUT, FULL)                                                                                                          \
  do {                                                                                                                                          \
    const size_t lds = (OUT) && NW > 1 ? (size_t)2 * NW * SC_TG * 64 * 4 : 0;                                                                    \
    KTX_HIP(ktx_set_max_lds((const void*)decay_scan_kernel<RR, PH, OUT, FULL>, 96 * 1024));                                                       \
    decay_scan_kernel<RR, PH, OUT, FULL><<<grid, NW * 64, lds, st>>>(c, d_q_indptr, d_pos0, d_slot, a->q, a->k, a->v, a->a, a->vmul, a->skip,     \
                                                                     a->S, delta, a->o);                                                        \
  } while (0)
#define KTX_SCAN_F(RR, PH, OUT)              \
  do {                                       \
    if (full) KTX_SCAN_GO(RR, PH, OUT, true); \
    else KTX_SCAN_GO(RR, PH, OUT, false);    \
  } while (0)
#define KTX_SCAN_P(RR, OUT)                       \
  do {                                            \
    if (a->a_per_head) KTX_SCAN_F(RR, true, OUT); \
    else KTX_SCAN_F(RR, false, OUT);              \
  } while (0)
#define KTX_SCAN(OUT)                     \
  do {                                    \
    if (R2 == 8) KTX_SCAN_P(8, OUT);      \
    else if (R2 == 16) KTX_SCAN_P(16, OUT); \
    else KTX_SCAN_P(32, OUT);             \
  } while (0)
  if (nch > 1) {
    if (mfma) KTX_SCANM(false);
    else KTX_SCAN(false);
    const int cols = a->a_per_head ? a->heads : a->heads * a->dim;
    chunk_decay_kernel<<<dim3((unsigned)B * nch, (cols + 255) / 256), 256, 0, st>>>(c, cols, d_q_indptr, a->a, lam);
    const int DV = a->dim * a->vdim;
    const bool v4 = a->vdim % 4 == 0 && aligned16(delta) && aligned16(a->S);
    const dim3 cg((unsigned)((DV / (v4 ? 4 : 1) + 255) / 256), a->heads, B);
    if (v4 && a->a_per_head) chunk_chain_kernel<float4, true><<<cg, 256, 0, st>>>(c, d_q_indptr, d_pos0, d_slot, a->S, lam, delta);
    else if (v4) chunk_chain_kernel<float4, false><<<cg, 256, 0, st>>>(c, d_q_indptr, d_pos0, d_slot, a->S, lam, delta);
    else if (a->a_per_head) chunk_chain_kernel<float, true><<<cg, 256, 0, st>>>(c, d_q_indptr, d_pos0, d_slot, a->S, lam, delta);
    else chunk_chain_kernel<float, false><<<cg, 256, 0, st>>>(c, d_q_indptr, d_pos0, d_slot, a->S, lam, delta);
  }
  if (mfma) KTX_SCANM(true);
  else KTX_SCAN(true);
#undef KTX_SCANM
#undef KTX_SCANM_N
#undef KTX_SCANM_P
#undef KTX_SCANM_GO
#undef KTX_SCAN
#undef KTX_SCAN_P
#undef KTX_SCAN_F
#undef KTX_SCAN_GO
  KTX_HIP(hipGetLastError());
  return 0;
}

int ktx_gate_segments(int T, int n_segs, const ktx_gate_seg* segs, void* d_out, int out_dtype, int64_t ldout, ktx_stream_t stream) {
  KTX_REQUIRE(T >= 0 && n_segs >= 1 && n_segs <= KTX_GATE_SEGS && segs && d_out && dtype_ok(out_dtype), "ktx_gate_segments: one or two segments");
  GateSegs sg;
  int units = 0;
  size_t lds = 0;
  for (int i = 0; i < n_segs; i++) {
    const ktx_gate_seg& s = segs[i];
    KTX_REQUIRE(s.o && s.gate && s.n > 0 && s.group >= 0 && dtype_ok(s.o_dtype) && s.ldo >= s.n && s.ldg >= s.n && s.out_off >= 0 &&
                    ldout >= s.out_off + s.n && (s.act == 0 || s.act == 1),
                "ktx_gate_segments: rows that hold the segment, a known activation");
    KTX_REQUIRE(s.group == 0 || (s.n % s.group == 0 && s.w && (s.w_mod == s.group || s.w_mod == s.n)), "ktx_gate_segments: groups divide the columns");
    if (s.group > GS_WAVE) lds = std::max(lds, (size_t)s.group * 4), units += 4 * (s.n / s.group);
    else units += s.group ? s.n / s.group : (s.n + GS_WAVE - 1) / GS_WAVE;
    sg.s[i] = s;
    const int osz = out_dtype == KTX_SEQ_F32 ? 4 : 2;
    sg.vec[i] = s.n % 8 == 0 && s.group % 8 == 0 && s.ldo % 8 == 0 && s.ldg % 4 == 0 && ldout % 8 == 0 && s.out_off % 8 == 0 && aligned16(s.o) &&
                aligned16(s.gate) && (!s.group || aligned16(s.w)) && aligned16(d_out) && ((size_t)ldout * osz) % 16 == 0;
  }
  KTX_REQUIRE(lds <= 150 * 1024, "ktx_gate_segments: a norm group must fit the LDS");
  if (T == 0) return 0;
  hipStream_t st = (hipStream_t)stream;
  KTX_HIP(ktx_set_max_lds((const void*)gate_segments_kernel<float>, 150 * 1024));
  KTX_HIP(ktx_set_max_lds((const void*)gate_segments_kernel<bf16_t>, 150 * 1024));
  // few tokens: the units of a token are spread over workgroups
  const int parts = std::max(1, std::min((units + 3) / 4, 1024 / std::max(T, 1)));
  const dim3 grid(T, parts);
  if (out_dtype == KTX_SEQ_F32) gate_segments_kernel<float><<<grid, 256, lds, st>>>(n_segs, sg, (float*)d_out, ldout);
  else gate_segments_kernel<bf16_t><<<grid, 256, lds, st>>>(n_segs, sg, (bf16_t*)d_out, ldout);
  KTX_HIP(hipGetLastError());
  return 0;
}

}  // extern "C"
