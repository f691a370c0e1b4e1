// Rotary positions, mainly in the "halves" layout: within a head, number i pairs with number i + half, and the pair (u, v) at
// position p becomes (u cos a - v sin a, v cos a + u sin a), a = p * freq[i]. The angle is formed and reduced to
// [-pi, pi] in 64-bit (a position in the thousands times a frequency near 1 would lose the low bits of a 32-bit angle),
// sine and cosine of the reduced angle are 32-bit.
//
//   hy_rope_prep    : the step after a fused q | k | v projection: bias per column, q and k heads rotated on their first
//                     2 qk_half numbers, optionally v heads rotated over 2 v_half numbers, q to a dense buffer, k / v into
//                     the caches at slot + s.
//   hy_rotate_heads : every head of a [M, H * n] activation rotated by sign * position and scaled (the inverse turn of
//                     an attention output whose values were cached rotated), written to a column slice. The rotated
//                     numbers may start at an offset within the head and may pair up as (2i, 2i + 1) instead (the
//                     interleaved layout: the rotated tail of a latent attention's queries, in place).
//   hy_qkv_prep     : the step after a fused q | k | v projection whose RMS norms run over the whole q and the whole k
//                     (before they are split into heads), with both pair layouts, and values blended with the same
//                     token's values of another layer. Heads may hold two maps (each rotated by itself), the values may
//                     be the key columns as projected, cosine and sine may carry a factor, and a layer may bring
//                     queries only.
#include "hy_util.h"
#include "hybrid.h"

namespace jla {

JLA_DEV void ro_sincos(int pos, double freq, float sign, float* s, float* c) {
  const double a = (double)pos * freq;
  const double r = a - 6.283185307179586476925 * rint(a * 0.159154943091895335769);
  sincosf((float)r, s, c);
  *s *= sign;
}

JLA_DEV void ro_st(float* p, float v) { *p = v; }
JLA_DEV void ro_st(bf16_t* p, float v) { *p = f2bf(v); }

// grid (M, ceil((H + 2G) / 4)), 4 waves: wave -> item: [0, H) q heads, [H, H + G) k heads, [H + G, H + 2G) v heads
template <typename CT>
__global__ void __launch_bounds__(256) rope_prep_kernel(RopePrep p) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int m = blockIdx.x, item = blockIdx.y * 4 + wave;
  if (item >= p.H + 2 * p.G) return;
  const int b = m / p.S, sidx = m - b * p.S;
  int kind, head, len, col, half;
  const double* freq;
  if (item < p.H) { kind = 0; head = item; len = p.dim; col = head * p.dim; half = p.qk_half; freq = p.qk_freq; }
  else if (item < p.H + p.G) {
    kind = 1; head = item - p.H; len = p.dim; col = (p.H + head) * p.dim; half = p.qk_half; freq = p.qk_freq;
  } else {
    kind = 2; head = item - p.H - p.G; len = p.vdim; col = (p.H + p.G) * p.dim + head * p.vdim;
    half = p.v_freq ? p.v_half : 0; freq = p.v_freq;
  }
  const float* row = p.proj + (size_t)m * p.ld + col;
  const float* bias = p.bias ? p.bias + col : nullptr;
  const int pos = p.positions[m];
  const int t = *p.slot + sidx;
  if (kind != 0 && (t < 0 || t >= p.T)) return;  // cache full: the write is dropped
  float* qd = p.q + ((size_t)m * p.H + head) * p.dim;
  CT* cd = kind == 0 ? nullptr
                     : (kind == 1 ? reinterpret_cast<CT*>(p.kc) : reinterpret_cast<CT*>(p.vc)) +
                           (((size_t)b * p.G + head) * p.T + t) * len;
  for (int i = lane; i < half; i += 64) {
    float sn, cs;
    ro_sincos(pos, freq[i], 1.f, &sn, &cs);
    const float u = row[i] + (bias ? bias[i] : 0.f), v = row[i + half] + (bias ? bias[i + half] : 0.f);
    const float a = u * cs - v * sn, c = v * cs + u * sn;
    if (kind == 0) { qd[i] = a; qd[i + half] = c; }
    else { ro_st(cd + i, a); ro_st(cd + i + half, c); }
  }
  for (int d = 2 * half + lane; d < len; d += 64) {
    const float v = row[d] + (bias ? bias[d] : 0.f);
    if (kind == 0) qd[d] = v;
    else ro_st(cd + d, v);
  }
}

int hy_rope_prep(const RopePrep& p, hipStream_t s) {
  if (p.B < 0 || p.S < 1 || p.H < 1 || p.G < 1 || p.H % p.G || p.dim < 1 || p.vdim < 1 || p.T < 1) return -1;
  if (p.qk_half < 0 || 2 * p.qk_half > p.dim || (p.qk_half > 0 && !p.qk_freq)) return -2;
  if (p.v_freq && (p.v_half < 0 || 2 * p.v_half > p.vdim)) return -2;
  if (p.ld < (p.H + p.G) * p.dim + p.G * p.vdim) return -3;
  const int M = p.B * p.S;
  if (M == 0) return 0;
  const int items = p.H + 2 * p.G;
  if ((items + 3) / 4 > 65535) return -4;
  dim3 grid(M, (items + 3) / 4);
  if (p.cbf16) rope_prep_kernel<bf16_t><<<grid, 256, 0, s>>>(p);
  else rope_prep_kernel<float><<<grid, 256, 0, s>>>(p);
  JLA_CHECK_LAUNCH();
  return 0;
}

// grid (M, Y), 4 waves. Every workgroup takes the token's two statistics (one read of q | k; a prompt's workgroup does a
// whole token, a decode step's token is shared by Y of them) and the token's sines and cosines once into LDS (they are the
// same for every head); the heads' pairs are then dealt to the threads.
constexpr int QP_MAX_HALF = 512;
constexpr int QP_UNR = 4;
template <typename CT>
__global__ void __launch_bounds__(256) qkv_prep_kernel(QkvPrep p) {
  __shared__ float red[8];
  __shared__ float cs[QP_MAX_HALF], sn[QP_MAX_HALF];
  const int tid = threadIdx.x;
  const int m = blockIdx.x, b = m / p.S, t = *p.slot + (m - b * p.S);
  const float* row = p.proj + (size_t)m * p.ld;
  const int qh = p.H * p.maps, kh = p.q_only ? 0 : p.G * p.maps;  // dim-sized parts of q and k
  const int nq = qh * p.dim, nk = kh * p.dim, ldk = p.maps * p.dim;
  const int pos = p.half > 0 ? p.positions[m] : 0;
  // both sums of squares in one walk over q | k, eight loads of a thread in flight, and the angle table behind them
  float sq = 0.f, sk = 0.f;
  if (p.q_w || p.k_w) {
    for (int d0 = 0; d0 < nq + nk; d0 += 2048) {
      float v[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const int d = min(d0 + tid + 256 * u, nq + nk - 1);
        v[u] = row[d] + (p.bias ? p.bias[d] : 0.f);
      }
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const int d = d0 + tid + 256 * u;
        if (d < nq) sq = fmaf(v[u], v[u], sq);
        else if (d < nq + nk) sk = fmaf(v[u], v[u], sk);
      }
    }
  }
  for (int i = tid; i < p.half; i += 256) {
    float si, co;
    ro_sincos(pos, p.freq[i], 1.f, &si, &co);
    sn[i] = si * p.rot_gain;
    cs[i] = co * p.rot_gain;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((tid & 63) == 0) {
    red[tid >> 6] = sq;
    red[4 + (tid >> 6)] = sk;
  }
  __syncthreads();  // (the angle table is complete too)
  sq = red[0] + red[1] + red[2] + red[3];
  sk = red[4] + red[5] + red[6] + red[7];
  const float rq = p.q_w ? 1.f / sqrtf(sq / (float)nq + p.eps) : 1.f;
  const float rk = p.k_w ? 1.f / sqrtf(sk / (float)nk + p.eps) : 1.f;
  const bool store = t >= 0 && t < p.T;  // (cache full: the write is dropped)
  const float lam = p.v_prev ? *p.lambda : 0.f;
  // q / k: an item is a rotated pair or a number that passes, (dim - half) of them per head; values: one number each. A
  // thread's items are taken QP_UNR at a time, all of their loads before the first use.
  const int per = p.dim - p.half, n_qk = (qh + kh) * per, n_v = p.q_only ? 0 : p.G * p.vdim;
  const int step = gridDim.y * 256, first = blockIdx.y * 256 + tid;
  for (int i0 = first; i0 < n_qk; i0 += QP_UNR * step) {
    float u[QP_UNR], v[QP_UNR];
    int head[QP_UNR], pair[QP_UNR], du[QP_UNR], dv[QP_UNR];
#pragma unroll
    for (int k = 0; k < QP_UNR; ++k) {
      const int idx = min(i0 + k * step, n_qk - 1);
      head[k] = idx / per;
      const int i = idx - head[k] * per;
      pair[k] = i < p.half ? i : -1;
      du[k] = i < p.half ? (p.halves ? i : 2 * i) : i + p.half;
      dv[k] = i < p.half ? (p.halves ? i + p.half : 2 * i + 1) : du[k];
      const int cu = head[k] * p.dim + du[k], cv = head[k] * p.dim + dv[k];
      const bool is_q = head[k] < qh;
      const float* gw = is_q ? p.q_w : (p.k_w ? p.k_w - nq : nullptr);
      const float rs = is_q ? rq : rk;
      u[k] = (row[cu] + (p.bias ? p.bias[cu] : 0.f)) * rs * (gw ? gw[cu] : 1.f);
      v[k] = (row[cv] + (p.bias ? p.bias[cv] : 0.f)) * rs * (gw ? gw[cv] : 1.f);
    }
#pragma unroll
    for (int k = 0; k < QP_UNR; ++k) {
      if (i0 + k * step >= n_qk) break;
      float a = u[k], c = v[k];
      if (pair[k] >= 0) {
        const float co = cs[pair[k]], si = sn[pair[k]];
        a = u[k] * co - v[k] * si;
        c = v[k] * co + u[k] * si;
      }
      if (head[k] < qh) {
        float* qd = p.q + (size_t)m * nq + head[k] * p.dim;
        qd[du[k]] = a;
        if (pair[k] >= 0) qd[dv[k]] = c;
      } else if (store) {
        const int part = head[k] - qh, g = part / p.maps;
        CT* cd = reinterpret_cast<CT*>(p.kc) + (((size_t)b * p.G + g) * p.T + t) * ldk + (part - g * p.maps) * p.dim;
        ro_st(cd + du[k], a);
        if (pair[k] >= 0) ro_st(cd + dv[k], c);
      }
    }
  }
  for (int i0 = first; i0 < n_v; i0 += QP_UNR * step) {
    float v[QP_UNR], vp[QP_UNR];
#pragma unroll
    for (int k = 0; k < QP_UNR; ++k) {
      const int d = min(i0 + k * step, n_v - 1), c = p.v_col + d;
      v[k] = row[c] + (p.bias ? p.bias[c] : 0.f);
      vp[k] = p.v_prev ? p.v_prev[(size_t)m * n_v + d] : 0.f;
    }
#pragma unroll
    for (int k = 0; k < QP_UNR; ++k) {
      const int d = i0 + k * step;
      if (d >= n_v) break;
      const float x = p.v_prev ? (1.f - lam) * v[k] + lam * vp[k] : v[k];
      if (p.v_out) p.v_out[(size_t)m * n_v + d] = x;
      const int g = d / p.vdim;
      if (store) ro_st(reinterpret_cast<CT*>(p.vc) + (((size_t)b * p.G + g) * p.T + t) * p.vdim + (d - g * p.vdim), x);
    }
  }
}

int hy_qkv_prep(const QkvPrep& p, hipStream_t s) {
  if (p.B < 0 || p.S < 1 || p.H < 1 || p.G < 1 || p.H % p.G || p.dim < 1 || p.vdim < 1 || p.T < 1) return -1;
  if (p.half < 0 || 2 * p.half > p.dim || p.half > QP_MAX_HALF || (p.half > 0 && !p.freq)) return -2;
  if (p.maps != 1 && p.maps != 2) return -6;
  const int parts = (p.H + (p.q_only ? 0 : p.G)) * p.maps;
  if ((long long)parts * p.dim > p.ld || (!p.q_only && (p.v_col < 0 || (long long)p.v_col + p.G * p.vdim > p.ld))) return -3;
  if (!p.q_only && (!p.kc || !p.vc)) return -7;
  if (p.v_prev && !p.lambda) return -4;
  const long long M = (long long)p.B * p.S;
  if (M == 0) return 0;
  if (M > 0x7fffffffLL) return -5;
  const dim3 grid((unsigned)M, M <= 8 ? (unsigned)min(8, (parts * (p.dim - p.half) + 255) / 256) : 1u);
  if (p.cbf16) qkv_prep_kernel<bf16_t><<<grid, 256, 0, s>>>(p);
  else qkv_prep_kernel<float><<<grid, 256, 0, s>>>(p);
  JLA_CHECK_LAUNCH();
  return 0;
}

// grid (M, ceil(H / 4)), one wave per (token, head)
__global__ void __launch_bounds__(256) rotate_heads_kernel(const float* a, int lda,
                                                           const int32_t* __restrict__ positions,
                                                           const double* __restrict__ freq, int half, int H, int n,
                                                           float sign, float gain, float* out, int ldo,
                                                           int offset, int interleaved) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int m = blockIdx.x, h = blockIdx.y * 4 + wave;
  if (h >= H) return;
  // (out may be a: a thread reads both numbers of its pair before it writes them, and no two threads share a number)
  const float* src = a + (size_t)m * lda + (size_t)h * n;
  float* dst = out + (size_t)m * ldo + (size_t)h * n;
  const int pos = half > 0 ? positions[m] : 0;
  for (int i = lane; i < half; i += 64) {
    float sn, cs;
    ro_sincos(pos, freq[i], sign, &sn, &cs);
    const int iu = offset + (interleaved ? 2 * i : i), iv = offset + (interleaved ? 2 * i + 1 : i + half);
    const float u = src[iu], v = src[iv];
    dst[iu] = (u * cs - v * sn) * gain;
    dst[iv] = (v * cs + u * sn) * gain;
  }
  if (src != dst || gain != 1.f) {
    for (int d = lane; d < offset; d += 64) dst[d] = src[d] * gain;
    for (int d = offset + 2 * half + lane; d < n; d += 64) dst[d] = src[d] * gain;
  }
}

int hy_rotate_heads(const float* a, int lda, const int32_t* positions, const double* freq, int half, int M, int H, int n,
                    float sign, float gain, float* out, int ldo, int offset, int interleaved, hipStream_t s) {
  if (M < 0 || H < 1 || n < 1 || lda < H * n || ldo < H * n) return -1;
  if (half < 0 || offset < 0 || offset + 2 * half > n || (half > 0 && !freq)) return -2;
  if (M == 0) return 0;
  if ((H + 3) / 4 > 65535) return -4;
  rotate_heads_kernel<<<dim3(M, (H + 3) / 4), 256, 0, s>>>(a, lda, positions, freq, half, H, n, sign, gain, out, ldo,
                                                             offset, interleaved);
  JLA_CHECK_LAUNCH();
  return 0;
}

}  // namespace jla
