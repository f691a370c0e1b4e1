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
//                     token's values of another layer.
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
// same for every head); the heads are then dealt to the waves.
constexpr int QP_MAX_HALF = 512;
template <typename CT>
__global__ void __launch_bounds__(256) qkv_prep_kernel(QkvPrep p) {
  __shared__ float red[16];
  __shared__ float cs[QP_MAX_HALF], sn[QP_MAX_HALF];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int m = blockIdx.x, b = m / p.S, t = *p.slot + (m - b * p.S);
  const float* row = p.proj + (size_t)m * p.ld;
  const int nq = p.H * p.dim, nk = p.G * p.dim;
  const int pos = p.half > 0 ? p.positions[m] : 0;
  for (int i = tid; i < p.half; i += 256) ro_sincos(pos, p.freq[i], 1.f, &sn[i], &cs[i]);
  float rq = 1.f, rk = 1.f;
  auto stat = [&](int c0, int n) {
    float ss = 0.f;
    for (int d0 = 0; d0 < n; d0 += 1024) {
      float v[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int d = c0 + min(d0 + tid + 256 * u, n - 1);
        v[u] = row[d] + (p.bias ? p.bias[d] : 0.f);
      }
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (d0 + tid + 256 * u < n) ss = fmaf(v[u], v[u], ss);
    }
    ss = block_sum(ss, red);
    return 1.f / sqrtf(ss / (float)n + p.eps);
  };
  if (p.q_w) rq = stat(0, nq);
  if (p.k_w) rk = stat(nq, nk);
  __syncthreads();  // (the angle table is complete)
  const bool store = t >= 0 && t < p.T;  // (cache full: the write is dropped)
  const float lam = p.v_prev ? *p.lambda : 0.f;
  for (int item = blockIdx.y * 4 + wave; item < p.H + 2 * p.G; item += gridDim.y * 4) {
    if (item >= p.H + p.G) {
      const int g = item - p.H - p.G, c0 = nq + nk + g * p.vdim;
      const size_t fl = ((size_t)m * p.G + g) * p.vdim;
      CT* cd = reinterpret_cast<CT*>(p.vc) + (((size_t)b * p.G + g) * p.T + (store ? t : 0)) * p.vdim;
      for (int d = lane; d < p.vdim; d += 64) {
        float v = row[c0 + d] + (p.bias ? p.bias[c0 + d] : 0.f);
        if (p.v_prev) v = (1.f - lam) * v + lam * p.v_prev[fl + d];
        if (p.v_out) p.v_out[fl + d] = v;
        if (store) ro_st(cd + d, v);
      }
      continue;
    }
    const bool is_q = item < p.H;
    const int head = is_q ? item : item - p.H, c0 = item * p.dim;
    const float rs = is_q ? rq : rk;
    const float* gw = is_q ? p.q_w : p.k_w;
    if (gw) gw += (size_t)head * p.dim;
    float* qd = p.q + ((size_t)m * p.H + head) * p.dim;
    CT* cd = reinterpret_cast<CT*>(p.kc) + (((size_t)b * p.G + head) * p.T + (store ? t : 0)) * p.dim;
    auto num = [&](int d) { return (row[c0 + d] + (p.bias ? p.bias[c0 + d] : 0.f)) * rs * (gw ? gw[d] : 1.f); };
    auto put = [&](int d, float v) {
      if (is_q) qd[d] = v;
      else if (store) ro_st(cd + d, v);
    };
    // the head's pairs, then the numbers that pass
    for (int i = lane; i < p.dim - p.half; i += 64) {
      if (i < p.half) {
        const int iu = p.halves ? i : 2 * i, iv = p.halves ? i + p.half : 2 * i + 1;
        const float u = num(iu), v = num(iv);
        put(iu, u * cs[i] - v * sn[i]);
        put(iv, v * cs[i] + u * sn[i]);
      } else {
        put(i + p.half, num(i + p.half));
      }
    }
  }
}

int hy_qkv_prep(const QkvPrep& p, hipStream_t s) {
  if (p.B < 0 || p.S < 1 || p.H < 1 || p.G < 1 || p.H % p.G || p.dim < 1 || p.vdim < 1 || p.T < 1) return -1;
  if (p.half < 0 || 2 * p.half > p.dim || p.half > QP_MAX_HALF || (p.half > 0 && !p.freq)) return -2;
  if (p.ld < (p.H + p.G) * p.dim + p.G * p.vdim) return -3;
  if (p.v_prev && !p.lambda) return -4;
  const long long M = (long long)p.B * p.S;
  if (M == 0) return 0;
  if (M > 0x7fffffffLL) return -5;
  const dim3 grid((unsigned)M, M <= 8 ? (unsigned)min(8, (p.H + 2 * p.G + 3) / 4) : 1u);
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
