// Softmax attention in two maps over the same values, the second subtracted from the first, over the
// paged cache (gfx950).  Query head h has two queries, a cached key row of a kv head holds two keys
// (K [G][16][2 dk], V [G][16][dv] inside a block), head h reads kv head h / (H / G):
//     a_m = softmax_j<=i ( cap(scale q_m . k_m,j) ) V     cap(s) = softcap tanh(s / softcap)
//     o = a_1 - lam a_2;  o / sqrt(mean(o^2) + eps) * out_scale per head;  times sigmoid(gate)
// Scores, weights, both sums, the difference and the norm are fp32.
//
// Matrix-core form (bf16): a workgroup owns 32 * NQ columns of one (sequence, kv head), a column being one
// (token, query head of the kv head), so that the heads of a kv head share every key and value that is
// staged.  Its 8 waves are 2 maps x NQ column groups x NK key groups: 4 x 1 for prompt chunks (each staged
// tile of 64 keys serves 128 columns), 1 x 4 for few columns (a tile of 128 keys, each wave a quarter of
// it).  Per 32 keys a wave multiplies S^T = K Q^T (v_mfma_f32_32x32x16_bf16, queries in registers), so a
// lane holds 16 keys of one column; turns them into weights in place; and multiplies O^T += V^T P^T with
// the weights straight from those registers, every weight as two bf16 halves.  The k order of that second
// product is the order in which a lane holds its keys; the values are staged transposed in the same order
// (within 16 keys: 0-3, 8-11, 4-7, 12-15), so that an operand is one 16-byte LDS read.
// A bounded score needs no running maximum: with softcap <= kMaxCap its exponential fits fp32 as it is,
// and partial sums over key groups or workgroups add up directly.  ONLINE keeps a running maximum for
// larger bounds and unbounded scores.
// The next tile's global loads are in flight while a tile is multiplied.  At the end the waves' sums meet in
// LDS, 32 value rows at a time: the difference, the norm and the gate are applied where they meet.  With
// nsplit > 1 a workgroup walks its share of the keys and leaves both maps' sums in `part`; a merge kernel
// does the rest.
//
// Rows form (fp32, sizes the matrix-core form does not take): a workgroup per (row, query head), keys in
// tiles of 256, a thread per key for both maps' scores, a wave's lanes across the value row.
#include <algorithm>

#include "mix_common.h"
#include "differential_attention.h"

namespace mxs {

typedef __bf16 bfx8_t __attribute__((ext_vector_type(8)));
typedef __bf16 bfx2_t __attribute__((ext_vector_type(2)));
typedef float fx2_t __attribute__((ext_vector_type(2)));
typedef float fx16_t __attribute__((ext_vector_type(16)));
typedef unsigned int ux4_t __attribute__((ext_vector_type(4)));

constexpr float kLog2e = 1.4426950408889634f;
constexpr float kMaxCap = 60.f;  // e^60 * (a million keys) * (values of 1e5) stays far inside fp32, e^-60 far above its smallest

__device__ __forceinline__ uint32_t cvt_pk(float a, float b) {
  return __builtin_bit_cast(uint32_t, __builtin_convertvector((fx2_t{a, b}), bfx2_t));
}

// scores -> log2 units, bounded when cap is: cap tanh(y) = cap - 2 cap / (1 + e^(2y))
struct Bound {
  float a, b, c;  // bounded: a - b / (1 + 2^(c s));  unbounded (b == 0): c s
  __device__ __forceinline__ float operator()(float s) const {
    if (b == 0.f) return c * s;
    return __builtin_fmaf(-b, __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(c * s)), a);
  }
};
__device__ __forceinline__ Bound make_bound(float scale, float cap) {
  Bound r;
  if (cap > 0.f) {
    r.a = cap * kLog2e;
    r.b = 2.f * r.a;
    r.c = 2.f * kLog2e * scale / cap;
  } else {
    r.a = r.b = 0.f;
    r.c = scale * kLog2e;
  }
  return r;
}

template <int KSM, int VTM, int NQ, int NK, bool ONLINE>
__global__ void __launch_bounds__(128 * NQ * NK, 2) differential_attention_mfma_kernel(const DiffArgs p) {
  constexpr int KSUB = NK == 1 ? 2 : 1;      // 32-key runs a wave takes of a tile
  constexpr int KT = 32 * KSUB * NK;         // keys per tile
  constexpr int NW = 2 * NQ * NK, NT = 64 * NW;
  constexpr int KP = (KT * 4 * KSM + NT - 1) / NT;         // 16-byte key pieces per thread (two maps of 16 KSM elements)
  constexpr int VP = (KT / 4 * 8 * VTM + NT - 1) / NT;     // 4 keys x 4 columns value units per thread
  constexpr bool PRE = !(VTM == 8 && NK > 1);              // next tile's loads wait in registers
  constexpr int VLD = KT + 8;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int dk = p.dk, dv = p.dv;
  const int KS = (dk + 15) >> 4, VT = (dv + 31) >> 5;
  const int KLD = KS * 16 + 8;               // padded LDS row of a key
  bf16_t* ks = reinterpret_cast<bf16_t*>(smem);            // [2][KT][KLD]
  bf16_t* vs = ks + 2 * KT * KLD;                          // [32 VT][VLD]
  float* xch = reinterpret_cast<float*>(smem);             // [NW][32][40], after the walk
  __shared__ float wsum[NW][32], wmax[ONLINE ? NW : 1][32];
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int c = lane & 31, hl = lane >> 5;
  // wave = map + 2 * (column group * NK + key group)
  const int map = wid & 1, wk = (wid >> 1) % NK, wq = (wid >> 1) / NK;
  const int s = blockIdx.z / p.nsplit, sp = blockIdx.z - s * p.nsplit, g = blockIdx.x;
  const int row0 = p.qsl[s];
  const int qlen = min(p.qsl[s + 1], p.n_rows) - row0;
  const int rep = p.H / p.G;
  // long walks first, the kv heads' workgroups of one tile side by side
  const int c0 = (static_cast<int>(gridDim.y) - 1 - static_cast<int>(blockIdx.y)) * 32 * NQ;
  if (row0 < 0 || qlen <= 0 || c0 >= qlen * rep) return;  // workgroup-uniform
  // the chunk's first position; its last row stays inside the block table whatever the metadata says
  const int pos0 = min(max(p.seq_lens[s] - qlen, 0), max(p.bt_stride * 16 - qlen, 0));
  const int ncol = qlen * rep;
  const int kend = min(pos0 + min(c0 + 32 * NQ - 1, ncol - 1) / rep + 1, p.bt_stride * 16);  // keys some column sees
  const int ntile = (kend + KT - 1) / KT;
  const int tile0 = ntile * sp / p.nsplit, tile1 = ntile * (sp + 1) / p.nsplit;
  const int* bt = p.block_tables + static_cast<long>(s) * p.bt_stride;
  // this lane's column
  const int col = c0 + wq * 32 + c;
  const bool ok = col < ncol;
  const int tok = min(col, ncol - 1) / rep, hd = g * rep + (ok ? col - tok * rep : 0);
  const int pq = pos0 + tok;
  const int p_first = pos0 + min(c0 + wq * 32, ncol - 1) / rep, p_last = pos0 + min(c0 + wq * 32 + 31, ncol - 1) / rep;
  const bool wave_on = c0 + wq * 32 < ncol;

  bfx8_t qf[KSM];
  {
    const bf16_t* qp = static_cast<const bf16_t*>(p.q) + static_cast<long>(row0 + tok) * p.q_stride + (2 * hd + map) * dk + 8 * hl;
#pragma unroll
    for (int k = 0; k < KSM; ++k) {
      ux4_t v = {0u, 0u, 0u, 0u};
      if (ok && k * 16 + 8 * hl < dk) v = *reinterpret_cast<const ux4_t*>(qp + 16 * k);
      qf[k] = __builtin_bit_cast(bfx8_t, v);
    }
  }
  // key columns past dk and value rows past dv stay zero for the whole walk
  {
    const int n16 = (2 * KT * KLD + 32 * VT * VLD) / 8;
    for (int i = tid; i < n16; i += NT) reinterpret_cast<uint4*>(smem)[i] = make_uint4(0, 0, 0, 0);
  }

  // ---- staging: keys as 16-byte pieces, values as 4 keys x 4 columns units
  const int kpr = 2 * dk / 8;                       // pieces per key row
  const int nkp = KT * kpr, vq = (dv + 3) >> 2, vhi = (vq + 7) >> 3, nvu = vhi * 8 * (KT / 4);
  const bf16_t* cache = static_cast<const bf16_t*>(p.cache);
  uint4 gk[PRE ? KP : 1];
  uint2 gv[PRE ? VP : 1][4];
  auto kload = [&](int t0, int i) {
    const int idx = tid + i * NT;
    uint4 v = make_uint4(0, 0, 0, 0);
    if (idx < nkp) {
      const int kr = idx / kpr, j = t0 + kr;
      if (j < kend)
        v = *reinterpret_cast<const uint4*>(cache + static_cast<long>(bt[j >> 4]) * p.block_stride + p.koff +
                                            (static_cast<long>(g) * 16 + (j & 15)) * (2 * dk) + (idx - kr * kpr) * 8);
    }
    return v;
  };
  auto kstore = [&](int i, uint4 v) {
    const int idx = tid + i * NT;
    if (idx < nkp) {
      const int kr = idx / kpr, e = (idx - kr * kpr) * 8, m = e >= dk ? 1 : 0;
      *reinterpret_cast<uint4*>(ks + (m * KT + kr) * KLD + e - m * dk) = v;
    }
  };
  auto vload = [&](int t0, int i, uint2* v) {
    const int u = tid + i * NT;
    const int kq = (u >> 3) % (KT / 4), dq = (u & 7) + 8 * ((u >> 3) / (KT / 4));
    const int j0 = t0 + 4 * kq;
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] = make_uint2(0, 0);
    if (u < nvu && dq < vq && j0 < kend) {  // 4 keys from a multiple of 4: one block
      const bf16_t* vp = cache + static_cast<long>(bt[j0 >> 4]) * p.block_stride + p.voff +
                         (static_cast<long>(g) * 16 + (j0 & 15)) * dv + 4 * dq;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (j0 + r < kend) v[r] = *reinterpret_cast<const uint2*>(vp + r * dv);  // rows past the last key may hold anything
    }
  };
  auto vstore = [&](int i, const uint2* v) {
    const int u = tid + i * NT;
    const int kq = (u >> 3) % (KT / 4), dq = (u & 7) + 8 * ((u >> 3) / (KT / 4));
    if (u < nvu && dq < vq) {
      const int a = kq & 3, at = 16 * (kq >> 2) + (a == 1 ? 8 : a == 2 ? 4 : 4 * a);
      bf16_t* d = vs + (4 * dq) * VLD + at;
      *reinterpret_cast<uint2*>(d) = make_uint2((v[0].x & 0xFFFFu) | (v[1].x << 16), (v[2].x & 0xFFFFu) | (v[3].x << 16));
      *reinterpret_cast<uint2*>(d + VLD) = make_uint2((v[0].x >> 16) | (v[1].x & 0xFFFF0000u), (v[2].x >> 16) | (v[3].x & 0xFFFF0000u));
      *reinterpret_cast<uint2*>(d + 2 * VLD) = make_uint2((v[0].y & 0xFFFFu) | (v[1].y << 16), (v[2].y & 0xFFFFu) | (v[3].y << 16));
      *reinterpret_cast<uint2*>(d + 3 * VLD) = make_uint2((v[0].y >> 16) | (v[1].y & 0xFFFF0000u), (v[2].y >> 16) | (v[3].y & 0xFFFF0000u));
    }
  };

  fx16_t o[VTM];
#pragma unroll
  for (int vt = 0; vt < VTM; ++vt)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[vt][i] = 0.f;
  float l = 0.f, m = ONLINE ? -INFINITY : 0.f;
  const Bound bound = make_bound(p.scale, p.softcap);

  if constexpr (PRE) {
    if (tile0 < tile1) {
#pragma unroll
      for (int i = 0; i < KP; ++i) gk[i] = kload(tile0 * KT, i);
#pragma unroll
      for (int i = 0; i < VP; ++i) vload(tile0 * KT, i, gv[i]);
    }
  }
  for (int tile = tile0; tile < tile1; ++tile) {
    __syncthreads();  // the tile before is no longer read (the first time: the zeros are in place)
    if constexpr (PRE) {
#pragma unroll
      for (int i = 0; i < KP; ++i) kstore(i, gk[i]);
#pragma unroll
      for (int i = 0; i < VP; ++i) vstore(i, gv[i]);
    } else {
#pragma unroll 2
      for (int i = 0; i < KP; ++i) kstore(i, kload(tile * KT, i));
#pragma unroll 2
      for (int i = 0; i < VP; ++i) {
        uint2 v[4];
        vload(tile * KT, i, v);
        vstore(i, v);
      }
    }
    __syncthreads();
    if constexpr (PRE) {
      if (tile + 1 < tile1) {
#pragma unroll
        for (int i = 0; i < KP; ++i) gk[i] = kload((tile + 1) * KT, i);
#pragma unroll
        for (int i = 0; i < VP; ++i) vload((tile + 1) * KT, i, gv[i]);
      }
    }
    if (!wave_on) continue;
#pragma unroll
    for (int sub = 0; sub < KSUB; ++sub) {
      const int kw = (wk * KSUB + sub) * 32, j0 = tile * KT + kw;
      if (j0 > p_last) continue;  // wave-uniform
      fx16_t acc;
#pragma unroll
      for (int i = 0; i < 16; ++i) acc[i] = 0.f;
      const bf16_t* kp = ks + (map * KT + kw + c) * KLD + 8 * hl;
#pragma unroll
      for (int k = 0; k < KSM; ++k)
        if (k < KS)
          acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bfx8_t, *reinterpret_cast<const ux4_t*>(kp + 16 * k)),
                                                        qf[k], acc, 0, 0, 0);
      const bool whole = j0 + 31 <= p_first;
      if constexpr (ONLINE) {
        float mx = -INFINITY;
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          const int j = j0 + 8 * (i >> 2) + 4 * hl + (i & 3);
          acc[i] = whole || j <= pq ? bound(acc[i]) : -INFINITY;
          mx = fmaxf(mx, acc[i]);
        }
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        const float m_new = fmaxf(m, mx);
        if (__builtin_amdgcn_ballot_w64(m_new > m) != 0) {
          const float corr = m_new == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(m - m_new);
          l *= corr;
#pragma unroll
          for (int vt = 0; vt < VTM; ++vt)
#pragma unroll
            for (int i = 0; i < 16; ++i) o[vt][i] *= corr;
          m = m_new;
        }
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          const float w = acc[i] == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(acc[i] - m);
          l += w;
          acc[i] = w;
        }
      } else {
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          float w = __builtin_amdgcn_exp2f(bound(acc[i]));
          if (!whole) {
            const int j = j0 + 8 * (i >> 2) + 4 * hl + (i & 3);
            w = j <= pq ? w : 0.f;
          }
          l += w;
          acc[i] = w;
        }
      }
#pragma unroll
      for (int h = 0; h < 2; ++h) {  // 16 keys: this lane's 8 weights as hi + lo
        ux4_t hi, lo;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float a = acc[8 * h + 2 * e], b = acc[8 * h + 2 * e + 1];
          const uint32_t w = cvt_pk(a, b);
          hi[e] = w;
          lo[e] = cvt_pk(a - bf2f_lo(w), b - bf2f_hi(w));
        }
        const bfx8_t ph = __builtin_bit_cast(bfx8_t, hi), pl = __builtin_bit_cast(bfx8_t, lo);
        const bf16_t* vp = vs + c * VLD + kw + 16 * h + 8 * hl;
#pragma unroll
        for (int vt = 0; vt < VTM; ++vt) {
          if (vt < VT) {
            const bfx8_t a = __builtin_bit_cast(bfx8_t, *reinterpret_cast<const ux4_t*>(vp + vt * 32 * VLD));
            o[vt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, ph, o[vt], 0, 0, 0);
            o[vt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, pl, o[vt], 0, 0, 0);
          }
        }
      }
    }
  }

  // ---- the waves of a column group meet
  l += __shfl_xor(l, 32, 64);
  if (hl == 0) {
    wsum[wid][c] = l;
    if (ONLINE) wmax[wid][c] = m;
  }
  __syncthreads();  // also: the last tile is no longer read
  float M[2] = {0.f, 0.f}, L[2] = {0.f, 0.f};
  auto wave_of = [&](int mp, int k) { return mp + 2 * (wq * NK + k); };
#pragma unroll
  for (int mp = 0; mp < 2; ++mp) {
    if constexpr (ONLINE) {
      M[mp] = -INFINITY;
#pragma unroll
      for (int k = 0; k < NK; ++k) M[mp] = fmaxf(M[mp], wmax[wave_of(mp, k)][c]);
    }
#pragma unroll
    for (int k = 0; k < NK; ++k) {
      const float w = wsum[wave_of(mp, k)][c];
      if constexpr (ONLINE) L[mp] += w == 0.f ? 0.f : w * __builtin_amdgcn_exp2f(wmax[wave_of(mp, k)][c] - M[mp]);
      else L[mp] += w;
    }
  }
  float f = 1.f;
  if constexpr (ONLINE) f = l == 0.f ? 0.f : __builtin_amdgcn_exp2f(m - M[map]);
  const bool split = p.nsplit > 1;
  if (!split) f *= (map == 0 ? 1.f : -p.lam) / L[map];
  float* xw = xch + wid * (32 * 40);
  float ss = 0.f;
#pragma unroll
  for (int vt = 0; vt < VTM; ++vt) {
    if (vt >= VT) continue;  // workgroup-uniform
    // waves whose sums another one gathers hand them over
    const bool gather = wk == 0 && (split || map == 0);
    if (!gather) {
#pragma unroll
      for (int i = 0; i < 16; ++i) xw[(8 * (i >> 2) + 4 * hl + (i & 3)) * 40 + c] = o[vt][i] * f;
    }
    __syncthreads();
    if (gather) {
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int at = (8 * (i >> 2) + 4 * hl + (i & 3)) * 40 + c;
        float v = o[vt][i] * f;
#pragma unroll
        for (int k = 1; k < NK; ++k) v += xch[wave_of(map, k) * (32 * 40) + at];
        if (!split) {
#pragma unroll
          for (int k = 0; k < NK; ++k) v += xch[wave_of(1, k) * (32 * 40) + at];
        }
        o[vt][i] = v;
        ss += v * v;
      }
    }
    __syncthreads();
  }
  if (wk != 0 || !ok) return;
  const long row = row0 + tok;
  if (split) {
    float* pr = p.part + (((row * p.H + hd) * 2 + map) * p.nsplit + sp) * (dv + 4);
#pragma unroll
    for (int vt = 0; vt < VTM; ++vt) {
#pragma unroll
      for (int b = 0; b < 4; ++b) {
        const int d = 32 * vt + 8 * b + 4 * hl;
        if (d < dv) *reinterpret_cast<float4*>(pr + d) = make_float4(o[vt][4 * b], o[vt][4 * b + 1], o[vt][4 * b + 2], o[vt][4 * b + 3]);
      }
    }
    if (hl == 0) {
      pr[dv] = L[map];
      pr[dv + 1] = M[map];
    }
    return;
  }
  if (map != 0) {
    return;
  }
  ss += __shfl_xor(ss, 32, 64);
  const float r = rsqrtf(ss / static_cast<float>(dv) + p.eps) * p.out_scale;
  bf16_t* op = static_cast<bf16_t*>(p.out) + row * (static_cast<long>(p.H) * dv) + hd * dv;
  const bf16_t* gp = p.gate ? static_cast<const bf16_t*>(p.gate) + row * p.gate_stride + hd * dv : nullptr;
#pragma unroll
  for (int vt = 0; vt < VTM; ++vt) {
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      const int d = 32 * vt + 8 * b + 4 * hl;
      if (d < dv) {
        float v[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = o[vt][4 * b + e] * r;
        if (gp) {
          const uint2 gw = *reinterpret_cast<const uint2*>(gp + d);
          v[0] *= sigmoid_f(bf2f_lo(gw.x));
          v[1] *= sigmoid_f(bf2f_hi(gw.x));
          v[2] *= sigmoid_f(bf2f_lo(gw.y));
          v[3] *= sigmoid_f(bf2f_hi(gw.y));
        }
        uint2 w;
        w.x = pack2(v[0], v[1]);
        w.y = pack2(v[2], v[3]);
        *reinterpret_cast<uint2*>(op + d) = w;
      }
    }
  }
}

// What the split workgroups left: per (row, head) and map nsplit sums of [dv values | weight sum | maximum].
__global__ void __launch_bounds__(64) differential_merge_kernel(const DiffArgs p, int S) {
  const long row = blockIdx.x;
  const int hd = blockIdx.y, lane = threadIdx.x, dv = p.dv;
  if (row < p.qsl[0] || row >= p.qsl[S]) return;
  const float* base = p.part + (row * p.H + hd) * 2 * p.nsplit * (dv + 4);
  float inv[2], M[2];
  for (int mp = 0; mp < 2; ++mp) {
    const float* b = base + mp * p.nsplit * (dv + 4);
    float mx = -INFINITY, L = 0.f;
    for (int k = 0; k < p.nsplit; ++k) mx = fmaxf(mx, b[k * (dv + 4) + dv + 1]);
    for (int k = 0; k < p.nsplit; ++k) {
      const float w = b[k * (dv + 4) + dv];
      L += w == 0.f ? 0.f : w * __builtin_amdgcn_exp2f(b[k * (dv + 4) + dv + 1] - mx);
    }
    M[mp] = mx;
    inv[mp] = (mp == 0 ? 1.f : -p.lam) / L;
  }
  constexpr int NC = 4;  // dv <= 256
  float o[NC], ss = 0.f;
#pragma unroll
  for (int n = 0; n < NC; ++n) {
    const int d = lane + 64 * n;
    o[n] = 0.f;
    if (d >= dv) continue;
    for (int mp = 0; mp < 2; ++mp) {
      const float* b = base + mp * p.nsplit * (dv + 4);
      float a = 0.f;
      for (int k = 0; k < p.nsplit; ++k) {
        const float* e = b + k * (dv + 4);
        if (e[dv] != 0.f) a += e[d] * __builtin_amdgcn_exp2f(e[dv + 1] - M[mp]);
      }
      o[n] += a * inv[mp];
    }
    ss += o[n] * o[n];
  }
  const float r = rsqrtf(wave_sum(ss) / static_cast<float>(dv) + p.eps) * p.out_scale;
  bf16_t* op = static_cast<bf16_t*>(p.out) + row * (static_cast<long>(p.H) * dv) + hd * dv;
  const bf16_t* gp = p.gate ? static_cast<const bf16_t*>(p.gate) + row * p.gate_stride + hd * dv : nullptr;
#pragma unroll
  for (int n = 0; n < NC; ++n) {
    const int d = lane + 64 * n;
    if (d < dv) op[d] = f2bf(gp ? o[n] * r * sigmoid_f(bf2f(gp[d])) : o[n] * r);
  }
}

// ---- rows form
constexpr int kDiffTile = 256;
constexpr int kDiffChunks = 8;  // dv <= 64 * 8

template <typename T>
__global__ void __launch_bounds__(256) differential_attention_rows_kernel(const DiffArgs p, int S, int bs, int vec) {
  extern __shared__ float lds[];
  const int dk = p.dk, dv = p.dv, dkp = (dk + 3) & ~3;
  float* qs = lds;                      // [2][dkp]
  float* w = qs + 2 * dkp;              // [2][kDiffTile]
  float* red = w + 2 * kDiffTile;       // [4][2][dv]
  __shared__ float scratch[16];
  const int t = blockIdx.x, hd = blockIdx.y;
  if (t < p.qsl[0] || t >= p.qsl[S]) return;
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int s = seq_of_row(p.qsl, S, t);
  const int qlen = p.qsl[s + 1] - p.qsl[s];
  const int pos = min(max(p.seq_lens[s] - qlen + (t - p.qsl[s]), 0), p.bt_stride * bs - 1);
  const int g = hd / (p.H / p.G);
  const int* bt = p.block_tables + static_cast<long>(s) * p.bt_stride;
  const T* cache = static_cast<const T*>(p.cache);
  for (int d = tid; d < 2 * dk; d += 256) {
    const int m = d >= dk ? 1 : 0;
    qs[m * dkp + d - m * dk] = ldf(static_cast<const T*>(p.q) + static_cast<long>(t) * p.q_stride + static_cast<long>(hd) * 2 * dk + d) * p.scale;
  }
  float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};
  float acc[2][kDiffChunks];
#pragma unroll
  for (int mp = 0; mp < 2; ++mp)
#pragma unroll
    for (int c = 0; c < kDiffChunks; ++c) acc[mp][c] = 0.f;
  const int nchunk = (dv + 63) >> 6;
  __syncthreads();
  for (int t0 = 0; t0 <= pos; t0 += kDiffTile) {
    const int nt = min(kDiffTile, pos + 1 - t0), j = t0 + tid;
    const T* kp = tid < nt ? cache + static_cast<long>(bt[j / bs]) * p.block_stride + p.koff + (static_cast<long>(g) * bs + j % bs) * (2 * dk)
                           : nullptr;
    for (int mp = 0; mp < 2; ++mp) {
      float sc = -INFINITY;
      if (tid < nt) {
        sc = dot_row<T>(qs + mp * dkp, kp + mp * dk, dk, vec);
        if (p.softcap > 0.f) sc = p.softcap * tanhf(sc / p.softcap);
      }
      const float m_new = fmaxf(m[mp], block_max(sc, scratch));
      const float e = tid < nt ? expf(sc - m_new) : 0.f;
      w[mp * kDiffTile + tid] = e;
      const float tsum = block_sum(e, scratch);  // its barriers also publish w
      const float corr = expf(m[mp] - m_new);    // first tile: exp(-inf) = 0
      l[mp] = l[mp] * corr + tsum;
      m[mp] = m_new;
#pragma unroll
      for (int c = 0; c < kDiffChunks; ++c) acc[mp][c] *= corr;
    }
    for (int n = wid; n < nt; n += 4) {
      const int jj = t0 + n;
      const T* vp = cache + static_cast<long>(bt[jj / bs]) * p.block_stride + p.voff + (static_cast<long>(g) * bs + jj % bs) * dv;
      const float w0 = w[n], w1 = w[kDiffTile + n];
#pragma unroll
      for (int c = 0; c < kDiffChunks; ++c) {
        const int d = lane + 64 * c;
        if (c < nchunk && d < dv) {
          const float v = ldf(vp + d);
          acc[0][c] += w0 * v;
          acc[1][c] += w1 * v;
        }
      }
    }
    __syncthreads();  // w is rewritten by the next tile
  }
#pragma unroll
  for (int mp = 0; mp < 2; ++mp)
#pragma unroll
    for (int c = 0; c < kDiffChunks; ++c) {
      const int d = lane + 64 * c;
      if (c < nchunk && d < dv) red[(wid * 2 + mp) * dv + d] = acc[mp][c];
    }
  __syncthreads();
  const float i0 = 1.f / l[0], i1 = p.lam / l[1];
  float ss = 0.f;
  for (int d = tid; d < dv; d += 256) {
    const float a = (red[d] + red[2 * dv + d]) + (red[4 * dv + d] + red[6 * dv + d]);
    const float b = (red[dv + d] + red[3 * dv + d]) + (red[5 * dv + d] + red[7 * dv + d]);
    const float o = a * i0 - b * i1;
    red[d] = o;  // read again by this thread only
    ss += o * o;
  }
  const float r = rsqrtf(block_sum(ss, scratch) / static_cast<float>(dv) + p.eps) * p.out_scale;
  T* op = static_cast<T*>(p.out) + static_cast<long>(t) * (static_cast<long>(p.H) * dv) + hd * dv;
  const T* gp = p.gate ? static_cast<const T*>(p.gate) + static_cast<long>(t) * p.gate_stride + static_cast<long>(hd) * dv : nullptr;
  for (int d = tid; d < dv; d += 256) stf(op + d, gp ? red[d] * r * sigmoid_f(ldf(gp + d)) : red[d] * r);
}

// Column tiles a chunk of max_q rows is cut into by the matrix-core form.
int differential_tiles(int max_q, int rep) {
  const int cols = max_q * rep;
  return cols <= 32 ? 1 : (cols + 127) / 128;
}

bool differential_takes_mfma(const DiffArgs& a, int bs) {
  auto al = [](const void* q, size_t n) { return reinterpret_cast<uintptr_t>(q) % n == 0; };
  return bs == 16 && a.dk % 8 == 0 && a.dk <= 128 && a.dv % 4 == 0 && a.dv <= 256 && a.q_stride % 8 == 0 && al(a.q, 16) &&
         al(a.cache, 16) && a.koff % 8 == 0 && a.voff % 4 == 0 && a.block_stride % 8 == 0 && al(a.out, 8) &&
         (a.gate == nullptr || (al(a.gate, 8) && a.gate_stride % 4 == 0)) && a.bt_stride >= 1;
}

template <int KSM, int VTM, int NQ, int NK, bool ONLINE>
static bool launch_mfma(const DiffArgs& a, int S, hipStream_t st) {
  constexpr int KT = 32 * (NK == 1 ? 2 : 1) * NK;
  const int KS = (a.dk + 15) / 16, VT = (a.dv + 31) / 32;
  const size_t stage = 2 * static_cast<size_t>(2 * KT * (KS * 16 + 8) + 32 * VT * (KT + 8));
  const size_t shm = std::max<size_t>(stage, 2 * NQ * NK * 32 * 40 * sizeof(float));
  if (shm > 64 * 1024 - 4096) {
    if (hipFuncSetAttribute(reinterpret_cast<const void*>(&differential_attention_mfma_kernel<KSM, VTM, NQ, NK, ONLINE>),
                            hipFuncAttributeMaxDynamicSharedMemorySize, 156 * 1024) != hipSuccess) {
      (void)hipGetLastError();
      return false;
    }
  }
  const int cols = a.max_q * (a.H / a.G);
  const dim3 grid(a.G, (cols + 32 * NQ - 1) / (32 * NQ), S * a.nsplit);
  if (grid.z > 65535u || grid.y > 65535u) return false;
  hipLaunchKernelGGL((differential_attention_mfma_kernel<KSM, VTM, NQ, NK, ONLINE>), grid, dim3(128 * NQ * NK), shm, st, a);
  MXS_CHECK_LAUNCH();
  return true;
}

template <int NQ, int NK, bool ONLINE>
static bool launch_sizes(const DiffArgs& a, int S, hipStream_t st) {
  if (a.dk <= 32 && a.dv <= 64) return launch_mfma<2, 2, NQ, NK, ONLINE>(a, S, st);
  if (a.dk <= 64 && a.dv <= 128) return launch_mfma<4, 4, NQ, NK, ONLINE>(a, S, st);
  return launch_mfma<8, 8, NQ, NK, ONLINE>(a, S, st);
}

bool launch_differential_attention(const DiffArgs& a0, int S, int bs, bool bf, hipStream_t st) {
  if (S == 0 || a0.n_rows == 0) return true;
  DiffArgs a = a0;
  if (bf && differential_takes_mfma(a, bs)) {
    const bool online = !(a.softcap > 0.f && a.softcap <= kMaxCap);
    const bool few = a.max_q * (a.H / a.G) <= 32;
    const bool done = few ? (online ? launch_sizes<1, 4, true>(a, S, st) : launch_sizes<1, 4, false>(a, S, st))
                          : (online ? launch_sizes<4, 1, true>(a, S, st) : launch_sizes<4, 1, false>(a, S, st));
    if (done) {
      if (a.nsplit > 1) {
        hipLaunchKernelGGL(differential_merge_kernel, dim3(a.n_rows, a.H), dim3(64), 0, st, a, S);
        MXS_CHECK_LAUNCH();
      }
      return true;
    }
  }
  if (a.dv > 64 * kDiffChunks) return false;
  const size_t shm = (2 * ((a.dk + 3) & ~3) + 2 * kDiffTile + 8 * static_cast<size_t>(a.dv)) * sizeof(float);
  if (shm > 60 * 1024) return false;
  const int el = bf ? 8 : 4;
  const int vec = a.dk % el == 0 && a.koff % el == 0 && a.block_stride % el == 0 && reinterpret_cast<uintptr_t>(a.cache) % 16 == 0;
  if (bf)
    hipLaunchKernelGGL(differential_attention_rows_kernel<bf16_t>, dim3(a.n_rows, a.H), dim3(256), shm, st, a, S, bs, vec);
  else
    hipLaunchKernelGGL(differential_attention_rows_kernel<float>, dim3(a.n_rows, a.H), dim3(256), shm, st, a, S, bs, vec);
  MXS_CHECK_LAUNCH();
  return true;
}

}  // namespace mxs
