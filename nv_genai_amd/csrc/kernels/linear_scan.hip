// Linear attention with a diagonal decay: a matrix state per head, carried across steps in state slots,
//
//   S_t = diag(w_t) S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t
//
//   CH true   w per key channel and row: log w = logsigmoid(z + bias) / tau
//   CH false  one constant w per head (its logarithm is given)
//
// q, k and v may pass silu first; q is multiplied by a constant.
//
// linear_rows: launches whose segments are single rows: o = (q w)^T S + (q . k) v and the update in one pass over
// the state.
//
// linear_prep + linear_walk: portions, in blocks of 16 rows. With c_t the running sum of the log decays inside
// a block (c of the last row: c_E), everything that does not depend on the state is formed ahead of time, one
// workgroup per (block, head):
//   R_t = q_t e^(c_t),  K'_s = k_s e^(c_E - c_s),  N_ts = sum_channels q_t k_s e^(c_t - c_s)  (s <= t)
// so that the walk over the blocks of a segment is
//   O = R S + N V,  S <- diag(e^(c_E)) S + K'^T V.
// The state enters linearly, so a launch with too few waves for the chip walks the segments in parts: one pass
// leaves what every part adds to the state and by how much it decays, a second one starts every part from the
// sum of what came before it and writes the outputs.
// No exponent above is positive. N of a constant decay takes its factor behind the product of q and k; N of
// channel decays is (q e^(c_t)) . (k e^(-c_s)) as long as no channel of the block decays by more than e^-SAFE
// (the factors stay far inside fp32), else the pairs of rows are summed one by one.
//
// All products run on mfma_f32_16x16x4_f32 (true fp32). The operands lie in the workspace in the order a lane
// needs them: a k-slot of step r is index 4 h + r (h = lane / 16), so an A operand of four steps is one float4
// per lane, and accumulators (row 4 h + r, column lane % 16) are B operands of the next product without moving
// between lanes: a wave keeps its 16 value columns of the state in registers for the whole segment.
//
// Workspace of (block, head), DT = tiles of 16 key channels: R [DT][64][4], K'^T [DT][64][4], N [64][4],
// e^(c_E) [16 DT]. Block c of segment b is entry cu[b] / 16 + b + c (cu counted from the launch's first row).
#include "common.h"
#include "gate_fn.h"
#include "kernels.h"

namespace nga {

namespace {

constexpr float SAFE = 30.f;

template <typename T> __device__ __forceinline__ float silu_(float z) { return z * GateFn<T>::sigmoid(z); }

// ---------------------------------------------------------------------------------------------
// Single rows. Workgroup = (value tile of TL * VEC columns, head, row); thread (rg, c) keeps rows
// rg + RG m (m < NR) of columns VEC c .. of the state.
template <typename T, bool CH, int TL, int VEC, int NR>
__global__ void __launch_bounds__(256) linear_rows_kernel(const LinearParams P) {
  using F = GateFn<T>;
  constexpr int RG = 256 / TL;
  __shared__ float wS[256], kS[256], rS[256];     // decay, key, query times decay
  __shared__ float red[4];
  __shared__ float part[4][TL][VEC];
  const int vt = blockIdx.x, h = blockIdx.y;
  const int64_t row = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int d = P.d, dv = P.dv;
  const int slot = P.slots[row];
  const bool fresh = slot < 0 || P.pos[row] == 0;
  const int c = tid % TL, rg = tid / TL;
  const int col = (vt * TL + c) * VEC;
  const bool colok = col < dv;
  float* sp = slot >= 0 ? P.state + ((int64_t)slot * P.H + h) * (int64_t)d * dv + col : nullptr;
  float S[NR][VEC];
#pragma unroll
  for (int m = 0; m < NR; ++m) {
    const int i = rg + RG * m;
    const bool ld = !fresh && colok && i < d;
    if constexpr (VEC == 4) {
      const float4 s4 = ld ? *reinterpret_cast<const float4*>(sp + (int64_t)i * dv) : make_float4(0.f, 0.f, 0.f, 0.f);
      S[m][0] = s4.x, S[m][1] = s4.y, S[m][2] = s4.z, S[m][3] = s4.w;
    } else {
      S[m][0] = ld ? sp[(int64_t)i * dv] : 0.f;
    }
  }
  // the row's vectors: one channel per thread (d <= 256)
  float kk = 0.f, qq = 0.f, ww = 1.f, vv[VEC];
  if (tid < d) {
    kk = ldf((const T*)P.k + row * P.ks + h * d + tid);
    qq = ldf((const T*)P.q + row * P.qs + h * d + tid);
    if (P.silu) {
      kk = silu_<T>(kk);
      qq = silu_<T>(qq);
    }
    qq *= P.q_scale;
    const float lw = CH ? -P.inv_tau * F::softplus(-(ldf((const T*)P.z + row * P.zs + h * d + tid) + P.vec[h * d + tid])) : P.vec[h];
    ww = F::exp(lw);
  }
#pragma unroll
  for (int e = 0; e < VEC; ++e) {
    vv[e] = colok ? ldf((const T*)P.v + row * P.vs + h * dv + col + e) : 0.f;
    if (P.silu) vv[e] = silu_<T>(vv[e]);
  }
  wS[tid] = ww;
  kS[tid] = kk;
  rS[tid] = qq * ww;
  const float s = wave_sum(qq * kk);
  if (lane == 0) red[wv] = s;
  __syncthreads();
  const float qk = red[0] + red[1] + red[2] + red[3];
  float o[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) o[e] = 0.f;
#pragma unroll
  for (int m = 0; m < NR; ++m) {
    const float r = rS[(rg + RG * m) & 255];      // (past d: zeros)
#pragma unroll
    for (int e = 0; e < VEC; ++e) o[e] += r * S[m][e];
  }
  if (sp && colok) {
#pragma unroll
    for (int m = 0; m < NR; ++m) {
      const int i = rg + RG * m;
      if (i < d) {
        const float wi = wS[i], ki = kS[i];
        float n[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) n[e] = wi * S[m][e] + ki * vv[e];
        if constexpr (VEC == 4)
          *reinterpret_cast<float4*>(sp + (int64_t)i * dv) = make_float4(n[0], n[1], n[2], n[3]);
        else
          sp[(int64_t)i * dv] = n[0];
      }
    }
  }
#pragma unroll
  for (int x = TL; x < 64; x <<= 1)
#pragma unroll
    for (int e = 0; e < VEC; ++e) o[e] += __shfl_xor(o[e], x, 64);
  if (lane < TL) {
#pragma unroll
    for (int e = 0; e < VEC; ++e) part[wv][c][e] = o[e];
  }
  __syncthreads();
  if (colok && rg == 0) {
    float* op = P.out + row * (int64_t)P.H * dv + h * dv + col;
#pragma unroll
    for (int e = 0; e < VEC; ++e) op[e] = part[0][c][e] + part[1][c][e] + part[2][c][e] + part[3][c][e] + vv[e] * qk;
  }
}

// ---------------------------------------------------------------------------------------------
// Block operands (see the head of the file). Workgroup = (block of a segment, head, segment).
template <typename T, bool CH, int DT>
__global__ void __launch_bounds__(256) linear_prep_kernel(const LinearParams P, float* __restrict__ ws) {
  using F = GateFn<T>;
  constexpr int D = 16 * DT, DS = D + 4;
  __shared__ __attribute__((aligned(16))) float Q[16 * DS], K[16 * DS], C[CH ? 16 * DS : 4];
  __shared__ __attribute__((aligned(16))) float part[4][256];
  const int blk = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int base = P.cu[0];
  const int t0 = P.cu[b], t1 = P.cu[b + 1];
  const int tc = t0 + blk * 16;
  if (tc >= t1) return;
  const int nrow = min(16, t1 - tc);
  const int d = P.d;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int t = tid >> 4, sub = tid & 15;
  const bool live = t < nrow;
  // rows past the segment read its last row, channels past d the first one (no branch around a load, so
  // that all of a thread's loads are in flight together), and count as zeros that do not decay
  const int64_t lrow = live ? tc + t : t1 - 1;
  {
    const T* kp = (const T*)P.k + lrow * P.ks + h * d;
    const T* qp = (const T*)P.q + lrow * P.qs + h * d;
    const T* zp = CH ? (const T*)P.z + lrow * P.zs + h * d : nullptr;
    T kr[DT], qr[DT], zr[CH ? DT : 1];
    float zb[CH ? DT : 1];
#pragma unroll
    for (int m = 0; m < DT; ++m) {
      const int i = sub + 16 * m, ii = i < d ? i : 0;
      kr[m] = kp[ii];
      qr[m] = qp[ii];
      if constexpr (CH) {
        zr[m] = zp[ii];
        zb[m] = P.vec[h * d + ii];
      }
    }
#pragma unroll
    for (int m = 0; m < DT; ++m) {
      const int i = sub + 16 * m;
      const bool ok = live && i < d;
      float kv = ldf(&kr[m]), qv = ldf(&qr[m]);
      if (P.silu) {
        kv = silu_<T>(kv);
        qv = silu_<T>(qv);
      }
      K[t * DS + i] = ok ? kv : 0.f;
      Q[t * DS + i] = ok ? qv * P.q_scale : 0.f;
      if constexpr (CH) C[t * DS + i] = ok ? -P.inv_tau * F::softplus(-(ldf(&zr[m]) + zb[m])) : 0.f;
    }
  }
  __syncthreads();
  bool steep = false;
  if constexpr (CH) {
    float l = 0.f;
    if (tid < D) {       // running sums of the log decays per channel
#pragma unroll
      for (int s = 0; s < 16; ++s) {
        l += C[s * DS + tid];
        C[s * DS + tid] = l;
      }
    }
    steep = __syncthreads_or(l < -SAFE);
  }
  const float lg = CH ? 0.f : P.vec[h];
  auto run = [&](int s) { return lg * (float)min(s + 1, nrow); };      // constant decay: c_s
  const int l15 = lane & 15, hh = lane >> 4;
  float* wp = ws + ((int64_t)((t0 - base) / 16 + b + blk) * P.H + h) * (int64_t)(33 * D + 256);
  f32x4 acc = (f32x4)(0.f);
  for (int j = wv; j < DT; j += 4) {
    const int at = l15 * DS + 16 * j + 4 * hh;       // row l15, channels 16 j + 4 hh ..
    const f32x4 qv = *reinterpret_cast<const f32x4*>(Q + at), kv = *reinterpret_cast<const f32x4*>(K + at);
    f32x4 rv, ko;
    const int ch = 16 * j + l15;
    if constexpr (CH) {
      const f32x4 cv = *reinterpret_cast<const f32x4*>(C + at);
      f32x4 ke;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        rv[r] = qv[r] * F::exp(cv[r]);
        ke[r] = kv[r] * F::exp(steep ? 0.f : -cv[r]);
      }
      if (!steep) {
#pragma unroll
        for (int r = 0; r < 4; ++r) acc = mfma32(rv[r], ke[r], acc);
      }
      const float cE = C[15 * DS + ch];
#pragma unroll
      for (int r = 0; r < 4; ++r) ko[r] = K[(4 * hh + r) * DS + ch] * F::exp(cE - C[(4 * hh + r) * DS + ch]);
      if (hh == 0) wp[32 * D + 256 + ch] = F::exp(cE);
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r) acc = mfma32(qv[r], kv[r], acc);
      rv = qv * F::exp(run(l15));
      const float cE = run(15);
#pragma unroll
      for (int r = 0; r < 4; ++r) ko[r] = K[(4 * hh + r) * DS + ch] * F::exp(cE - run(4 * hh + r));
      if (hh == 0) wp[32 * D + 256 + ch] = F::exp(cE);
    }
    *reinterpret_cast<f32x4*>(wp + (j * 64 + lane) * 4) = rv;
    *reinterpret_cast<f32x4*>(wp + 16 * D + (j * 64 + lane) * 4) = ko;
  }
  // the waves' parts of N, then one entry (row n_t, column n_s) per thread
  if (!steep) *reinterpret_cast<f32x4*>(part[wv] + 4 * lane) = acc;     // part[4 lane + r]: row 4 hh + r, column l15
  __syncthreads();
  const int n_t = tid >> 4, n_s = tid & 15;
  float n = 0.f;
  if (n_s <= n_t) {
    if (steep) {
      if constexpr (CH) {
        for (int i = 0; i < d; ++i)
          n += Q[n_t * DS + i] * K[n_s * DS + i] * F::exp(C[n_t * DS + i] - C[n_s * DS + i]);
      }
    } else {
      const int at = 4 * (16 * (n_t >> 2) + n_s) + (n_t & 3);
      n = part[0][at] + part[1][at] + part[2][at] + part[3][at];
      if (!CH) n *= F::exp(run(n_t) - run(n_s));
    }
  }
  // A operand of N V: lane (row l15, hh), element r = column 4 hh + r
  wp[32 * D + 4 * ((n_s >> 2) * 16 + n_t) + (n_s & 3)] = n;
}

// One wave = 16 value columns of one head of one segment (PASS 0), or of one of the n_split parts of its blocks
// (PASS 1: the state each part adds, PASS 2: the outputs). Up to 8 key tiles the next block's operands are
// loaded into a second register set while the current one is used.
template <typename T, int DT, bool OUT>
struct LinearRegs {
  f32x4 k[DT], p[DT], r[OUT ? DT : 1], n;
  T v[4];      // raw values (converted at their use: a conversion behind the load would wait for it)
};

template <typename T, int DT, int PASS, bool SILU>
__global__ void __launch_bounds__(64) __attribute__((amdgpu_waves_per_eu(1, 1))) linear_walk_kernel(
    const LinearParams P, const float* __restrict__ ws, float* __restrict__ es, float* __restrict__ ps, int n_split) {
  constexpr int D = 16 * DT;
  constexpr bool OUT = PASS != 1;
  const int h = blockIdx.x % P.H, b = blockIdx.x / P.H, tile = blockIdx.y, part = PASS ? blockIdx.z : 0;
  const int lane = threadIdx.x, l15 = lane & 15, hh = lane >> 4;
  const int t0 = P.cu[b], t1 = P.cu[b + 1];
  if (t1 <= t0) return;
  const int nblk = (t1 - t0 + 15) / 16;
  const int per = PASS ? (nblk + n_split - 1) / n_split : nblk;
  const int b0 = part * per, b1 = min(nblk, b0 + per);
  if (b0 >= b1) return;
  if (PASS == 1 && part > 0 && b1 == nblk) return;       // nothing follows the last part
  const int slot = P.slots[b];
  const bool fresh = slot < 0 || P.pos[t0] == 0;
  const int d = P.d, dv = P.dv, col = tile * 16 + l15;
  const bool colok = col < dv;
  float* sp = slot >= 0 ? P.state + ((int64_t)slot * P.H + h) * (int64_t)d * dv + col : nullptr;
  // states of the parts in lane order: entry 0 the segment's first state, entry c > 0 what part c - 1 leaves (part 0
  // from the first state, the others from zero); ps: the parts' whole decays
  float* ep = PASS ? es + (((int64_t)b * P.H + h) * gridDim.y + tile) * n_split * (int64_t)(16 * D) + 4 * lane : nullptr;
  float* pp = PASS ? ps + ((int64_t)b * P.H + h) * n_split * (int64_t)D + 4 * hh : nullptr;
  f32x4 S[DT], pt[PASS == 1 ? DT : 1];
  if (PASS == 2) {
    const float* e = ep + (part ? 16 * D : 0);
#pragma unroll
    for (int i = 0; i < DT; ++i) S[i] = *reinterpret_cast<const f32x4*>(e + 256 * i);
    for (int c = 1; c < part; ++c) {
      e += 16 * D;
#pragma unroll
      for (int i = 0; i < DT; ++i)
        S[i] = S[i] * *reinterpret_cast<const f32x4*>(pp + (int64_t)c * D + 16 * i) + *reinterpret_cast<const f32x4*>(e + 256 * i);
    }
  } else {
    const bool load = !fresh && part == 0 && colok;
#pragma unroll
    for (int i = 0; i < DT; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int ch = 16 * i + 4 * hh + r;
        S[i][r] = (load && ch < d) ? sp[(int64_t)ch * dv] : 0.f;
      }
    if (PASS == 1) {
      if (part == 0) {
#pragma unroll
        for (int i = 0; i < DT; ++i) *reinterpret_cast<f32x4*>(ep + 256 * i) = S[i];
        if (b1 == nblk) return;
      }
#pragma unroll
      for (int i = 0; i < DT; ++i) pt[i] = (f32x4)(1.f);
    }
  }
  const int64_t ent = (int64_t)P.H * (33 * D + 256);       // one block of all heads
  const float* wp = ws + ((int64_t)((t0 - P.cu[0]) / 16 + b) * P.H + h) * (int64_t)(33 * D + 256);
  // no branch around a load (each would wait for all loads in flight): rows past the segment read its
  // last row - the block operands are zero there -, columns past dv the first one, and are not stored
  const T* vp = (const T*)P.v + (int64_t)t0 * P.vs + h * dv + (colok ? col : 0);
  auto load = [&](LinearRegs<T, DT, OUT>& B, int blk) {
    const float* w = wp + blk * ent;
    if constexpr (OUT) {
#pragma unroll
      for (int i = 0; i < DT; ++i) B.r[i] = *reinterpret_cast<const f32x4*>(w + (i * 64 + lane) * 4);
      B.n = *reinterpret_cast<const f32x4*>(w + 32 * D + 4 * lane);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = min(blk * 16 + 4 * hh + r, t1 - t0 - 1);
      B.v[r] = vp[(int64_t)t * P.vs];
    }
#pragma unroll
    for (int i = 0; i < DT; ++i) {
      B.k[i] = *reinterpret_cast<const f32x4*>(w + 16 * D + (i * 64 + lane) * 4);
      B.p[i] = *reinterpret_cast<const f32x4*>(w + 32 * D + 256 + 16 * i + 4 * hh);
    }
  };
  auto step = [&](const LinearRegs<T, DT, OUT>& B, int blk) {
    f32x4 o = (f32x4)(0.f), o2 = (f32x4)(0.f);
    if constexpr (OUT) {
#pragma unroll
      for (int i = 0; i < DT; ++i) {
        o = mfma32(B.r[i][0], S[i][0], o);
        o2 = mfma32(B.r[i][1], S[i][1], o2);
        o = mfma32(B.r[i][2], S[i][2], o);
        o2 = mfma32(B.r[i][3], S[i][3], o2);
      }
    }
#pragma unroll
    for (int i = 0; i < DT; ++i) {
      S[i] *= B.p[i];
      if constexpr (PASS == 1) pt[i] *= B.p[i];
    }
    float v[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      v[r] = ldf(&B.v[r]);
      if constexpr (SILU) v[r] = silu_<T>(v[r]);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      if constexpr (OUT) {
        if (r & 1) o2 = mfma32(B.n[r], v[r], o2);
        else o = mfma32(B.n[r], v[r], o);
      }
#pragma unroll
      for (int i = 0; i < DT; ++i) S[i] = mfma32(B.k[i][r], v[r], S[i]);
    }
    if constexpr (DT <= 8) {
      // the next block's loads (issued in front of this step in program order) between the MFMAs: a
      // wave issues in order, and loads in a row would leave the matrix pipe idle
#pragma unroll
      for (int g = 0; g < (OUT ? 3 * DT + 5 : 2 * DT + 4); ++g) {
        __builtin_amdgcn_sched_group_barrier(0x008, 2, 0);   // MFMA
        __builtin_amdgcn_sched_group_barrier(0x020, 1, 0);   // VMEM read
      }
    }
    if constexpr (OUT) {
      o += o2;
      float* op = P.out + (int64_t)(t0 + blk * 16) * P.H * dv + h * dv + col;
      if (blk * 16 + 16 <= t1 - t0) {
        if (colok) {
#pragma unroll
          for (int r = 0; r < 4; ++r) op[(int64_t)(4 * hh + r) * P.H * dv] = o[r];
        }
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (colok && blk * 16 + 4 * hh + r < t1 - t0) op[(int64_t)(4 * hh + r) * P.H * dv] = o[r];
      }
    }
  };
  if constexpr (DT <= 8) {
    LinearRegs<T, DT, OUT> A, B;
    load(A, b0);
    int blk = b0;
    for (; blk + 1 < b1; blk += 2) {
      load(B, blk + 1);
      step(A, blk);
      load(A, min(blk + 2, b1 - 1));
      step(B, blk + 1);
    }
    if (blk < b1) step(A, blk);
  } else {
    LinearRegs<T, DT, OUT> A;
    for (int blk = b0; blk < b1; ++blk) {
      load(A, blk);
      step(A, blk);
    }
  }
  if (PASS == 1) {
#pragma unroll
    for (int i = 0; i < DT; ++i) {
      *reinterpret_cast<f32x4*>(ep + (int64_t)(part + 1) * (16 * D) + 256 * i) = S[i];
      if (tile == 0 && l15 == 0) *reinterpret_cast<f32x4*>(pp + (int64_t)part * D + 16 * i) = pt[i];
    }
    return;
  }
  if (sp && colok && b1 == nblk) {
#pragma unroll
    for (int i = 0; i < DT; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int ch = 16 * i + 4 * hh + r;
        if (ch < d) sp[(int64_t)ch * dv] = S[i][r];
      }
  }
}

template <typename T, bool CH, int TL, int VEC>
void launch_rows_nr(const LinearParams& P, int n, hipStream_t stream) {
  constexpr int RG = 256 / TL;
  const dim3 grid((unsigned)((P.dv + TL * VEC - 1) / (TL * VEC)), (unsigned)P.H, (unsigned)n);
  const int nr = (P.d + RG - 1) / RG;
  if (nr <= 2)
    linear_rows_kernel<T, CH, TL, VEC, 2><<<grid, 256, 0, stream>>>(P);
  else if (nr <= 4)
    linear_rows_kernel<T, CH, TL, VEC, 4><<<grid, 256, 0, stream>>>(P);
  else if (nr <= 8)
    linear_rows_kernel<T, CH, TL, VEC, 8><<<grid, 256, 0, stream>>>(P);
  else
    linear_rows_kernel<T, CH, TL, VEC, 16><<<grid, 256, 0, stream>>>(P);
}

template <typename T, bool CH>
void launch_rows_t(const LinearParams& P, int n, hipStream_t stream) {
  const bool vec = P.dv % 4 == 0 && ((uintptr_t)P.state % 16) == 0;
  if (vec && P.dv > 32)
    launch_rows_nr<T, CH, 16, 4>(P, n, stream);
  else if (vec)
    launch_rows_nr<T, CH, 8, 4>(P, n, stream);
  else
    launch_rows_nr<T, CH, 16, 1>(P, n, stream);
}

// parts a segment's blocks are walked in: enough waves for every SIMD (256 CUs x 4), at least PART_ROWS rows each;
// fewer than four do not pay for the second pass (measured)
constexpr int PART_ROWS = 128, SIMDS = 1024;
int linear_parts(int waves, int max_q) {
  const int p = SIMDS / (waves > 0 ? waves : 1), q = max_q / PART_ROWS;
  const int n = p < q ? p : q;
  return n < 4 ? 1 : (n > 32 ? 32 : n);
}

template <typename T, int DT, bool SILU>
void launch_walk(const LinearParams& P, float* ws, int64_t entries, int n_seg, int max_q, hipStream_t stream) {
  const int tiles = (P.dv + 15) / 16, parts = linear_parts(n_seg * P.H * tiles, max_q);
  dim3 walk((unsigned)(P.H * n_seg), (unsigned)tiles);
  if (parts == 1) {
    linear_walk_kernel<T, DT, 0, SILU><<<walk, 64, 0, stream>>>(P, ws, nullptr, nullptr, 1);
    return;
  }
  float* es = ws + entries * P.H * (33 * 16 * DT + 256);
  float* ps = es + (int64_t)n_seg * P.H * tiles * parts * (256 * DT);
  walk.z = (unsigned)(parts - 1);
  linear_walk_kernel<T, DT, 1, SILU><<<walk, 64, 0, stream>>>(P, ws, es, ps, parts);
  walk.z = (unsigned)parts;
  linear_walk_kernel<T, DT, 2, SILU><<<walk, 64, 0, stream>>>(P, ws, es, ps, parts);
}

template <typename T, int DT>
void launch_blocks_dt(const LinearParams& P, float* ws, int64_t entries, int n_seg, int max_q, hipStream_t stream) {
  const dim3 grid((unsigned)((max_q + 15) / 16), (unsigned)P.H, (unsigned)n_seg);
  if (P.z)
    linear_prep_kernel<T, true, DT><<<grid, 256, 0, stream>>>(P, ws);
  else
    linear_prep_kernel<T, false, DT><<<grid, 256, 0, stream>>>(P, ws);
  P.silu ? launch_walk<T, DT, true>(P, ws, entries, n_seg, max_q, stream)
         : launch_walk<T, DT, false>(P, ws, entries, n_seg, max_q, stream);
}

template <typename T>
bool launch_blocks_t(const LinearParams& P, float* ws, int64_t entries, int n_seg, int max_q, hipStream_t stream) {
  switch (delta_key_tiles(P.d)) {
#define NGA_LINEAR(N) case N: launch_blocks_dt<T, N>(P, ws, entries, n_seg, max_q, stream); return true;
    NGA_LINEAR(1) NGA_LINEAR(2) NGA_LINEAR(3) NGA_LINEAR(4) NGA_LINEAR(6) NGA_LINEAR(8) NGA_LINEAR(12) NGA_LINEAR(16)
#undef NGA_LINEAR
    default: return false;
  }
}

}  // namespace

void launch_linear_rows(const LinearParams& P, int n, bool f32, hipStream_t stream) {
  if (n == 0) return;
  if (f32)
    P.z ? launch_rows_t<float, true>(P, n, stream) : launch_rows_t<float, false>(P, n, stream);
  else
    P.z ? launch_rows_t<uint16_t, true>(P, n, stream) : launch_rows_t<uint16_t, false>(P, n, stream);
}

// Floats of the workspace of a launch over T rows: block operands, then, when the segments are walked in parts,
// the parts' states and decays.
int64_t linear_workspace(int64_t T, int n_seg, int H, int d, int dv, int max_q) {
  const int64_t D = 16 * delta_key_tiles(d), tiles = (dv + 15) / 16;
  const int64_t parts = linear_parts((int)(n_seg * H * tiles), max_q);
  return (T / 16 + n_seg) * H * (33 * D + 256) + (parts > 1 ? n_seg * H * parts * (tiles * 16 * D + D) : 0);
}

void launch_linear_blocks(const LinearParams& P, float* ws, int64_t T, int n_seg, int max_q, bool f32, hipStream_t stream) {
  if (n_seg == 0 || max_q == 0) return;
  const int64_t entries = T / 16 + n_seg;
  if (!(f32 ? launch_blocks_t<float>(P, ws, entries, n_seg, max_q, stream)
            : launch_blocks_t<uint16_t>(P, ws, entries, n_seg, max_q, stream)))
    abort();   // the binding checks d
}

}  // namespace nga
