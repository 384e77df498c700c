// Delta-rule recurrences with a matrix state per head, carried across steps in state slots.
//
//   mode 0   gated delta rule: one decay g and one step size beta per head and token, unit keys and
//            queries: S <- g S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q
//   mode 1   decay w and removal rate a per key channel, unit key u = k / |k|:
//            S <- diag(w) S - (a u)(u^T S) + k v^T (both terms on the old state), o = S^T r
//
// Both are  S_t = diag(w_t) S_(t-1) + A_t (b_t^T S_(t-1)) + k_t v_t^T,  o_t = S_t^T r_t  with
//   mode 0   w = g, A = -beta g k, b = k, k_t = beta k, r = q d^(-1/2)
//   mode 1   w per channel, A = -a u, b = u, k_t = k, r as projected.
//
// delta_rows: launches whose segments are single rows. One pass over the state of a head: with
// y = b^T S and z = (r w)^T S (one reduction), o = z + y (r . A) + v (r . k_t), then the update.
//
// delta_prep + delta_walk: portions, in blocks of 16 rows. With P_t the running product of the
// decays inside a block (P_0 = 1), S_t = diag(P_t) Z_t turns the block into matrix products:
//   c_t = b_t P_(t-1), rho_t = r_t P_t, alpha_t = A_t / P_t, kappa_t = k_t / P_t
//   Y = C Z_0 + L_A Y + L_K V   (L_A, L_K: strictly lower parts of C alpha^T and C kappa^T)
//   O = R Z_0 + G_A Y + G_K V   (lower parts of R alpha^T and R kappa^T)
//   S_16 = diag(P_16) (Z_0 + alpha^T Y + kappa^T V)
// and with T = (I - L_A)^(-1), M = T L_K everything that does not depend on the state is folded
// ahead of time, one workgroup per (block, head):
//   C' = T C, R' = R + G_A C', N = G_K + G_A M, alpha' = alpha P_16, kappa' = kappa P_16 + M^T alpha'
// so that the walk over the blocks of a segment is
//   Y' = C' S, O = R' S + N V, S <- diag(P_16) S + alpha'^T Y' + kappa'^T V.
// In mode 0 the decays are scalars of any size and enter as differences of logarithms (never above
// 0) on the products; in mode 1 they divide the vectors (a block's decays are bounded: 16 rows of
// exp(-decay), decay <= 4).
//
// All products run on mfma_f32_16x16x4_f32 (true fp32). The operands lie in the workspace in the
// order a lane needs them: a k-slot of step r is index 4 h + r (h = lane / 16), so an A operand of
// four steps is one float4 per lane, and accumulators (row 4 h + r, column lane % 16) are B operands of
// the next product without moving between lanes: a wave keeps its 16 value columns of the state
// in registers for the whole segment and needs neither LDS nor barriers.
//
// Workspace of (block, head), DT = tiles of 16 key channels: C' [DT][64][4], R' [DT][64][4],
// alpha'^T [DT][64][4], kappa'^T [DT][64][4], N [64][4], P_16 [16 DT]. Block c of segment b is entry
// cu[b] / 16 + b + c (cu counted from the launch's first row).
#include "common.h"
#include "gate_fn.h"
#include "kernels.h"

namespace nga {

namespace {

// ---------------------------------------------------------------------------------------------
// Single rows. Workgroup = (value tile of TL * VEC columns, head, row); thread (rg, c) keeps rows
// rg + RG m (m < NR) of columns VEC c .. of the state.
template <typename T, int MODE, int TL, int VEC, int NR>
__global__ void __launch_bounds__(256) delta_rows_kernel(const DeltaParams P) {
  using F = GateFn<T>;
  constexpr int RG = 256 / TL;
  __shared__ float wS[256], aS[256], bS[256], kS[256], rS[256];
  __shared__ float red[4][3];
  __shared__ float part[4][TL][2 * VEC];
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
  float kk = 0.f, rr = 0.f, aa = 0.f, ww = 1.f, vv[VEC];
  if (tid < d) {
    const int g = MODE == 0 ? h / (P.H / P.G) : h;
    kk = ldf((const T*)P.k + row * P.ks + g * d + tid);
    rr = ldf((const T*)P.q + row * P.qs + g * d + tid);
    if (MODE == 1) {
      aa = F::sigmoid(ldf((const T*)P.b + row * P.bs + h * d + tid) + P.b_vec[h * d + tid]);
      ww = F::exp(-P.decay * F::sigmoid(ldf((const T*)P.w + row * P.ws + h * d + tid) + P.w_vec[h * d + tid]));
    }
  }
#pragma unroll
  for (int e = 0; e < VEC; ++e) vv[e] = colok ? ldf((const T*)P.v + row * P.vs + h * dv + col + e) : 0.f;
  {
    const float s0 = wave_sum(kk * kk);
    const float s1 = wave_sum(MODE == 0 ? rr * rr : rr * aa * kk);
    const float s2 = wave_sum(rr * kk);
    if (lane == 0) {
      red[wv][0] = s0;
      red[wv][1] = s1;
      red[wv][2] = s2;
    }
  }
  __syncthreads();
  const float s0 = red[0][0] + red[1][0] + red[2][0] + red[3][0];
  const float s1 = red[0][1] + red[1][1] + red[2][1] + red[3][1];
  const float s2 = red[0][2] + red[1][2] + red[2][2] + red[3][2];
  const float ik = 1.0f / sqrtf(s0 + 1e-6f);
  float rA, rK;      // r . A and r . k_t
  if (MODE == 0) {
    const float iq = 1.0f / sqrtf(s1 + 1e-6f) / sqrtf((float)d);
    const float beta = F::sigmoid(ldf((const T*)P.b + row * P.bs + h));
    const float g = F::exp(-F::exp(P.w_vec[h]) * F::softplus(ldf((const T*)P.w + row * P.ws + h) + P.b_vec[h]));
    rK = beta * s2 * ik * iq;
    rA = -g * rK;
    kk *= ik;
    wS[tid] = g;
    bS[tid] = kk;
    aS[tid] = -beta * g * kk;
    kS[tid] = beta * kk;
    rS[tid] = rr * iq;
  } else {
    rK = s2;
    rA = -s1 * ik;
    wS[tid] = ww;
    bS[tid] = kk * ik;
    aS[tid] = -aa * kk * ik;
    kS[tid] = kk;
    rS[tid] = rr;
  }
  __syncthreads();
  float y[VEC], z[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) y[e] = z[e] = 0.f;
#pragma unroll
  for (int m = 0; m < NR; ++m) {
    const int i = rg + RG * m;      // (RG NR can exceed 256 only past d: those rows are zeros)
    const float bi = bS[i & 255], rw = rS[i & 255] * wS[i & 255];
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      y[e] += bi * S[m][e];
      z[e] += rw * S[m][e];
    }
  }
#pragma unroll
  for (int o = TL; o < 64; o <<= 1)
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      y[e] += __shfl_xor(y[e], o, 64);
      z[e] += __shfl_xor(z[e], o, 64);
    }
  if (lane < TL) {
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      part[wv][c][e] = y[e];
      part[wv][c][VEC + e] = z[e];
    }
  }
  __syncthreads();
#pragma unroll
  for (int e = 0; e < VEC; ++e) {
    y[e] = part[0][c][e] + part[1][c][e] + part[2][c][e] + part[3][c][e];
    z[e] = part[0][c][VEC + e] + part[1][c][VEC + e] + part[2][c][VEC + e] + part[3][c][VEC + e];
  }
  if (!colok) return;
  if (rg == 0) {
    float* op = P.out + row * (int64_t)P.H * dv + h * dv + col;
#pragma unroll
    for (int e = 0; e < VEC; ++e) op[e] = z[e] + y[e] * rA + vv[e] * rK;
  }
  if (sp) {
#pragma unroll
    for (int m = 0; m < NR; ++m) {
      const int i = rg + RG * m;
      if (i < d) {
        const float wi = wS[i], ai = aS[i], ki = kS[i];
        float s[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) s[e] = wi * S[m][e] + ai * y[e] + ki * vv[e];
        if constexpr (VEC == 4)
          *reinterpret_cast<float4*>(sp + (int64_t)i * dv) = make_float4(s[0], s[1], s[2], s[3]);
        else
          sp[(int64_t)i * dv] = s[0];
      }
    }
  }
}

// ---------------------------------------------------------------------------------------------
// Block operands (see the head of the file). Workgroup = (block of a segment, head, segment).
constexpr int ML = 20;    // row stride of the 16 x 16 matrices in LDS

template <typename T, int MODE, int DT>
__global__ void __launch_bounds__(256) delta_prep_kernel(const DeltaParams P, float* __restrict__ ws) {
  using F = GateFn<T>;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ __attribute__((aligned(16))) float LA[16 * ML], LK[16 * ML], GA[16 * ML], GK[16 * ML], Tm[16 * ML];
  __shared__ float cl[16], beta_s[16];
  const int blk = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int base = P.cu[0];
  const int t0 = P.cu[b], t1 = P.cu[b + 1];
  const int tc = t0 + blk * 16;
  if (tc >= t1) return;
  const int nrow = min(16, t1 - tc);
  constexpr int D = 16 * DT, DS = D + 4;
  const int d = P.d;
  // mode 0: rows K, Q; mode 1: rows C, R, alpha, kappa, running log decays, then P_16
  float* X0 = lds;
  float* X1 = lds + 16 * DS;
  float* X2 = lds + 32 * DS;
  float* X3 = lds + 48 * DS;
  float* X4 = lds + 64 * DS;
  float* pc = lds + 80 * DS;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int t = tid >> 4, sub = tid & 15;
  const int64_t row = tc + t;
  const bool live = t < nrow;
  // rows past the segment read its last row, channels past d the first one (no branch around a load, so
  // that all of a thread's loads are in flight together), and count as zeros
  const int64_t lrow = live ? row : t1 - 1;
  if (MODE == 0) {
    const int g = h / (P.H / P.G);
    const T* kp = (const T*)P.k + lrow * P.ks + g * d;
    const T* qp = (const T*)P.q + lrow * P.qs + g * d;
    T kr[DT], qr[DT];
#pragma unroll
    for (int m = 0; m < DT; ++m) {
      const int i = sub + 16 * m, ii = i < d ? i : 0;
      kr[m] = kp[ii];
      qr[m] = qp[ii];
    }
    float kf[DT], qf[DT], sk = 0.f, sq = 0.f;
#pragma unroll
    for (int m = 0; m < DT; ++m) {
      const bool ok = live && sub + 16 * m < d;
      kf[m] = ok ? ldf(&kr[m]) : 0.f;
      qf[m] = ok ? ldf(&qr[m]) : 0.f;
      sk += kf[m] * kf[m];
      sq += qf[m] * qf[m];
    }
#pragma unroll
    for (int o = 8; o > 0; o >>= 1) {
      sk += __shfl_xor(sk, o, 64);
      sq += __shfl_xor(sq, o, 64);
    }
    const float ik = 1.0f / sqrtf(sk + 1e-6f), iq = 1.0f / sqrtf(sq + 1e-6f) / sqrtf((float)d);
#pragma unroll
    for (int m = 0; m < DT; ++m) {
      X0[t * DS + sub + 16 * m] = kf[m] * ik;
      X1[t * DS + sub + 16 * m] = qf[m] * iq;
    }
    if (tid < 16) {      // running log decay and step size of the block's rows, one row per lane
      const int64_t r2 = tc + tid;
      float lg = 0.f, be = 0.f;
      if (tid < nrow) {
        be = F::sigmoid(ldf((const T*)P.b + r2 * P.bs + h));
        lg = -F::exp(P.w_vec[h]) * F::softplus(ldf((const T*)P.w + r2 * P.ws + h) + P.b_vec[h]);
      }
#pragma unroll
      for (int o = 1; o < 16; o <<= 1) {
        const float up = __shfl_up(lg, o, 16);
        if (tid >= o) lg += up;
      }
      cl[tid] = lg;
      beta_s[tid] = be;
    }
    __syncthreads();
  } else {
    const T* kp = (const T*)P.k + lrow * P.ks + h * d;
    const T* qp = (const T*)P.q + lrow * P.qs + h * d;
    const T* bp = (const T*)P.b + lrow * P.bs + h * d;
    const T* wq = (const T*)P.w + lrow * P.ws + h * d;
    T kr[DT], qr[DT], br[DT], wr[DT];
    float bb[DT], wb[DT];
#pragma unroll
    for (int m = 0; m < DT; ++m) {
      const int i = sub + 16 * m, ii = i < d ? i : 0;
      kr[m] = kp[ii];
      qr[m] = qp[ii];
      br[m] = bp[ii];
      wr[m] = wq[ii];
      bb[m] = P.b_vec[h * d + ii];
      wb[m] = P.w_vec[h * d + ii];
    }
    float kf[DT], sk = 0.f;
#pragma unroll
    for (int m = 0; m < DT; ++m) {
      const int i = sub + 16 * m;
      const bool ok = live && i < d;
      kf[m] = ok ? ldf(&kr[m]) : 0.f;
      sk += kf[m] * kf[m];
      X1[t * DS + i] = ok ? ldf(&qr[m]) : 0.f;
      X2[t * DS + i] = ok ? F::sigmoid(ldf(&br[m]) + bb[m]) : 0.f;
      X4[t * DS + i] = ok ? -P.decay * F::sigmoid(ldf(&wr[m]) + wb[m]) : 0.f;
    }
#pragma unroll
    for (int o = 8; o > 0; o >>= 1) sk += __shfl_xor(sk, o, 64);
    const float ik = 1.0f / sqrtf(sk + 1e-6f);
    __syncthreads();
    if (tid < D) {       // running sums of the log decays per channel
      float l[16];
#pragma unroll
      for (int s = 0; s < 16; ++s) l[s] = X4[s * DS + tid];
#pragma unroll
      for (int s = 1; s < 16; ++s) {
        l[s] += l[s - 1];
        X4[s * DS + tid] = l[s];
      }
      pc[tid] = F::exp(l[15]);
    }
    __syncthreads();
#pragma unroll
    for (int m = 0; m < DT; ++m) {
      const int i = sub + 16 * m;
      const float c1 = X4[t * DS + i], c0 = t > 0 ? X4[(t - 1) * DS + i] : 0.f;
      const float kv = kf[m], u = kv * ik, down = F::exp(-c1);
      X0[t * DS + i] = u * F::exp(c0);
      X1[t * DS + i] *= F::exp(c1);
      X2[t * DS + i] *= -u * down;
      X3[t * DS + i] = kv * down;
    }
    __syncthreads();
  }
  // products of the block's rows: one 16 x 16 matrix per wave (mode 0: waves 0 and 1)
  const int l15 = lane & 15, hh = lane >> 4;
  if (MODE == 1 || wv < 2) {
    const float* Ar = MODE == 0 ? (wv == 0 ? X0 : X1) : (wv < 2 ? X0 : X1);
    const float* Br = MODE == 0 ? X0 : ((wv & 1) ? X3 : X2);
    f32x4 acc0 = (f32x4)(0.f), acc1 = (f32x4)(0.f);
#pragma unroll
    for (int i = 0; i < DT; ++i) {
      const f32x4 av = *reinterpret_cast<const f32x4*>(Ar + l15 * DS + 16 * i + 4 * hh);
      const f32x4 bv = *reinterpret_cast<const f32x4*>(Br + l15 * DS + 16 * i + 4 * hh);
      acc0 = mfma32(av[0], bv[0], acc0);
      acc1 = mfma32(av[1], bv[1], acc1);
      acc0 = mfma32(av[2], bv[2], acc0);
      acc1 = mfma32(av[3], bv[3], acc1);
    }
    acc0 += acc1;
#pragma unroll
    for (int r = 0; r < 4; ++r) {     // entry (row tt, column s) of the product
      const int tt = 4 * hh + r, s = l15, at = tt * ML + s;
      if (MODE == 1) {
        float* M = wv == 0 ? LA : wv == 1 ? LK : wv == 2 ? GA : GK;
        M[at] = (wv < 2 ? s < tt : s <= tt) ? acc0[r] : 0.f;
      } else {
        const float ct = wv == 0 ? (tt > 0 ? cl[tt - 1] : 0.f) : cl[tt];     // log decay in front of the row's read-out
        const float cs = cl[s], cp = s > 0 ? cl[s - 1] : 0.f;
        const bool in = wv == 0 ? s < tt : s <= tt;
        const float v = acc0[r] * beta_s[s];
        (wv == 0 ? LA : GA)[at] = in ? -v * F::exp(ct - cp) : 0.f;
        (wv == 0 ? LK : GK)[at] = in ? v * F::exp(ct - cs) : 0.f;
      }
    }
  }
  __syncthreads();
  if (tid < 16) {     // T = (I - L_A)^(-1), one column per lane by forward substitution
    float x[16];
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      float a = r == tid ? 1.f : 0.f;
#pragma unroll
      for (int s = 0; s < r; ++s) a += LA[r * ML + s] * x[s];
      x[r] = a;
      Tm[r * ML + tid] = a;
    }
  }
  __syncthreads();
  const f32x4 trow = *reinterpret_cast<const f32x4*>(Tm + l15 * ML + 4 * hh);      // T[l15][4 hh + r]
  const f32x4 garow = *reinterpret_cast<const f32x4*>(GA + l15 * ML + 4 * hh);
  f32x4 M = (f32x4)(0.f), qt = (f32x4)(0.f);     // M[4 hh + r][l15]; (G_A T)[l15][4 hh + r]
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    M = mfma32(trow[r], LK[(4 * hh + r) * ML + l15], M);
    qt = mfma32(Tm[(4 * hh + r) * ML + l15], garow[r], qt);
  }
  float* wp = ws + ((int64_t)((t0 - base) / 16 + b + blk) * P.H + h) * (int64_t)(65 * D + 256);
  if (wv == 0) {
    f32x4 n = *reinterpret_cast<const f32x4*>(GK + l15 * ML + 4 * hh);
#pragma unroll
    for (int r = 0; r < 4; ++r) n = mfma32(M[r], garow[r], n);
    *reinterpret_cast<f32x4*>(wp + 64 * D + 4 * lane) = n;
  }
  float sC[4], sA[4], sK[4], sR = 1.f, pC = 1.f;      // mode 0: factors of the rows
  if (MODE == 0) {
    const float cE = cl[15];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int s = 4 * hh + r;
      const float cp = s > 0 ? cl[s - 1] : 0.f;
      sC[r] = F::exp(cp);
      sA[r] = -beta_s[s] * F::exp(cE - cp);
      sK[r] = beta_s[s] * F::exp(cE - cl[s]);
    }
    sR = F::exp(cl[l15]);
    pC = F::exp(cE);
  }
  for (int j = wv; j < DT; j += 4) {
    const int ch = 16 * j + l15;
    f32x4 cT, aT, kT;
    const float pj = MODE == 1 ? pc[ch] : 1.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int at = (4 * hh + r) * DS + ch;
      if (MODE == 0) {
        const float kv = X0[at];
        cT[r] = kv * sC[r];
        aT[r] = kv * sA[r];
        kT[r] = kv * sK[r];
      } else {
        cT[r] = X0[at];
        aT[r] = X2[at] * pj;
        kT[r] = X3[at] * pj;
      }
    }
    f32x4 co = (f32x4)(0.f);
    f32x4 ro = *reinterpret_cast<const f32x4*>(X1 + l15 * DS + 16 * j + 4 * hh);
    if (MODE == 0) ro *= sR;
    f32x4 ko = kT;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      co = mfma32(cT[r], trow[r], co);
      ro = mfma32(cT[r], qt[r], ro);
      ko = mfma32(M[r], aT[r], ko);
    }
    *reinterpret_cast<f32x4*>(wp + (j * 64 + lane) * 4) = co;
    *reinterpret_cast<f32x4*>(wp + 16 * D + (j * 64 + lane) * 4) = ro;
    *reinterpret_cast<f32x4*>(wp + 32 * D + (j * 64 + lane) * 4) = aT;
    *reinterpret_cast<f32x4*>(wp + 48 * D + (j * 64 + lane) * 4) = ko;
    if (hh == 0) wp[64 * D + 256 + ch] = MODE == 0 ? pC : pj;
  }
}

// One wave = 16 value columns of one head of one segment, over all its blocks. Up to 8 key tiles the
// next block's operands are loaded into a second register set while the current one is used.
template <typename T, int DT>
struct BlockRegs {
  f32x4 c[DT], r[DT], a[DT], k[DT], p[DT], n;
  T v[4];      // raw values (converted at their use: a conversion behind the load would wait for it)
};

template <typename T, int DT>
__global__ void __launch_bounds__(64) __attribute__((amdgpu_waves_per_eu(1, 1))) delta_walk_kernel(
    const DeltaParams P, const float* __restrict__ ws) {
  constexpr int D = 16 * DT;
  const int h = blockIdx.x % P.H, b = blockIdx.x / P.H, tile = blockIdx.y;
  const int lane = threadIdx.x, l15 = lane & 15, hh = lane >> 4;
  const int t0 = P.cu[b], t1 = P.cu[b + 1];
  if (t1 <= t0) return;
  const int slot = P.slots[b];
  const bool fresh = slot < 0 || P.pos[t0] == 0;
  const int d = P.d, dv = P.dv, col = tile * 16 + l15;
  const bool colok = col < dv;
  float* sp = slot >= 0 ? P.state + ((int64_t)slot * P.H + h) * (int64_t)d * dv + col : nullptr;
  f32x4 S[DT];
#pragma unroll
  for (int i = 0; i < DT; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int ch = 16 * i + 4 * hh + r;
      S[i][r] = (!fresh && colok && ch < d) ? sp[(int64_t)ch * dv] : 0.f;
    }
  const int64_t ent = (int64_t)P.H * (65 * D + 256);       // one block of all heads
  const float* wp = ws + ((int64_t)((t0 - P.cu[0]) / 16 + b) * P.H + h) * (int64_t)(65 * D + 256);
  // no branch around a load (each would wait for all loads in flight): rows past the segment read its
  // last row - the block operands are zero there -, columns past dv the first one, and are not stored
  const T* vp = (const T*)P.v + (int64_t)t0 * P.vs + h * dv + (colok ? col : 0);
  auto load = [&](BlockRegs<T, DT>& B, int blk) {
    const float* w = wp + blk * ent;
#pragma unroll
    for (int i = 0; i < DT; ++i) {
      B.c[i] = *reinterpret_cast<const f32x4*>(w + (i * 64 + lane) * 4);
      B.r[i] = *reinterpret_cast<const f32x4*>(w + 16 * D + (i * 64 + lane) * 4);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = min(blk * 16 + 4 * hh + r, t1 - t0 - 1);
      B.v[r] = vp[(int64_t)t * P.vs];
    }
    B.n = *reinterpret_cast<const f32x4*>(w + 64 * D + 4 * lane);
#pragma unroll
    for (int i = 0; i < DT; ++i) {
      B.a[i] = *reinterpret_cast<const f32x4*>(w + 32 * D + (i * 64 + lane) * 4);
      B.k[i] = *reinterpret_cast<const f32x4*>(w + 48 * D + (i * 64 + lane) * 4);
      B.p[i] = *reinterpret_cast<const f32x4*>(w + 64 * D + 256 + 16 * i + 4 * hh);
    }
  };
  auto step = [&](const BlockRegs<T, DT>& B, int blk) {
    f32x4 y = (f32x4)(0.f), o = (f32x4)(0.f);
#pragma unroll
    for (int i = 0; i < DT; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        y = mfma32(B.c[i][r], S[i][r], y);
        o = mfma32(B.r[i][r], S[i][r], o);
      }
#pragma unroll
    for (int i = 0; i < DT; ++i) S[i] *= B.p[i];
    float v[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] = ldf(&B.v[r]);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      o = mfma32(B.n[r], v[r], o);
#pragma unroll
      for (int i = 0; i < DT; ++i) S[i] = mfma32(B.k[i][r], v[r], S[i]);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int i = 0; i < DT; ++i) S[i] = mfma32(B.a[i][r], y[r], S[i]);
    if constexpr (DT <= 8) {
      // the next block's loads (issued in front of this step in program order) between the MFMAs: a
      // wave issues in order, and loads in a row would leave the matrix pipe idle
#pragma unroll
      for (int g = 0; g < 5 * DT + 5; ++g) {
        __builtin_amdgcn_sched_group_barrier(0x008, 2, 0);   // MFMA
        __builtin_amdgcn_sched_group_barrier(0x020, 1, 0);   // VMEM read
      }
    }
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
  };
  const int nblk = (t1 - t0 + 15) / 16;
  if constexpr (DT <= 8) {
    BlockRegs<T, DT> A, B;
    load(A, 0);
    int blk = 0;
    for (; blk + 1 < nblk; blk += 2) {
      load(B, blk + 1);
      step(A, blk);
      load(A, min(blk + 2, nblk - 1));
      step(B, blk + 1);
    }
    if (blk < nblk) step(A, blk);
  } else {
    BlockRegs<T, DT> A;
    for (int blk = 0; blk < nblk; ++blk) {
      load(A, blk);
      step(A, blk);
    }
  }
  if (sp && colok) {
#pragma unroll
    for (int i = 0; i < DT; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int ch = 16 * i + 4 * hh + r;
        if (ch < d) sp[(int64_t)ch * dv] = S[i][r];
      }
  }
}

template <typename T, int MODE, int TL, int VEC>
void launch_rows_nr(const DeltaParams& P, int n, hipStream_t stream) {
  constexpr int RG = 256 / TL;
  const dim3 grid((unsigned)((P.dv + TL * VEC - 1) / (TL * VEC)), (unsigned)P.H, (unsigned)n);
  const int nr = (P.d + RG - 1) / RG;
  if (nr <= 2)
    delta_rows_kernel<T, MODE, TL, VEC, 2><<<grid, 256, 0, stream>>>(P);
  else if (nr <= 4)
    delta_rows_kernel<T, MODE, TL, VEC, 4><<<grid, 256, 0, stream>>>(P);
  else if (nr <= 8)
    delta_rows_kernel<T, MODE, TL, VEC, 8><<<grid, 256, 0, stream>>>(P);
  else
    delta_rows_kernel<T, MODE, TL, VEC, 16><<<grid, 256, 0, stream>>>(P);
}

template <typename T, int MODE>
void launch_rows_t(const DeltaParams& P, int n, hipStream_t stream) {
  const bool vec = P.dv % 4 == 0 && ((uintptr_t)P.state % 16) == 0;
  if (vec && P.dv > 32)
    launch_rows_nr<T, MODE, 16, 4>(P, n, stream);
  else if (vec)
    launch_rows_nr<T, MODE, 8, 4>(P, n, stream);
  else
    launch_rows_nr<T, MODE, 16, 1>(P, n, stream);
}

template <typename T>
bool launch_walk_t(const DeltaParams& P, const float* ws, int dt, int n_seg, hipStream_t stream) {
  const dim3 grid((unsigned)(P.H * n_seg), (unsigned)((P.dv + 15) / 16));
  switch (dt) {
#define NGA_WALK(N) case N: delta_walk_kernel<T, N><<<grid, 64, 0, stream>>>(P, ws); return true;
    NGA_WALK(1) NGA_WALK(2) NGA_WALK(3) NGA_WALK(4) NGA_WALK(6) NGA_WALK(8) NGA_WALK(12) NGA_WALK(16)
#undef NGA_WALK
    default: return false;
  }
}

template <typename T, int MODE, int DT>
void launch_prep_dt(const DeltaParams& P, float* ws, dim3 grid, hipStream_t stream) {
  constexpr int D = 16 * DT;
  constexpr size_t smem = (size_t)((MODE == 0 ? 32 : 80) * (D + 4) + (MODE == 0 ? 0 : D)) * sizeof(float);
  static bool attr_set = false;
  if (smem > 49152 && !attr_set) {     // (with the static part above the default limit: the attribute once)
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&delta_prep_kernel<T, MODE, DT>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
    attr_set = true;
  }
  delta_prep_kernel<T, MODE, DT><<<grid, 256, smem, stream>>>(P, ws);
}

template <typename T, int MODE>
void launch_prep_t(const DeltaParams& P, float* ws, int dt, int n_seg, int max_q, hipStream_t stream) {
  const dim3 grid((unsigned)((max_q + 15) / 16), (unsigned)P.H, (unsigned)n_seg);
  switch (dt) {
#define NGA_PREP(N) case N: launch_prep_dt<T, MODE, N>(P, ws, grid, stream); return;
    NGA_PREP(1) NGA_PREP(2) NGA_PREP(3) NGA_PREP(4) NGA_PREP(6) NGA_PREP(8) NGA_PREP(12) NGA_PREP(16)
#undef NGA_PREP
    default: return;      // (the walk's launch reports a size that is not compiled)
  }
}

}  // namespace

// key tiles of 16 a head of d channels takes (sizes the walk kernel is compiled for); 0: too wide
int delta_key_tiles(int d) {
  static const int sizes[] = {1, 2, 3, 4, 6, 8, 12, 16};
  for (int s : sizes)
    if (d <= 16 * s) return s;
  return 0;
}

void launch_delta_rows(const DeltaParams& P, int n, bool f32, hipStream_t stream) {
  if (n == 0) return;
  if (f32)
    P.mode == 0 ? launch_rows_t<float, 0>(P, n, stream) : launch_rows_t<float, 1>(P, n, stream);
  else
    P.mode == 0 ? launch_rows_t<uint16_t, 0>(P, n, stream) : launch_rows_t<uint16_t, 1>(P, n, stream);
}

// ws: (rows / 16 + n_seg) * H * (65 * 16 * delta_key_tiles(d) + 256) floats, 16-byte aligned
void launch_delta_blocks(const DeltaParams& P, float* ws, int n_seg, int max_q, bool f32, hipStream_t stream) {
  if (n_seg == 0 || max_q == 0) return;
  const int dt = delta_key_tiles(P.d);
  bool ok;
  if (f32) {
    P.mode == 0 ? launch_prep_t<float, 0>(P, ws, dt, n_seg, max_q, stream)
                : launch_prep_t<float, 1>(P, ws, dt, n_seg, max_q, stream);
    ok = launch_walk_t<float>(P, ws, dt, n_seg, stream);
  } else {
    P.mode == 0 ? launch_prep_t<uint16_t, 0>(P, ws, dt, n_seg, max_q, stream)
                : launch_prep_t<uint16_t, 1>(P, ws, dt, n_seg, max_q, stream);
    ok = launch_walk_t<uint16_t>(P, ws, dt, n_seg, stream);
  }
  if (!ok) abort();   // the binding checks d
}

}  // namespace nga
