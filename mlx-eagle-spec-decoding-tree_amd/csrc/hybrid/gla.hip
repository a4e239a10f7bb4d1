// Gated linear attention with a decay per key channel:
//   S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,  o_t = S_t^T (q_t dim^-1/2),
//   alpha = sigmoid(z)^(1/tau),  result = rms_norm(o) * w * silu(gate)  per head.
// Everything of the recurrence is fp32, matrix products included.
//
// One to a few rows: one workgroup per head walks the rows with the state in registers.
// A prompt portion: chunks of 64 rows in four sub-chunks of 16.  With L the running sum of
// log alpha inside a sub-chunk and T its total, every factor used is exp of a sum of such terms
// that is never positive, whatever the decays are:
//   (1) per chunk: A[i][j] = sum_d q_id k_jd exp(decay from j to i), U = sum_j k_j v_j^T decayed to the
//       chunk's end, and the chunk's total decay;
//   (2) a scan over the chunks turns U into the state before each chunk and leaves the last state;
//   (3) per chunk: o = (q decayed from the chunk's start) S + A V, then norm and gate.
#include "hybrid.h"

#include <math.h>

namespace {

constexpr int CH = HYB_GLA_CHUNK, SUBC = 16;

// ------------------------------------------------------------------------------------
// Few rows.
// ------------------------------------------------------------------------------------
struct StepP {
  const void* x;           // projections [R][ldx]: q, k, v, gate, a1 at their offsets
  const void* a2;          // [H dkp][rp]
  const float* a2_bias;    // [H dkp]
  const float* norm_w;     // [dvp]
  float* state;            // [H][dkp][dvp]
  void* out;
  const int32_t* n_dev;
  long ldx, ldo;
  int R, H, dkp, dvp, rp, dv_true, oq, ok, ov, og, oa;
  float qscale, inv_tau, eps;
};

// ND: state rows per thread kept in registers (0: any number, the state stays in memory)
template <typename T, int ND>
__global__ __launch_bounds__(1024) void gla_step_kernel(StepP p) {
  extern __shared__ __align__(16) float sm[];
  float* part = sm;                       // [TY][dvp] = 4 * threads
  float* qs = part + 4 * blockDim.x;      // [dkp] x 3: q, k, alpha
  float* ks = qs + p.dkp;
  float* as = ks + p.dkp;
  __shared__ float red[16];
  const int h = blockIdx.x, tid = threadIdx.x;
  const int live = hyb_live(p.n_dev, p.R);
  if (live == 0) return;
  const int NV = p.dvp >> 2, TY = blockDim.x / NV;
  const int ty = tid / NV, tx = tid % NV;
  const bool work = ty < TY;
  float* st = p.state + (size_t)h * p.dkp * p.dvp + tx * 4;
  f32x4_t s[ND > 0 ? ND : 1];
  if (ND > 0) {
#pragma unroll
    for (int i = 0; i < ND; ++i) {
      const int d = ty + i * TY;
      s[i] = work && d < p.dkp ? load4(st + (size_t)d * p.dvp) : f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
  }
  for (int r = 0; r < live; ++r) {
    const T* x = reinterpret_cast<const T*>(p.x) + (size_t)r * p.ldx;
    // gate of the recurrence: eight lanes per key channel
    for (int d0 = 0; d0 < p.dkp; d0 += blockDim.x >> 3) {
      const int d = d0 + (tid >> 3);
      if (d < p.dkp) {
        const T* a2 = reinterpret_cast<const T*>(p.a2) + ((size_t)h * p.dkp + d) * p.rp;
        float z = 0.f;
        for (int c = (tid & 7) * 8; c < p.rp; c += 64) {
          const Frag<T> w = Frag<T>::load(a2 + c), a = Frag<T>::load(x + p.oa + c);
#pragma unroll
          for (int e = 0; e < 8; ++e) z = fmaf(w.at(e), a.at(e), z);
        }
        z += __shfl_xor(z, 1, 64);
        z += __shfl_xor(z, 2, 64);
        z += __shfl_xor(z, 4, 64);
        if ((tid & 7) == 0) {
          z += p.a2_bias[(size_t)h * p.dkp + d];
          as[d] = expf(hyb_log_sigmoid(z) * p.inv_tau);
          qs[d] = (float)x[p.oq + h * p.dkp + d] * p.qscale;
          ks[d] = (float)x[p.ok + h * p.dkp + d];
        }
      }
    }
    __syncthreads();
    f32x4_t o = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (work) {
      const f32x4_t v = load4(x + p.ov + h * p.dvp + tx * 4);
      if (ND > 0) {
#pragma unroll
        for (int i = 0; i < ND; ++i) {
          const int d = ty + i * TY;
          if (d < p.dkp) {
            s[i] = s[i] * as[d] + v * ks[d];
            o += s[i] * qs[d];
          }
        }
      } else {
        for (int d = ty; d < p.dkp; d += TY) {
          f32x4_t c = load4(st + (size_t)d * p.dvp);
          c = c * as[d] + v * ks[d];
          *reinterpret_cast<f32x4_t*>(st + (size_t)d * p.dvp) = c;
          o += c * qs[d];
        }
      }
      *reinterpret_cast<f32x4_t*>(part + (size_t)ty * p.dvp + tx * 4) = o;
    }
    __syncthreads();
    float ov = 0.f;
    if (tid < p.dvp)
      for (int y = 0; y < TY; ++y) ov += part[(size_t)y * p.dvp + tid];
    float ss = hyb_wave_sum(ov * ov);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    ss = 0.f;
    for (int i = 0; i < (int)(blockDim.x >> 6); ++i) ss += red[i];
    if (tid < p.dvp) {
      const float rstd = 1.f / sqrtf(ss / (float)p.dv_true + p.eps);
      const float gt = (float)x[p.og + h * p.dvp + tid];
      reinterpret_cast<T*>(p.out)[(size_t)r * p.ldo + h * p.dvp + tid] = (T)(ov * rstd * p.norm_w[tid] * gt * hyb_sigmoid(gt));
    }
    __syncthreads();
  }
  if (ND > 0 && work) {
#pragma unroll
    for (int i = 0; i < ND; ++i) {
      const int d = ty + i * TY;
      if (d < p.dkp) *reinterpret_cast<f32x4_t*>(st + (size_t)d * p.dvp) = s[i];
    }
  }
}

// ------------------------------------------------------------------------------------
// Prompt portions.  z [R][H dkp] fp32 becomes L in place; rows past the live ones decay by 1 and
// carry nothing.
// ------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void gla_decay_kernel(float* __restrict__ z, const int32_t* __restrict__ n_dev, int R, int W,
                                                        float inv_tau) {
  const int c = blockIdx.x * 256 + threadIdx.x, r0 = blockIdx.y * SUBC;
  const int live = hyb_live(n_dev, R);
  // whole chunks are read by the kernels below
  if (c >= W || r0 >= (live + CH - 1) / CH * CH) return;
  float v[SUBC];
#pragma unroll
  for (int i = 0; i < SUBC; ++i) v[i] = r0 + i < live ? z[(size_t)(r0 + i) * W + c] : 0.f;
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < SUBC; ++i) {
    if (r0 + i < live) s += hyb_log_sigmoid(v[i]) * inv_tau;
    z[(size_t)(r0 + i) * W + c] = s;
  }
}

// e^x for sums of log decays (x <= 0): the error grows with |x| where the result vanishes
__device__ inline float decay_exp(float x) { return __builtin_amdgcn_exp2f(x * 1.4426950408889634f); }

struct ChunkP {
  const void* x;
  const float* L;          // [R][H dkp]
  const float* norm_w;
  float* state;            // [H][dkp][dvp]
  float* A;                // [chunks][H][64][64]
  float* U;                // [chunks][H][dkp][dvp]
  float* decay;            // [chunks][H][dkp]
  void* out;
  const int32_t* n_dev;
  long ldx, ldo;
  int R, H, dkp, dvp, dv_true, oq, ok, ov, og;
  float qscale, eps;
};

// a row of the projections, zero past the live rows
template <typename T>
__device__ inline Frag<T> row8(const ChunkP& p, int row, int live, int off) {
  return row < live ? Frag<T>::load(reinterpret_cast<const T*>(p.x) + (size_t)row * p.ldx + off) : Frag<T>::zero();
}

template <typename T>
__global__ __launch_bounds__(256, 2) void gla_chunk_kernel(ChunkP p) {
  extern __shared__ __align__(16) float sm[];
  const int c = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int live = hyb_live(p.n_dev, p.R), r0 = c * CH;
  if (r0 >= live) return;
  const int dkp = p.dkp, ldl = dkp + 16;
  float* Ls = sm;                         // [64][ldl]: L, later the decayed keys
  float* Ts = sm + CH * ldl;              // [4][dkp]: totals of the sub-chunks
  const int lane = tid & 63, wave = tid >> 6, col = lane & 15, g = lane >> 4;
  const int W = p.H * dkp;
  for (int i = tid; i < CH * (dkp >> 2); i += 256) {
    const int r = i / (dkp >> 2), d = (i % (dkp >> 2)) * 4;
    const f32x4_t v = load4(p.L + (size_t)(r0 + r) * W + h * dkp + d);
    *reinterpret_cast<f32x4_t*>(Ls + r * ldl + d) = v;
    if ((r & 15) == 15) *reinterpret_cast<f32x4_t*>(Ts + (r >> 4) * dkp + d) = v;
  }
  __syncthreads();
  float* A = p.A + ((size_t)c * p.H + h) * CH * CH;
  // off-diagonal tiles (I, J < I), one or two per wave
  for (int pr = wave; pr < 6; pr += 4) {
    const int I = pr < 1 ? 1 : (pr < 3 ? 2 : 3), J = pr < 1 ? 0 : (pr < 3 ? pr - 1 : pr - 3);
    f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const int ri = I * SUBC + col, rj = J * SUBC + col;
    for (int d = g * 8; d < (dkp + 31) / 32 * 32; d += 32) {
      Frag<float> a = Frag<float>::zero(), b = Frag<float>::zero();
      if (d < dkp) {
        const Frag<T> q = row8<T>(p, r0 + ri, live, p.oq + h * dkp + d), k = row8<T>(p, r0 + rj, live, p.ok + h * dkp + d);
        const Frag<float> li = Frag<float>::load(Ls + ri * ldl + d), lj = Frag<float>::load(Ls + rj * ldl + d);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          float mid = 0.f;
          for (int M = J + 1; M < I; ++M) mid += Ts[M * dkp + d + e];
          a.set(e, q.at(e) * p.qscale * decay_exp(li.at(e) + mid));
          b.set(e, k.at(e) * decay_exp(Ts[J * dkp + d + e] - lj.at(e)));
        }
      }
      acc = mma(a, b, acc);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) A[(I * SUBC + g * 4 + i) * CH + J * SUBC + col] = acc[i];
  }
  // Diagonal tile of this wave: lane = (j, quarter of d), one row i after the other.  128 columns at a time
  // with this lane's keys and decays in registers; the next row's queries are requested ahead.
  {
    constexpr int DB = 4;
    const int b0 = wave * SUBC, rj = b0 + col;
    for (int d0 = 0; d0 < dkp; d0 += 32 * DB) {
      Frag<T> k[DB], q[DB];
      Frag<float> lj[DB];
      int at[DB];
#pragma unroll
      for (int t = 0; t < DB; ++t) {
        const int d = d0 + t * 32 + g * 8;
        at[t] = d < dkp ? d : dkp - 8;
        k[t] = d < dkp ? row8<T>(p, r0 + rj, live, p.ok + h * dkp + d) : Frag<T>::zero();
        lj[t] = Frag<float>::load(Ls + rj * ldl + at[t]);
      }
      auto queries = [&](int i) {
        const int r = r0 + b0 + i < live ? r0 + b0 + i : live - 1;      // rows past the live ones are not used
        const T* x = reinterpret_cast<const T*>(p.x) + (size_t)r * p.ldx + p.oq + h * dkp;
#pragma unroll
        for (int t = 0; t < DB; ++t) q[t] = Frag<T>::load(x + at[t]);
      };
      queries(0);
#pragma unroll 1
      for (int i = 0; i < SUBC; ++i) {
        float s = 0.f;
        Frag<T> now[DB];
#pragma unroll
        for (int t = 0; t < DB; ++t) now[t] = q[t];
        if (i + 1 < SUBC) queries(i + 1);
#pragma unroll
        for (int t = 0; t < DB; ++t) {
          const Frag<float> li = Frag<float>::load(Ls + (b0 + i) * ldl + at[t]);
#pragma unroll
          for (int e = 0; e < 8; ++e)       // j > i is dropped below: only keep the exponent in range
            s = fmaf(now[t].at(e) * k[t].at(e), decay_exp(fminf(li.at(e) - lj[t].at(e), 0.f)), s);
        }
        s *= p.qscale;
        s += __shfl_xor(s, 16, 64);
        s += __shfl_xor(s, 32, 64);
        if (g == 0) {
          float* o = A + (b0 + i) * CH + rj;
          *o = (d0 ? *o : 0.f) + (col <= i ? s : 0.f);
        }
      }
    }
  }
  __syncthreads();
  // keys decayed to the end of the chunk, in place of L
  for (int i = tid; i < CH * (dkp >> 3); i += 256) {
    const int r = i / (dkp >> 3), d = (i % (dkp >> 3)) * 8, J = r >> 4;
    const Frag<T> k = row8<T>(p, r0 + r, live, p.ok + h * dkp + d);
    float* dst = Ls + r * ldl + d;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      float t = Ts[J * dkp + d + e] - dst[e];
      for (int M = J + 1; M < 4; ++M) t += Ts[M * dkp + d + e];
      dst[e] = k.at(e) * decay_exp(t);
    }
  }
  if (tid < dkp || dkp > 256)
    for (int d = tid; d < dkp; d += 256)
      p.decay[((size_t)c * p.H + h) * dkp + d] = decay_exp(Ts[d] + Ts[dkp + d] + Ts[2 * dkp + d] + Ts[3 * dkp + d]);
  __syncthreads();
  // U = K^T V.  Value columns go in groups of 64: tile j of a group holds columns 4 c + j, so that a lane
  // reads and writes four columns at once.  The waves share a group's key tiles where there are few groups.
  float* U = p.U + ((size_t)c * p.H + h) * dkp * p.dvp;
  const int groups = (p.dvp + 63) >> 6, share = groups == 1 ? 4 : (groups == 2 ? 2 : 1);
  for (int vg = wave / share; vg < groups; vg += 4 / share) {
    const int v0 = vg * 64 + col * 4, vc = v0 < p.dvp ? v0 : p.dvp - 4;
    f32x4_t vv[16];
#pragma unroll
    for (int s = 0; s < 16; ++s) {
      const int r = r0 + 4 * s + g;       // keys past the live rows are zero
      vv[s] = load4(reinterpret_cast<const T*>(p.x) + (size_t)(r < live ? r : live - 1) * p.ldx + p.ov + h * p.dvp + vc);
    }
    for (int dt = wave % share; dt < (dkp >> 4); dt += share) {
      f32x4_t acc[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < 16; ++s) {
        const float k = Ls[(4 * s + g) * ldl + dt * 16 + col];
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(k, vv[s][j], acc[j], 0, 0, 0);
      }
      if (v0 < p.dvp) {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          *reinterpret_cast<f32x4_t*>(U + (size_t)(dt * 16 + g * 4 + i) * p.dvp + v0) =
              f32x4_t{acc[0][i], acc[1][i], acc[2][i], acc[3][i]};
      }
    }
  }
}

// U[c] <- state before chunk c; state <- state after the last chunk.  Eight chunks requested at a time.
__global__ __launch_bounds__(256) void gla_scan_kernel(ChunkP p) {
  const int live = hyb_live(p.n_dev, p.R), chunks = (live + CH - 1) / CH;
  if (chunks == 0) return;
  const long per = (long)p.H * p.dkp * p.dvp;
  const long at = ((long)blockIdx.x * 256 + threadIdx.x) * 4;
  if (at >= per) return;
  const long hd = at / p.dvp;                 // h dkp + d
  const long hk = (long)p.H * p.dkp;
  f32x4_t s = load4(p.state + at);
  for (int c0 = 0; c0 < chunks; c0 += 8) {
    f32x4_t u[8];
    float a[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int c = c0 + i < chunks ? c0 + i : chunks - 1;
      u[i] = load4(p.U + (size_t)c * per + at);
      a[i] = p.decay[(size_t)c * hk + hd];
    }
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (c0 + i < chunks) {
        *reinterpret_cast<f32x4_t*>(p.U + (size_t)(c0 + i) * per + at) = s;
        s = s * a[i] + u[i];
      }
  }
  *reinterpret_cast<f32x4_t*>(p.state + at) = s;
}

// NG: groups of 64 value columns (tile j of a group: columns 4 c + j)
template <typename T, int NG>
__global__ __launch_bounds__(256) void gla_out_kernel(ChunkP p) {
  extern __shared__ __align__(16) float sm[];
  const int c = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int live = hyb_live(p.n_dev, p.R), r0 = c * CH;
  if (r0 >= live) return;
  const int dkp = p.dkp, dvp = p.dvp, ldq = dkp + 4, W = p.H * dkp;
  float* Qs = sm;                          // [64][ldq]: queries decayed from the chunk's start
  const int lane = tid & 63, wave = tid >> 6, col = lane & 15, g = lane >> 4;
  for (int i = tid; i < CH * (dkp >> 3); i += 256) {
    const int r = i / (dkp >> 3), d = (i % (dkp >> 3)) * 8, I = r >> 4;
    const Frag<T> q = row8<T>(p, r0 + r, live, p.oq + h * dkp + d);
    Frag<float> l = Frag<float>::load(p.L + (size_t)(r0 + r) * W + h * dkp + d);
    for (int M = 0; M < I; ++M) {
      const Frag<float> t = Frag<float>::load(p.L + (size_t)(r0 + M * SUBC + SUBC - 1) * W + h * dkp + d);
      l.lo += t.lo;
      l.hi += t.hi;
    }
    Frag<float> o;
#pragma unroll
    for (int e = 0; e < 8; ++e) o.set(e, q.at(e) * p.qscale * decay_exp(l.at(e)));
    o.store(Qs + r * ldq + d);
  }
  __syncthreads();
  const float* S = p.U + ((size_t)c * p.H + h) * dkp * dvp;
  const float* A = p.A + ((size_t)c * p.H + h) * CH * CH + (wave * SUBC + col) * CH + g * 8;
  const T* V = reinterpret_cast<const T*>(p.x) + p.ov + h * dvp;
  int vc[NG];                              // this lane's columns (groups past the last repeat it)
#pragma unroll
  for (int v = 0; v < NG; ++v) vc[v] = v * 64 + col * 4 < dvp ? v * 64 + col * 4 : dvp - 4;
  f32x4_t acc[NG][4];
#pragma unroll
  for (int v = 0; v < NG; ++v)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[v][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  auto add = [&](const Frag<float>& a, const f32x4_t (&b)[8], f32x4_t (&o)[4]) {
#pragma unroll
    for (int e = 0; e < 8; ++e)
#pragma unroll
      for (int j = 0; j < 4; ++j) o[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a.at(e), b[e][j], o[j], 0, 0, 0);
  };
  for (int d = g * 8; d < (dkp + 31) / 32 * 32; d += 32) {
    const bool in = d < dkp;
    const Frag<float> q = in ? Frag<float>::load(Qs + (wave * SUBC + col) * ldq + d) : Frag<float>::zero();
    const float* Sr = S + (size_t)(in ? d : 0) * dvp;
#pragma unroll
    for (int v = 0; v < NG; ++v) {
      f32x4_t b[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) b[e] = load4(Sr + e * dvp + vc[v]);
      add(q, b, acc[v]);
    }
  }
  // within the chunk: rows of A against V (32 rows at a time, no further than this wave's rows)
  for (int j0 = 0; j0 < (wave < 2 ? 32 : 64); j0 += 32) {
    Frag<float> a = Frag<float>::load(A + j0);
    const int jr = j0 + g * 8;
    // tiles above the diagonal are never written
    if ((jr >> 4) > wave) a = Frag<float>::zero();
#pragma unroll
    for (int v = 0; v < NG; ++v) {
      f32x4_t b[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int r = r0 + jr + e < live ? r0 + jr + e : live - 1;      // a's columns past the live rows are zero
        b[e] = load4(V + (size_t)r * p.ldx + vc[v]);
      }
      add(a, b, acc[v]);
    }
  }
  float ss[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int v = 0; v < NG; ++v)
    if (v * 64 + col * 4 < dvp) {
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) ss[i] += acc[v][j][i] * acc[v][j][i];
    }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
#pragma unroll
    for (int o = 8; o > 0; o >>= 1) ss[i] += __shfl_xor(ss[i], o, 64);
    ss[i] = 1.f / sqrtf(ss[i] / (float)p.dv_true + p.eps);
  }
#pragma unroll
  for (int v = 0; v < NG; ++v)
    if (v * 64 + col * 4 < dvp) {
      const f32x4_t w = load4(p.norm_w + vc[v]);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = r0 + wave * SUBC + g * 4 + i;
        if (r < live) {
          const int at = h * dvp + vc[v];
          const f32x4_t gt = load4(reinterpret_cast<const T*>(p.x) + (size_t)r * p.ldx + p.og + at);
          f32x4_t o;
#pragma unroll
          for (int j = 0; j < 4; ++j) o[j] = acc[v][j][i] * ss[i] * w[j] * gt[j] * hyb_sigmoid(gt[j]);
          store4<T>(reinterpret_cast<T*>(p.out) + (size_t)r * p.ldo + at, o);
        }
      }
    }
}

template <typename K>
void allow_lds(K kernel, size_t lds) {
  if (lds > 65536) (void)hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
}

template <typename T>
void launch_step(const StepP& p, hipStream_t st) {
  // threads: whole waves, at least one row of float4 columns, enough to hold the state in registers
  const int threads = p.dkp * p.dvp <= 4096 ? 256 : 1024;
  const int ty = threads / (p.dvp / 4);
  const int nd = (p.dkp + ty - 1) / ty;
  const size_t lds = (size_t)(4 * threads + 3 * p.dkp) * 4;
#define STEP(N) gla_step_kernel<T, N><<<p.H, threads, lds, st>>>(p)
  if (nd <= 2)
    STEP(2);
  else if (nd <= 4)
    STEP(4);
  else
    STEP(0);
#undef STEP
}

template <typename T>
void launch_chunks(const ChunkP& p, hipStream_t st) {
  const int chunks = (p.R + CH - 1) / CH;
  const dim3 grid(chunks, p.H);
  const size_t lds1 = (size_t)(CH * (p.dkp + 16) + 4 * p.dkp) * 4, lds3 = (size_t)CH * (p.dkp + 4) * 4;
  allow_lds(gla_chunk_kernel<T>, lds1);
  gla_chunk_kernel<T><<<grid, 256, lds1, st>>>(p);
  const long per = (long)p.H * p.dkp * p.dvp / 4;
  gla_scan_kernel<<<(unsigned)((per + 255) / 256), 256, 0, st>>>(p);
#define OUT(N)                             \
  allow_lds(gla_out_kernel<T, N>, lds3);   \
  gla_out_kernel<T, N><<<grid, 256, lds3, st>>>(p)
  const int ng = (p.dvp + 63) / 64;
  if (ng == 1) {
    OUT(1);
  } else if (ng == 2) {
    OUT(2);
  } else if (ng <= 4) {
    OUT(4);
  } else {
    OUT(8);
  }
#undef OUT
}

int check_gla(const hyb_gla_args* a) {
  if (!a || !a->x || !a->norm_w || !a->state || !a->out) return HYB_ERR_NULL;
  if (a->dtype != HYB_BF16 && a->dtype != HYB_F32) return HYB_ERR_UNSUPPORTED;
  if (a->R < 1 || a->H < 1 || a->dkp < 16 || a->dkp % 16 || a->dkp > 512 || a->dvp < 16 || a->dvp % 16 || a->dvp > 512 ||
      a->dv_true < 1 || a->dv_true > a->dvp || a->tau <= 0.f || a->ldx % 8 || a->ldo < (long)a->H * a->dvp)
    return HYB_ERR_SHAPE;
  if (a->off_q % 8 || a->off_k % 8 || a->off_v % 8 || a->off_g % 8 || a->off_a % 8) return HYB_ERR_ALIGN;
  if (!hyb_aligned16(a->x) || !hyb_aligned16(a->state) || !hyb_aligned16(a->a2) || !hyb_aligned16(a->norm_w) ||
      !hyb_aligned16(a->out) || a->ldo % 8)
    return HYB_ERR_ALIGN;
  return HYB_OK;
}

}  // namespace

HYB_EXPORT int hyb_gla_step(const hyb_gla_args* a, hyb_stream_t stream) {
  const int rc = check_gla(a);
  if (rc != HYB_OK) return rc;
  if (!a->a2 || !a->a2_bias) return HYB_ERR_NULL;
  if (a->rp < 8 || a->rp % 8) return HYB_ERR_SHAPE;
  StepP p{a->x,   a->a2, a->a2_bias, a->norm_w, a->state, a->out,     a->n_dev, a->ldx,   a->ldo,   a->R,     a->H,      a->dkp,
          a->dvp, a->rp, a->dv_true, a->off_q,  a->off_k, a->off_v,   a->off_g, a->off_a, a->qscale, 1.f / a->tau, a->eps};
  HYB_DISPATCH(a->dtype, launch_step<T>(p, (hipStream_t)stream);)
  return hyb_launch_status();
}

HYB_EXPORT size_t hyb_gla_chunk_workspace_bytes(int R, int H, int dkp, int dvp) {
  if (R < 1 || H < 1 || dkp < 16 || dvp < 16) return 0;
  const size_t chunks = (R + CH - 1) / CH;
  return chunks * H * ((size_t)CH * CH + (size_t)dkp * dvp + dkp) * 4;
}

HYB_EXPORT int hyb_gla_chunks(const hyb_gla_args* a, hyb_stream_t stream) {
  const int rc = check_gla(a);
  if (rc != HYB_OK) return rc;
  if (!a->z) return HYB_ERR_NULL;
  if (a->R % CH) return HYB_ERR_SHAPE;            // whole chunks of rows; n_dev says how many are live
  if (!hyb_aligned16(a->z)) return HYB_ERR_ALIGN;
  if (!a->workspace || a->workspace_bytes < hyb_gla_chunk_workspace_bytes(a->R, a->H, a->dkp, a->dvp)) return HYB_ERR_WORKSPACE;
  const size_t chunks = a->R / CH;
  float* A = (float*)a->workspace;
  float* U = A + chunks * a->H * CH * CH;
  float* decay = U + chunks * a->H * (size_t)a->dkp * a->dvp;
  hipStream_t st = (hipStream_t)stream;
  const int W = a->H * a->dkp;
  gla_decay_kernel<<<dim3((W + 255) / 256, a->R / SUBC), 256, 0, st>>>(a->z, a->n_dev, a->R, W, 1.f / a->tau);
  ChunkP p{a->x,   a->z,   a->norm_w, a->state, A,          U,        decay,    a->out,   a->n_dev, a->ldx,    a->ldo, a->R,
           a->H,   a->dkp, a->dvp,    a->dv_true, a->off_q, a->off_k, a->off_v, a->off_g, a->qscale, a->eps};
  HYB_DISPATCH(a->dtype, launch_chunks<T>(p, st);)
  return hyb_launch_status();
}
