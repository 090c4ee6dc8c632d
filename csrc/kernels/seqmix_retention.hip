// Recurrence with one fixed decay per head over chunks of tokens (retention, long segments):
//
//   S_t = g S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t        S fp32 [dim, vdim] per head, g in [0, 1]
//
// A chunk of CT tokens is one set of matrix products instead of CT steps; with S the state in
// front of the chunk and r = 0, 1, ... the token's place in it,
//
//   o_r = g^(r + 1) S^T q_r + sum_(s <= r) g^(r - s) (q_r . k_s) v_s
//   S  <- g^n S + sum_s g^(n - 1 - s) k_s v_s^T            (n tokens in the chunk)
//
// Everything is fp32 (true-fp32 MFMAs, `mma16`); v is read in the activation type T.  The powers of g
// come from a table of repeated products (g = 0 gives 1, 0, 0, ...).  The token-by-token form of
// seqmix_state.hip serves short segments; both leave the same state up to rounding.
//
// One workgroup per (segment, head, VT value columns), four waves.  The chunk's keys lie in LDS as
// rows, its values transposed, the state transposed (value column by value column).  Wave w owns the
// chunk's queries 16 w .. 16 w + 15 and the state's key-feature tiles w, w + 4, ...  The products are
// arranged so that a result in C registers is the next product's B operand (no shuffle):
//   S^T Q^T       [value column x query]   from the state in LDS
//   K Q^T         [key x query]            weighted by g^(r - s), zero above the diagonal
//   V^T (K Q^T)   [value column x query]   added to it
//   V^T K         [value column x key feature], keys weighted by g^(n - 1 - s): the state's update
#include <algorithm>

#include "seqmix_common.h"

namespace {

constexpr int CT = 64, VT = 64, NTH = 256;
constexpr int MIN_LEN = 16;   // shorter segments are faster token by token

struct ChunkArgs {
  const float* q; const float* k;                   // [T, Gq, dim]
  const float* decay;                               // [H]
  const void* v; int64_t v_stride;                  // [T, >= H vdim]
  const int* positions; const int* q_start; const int* state_rows;
  float* state;                                     // [n_rows, H, dim, vdim]
  float* out;                                       // [T, H, vdim]
  int n_rows, H, Gq, dim, vdim, vec;                // vec: rows of q / k are 16-byte aligned
};

// four fp32 at p[0..3], zero from n_valid on
__device__ __forceinline__ f32x4 load4(const float* p, int n_valid, bool vec) {
  f32x4 r = {0.f, 0.f, 0.f, 0.f};
  if (n_valid >= 4 && vec) return *reinterpret_cast<const f32x4*>(p);
#pragma unroll
  for (int j = 0; j < 4; ++j)
    if (j < n_valid) r[j] = p[j];
  return r;
}

// DC: 16-wide tiles of key features (dim <= 16 DC).
template <typename T, int DC, int OCC>
__global__ __launch_bounds__(NTH, OCC) void retention_chunk_kernel(ChunkArgs a) {
  typedef typename Elem<T>::frag F;
  constexpr int LDK = 16 * DC + 4, LDV = CT + 4, ND = (DC + 3) / 4;
  __shared__ __attribute__((aligned(16))) float Ks[CT * LDK];   // [token][feature]
  __shared__ __attribute__((aligned(16))) float Ss[VT * LDK];   // [value column][feature]
  __shared__ __attribute__((aligned(16))) T Vs[VT * LDV];       // [value column][token]
  __shared__ float pw[CT + 1];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, grp = lane >> 4;
  const int b = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * VT;
  const int t0 = a.q_start[b], t1 = a.q_start[b + 1], sr = a.state_rows[b];
  if (t1 - t0 < MIN_LEN || sr < 0 || sr >= a.n_rows) return;
  const int gq = h / (a.H / a.Gq), dim = a.dim, vdim = a.vdim;
  if (tid <= CT) {
    const float g = a.decay[h];
    float p = 1.0f;
    for (int i = 0; i < tid; ++i) p *= g;
    pw[tid] = p;
  }
  float* Sg = a.state + (static_cast<size_t>(sr) * a.H + h) * dim * vdim + v0;
  const bool carry = a.positions[t0] != 0;
  const bool vec_s = (vdim & 3) == 0;
  f32x4 S[ND][4];   // lane: S^T[value column 16 u + 4 grp + i][feature 16 (wave + 4 m) + col]
#pragma unroll
  for (int m = 0; m < ND; ++m) {
    const int d = 16 * (wave + 4 * m) + col;
#pragma unroll
    for (int u = 0; u < 4; ++u)
      S[m][u] = (carry && d < dim) ? load4(Sg + static_cast<size_t>(d) * vdim + 16 * u + 4 * grp, vdim - v0 - 16 * u - 4 * grp, vec_s)
                                   : f32x4{0.f, 0.f, 0.f, 0.f};
  }
  auto stage_state = [&]() {
#pragma unroll
    for (int m = 0; m < ND; ++m) {
      const int dt = wave + 4 * m;
      if (dt < DC) {
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
          for (int i = 0; i < 4; ++i) Ss[(16 * u + 4 * grp + i) * LDK + 16 * dt + col] = S[m][u][i];
      }
    }
  };
  auto value_frag = [&](int u, int tok) {   // V^T[value column 16 u + col][tokens tok .. tok + 3] as fp32
    const F f = *reinterpret_cast<const F*>(&Vs[(16 * u + col) * LDV + tok]);
    f32x4 r;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if constexpr (sizeof(T) == 2) r[j] = bf2f(static_cast<bf16_t>(f[j])); else r[j] = f[j];
    }
    return r;
  };
  stage_state();
  const T* vbase = static_cast<const T*>(a.v) + static_cast<size_t>(h) * vdim + v0;
  for (int first = t0; first < t1; first += CT) {
    const int n = min(CT, t1 - first);
    // ---- the chunk's keys and values; rows past the segment are zero ----
    for (int e = tid; e < CT * 4 * DC; e += NTH) {
      const int r = e / (4 * DC), f = 4 * (e - r * 4 * DC);
      const f32x4 x = r < n ? load4(a.k + (static_cast<size_t>(first + r) * a.Gq + gq) * dim + f, dim - f, a.vec) : f32x4{0.f, 0.f, 0.f, 0.f};
      *reinterpret_cast<f32x4*>(&Ks[r * LDK + f]) = x;
    }
#pragma unroll
    for (int p = 0; p < 4; ++p) {
      const int r = 16 * wave + 4 * p;
      F f = zero_frag<T>();
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (r + j < n && v0 + lane < vdim) {
          const T x = vbase[static_cast<size_t>(first + r + j) * a.v_stride + lane];
          if constexpr (sizeof(T) == 2) f[j] = static_cast<short>(x); else f[j] = x;
        }
      *reinterpret_cast<F*>(&Vs[lane * LDV + r]) = f;
    }
    const int place = 16 * wave + col;   // this lane's query
    f32x4 qf[DC];
    {
      const float* qrow = a.q + (static_cast<size_t>(first + min(place, n - 1)) * a.Gq + gq) * dim;
#pragma unroll
      for (int c = 0; c < DC; ++c) qf[c] = load4(qrow + 16 * c + 4 * grp, dim - 16 * c - 4 * grp, a.vec);
    }
    __syncthreads();
    const bool live = 16 * wave < n;   // (wave-uniform) some query of the wave
    f32x4 o[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) o[u] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (live) {
      if (carry || first > t0) {
#pragma unroll
        for (int c = 0; c < DC; ++c)
#pragma unroll
          for (int u = 0; u < 4; ++u)
            o[u] = mma16(*reinterpret_cast<const f32x4*>(&Ss[(16 * u + col) * LDK + 16 * c + 4 * grp]), qf[c], o[u]);
        const float g = pw[place + 1];
#pragma unroll
        for (int u = 0; u < 4; ++u) o[u] *= g;
      }
      for (int kt = 0; kt <= wave; ++kt) {
        f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = s0;   // (two chains)
#pragma unroll
        for (int c = 0; c < DC; ++c) {
          const f32x4 kf = *reinterpret_cast<const f32x4*>(&Ks[(16 * kt + col) * LDK + 16 * c + 4 * grp]);
          if (c & 1) s1 = mma16(kf, qf[c], s1); else s0 = mma16(kf, qf[c], s0);
        }
        f32x4 s = s0 + s1;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int back = place - (16 * kt + 4 * grp + i);
          s[i] = back >= 0 ? s[i] * pw[back] : 0.f;
        }
#pragma unroll
        for (int u = 0; u < 4; ++u) o[u] = mma16(value_frag(u, 16 * kt + 4 * grp), s, o[u]);
      }
      if (place < n) {
        float* orow = a.out + (static_cast<size_t>(first + place) * a.H + h) * vdim + v0;
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          const int e = 16 * u + 4 * grp;
          if (vec_s && v0 + e + 3 < vdim) {
            *reinterpret_cast<f32x4*>(orow + e) = o[u];
          } else {
#pragma unroll
            for (int i = 0; i < 4; ++i)
              if (v0 + e + i < vdim) orow[e + i] = o[u][i];
          }
        }
      }
    }
    // ---- the state behind the chunk ----
    const float gn = pw[n];
#pragma unroll
    for (int m = 0; m < ND; ++m)
#pragma unroll
      for (int u = 0; u < 4; ++u) S[m][u] *= gn;
    for (int tt = 0; 16 * tt < n; ++tt) {
      f32x4 vf[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) vf[u] = value_frag(u, 16 * tt + 4 * grp);
      float w[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) w[j] = pw[max(n - 1 - (16 * tt + 4 * grp + j), 0)];   // (keys past the segment are zero)
#pragma unroll
      for (int m = 0; m < ND; ++m) {
        const int dt = wave + 4 * m;
        if (dt < DC) {
          f32x4 kf;
#pragma unroll
          for (int j = 0; j < 4; ++j) kf[j] = Ks[(16 * tt + 4 * grp + j) * LDK + 16 * dt + col] * w[j];
#pragma unroll
          for (int u = 0; u < 4; ++u) S[m][u] = mma16(vf[u], kf, S[m][u]);
        }
      }
    }
    __syncthreads();   // every reader of the chunk and of the old state is done
    if (first + CT < t1) stage_state();
  }
#pragma unroll
  for (int m = 0; m < ND; ++m) {
    const int d = 16 * (wave + 4 * m) + col;
    if (d >= dim) continue;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int e = 16 * u + 4 * grp;
      float* p = Sg + static_cast<size_t>(d) * vdim + e;
      if (vec_s && v0 + e + 3 < vdim) {
        *reinterpret_cast<f32x4*>(p) = S[m][u];
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (v0 + e + i < vdim) p[i] = S[m][u][i];
      }
    }
  }
}

template <typename T>
int launch_chunks(const ChunkArgs& a, int B, hipStream_t s) {
  const dim3 grid(B, a.H, (a.vdim + VT - 1) / VT);
  if (a.dim <= 32) retention_chunk_kernel<T, 2, 2><<<grid, NTH, 0, s>>>(a);
  else if (a.dim <= 64) retention_chunk_kernel<T, 4, 2><<<grid, NTH, 0, s>>>(a);
  else if (a.dim <= 128) retention_chunk_kernel<T, 8, sizeof(T) == 2 ? 2 : 1><<<grid, NTH, 0, s>>>(a);
  else retention_chunk_kernel<T, 16, 1><<<grid, NTH, 0, s>>>(a);
  return BCG_CHECK_LAUNCH();
}

}  // namespace

// Segments shorter than this are left alone by `bcg_retention_chunks`.
BCG_API int bcg_retention_min_len() { return MIN_LEN; }

BCG_API int bcg_retention_chunks(const void* q32, const void* k32, const void* decay, const void* v, int64_t v_stride,
                                 const void* positions, const void* q_start, const void* state_rows, void* state, int n_rows,
                                 void* out, int B, int H, int Gq, int dim, int vdim, int is_f32, void* stream) {
  if (B <= 0) return 0;
  if (dim < 1 || dim > 256 || vdim < 1 || H <= 0 || Gq <= 0 || H % Gq || H > 65535 || (vdim + VT - 1) / VT > 65535) return -2;
  auto al16 = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  if (!al16(state) || !al16(out)) return -2;
  ChunkArgs a;
  a.q = static_cast<const float*>(q32); a.k = static_cast<const float*>(k32); a.decay = static_cast<const float*>(decay);
  a.v = v; a.v_stride = v_stride;
  a.positions = static_cast<const int*>(positions); a.q_start = static_cast<const int*>(q_start);
  a.state_rows = static_cast<const int*>(state_rows);
  a.state = static_cast<float*>(state); a.out = static_cast<float*>(out);
  a.n_rows = n_rows; a.H = H; a.Gq = Gq; a.dim = dim; a.vdim = vdim;
  a.vec = dim % 4 == 0 && al16(q32) && al16(k32);
  hipStream_t s = static_cast<hipStream_t>(stream);
  return is_f32 ? launch_chunks<float>(a, B, s) : launch_chunks<bf16_t>(a, B, s);
}
