// Retention: linear attention whose state S [dk, dv] per head (fp32) forgets with a fixed decay. Over a step's
// per-sequence token runs, each continuing the state in its slot (seq_slot) or starting from zero (seq_init == 0):
//
//   q, k rotated on their first rot_dims dimensions (pairs (i, i + rot_dims / 2)), k times dk^-1/2
//   S <- decay S + k v^T;  o = S^T q;  out = o / rms(o) * silu(g)
//
// from the fused projection rows [q | k | v (| g)]; everything between the projections and ``out`` is fp32.
//
// retention_step  : sequences that bring one token. One workgroup per (head, sequence) rotates q and k, streams S
//                   once (16-byte pieces, a thread keeps its columns), and norms and gates the read-out.
// Longer runs are cut into chunks of at most C = 64 tokens. A chunk of n tokens that starts from S gives
//   o_i = decay^(i+1) S^T q_i + sum_{j <= i} decay^(i-j) (q_i . k_j) v_j,   S' = decay^n S + sum_j decay^(n-1-j) k_j v_j^T
// so all products are matrix products. They run on v_mfma_f32_16x16x4_f32: operands and sums are fp32.
// retention_chunk : every chunk's own part of its final state, L = sum_j decay^(n-1-j) k_j v_j^T.
// retention_link  : walks a sequence's chunks in order, S_(c+1) = decay^n S_c + L_c; leaves every chunk's start
//                   state where its L was and the run's final state in the slot.
// retention_out   : a chunk's read-outs; workgroup = 64 queries (16 per wave) x up to 256 columns. The weights of the
//                   second product stay in the registers the scores arrive in. Norm and gate are fused when one
//                   workgroup holds all of a head's columns, else retention_norm follows.
// In all of them the contraction index is dealt so that an operand's four consecutive elements belong to one lane:
// step e of a group of 16 takes element 4 kq + e from lane group kq, on both sides.
#include "seqmix_common.h"
#include <algorithm>

using namespace sm;

namespace {

constexpr int NT = 256;
constexpr int C = 64;         // tokens per chunk
constexpr int DB = 64;        // key dimensions staged at a time
constexpr int QS = DB + 4;    // LDS row stride of the keys
constexpr int MAXCOLS = 256;  // value columns of a workgroup

typedef float f32x4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ void ld4(const float* p, float (&v)[4]) {
  const float4 t = *reinterpret_cast<const float4*>(p);
  v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
}
__device__ __forceinline__ void ld4(const bf16_t* p, float (&v)[4]) {
  const uint2 t = *reinterpret_cast<const uint2*>(p);
  v[0] = __uint_as_float(t.x << 16); v[1] = __uint_as_float(t.x & 0xffff0000u);
  v[2] = __uint_as_float(t.y << 16); v[3] = __uint_as_float(t.y & 0xffff0000u);
}

struct Rot {
  const int64_t* positions;
  const float* cos_sin;  // [max_pos, dims] = [cos | sin]
  int dims;              // 0: no rotation
};

// Element e of a head's rotated row.
template <typename T>
__device__ __forceinline__ float rot1(const T* row, int e, const float* cs, int half) {
  const float x = ld(row + e);
  if (e >= 2 * half) return x;
  const bool first = e < half;
  const float xp = ld(row + (first ? e + half : e - half));
  const int f = first ? e : e - half;
  const float c = cs[f], s = cs[half + f];
  return first ? x * c - xp * s : x * c + xp * s;
}

// Elements e .. e + 3, zero past dk. VEC (dk and half multiples of four, rows aligned for it): all loads are
// unconditional, from clamped places, so that those of several calls are in flight together.
template <typename T, bool VEC>
__device__ __forceinline__ void rot4(const T* row, int e, int dk, const float* cs, int half, float (&v)[4]) {
  if constexpr (!VEC) {
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = e + i < dk ? rot1(row, e + i, cs, half) : 0.f;
  } else {
    const int ec = min(e, dk - 4);
    ld4(row + ec, v);
    if (half > 0) {
      const bool first = ec < half, in = ec < 2 * half;
      const int f = in ? (first ? ec : ec - half) : 0;
      float p[4], c[4], s[4];
      ld4(row + (in ? (first ? ec + half : ec - half) : ec), p);
      ld4(cs + f, c);
      ld4(cs + half + f, s);
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] = in ? (first ? v[i] * c[i] - p[i] * s[i] : v[i] * c[i] + p[i] * s[i]) : v[i];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = e < dk ? v[i] : 0.f;
  }
}

// ---------------------------------------------------------------------------------------------
// VEC columns per thread; ncg = column groups side by side, RG = row groups (threads past RG * ncg idle).
template <typename T, int VEC>
__global__ __launch_bounds__(NT) void retention_step_kernel(const T* __restrict__ p, int64_t stride, int H, int dk,
                                                            int dv, int gate, Rot rot, const float* __restrict__ powers,
                                                            int pw_stride, float eps, float* __restrict__ state,
                                                            const int* __restrict__ seq_start,
                                                            const int* __restrict__ seq_slot,
                                                            const int* __restrict__ seq_init, T* __restrict__ out,
                                                            int ncg, int RG) {
  extern __shared__ float lds[];
  __shared__ float red[NT / 64];
  const int h = blockIdx.x, s = blockIdx.y;
  const int64_t t = seq_start[s];
  const bool init = seq_init[s] != 0;
  float* sp = state + ((int64_t)seq_slot[s] * H + h) * dk * dv;
  float *sq = lds, *sk = lds + dk, *so = lds + 2 * dk;  // so [RG, dv]
  const T* row = p + t * stride;
  const int rg = threadIdx.x / ncg, cg = threadIdx.x - rg * ncg;
  constexpr int U = 8;  // rows of the state in flight
  float S[U][VEC];
  auto load = [&](int r0, int col) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int r = r0 + u * RG;
#pragma unroll
      for (int i = 0; i < VEC; ++i) S[u][i] = 0.f;
      if (init && r < dk) {
        if constexpr (VEC == 4) ld4(sp + (int64_t)r * dv + col, S[u]);
        else S[u][0] = sp[(int64_t)r * dv + col];
      }
    }
  };
  if (rg < RG) load(rg, cg * VEC);  // the first piece is on its way while the keys and queries are rotated
  const int half = rot.dims >> 1;
  const float* cs = rot.dims ? rot.cos_sin + rot.positions[t] * rot.dims : nullptr;
  const float kscale = 1.f / sqrtf((float)dk);
  const float decay = powers[h * pw_stride + 1];
  for (int e = threadIdx.x; e < 2 * dk; e += NT) {
    const bool is_q = e < dk;
    const int d = is_q ? e : e - dk;
    const float x = rot1(row + (is_q ? h : H + h) * dk, d, cs, half);
    lds[e] = is_q ? x : x * kscale;
  }
  __syncthreads();
  const T* vrow = row + 2 * H * dk + h * dv;
  if (rg < RG) {
    for (int col = cg * VEC; col < dv; col += ncg * VEC) {
      if (col != cg * VEC) load(rg, col);
      float v[VEC], o[VEC];
#pragma unroll
      for (int i = 0; i < VEC; ++i) {
        v[i] = ld(vrow + col + i);
        o[i] = 0.f;
      }
      for (int r0 = rg; r0 < dk; r0 += RG * U) {
        if (r0 != rg) load(r0, col);
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const int r = r0 + u * RG;
          if (r >= dk) continue;
          const float k = sk[r], q = sq[r];
#pragma unroll
          for (int i = 0; i < VEC; ++i) {
            S[u][i] = decay * S[u][i] + k * v[i];
            o[i] += S[u][i] * q;
          }
          if constexpr (VEC == 4)
            *reinterpret_cast<float4*>(sp + (int64_t)r * dv + col) = make_float4(S[u][0], S[u][1], S[u][2], S[u][3]);
          else
            sp[(int64_t)r * dv + col] = S[u][0];
        }
      }
#pragma unroll
      for (int i = 0; i < VEC; ++i) so[rg * dv + col + i] = o[i];
    }
  }
  __syncthreads();
  const T* grow = row + 2 * H * dk + H * dv + h * dv;
  const float g0 = gate && (int)threadIdx.x < dv ? ld(grow + threadIdx.x) : 0.f;
  float ss = 0.f;
  for (int e = threadIdx.x; e < dv; e += NT) {  // a thread reads back only what it sums here
    float a = 0.f;
    for (int g = 0; g < RG; ++g) a += so[g * dv + e];
    so[e] = a;
    ss += a * a;
  }
  const float inv = 1.f / sqrtf(block_sum<NT>(ss, red) / (float)dv + eps);
  for (int e = threadIdx.x; e < dv; e += NT) {
    float o = so[e] * inv;
    if (gate) o *= Fn<T>::silu(e < NT ? g0 : ld(grow + e));
    st(out + (t * H + h) * dv + e, o);
  }
}

// ---------------------------------------------------------------------------------------------
// Stage CB value columns [col0, col0 + CB) of ROWS tokens t0 .. (rows past n and columns past dv are zero).
template <typename T, int CB, int ROWS, bool VEC>
__device__ __forceinline__ void stage_v(const T* __restrict__ p, int64_t stride, int64_t t0, int n, int voff, int col0,
                                        int dv, float* sV) {
  constexpr int BS = CB + 4;
#pragma unroll
  for (int e0 = 0; e0 < ROWS * (CB / 4); e0 += NT) {
    const int e = e0 + threadIdx.x;
    const int j = e / (CB / 4), c = (e - j * (CB / 4)) * 4;
    const T* src = p + (t0 + min(j, n - 1)) * stride + voff;
    float v[4] = {0.f, 0.f, 0.f, 0.f};
    if constexpr (VEC) {
      ld4(src + min(col0 + c, dv - 4), v);
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] = j < n && col0 + c < dv ? v[i] : 0.f;
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (j < n && col0 + c + i < dv) v[i] = ld(src + col0 + c + i);
    }
    *reinterpret_cast<float4*>(&sV[j * BS + c]) = make_float4(v[0], v[1], v[2], v[3]);
  }
}

// L = sum_j decay^(n-1-j) k_j v_j^T of chunk c0 + blockIdx.x, head blockIdx.y; blockIdx.z: block of DB key rows x CB columns.
template <typename T, int NCB, bool VEC>
__global__ __launch_bounds__(NT) void retention_chunk_kernel(const T* __restrict__ p, int64_t stride, int H, int dk,
                                                             int dv, Rot rot, const float* __restrict__ powers,
                                                             int pw_stride, const int* __restrict__ c_start, int c0,
                                                             float* __restrict__ c_state) {
  constexpr int CB = 16 * NCB, BS = CB + 4;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float *sK = lds, *sV = lds + C * QS;
  const int c = blockIdx.x, h = blockIdx.y;
  const int ncb = (dv + CB - 1) / CB;
  const int d0 = (int)(blockIdx.z / ncb) * DB, col0 = (int)(blockIdx.z % ncb) * CB;
  const int64_t t0 = c_start[c0 + c];
  const int n = c_start[c0 + c + 1] - (int)t0;
  const int half = rot.dims >> 1;
  const float kscale = 1.f / sqrtf((float)dk);
  const float* pw = powers + (int64_t)h * pw_stride;
  const int64_t pos0 = rot.positions[t0];  // a chunk's positions follow each other
#pragma unroll
  for (int e0 = 0; e0 < C * (DB / 4); e0 += NT) {
    const int e = e0 + threadIdx.x;
    const int j = e / (DB / 4), d = (e - j * (DB / 4)) * 4, jc = min(j, n - 1);
    float v[4];
    rot4<T, VEC>(p + (t0 + jc) * stride + (H + h) * dk, d0 + d, dk, rot.cos_sin + (pos0 + jc) * rot.dims, half, v);
    const float w = j < n ? kscale * pw[n - 1 - jc] : 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = j < n ? v[i] * w : 0.f;
    *reinterpret_cast<float4*>(&sK[j * QS + d]) = make_float4(v[0], v[1], v[2], v[3]);
  }
  stage_v<T, CB, C, VEC>(p, stride, t0, n, 2 * H * dk + h * dv, col0, dv, sV);
  __syncthreads();
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int r16 = lane & 15, kq = lane >> 4;
  if (d0 + wave * 16 >= dk) return;
  f32x4_t acc[NCB];
#pragma unroll
  for (int m = 0; m < NCB; ++m) acc[m] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int j0 = 0; j0 < n; j0 += 16) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int j = j0 + 4 * kq + e;
      const float a = sK[j * QS + wave * 16 + r16];
#pragma unroll
      for (int m = 0; m < NCB; ++m) acc[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, sV[j * BS + m * 16 + r16], acc[m], 0, 0, 0);
    }
  }
  float* dst = c_state + ((int64_t)c * H + h) * dk * dv;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int d = d0 + wave * 16 + kq * 4 + r;
    if (d >= dk) continue;
#pragma unroll
    for (int m = 0; m < NCB; ++m) {
      const int col = col0 + m * 16 + r16;
      if (col < dv) dst[(int64_t)d * dv + col] = acc[m][r];
    }
  }
}

// Sequence s0 + blockIdx.y: its chunks in order, VEC elements of the state per thread.
template <int VEC>
__global__ __launch_bounds__(NT) void retention_link_kernel(float* __restrict__ c_state, const int* __restrict__ c_start,
                                                            const int* __restrict__ s_chunk0, int c0, int s0, int H,
                                                            int64_t per_head, const float* __restrict__ powers,
                                                            int pw_stride, float* __restrict__ state,
                                                            const int* __restrict__ seq_slot,
                                                            const int* __restrict__ seq_init) {
  const int s = s0 + blockIdx.y;
  const int64_t total = per_head * H;
  const int64_t e = ((int64_t)blockIdx.x * NT + threadIdx.x) * VEC;
  if (e >= total) return;
  const float* pw = powers + (e / per_head) * pw_stride;  // VEC divides a head's elements
  const int lo = s_chunk0[s], hi = s_chunk0[s + 1];
  if (lo >= hi) return;
  float* sp = state + (int64_t)seq_slot[s] * total + e;
  float S[VEC];
#pragma unroll
  for (int i = 0; i < VEC; ++i) S[i] = 0.f;
  if (seq_init[s]) {
    if constexpr (VEC == 4) ld4(sp, S);
    else S[0] = sp[0];
  }
  constexpr int U = 16;  // chunks in flight
  const float d_full = pw[C], d_last = pw[c_start[hi] - c_start[hi - 1]];  // all chunks but a run's last are whole
  for (int cb = lo; cb < hi; cb += U) {
    float L[U][VEC];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const float* src = c_state + (int64_t)(min(cb + u, hi - 1) - c0) * total + e;
      if constexpr (VEC == 4) ld4(src, L[u]);
      else L[u][0] = src[0];
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (cb + u < hi) {
        float* dst = c_state + (int64_t)(cb + u - c0) * total + e;
        if constexpr (VEC == 4) *reinterpret_cast<float4*>(dst) = make_float4(S[0], S[1], S[2], S[3]);
        else dst[0] = S[0];
        const float d = cb + u == hi - 1 ? d_last : d_full;
#pragma unroll
        for (int i = 0; i < VEC; ++i) S[i] = d * S[i] + L[u][i];
      }
  }
  if constexpr (VEC == 4) *reinterpret_cast<float4*>(sp) = make_float4(S[0], S[1], S[2], S[3]);
  else sp[0] = S[0];
}

// The read-outs of chunk c0 + blockIdx.x, head blockIdx.y, columns CB blockIdx.z ..; c_state holds the chunks' start states.
// A wave's 16 rotated queries go from global memory to its registers; keys (OB dimensions at a time), the state's
// rows (OB at a time) and the values (OB tokens at a time) pass through LDS in small pieces, so that several
// workgroups share a CU and hide each other's loads.
constexpr int OB = 32, OS = OB + 4;

template <typename T, int NCB, bool VEC>
__global__ __launch_bounds__(NT, NCB <= 4 ? 4 : NCB <= 8 ? 3 : 2) void retention_out_kernel(const T* __restrict__ p, int64_t stride, int H, int dk,
                                                           int dv, int gate, Rot rot, const float* __restrict__ powers,
                                                           int pw_stride, float eps, const int* __restrict__ c_start,
                                                           int c0, const float* __restrict__ c_state,
                                                           T* __restrict__ out, float* __restrict__ o_raw) {
  constexpr int CB = 16 * NCB, BS = CB + 4;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float sP[C + 1];
  float *sK = lds, *sB = lds + C * OS;  // sK [64 keys, OB]; sB [OB, CB]: a piece of the state, then of the values
  const int c = blockIdx.x, h = blockIdx.y, col0 = blockIdx.z * CB;
  const int64_t t0 = c_start[c0 + c];
  const int n = c_start[c0 + c + 1] - (int)t0;
  const int half = rot.dims >> 1;
  const float kscale = 1.f / sqrtf((float)dk);
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int r16 = lane & 15, kq = lane >> 4;
  if (threadIdx.x <= C) sP[threadIdx.x] = powers[(int64_t)h * pw_stride + threadIdx.x];
  const float* S0 = c_state + ((int64_t)c * H + h) * dk * dv;
  const int64_t pos0 = rot.positions[t0];  // a chunk's positions follow each other
  const int qi = wave * 16 + r16, qc = min(qi, n - 1);
  const T* q_row = p + (t0 + qc) * stride + h * dk;
  const float* q_cs = rot.cos_sin + (pos0 + qc) * rot.dims;
  f32x4_t o[NCB], w[4];  // o: rows 16 wave + 4 kq + r, column 16 m + r16; w[jb]: key 16 jb + 4 kq + r of query 16 wave + r16
#pragma unroll
  for (int m = 0; m < NCB; ++m) o[m] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int jb = 0; jb < 4; ++jb) w[jb] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int d0 = 0; d0 < dk; d0 += OB) {
    float a[OB / 16][4];  // this lane's query, dimensions d0 + 16 i + 4 kq .. (a row past n repeats the last one)
#pragma unroll
    for (int i = 0; i < OB / 16; ++i) rot4<T, VEC>(q_row, d0 + 16 * i + 4 * kq, dk, q_cs, half, a[i]);
    if (d0 > 0) __syncthreads();  // the previous piece is read
#pragma unroll
    for (int e0 = 0; e0 < C * (OB / 4); e0 += NT) {
      const int e = e0 + threadIdx.x;
      const int j = e / (OB / 4), d = (e - j * (OB / 4)) * 4, jc = min(j, n - 1);
      float b[4];
      rot4<T, VEC>(p + (t0 + jc) * stride + (H + h) * dk, d0 + d, dk, rot.cos_sin + (pos0 + jc) * rot.dims, half, b);
#pragma unroll
      for (int i = 0; i < 4; ++i) b[i] = j < n ? b[i] * kscale : 0.f;
      *reinterpret_cast<float4*>(&sK[j * OS + d]) = make_float4(b[0], b[1], b[2], b[3]);
    }
#pragma unroll
    for (int e0 = 0; e0 < OB * (CB / 4); e0 += NT) {
      const int e = e0 + threadIdx.x;
      const int d = e / (CB / 4), cc = (e - d * (CB / 4)) * 4;
      const float* src = S0 + (int64_t)min(d0 + d, dk - 1) * dv;
      float v[4] = {0.f, 0.f, 0.f, 0.f};
      if constexpr (VEC) {
        ld4(src + min(col0 + cc, dv - 4), v);
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = d0 + d < dk && col0 + cc < dv ? v[i] : 0.f;
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (d0 + d < dk && col0 + cc + i < dv) v[i] = src[col0 + cc + i];
      }
      *reinterpret_cast<float4*>(&sB[d * BS + cc]) = make_float4(v[0], v[1], v[2], v[3]);
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < OB / 16; ++i) {
      if (d0 + 16 * i >= dk) break;
#pragma unroll
      for (int jb = 0; jb < 4; ++jb) {
        if (jb > wave) break;  // keys after every query of this wave
        float b[4];
        ld4(&sK[(jb * 16 + r16) * OS + 16 * i + 4 * kq], b);
#pragma unroll
        for (int e = 0; e < 4; ++e) w[jb] = __builtin_amdgcn_mfma_f32_16x16x4f32(b[e], a[i][e], w[jb], 0, 0, 0);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e)
#pragma unroll
        for (int m = 0; m < NCB; ++m)
          o[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i][e], sB[(16 * i + 4 * kq + e) * BS + m * 16 + r16], o[m], 0, 0, 0);
    }
  }
  // decay of the state's part by the row, of a weight by the distance
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const float d = sP[wave * 16 + kq * 4 + r + 1];
#pragma unroll
    for (int m = 0; m < NCB; ++m) o[m][r] *= d;
  }
#pragma unroll
  for (int jb = 0; jb < 4; ++jb)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int dist = wave * 16 + r16 - (jb * 16 + kq * 4 + r);
      w[jb][r] = dist >= 0 ? w[jb][r] * sP[max(dist, 0)] : 0.f;
    }
#pragma unroll
  for (int j0 = 0; j0 < C; j0 += OB) {
    if (j0 >= n) break;
    __syncthreads();  // the previous piece is read
    stage_v<T, CB, OB, VEC>(p, stride, t0 + j0, n - j0, 2 * H * dk + h * dv, col0, dv, sB);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < OB / 16; ++i) {
      const int jb = j0 / 16 + i;
      if (jb > wave) break;
#pragma unroll
      for (int e = 0; e < 4; ++e)
#pragma unroll
        for (int m = 0; m < NCB; ++m)
          o[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(w[jb][e], sB[(16 * i + 4 * kq + e) * BS + m * 16 + r16], o[m], 0, 0, 0);
    }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int i = wave * 16 + kq * 4 + r;
    const int64_t t = t0 + i;
    if (o_raw != nullptr) {
      if (i < n) {
#pragma unroll
        for (int m = 0; m < NCB; ++m) {
          const int col = col0 + m * 16 + r16;
          if (col < dv) o_raw[(t * H + h) * dv + col] = o[m][r];
        }
      }
      continue;
    }
    float ss = 0.f;  // columns past dv are zero
#pragma unroll
    for (int m = 0; m < NCB; ++m) ss += o[m][r] * o[m][r];
#pragma unroll
    for (int x = 8; x > 0; x >>= 1) ss += __shfl_xor(ss, x, 64);
    const float inv = 1.f / sqrtf(ss / (float)dv + eps);
    float g[NCB];  // the row's gates: loads from clamped places, all in flight together
    if (gate) {
      const T* grow = p + (t0 + min(i, n - 1)) * stride + 2 * H * dk + H * dv + h * dv;
#pragma unroll
      for (int m = 0; m < NCB; ++m) g[m] = ld(grow + min(m * 16 + r16, dv - 1));
#pragma unroll
      for (int m = 0; m < NCB; ++m) o[m][r] *= Fn<T>::silu(g[m]);
    }
    if (i >= n) continue;
#pragma unroll
    for (int m = 0; m < NCB; ++m) {
      const int col = m * 16 + r16;
      if (col < dv) st(out + (t * H + h) * dv + col, o[m][r] * inv);
    }
  }
}

// out = o / rms(o) * silu(g) for tokens t0 + blockIdx.x; a wave per head.
template <typename T>
__global__ __launch_bounds__(NT) void retention_norm_kernel(const float* __restrict__ o_raw, const T* __restrict__ p,
                                                            int64_t stride, int H, int dk, int dv, int gate, float eps,
                                                            const int* __restrict__ first, T* __restrict__ out) {
  const int64_t t = *first + (int64_t)blockIdx.x;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  for (int h = blockIdx.y * (NT / 64) + wave; h < H; h += gridDim.y * (NT / 64)) {
    const float* orow = o_raw + (t * H + h) * dv;
    float ss = 0.f;
    for (int e = lane; e < dv; e += 64) ss += orow[e] * orow[e];
    const float inv = 1.f / sqrtf(wave_sum(ss) / (float)dv + eps);
    for (int e = lane; e < dv; e += 64) {
      float v = orow[e] * inv;
      if (gate) v *= Fn<T>::silu(ld(p + t * stride + 2 * H * dk + H * dv + h * dv + e));
      st(out + (t * H + h) * dv + e, v);
    }
  }
}

template <typename T>
int launch(const T* p, int64_t stride, int H, int dk, int dv, int gate, const Rot& rot, const float* powers, int pw_stride,
           float eps, float* state, const int* seq_start, const int* seq_slot, const int* seq_init, T* out, int T_rows,
           int nseq, int nd, int nc, const int* c_start, const int* s_chunk0, float* c_state, float* o_raw,
           hipStream_t stream) {
  const size_t es = sizeof(T);
  if (nd > 0) {
    const bool v4 = dv % 4 == 0 && ((uintptr_t)state & 15) == 0;
    const int cols = v4 ? dv / 4 : dv, ncg = std::min(cols, NT), RG = std::min(NT / ncg, dk);
    const size_t lds = (size_t)(2 * dk + RG * dv) * sizeof(float);
    if (lds > 64 * 1024) return 1;
    const dim3 grid(H, nd);
    if (v4)
      hipLaunchKernelGGL((retention_step_kernel<T, 4>), grid, dim3(NT), lds, stream, p, stride, H, dk, dv, gate, rot,
                         powers, pw_stride, eps, state, seq_start, seq_slot, seq_init, out, ncg, RG);
    else
      hipLaunchKernelGGL((retention_step_kernel<T, 1>), grid, dim3(NT), lds, stream, p, stride, H, dk, dv, gate, rot,
                         powers, pw_stride, eps, state, seq_start, seq_slot, seq_init, out, ncg, RG);
  }
  if (nd >= nseq) return 0;
  const int n = nc - nd;  // chunks of the longer runs
  // 16-byte pieces of the state, four elements of a projection row at a time
  const bool vec = dk % 4 == 0 && dv % 4 == 0 && (rot.dims >> 1) % 4 == 0 && stride % 4 == 0 &&
                   ((uintptr_t)p & (4 * es - 1)) == 0 && ((uintptr_t)rot.cos_sin & 15) == 0;
  auto set = [](const void* k, size_t lds) {
    if (lds > 64 * 1024) (void)hipFuncSetAttribute(k, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  };
#define SM_CHUNK(NCB, VEC)                                                                                            \
  {                                                                                                                   \
    const size_t lds = (size_t)(C * QS + C * (16 * NCB + 4)) * sizeof(float);                                         \
    const dim3 grid(n, H, ((dk + DB - 1) / DB) * ((dv + 16 * NCB - 1) / (16 * NCB)));                                 \
    set((const void*)retention_chunk_kernel<T, NCB, VEC>, lds);                                                       \
    hipLaunchKernelGGL((retention_chunk_kernel<T, NCB, VEC>), grid, dim3(NT), lds, stream, p, stride, H, dk, dv, rot, \
                       powers, pw_stride, c_start, nd, c_state);                                                      \
  }
  if (dv <= 64 && vec) SM_CHUNK(4, true)
  else if (dv <= 64) SM_CHUNK(4, false)
  else if (vec) SM_CHUNK(8, true)
  else SM_CHUNK(8, false)
#undef SM_CHUNK
  const int64_t per_head = (int64_t)dk * dv;
  // 16-byte pieces when that still leaves enough threads to fill the chip
  if (per_head % 4 == 0 && per_head * H * (nseq - nd) >= (int64_t)4 * 65536 && ((uintptr_t)state & 15) == 0 &&
      ((uintptr_t)c_state & 15) == 0)
    hipLaunchKernelGGL((retention_link_kernel<4>), dim3((unsigned)((per_head * H / 4 + NT - 1) / NT), nseq - nd), dim3(NT),
                       0, stream, c_state, c_start, s_chunk0, nd, nd, H, per_head, powers, pw_stride, state, seq_slot,
                       seq_init);
  else
    hipLaunchKernelGGL((retention_link_kernel<1>), dim3((unsigned)((per_head * H + NT - 1) / NT), nseq - nd), dim3(NT), 0,
                       stream, c_state, c_start, s_chunk0, nd, nd, H, per_head, powers, pw_stride, state, seq_slot,
                       seq_init);
#define SM_OUT(NCB, VEC)                                                                                              \
  {                                                                                                                   \
    const size_t lds = (size_t)(C * OS + OB * (16 * NCB + 4)) * sizeof(float);                                        \
    const dim3 grid(n, H, (dv + 16 * NCB - 1) / (16 * NCB));                                                          \
    set((const void*)retention_out_kernel<T, NCB, VEC>, lds);                                                         \
    hipLaunchKernelGGL((retention_out_kernel<T, NCB, VEC>), grid, dim3(NT), lds, stream, p, stride, H, dk, dv, gate,  \
                       rot, powers, pw_stride, eps, c_start, nd, c_state, out, o_raw);                                \
  }
#define SM_OUT2(VEC)                  \
  if (dv <= 64) SM_OUT(4, VEC)        \
  else if (dv <= 128) SM_OUT(8, VEC)  \
  else SM_OUT(16, VEC)
  if (vec) { SM_OUT2(true) }
  else { SM_OUT2(false) }
#undef SM_OUT2
#undef SM_OUT
  if (o_raw != nullptr) {
    const int rows = T_rows - nd;  // the longer runs' tokens follow the nd single ones
    hipLaunchKernelGGL((retention_norm_kernel<T>), dim3(rows, std::max(1, std::min((H + 3) / 4, 4096 / rows))), dim3(NT), 0,
                       stream, o_raw, p, stride, H, dk, dv, gate, eps, c_start + nd, out);
  }
  return 0;
}

}  // namespace

extern "C" {

int sm_retention_chunk() { return C; }
int sm_retention_cols() { return MAXCOLS; }

// The first nd sequences bring one token each; the chunks of the others are numbers nd .. nc - 1 of c_start [nc + 1],
// s_chunk0 [nseq + 1] bounds each sequence's chunks. Workspaces (fp32): c_state [nc - nd, H, dk, dv]; o_raw
// [T, H, dv] when dv > sm_retention_cols(), else null. Returns 0, or 1 when the sizes do not fit.
int sm_retention(const void* p, int64_t stride, int H, int dk, int dv, int gate, const int64_t* positions,
                 const float* cos_sin, int rot_dims, const float* powers, int pw_stride, float eps, float* state,
                 const int* seq_start, const int* seq_slot, const int* seq_init, void* out, int T, int nseq, int nd,
                 int f32, int nc, const int* c_start, const int* s_chunk0, float* c_state, float* o_raw,
                 hipStream_t stream) {
  const Rot rot{positions, cos_sin, rot_dims};
  if (f32)
    return launch<float>((const float*)p, stride, H, dk, dv, gate, rot, powers, pw_stride, eps, state, seq_start, seq_slot,
                         seq_init, (float*)out, T, nseq, nd, nc, c_start, s_chunk0, c_state, o_raw, stream);
  return launch<bf16_t>((const bf16_t*)p, stride, H, dk, dv, gate, rot, powers, pw_stride, eps, state, seq_start, seq_slot,
                        seq_init, (bf16_t*)out, T, nseq, nd, nc, c_start, s_chunk0, c_state, o_raw, stream);
}

}  // extern "C"
