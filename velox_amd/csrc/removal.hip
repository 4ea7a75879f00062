// The generalized delta rule over long portions of prompts, in chunks of 16 tokens on the float32 matrix instructions.
//
// Per head, with decay w_t, unit key u_t, removal vector b_t = a_t * u_t, key k_t, value v_t and read vector r_t:
//     S_t = diag(w_t) S_(t-1) - b_t (u_t^T S_(t-1)) + k_t v_t^T,   o_t = S_t^T r_t.
// Inside a chunk let P_t = w_1 * .. * w_t (per channel, P_0 = 1) and S_t = diag(P_t) Z_t.  With
//     U_t = u_t * P_(t-1),  R_t = r_t * P_t,  B_t = b_t / P_t,  K_t = k_t / P_t       (rows of 16 x dim matrices)
// the rule reads Z_t = Z_(t-1) - B_t d_t + K_t v_t^T with the removed rows d_t = U_t Z_(t-1), so that
//     D = U Z_0 + M1 V - M2 D,   O = R Z_0 + M3 V - M4 D,   Z_16 = Z_0 + K^T V - B^T D,
// M1 = U K^T and M2 = U B^T below the diagonal, M3 = R K^T and M4 = R B^T with it.  With T = (I + M2)^-1 (unit lower
// triangular, by substitution) everything that does not touch the state is worked for all chunks at the same time:
//     U' = T U,   Dv = T M1 V,   R' = R - M4 T U,   Ov = M3 V - M4 Dv,
// and what is left of the dependent chain is, per chunk,   D = U' Z_0 + Dv,   O = R' Z_0 + Ov,   S = diag(P_16) (Z_0 + K^T V - B^T D).
// All of it is float32.  A decay is at least exp(-scale), so P_16 is at least exp(-16 scale); the host takes these kernels only while
// 16 scale < 13 (P_16 > 2e-6), and products of rows hold P_t / P_j <= 1 for j <= t: nothing overflows and nothing cancels.
//
//   removal_chunk_prepare_kernel   a workgroup per chunk and head: unit keys, removal vectors, the decay's low-rank map, the four
//                                  products, T, and the matrices above into `scratch`
//   removal_chunk_scan_kernel      a workgroup per 16 value columns, head and sequence; a wave holds 16 rows of the state in the
//                                  matrix instructions' result layout, which is also their operand layout, so that the state
//                                  never leaves the registers; the waves exchange their parts of D and O through LDS
#include "common.h"

#define CHUNK 16
#define CHUNK_STRIDE 20  // floats between the rows of a 16 x 16 matrix in LDS (16-byte aligned, rows on different banks)

struct RemovalChunkArgs {
  const void* main;  // [T, ld]
  int ld, r_at, k_at, v_at, a_at, low_at, rank, heads, dim, vdim;
  const float* a_bias;
  const void* w2;
  const float* w0;
  float scale;
  float* scratch;
  float* state;  // [slots, heads, dim, vdim]
  const int* slots;
  const int* cu_q;
  float* out;  // [T, heads * vdim]
};

// A chunk and head in `scratch`, in floats: U' | R' | -B | K (each 16 * dim), P_16 (dim), Dv | Ov (each 16 * columns).  U' and R' as
// [dim / 16][16 tokens][16 channels], B and K as [dim][16 tokens], Dv and Ov as [columns][16 tokens]: what a wave reads of one
// of them is one contiguous kilobyte, 16 bytes a lane.
__host__ __device__ __forceinline__ int removal_columns(int vdim) { return (vdim + 15) / 16 * 16; }
__host__ __device__ __forceinline__ size_t removal_record(int dim, int vdim) { return (size_t)65 * dim + 32 * removal_columns(vdim); }
// the first record of a sequence: sequences' chunks never overlap, because floor((a + n) / 16) + 1 >= floor(a / 16) + ceil(n / 16)
__device__ __forceinline__ int removal_first_chunk(int first_token, int sequence) { return first_token / CHUNK + sequence; }

__device__ __forceinline__ float removal_sigmoid(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float4_t mfma4(float a, float b, float4_t c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
__device__ __forceinline__ float4_t lds4(const float* p) { return *reinterpret_cast<const float4_t*>(p); }

template <typename T>
__global__ void __launch_bounds__(256) removal_chunk_prepare_kernel(const RemovalChunkArgs a) {
  extern __shared__ float4_t lds_pieces[];
  float* lds = reinterpret_cast<float*>(lds_pieces);
  const int h = blockIdx.x, b = blockIdx.z;
  const int lo = a.cu_q[b], hi = a.cu_q[b + 1];
  const int t0 = lo + blockIdx.y * CHUNK;
  if (t0 >= hi) return;  // (the whole workgroup)
  const int count = hi - t0 < CHUNK ? hi - t0 : CHUNK;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int n = lane & 15, g = lane >> 4;  // column and group of four rows in the matrix instructions' layouts
  const int dim = a.dim, rank = a.rank, row = dim + 4;
  const int padded_rank = (rank + 15) / 16 * 16, inner_row = padded_rank + 4;
  // four matrices of 16 rows (U, R, B, K), the decays, the map's inner rows, and 16 x 16 matrices: M1..M4, T, M4 T, T M1
  float* matrix[4] = {lds, lds + CHUNK * row, lds + 2 * CHUNK * row, lds + 3 * CHUNK * row};
  float* decays = lds + 4 * CHUNK * row;
  float* inner = decays + CHUNK * row;
  float* small = inner + CHUNK * inner_row;
  const T* rows = (const T*)a.main + (size_t)t0 * a.ld;

  for (int i = tid; i < CHUNK * padded_rank; i += 256) {
    const int j = i / padded_rank, m = i - j * padded_rank;
    inner[j * inner_row + m] = j < count && m < rank ? tanhf(to_f32(rows[(size_t)j * a.ld + a.low_at + m])) : 0.f;
  }
  const float* bias = a.a_bias + (size_t)h * dim;
  for (int j = wave; j < CHUNK; j += 4) {  // (tokens beyond the portion: zeros, with decays of 1)
    const T* mine = rows + (size_t)j * a.ld + (size_t)h * dim;
    float s = 0.f;
    if (j < count)
      for (int c = lane; c < dim; c += 64) { const float v = to_f32(mine[a.k_at + c]); s += v * v; }
    const float inv = 1.f / sqrtf(wave_sum(s) + 1e-6f);
    for (int c = lane; c < dim; c += 64) {
      float r = 0.f, k = 0.f, u = 0.f, removal = 0.f;
      if (j < count) {
        r = to_f32(mine[a.r_at + c]);
        k = to_f32(mine[a.k_at + c]);
        u = k * inv;
        removal = removal_sigmoid(to_f32(mine[a.a_at + c]) + bias[c]) * u;
      }
      matrix[0][j * row + c] = u;
      matrix[1][j * row + c] = r;
      matrix[2][j * row + c] = removal;
      matrix[3][j * row + c] = k;
    }
  }
  __syncthreads();
  // the decays: 16 channels x 16 tokens at a time, w2 [channel, m] times the inner rows; a lane ends with four neighbouring channels
  // of token n
  for (int tile = wave; tile < dim / 16; tile += 4) {
    const size_t channel = (size_t)h * dim + tile * 16;
    const T* w = (const T*)a.w2 + (channel + n) * rank;
    float4_t z = {0.f, 0.f, 0.f, 0.f};
    for (int m = 4 * g; m < padded_rank; m += 16) {
      const float4_t x = lds4(inner + n * inner_row + m);
#pragma unroll
      for (int e = 0; e < 4; ++e) z = mfma4(m + e < rank ? to_f32(w[m + e]) : 0.f, x[e], z);
    }
    float4_t dec;
#pragma unroll
    for (int i = 0; i < 4; ++i) dec[i] = n < count ? expf(-a.scale * removal_sigmoid(a.w0[channel + 4 * g + i] + z[i])) : 1.f;
    *reinterpret_cast<float4_t*>(decays + n * row + tile * 16 + 4 * g) = dec;
  }
  __syncthreads();
  // the running products and the scaled rows; a lane walks one channel of one of the four matrices
  const int record_at = removal_first_chunk(lo, b) + blockIdx.y;
  float* record = a.scratch + ((size_t)record_at * a.heads + h) * removal_record(dim, a.vdim);
  float* record_b = record + 32 * dim;
  float* record_k = record + 48 * dim;
  float* record_p = record + 64 * dim;
  for (int i = tid; i < 4 * dim; i += 256) {
    const int which = i / dim, c = i - which * dim;
    float* column = matrix[which] + c;
    float p = 1.f;
    float4_t kept[4];
#pragma unroll
    for (int t = 0; t < CHUNK; ++t) {
      const float before = p;
      p *= decays[t * row + c];
      const float v = column[t * row] * (which == 0 ? before : which == 1 ? p : 1.f / p);
      column[t * row] = v;
      kept[t >> 2][t & 3] = which == 2 ? -v : v;
    }
    if (which >= 2) {
      float* to = (which == 2 ? record_b : record_k) + (size_t)c * CHUNK;
#pragma unroll
      for (int q = 0; q < 4; ++q) *reinterpret_cast<float4_t*>(to + 4 * q) = kept[q];
    }
    if (which == 0) record_p[c] = p;
  }
  __syncthreads();
  // M1 = U K^T, M2 = U B^T (below the diagonal), M3 = R K^T, M4 = R B^T (with it): a wave each
  {
    const float* left = matrix[wave < 2 ? 0 : 1] + n * row;
    const float* right = matrix[(wave & 1) ? 2 : 3] + n * row;
    float4_t m = {0.f, 0.f, 0.f, 0.f};
    for (int c = 4 * g; c < dim; c += 16) {
      const float4_t x = lds4(left + c), y = lds4(right + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) m = mfma4(x[e], y[e], m);
    }
    float* to = small + wave * CHUNK * CHUNK_STRIDE;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 4 * g + i;
      to[t * CHUNK_STRIDE + n] = n < t || (wave >= 2 && n == t) ? m[i] : 0.f;
    }
  }
  __syncthreads();
  const float* M1 = small;
  const float* M2 = small + CHUNK * CHUNK_STRIDE;
  const float* M3 = small + 2 * CHUNK * CHUNK_STRIDE;
  const float* M4 = small + 3 * CHUNK * CHUNK_STRIDE;
  float* inverse = small + 4 * CHUNK * CHUNK_STRIDE;
  float* M4T = small + 5 * CHUNK * CHUNK_STRIDE;
  float* TM1 = small + 6 * CHUNK * CHUNK_STRIDE;
  if (wave == 0) {  // column n of T, by substitution (the four groups of lanes do the same)
    float x[CHUNK];
#pragma unroll
    for (int t = 0; t < CHUNK; ++t) {
      float v = t == n ? 1.f : 0.f;
#pragma unroll
      for (int q = 0; q < (t + 3) / 4; ++q) {
        const float4_t m = lds4(M2 + t * CHUNK_STRIDE + 4 * q);
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (4 * q + e < t) v -= m[e] * x[4 * q + e];
      }
      x[t] = v;
    }
    if (g == 0) {
#pragma unroll
      for (int t = 0; t < CHUNK; ++t) inverse[t * CHUNK_STRIDE + n] = x[t];
    }
  }
  __syncthreads();
  if (wave < 2) {  // M4 T and T M1
    const float4_t x = lds4((wave == 0 ? M4 : inverse) + n * CHUNK_STRIDE + 4 * g);
    const float* y = (wave == 0 ? inverse : M1) + 4 * g * CHUNK_STRIDE + n;
    float4_t m = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e) m = mfma4(x[e], y[e * CHUNK_STRIDE], m);
    float* to = wave == 0 ? M4T : TM1;
#pragma unroll
    for (int i = 0; i < 4; ++i) to[(4 * g + i) * CHUNK_STRIDE + n] = m[i];
  }
  __syncthreads();
  const float4_t t4 = lds4(inverse + n * CHUNK_STRIDE + 4 * g), m4t = lds4(M4T + n * CHUNK_STRIDE + 4 * g);
  for (int tile = wave; tile < dim / 16; tile += 4) {  // U' and R', 16 channels at a time
    float4_t up = {0.f, 0.f, 0.f, 0.f}, rp;
#pragma unroll
    for (int i = 0; i < 4; ++i) rp[i] = matrix[1][(4 * g + i) * row + tile * 16 + n];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float y = matrix[0][(4 * g + e) * row + tile * 16 + n];
      up = mfma4(t4[e], y, up);
      rp = mfma4(-m4t[e], y, rp);
    }
    float* to = record + tile * 256 + n;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      to[(4 * g + i) * 16] = up[i];
      to[16 * dim + (4 * g + i) * 16] = rp[i];
    }
  }
  const float4_t m3 = lds4(M3 + n * CHUNK_STRIDE + 4 * g), m4 = lds4(M4 + n * CHUNK_STRIDE + 4 * g), tm1 = lds4(TM1 + n * CHUNK_STRIDE + 4 * g);
  const int columns = removal_columns(a.vdim);
  float* record_d = record + 65 * dim;
  for (int tile = wave; tile < columns / 16; tile += 4) {  // Dv and Ov, 16 columns of values at a time
    const int column = tile * 16 + n;
    const T* values = rows + a.v_at + (size_t)h * a.vdim + (column < a.vdim ? column : a.vdim - 1);
    float4_t v, dv = {0.f, 0.f, 0.f, 0.f}, ov = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = 4 * g + e < count ? to_f32(values[(size_t)(4 * g + e) * a.ld]) : 0.f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      dv = mfma4(tm1[e], v[e], dv);
      ov = mfma4(m3[e], v[e], ov);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) ov = mfma4(-m4[e], dv[e], ov);
    *reinterpret_cast<float4_t*>(record_d + (size_t)column * CHUNK + 4 * g) = dv;
    *reinterpret_cast<float4_t*>(record_d + (size_t)(columns + column) * CHUNK + 4 * g) = ov;
  }
}

// What a wave reads of one chunk, in registers: loaded SCAN_AHEAD chunks before it is worked.
struct RemovalOperands {
  float4_t up, rp, nb, k, p, dv;
  float v[4];
};
#define SCAN_AHEAD 4

template <typename T, int WAVES>
__global__ void __launch_bounds__(64 * WAVES) removal_chunk_scan_kernel(const RemovalChunkArgs a) {
  __shared__ float4_t parts[2][2][WAVES][64];  // [buffer][D, O][wave][lane]
  const int tile = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
  const int lo = a.cu_q[b], hi = a.cu_q[b + 1];
  if (hi <= lo) return;  // (the whole workgroup)
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int n = lane & 15, g = lane >> 4;
  constexpr int dim = 16 * WAVES;
  const int vdim = a.vdim, columns = removal_columns(vdim);
  const int column = tile * 16 + n;
  const bool live = column < vdim;
  const int col = live ? column : vdim - 1;
  const int chunks = (hi - lo + CHUNK - 1) / CHUNK;
  const size_t stride = (size_t)a.heads * removal_record(dim, vdim);  // between a sequence's records of this head
  const float* records = a.scratch + ((size_t)removal_first_chunk(lo, b) * a.heads + h) * removal_record(dim, vdim);
  const T* values = (const T*)a.main + (size_t)lo * a.ld + a.v_at + (size_t)h * vdim + col;
  const int last_row = hi - lo - 1;

  auto load = [&](int c, RemovalOperands& o) {
    const float* record = records + (size_t)c * stride;
    const int at = wave * 256 + n * 16 + 4 * g;
    o.up = lds4(record + at);
    o.rp = lds4(record + 16 * dim + at);
    o.nb = lds4(record + 32 * dim + at);
    o.k = lds4(record + 48 * dim + at);
    o.p = lds4(record + 64 * dim + wave * 16 + 4 * g);
    o.dv = lds4(record + 65 * dim + (size_t)column * CHUNK + 4 * g);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = c * CHUNK + 4 * g + e;  // (rows beyond the portion follow its last one: their keys are zero)
      o.v[e] = to_f32(values[(size_t)(t < last_row ? t : last_row) * a.ld]);
    }
  };

  float* S = a.state + (((size_t)a.slots[b] * a.heads + h) * dim + wave * 16 + 4 * g) * vdim + col;
  float4_t z;
#pragma unroll
  for (int i = 0; i < 4; ++i) z[i] = S[(size_t)i * vdim];

  RemovalOperands ops[SCAN_AHEAD];
#pragma unroll
  for (int c = 0; c < SCAN_AHEAD; ++c)
    if (c < chunks) load(c, ops[c]);
  for (int c0 = 0; c0 < chunks; c0 += SCAN_AHEAD) {
#pragma unroll
    for (int j = 0; j < SCAN_AHEAD; ++j) {
      const int c = c0 + j;
      if (c >= chunks) break;  // (the same for the whole workgroup)
      RemovalOperands& o = ops[j];
      float4_t d = {0.f, 0.f, 0.f, 0.f}, read = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        d = mfma4(o.up[e], z[e], d);
        read = mfma4(o.rp[e], z[e], read);
      }
      parts[j & 1][0][wave][lane] = d;
      parts[j & 1][1][wave][lane] = read;
#pragma unroll
      for (int e = 0; e < 4; ++e) z = mfma4(o.k[e], o.v[e], z);
      __syncthreads();  // (one a chunk: a buffer is written again behind the next chunk's barrier)
      d = o.dv;
#pragma unroll
      for (int w = 0; w < WAVES; ++w) d += parts[j & 1][0][w][lane];
#pragma unroll
      for (int e = 0; e < 4; ++e) z = mfma4(o.nb[e], d[e], z);
      z *= o.p;
      // the chunk's read-outs: 256 of them over the workgroup's lanes
      const float* sums = reinterpret_cast<const float*>(parts[j & 1][1]);
      const float* ov = records + (size_t)c * stride + 65 * dim + (size_t)(columns + tile * 16) * CHUNK;
      for (int i = tid; i < 256; i += 64 * WAVES) {
        const int t = (i >> 6) * 4 + (i & 3), e = (i >> 2) & 15;  // (the order in which the parts lie in LDS)
        float v = ov[e * CHUNK + t];
#pragma unroll
        for (int w = 0; w < WAVES; ++w) v += sums[w * 256 + i];
        const int token = c * CHUNK + t;
        if (token <= last_row && tile * 16 + e < vdim) a.out[((size_t)(lo + token) * a.heads + h) * vdim + tile * 16 + e] = v;
      }
      if (c + SCAN_AHEAD < chunks) load(c + SCAN_AHEAD, o);
    }
  }
  if (live) {
#pragma unroll
    for (int i = 0; i < 4; ++i) S[(size_t)i * vdim] = z[i];
  }
}

static size_t removal_prepare_lds(int dim, int rank) {
  const int padded_rank = (rank + 15) / 16 * 16;
  return (size_t)CHUNK * (5 * (dim + 4) + padded_rank + 4 + 7 * CHUNK_STRIDE) * sizeof(float);
}

// float32 elements of the scratch of a step; 0: these sizes are not for these kernels
extern "C" long long velox_removal_chunk_scratch_elems(int tokens, int num_seqs, int heads, int dim, int vdim, int rank) {
  if (dim % 16 != 0 || dim < 16 || dim > 128 || vdim < 1 || rank < 1 || removal_prepare_lds(dim, rank) > 64 * 1024) return 0;
  return ((long long)tokens / CHUNK + num_seqs + 1) * heads * (long long)removal_record(dim, vdim);
}

template <typename T>
static void removal_chunk_launch(const RemovalChunkArgs& a, int num_seqs, int max_q_len, hipStream_t stream) {
  const int chunks = (max_q_len + CHUNK - 1) / CHUNK;
  removal_chunk_prepare_kernel<T><<<dim3(a.heads, chunks, num_seqs), 256, removal_prepare_lds(a.dim, a.rank), stream>>>(a);
  const dim3 grid(removal_columns(a.vdim) / 16, a.heads, num_seqs);
  switch (a.dim / 16) {
    case 1: removal_chunk_scan_kernel<T, 1><<<grid, 64, 0, stream>>>(a); break;
    case 2: removal_chunk_scan_kernel<T, 2><<<grid, 128, 0, stream>>>(a); break;
    case 3: removal_chunk_scan_kernel<T, 3><<<grid, 192, 0, stream>>>(a); break;
    case 4: removal_chunk_scan_kernel<T, 4><<<grid, 256, 0, stream>>>(a); break;
    case 5: removal_chunk_scan_kernel<T, 5><<<grid, 320, 0, stream>>>(a); break;
    case 6: removal_chunk_scan_kernel<T, 6><<<grid, 384, 0, stream>>>(a); break;
    case 7: removal_chunk_scan_kernel<T, 7><<<grid, 448, 0, stream>>>(a); break;
    default: removal_chunk_scan_kernel<T, 8><<<grid, 512, 0, stream>>>(a); break;
  }
}

extern "C" int velox_removal_chunk_scan(const void* main, int dtype, int ld, int r_at, int k_at, int v_at, int a_at, int low_at, int rank, int heads, int dim,
                                        int vdim, const float* a_bias, const void* w2, const float* w0, float scale, float* scratch, float* state,
                                        const int* slots, const int* cu_q, float* out, int num_seqs, int max_q_len, hipStream_t stream) {
  if (num_seqs <= 0 || max_q_len <= 0) return 0;
  if (velox_removal_chunk_scratch_elems(max_q_len, num_seqs, heads, dim, vdim, rank) == 0 || heads < 1 || heads > 65535 || num_seqs > 65535 ||
      max_q_len > 65535 * CHUNK || !scratch || !(scale * CHUNK < 13.f))
    return (int)hipErrorInvalidValue;
  RemovalChunkArgs a{main, ld, r_at, k_at, v_at, a_at, low_at, rank, heads, dim, vdim, a_bias, w2, w0, scale, scratch, state, slots, cu_q, out};
  if (dtype == VELOX_BF16) removal_chunk_launch<bf16_t>(a, num_seqs, max_q_len, stream);
  else removal_chunk_launch<float>(a, num_seqs, max_q_len, stream);
  VELOX_RETURN_LAUNCH_STATUS();
}
