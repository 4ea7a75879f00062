// gated_scan: a recurrence on every channel by itself, S_t = (1 - z_t) S_(t-1) + z_t c_t, with gates that do not depend on the state.
//   A row of `proj` holds z, u and g, `width` channels each:  z = sigmoid(proj_z + bias_z);  u = proj_u + bias_u;
//   c = u + shift (u >= 0) or sigmoid(u) (u < 0);  out[t] = S_t * silu(g).  The state is float32 [slots, width].
// Everything between a load and a store is float32.
//
// Steps whose portions fit one piece of GATED_PIECE tokens (decoding, short portions): one lane per channel walks the
// portion from the slot's state.  Longer portions are cut into pieces that are worked at the same time, in two passes over
// the rows:
//   gated_pieces_kernel: per piece and channel A = product of (1 - z) and B = the state the piece reaches from zero, into `scratch`
//     [sequence][1 + pieces][2][width]; the first entry is (0, the slot's state), which only this pass reads;
//   gated_scan_kernel: every piece folds the entries before it into the state it starts from, walks its tokens and writes
//     the outputs; a sequence's last piece writes the slot's state.
// (A lane with two neighbouring channels reads wider but leaves half the waves: 53 us for 2,048 tokens of 3,072 channels where
// one channel a lane takes 48.)
#include "common.h"

#define GATED_PIECE 32
#define GATED_AHEAD 4  // tokens whose loads are in flight together

struct GatedArgs {
  const void* proj;
  int width;
  const float* bias_z;
  const float* bias_u;
  float shift;
  float* state;
  const int* slots;
  const int* cu_q;
  void* out;
  float* scratch;  // nullptr: portions of one piece
  int entries;     // 1 + the pieces of the longest portion
};

// sigmoid(x) and 1 - sigmoid(x) = sigmoid(-x) (taken so, nothing is lost near 0) from one exponential and one reciprocal of a
// number between 1 and 2 (the hardware's, correct to one unit in the last place)
__device__ __forceinline__ void gated_sigmoids(float x, float& s, float& rest) {
  const float e = expf(-fabsf(x));
  const float large = __builtin_amdgcn_rcpf(1.f + e), small = e * large;
  s = x >= 0.f ? large : small;
  rest = x >= 0.f ? small : large;
}

// keep = 1 - z and add = z * candidate of one token and channel
__device__ __forceinline__ void gated_token(float xz, float xu, float shift, float& keep, float& add) {
  float z, below, unused;
  gated_sigmoids(xz, z, keep);
  gated_sigmoids(xu, below, unused);
  add = z * (xu >= 0.f ? xu + shift : below);
}

template <typename T>
__global__ void __launch_bounds__(128) gated_pieces_kernel(const GatedArgs a) {
  const int c = blockIdx.x * 128 + threadIdx.x;
  const int b = blockIdx.z, piece = blockIdx.y, W = a.width;
  const int lo = a.cu_q[b], hi = a.cu_q[b + 1];
  const int first = lo + piece * GATED_PIECE;
  if (c >= W || first >= hi) return;
  float* entry = a.scratch + (size_t)b * a.entries * 2 * W + c;
  if (piece == 0) {
    entry[0] = 0.f;
    entry[W] = a.state[(size_t)a.slots[b] * W + c];
  }
  if (first + GATED_PIECE >= hi) return;  // (a last piece: nobody folds it)
  const float bz = a.bias_z[c], bu = a.bias_u[c];
  float A = 1.f, B = 0.f;
  const T* row = (const T*)a.proj + (size_t)first * 3 * W + c;
  for (int t = 0; t < GATED_PIECE; t += GATED_AHEAD) {
    float z[GATED_AHEAD], u[GATED_AHEAD];
#pragma unroll
    for (int j = 0; j < GATED_AHEAD; ++j) {
      z[j] = to_f32(row[(size_t)(t + j) * 3 * W]);
      u[j] = to_f32(row[(size_t)(t + j) * 3 * W + W]);
    }
#pragma unroll
    for (int j = 0; j < GATED_AHEAD; ++j) {
      float keep, add;
      gated_token(z[j] + bz, u[j] + bu, a.shift, keep, add);
      A *= keep;
      B = keep * B + add;
    }
  }
  entry += (size_t)(piece + 1) * 2 * W;
  entry[0] = A;
  entry[W] = B;
}

template <typename T>
__global__ void __launch_bounds__(128) gated_scan_kernel(const GatedArgs a) {
  const int c = blockIdx.x * 128 + threadIdx.x;
  const int b = blockIdx.z, piece = blockIdx.y, W = a.width;
  const int lo = a.cu_q[b], hi = a.cu_q[b + 1];
  const int first = lo + piece * GATED_PIECE;
  if (c >= W || first >= hi) return;
  const int last = first + GATED_PIECE < hi ? first + GATED_PIECE : hi;
  float* my_state = a.state + (size_t)a.slots[b] * W + c;
  const float bz = a.bias_z[c], bu = a.bias_u[c];
  float s = 0.f;
  if (a.scratch) {
    const float* entry = a.scratch + (size_t)b * a.entries * 2 * W + c;
#pragma unroll 4
    for (int p = 0; p <= piece; ++p) s = entry[(size_t)p * 2 * W] * s + entry[(size_t)p * 2 * W + W];
  } else {
    s = *my_state;
  }
  const T* row = (const T*)a.proj + c;
  T* out = (T*)a.out + c;
  for (int t = first; t < last; t += GATED_AHEAD) {
    float z[GATED_AHEAD], u[GATED_AHEAD], g[GATED_AHEAD];
#pragma unroll
    for (int j = 0; j < GATED_AHEAD; ++j) {
      const size_t at = (size_t)(t + j < last ? t + j : last - 1) * 3 * W;  // (a place beyond the portion follows its last token and is not worked)
      z[j] = to_f32(row[at]);
      u[j] = to_f32(row[at + W]);
      g[j] = to_f32(row[at + 2 * W]);
    }
#pragma unroll
    for (int j = 0; j < GATED_AHEAD; ++j) {
      if (t + j < last) {
        float keep, add, open, unused;
        gated_token(z[j] + bz, u[j] + bu, a.shift, keep, add);
        gated_sigmoids(g[j], open, unused);
        s = keep * s + add;
        out[(size_t)(t + j) * W] = from_f32<T>(s * (g[j] * open));
      }
    }
  }
  if (last == hi) *my_state = s;
}

// float32 elements of the scratch that a step with portions of at most max_q_len tokens needs (0: none)
extern "C" long long velox_gated_scan_scratch_elems(int num_seqs, int max_q_len, int width) {
  const long long pieces = (max_q_len + GATED_PIECE - 1) / GATED_PIECE;
  return pieces <= 1 ? 0 : (long long)num_seqs * (1 + pieces) * 2 * width;
}

template <typename T>
static void gated_scan_launch(const GatedArgs& a, int pieces, int num_seqs, hipStream_t stream) {
  const dim3 grid((a.width + 127) / 128, pieces, num_seqs);
  if (a.scratch) gated_pieces_kernel<T><<<grid, 128, 0, stream>>>(a);
  gated_scan_kernel<T><<<grid, 128, 0, stream>>>(a);
}

extern "C" int velox_gated_scan(const void* proj, int dtype, int width, const float* bias_z, const float* bias_u, float shift, float* state, const int* slots,
                                const int* cu_q, void* out, float* scratch, int num_seqs, int max_q_len, hipStream_t stream) {
  if (num_seqs <= 0 || max_q_len <= 0) return 0;
  const int pieces = (max_q_len + GATED_PIECE - 1) / GATED_PIECE;
  if (width < 1 || num_seqs > 65535 || pieces > 65535 || (pieces > 1 && !scratch)) return (int)hipErrorInvalidValue;
  GatedArgs a{proj, width, bias_z, bias_u, shift, state, slots, cu_q, out, pieces > 1 ? scratch : nullptr, 1 + pieces};
  if (dtype == VELOX_BF16) gated_scan_launch<bf16_t>(a, pieces, num_seqs, stream);
  else gated_scan_launch<float>(a, pieces, num_seqs, stream);
  VELOX_RETURN_LAUNCH_STATUS();
}
