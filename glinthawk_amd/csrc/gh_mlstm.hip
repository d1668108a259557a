// Matrix-memory LSTM (the mLSTM of xLSTM: Beck et al., "xLSTM: Extended Long Short-Term Memory"): exponential input gate and sigmoid
// forget gate in log space with a running maximum m (starting at 0), a matrix S and a vector n per head.
//
//   m' = max(f + m, i);  S' = e^(f + m - m') S + e^(i - m') k v^T;  n' likewise with k;  o = S'^T q / (max(|n' . q|, e^(-m')) + 1e-6)
//
// gates   i = cap tanh((. + b) / cap), f = logsigmoid(cap tanh((. + b) / cap))
// state   fp32, per context and head: S (dim x vdim_padded), then n (heads x dim), then m (heads); zero at position 0, which the kernels
//         take from the position (a slot that is used again needs no clearing)
// walk    work-group = 64 columns of v of one (context, head); it keeps its (dim x 64) part of S in registers over all the tokens of the
//         call (one for decode) and streams it in and out of memory once.  n and m are needed by every column slice: each slice carries
//         its own copy and the finishing kernel writes them back, so no slice reads what another one has already replaced.
// finish  one work-group per token: each head's output divided by its root mean square, times a weight, times sigmoid(g)
#include "gh_product.h"

#include <algorithm>

namespace gh {
namespace {

constexpr uint32_t SLICE = 64; // columns of v per work-group of the walk

struct MlstmShape
{
  uint32_t heads, dim, vdim, vpad;
  float cap, eps, q_scale;
  // elements of the state of one context
  __host__ __device__ uint64_t n_off() const { return (uint64_t)heads * dim * vpad; }
  __host__ __device__ uint64_t m_off() const { return n_off() + (uint64_t)heads * dim; }
  __host__ __device__ uint64_t elements() const { return m_off() + heads; }
};

__device__ __forceinline__ float soft_cap( float z, float cap ) { return cap * tanhf( z / cap ); }
// log(sigmoid(z)), stable for either sign
__device__ __forceinline__ float log_sigmoid( float z ) { return fminf( z, 0.0f ) - log1pf( expf( -fabsf( z ) ) ); }

// columns of the products: [q | k | v | g] in one, [i | f] in the other
struct MlstmCols
{
  uint32_t q, k, v, g, i, f;
};

template<typename E, typename View>
struct MlstmIn
{
  View main;
  ProductView<float> gates;
  MlstmCols col;
  const E *bias_i, *bias_f;
};

struct MlstmState
{
  void* const* rows;         // state region of each context; NULL: no context
  uint64_t offset;           // bytes from there to this layer's state
  const uint32_t* start_pos; // position of the first token of the call
  uint32_t n_tokens;
};

// RPT: rows of S per thread kept in registers (0: S stays in memory, any dim)
template<typename E, typename View, int RPT>
__global__ __launch_bounds__( 256 ) void mlstm_walk_kernel( float* __restrict__ o_out, float* __restrict__ nm_out, MlstmIn<E, View> in, MlstmState st, MlstmShape s )
{
  extern __shared__ float lds[];
  const uint32_t dim4 = ( s.dim + 3 ) / 4 * 4; // v_s and red are read as float4
  float* q_s = lds;               // dim
  float* k_s = q_s + dim4;        // dim
  float* n_s = k_s + dim4;        // dim
  float* v_s = n_s + s.dim;       // SLICE
  float* nq_s = v_s + SLICE;      // 16
  float* red = nq_s + 16;         // 16 x SLICE
  const uint32_t slice = blockIdx.x, h = blockIdx.y, ctx = blockIdx.z;
  uint8_t* base = static_cast<uint8_t*>( st.rows[ctx] );
  if ( base == nullptr ) {
    return;
  }
  float* S = reinterpret_cast<float*>( base + st.offset );
  const float* n_in = S + s.n_off() + (uint64_t)h * s.dim;
  const float* m_in = S + s.m_off() + h;
  S += (uint64_t)h * s.dim * s.vpad;
  const bool fresh = st.start_pos[ctx] == 0;
  const uint32_t t = threadIdx.x;
  const uint32_t cl = t & 15, rg = t >> 4;
  const uint32_t c0 = slice * SLICE + cl * 4;
  const bool col_live = c0 < s.vpad;
  constexpr int R = RPT > 0 ? RPT : 1;
  float4 reg[R];
  if constexpr ( RPT > 0 ) {
#pragma unroll
    for ( int r = 0; r < RPT; r++ ) {
      const uint32_t row = rg + 16 * r;
      reg[r] = make_float4( 0.0f, 0.0f, 0.0f, 0.0f );
      if ( !fresh && row < s.dim && col_live ) {
        reg[r] = *reinterpret_cast<const float4*>( S + (uint64_t)row * s.vpad + c0 );
      }
    }
  } else if ( fresh && col_live ) {
    for ( uint32_t row = rg; row < s.dim; row += 16 ) {
      *reinterpret_cast<float4*>( S + (uint64_t)row * s.vpad + c0 ) = make_float4( 0.0f, 0.0f, 0.0f, 0.0f );
    }
  }
  for ( uint32_t d = t; d < s.dim; d += 256 ) {
    n_s[d] = fresh ? 0.0f : n_in[d];
  }
  float m = fresh ? 0.0f : *m_in;
  const float bi = in.bias_i != nullptr ? to_f32( in.bias_i[h] ) : 0.0f, bf = in.bias_f != nullptr ? to_f32( in.bias_f[h] ) : 0.0f;

  for ( uint32_t tok = 0; tok < st.n_tokens; tok++ ) {
    const uint64_t row_in = (uint64_t)ctx * st.n_tokens + tok;
    __syncthreads(); // the previous token's readers are done (and n_s is written)
    for ( uint32_t d = t; d < s.dim; d += 256 ) {
      q_s[d] = in.main.at( row_in, in.col.q + h * s.dim + d ) * s.q_scale;
      k_s[d] = in.main.at( row_in, in.col.k + h * s.dim + d );
    }
    if ( t < SLICE ) {
      const uint32_t c = slice * SLICE + t;
      v_s[t] = c < s.vdim ? in.main.at( row_in, in.col.v + h * s.vdim + c ) : 0.0f;
    }
    const float gi = soft_cap( in.gates.at( row_in, in.col.i + h ) + bi, s.cap );
    const float gf = log_sigmoid( soft_cap( in.gates.at( row_in, in.col.f + h ) + bf, s.cap ) );
    const float m_new = fmaxf( gf + m, gi );
    const float decay = expf( gf + m - m_new ), inp = expf( gi - m_new );
    m = m_new;
    __syncthreads();
    const float4 v4 = *reinterpret_cast<const float4*>( v_s + cl * 4 );
    float4 acc = make_float4( 0.0f, 0.0f, 0.0f, 0.0f );
    auto row_step = [&]( float4& x, uint32_t row ) {
      const float kk = inp * k_s[row], qq = q_s[row];
      x.x = decay * x.x + kk * v4.x;
      x.y = decay * x.y + kk * v4.y;
      x.z = decay * x.z + kk * v4.z;
      x.w = decay * x.w + kk * v4.w;
      acc.x += qq * x.x;
      acc.y += qq * x.y;
      acc.z += qq * x.z;
      acc.w += qq * x.w;
    };
    if constexpr ( RPT > 0 ) {
#pragma unroll
      for ( int r = 0; r < RPT; r++ ) {
        const uint32_t row = rg + 16 * r;
        if ( row < s.dim ) {
          row_step( reg[r], row );
        }
      }
    } else if ( col_live ) {
      for ( uint32_t row = rg; row < s.dim; row += 16 ) {
        float4* p = reinterpret_cast<float4*>( S + (uint64_t)row * s.vpad + c0 );
        float4 x = *p;
        row_step( x, row );
        *p = x;
      }
    }
    // n: one owner per element; its product with q by the sixteen row groups
    float nq = 0.0f;
    for ( uint32_t row = rg + 16 * cl; row < s.dim; row += 256 ) {
      const float x = decay * n_s[row] + inp * k_s[row];
      n_s[row] = x;
      nq += x * q_s[row];
    }
    nq = row16_sum( nq );
    if ( cl == 0 ) {
      nq_s[rg] = nq;
    }
    *reinterpret_cast<float4*>( red + rg * SLICE + cl * 4 ) = acc;
    __syncthreads();
    if ( t < SLICE && slice * SLICE + t < s.vdim ) {
      float num = 0.0f, den = 0.0f;
#pragma unroll
      for ( int r = 0; r < 16; r++ ) {
        num += red[r * SLICE + t];
        den += nq_s[r];
      }
      o_out[row_in * s.heads * s.vdim + h * s.vdim + slice * SLICE + t] = num / ( fmaxf( fabsf( den ), expf( -m ) ) + 1e-6f );
    }
  }
  if constexpr ( RPT > 0 ) {
#pragma unroll
    for ( int r = 0; r < RPT; r++ ) {
      const uint32_t row = rg + 16 * r;
      if ( row < s.dim && col_live ) {
        *reinterpret_cast<float4*>( S + (uint64_t)row * s.vpad + c0 ) = reg[r];
      }
    }
  }
  if ( slice == 0 ) {
    float* dst = nm_out + ( (uint64_t)ctx * s.heads + h ) * ( s.dim + 1 );
    for ( uint32_t row = t; row < s.dim; row += 256 ) { // (the owners wrote before the last barrier)
      dst[row] = n_s[row];
    }
    if ( t == 0 ) {
      dst[s.dim] = m;
    }
  }
}

// one work-group per token, one wave per head in turn
template<typename E, typename View>
__global__ __launch_bounds__( 256 ) void mlstm_finish_kernel( E* __restrict__ out,
                                                              const float* __restrict__ o,
                                                              const float* __restrict__ nm,
                                                              MlstmIn<E, View> in,
                                                              const E* __restrict__ norm,
                                                              MlstmState st,
                                                              MlstmShape s )
{
  const uint64_t row = blockIdx.x;
  const uint32_t ctx = (uint32_t)( row / st.n_tokens ), tok = (uint32_t)( row % st.n_tokens );
  uint8_t* base = static_cast<uint8_t*>( st.rows[ctx] );
  if ( base == nullptr ) {
    return;
  }
  const uint32_t wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  for ( uint32_t h = wave; h < s.heads; h += 4 ) {
    const float* oh = o + row * s.heads * s.vdim + (uint64_t)h * s.vdim;
    float ss = 0.0f;
    for ( uint32_t c = lane; c < s.vdim; c += 64 ) {
      ss += oh[c] * oh[c];
    }
    const float inv = 1.0f / sqrtf( wave_sum( ss ) / (float)s.vdim + s.eps );
    for ( uint32_t c = lane; c < s.vdim; c += 64 ) {
      const uint32_t hc = h * s.vdim + c;
      const float g = in.main.at( row, in.col.g + hc );
      out[row * s.heads * s.vdim + hc] = from_f32<E>( oh[c] * inv * to_f32( norm[hc] ) / ( 1.0f + expf( -g ) ) );
    }
  }
  if ( tok + 1 == st.n_tokens ) {
    float* S = reinterpret_cast<float*>( base + st.offset );
    for ( uint32_t h = 0; h < s.heads; h++ ) {
      const float* src = nm + ( (uint64_t)ctx * s.heads + h ) * ( s.dim + 1 );
      for ( uint32_t d = threadIdx.x; d <= s.dim; d += blockDim.x ) {
        if ( d < s.dim ) {
          S[s.n_off() + (uint64_t)h * s.dim + d] = src[d];
        } else {
          S[s.m_off() + h] = src[d];
        }
      }
    }
  }
}

MlstmShape shape_of( const gh_mlstm* m )
{
  MlstmShape s;
  s.heads = m->heads;
  s.dim = m->dim;
  s.vdim = m->vdim;
  s.vpad = ( m->vdim + 3 ) / 4 * 4;
  s.cap = m->gate_cap;
  s.eps = m->eps;
  s.q_scale = 1.0f / sqrtf( (float)m->dim );
  return s;
}

} // namespace
} // namespace gh

using namespace gh;

extern "C" {

uint64_t gh_mlstm_state_bytes( const gh_mlstm* m ) { return shape_of( m ).elements() * sizeof( float ); }

uint64_t gh_mlstm_weight_rows( const gh_mlstm* m, uint64_t* gate_row )
{
  const uint64_t main = 2ull * m->heads * m->dim + 2ull * m->heads * m->vdim;
  const uint64_t first = ( main + 7 ) / 8 * 8;
  if ( gate_row != nullptr ) {
    *gate_row = first;
  }
  return first + ( 2ull * m->heads + 7 ) / 8 * 8;
}

int gh_mlstm_forward( void* out, const void* x, const void* w, uint64_t width, const gh_mlstm* m, const void* bias_i, const void* bias_f, const void* norm,
                      void* const* context_rows_dev, uint64_t state_offset, const uint32_t* start_pos_dev, uint64_t batch, uint32_t n_tokens, gh_dtype dt,
                      gh_stream stream )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  const uint64_t rows = batch * n_tokens;
  if ( rows == 0 ) {
    return GH_OK;
  }
  GH_REQUIRE( out && x && w && m && norm && context_rows_dev && start_pos_dev, "gh_mlstm_forward: NULL pointer" );
  GH_REQUIRE( dt == GH_BF16 || dt == GH_F32, "gh_mlstm_forward: unsupported dtype %d", (int)dt );
  GH_REQUIRE( m->heads > 0 && m->dim > 0 && m->vdim > 0 && m->heads <= 65535 && batch <= 65535 && m->dim <= 4096, "gh_mlstm_forward: bad shape" );
  GH_REQUIRE( m->gate_cap > 0.0f && state_offset % 16 == 0, "gh_mlstm_forward: bad gate cap or state offset" );
  const MlstmShape s = shape_of( m );
  hipStream_t st = as_stream( stream );
  uint64_t gate_row = 0;
  const uint64_t r = gh_mlstm_weight_rows( m, &gate_row );
  const uint32_t hd = s.heads * s.dim, hv = s.heads * s.vdim;
  MlstmCols col { 0, hd, 2 * hd, 2 * hd + hv, (uint32_t)gate_row, (uint32_t)gate_row + s.heads };
  Product y, gates;
  if ( dt == GH_BF16 && rows >= PRODUCT_ROUNDED_ROWS ) { // the gates stay fp32 sums
    if ( int rc = make_product( x, w, width, gate_row, rows, dt, false, st, &y ) ) {
      return rc;
    }
    if ( int rc = make_product( x, static_cast<const char*>( w ) + gate_row * width * dtype_size( dt ), width, r - gate_row, rows, dt, true, st, &gates ) ) {
      return rc;
    }
    col.i = 0;
    col.f = s.heads;
  } else {
    if ( int rc = make_product( x, w, width, r, rows, dt, false, st, &y ) ) {
      return rc;
    }
    gates = y;
  }
  void* scratch = nullptr;
  const uint64_t o_bytes = ( rows * hv * sizeof( float ) + 255 ) / 256 * 256;
  if ( int rc = stream_scratch( st, SCRATCH_MIXER, o_bytes + batch * s.heads * ( s.dim + 1ull ) * sizeof( float ), 1ull << 20, &scratch ) ) {
    return rc;
  }
  float* o = static_cast<float*>( scratch );
  float* nm = reinterpret_cast<float*>( static_cast<char*>( scratch ) + o_bytes );
  const MlstmState state { context_rows_dev, state_offset, start_pos_dev, n_tokens };
  return with_product( dt, y, [&]( auto tag, auto view ) -> int {
    using E = decltype( tag );
    using View = decltype( view );
    const MlstmIn<E, View> in { view, ProductView<float>( gates ), col, static_cast<const E*>( bias_i ), static_cast<const E*>( bias_f ) };
    const dim3 grid( ( s.vpad + SLICE - 1 ) / SLICE, s.heads, (unsigned)batch );
    const size_t lds = ( 3 * ( ( s.dim + 3 ) / 4 * 4 ) + SLICE + 16 + 16 * SLICE ) * sizeof( float );
    if ( s.dim <= 64 ) {
      mlstm_walk_kernel<E, View, 4><<<grid, 256, lds, st>>>( o, nm, in, state, s );
    } else if ( s.dim <= 128 ) {
      mlstm_walk_kernel<E, View, 8><<<grid, 256, lds, st>>>( o, nm, in, state, s );
    } else if ( s.dim <= 256 ) {
      mlstm_walk_kernel<E, View, 16><<<grid, 256, lds, st>>>( o, nm, in, state, s );
    } else {
      mlstm_walk_kernel<E, View, 0><<<grid, 256, lds, st>>>( o, nm, in, state, s );
    }
    GH_LAUNCH_CHECK();
    mlstm_finish_kernel<E, View><<<(unsigned)rows, 256, 0, st>>>( static_cast<E*>( out ), o, nm, in, static_cast<const E*>( norm ), state, s );
    GH_LAUNCH_CHECK();
    return GH_OK;
  } );
}

} // extern "C"
