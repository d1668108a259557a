// Driver of the Dirozen design for the hip target: weights, scratch, and the ops of one step.
//
//   embedding        x = embed[token]
//   layer            h = norm1(x); x += attention(h) + W_down (silu(W_gate h) * (W_up h)), the feed-forward optional
//   attention        q, k per head over their root mean square, q times its position's temperature; values are the keys as projected;
//                    each head's output times a sigmoid gate of h
//   output           logits = head . final_norm(x) (fp32) -> (Gumbel noise if temperature > 0) -> argmax
//
// Norms' weights are stored around zero.  The residual stream x is fp32.  Both sides of a layer are one product each: all that reads h
// (q, k, head gates, gate, up) on the way in, and on the way out [W_o | W_down] over [attention | hidden], which the attention and the
// feed-forward write side by side; the residual update and the next norm follow it.
#pragma once

#include <algorithm>
#include <string>
#include <vector>

#include "glint/design_driver.hh"
#include "glint/dirozen_config.hh"

namespace glint {

template<typename DType, typename Context = hip::LayeredContext>
class Dirozen : public DesignDriver<configs::Dirozen, DType, Context>
{
  using Base = DesignDriver<configs::Dirozen, DType, Context>;
  using Base::DT;
  using Base::ops_, Base::x_, Base::h_, Base::final_norm_, Base::settings_, Base::max_start_;
  using Base::tokens_dev, Base::pos_dev, Base::contexts_dev, Base::no_step, Base::lead_to, Base::lead_out;

public:
  Dirozen( const DirozenConfig& config, DesignSettings settings, const ModelOptions options = {} )
    : Base( { config.width, config.vocab, config.max_positions, config.eps, 1.0f }, std::move( settings ), options, plan( config ) )
    , config_( config )
  {
    describe_layers();
    this->allocate();
  }

  // per layer the cache rows, then the keys' factors
  static ContextPlan plan( const DirozenConfig& config )
  {
    ContextPlan p( config.max_positions );
    for ( const auto& layer : config.layers ) {
      const gh_window_attn a = attention_shape( layer );
      p.add_rows( gh_window_row_bytes( &a, DT ) );
      p.add_rows( gh_window_factor_bytes( &a ), GH_WINDOW_FACTOR_GROUP );
    }
    return p;
  }

  const DirozenConfig& config() const { return config_; }
  size_t n_runs() const override { return layers_.size(); }

private:
  struct Layer
  {
    DType *norm1 {}, *in {}, *out {};
    gh_window_attn attention {};
    gh_unit_heads unit_heads {};
    uint64_t hidden_col {}; // of the feed-forward in the rows `out` reads
    uint64_t out_cols {};
  };

  static gh_window_attn attention_shape( const DirozenConfig::Layer& l ) { return { l.heads, l.kv_heads, l.dim, l.dim, 0, 0, 0, l.scale, 1 }; }

  void describe_layers()
  {
    auto whole = []( const uint64_t n ) { return ( n + 7 ) / 8 * 8; }; // both parts of a row start at a whole load
    for ( const auto& c : config_.layers ) {
      Layer w;
      w.attention = attention_shape( c );
      w.unit_heads = { config_.eps, c.temp_coef, c.temp_every };
      w.hidden_col = whole( (uint64_t)c.heads * c.dim );
      w.out_cols = w.hidden_col + whole( c.ff );
      out_max_ = std::max( out_max_, w.out_cols );
      query_max_ = std::max( query_max_, gh_window_query_elements( &w.attention ) );
      heads_max_ = std::max<uint64_t>( heads_max_, c.heads );
      layers_.push_back( w );
    }
  }

  void lay_out( WeightCursor<DType>& cursor ) override
  {
    const uint64_t width = config_.width;
    embed_ = cursor.alone( "embed", { config_.vocab, width } );
    head_ = cursor.alone( "head", { config_.vocab, width } );
    final_norm_ = cursor.alone( "final.norm", { width } );
    for ( size_t l = 0; l < layers_.size(); l++ ) {
      auto& w = layers_[l];
      const auto& c = config_.layers[l];
      const std::string p = "l" + std::to_string( l ) + ".";
      const uint64_t hd = (uint64_t)c.heads * c.dim, gd = (uint64_t)c.kv_heads * c.dim, ff = c.ff;
      uint64_t ff_row = 0;
      const uint64_t rows = gh_parallel_weight_rows( &w.attention, 1, ff, &ff_row );
      w.norm1 = cursor.alone( p + "norm1", { width } );
      w.in = cursor.alone( p + "mix.q", { hd, width } );
      cursor.tensor( p + "mix.k", { gd, width } );
      cursor.tensor( p + "mix.g", { c.heads, width } );
      cursor.take( ( ff_row - hd - gd - c.heads ) * width );
      if ( ff > 0 ) {
        cursor.tensor( p + "mlp.gate", { ff, width } );
        cursor.tensor( p + "mlp.up", { ff, width } );
      }
      cursor.take( ( rows - ff_row - 2 * ff ) * width );
      cursor.align();
      w.out = cursor.take( width * w.out_cols );
      cursor.columns( p + "mix.o", { width, hd }, w.out, 0, w.out_cols );
      if ( ff > 0 ) {
        cursor.columns( p + "mlp.down", { width, ff }, w.out, w.hidden_col, w.out_cols );
      }
    }
  }

  void allocate_layer_scratch( const uint64_t rows ) override
  {
    q_ = ops_.device_allocate( rows * query_max_ * sizeof( DType ) );
    gates_ = this->logit_ops_.device_allocate( rows * heads_max_ * sizeof( float ) );
    joined_ = ops_.device_allocate( rows * out_max_ * sizeof( DType ) );
    // columns between the parts are read, against weights of zero, and never written
    GLINT_GH( gh_memset_zero( joined_.get(), rows * out_max_ * sizeof( DType ), ops_.stream() ) );
  }

  void run_layers( const uint64_t batch, const uint32_t n_tokens, const bool all_rows_classified, float* residuals_out ) override
  {
    const uint64_t rows = batch * n_tokens, width = config_.width;
    const gh_stream stream = ops_.stream();
    GLINT_GH( gh_embed_positions( x_.get(), tokens_dev(), pos_dev(), batch, n_tokens, embed_, nullptr, width, config_.vocab, 1, nullptr, 0, DT, stream ) );
    {
      gh_stream_step first = no_step();
      lead_to( first, layers_[0].norm1 );
      GLINT_GH( gh_stream_out( x_.get(), width, rows, &first, DT, stream ) );
    }
    for ( size_t l = 0; l < layers_.size(); l++ ) {
      const auto& w = layers_[l];
      const uint64_t ff = config_.layers[l].ff, keys = settings_.plan->parts[2 * l].offset, factors = settings_.plan->parts[2 * l + 1].offset;
      GLINT_GH( gh_matmul_parallel( q_.get(), gates_.get(), joined_.get() + w.hidden_col, w.out_cols, h_.get(), w.in, width, &w.attention, &w.unit_heads, ff, GH_ACT_SILU,
                                    contexts_dev(), keys, factors, pos_dev(), batch, n_tokens, DT, stream ) );
      GLINT_GH( gh_attn_window( joined_.get(), w.out_cols, gates_.get(), q_.get(), &w.attention, nullptr, contexts_dev(), keys, factors, pos_dev(), batch, n_tokens,
                                max_start_, DT, stream ) );
      gh_stream_step step = no_step();
      step.accumulate = 1;
      if ( l + 1 < layers_.size() ) {
        lead_to( step, layers_[l + 1].norm1 );
      } else if ( all_rows_classified ) {
        lead_out( step );
      }
      GLINT_GH( gh_matmul_stream( x_.get(), joined_.get(), w.out, w.out_cols, width, rows, &step, DT, stream ) );
      this->copy_residuals( residuals_out, l, rows );
    }
  }

  void classify( const uint64_t n ) override
  {
    GLINT_GH( gh_matmul_scaled( this->logits_.get(), h_.get(), head_, config_.width, config_.vocab, n, 1.0f, DT, ops_.stream() ) );
  }

  DirozenConfig config_;
  std::vector<Layer> layers_ {};
  uint64_t out_max_ { 0 }, query_max_ { 0 }, heads_max_ { 0 };
  DType *embed_ {}, *head_ {};
  typename Base::Operations::DeviceUniquePtr q_ {}, joined_ {};
  hip::Operations<float>::DeviceUniquePtr gates_ {};
};

} // namespace glint
